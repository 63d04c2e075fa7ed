"""Each Bolatar mechanism alone, CPU form and HIP kernels, against the plain
equations: delta rule and its convolution, mLSTM, RWKV-style recurrence,
biased attention, token mixing, merged outputs, clamped feed-forward, soft
cap.  Inputs are made so that one wrong key, row, decay or maximum shows."""

import math

import pytest
import torch

import bolatar_plain as plain
import resilient_llm_amd.ops as ops
from nesizen_util import BF16, F32, GPU, TARGETS
from resilient_llm_amd.engine.batch import Portion, PromptRows

NAN = float("nan")


def rel(got, want):
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all()
    return float((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())


def tol(dtype):
    return 4e-6 if dtype == F32 else 8e-3


def rnd(shape, seed, dtype, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(dtype)


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=device)


CUTS = [[150], [1] * 20, [2, 63, 1, 1, 64, 19], [3, 5, 1, 16, 2, 65, 58]]


def pieces(T, cut):
    p = 0
    for n in cut:
        n = min(n, T - p)
        if n:
            yield p, n
        p += n


# ------------------------------------------------------------ delta rule
class Delta:
    def __init__(self, T, H, G, dim, vdim, taps, device, dtype, seed=0):
        self.H, self.G, self.dim, self.vdim = H, G, dim, vdim
        self.device, self.dtype, self.eps = device, dtype, 1e-4
        self.C = 2 * G * dim + H * vdim
        pad = 3 if dim % 8 else -(self.C + H * vdim + 2 * H) % 8
        self.proj = rnd((T, self.C + H * vdim + 2 * H + pad), seed, dtype)
        self.w = rnd((self.C, taps), seed + 1, F32, 0.6)
        self.A_log = torch.linspace(-4.0, 1.0, H)
        self.dt_bias = torch.linspace(-4.0, 1.0, H)
        self.norm = 1 + rnd((vdim,), seed + 2, F32, 0.3)
        self.state = torch.full((3, H, dim, -(-vdim // 4) * 4), NAN,
                                device=device)
        self.tail = torch.full((3, taps, self.C), NAN, dtype=dtype,
                               device=device) if taps > 1 else None

    def want(self, round_x=True):
        """o after norm and gate; the convolved rows are activations."""
        p, H, G, hv = self.proj.double(), self.H, self.G, self.H * self.vdim
        T = p.shape[0]
        x = plain.silu(plain.short_conv(p[:, :self.C], self.w.double()))
        if round_x:
            x = x.to(self.dtype).double()
        qk = G * self.dim
        q, k, v = x[:, :qk], x[:, qk:2 * qk], x[:, 2 * qk:]
        of = [h // (H // G) for h in range(H)]
        q = plain.unit(q.view(T, G, -1))[:, of] * self.dim ** -0.5
        k = plain.unit(k.view(T, G, -1))[:, of]
        at = self.C
        gate, b, a = (p[:, at:at + hv], p[:, at + hv:at + hv + H],
                      p[:, at + hv + H:at + hv + 2 * H])
        g = plain.delta_decay(a, self.A_log.double(), self.dt_bias.double())
        o, S = plain.delta_recur(q, k, v.reshape(T, H, -1), torch.sigmoid(b),
                                 g)
        o = plain.rms(o, self.eps) * self.norm.double() \
            * plain.silu(gate).view(T, H, -1)
        return o.reshape(T, -1), S

    def call(self, p, n, slot, seqs=1):
        d = self.device
        rows = self.proj[p:p + n].contiguous().to(d)
        out = torch.full((n, self.H * self.vdim), NAN, dtype=self.dtype,
                         device=d)
        args = (self.w.t().contiguous().to(d), self.tail,
                torch.exp(self.A_log).to(d), self.dt_bias.to(d),
                self.norm.to(d), self.state)
        if n == 1 and p > 0:
            ops.delta_decode(rows, *args, i32([slot], d), i32([p], d), self.G,
                             self.vdim, self.eps, out)
        else:
            ops.delta_prefill(rows, *args, PromptRows(
                [Portion(0, p, n, 0, slot)], d), self.G, self.vdim, self.eps,
                out)
        return out


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("cut", CUTS, ids=lambda c: f"{len(c)}-{c[0]}")
@pytest.mark.parametrize("shape", [(2, 1, 16, 24, 4), (3, 3, 20, 18, 1),
                                   (4, 2, 64, 64, 2), (6, 2, 128, 48, 3),
                                   (1, 1, 200, 33, 7), (5, 1, 7, 300, 3)],
                         ids=str)
def test_delta_rule(shape, cut, device, dtype):
    """Any cut into portions and tokens, slots that hold NaN, shared key
    heads, slow and steep decays; the state at the end."""
    T = sum(cut)
    a = Delta(T, *shape, device, dtype, seed=sum(shape))
    want, S = a.want()
    got = torch.cat([a.call(p, n, 2) for p, n in pieces(T, cut)])
    assert rel(got, want) < tol(dtype)
    s = a.state[2, :, :, :a.vdim].cpu()
    assert rel(s, S) < (5e-6 if dtype == F32 else 2e-3)


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_delta_rule_repeated_keys(device, dtype):
    """The same key again and again: only what is new is learned, across
    sub-chunk and chunk borders."""
    T = 150
    a = Delta(T, 2, 1, 32, 16, 1, device, dtype)
    a.w.fill_(1)
    a.proj[:, :64] = a.proj[:1, :64]
    a.proj[:, a.C + 32:a.C + 34] = 4.0           # strong writes
    a.A_log.fill_(-6.0)
    want, _ = a.want()
    for cut in ([T], [70, 2, 1, 77]):
        a.state.fill_(NAN)
        got = torch.cat([a.call(p, n, 0) for p, n in pieces(T, cut)])
        assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_delta_rule_several_sequences(device, dtype):
    """Portions of two sequences in one call, then one token of each in one
    batch that shares key heads."""
    H, G, dim, vdim = 4, 2, 16, 20
    a, b = (Delta(80, H, G, dim, vdim, 3, device, dtype, seed=s)
            for s in (0, 0))
    b.proj = rnd(b.proj.shape, 9, dtype)
    b.state, b.tail = a.state, a.tail
    d = device
    want = [x.want()[0] for x in (a, b)]
    args = (a.w.t().contiguous().to(d), a.tail, torch.exp(a.A_log).to(d),
            a.dt_bias.to(d), a.norm.to(d), a.state)
    rows = torch.cat([a.proj[:70], b.proj[:5]]).to(d)
    out = torch.empty((75, H * vdim), dtype=dtype, device=d)
    ops.delta_prefill(rows, *args, PromptRows(
        [Portion(0, 0, 70, 0, 2), Portion(70, 0, 5, 1, 0)], d), G, vdim,
        a.eps, out)
    assert rel(out, torch.cat([want[0][:70], want[1][:5]])) < tol(dtype)
    for k in range(5):
        rows = torch.stack([b.proj[5 + k], a.proj[70 + k]]).to(d)
        out = torch.empty((2, H * vdim), dtype=dtype, device=d)
        ops.delta_decode(rows, *args, i32([0, 2], d), i32([5 + k, 70 + k], d),
                         G, vdim, a.eps, out)
        assert rel(out, torch.stack([want[1][5 + k], want[0][70 + k]])) \
            < 2 * tol(dtype)


# ----------------------------------------------------------------- mLSTM
class Mlstm:
    def __init__(self, T, H, dim, vdim, cap, device, dtype, seed=0):
        self.H, self.dim, self.vdim, self.cap = H, dim, vdim, cap
        self.device, self.dtype, self.eps = device, dtype, 1e-5
        w = 2 * H * (dim + vdim) + 2 * H
        self.proj = rnd((T, w + (3 if dim % 8 else -w % 8)), seed, dtype)
        self.at = 2 * H * (dim + vdim)
        self.proj[:, self.at:self.at + 2 * H] *= 3
        self.i_b = torch.linspace(-3.0, 3.0, H)
        self.f_b = torch.linspace(6.0, -2.0, H)
        self.norm = 1 + rnd((H * vdim,), seed + 1, F32, 0.3)
        self.state = torch.full((3, H, dim, (vdim + 4) // 4 * 4), NAN,
                                device=device)
        self.m = torch.full((3, H), NAN, device=device)

    def want(self):
        p, H, T = self.proj.double(), self.H, self.proj.shape[0]
        q, k, v, g, i, f = torch.split(
            p[:, :self.at + 2 * H],
            [H * self.dim, H * self.dim, H * self.vdim, H * self.vdim, H, H],
            1)
        i = plain.soft_cap(i + self.i_b.double(), self.cap)
        f = -plain.softplus(-plain.soft_cap(f + self.f_b.double(), self.cap))
        o, S, n, m = plain.mlstm_recur(
            q.reshape(T, H, -1) * self.dim ** -0.5, k.reshape(T, H, -1),
            v.reshape(T, H, -1), i, f)
        o = plain.rms(o, self.eps).reshape(T, -1) * self.norm.double()
        return o * torch.sigmoid(g), torch.cat([S, n[..., None]], -1), m

    def call(self, p, n, slot):
        d = self.device
        rows = self.proj[p:p + n].contiguous().to(d)
        out = torch.full((n, self.H * self.vdim), NAN, dtype=self.dtype,
                         device=d)
        args = (self.i_b.to(d), self.f_b.to(d), self.norm.to(d), self.state,
                self.m)
        if n == 1 and p > 0:
            ops.mlstm_decode(rows, *args, i32([slot], d), i32([p], d),
                             self.vdim, self.cap, self.eps, out)
        else:
            ops.mlstm_prefill(rows, *args, PromptRows(
                [Portion(0, p, n, 0, slot)], d), self.vdim, self.cap,
                self.eps, out)
        return out


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("cut", CUTS, ids=lambda c: f"{len(c)}-{c[0]}")
@pytest.mark.parametrize("shape", [(2, 16, 24, 6.0), (3, 20, 17, 1.5),
                                   (4, 64, 64, 15.0), (1, 128, 80, 12.0),
                                   (2, 200, 1, 4.0), (1, 5, 260, 9.0)],
                         ids=str)
def test_mlstm(shape, cut, device, dtype):
    """Any cut, slots that hold NaN; state, normalizer and maximum at the
    end."""
    T = sum(cut)
    a = Mlstm(T, *shape, device, dtype, seed=T)
    want, S, m = a.want()
    got = torch.cat([a.call(p, n, 1) for p, n in pieces(T, cut)])
    # (heads that forget almost all a token lose digits in the exponents)
    assert rel(got, want) < (2e-5 if dtype == F32 else 1e-2)
    assert rel(a.m[1], m) < 1e-5
    assert rel(a.state[1, :, :, :a.vdim + 1].cpu(), S) < 2e-5


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("loud", [0, 1, 15, 16, 63, 64, 127, 128, 140])
def test_mlstm_one_loud_input(loud, device, dtype):
    """The running maximum jumps once, anywhere in a chunk, and then slowly
    falls; before that it only falls from where it started, zero."""
    T = 150
    a = Mlstm(T, 2, 16, 16, 20.0, device, dtype)
    a.f_b.fill_(4.0)
    a.proj[:, a.at:a.at + 4] = 0
    a.i_b.fill_(-8.0)
    a.proj[loud, a.at:a.at + 2] = 24.0
    want, _, m = a.want()
    for cut in ([T], [62, 2, 1, 85]):
        got = torch.cat([a.call(p, n, 2) for p, n in pieces(T, cut)])
        assert rel(got, want) < (1e-5 if dtype == F32 else 1e-2), cut
        assert rel(a.m[2], m) < 1e-5


# ------------------------------------------------------------------ RWKV
class Rwkv:
    def __init__(self, T, H, dim, rank, device, dtype, seed=0):
        n = H * dim
        self.H, self.dim, self.device, self.dtype = H, dim, device, dtype
        self.eps = 1e-4
        self.rkvg = rnd((4, T, n), seed, dtype)
        self.low = rnd((T, rank), seed + 1, dtype)
        self.w2 = rnd((n, rank), seed + 2, dtype, rank ** -0.5)
        self.w0 = torch.linspace(-7.0, 1.5, n)
        self.u = rnd((n,), seed + 3, F32)
        self.norm = 1 + rnd((n,), seed + 4, F32, 0.3)
        self.state = torch.full((3, H, dim, -(-dim // 4) * 4), NAN,
                                device=device)

    def want(self):
        T = self.low.shape[0]
        r, k, v, g = (x.double().view(T, self.H, self.dim)
                      for x in self.rkvg)
        z = torch.tanh(self.low.double()) @ self.w2.double().T + self.w0
        w = torch.exp(-torch.exp(z)).view(T, self.H, self.dim)
        o, S = plain.rwkv_recur(r, k, v, w,
                                self.u.double().view(self.H, self.dim))
        o = plain.rms(o, self.eps).reshape(T, -1) * self.norm.double()
        return o * plain.silu(g.reshape(T, -1)), S

    def call(self, p, n, slot):
        d = self.device
        # a range of a longer batch, as in a mixed step
        wide = torch.full((4, n + 2, self.H * self.dim), NAN,
                          dtype=self.dtype)
        wide[:, 2:] = self.rkvg[:, p:p + n]
        rkvg = wide.to(d)[:, 2:]
        out = torch.full((n, self.H * self.dim), NAN, dtype=self.dtype,
                         device=d)
        args = (self.low[p:p + n].to(d), self.w2.to(d), self.w0.to(d),
                self.u.to(d), self.norm.to(d), self.state)
        if n == 1 and p > 0:
            ops.rwkv_decode(rkvg, *args, i32([slot], d), i32([p], d),
                            self.eps, out)
        else:
            ops.rwkv_prefill(rkvg, *args, PromptRows(
                [Portion(0, p, n, 0, slot)], d), self.eps, out)
        return out


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("cut", CUTS, ids=lambda c: f"{len(c)}-{c[0]}")
@pytest.mark.parametrize("shape", [(2, 16, 4), (3, 20, 5), (2, 64, 16),
                                   (1, 128, 12), (1, 144, 64), (4, 6, 3)],
                         ids=str)
def test_rwkv(shape, cut, device, dtype):
    """Decays from nearly none to nearly all per token in every head; the
    bonus for the present token only."""
    T = sum(cut)
    a = Rwkv(T, *shape, device, dtype, seed=T)
    want, S = a.want()
    got = torch.cat([a.call(p, n, 0) for p, n in pieces(T, cut)])
    assert rel(got, want) < (1e-5 if dtype == F32 else 8e-3)
    assert rel(a.state[0, :, :, :a.dim].cpu(), S) < 2e-5


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("w0", [-9.0, -1.0, 1.0, 2.5, 5.0])
def test_rwkv_gentle_and_steep_decays(w0, device, dtype):
    T = 150
    a = Rwkv(T, 2, 64, 8, device, dtype)
    a.w0.fill_(w0)
    want, _ = a.want()
    got = torch.cat([a.call(p, n, 1) for p, n in pieces(T, [80, 1, 2, 67])])
    assert rel(got, want) < (2e-5 if dtype == F32 else 8e-3)


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_rwkv_bonus_and_first_row(device, dtype):
    """Without a past only the bonus speaks; without a bonus the present is
    not seen."""
    a = Rwkv(70, 2, 16, 4, device, dtype)
    a.u.zero_()
    assert float(a.call(0, 1, 0).abs().max()) < 1e-6
    want, _ = a.want()
    got = a.call(0, 70, 0)
    assert rel(got[1:], want[1:]) < tol(dtype) * 2


# ------------------------------------------------------ biased attention
class Biased:
    """Paged keys and values with scattered, poisoned pages."""

    def __init__(self, T, H, G, dim, vdim, device, dtype, seed=0, coef=0.5,
                 every=9, scale=None, cache_dtype=None):
        self.H, self.G, self.dim, self.vdim = H, G, dim, vdim
        self.device, self.dtype, self.eps = device, dtype, 1e-3
        self.coef, self.every = coef, every
        self.scale = dim ** -0.5 if scale is None else scale
        self.qkv = rnd((T, H * dim + G * (dim + vdim)), seed, dtype)
        self.r1 = torch.linspace(0.02, 2.0, H)
        self.r2 = torch.linspace(1.0, 0.05, H)
        n = -(-T // 16)
        perm = torch.randperm(n + 3, generator=torch.Generator()
                              .manual_seed(seed))[:n]
        self.table = perm.to(torch.int32)[None].contiguous()
        cd = cache_dtype or dtype
        self.k = torch.full((n + 3, G, 16, dim), NAN).to(cd).to(device)
        self.v = torch.full((n + 3, G, 16, vdim), NAN).to(cd).to(device)

    def want(self):
        T, H, G = self.qkv.shape[0], self.H, self.G
        q, k, v = torch.split(self.qkv.double(), [
            H * self.dim, G * self.dim, G * self.vdim], 1)
        t = torch.tensor([plain.query_temperature(p, self.coef, self.every)
                          for p in range(T)]).double()
        return plain.biased_attention(
            q.view(T, H, -1) * t[:, None, None], k.view(T, G, -1),
            plain.rms(v.view(T, G, -1), self.eps), self.scale,
            self.r1.double(), self.r2.double()).reshape(T, -1)

    def call(self, p, n):
        d = self.device
        pos = range(p, p + n)
        slots = [int(self.table[0, x // 16]) * 16 + x % 16 for x in pos]
        args = (self.qkv[p:p + n].contiguous().to(d), self.k, self.v,
                i32(list(pos), d), i32(slots, d), self.table.to(d))
        score = (self.scale, self.H, self.r1.to(d), self.r2.to(d), self.coef,
                 self.every, self.eps)
        if n == 1 and p > 0:
            return ops.biased_decode(*args, *score)
        return ops.biased_prefill(*args, PromptRows([Portion(0, p, n, 0)], d),
                                  *score)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("cut", CUTS, ids=lambda c: f"{len(c)}-{c[0]}")
@pytest.mark.parametrize("shape", [(2, 1, 16, 24), (3, 3, 20, 9),
                                   (8, 2, 64, 64), (6, 2, 128, 72),
                                   (5, 1, 40, 200), (1, 1, 3, 5)], ids=str)
def test_biased_attention(shape, cut, device, dtype):
    T = sum(cut)
    a = Biased(T, *shape, device, dtype, seed=T)
    got = torch.cat([a.call(p, n) for p, n in pieces(T, cut)])
    assert rel(got, a.want()) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("H,G,dim", [(2, 1, 32), (3, 3, 12)])
def test_one_loud_key_and_its_distance(H, G, dim, device, dtype):
    """Every query asks for one key; how loudly it answers depends on the
    distance alone, and a key behind the query stays unseen."""
    T = 300
    a = Biased(T, H, G, dim, 16, device, dtype, scale=1.0, every=64)
    q, k = a.qkv[:, :H * dim], a.qkv[:, H * dim:(H + G) * dim]
    q.zero_()
    q.view(T, H, dim)[:, :, 0] = 1
    k.zero_()
    for loud in (0, 15, 16, 63, 64, 128, 255, 270):
        k.view(T, G, dim)[:, :, 0] = 0
        k.view(T, G, dim)[loud, :, 0] = 8
        want = a.want()
        assert rel(a.call(0, T), want) < tol(dtype), loud
        for p in {max(1, loud - 1), loud + 1, loud + 17, T - 1}:
            assert rel(a.call(p, 1), want[p:p + 1]) < tol(dtype), (loud, p)
        p = max(0, loud - 2)
        assert rel(a.call(p, 5), want[p:p + 5]) < tol(dtype), loud


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_query_temperature_steps(device, dtype):
    """The temperature moves at positions every - 1, 2 every - 1, ..., and
    not one off."""
    for every in (1, 16, 31):
        a = Biased(100, 2, 1, 16, 16, device, dtype, coef=2.0, every=every)
        a.qkv[:, :32] *= 2
        want = a.want()
        assert rel(a.call(0, 100), want) < tol(dtype) * 2
        for p in (every - 2, every - 1, every, 2 * every - 1):
            if 0 < p < 100:
                assert rel(a.call(p, 1), want[p:p + 1]) < tol(dtype) * 2


@GPU
def test_biased_decode_batches_and_splits():
    """Unequal sequences in one batch, splits that some do not reach."""
    lens = [1, 700, 17, 64, 65, 1500, 128, 300]
    d, H, G, dim, vdim = "cuda:0", 8, 2, 32, 40
    parts = [Biased(n, H, G, dim, vdim, d, BF16, seed=i)
             for i, n in enumerate(lens)]
    width = max(p.table.shape[1] for p in parts)
    tables, at = [], 0
    for p in parts:
        p.call(0, len(p.qkv))                       # fill the cache
        row = torch.zeros(1, width, dtype=torch.int32)
        row[:, :p.table.shape[1]] = p.table + at
        at += p.k.shape[0]
        tables.append(row)
    tables = torch.cat(tables)
    a = parts[0]
    pos = [n - 1 for n in lens]
    slots = [int(tables[i, p // 16]) * 16 + p % 16 for i, p in enumerate(pos)]
    out = ops.biased_decode(
        torch.stack([p.qkv[-1] for p in parts]).to(d),
        torch.cat([p.k for p in parts]), torch.cat([p.v for p in parts]),
        i32(pos, d), i32(slots, d), tables.to(d), a.scale, H, a.r1.to(d),
        a.r2.to(d), a.coef, a.every, a.eps)
    for i, p in enumerate(parts):
        want = last_row(p)
        assert rel(out[i], want) < tol(BF16), lens[i]


def last_row(a):
    """The plain attention of the last query only."""
    T, H, G = len(a.qkv), a.H, a.G
    q, k, v = torch.split(a.qkv.double(),
                          [H * a.dim, G * a.dim, G * a.vdim], 1)
    q = q[-1].view(H, -1) * plain.query_temperature(T - 1, a.coef, a.every)
    k, v = k.view(T, G, -1), plain.rms(v.view(T, G, -1), a.eps)
    back = torch.arange(T - 1, -1, -1).double()
    out = []
    for h in range(H):
        s = k[:, h // (H // G)] @ q[h] * a.scale \
            - a.r1[h] * torch.log(1 + a.r2[h] * back)
        out.append(torch.softmax(s, 0) @ v[:, h // (H // G)])
    return torch.cat(out)


# ---------------------------------------------- token mixing, merged norms
@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("W", [24, 64, 78, 1028, 2048])
def test_token_mixes(W, device, dtype):
    """Five mixes of a row with the one before it, through portions and,
    fused behind the norm, single tokens."""
    N = 40
    h = rnd((2, N, W), 1, dtype)
    mu = torch.rand(5, W, generator=torch.Generator().manual_seed(2))
    taps = torch.stack([mu, -mu], 1).contiguous().to(device)
    want = torch.stack([torch.stack([plain.shift_mix(h[s].double(), m)
                                     for m in mu.double()])
                        for s in range(2)])
    tail = torch.full((3, 1, W), NAN, dtype=dtype, device=device)
    slots, got, p = [2, 0], [[], []], 0
    for n in [2, 1, 17, 1, 1, 3, 13, 2]:
        if n > 1 or p == 0:
            rows = torch.cat([h[0, p:p + n], h[1, p:p + n]]).to(device)
            out = torch.full((5, 2 * n + 1, W), NAN, dtype=dtype,
                             device=device)
            ops.conv_prompt(rows, taps, tail, PromptRows(
                [Portion(0, p, n, 0, slots[0]),
                 Portion(n, p, n, 1, slots[1])], device), out[:, 1:])
            got[0].append(out[:, 1:n + 1])
            got[1].append(out[:, n + 1:])
        else:
            # rows of unit mean square are their own norm
            x = h[:, p].to(device).float()
            size = x.pow(2).mean(-1, keepdim=True).sqrt()
            hn, hc = ops.block_step(
                x.clone(), torch.zeros_like(x).to(dtype),
                torch.ones(W, device=device), 1, 1e-12,
                i32([p, p], device), taps, tail, i32(slots, device), 2)
            assert hc.shape == (5, 2, W)
            # put the sequence's own rows in the place of the normed ones
            assert torch.equal(tail[torch.tensor(slots), 0], hn)
            tail[torch.tensor(slots), 0] = h[:, p].to(device)
            own = (1 - mu.to(device))[:, None] * (x - hn.float())
            for s in range(2):
                got[s].append((hc[:, s].float() + own[:, s])[:, None])
            assert float(size.min()) > 0
        p += n
    assert p == N
    for s in range(2):
        assert rel(torch.cat([t.double() for t in got[s]], 1), want[s]) \
            < 2 * tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("W", [5, 40, 256, 1024, 1032, 2048, 4100, 8192,
                               8200])
def test_merged_outputs(W, device, dtype):
    """Two outputs of very different size, normed apart and averaged into
    the residual; rows for the last norm."""
    T, eps = 5, 3e-4
    x0 = rnd((T, W), 1, F32)
    y1, y2 = rnd((T, W), 2, dtype, 0.02), rnd((T, W), 3, dtype, 30.0)
    g1, g2, g = (1 + rnd((W,), s, F32, 0.3) for s in (4, 5, 6))
    new = x0.double() + 0.5 * (plain.rms(y1.double(), eps) * g1
                               + plain.rms(y2.double(), eps) * g2)
    d = device
    x = x0.clone().to(d)
    two = dict(y2=y2.to(d), gain1=g1.to(d), gain2=g2.to(d))
    rows = torch.tensor([4, 1])
    last, _ = ops.block_step(x, y1.to(d), g.to(d), 1, eps, i32([0] * T, d),
                             rows=rows.to(d), keep=False, **two)
    assert rel(last, (plain.rms(new, eps) * g)[rows]) < tol(dtype)
    assert torch.equal(x.cpu(), x0)                     # left alone
    h, _ = ops.block_step(x, y1.to(d), g.to(d), 1, eps, i32([0] * T, d),
                          **two)
    assert rel(x, new) < 3e-6
    assert rel(h, plain.rms(new, eps) * g) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_scaled_embedding_and_positions(device, dtype):
    W, scale = 40, 3.25
    table, pos = rnd((11, W), 1, dtype), rnd((9, W), 2, dtype)
    ids, at = [3, 0, 10], [8, 0, 3]
    x = torch.empty(3, W, device=device)
    h, _ = ops.block_embed(i32(ids, device), table.to(device),
                           pos.to(device), i32(at, device), x,
                           torch.ones(W, device=device), 1, 1e-5,
                           scale=scale)
    want = table.double()[ids] * scale + pos.double()[at]
    assert rel(x, want) < 1e-6
    assert rel(h, plain.rms(want, 1e-5)) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("ff", [64, 41, 2056])
@pytest.mark.parametrize("limit", [0.3, 7.0])
def test_clamped_feed_forward(ff, limit, device, dtype):
    gu = rnd((5, 2 * ff), 1, dtype, 2.0)
    gu[0, :4] = torch.tensor([-90.0, 50.0, -0.0, limit])
    out = torch.empty((5, ff), dtype=dtype, device=device)
    ops.gate_act(gu.to(device), out, "clamp_glu", limit)
    eye = torch.eye(2 * ff, dtype=torch.float64)
    want = plain.clamped_ff(gu.double(), {
        "gate": eye[:ff], "up": eye[ff:], "down": eye[:ff, :ff]}, limit)
    assert rel(out, want) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_soft_cap(device, dtype):
    x = rnd((7, 37), 1, dtype, 20.0)
    got = ops.soft_cap(x.to(device), 6.5)
    assert got.dtype == F32
    assert rel(got, plain.soft_cap(x.double(), 6.5)) < 2e-6
    assert math.isclose(float(got.abs().max()), 6.5, rel_tol=1e-3)
