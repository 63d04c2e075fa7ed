"""Each Riruzen mechanism alone, CPU form and HIP kernels, against the plain
equations: residual and grouped norms, the short convolution and its tails,
latent attention in its forms, HGRN2.  Inputs are made so that one wrong
key, row, tap or decay shows."""


import pytest
import torch

import resilient_llm_amd.ops as ops
import riruzen_plain as plain
from nesizen_util import BF16, F32, GPU, TARGETS
from resilient_llm_amd.engine.batch import Portion, PromptRows

D64 = torch.float64
NAN = float("nan")


def rel(got, want):
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all()
    return float((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())


def tol(dtype):
    return 3e-6 if dtype == F32 else 8e-3


def rnd(shape, seed, dtype, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(dtype)


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=device)


# ------------------------------------------------- residual and norms
@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("W,G", [(40, 1), (96, 3), (200, 25), (256, 2),
                                 (1024, 8), (1032, 6), (2048, 4), (4100, 5),
                                 (8192, 16), (8200, 2), (78, 3), (5, 5)])
def test_residual_and_grouped_norm(W, G, device, dtype):
    T, V, eps = 5, 11, 3e-4
    table, pos_table = rnd((V, W), 1, dtype, 0.05), rnd((9, W), 2, dtype, 0.05)
    # parts of very different size: a norm over the wrong part shows
    size = torch.repeat_interleave(
        torch.logspace(-1, 1, G), W // G).to(dtype)
    table, pos_table = table * size, pos_table * size
    ids, pos = [3, 0, 10, 3, 7], [8, 0, 3, 1, 5]
    g1, g2 = (1 + rnd((W,), s, F32, 0.3) for s in (3, 4))
    x = torch.empty(T, W, dtype=F32, device=device)

    def dev(t):
        return t.to(device)
    h, _ = ops.block_embed(i32(ids, device), dev(table), dev(pos_table),
                           i32(pos, device), x, dev(g1), G, eps)
    want = table.double()[ids] + pos_table.double()[pos]
    assert rel(x, want) < 3e-6
    assert rel(h, plain.group_norm(want, g1.double(), G, eps)) < tol(dtype)
    y = rnd((T, W), 5, dtype)
    new = want + y.double()
    rows = torch.tensor([4, 1])
    last, _ = ops.block_step(x, dev(y), dev(g2), G, eps, i32(pos, device),
                             rows=dev(rows), keep=False)
    assert rel(last, plain.group_norm(new, g2.double(), G, eps)[rows]) \
        < tol(dtype)
    assert rel(x, want) < 3e-6                          # left alone
    h, _ = ops.block_step(x, dev(y), dev(g2), G, eps, i32(pos, device))
    assert rel(x, new) < 3e-6
    assert rel(h, plain.group_norm(new, g2.double(), G, eps)) < tol(dtype)


# ---------------------------------------------------- short convolution
@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("W,taps", [(64, 1), (64, 2), (72, 3), (1028, 4),
                                    (30, 3), (40, 7), (7, 1)])
def test_convolution_portions_and_tokens(W, taps, device, dtype):
    """Any cut of a sequence into portions and single tokens, two sequences
    in one call, tails that hold an earlier owner's values."""
    N, eps = 61, 1e-5
    h = rnd((2, N, W), 1, dtype)
    w = rnd((W, taps), 2, F32)
    wt = w.t().contiguous().to(device)
    gain = torch.ones(W, device=device)
    want = torch.stack([h[s].double() + plain.short_conv(
        h[s].double(), w.double()) for s in range(2)])
    tail = torch.full((3, taps - 1, W), NAN, dtype=dtype, device=device) \
        if taps > 1 else None
    slots = [2, 0]
    got = [[], []]
    p = 0
    for n in [2, 1, 17, 1, 1, 3, 2, 16, 1, 15, 2]:
        if n > 1 or p == 0:
            a, b = h[0, p:p + n], h[1, p:p + n]
            rows = torch.cat([a, b]).contiguous().to(device)
            out = torch.empty_like(rows)
            ops.conv_prompt(rows, wt, tail, PromptRows(
                [Portion(0, p, n, 0, slots[0]),
                 Portion(n, p, n, 1, slots[1])], device), out)
            got[0].append(out[:n])
            got[1].append(out[n:])
        else:
            # through the fused step: rows of unit mean square are their
            # own norm
            rows = h[:, p].to(device)
            x = rows.float()
            ms = x.pow(2).mean(-1, keepdim=True)
            unit = (x / torch.sqrt(ms + eps)).to(dtype)
            hn, hc = ops.block_step(
                x.clone(), torch.zeros_like(rows), gain, 1, eps,
                i32([p, p], device), wt, tail, i32(slots, device), 2)
            assert rel(hn, unit.cpu().double()) < tol(dtype)
            if tail is not None:
                # what the convolution sees is the normed row; put the
                # sequence's own row in its place for the steps to come
                ring = tail[torch.tensor(slots), p % (taps - 1)]
                assert torch.equal(ring, hn)
                tail[torch.tensor(slots), p % (taps - 1)] = rows
            fix = (1 + wt[-1]) * (rows.float() - hn.float())
            for s in range(2):
                got[s].append((hc[s].float() + fix[s])[None])
        p += n
    assert p == N
    for s in range(2):
        assert rel(torch.cat([t.double() for t in got[s]]), want[s]) \
            < 2 * tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("act", ["relu", "silu"])
@pytest.mark.parametrize("ff,width", [(64, 96), (41, 41), (2056, 2064),
                                      (40, 43)])
def test_gated_activation(ff, width, act, device, dtype):
    gu = rnd((5, 2 * ff), 1, dtype)
    out = torch.full((5, width), NAN, dtype=dtype, device=device)
    ops.gate_act(gu.to(device), out[:, width - ff:], act)
    g, u = gu.double().chunk(2, 1)
    f = torch.relu(g) if act == "relu" else g * torch.sigmoid(g)
    assert rel(out[:, width - ff:], f * u) < tol(dtype)
    assert torch.isnan(out[:, :width - ff]).all()


# ---------------------------------------------------- latent attention
class Latent:
    """A paged latent cache with scattered, poisoned pages and the op
    calls; keys and values per head come from the latents."""

    def __init__(self, T, H, dim, vdim, rank, device, dtype, scale=None,
                 seed=0, cache_dtype=None, block=16, wide=3):
        self.H, self.dim, self.vdim, self.R = H, dim, vdim, rank
        self.device, self.dtype, self.block = device, dtype, block
        self.scale = dim ** -0.5 if scale is None else scale
        self.q = rnd((T, H * dim), seed, dtype)
        self.c = rnd((T, rank), seed + 1, dtype)
        self.gate = rnd((T, H * vdim + wide), seed + 2, dtype)
        self.uk = rnd((H * dim, rank), seed + 3, dtype, rank ** -0.5)
        self.uv = rnd((H * vdim, rank), seed + 4, dtype, rank ** -0.5)
        n = -(-T // block)
        perm = torch.randperm(n + 3, generator=torch.Generator()
                              .manual_seed(seed))[:n]
        self.table = perm.to(torch.int32)[None].contiguous()
        self.cache = torch.full((n + 3, 1, block, rank), NAN).to(
            cache_dtype or dtype).to(device)

    def want(self):
        T, f = self.q.shape[0], torch.Tensor.double
        k = (f(self.c) @ f(self.uk).T).view(T, self.H, self.dim)
        v = (f(self.c) @ f(self.uv).T).view(T, self.H, self.vdim)
        o = plain.attend(f(self.q).view(T, self.H, self.dim), k, v,
                         self.scale)
        return o.reshape(T, -1) * torch.sigmoid(f(self.gate)
                                                [:, :self.H * self.vdim])

    def put(self, p0, n):
        for p in range(p0, p0 + n):
            self.cache[int(self.table[0, p // self.block]), 0,
                       p % self.block] = self.c[p].to(self.cache.dtype)

    def call(self, p0, n, expand=None):
        """Rows p0 .. p0 + n on what was put before."""
        d = self.device
        hv = self.H * self.vdim
        out = torch.full((n, hv + 4), NAN, dtype=self.dtype, device=d)
        q = self.q[p0:p0 + n].contiguous().to(d)
        gate = self.gate[p0:p0 + n].to(d)[:, :hv]
        uk, uv = self.uk.to(d), self.uv.to(d)
        uk_t = uk.view(self.H, self.dim, self.R).transpose(1, 2).contiguous()
        uv3 = uv.view(self.H, self.vdim, self.R)
        if n == 1 and expand is None:
            ops.latent_decode(q, gate, self.cache, i32([p0], d),
                              self.table.to(d), self.scale, uk_t, uv3,
                              out[:, :hv])
        else:
            ops.latent_prefill(
                q, gate, self.cache, self.table.to(d),
                PromptRows([Portion(0, p0, n, 0)], d), self.scale, uk_t, uv3,
                uk, uv, out[:, :hv], expand)
        assert torch.isnan(out[:, hv:]).all()
        return out[:, :hv]


# heads, dim, vdim, rank
SHAPES = [(4, 32, 32, 64), (6, 16, 24, 40), (3, 12, 20, 27), (16, 64, 64, 128),
          (17, 24, 8, 136), (40, 16, 16, 256), (66, 8, 16, 320),
          (2, 128, 96, 512), (1, 72, 200, 384), (2, 192, 256, 96),
          (5, 40, 48, 520), (1, 1, 1, 8)]


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("shape", SHAPES, ids=str)
def test_latent_attention_sizes(shape, device, dtype):
    T = 147
    a = Latent(T, *shape, device, dtype, seed=sum(shape))
    want, t = a.want(), 2 * tol(dtype)
    a.put(0, T)
    assert rel(a.call(0, T, expand=False), want) < t
    assert rel(a.call(0, T, expand=True), want) < t
    for p in (0, 15, 16, 63, 64, 146):
        assert rel(a.call(p, 1), want[p:p + 1]) < t, p
    for p, n in ((1, 2), (31, 34), (60, 70), (128, 19)):
        for expand in (False, True):
            assert rel(a.call(p, n, expand), want[p:p + n]) < t, (p, n)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("H,dim,vdim,rank", [(4, 32, 32, 64),
                                             (18, 16, 24, 512),
                                             (2, 12, 12, 20)])
def test_one_loud_key_is_found_and_the_next_is_not(H, dim, vdim, rank, device,
                                                   dtype):
    """Every query asks for one far key, among others at page and tile
    borders; a key just behind the query must stay unseen however loud."""
    T = 330
    a = Latent(T, H, dim, vdim, rank, device, dtype, scale=1.0)
    a.q.zero_()
    a.uk.zero_()
    a.uk.view(H, dim, rank)[:, 0, 0] = 1
    a.q.view(T, H, dim)[:, :, 0] = 1         # score = c[:, 0]
    for loud in (0, 1, 15, 16, 63, 64, 127, 128, 255, 256, 300):
        a.c[:, 0] = 0
        a.c[loud, 0] = 24.0
        a.put(0, T)
        want = a.want()
        for p in {max(0, loud - 1), loud, loud + 1, 299, T - 1}:
            assert rel(a.call(p, 1), want[p:p + 1]) < 2 * tol(dtype), (loud, p)
        for expand in (False, True):
            assert rel(a.call(0, T, expand), want) < 2 * tol(dtype), loud
            p0 = max(0, loud - 3)
            n = min(20, T - p0)
            assert rel(a.call(p0, n, expand), want[p0:p0 + n]) \
                < 2 * tol(dtype), loud


@GPU
@pytest.mark.parametrize("H,rank", [(8, 96), (24, 512), (70, 64)])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_latent_decode_batches_and_splits(H, rank, dtype):
    """Unequal sequences in one batch, splits that some of them do not
    reach, other pages."""
    lens = [1, 700, 17, 64, 65, 2000, 128, 300]
    d = "cuda:0"
    parts = [Latent(n, H, 16, 16, rank, d, dtype, seed=i)
             for i, n in enumerate(lens)]
    width = max(p.table.shape[1] for p in parts)
    tables, caches, at = [], [], 0
    for p in parts:
        p.put(0, p.q.shape[0])
        row = torch.zeros(1, width, dtype=torch.int32)
        row[:, :p.table.shape[1]] = p.table + at
        at += p.cache.shape[0]
        tables.append(row)
        caches.append(p.cache)
    a = parts[0]
    uk_t = a.uk.to(d).view(H, 16, rank).transpose(1, 2).contiguous()
    out = torch.empty((len(lens), H * 16), dtype=dtype, device=d)
    ops.latent_decode(
        torch.cat([p.q[-1:] for p in parts]).to(d),
        torch.cat([p.gate[-1:, :H * 16] for p in parts]).to(d),
        torch.cat(caches), i32([n - 1 for n in lens], d),
        torch.cat(tables).to(d), a.scale, uk_t,
        a.uv.to(d).view(H, 16, rank), out)
    for i, p in enumerate(parts):
        p.uk, p.uv = a.uk, a.uv
        T, f = p.q.shape[0], torch.Tensor.double
        k = (f(p.c) @ f(p.uk).T).view(T, H, 16)
        v = (f(p.c) @ f(p.uv).T).view(T, H, 16)
        s = torch.softmax((k * f(p.q[-1]).view(1, H, 16)).sum(-1) * p.scale,
                          0)
        want = (s[:, :, None] * v).sum(0).reshape(1, -1) * torch.sigmoid(
            f(p.gate[-1:, :H * 16]))
        assert rel(out[i:i + 1], want) < 2 * tol(dtype), lens[i]


@GPU
def test_several_portions_in_one_prompt_call():
    """Portions of three sequences at different positions, both forms."""
    d, H, dim, vdim, rank = "cuda:0", 4, 32, 40, 96
    a = [Latent(200, H, dim, vdim, rank, d, BF16, seed=s, wide=0)
         for s in range(3)]
    for x in a:
        x.uk, x.uv = a[0].uk, a[0].uv
        x.put(0, 200)
    at, tables = 0, []
    for x in a:
        tables.append(x.table + at)
        at += x.cache.shape[0]
    cuts = [(0, 70), (130, 2), (61, 139)]
    uk, uv = a[0].uk.to(d), a[0].uv.to(d)
    uk_t = uk.view(H, dim, rank).transpose(1, 2).contiguous()
    portions, row = [], 0
    for s, (p0, n) in enumerate(cuts):
        portions.append(Portion(row, p0, n, s))
        row += n
    for expand in (False, True):
        out = torch.empty((row, H * vdim), dtype=BF16, device=d)
        ops.latent_prefill(
            torch.cat([x.q[p:p + n] for x, (p, n) in zip(a, cuts)]).to(d),
            torch.cat([x.gate[p:p + n] for x, (p, n) in zip(a, cuts)]).to(d),
            torch.cat([x.cache for x in a]), torch.cat(tables).to(d),
            PromptRows(portions, d), a[0].scale, uk_t,
            uv.view(H, vdim, rank), uk, uv, out, expand)
        for x, p in zip(a, portions):
            assert rel(out[p.row0:p.row0 + p.n],
                       x.want()[p.pos0:p.pos0 + p.n]) < 2 * tol(BF16)


def test_the_cheaper_form_is_chosen_by_cost():
    def one(pos0, n):
        return ops.expands(PromptRows([Portion(0, pos0, n, 0)], "cpu"),
                           512, 128, 128)
    assert one(0, 2048) and one(4096, 512)
    assert not one(4096, 2) and not one(30000, 16)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("q_rank,kv_rank", [(48, 64), (19, 27), (1536, 512),
                                            (1, 520)])
def test_latent_norms_and_cache(q_rank, kv_rank, device, dtype):
    T, eps = 7, 2e-3
    proj = rnd((T, q_rank + kv_rank + 8), 1, dtype, 0.05)
    wq, wk = 1 + rnd((q_rank,), 2, F32, 0.3), 1 + rnd((kv_rank,), 3, F32, 0.3)
    cache = torch.full((4, 1, 16, kv_rank), NAN, dtype=dtype, device=device)
    slots = [5, 63, 16, 0, 31, 32, 47]
    cq = ops.latent_prep(proj.to(device), wq.to(device), wk.to(device), eps,
                         cache, i32(slots, device))
    p = proj.double()
    assert rel(cq, plain.rms(p[:, :q_rank], eps) * wq) < tol(dtype)
    flat = cache.view(64, kv_rank)
    assert rel(flat[slots], plain.rms(p[:, q_rank:q_rank + kv_rank], eps)
               * wk) < tol(dtype)
    assert int(torch.isnan(flat[:, 0]).sum()) == 64 - T


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("T,H,N,K", [(1, 3, 64, 128), (16, 2, 40, 24),
                                     (33, 5, 17, 256), (70, 4, 96, 512),
                                     (130, 1, 7, 5), (17, 16, 512, 64)])
def test_head_linear(T, H, N, K, device, dtype):
    x = rnd((T, H * K + 8), 1, dtype)
    w = rnd((H, N, K), 2, dtype, K ** -0.5)
    gate = rnd((T, H * N + 8), 3, dtype)
    out = torch.full((T, H * N + 8), NAN, dtype=dtype, device=device)
    xs = x.to(device)[:, :H * K]
    want = (x[:, :H * K].double().view(T, H, 1, K)
            * w.double()[None]).sum(-1).flatten(1)
    assert rel(ops.head_linear(xs, w.to(device)), want) < tol(dtype)
    ops.head_linear(xs, w.to(device), gate.to(device)[:, 8:],
                    out[:, 8:])
    assert rel(out[:, 8:], want * torch.sigmoid(gate[:, 8:].double())) \
        < tol(dtype)
    assert torch.isnan(out[:, :8]).all()


@GPU
def test_fp8_latents():
    T = 200
    a = Latent(T, 8, 32, 32, 128, "cuda:0", BF16,
               cache_dtype=torch.float8_e4m3fn)
    a.put(0, T)
    a.c = a.cache.float().cpu()[a.table[0].long(), 0].reshape(-1, 128)[:T] \
        .to(BF16)
    want = a.want()
    for expand in (False, True):
        assert rel(a.call(0, T, expand), want) < 2 * tol(BF16)
    assert rel(a.call(T - 1, 1), want[-1:]) < 2 * tol(BF16)


# --------------------------------------------------------------- HGRN2
def hgrn2_case(T, H, dim, vdim, bias, low, seed, dtype):
    """low: bounds up to this; bias: of the forget gate (steep below 0)."""
    proj = rnd((T, H * (2 * dim + vdim)), seed, dtype)
    b = rnd((H * dim,), seed + 1, F32) + bias
    lower = torch.rand(H * dim, generator=torch.Generator()
                       .manual_seed(seed + 2)) * low
    norm, eps = 1 + rnd((vdim,), seed + 3, F32, 0.2), 1e-4
    q, z, v = torch.split(proj.double(), [H * dim, H * dim, H * vdim], 1)
    q = (q * torch.sigmoid(q)).view(T, H, dim)
    f = plain.forget(z + b.double(), lower.double()).view(T, H, dim)
    o, S = plain.recur(q, v.reshape(T, H, vdim), f)
    want = (plain.rms(o, eps) * norm).reshape(T, -1)
    return proj, b, lower, norm, eps, want, S


HGRN2 = [(129, 3, 32, 48, 2.0, 0.9), (150, 2, 20, 18, 0.0, 0.0),
         (97, 2, 128, 64, 6.0, 0.99), (80, 1, 256, 33, 1.0, 0.5),
         (200, 2, 64, 160, -4.0, 0.0), (70, 1, 33, 17, -12.0, 0.0),
         (66, 1, 8, 8, 9.0, 1.0), (131, 1, 48, 300, -6.0, 0.1)]


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("case", HGRN2, ids=str)
def test_hgrn2(case, device, dtype):
    T, H, dim, vdim, bias, low = case
    proj, b, lower, norm, eps, want, S = hgrn2_case(
        T, H, dim, vdim, bias, low, dim + T, dtype)
    proj, b, lower, norm = (t.to(device) for t in (proj, b, lower, norm))
    # steep decays: what is left is the rounding of the running log-decay
    t = max(tol(dtype), 3e-5 if bias < -2 else 1e-5)

    def start():
        # a used slot: what the last owner left must not be seen
        return torch.full((3, H, dim, -(-vdim // 4) * 4), NAN, device=device)

    def prompt(state, p0, n):
        return ops.hgrn2_prefill(
            proj[p0:p0 + n].contiguous(), b, lower, norm, state,
            PromptRows([Portion(0, p0, n, 0, 2)], device), vdim, eps)

    def token(state, p):
        return ops.hgrn2_decode(
            proj[p:p + 1].contiguous(), b, lower, norm, state,
            i32([2], device), i32([p], device), vdim, eps)

    st = start()
    assert rel(prompt(st, 0, T), want) < t
    assert rel(st[2, :, :, :vdim], S) < 3e-5
    st = start()
    assert rel(torch.cat([token(st, p) for p in range(T)]), want) < t
    assert rel(st[2, :, :, :vdim], S) < 3e-5
    st, got, p = start(), [], 0
    for n in [2, 17, 1, 3, 15, 16, 1, T - 55]:
        got.append(token(st, p) if n == 1 else prompt(st, p, n))
        p += n
    assert rel(torch.cat(got), want) < t
    assert rel(st[2, :, :, :vdim], S) < 3e-5


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_hgrn2_writes_a_column_range(device, dtype):
    """Unequal sequences in one launch, output beside something else."""
    H, dim, vdim = 2, 24, 20
    cases = [hgrn2_case(n, H, dim, vdim, 1.0, 0.8, 7, dtype)
             for n in (5, 130, 64)]
    _, b, lower, norm, eps, _, _ = cases[0]
    proj = torch.cat([c[0] for c in cases]).to(device)
    out = torch.full((199, H * vdim + 8), NAN, dtype=dtype, device=device)
    st = torch.full((4, H, dim, vdim), NAN, device=device)
    rows = [Portion(0, 0, 5, 0, 3), Portion(5, 0, 130, 1, 0),
            Portion(135, 0, 64, 2, 1)]
    ops.hgrn2_prefill(proj, b.to(device), lower.to(device), norm.to(device),
                      st, PromptRows(rows, device), vdim, eps,
                      out[:, :H * vdim])
    for c, p in zip(cases, rows):
        assert rel(out[p.row0:p.row0 + p.n, :H * vdim], c[5]) \
            < max(tol(dtype), 1e-5)
        assert rel(st[p.slot], c[6]) < 1e-5
    assert torch.isnan(out[:, H * vdim:]).all()


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_hgrn2_remembers_over_a_long_sequence(device, dtype):
    """One loud value far back, gates that forget almost nothing since."""
    T, H, dim, vdim = 900, 1, 16, 16
    proj = torch.zeros(T, H * (2 * dim + vdim), dtype=dtype)
    proj[:, :dim] = 1.0
    proj[:, dim:2 * dim] = 14.0
    proj[3, dim:2 * dim] = -14.0
    proj[3, 2 * dim:] = rnd((vdim,), 1, dtype, 4.0)
    b, lower = torch.zeros(dim), torch.linspace(0, 0.5, dim)
    norm, eps = torch.ones(vdim), 1e-3
    q, z, v = torch.split(proj.double(), [dim, dim, vdim], 1)
    o, _ = plain.recur((q * torch.sigmoid(q))[:, None], v[:, None],
                       plain.forget(z + b, lower.double())[:, None])
    want = plain.rms(o, eps).reshape(T, -1)
    st = torch.full((1, H, dim, vdim), NAN, device=device)
    args = [t.to(device) for t in (b, lower, norm)]
    got = ops.hgrn2_prefill(proj[:-1].contiguous().to(device), *args, st,
                            PromptRows([Portion(0, 0, T - 1, 0, 0)], device),
                            vdim, eps)
    last = ops.hgrn2_decode(proj[-1:].contiguous().to(device), *args, st,
                            i32([0], device), i32([T - 1], device), vdim, eps)
    assert float(want[-1].abs().mean()) > 0.3
    assert rel(got, want[:-1]) < max(tol(dtype), 1e-5)
    assert rel(last, want[-1:]) < max(tol(dtype), 1e-5)
