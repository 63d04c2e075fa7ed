"""Each Fimunex mechanism alone, CPU form and HIP kernels, against the plain
equations: YaRN angles, differential attention in chunks, the router and its
experts, biases and parts in the residual step.  Inputs are made so that one
wrong key, edge, map, bias, group or route shows."""

import math

import pytest
import torch

import fimunex_plain as plain
import resilient_llm_amd.ops as ops
from nesizen_util import BF16, DEVICES, F32, GPU, TARGETS
from resilient_llm_amd.engine.batch import Portion, PromptRows

D64 = torch.float64


def rel(got, want):
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all()
    return float((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())


def tol(dtype):
    return 3e-6 if dtype == F32 else 1.2e-2


def rnd(shape, seed, dtype, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(dtype)


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=device)


# ----------------------------------------------------------------- angles
YARN = [(32, 10000.0, 5.0, 2048, 24.0, 1.5), (8, 500.0, 1.0, 64, 4.0, 0.5),
        (64, 1e6, 16.0, 4096, 32.0, 1.0), (2, 100.0, 3.0, 50, 2.0, 1.0),
        # both ends beyond the pairs, and a ramp of no width
        (16, 1000.0, 8.0, 1 << 20, 1e5, 1e4), (16, 1000.0, 8.0, 2, 8.0, 4.0),
        (24, 10000.0, 2.5, 512, 7.0, 7.0)]


@pytest.mark.parametrize("case", YARN, ids=str)
def test_yarn_angles(case):
    dims, _, factor = case[:3]
    table = ops.yarn_cos_sin(40, *case)
    assert table.shape == (40, dims) and table.dtype == F32
    freqs = plain.yarn_frequencies(*case)
    gain = 0.1 * math.log(factor) + 1
    for pos in (0, 1, 17, 39):
        x = rnd((dims + 3,), pos, D64)
        want = plain.rotate_halves(x, pos, freqs, gain)
        c, s = table[pos].double().chunk(2)
        u, v = x[:dims // 2], x[dims // 2:dims]
        got = torch.cat([u * c - v * s, v * c + u * s, x[dims:]])
        assert rel(got, want) < 1e-6
    whole = rnd((40, 2, dims + 3), 5, D64)
    want = plain.rotate_all(whole, freqs, gain)
    assert rel(want[17, 1], plain.rotate_halves(whole[17, 1], 17, freqs,
                                                gain)) < 1e-12


# --------------------------------------------------- differential attention
class Diff:
    """A paged cache with scattered, poisoned pages and the op calls."""

    def __init__(self, T, H, G, dim, vdim, rot, chunk, device, dtype, cap=9.0,
                 lam=0.4, out_scale=0.7, eps=1e-3, scale=None, seed=0,
                 bias=True, gate=True, extra=0, cache_dtype=None, size=1.0):
        self.T, self.H, self.G, self.dim, self.vdim = T, H, G, dim, vdim
        self.device, self.dtype, self.rot = device, dtype, rot
        self.chunk, self.cap, self.lam = chunk, cap, lam
        self.out_scale, self.eps = out_scale, eps
        self.scale = dim ** -0.5 if scale is None else scale
        n = 2 * dim * (H + G) + G * vdim
        cols = n + (H if gate else 0) + extra
        self.rows = rnd((T, cols + -cols % 8 if extra == 0 else cols), seed,
                        dtype, size)
        self.gate = gate
        self.n = n
        self.bias = rnd((n,), seed + 1, F32, 0.5 * size) if bias else None
        self.qn = 1.3 + rnd((dim,), seed + 2, F32, 0.3)
        self.kn = 1.3 + rnd((dim,), seed + 3, F32, 0.3)
        self.yarn = (rot, 100.0, 4.0, 40, 4.0, 0.5)
        self.cs = ops.yarn_cos_sin(T + 1, *self.yarn, device=device) \
            if rot else None
        pages = -(-T // 16)
        perm = torch.randperm(pages + 3, generator=torch.Generator()
                              .manual_seed(seed))[:pages]
        self.table = perm.to(torch.int32)[None].contiguous().to(device)
        cd = cache_dtype or dtype
        self.kc = torch.full((pages + 3, G, 16, 2 * dim), float("nan")) \
            .to(cd).to(device)
        self.vc = torch.full((pages + 3, G, 16, vdim), float("nan")) \
            .to(cd).to(device)

    def slots(self, p0, n):
        p = torch.arange(p0, p0 + n)
        t = self.table[0].cpu()[p // 16].long()
        return (t * 16 + p % 16).to(torch.int32).to(self.device)

    def tail(self):
        dev = self.device
        return (self.H, None if self.bias is None else self.bias.to(dev),
                self.qn.to(dev), self.kn.to(dev), self.scale, self.chunk,
                self.cap, self.lam, self.out_scale, self.eps)

    def run(self, p0, n, decode=False):
        x = self.rows[p0:p0 + n].clone().to(self.device)
        gate = x[:, self.n:self.n + self.H] if self.gate else None
        pos = torch.arange(p0, p0 + n, dtype=torch.int32, device=self.device)
        if decode:
            return ops.diff_decode(
                x, gate, self.kc, self.vc, pos, self.cs, self.slots(p0, n),
                self.table.expand(n, -1).contiguous(), *self.tail())
        return ops.diff_prefill(
            x, gate, self.kc, self.vc, pos, self.cs, self.slots(p0, n),
            self.table, PromptRows([Portion(0, p0, n, 0)], self.device),
            *self.tail())

    def want(self):
        T, H, G, dim, vdim = self.T, self.H, self.G, self.dim, self.vdim
        x = self.rows[:, :self.n].double()
        if self.bias is not None:
            x = x + self.bias.double()
        q, k, v = torch.split(x, [2 * H * dim, 2 * G * dim, G * vdim], 1)
        q = plain.rms(q.view(T, H, 2, dim), self.eps) * self.qn.double()
        k = plain.rms(k.view(T, G, 2, dim), self.eps) * self.kn.double()
        if self.rot:
            f = plain.yarn_frequencies(*self.yarn)
            gain = 0.1 * math.log(self.yarn[2]) + 1
            q, k = (plain.rotate_all(t, f, gain) for t in (q, k))
        out = []
        for h in range(H):
            g = h // (H // G)
            a1, a2 = (plain.softmax_map(
                q[:, h, i], k[:, g, i], v.view(T, G, vdim)[:, g], self.scale,
                self.cap, self.chunk) for i in range(2))
            o = plain.rms(a1 - self.lam * a2, self.eps) * self.out_scale
            if self.gate:
                o = o * torch.sigmoid(self.rows[:, self.n + h].double())[:,
                                                                         None]
            out.append(o)
        return torch.cat(out, 1)


# heads, kv heads, dim of a map, vdim, rotation
SHAPES = [(3, 1, 10, 14, 6), (2, 2, 8, 8, 8), (4, 2, 32, 64, 32),
          (8, 2, 64, 128, 64), (6, 2, 48, 96, 16), (5, 1, 24, 72, 20),
          (10, 1, 64, 64, 32), (9, 1, 48, 48, 0), (2, 1, 80, 200, 80),
          (17, 1, 128, 256, 128), (1, 1, 96, 136, 2), (12, 4, 16, 24, 16),
          (4, 4, 128, 32, 48), (2, 1, 16, 256, 16), (2, 1, 160, 40, 64)]


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("shape", SHAPES, ids=str)
def test_attention_sizes(shape, device, dtype):
    H, G, dim, vdim, rot = shape
    T = 150
    for k, chunk in enumerate((30, 64, 1000)):
        a = Diff(T, H, G, dim, vdim, rot, chunk, device, dtype, seed=dim + k)
        want = a.want()
        assert rel(a.run(0, T), want) < tol(dtype)
        got = torch.cat([a.run(0, 41), a.run(41, 1, decode=True),
                         a.run(42, 2), a.run(44, 1, decode=True),
                         a.run(45, T - 46), a.run(T - 1, 1, decode=True)])
        assert rel(got, want) < tol(dtype), chunk


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("shape", [(3, 1, 10, 14, 6), (6, 2, 32, 40, 16)],
                         ids=str)
def test_token_by_token(shape, device, dtype):
    """Decoding alone fills the cache, over edges of chunks and pages."""
    a = Diff(140, *shape, 37, device, dtype, seed=3)
    got = torch.cat([a.run(p, 1, decode=True) for p in range(140)])
    assert rel(got, a.want()) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("bias,gate,extra", [(False, True, 0),
                                             (True, False, 0), (True, True, 3),
                                             (False, False, 0)])
def test_bias_gate_and_odd_row_widths(bias, gate, extra, device, dtype):
    a = Diff(50, 4, 2, 16, 32, 16, 20, device, dtype, bias=bias, gate=gate,
             extra=extra, seed=1)
    got = torch.cat([a.run(0, 33), a.run(33, 1, decode=True), a.run(34, 16)])
    assert rel(got, a.want()) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("cap,scale", [(0.5, 1.0), (3.0, 0.1), (50.0, 4.0)])
def test_caps_and_scales(cap, scale, device, dtype):
    """Scores far above the cap, around it, and far below."""
    a = Diff(90, 2, 1, 32, 32, 32, 60, device, dtype, cap=cap, scale=scale,
             seed=4)
    got = torch.cat([a.run(0, 70), *[a.run(p, 1, decode=True)
                                     for p in range(70, 90)]])
    # at 16 bits a rounded query moves a sharp score by its own size
    assert rel(got, a.want()) < (tol(dtype) if scale < 2 or dtype == F32
                                 else 0.15)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("lam,size", [(0.0, 1.0), (-0.6, 1.0), (1.7, 1.0),
                                      (0.3, 0.02)])
def test_difference_and_its_norm(lam, size, device, dtype):
    """Any lambda; outputs so small that eps matters."""
    a = Diff(60, 3, 1, 16, 24, 16, 40, device, dtype, lam=lam, size=size,
             eps=2e-3, seed=6)
    got = torch.cat([a.run(0, 45), *[a.run(p, 1, decode=True)
                                     for p in range(45, 60)]])
    assert rel(got, a.want()) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("chunk", [1, 2, 15, 16, 17, 40, 64, 65, 100, 128,
                                   10**9])
@pytest.mark.parametrize("dim,vdim", [(32, 32), (12, 20)])
def test_chunk_edges_show(dim, vdim, chunk, device, dtype):
    """One loud key per case, in one map, at and around the edges of chunks:
    let in or left out by one position it changes the output at order one.
    Prompt, portions and decode."""
    T = 160
    edges = {0, 1, 15, 16, 63, 64, 127, 128, T - 1}
    for c in range(1, 3):
        edges |= {c * chunk - 1, c * chunk, c * chunk + 1}
    for map_ in range(2):
        a = Diff(T, 2, 1, dim, vdim, 0, chunk, device, dtype, cap=30.0,
                 scale=0.5, bias=False, gate=False, lam=0.5, seed=chunk % 97)
        x = a.rows.float()
        x[:, :4 * dim] = 1.0                              # every query alike
        k = torch.ones(T, 2, dim)
        k[:, :, ::2] = -1.0                               # keys across it
        for j in edges:
            if 0 <= j < T:
                k[j, map_] = 1.0                          # but these along
        x[:, 4 * dim:6 * dim] = k.reshape(T, -1)
        a.rows = x.to(dtype)
        want = a.want()
        assert rel(a.run(0, T), want) < tol(dtype)
        for p in (0, 1, 15, 16, 17, 39, 40, 41, 63, 64, 65, 80, 127, 128, 129,
                  159):
            d = a.run(p, 1, decode=True)
            assert rel(d, want[p:p + 1]) < tol(dtype), p
        for p0, n in ((89, 2), (90, 3), (64, 1), (63, 2), (100, 60), (31, 97)):
            assert rel(a.run(p0, n), want[p0:p0 + n]) < tol(dtype), (p0, n)


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_a_far_key_is_found(device, dtype):
    """One loud key hundreds back, in map 1 only."""
    T, dim = 700, 32
    a = Diff(T, 2, 1, dim, 32, 8, 1024, device, dtype, cap=30.0, scale=0.6,
             bias=False, seed=2)
    a.rows[:, 8:32] = 1.0
    k = a.rows[:, 4 * dim:4 * dim + 32]
    k[:, 8::2], k[:, 9::2] = 1.0, -1.0
    quiet = a.want()
    k[23, 8:] = 3.0
    want = a.want()
    assert rel(quiet[100:], want[100:]) > 0.1
    assert rel(a.run(0, T), want) < tol(dtype)
    for p in (300, 648, 690, 699):
        assert rel(a.run(p, 1, decode=True), want[p:p + 1]) < tol(dtype)
    for p0, n in ((500, 2), (640, 60)):
        assert rel(a.run(p0, n), want[p0:p0 + n]) < tol(dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("dim,vdim", [(32, 48), (10, 18)])
def test_several_portions_in_one_call(dim, vdim, device, dtype):
    """Sequences at different places of their chunks, gathered together."""
    T, chunk = 260, 100
    cases = [Diff(T, 4, 2, dim, vdim, 4, chunk, device, dtype, seed=9)
             for _ in range(4)]
    a = cases[0]
    spans = [(0, 40), (90, 30), (199, 2), (230, 30)]
    want = a.want()
    P = a.kc.shape[0]
    for c, (p0, _) in zip(cases, spans):
        if p0:
            c.run(0, p0)
    kc, vc = (torch.cat([getattr(c, x) for c in cases]) for x in ("kc", "vc"))
    tables = torch.cat([a.table + P * i for i in range(4)]).contiguous()
    rows = torch.cat([a.rows[p:p + n] for p, n in spans]).to(device)
    slots = torch.cat([a.slots(p, n) + 16 * P * i
                       for i, (p, n) in enumerate(spans)]).to(torch.int32)
    pos = torch.cat([torch.arange(p, p + n) for p, n in spans])
    portions, at = [], 0
    for i, (p, n) in enumerate(spans):
        portions.append(Portion(at, p, n, i))
        at += n
    got = ops.diff_prefill(
        rows, rows[:, a.n:a.n + a.H], kc, vc,
        pos.to(torch.int32).to(device), a.cs, slots, tables,
        PromptRows(portions, device), *a.tail())
    assert rel(got, want[pos]) < tol(dtype)


def test_gathered_rows_start_with_the_chunk():
    rows = PromptRows([Portion(0, 230, 30, 0), Portion(30, 0, 5, 2),
                       Portion(35, 64, 1, 1)], "cpu")
    blocks, off, total = rows.gathered(64, 100)
    # from 200 on, aligned down to 192; from 0; from 0 (64 lies in chunk 0)
    assert blocks.t().tolist() == [[0, 192, 64, 0], [0, 256, 4, 64],
                                   [2, 0, 5, 128], [1, 0, 64, 192],
                                   [1, 64, 1, 256]]
    assert off.tolist() == [-192, 192, 128] and total == 320
    assert rows.gathered(64)[2] == 320 + 64 + 128


@GPU
@pytest.mark.parametrize("shape", [(8, 2, 32, 64, 32), (16, 1, 64, 128, 32),
                                   (5, 1, 16, 200, 16)], ids=str)
def test_decode_batches_and_splits(shape):
    """Many sequences in one decode launch, few enough for key splits and
    enough for none, lengths from 1 up."""
    H, G, dim, vdim, rot = shape
    a = Diff(300, H, G, dim, vdim, rot, 270, "cuda:0", BF16)
    a.run(0, 300)
    want = a.want()
    n = a.table.shape[1]
    for B in (1, 3, 40, 300):
        lens = [1 + (37 * b + 290 * (B == 1)) % 300 for b in range(B)]
        kc = a.kc[a.table[0].long()].repeat(B, 1, 1, 1)
        vc = a.vc[a.table[0].long()].repeat(B, 1, 1, 1)
        pos = torch.tensor(lens, dtype=torch.int32) - 1
        tab = torch.arange(B * n, dtype=torch.int32).view(B, n)
        slots = tab[torch.arange(B), pos.long() // 16] * 16 + pos % 16
        x = a.rows[pos.long()].cuda()
        got = ops.diff_decode(
            x, x[:, a.n:a.n + H], kc, vc, pos.cuda(), a.cs,
            slots.to(torch.int32).cuda(), tab.cuda(), *a.tail())
        assert rel(got, want[pos.long()]) < tol(BF16), B


@GPU
def test_fp8_cache():
    a = Diff(120, 8, 2, 64, 64, 32, 70, "cuda:0", BF16,
             cache_dtype=torch.float8_e4m3fn)
    got = torch.cat([a.run(0, 100), *[a.run(i, 1, decode=True)
                                      for i in range(100, 120)]])
    assert rel(got, a.want()) < 0.12


# ---------------------------------------------------------------- experts
def moe_case(T, W, E, I, ff, seed, dtype):
    h = rnd((T, W), seed, dtype)
    router = rnd((E + I, W), seed + 1, dtype, 2.0 * W ** -0.5)
    # choice scores of both signs
    correction = rnd((E + I,), seed + 2, F32, 0.3) - 0.2
    up = rnd((E, ff, W), seed + 3, dtype, 1.5 * W ** -0.5)
    down = rnd((E, W, ff), seed + 4, dtype, ff ** -0.5)
    return h, router, correction, up, down


def pad_experts(up, down):
    n = -up.shape[1] % 64
    return (torch.nn.functional.pad(up, (0, 0, 0, n)).contiguous(),
            torch.nn.functional.pad(down, (0, n)).contiguous())


# tokens, width, experts, identities, top, ff, groups, kept
MOE = [(1, 64, 4, 0, 1, 64, 1, 1), (5, 72, 5, 1, 3, 40, 3, 2),
       (33, 128, 8, 4, 2, 96, 4, 2), (64, 256, 40, 5, 8, 64, 9, 4),
       (7, 64, 2, 1, 3, 16, 1, 1), (50, 64, 100, 30, 2, 32, 13, 5),
       (20, 64, 200, 50, 70, 16, 5, 3), (16, 64, 40, 8, 1, 16, 48, 1),
       (300, 128, 4, 1, 2, 80, 5, 3), (1500, 64, 5, 0, 3, 64, 5, 4),
       (2100, 128, 9, 3, 2, 200, 3, 1), (30, 1088, 20, 4, 4, 192, 6, 2),
       (9, 64, 3, 3, 4, 24, 2, 2)]


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("case", MOE, ids=str)
def test_router_and_experts(case, device, dtype):
    T, W, E, I, top, ff, count, keep = case
    h, router, correction, up, down = moe_case(T, W, E, I, ff, T + E, dtype)
    dev = [t.to(device) for t in (h, router, correction)]
    ids, wts = (t.cpu() for t in ops.moe_route_softmax(*dev, top, count,
                                                       keep))
    z = h.double() @ router.double().T
    for t in range(T):
        want, w = plain.choose(z[t], correction.double(), top, count, keep)
        assert ids[t].tolist() == want, t
        assert torch.allclose(wts[t].double(), w, atol=1e-5)
    packed = [t.to(device) for t in pad_experts(up, down)]
    y, ids2, wts2 = ops.moe_relu2(*dev, *packed, top, count, keep)
    assert torch.equal(ids2.cpu(), ids) and torch.equal(wts2.cpu(), wts)
    parts = torch.zeros(T, top, W, dtype=D64)
    for e in range(E):
        t, c = torch.nonzero(ids == e, as_tuple=True)
        parts[t, c] = wts[t, c][:, None].double() * plain.expert(
            h[t].double(), up[e].double(), down[e].double())
    own = (ids < E)[..., None]
    got = y.cpu().masked_fill(~own, 0)
    if own.any():
        assert rel(got, parts) < tol(dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_closed_groups_lose_also_where_choice_scores_are_negative(device):
    """All choice scores below zero: a closed group is not chosen, however
    much that would gain."""
    h = torch.ones(1, 64)
    router = torch.zeros(12, 64)
    correction = torch.tensor([-9.0, -1, -8, -7, -2, -3, -6, -5, -4, -1.5,
                               -20, -30])
    # groups of three lead with -1, -2, -4, -1.5: the first and last stay
    ids, w = ops.moe_route_softmax(h.to(device), router.to(device),
                                   correction.to(device), 5, 4, 2)
    assert ids.tolist() == [[1, 9, 2, 0, 10]]
    assert torch.allclose(w.cpu(), torch.full((1, 5), 0.2))


@pytest.mark.parametrize("device", DEVICES)
def test_router_ties_go_to_the_lower_route_and_group(device):
    h = torch.ones(3, 64).to(device)
    router = torch.zeros(70, 64)
    router[[66, 5, 20]] = 0.1
    none = torch.zeros(70)
    ids, _ = ops.moe_route_softmax(h, router.to(device), none.to(device), 4,
                                   1, 1)
    assert ids.tolist() == [[5, 20, 66, 0]] * 3
    ids, _ = ops.moe_route_softmax(h, router.to(device), None, 4, 7, 2)
    assert ids.tolist() == [[5, 20, 0, 1]] * 3


# ----------------------------------------------------------- residual step
@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("W,taps", [(40, 1), (256, 4), (264, 3), (1028, 2),
                                    (2048, 4), (4100, 4), (8200, 2), (30, 6)])
def test_parts_and_biases_in_the_residual_step(W, taps, device, dtype):
    """Identity parts read the block's input, whatever their rows of y hold;
    norm and (for the decoded rows) convolution follow in the same pass."""
    T, parts, E, eps, nd = 7, 5, 4, 1e-3, 4
    x0 = rnd((T, W), 1, F32)
    y = rnd((T, parts, W), 2, dtype)
    h = rnd((T, W), 3, dtype)
    wts = torch.rand(T, parts, generator=torch.Generator().manual_seed(4))
    ids = torch.randint(0, E + 3, (T, parts), dtype=torch.int32,
                        generator=torch.Generator().manual_seed(5))
    ids[0], ids[1] = 1, E                       # all experts, all identities
    same = (ids >= E)[..., None]
    y = y.masked_fill(same, float("nan"))
    gain = 1 + rnd((W,), 6, F32, 0.3)
    w = rnd((taps, W), 7, F32, 0.5)
    ring = max(taps - 1, 1)
    tail = rnd((T, ring, W), 8, dtype)
    pos = i32([0, 1, 5, 9, 3, 2, 7], device)
    slots = i32([3, 0, 5, 1], device)

    def dev(t):
        return t.to(device)

    def check(new, x, hh, hc, t0):
        assert rel(x, new) < 3e-6
        n = plain.rms(new, eps) * gain.double()
        assert rel(hh, n) < tol(dtype)
        for r in range(nd):
            p, s = int(pos[r]), int(slots[r])
            past = [hh[r].double().cpu()]
            past += [t0[s, (p - k) % ring].double() if p >= k else
                     torch.zeros(W, dtype=D64) for k in range(1, taps)]
            seq = torch.stack(past[::-1])
            want = plain.with_past(seq, w.double().T)[-1]
            assert rel(hc[r], want) < tol(dtype), r
    new = x0.double() + torch.where(
        same, wts[..., None].double() * h.double()[:, None],
        y.double()).sum(1)
    x, tl = dev(x0.clone()), dev(tail.clone())
    hh, hc = ops.block_step(
        x, dev(y), dev(gain), 1, eps, pos, dev(w), tl, slots, nd,
        part_ids=dev(ids), part_w=dev(wts), part_h=dev(h), part_limit=E)
    check(new, x, hh, hc, tail)
    rows = torch.tensor([4, 1])
    x = dev(x0.clone())
    last, _ = ops.block_step(
        x, dev(y), dev(gain), 1, eps, pos, rows=dev(rows), keep=False,
        part_ids=dev(ids), part_w=dev(wts), part_h=dev(h), part_limit=E)
    assert rel(last, (plain.rms(new, eps) * gain.double())[rows]) < tol(dtype)
    assert torch.equal(x.cpu(), x0)
    one, bias = rnd((T, W), 9, dtype), rnd((W,), 10, F32)
    x, tl = dev(x0.clone()), dev(tail.clone())
    hh, hc = ops.block_step(x, dev(one), dev(gain), 1, eps, pos, dev(w), tl,
                            slots, nd, y_bias=dev(bias))
    check(x0.double() + one.double() + bias.double(), x, hh, hc, tail)
