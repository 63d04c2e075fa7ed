"""CPU forms of the mixed-layer ops (same signatures and layouts as
torch.ops.rlli_mix), in f32 PyTorch: the no-GPU path of the engine tests
and what the HIP kernels' op tests are compared with."""

from __future__ import annotations

import torch
import torch.nn.functional as F

GLA_CHUNK = 64


def _norm(x, gain, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * gain


def hyper_embed(ids, table, w_embed, x, in_w, gain, eps):
    e = _norm(table[ids.long()].float(), w_embed, eps)
    x.copy_(e.unsqueeze(1).expand_as(x))
    return _norm(torch.einsum("s,tsw->tw", in_w, x), gain, eps) \
        .to(table.dtype)


def hyper_step(x, y, mix, out_w, in_w, gain, eps, rows, keep):
    dtype = y.dtype
    y = y.float()
    if y.dim() == 3:
        y = y.sum(1)
    new = torch.einsum("st,nsw->ntw", mix, x) \
        + out_w[None, :, None] * y[:, None]
    if keep:
        x.copy_(new)
    if rows is not None:
        new = new[rows]
    u = new.sum(1) if in_w is None else torch.einsum("s,tsw->tw", in_w, new)
    return _norm(u, gain, eps).to(dtype)


def relu2(x):
    r = torch.relu(x.float())
    return (r * r).to(x.dtype)


# ------------------------------------------------------ window attention
def rotate_pairs(x, positions, cos_sin):
    """x [T, H, D]; pairs (2i, 2i+1) of the first cos_sin.shape[1] dims."""
    rot = cos_sin.shape[1]
    cs = cos_sin[positions.long()]
    c, s = cs[:, None, :rot // 2], cs[:, None, rot // 2:]
    xf = x.float()
    u, v = xf[..., 0:rot:2], xf[..., 1:rot:2]
    turned = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)
    return torch.cat([turned, xf[..., rot:]], -1).to(x.dtype)


def _split_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                  has_kv):
    T = qkv.shape[0]
    _, G, bs, D = k_cache.shape
    V = v_cache.shape[3]
    q = rotate_pairs(qkv[:, :n_q * D].reshape(T, n_q, D), positions, cos_sin)
    if has_kv:
        k = rotate_pairs(qkv[:, n_q * D:(n_q + G) * D].reshape(T, G, D),
                         positions, cos_sin)
        v = qkv[:, (n_q + G) * D:].reshape(T, G, V)
        b, o = slots.long() // bs, slots.long() % bs
        k_cache[b, :, o] = k.to(k_cache.dtype)
        v_cache[b, :, o] = v.to(v_cache.dtype)
    return q


def _attend(q, qpos, k_cache, v_cache, table, sink, scale, window,
            keep_first):
    """q [n, H, D] at positions qpos over one sequence's cached tokens."""
    _, G, bs, D = k_cache.shape
    n_kv = int(qpos[-1]) + 1
    blocks = table[:-(-n_kv // bs)].long()
    k = k_cache[blocks].float().transpose(1, 2).reshape(-1, G, D)[:n_kv]
    v = v_cache[blocks].float().transpose(1, 2) \
        .reshape(-1, G, v_cache.shape[3])[:n_kv]
    H = q.shape[1]
    k = k.repeat_interleave(H // G, 1)
    v = v.repeat_interleave(H // G, 1)
    s = torch.einsum("nhd,mhd->hnm", q.float(), k) * scale
    i, j = qpos[:, None].long(), torch.arange(n_kv)[None]
    ok = (j <= i) & ((i - j < window) | (j < keep_first))
    s = s.masked_fill(~ok, float("-inf"))
    if sink is not None:
        s = torch.cat([s, sink[:, None, None].expand(-1, s.shape[1], 1)], -1)
    p = torch.softmax(s, -1)[..., :n_kv]
    return torch.einsum("hnm,mhd->nhd", p, v).reshape(q.shape[0], -1)


def window_prefill(qkv, k_cache, v_cache, positions, cos_sin, slots,
                   block_tables, prompt, sink, scale, n_q, window,
                   keep_first, has_kv):
    q = _split_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                      has_kv)
    out = torch.empty(qkv.shape[0], n_q * v_cache.shape[3], dtype=qkv.dtype)
    for p in prompt.portions:
        r = slice(p.row0, p.row0 + p.n)
        out[r] = _attend(q[r], positions[r], k_cache, v_cache,
                         block_tables[p.seq], sink, scale, window,
                         keep_first).to(qkv.dtype)
    return out


def window_decode(qkv, k_cache, v_cache, positions, cos_sin, slots,
                  block_tables, sink, scale, n_q, window, keep_first,
                  has_kv):
    q = _split_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                      has_kv)
    return torch.cat([
        _attend(q[b:b + 1], positions[b:b + 1], k_cache, v_cache,
                block_tables[b], sink, scale, window, keep_first)
        for b in range(qkv.shape[0])]).to(qkv.dtype)


# ------------------------------------------------- gated linear attention
def _gla_parts(proj, a2, a2_bias, state, vdim, tau):
    T = proj.shape[0]
    _, H, D, _ = state.shape
    pf = proj.float()
    q, k, v, g, a1 = torch.split(
        pf, [H * D, H * D, H * vdim, H * vdim, a2.shape[1]], dim=1)
    z = a1 @ a2.float().T + a2_bias
    alpha = torch.exp(F.logsigmoid(z) / tau).view(T, H, D)
    return (q.view(T, H, D) * D ** -0.5, k.view(T, H, D),
            v.view(T, H, vdim), g.view(T, H, vdim), alpha)


def _gla_out(o, g, norm, eps, dtype):
    return (_norm(o, norm, eps) * F.silu(g)).flatten(1).to(dtype)


def _step_states(q, k, v, alpha, state, slots, positions, vdim):
    S = state[slots.long()][..., :vdim]
    S[positions == 0] = 0.0               # a fresh sequence, a used slot
    S = alpha[..., None] * S + k[..., None] * v[:, :, None]
    state[slots.long(), :, :, :vdim] = S
    return torch.einsum("bhd,bhdv->bhv", q, S)


def _scan_states(q, k, v, alpha, state, tiles, seqs, vdim):
    o = torch.empty_like(v)
    for first, count, pos0, slot in seqs.t().tolist():
        S = state[slot, :, :, :vdim].clone()
        if pos0 == 0:
            S.zero_()
        row = int(tiles[0, first])
        n = int(tiles[2, first:first + count].sum())
        for t in range(row, row + n):
            S = alpha[t][..., None] * S + k[t][..., None] * v[t][:, None]
            o[t] = torch.einsum("hd,hdv->hv", q[t], S)
        state[slot, :, :, :vdim] = S
    return o


def gla_decode(proj, a2, a2_bias, norm, state, slots, positions, vdim, tau,
               eps, out):
    q, k, v, g, alpha = _gla_parts(proj, a2, a2_bias, state, vdim, tau)
    o = _step_states(q, k, v, alpha, state, slots, positions, vdim)
    out.copy_(_gla_out(o, g, norm, eps, proj.dtype))


def gla_prefill(proj, a2, a2_bias, norm, state, tiles, seqs, vdim, tau, eps,
                out):
    q, k, v, g, alpha = _gla_parts(proj, a2, a2_bias, state, vdim, tau)
    o = _scan_states(q, k, v, alpha, state, tiles, seqs, vdim)
    out.copy_(_gla_out(o, g, norm, eps, proj.dtype))


def _hgrn2_parts(proj, bias, lower, state, vdim):
    T = proj.shape[0]
    _, H, D, _ = state.shape
    q, z, v = torch.split(proj.float(), [H * D, H * D, H * vdim], dim=1)
    z = z + bias
    k = (1 - lower) * torch.sigmoid(-z)
    alpha = lower + (1 - lower) * torch.sigmoid(z)
    return (F.silu(q).view(T, H, D), k.view(T, H, D), v.view(T, H, vdim),
            alpha.view(T, H, D))


def hgrn2_decode(proj, bias, lower, norm, state, slots, positions, vdim, eps,
                 out):
    parts = _hgrn2_parts(proj, bias, lower, state, vdim)
    o = _step_states(*parts, state, slots, positions, vdim)
    out.copy_(_norm(o, norm, eps).flatten(1))


def hgrn2_prefill(proj, bias, lower, norm, state, tiles, seqs, vdim, eps,
                  out):
    parts = _hgrn2_parts(proj, bias, lower, state, vdim)
    o = _scan_states(*parts, state, tiles, seqs, vdim)
    out.copy_(_norm(o, norm, eps).flatten(1))


# ---------------------------------------------------------------- experts
def moe_route(h, router, top):
    s = torch.sigmoid(h.float() @ router.float().T)
    # stable sort: equal scores go to the lower expert, as on the GPU
    w, ids = torch.sort(s, dim=-1, descending=True, stable=True)
    return ids[:, :top].to(torch.int32).contiguous(), w[:, :top].contiguous()


def moe_experts(h, router, w_up, w_down, top, limit):
    ids, w = moe_route(h, router, top)
    T, W = h.shape
    y = torch.zeros(T, top, W)
    hf = h.float()
    for e in range(router.shape[0]):
        t, c = torch.nonzero(ids == e, as_tuple=True)
        if not len(t):
            continue
        x = hf[t] * w[t, c][:, None]
        up = w_up[e].float()                     # [ffp/16, 2, 16, W]
        gate = torch.clamp(x @ up[:, 0].reshape(-1, W).T, max=limit)
        u = torch.clamp(x @ up[:, 1].reshape(-1, W).T, -limit, limit)
        y[t, c] = (gate * torch.sigmoid(1.702 * gate) * (u + 1)) \
            @ w_down[e].float().T
    return y.to(h.dtype)
