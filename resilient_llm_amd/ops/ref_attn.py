"""CPU forms of paged softmax attention (same signatures and layouts as the
ops of torch.ops.rlli_attn that they stand for), in f32 PyTorch."""

from __future__ import annotations

import torch


def rotate_pairs(x, positions, cos_sin):
    """x [T, H, D]; pairs (2i, 2i+1) of the first cos_sin.shape[1] dims
    (None: no rotation)."""
    if cos_sin is None:
        return x
    rot = cos_sin.shape[1]
    cs = cos_sin[positions.long()]
    c, s = cs[:, None, :rot // 2], cs[:, None, rot // 2:]
    xf = x.float()
    u, v = xf[..., 0:rot:2], xf[..., 1:rot:2]
    turned = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)
    return torch.cat([turned, xf[..., rot:]], -1).to(x.dtype)


def _split_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                  has_kv, v_eps):
    T = qkv.shape[0]
    _, G, bs, D = k_cache.shape
    V = v_cache.shape[3]
    q = rotate_pairs(qkv[:, :n_q * D].reshape(T, n_q, D), positions, cos_sin)
    if has_kv:
        k = rotate_pairs(qkv[:, n_q * D:(n_q + G) * D].reshape(T, G, D),
                         positions, cos_sin)
        v = qkv[:, (n_q + G) * D:].reshape(T, G, V)
        if v_eps is not None:
            v = v.float()
            v = v * torch.rsqrt(v.pow(2).mean(-1, keepdim=True) + v_eps)
        b, o = slots.long() // bs, slots.long() % bs
        k_cache[b, :, o] = k.to(k_cache.dtype)
        v_cache[b, :, o] = v.to(v_cache.dtype)
    return q


def _attend(q, qpos, k_cache, v_cache, table, sink, scale, window,
            keep_first, r1, r2, temp_coef, temp_every):
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
    if temp_every:
        t = (qpos.long() + 1) // temp_every + 1
        s = s * (1 + temp_coef * torch.log(t.float()))[None, :, None]
    i, j = qpos[:, None].long(), torch.arange(n_kv)[None]
    ok = (j <= i) & ((i - j < window) | (j < keep_first))
    if r1 is not None:
        s = s - r1[:, None, None] * torch.log(
            1 + r2[:, None, None] * (i - j).clamp(min=0).float())
    s = s.masked_fill(~ok, float("-inf"))
    if sink is not None:
        s = torch.cat([s, sink[:, None, None].expand(-1, s.shape[1], 1)], -1)
    p = torch.softmax(s, -1)[..., :n_kv]
    return torch.einsum("hnm,mhd->nhd", p, v).reshape(q.shape[0], -1)


def window_prefill(qkv, k_cache, v_cache, positions, cos_sin, slots,
                   block_tables, prompt, sink, scale, n_q, window,
                   keep_first, has_kv, r1, r2, temp_coef, temp_every, v_eps):
    q = _split_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                      has_kv, v_eps)
    out = torch.empty(qkv.shape[0], n_q * v_cache.shape[3], dtype=qkv.dtype)
    for p in prompt.portions:
        r = slice(p.row0, p.row0 + p.n)
        out[r] = _attend(q[r], positions[r], k_cache, v_cache,
                         block_tables[p.seq], sink, scale, window, keep_first,
                         r1, r2, temp_coef, temp_every).to(qkv.dtype)
    return out


def window_decode(qkv, k_cache, v_cache, positions, cos_sin, slots,
                  block_tables, sink, scale, n_q, window, keep_first, has_kv,
                  r1, r2, temp_coef, temp_every, v_eps):
    q = _split_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                      has_kv, v_eps)
    return torch.cat([
        _attend(q[b:b + 1], positions[b:b + 1], k_cache, v_cache,
                block_tables[b], sink, scale, window, keep_first, r1, r2,
                temp_coef, temp_every)
        for b in range(qkv.shape[0])]).to(qkv.dtype)
