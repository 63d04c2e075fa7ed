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


# ---------------------------------------------- differential attention
def _turn_halves(x, positions, cos_sin):
    """x [T, ..., D] f32; pairs (i, i + rot / 2)."""
    if cos_sin is None:
        return x
    rot = cos_sin.shape[1]
    cs = cos_sin[positions.long()].view(-1, *[1] * (x.dim() - 2), rot)
    c, s = cs.chunk(2, -1)
    u, v = x[..., :rot // 2], x[..., rot // 2:rot]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., rot:]], -1)


def _normed(x, gain, eps):
    x = x.float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * gain


def diff_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q, bias,
                q_norm, k_norm, eps):
    T = qkv.shape[0]
    _, G, bs, D2 = k_cache.shape
    V, D = v_cache.shape[3], D2 // 2
    n_k, n_v = (n_q + G) * D2, (n_q + G) * D2 + G * V
    x = qkv[:, :n_v].float()
    if bias is not None:
        x = x + bias
    q, k, v = (x[:, :n_q * D2].view(T, n_q, 2, D),
               x[:, n_q * D2:n_k].view(T, G, 2, D), x[:, n_k:])
    b, o = slots.long() // bs, slots.long() % bs
    k = _turn_halves(_normed(k, k_norm, eps), positions, cos_sin)
    k_cache[b, :, o] = k.reshape(T, G, D2).to(k_cache.dtype)
    v_cache[b, :, o] = v.reshape(T, G, V).to(v_cache.dtype)
    qkv[:, :n_q * D2] = _turn_halves(_normed(q, q_norm, eps), positions,
                                     cos_sin).flatten(1).to(qkv.dtype)


def _diff_attend(q, gate, qpos, k_cache, v_cache, table, scale, chunk, cap,
                 lam, out_scale, eps):
    """q [n, H, 2, D] at positions qpos over one sequence's cache."""
    _, G, bs, D2 = k_cache.shape
    n_kv = int(qpos[-1]) + 1
    blocks = table[:-(-n_kv // bs)].long()
    k = k_cache[blocks].float().transpose(1, 2).reshape(-1, G, D2)[:n_kv]
    v = v_cache[blocks].float().transpose(1, 2) \
        .reshape(-1, G, v_cache.shape[3])[:n_kv]
    H = q.shape[1]
    i, j = qpos[:, None].long(), torch.arange(n_kv)[None]
    ok = (j <= i) & (j >= i // chunk * chunk)
    seen = ok.any(0)                 # the rest may hold anything
    k, v, ok = k[seen], v[seen], ok[:, seen]
    k = k.view(len(k), G, 2, -1).repeat_interleave(H // G, 1)
    v = v.repeat_interleave(H // G, 1)
    s = torch.einsum("nhad,mhad->ahnm", q.float(), k) * scale
    if cap > 0:
        s = cap * torch.tanh(s / cap)
    p = torch.softmax(s.masked_fill(~ok, float("-inf")), -1)
    a1, a2 = torch.einsum("ahnm,mhd->anhd", p, v)
    o = _normed(a1 - lam * a2, out_scale, eps)
    if gate is not None:
        o = o * torch.sigmoid(gate.float())[..., None]
    return o.reshape(q.shape[0], -1)


def _diff_queries(qkv, k_cache, n_q):
    D2 = k_cache.shape[3]
    return qkv[:, :n_q * D2].view(-1, n_q, 2, D2 // 2)


def diff_prefill(qkv, gate, k_cache, v_cache, positions, cos_sin, slots,
                 block_tables, prompt, n_q, bias, q_norm, k_norm, scale,
                 chunk, cap, lam, out_scale, eps):
    diff_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q, bias,
                q_norm, k_norm, eps)
    q = _diff_queries(qkv, k_cache, n_q)
    out = torch.empty(qkv.shape[0], n_q * v_cache.shape[3], dtype=qkv.dtype)
    for p in prompt.portions:
        r = slice(p.row0, p.row0 + p.n)
        out[r] = _diff_attend(
            q[r], None if gate is None else gate[r], positions[r], k_cache,
            v_cache, block_tables[p.seq], scale, chunk, cap, lam, out_scale,
            eps).to(qkv.dtype)
    return out


def diff_decode(qkv, k_cache, v_cache, positions, cos_sin, slots,
                block_tables, gate, scale, n_q, bias, q_norm, k_norm, chunk,
                cap, lam, out_scale, eps):
    diff_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q, bias,
                q_norm, k_norm, eps)
    q = _diff_queries(qkv, k_cache, n_q)
    return torch.cat([
        _diff_attend(q[b:b + 1], None if gate is None else gate[b:b + 1],
                     positions[b:b + 1], k_cache, v_cache, block_tables[b],
                     scale, chunk, cap, lam, out_scale, eps)
        for b in range(qkv.shape[0])]).to(qkv.dtype)


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
