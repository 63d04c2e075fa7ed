"""CPU forms of the parallel-block and latent-attention ops (same
signatures and layouts as torch.ops.rlli_lat), in f32 PyTorch.  Attention
has the absorbed form only; the expanded one is a GPU choice."""

from __future__ import annotations

import torch


def _group_norm(x, gain, groups, eps):
    p = x.view(x.shape[0], groups, x.shape[1] // groups)
    p = p * torch.rsqrt(p.pow(2).mean(-1, keepdim=True) + eps)
    return p.view_as(x) * gain


def _norm_conv(x, gain, groups, eps, dtype, positions, taps, tail, slots,
               n_decode):
    h = _group_norm(x, gain, groups, eps).to(dtype)
    if taps is None:
        return h, h.new_empty(0)
    hc = torch.empty_like(h)
    back = taps.shape[0] - 1
    for n in range(n_decode):
        p = int(positions[n])
        o = h[n].float() * (1 + taps[back])
        for k in range(1, min(back, p) + 1):
            o = o + taps[back - k] * tail[int(slots[n]), (p - k) % back] \
                .float()
        hc[n] = o.to(dtype)
        if back:
            tail[int(slots[n]), p % back] = h[n]
    return h, hc


def block_embed(ids, table, pos_table, positions, x, gain, groups, eps, taps,
                tail, slots, n_decode):
    e = table[ids.long()].float()
    if pos_table is not None:
        last = pos_table.shape[0] - 1
        e = e + pos_table[positions.long().clamp(max=last)].float()
    x.copy_(e)
    return _norm_conv(x, gain, groups, eps, table.dtype, positions, taps,
                      tail, slots, n_decode)


def block_step(x, y, gain, groups, eps, positions, taps, tail, slots,
               n_decode, rows, keep):
    new = x + y.float()
    if keep:
        x.copy_(new)
    if rows is not None:
        new = new[rows]
    return _norm_conv(new, gain, groups, eps, y.dtype, positions, taps, tail,
                      slots, n_decode)


def conv_prompt(h, taps, tail, spans, portions, out):
    back = taps.shape[0] - 1
    for row0, pos0, n, _, slot in portions.t().tolist():
        past = torch.zeros(back, h.shape[1])
        for k in range(1, min(back, pos0) + 1):
            past[back - k] = tail[slot, (pos0 - k) % back].float()
        own = h[row0:row0 + n]
        seq = torch.cat([past, own.float()])
        o = own.float()
        for j in range(back + 1):
            o = o + taps[j] * seq[j:j + n]
        out[row0:row0 + n] = o.to(h.dtype)
        for r in range(max(0, n - back), n):
            tail[slot, (pos0 + r) % back] = own[r]


def gate_act(gate_up, out, act):
    g, u = gate_up.float().chunk(2, dim=1)
    f = {"relu": torch.relu, "silu": torch.nn.functional.silu}[act]
    out.copy_(f(g) * u)


def latent_prep(proj, q_norm, kv_norm, eps, cache, slots):
    def norm(x, w):
        return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w
    q, r, bs = q_norm.numel(), cache.shape[3], cache.shape[2]
    c = norm(proj[:, q:q + r].float(), kv_norm)
    cache[slots.long() // bs, 0, slots.long() % bs] = c.to(cache.dtype)
    return norm(proj[:, :q].float(), q_norm).to(proj.dtype)


def head_linear(x, w, gate, out):
    H, N, K = w.shape
    y = torch.einsum("thk,hnk->thn", x.reshape(-1, H, K).float(),
                     w.float()).flatten(1)
    if gate is not None:
        y = y * torch.sigmoid(gate.float())
    out.copy_(y)


def _over_latents(q, pos, cache, table, scale):
    """q [n, H, R] at positions pos over one sequence's latents."""
    bs, n_kv = cache.shape[2], int(pos[-1]) + 1
    c = cache[table[:-(-n_kv // bs)].long(), 0].float() \
        .reshape(-1, cache.shape[3])[:n_kv]
    s = torch.einsum("nhr,mr->hnm", q.float(), c) * scale
    seen = torch.arange(n_kv)[None] <= pos[:, None].long()
    p = torch.softmax(s.masked_fill(~seen, float("-inf")), -1)
    return torch.einsum("hnm,mr->nhr", p, c).reshape(q.shape[0], -1)


def latent_attn(q, cache, block_tables, scale, heads, positions, tiles,
                pos0):
    T, R = q.shape[0], cache.shape[3]
    q3 = q.view(T, heads, R)
    out = torch.empty_like(q)
    if tiles is None:
        for b in range(T):
            out[b] = _over_latents(q3[b:b + 1], positions[b:b + 1], cache,
                                   block_tables[b], scale)[0].to(q.dtype)
        return out
    for row0, pos, n, seq in tiles.t().tolist():
        out[row0:row0 + n] = _over_latents(
            q3[row0:row0 + n], torch.arange(pos, pos + n), cache,
            block_tables[seq], scale).to(q.dtype)
    return out
