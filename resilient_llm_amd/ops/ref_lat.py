"""CPU forms of the latent-attention ops (same signatures and layouts as
torch.ops.rlli_lat), in f32 PyTorch.  Attention has the absorbed form only;
the expanded one is a GPU choice."""

from __future__ import annotations

import torch


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
