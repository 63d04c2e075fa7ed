"""CPU forms of the residual-block ops (same signatures and layouts as
torch.ops.rlli_blk), in f32 PyTorch."""

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
    branches = taps if taps.dim() == 3 else taps[None]
    hc = h.new_empty((len(branches), *h.shape))
    back = taps.shape[-2] - 1
    for n in range(n_decode):
        p = int(positions[n])
        o = h[n].float() * (1 + branches[:, back])
        for k in range(1, min(back, p) + 1):
            o = o + branches[:, back - k] \
                * tail[int(slots[n]), (p - k) % tail.shape[1]].float()
        hc[:, n] = o.to(dtype)
        if back:
            tail[int(slots[n]), p % tail.shape[1]] = h[n]
    return h, hc if taps.dim() == 3 else hc[0]


def block_embed(ids, table, pos_table, positions, x, gain, groups, eps, taps,
                tail, slots, n_decode, scale):
    e = table[ids.long()].float() * scale
    if pos_table is not None:
        last = pos_table.shape[0] - 1
        e = e + pos_table[positions.long().clamp(max=last)].float()
    x.copy_(e)
    return _norm_conv(x, gain, groups, eps, table.dtype, positions, taps,
                      tail, slots, n_decode)


def block_step(x, y, gain, groups, eps, positions, taps, tail, slots,
               n_decode, rows, keep, y2, gain1, gain2, part_ids=None,
               part_w=None, part_h=None, part_limit=0, y_bias=None):
    if part_ids is not None:
        own = (part_ids < part_limit)[..., None]
        new = x + torch.where(own, y.float(), part_w[..., None]
                              * part_h.float()[:, None]).sum(1)
    elif y2 is None:
        new = x + y.float()
        if y_bias is not None:
            new = new + y_bias
    else:
        new = x + 0.5 * (_group_norm(y.float(), gain1, 1, eps)
                         + _group_norm(y2.float(), gain2, 1, eps))
    if keep:
        x.copy_(new)
    if rows is not None:
        new = new[rows]
    return _norm_conv(new, gain, groups, eps, y.dtype, positions, taps, tail,
                      slots, n_decode)


def conv_prompt(h, taps, tail, spans, portions, out, silu):
    back = taps.shape[-2] - 1
    ring = tail.shape[1] if back else 1
    for row0, pos0, n, _, slot in portions.t().tolist():
        past = torch.zeros(back, h.shape[1])
        for k in range(1, min(back, pos0) + 1):
            past[back - k] = tail[slot, (pos0 - k) % ring].float()
        own = h[row0:row0 + n]
        seq = torch.cat([past, own.float()])
        for b, w in enumerate(taps if taps.dim() == 3 else taps[None]):
            o = torch.zeros_like(own, dtype=torch.float32)
            for j in range(back + 1):
                o = o + w[j] * seq[j:j + n]
            o = torch.nn.functional.silu(o) if silu else own.float() + o
            (out[b] if taps.dim() == 3 else out)[row0:row0 + n] = \
                o.to(h.dtype)
        if back:
            for r in range(max(0, n - ring), n):
                tail[slot, (pos0 + r) % ring] = own[r]


def gate_act(gate_up, out, act, limit):
    g, u = gate_up.float().chunk(2, dim=1)
    if act == "clamp_glu":
        g, u = g.clamp(max=limit), u.clamp(-limit, limit)
        out.copy_(g * torch.sigmoid(1.702 * g) * (u + 1))
        return
    f = {"relu": torch.relu, "silu": torch.nn.functional.silu}[act]
    out.copy_(f(g) * u)


def soft_cap(x, cap):
    return cap * torch.tanh(x.float() / cap)
