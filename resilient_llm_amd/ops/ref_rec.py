"""CPU forms of the linear recurrences (same signatures and layouts as
torch.ops.rlli_rec), in f32 PyTorch, token by token."""

from __future__ import annotations

import torch
import torch.nn.functional as F

REC_CHUNK = 64


def _norm(x, gain, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * gain


# ----------------------------------------- decays per key channel
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


def _over_sequences(step, state, tiles, seqs, v):
    """Rows of every portion through ``step(carry, t)``; ``carry`` is what
    the slot holds, zeros for a new sequence."""
    o = torch.empty_like(v)
    for first, count, pos0, slot in seqs.t().tolist():
        carry = [s[slot].clone() for s in state]
        if pos0 == 0:
            carry = _zeros(carry)
        row = int(tiles[0, first])
        n = int(tiles[2, first:first + count].sum())
        for t in range(row, row + n):
            o[t] = step(carry, t)
        for s, c in zip(state, carry):
            s[slot] = c
    return o


def _zeros(carry):
    return [torch.zeros_like(c) for c in carry]


def _rows(step, state, slots, positions, v):
    """One row per sequence."""
    o = torch.empty_like(v)
    for b in range(v.shape[0]):
        carry = [s[int(slots[b])].clone() for s in state]
        if int(positions[b]) == 0:
            carry = _zeros(carry)
        o[b] = step(carry, b)
        for s, c in zip(state, carry):
            s[int(slots[b])] = c
    return o


def _rwkv(rkvg, low, w2, w0, bonus, state):
    _, T, _ = rkvg.shape
    _, H, D, _ = state.shape
    r, k, v, g = (x.float().reshape(T, H, D) for x in rkvg)
    z = torch.tanh(low.float()) @ w2.float().T + w0
    w = torch.exp(-torch.exp(z)).view(T, H, D)
    u = bonus.view(H, D)

    def step(carry, t):
        S = carry[0][..., :D]
        kv = k[t][..., None] * v[t][:, None]
        o = torch.einsum("hd,hdv->hv", r[t], S + u[..., None] * kv)
        carry[0] = F.pad(w[t][..., None] * S + kv,
                         (0, state.shape[3] - D))
        return o
    return step, v, g


def _rwkv_out(o, g, norm, eps, out):
    D = o.shape[2]
    o = _norm(o, norm.view(-1, D), eps) * F.silu(g)
    out.copy_(o.flatten(1))


def rwkv_decode(rkvg, low, w2, w0, bonus, norm, state, slots, positions, eps,
                out):
    step, v, g = _rwkv(rkvg, low, w2, w0, bonus, state)
    _rwkv_out(_rows(step, [state], slots, positions, v), g, norm, eps, out)


def rwkv_prefill(rkvg, low, w2, w0, bonus, norm, state, tiles, seqs, eps,
                 out):
    step, v, g = _rwkv(rkvg, low, w2, w0, bonus, state)
    _rwkv_out(_over_sequences(step, [state], tiles, seqs, v), g,
              norm, eps, out)


# ------------------------------------------------------------ delta rule
def _delta(proj, x, a_rate, dt_bias, state, kv_heads, vdim):
    """``x``: q | k | v after convolution and silu."""
    T = proj.shape[0]
    _, H, D, P = state.shape
    G, per = kv_heads, H // kv_heads
    qk, hv = G * D, H * vdim
    q, k, v = torch.split(x.float(), [qk, qk, hv], dim=1)
    g, b, a = torch.split(proj[:, 2 * qk + hv:2 * qk + 2 * hv + 2 * H].float(),
                          [hv, H, H], dim=1)

    def unit(y):
        y = y.reshape(T, G, D)
        y = y * torch.rsqrt(y.pow(2).sum(-1, keepdim=True) + 1e-6)
        return y.repeat_interleave(per, 1)
    q, k = unit(q) * D ** -0.5, unit(k)
    v = v.reshape(T, H, vdim)
    beta = torch.sigmoid(b)
    decay = torch.exp(-a_rate * F.softplus(a + dt_bias))

    def step(carry, t):
        S = decay[t][:, None, None] * carry[0][..., :vdim]
        u = beta[t][:, None] * (v[t] - torch.einsum("hd,hdv->hv", k[t], S))
        S = S + k[t][..., None] * u[:, None]
        carry[0] = F.pad(S, (0, P - vdim))
        return torch.einsum("hd,hdv->hv", q[t], S)
    return step, v, g.reshape(T, H, vdim)


def _delta_out(o, g, norm, eps, out):
    out.copy_((_norm(o, norm, eps) * F.silu(g)).flatten(1))


def delta_decode(proj, taps, tail, a_rate, dt_bias, norm, state, slots,
                 positions, kv_heads, vdim, eps, out):
    back, C = taps.shape[0] - 1, taps.shape[1]
    x = proj[:, :C].float() * taps[back]
    for n in range(proj.shape[0]):
        p, s = int(positions[n]), int(slots[n])
        for k in range(1, min(back, p) + 1):
            x[n] += taps[back - k] * tail[s, (p - k) % tail.shape[1]].float()
        if back:
            tail[s, p % tail.shape[1]] = proj[n, :C]
    x = F.silu(x).to(proj.dtype)
    step, v, g = _delta(proj, x, a_rate, dt_bias, state, kv_heads, vdim)
    _delta_out(_rows(step, [state], slots, positions, v), g, norm, eps, out)


def delta_prefill(proj, x, a_rate, dt_bias, norm, state, tiles, seqs,
                  kv_heads, vdim, eps, out):
    step, v, g = _delta(proj, x, a_rate, dt_bias, state, kv_heads, vdim)
    _delta_out(_over_sequences(step, [state], tiles, seqs, v), g,
               norm, eps, out)


# ----------------------------------------------------------------- mLSTM
def _mlstm(proj, i_bias, f_bias, state, vdim, cap):
    T = proj.shape[0]
    _, H, D, P = state.shape
    q, k, v, g, i, f = torch.split(
        proj[:, :2 * H * (D + vdim) + 2 * H].float(),
        [H * D, H * D, H * vdim, H * vdim, H, H], dim=1)
    q = q.reshape(T, H, D) * D ** -0.5
    k, v = k.reshape(T, H, D), v.reshape(T, H, vdim)
    i = cap * torch.tanh((i + i_bias) / cap)
    f = F.logsigmoid(cap * torch.tanh((f + f_bias) / cap))
    ones = torch.ones(H, 1)

    def step(carry, t):
        S, m = carry[0][..., :vdim + 1], carry[1]
        new = torch.maximum(f[t] + m, i[t])
        vn = torch.cat([v[t], ones], -1)
        S = torch.exp(f[t] + m - new)[:, None, None] * S \
            + torch.exp(i[t] - new)[:, None, None] \
            * k[t][..., None] * vn[:, None]
        carry[0], carry[1] = F.pad(S, (0, P - vdim - 1)), new
        o = torch.einsum("hd,hdv->hv", q[t], S)
        den = torch.maximum(o[:, vdim].abs(), torch.exp(-new)) + 1e-6
        return o[:, :vdim] / den[:, None]
    return step, v, g.reshape(T, H, vdim)


def _mlstm_out(o, g, norm, eps, out):
    out.copy_((_norm(o, norm.view(o.shape[1:]), eps)
               * torch.sigmoid(g)).flatten(1))


def mlstm_decode(proj, i_bias, f_bias, norm, state, m, slots, positions, vdim,
                 cap, eps, out):
    step, v, g = _mlstm(proj, i_bias, f_bias, state, vdim, cap)
    _mlstm_out(_rows(step, [state, m], slots, positions, v), g, norm, eps,
               out)


def mlstm_prefill(proj, i_bias, f_bias, norm, state, m, tiles, seqs, vdim,
                  cap, eps, out):
    step, v, g = _mlstm(proj, i_bias, f_bias, state, vdim, cap)
    _mlstm_out(_over_sequences(step, [state, m], tiles, seqs, v), g,
               norm, eps, out)
