"""CPU forms of the mixed-layer ops (same signatures and layouts as
torch.ops.rlli_mix), in f32 PyTorch: the no-GPU path of the engine tests
and what the HIP kernels' op tests are compared with."""

from __future__ import annotations

import torch

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


# ---------------------------------------------------------------- experts
def moe_route(h, router, top):
    s = torch.sigmoid(h.float() @ router.float().T)
    # stable sort: equal scores go to the lower expert, as on the GPU
    w, ids = torch.sort(s, dim=-1, descending=True, stable=True)
    return ids[:, :top].to(torch.int32).contiguous(), w[:, :top].contiguous()


def moe_route_softmax(h, router, correction, top, groups, keep):
    s = torch.softmax(h.float() @ router.float().T, -1)
    choice = s if correction is None else s + correction
    g = choice.view(-1, groups, choice.shape[1] // groups)
    order = torch.sort(g.amax(-1), dim=-1, descending=True,
                       stable=True).indices[:, :keep]
    stays = torch.zeros(g.shape[:2], dtype=torch.bool).scatter_(1, order, True)
    choice = g.masked_fill(~stays[..., None], float("-inf")).flatten(1)
    ids = torch.sort(choice, dim=-1, descending=True,
                     stable=True).indices[:, :top]
    w = s.gather(1, ids)
    return (ids.to(torch.int32).contiguous(),
            w / (w.sum(-1, keepdim=True) + 1e-20))


def moe_relu2(h, router, correction, w_up, w_down, top, groups, keep):
    ids, w = moe_route_softmax(h, router, correction, top, groups, keep)
    # identity experts' rows stay unwritten, as on the GPU
    y = torch.full((h.shape[0], top, h.shape[1]), float("nan"))
    for e in range(w_up.shape[0]):
        t, c = torch.nonzero(ids == e, as_tuple=True)
        if len(t):
            r = torch.relu(h[t].float() @ w_up[e].float().T)
            y[t, c] = (r * r * w[t, c][:, None]) @ w_down[e].float().T
    return y.to(h.dtype), ids, w


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
