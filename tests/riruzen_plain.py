"""Plain, slow Riruzen: the equations one by one, one function per
mechanism, one sequence at a time.

This is the yardstick of the Riruzen tests.  It shares no code with the
package: weights come in as a dict of tensors under their checkpoint
names, the configuration as the parsed config.json, and everything is
computed in ``dtype`` (float64 unless asked otherwise).
"""

from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square (last axis), eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    """Consecutive equal parts of the last axis, each over its own root
    mean square; one weight vector for the whole."""
    n = x.shape[-1] // groups
    parts = [rms(x[..., g * n:(g + 1) * n], eps) for g in range(groups)]
    return torch.cat(parts, -1) * w


def short_conv(h, w):
    """Causal depthwise convolution over time; w [width, taps], the last
    tap meets the present row; nothing comes before the first row."""
    T, taps = h.shape[0], w.shape[1]
    out = torch.zeros_like(h)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


def latent(h, w_dkv, w_norm, eps):
    return rms(h @ w_dkv.T, eps) * w_norm


def latent_queries(h, w_dq, w_norm, w_uq, heads, eps):
    c = rms(h @ w_dq.T, eps) * w_norm
    return (c @ w_uq.T).view(h.shape[0], heads, -1)


def attend(q, k, v, scale):
    """q, k [T, heads, dim], v [T, heads, vdim] from position 0; every
    earlier key and the own one are seen."""
    T, H = q.shape[:2]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        for h in range(H):
            sc = (k[:i + 1, h] @ q[i, h]) * scale
            e = torch.exp(sc - sc.max())
            out[i, h] = (e[:, None] * v[:i + 1, h]).sum(0) / e.sum()
    return out


def latent_attention_mixer(h, w, mc, eps):
    T, H = h.shape[0], mc["heads"]
    q = latent_queries(h, w["dq"], w["dq.norm"], w["uq"], H, eps)
    c = latent(h, w["dkv"], w["dkv.norm"], eps)
    k = (c @ w["uk"].T).view(T, H, mc["dim"])
    v = (c @ w["uv"].T).view(T, H, mc["vdim"])
    o = attend(q, k, v, mc["scale"]).reshape(T, H * mc["vdim"])
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def forget(z, lower):
    return lower + (1 - lower) * torch.sigmoid(z)


def recur(q, v, f):
    """S <- diag(f_t) S + (1 - f_t) v_t^T from zero; o_t = S^T q_t."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        S = f[t][:, :, None] * S + (1 - f[t])[:, :, None] * v[t][:, None, :]
        out.append((q[t][:, :, None] * S).sum(1))
    return torch.stack(out), S


def hgrn2_mixer(h, w, mc, eps):
    T, H, dim, vdim = h.shape[0], mc["heads"], mc["dim"], mc["vdim"]
    q = h @ w["q"].T
    q = (q * torch.sigmoid(q)).view(T, H, dim)
    f = forget(h @ w["f"].T + w["f.b"], w["lower"]).view(T, H, dim)
    v = (h @ w["v"].T).view(T, H, vdim)
    o, _ = recur(q, v, f)
    return (rms(o, eps) * w["norm"]).reshape(T, H * vdim) @ w["o"].T


def relu_gated_ff(h, w):
    return (torch.relu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def run(config, weights, tokens, dtype=torch.float64):
    """One sequence through the whole model.  Returns logits [T, vocab]
    and the residual after every layer."""
    eps, groups = config["norm"]["eps"], config["norm"]["groups"]
    W = {k: v.to(dtype) for k, v in weights.items()}

    def under(prefix):
        return {k[len(prefix):]: v for k, v in W.items()
                if k.startswith(prefix)}

    T = len(tokens)
    x = W["embed"][torch.as_tensor(tokens)] + W["pos"][:T]
    after = []
    for i, layer in enumerate(config["layers"]):
        h = group_norm(x, W[f"l{i}.norm1"], groups, eps)
        hm = h + short_conv(h, W[f"l{i}.canon1"])
        w = under(f"l{i}.mix.")
        mix = {"latent_attention": latent_attention_mixer,
               "hgrn2": hgrn2_mixer}[layer["type"]]
        y = mix(hm, w, layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + relu_gated_ff(h, under(f"l{i}.mlp."))
        x = x + y
        after.append(x)
    h = group_norm(x, W["final.norm"], groups, eps)
    return (h @ W["embed"].T) * config["logit_scale"], after


def make_config(layers, width=64, vocab=97, groups=2, taps=4, eps=1e-5,
                logit_scale=0.7, max_positions=512):
    return {"architecture": "Riruzen", "canon": {"taps": taps},
            "layers": layers, "logit_scale": logit_scale,
            "max_positions": max_positions,
            "norm": {"eps": eps, "groups": groups}, "vocab": vocab,
            "width": width}


def tensor_shapes(config):
    """Checkpoint names and shapes that a configuration implies."""
    d = config["width"]
    out = {"embed": (config["vocab"], d),
           "pos": (config["max_positions"], d), "final.norm": (d,)}
    for i, layer in enumerate(config["layers"]):
        m, f, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        H, dim, vdim = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (d,)
        out[p + "canon1"] = (d, config["canon"]["taps"])
        if layer["type"] == "latent_attention":
            R, Q = m["kv_rank"], m["q_rank"]
            out.update({
                p + "mix.dq": (Q, d), p + "mix.dq.norm": (Q,),
                p + "mix.uq": (H * dim, Q), p + "mix.dkv": (R, d),
                p + "mix.dkv.norm": (R,), p + "mix.uk": (H * dim, R),
                p + "mix.uv": (H * vdim, R), p + "mix.g": (H * vdim, d)})
        else:
            out.update({
                p + "mix.q": (H * dim, d), p + "mix.f": (H * dim, d),
                p + "mix.f.b": (H * dim,), p + "mix.lower": (H * dim,),
                p + "mix.v": (H * vdim, d), p + "mix.norm": (vdim,)})
        out[p + "mix.o"] = (d, H * vdim)
        if f is not None:
            out.update({p + "mlp.gate": (f["ff"], d),
                        p + "mlp.up": (f["ff"], d),
                        p + "mlp.down": (d, f["ff"])})
    return out


def random_weights(config, seed=0):
    """bfloat16 weights that keep every mechanism audible: unit-gain
    linears, norms a little off one, audible taps, lower bounds over the
    whole range, forget gates from slow to fast."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config).items():
        t = torch.randn(shape, generator=g)
        if name.endswith("norm") or name.endswith("norm1"):
            t = 1 + 0.2 * t
        elif name.endswith("canon1"):
            t = 0.4 * t
        elif name.endswith("lower"):
            t = torch.rand(shape, generator=g) ** 0.5 * 0.99
        elif name.endswith("f.b"):
            t = 1.0 + 1.5 * t
        elif name == "pos":
            t = 0.5 * t
        elif name.endswith(("mix.uq", "mix.uk")):
            t = t * 1.5 / math.sqrt(shape[-1])
        elif name != "embed":
            t = t * 1.2 / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    return out
