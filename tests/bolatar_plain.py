"""Plain, slow Bolatar: the equations one by one, one function per
mechanism, one sequence at a time.

This is the yardstick of the Bolatar tests.  It shares no code with the
package: weights come in as a dict of tensors under their checkpoint
names, the configuration as the parsed config.json, and everything is
computed in ``dtype`` (float64 unless asked otherwise).
"""

from __future__ import annotations

import math

import torch

UNIT_EPS = 1e-6        # inside the root of the delta rule's unit vectors
MLSTM_EPS = 1e-6       # added to the mLSTM's denominator


def rms(x, eps):
    """x over its root mean square (last axis), eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


# ------------------------------------------------------------ delta rule
def short_conv(h, w):
    """Causal depthwise convolution over time; w [channels, taps], the last
    tap meets the present row; nothing comes before the first row."""
    T, taps = h.shape[0], w.shape[1]
    out = torch.zeros_like(h)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def delta_decay(a, A_log, dt_bias):
    return torch.exp(-torch.exp(A_log) * softplus(a + dt_bias))


def delta_recur(q, k, v, beta, g):
    """q, k [T, H, dim], v [T, H, vdim], beta, g [T, H].  The state first
    decays, then learns what it got wrong about v, then is read."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        S = g[t][:, None, None] * S
        guess = (S * k[t][:, :, None]).sum(1)
        u = beta[t][:, None] * (v[t] - guess)
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def delta_mixer(h, w, mc, eps):
    T, H, G = h.shape[0], mc["heads"], mc["kv_heads"]
    dim, vdim = mc["dim"], mc["vdim"]

    def branch(name, heads):
        x = silu(short_conv(h @ w[name].T, w[name + ".conv"]))
        return x.view(T, heads, -1)
    q = unit(branch("q", G)) * dim ** -0.5
    k = unit(branch("k", G))
    v = branch("v", H)
    of_head = [n // (H // G) for n in range(H)]
    beta = torch.sigmoid(h @ w["b"].T)
    g = delta_decay(h @ w["a"].T, w["A_log"], w["dt_bias"])
    o, _ = delta_recur(q[:, of_head], k[:, of_head], v, beta, g)
    o = rms(o, eps) * w["norm"] * silu(h @ w["g"].T).view(T, H, vdim)
    return o.reshape(T, H * vdim) @ w["o"].T


# ------------------------------------------------------- parallel: left
def query_temperature(p, coef, every):
    return 1 + coef * math.log((p + 1) // every + 1)


def biased_attention(q, k, v, scale, r1, r2):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] from position 0, every
    earlier key and the own one seen; a score loses r1 ln(1 + r2 distance)."""
    T, H = q.shape[:2]
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        back = torch.arange(i, -1, -1, dtype=q.dtype)
        for h in range(H):
            sc = (k[:i + 1, h // per] @ q[i, h]) * scale
            sc = sc - r1[h] * torch.log(1 + r2[h] * back)
            e = torch.exp(sc - sc.max())
            out[i, h] = (e[:, None] * v[:i + 1, h // per]).sum(0) / e.sum()
    return out


def left_mixer(h, w, mc, eps):
    T, H, G = h.shape[0], mc["heads"], mc["kv_heads"]
    q = (h @ w["q"].T).view(T, H, mc["dim"])
    k = (h @ w["k"].T).view(T, G, mc["dim"])
    v = rms((h @ w["v"].T).view(T, G, mc["vdim"]), eps)
    t = mc["q_temp"]
    temp = [query_temperature(p, t["coef"], t["every"]) for p in range(T)]
    q = q * torch.tensor(temp, dtype=q.dtype)[:, None, None]
    o = biased_attention(q, k, v, mc["scale"], w["r1"], w["r2"])
    return o.reshape(T, H * mc["vdim"]) @ w["o"].T


# ------------------------------------------------------ parallel: right
def shifted(h):
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def shift_mix(h, mu):
    return h + (shifted(h) - h) * mu


def rwkv_decay(x, w1, w2, w0):
    return torch.exp(-torch.exp(torch.tanh(x @ w1.T) @ w2.T + w0))


def rwkv_recur(r, k, v, w, u):
    """r, k, w [T, H, dim], v [T, H, vdim], u [H, dim].  The read-out sees
    the past and, through the bonus, the present; then the state moves on."""
    T, H, dim = r.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=r.dtype)
    out = []
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out.append(((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1))
        S = w[t][:, :, None] * S + kv
    return torch.stack(out), S


def right_mixer(h, w, mc, eps):
    T, H, dim = h.shape[0], mc["heads"], mc["dim"]
    mixed = {n: shift_mix(h, w["mu." + n]) for n in "rkvgw"}
    r, k, v = ((mixed[n] @ w[n].T).view(T, H, dim) for n in "rkv")
    gate = silu(mixed["g"] @ w["g"].T)
    decay = rwkv_decay(mixed["w"], w["w1"], w["w2"], w["w0"])
    o, _ = rwkv_recur(r, k, v, decay.view(T, H, dim), w["u"])
    o = rms(o, eps).reshape(T, H * dim) * w["norm"] * gate
    return o @ w["o"].T


def parallel_mixer(h, w, mc, eps):
    def side(name):
        return {k[len(name) + 1:]: v for k, v in w.items()
                if k.startswith(name + ".")}
    lw, rw = side("left"), side("right")
    yl = rms(left_mixer(h, lw, mc["left"], eps), eps) * lw["out"]
    yr = rms(right_mixer(h, rw, mc["right"], eps), eps) * rw["out"]
    return 0.5 * (yl + yr)


# ----------------------------------------------------------------- mLSTM
def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


def mlstm_recur(q, k, v, i, f):
    """q, k [T, H, dim], v [T, H, vdim], log gates i, f [T, H]; q already
    scaled.  Matrix and normalizer are kept relative to e^m."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype)
    n = torch.zeros(H, dim, dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = []
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        S = keep[:, None, None] * S + take[:, None, None] * (
            k[t][:, :, None] * v[t][:, None, :])
        n = keep[:, None] * n + take[:, None] * k[t]
        m = new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m))
        out.append((S * q[t][:, :, None]).sum(1) / (den + MLSTM_EPS)[:, None])
    return torch.stack(out), S, n, m


def mlstm_mixer(h, w, mc, eps):
    T, H, dim, vdim = h.shape[0], mc["heads"], mc["dim"], mc["vdim"]
    q = (h @ w["q"].T).view(T, H, dim) * dim ** -0.5
    k = (h @ w["k"].T).view(T, H, dim)
    v = (h @ w["v"].T).view(T, H, vdim)
    cap = mc["gate_cap"]
    i = soft_cap(h @ w["i"].T + w["i.b"], cap)
    f = -softplus(-soft_cap(h @ w["f"].T + w["f.b"], cap))
    o = mlstm_recur(q, k, v, i, f)[0]
    o = rms(o, eps).reshape(T, H * vdim) * w["norm"]
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ----------------------------------------------------- feed-forward, model
def clamped_ff(h, w, limit):
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w["down"].T


MIXERS = {"delta": delta_mixer, "parallel": parallel_mixer,
          "mlstm": mlstm_mixer}


def run(config, weights, tokens, dtype=torch.float64):
    """One sequence through the whole model.  Returns logits [T, vocab]
    and the residual after every layer."""
    eps = config["norm"]["eps"]
    W = {k: v.to(dtype) for k, v in weights.items()}

    def under(prefix):
        return {k[len(prefix):]: v for k, v in W.items()
                if k.startswith(prefix)}

    x = W["embed"][torch.as_tensor(tokens)] * config["embedding"]["scale"] \
        + W["pos"][:len(tokens)]
    after = []
    for i, layer in enumerate(config["layers"]):
        h = rms(x, eps) * W[f"l{i}.norm1"]
        x = x + MIXERS[layer["type"]](h, under(f"l{i}.mix."), layer["mixer"],
                                      eps)
        f = layer.get("mlp")
        if f is not None:
            h = rms(x, eps) * W[f"l{i}.norm2"]
            x = x + clamped_ff(h, under(f"l{i}.mlp."), f["limit"])
        after.append(x)
    h = rms(x, eps) * W["final.norm"]
    return soft_cap(h @ W["head"].T, config["logit_softcap"]), after


# ------------------------------------------------------------ test models
def make_config(layers, width=64, vocab=97, eps=1e-5, scale=0.8,
                softcap=9.0, max_positions=512):
    return {"architecture": "Bolatar", "embedding": {"scale": scale},
            "layers": layers, "logit_softcap": softcap,
            "max_positions": max_positions, "norm": {"eps": eps},
            "vocab": vocab, "width": width}


def tensor_shapes(config, rank=8):
    """Checkpoint names and shapes that a configuration implies; ``rank``
    is the width of the decay's low-rank projection."""
    d = config["width"]
    out = {"embed": (config["vocab"], d), "head": (config["vocab"], d),
           "pos": (config["max_positions"], d), "final.norm": ()}
    for n, layer in enumerate(config["layers"]):
        m, f, p = layer["mixer"], layer.get("mlp"), f"l{n}."
        out[p + "norm1"] = ()
        if layer["type"] == "delta":
            H, qk, vo = m["heads"], m["kv_heads"] * m["dim"], \
                m["heads"] * m["vdim"]
            for x, rows in (("q", qk), ("k", qk), ("v", vo)):
                out[f"{p}mix.{x}"] = (rows, d)
                out[f"{p}mix.{x}.conv"] = (rows, m["conv"])
            out.update({p + "mix.b": (H, d), p + "mix.a": (H, d),
                        p + "mix.A_log": (H,), p + "mix.dt_bias": (H,),
                        p + "mix.norm": (m["vdim"],), p + "mix.g": (vo, d),
                        p + "mix.o": (d, vo)})
        elif layer["type"] == "mlstm":
            H, qk, vo = m["heads"], m["heads"] * m["dim"], \
                m["heads"] * m["vdim"]
            out.update({p + "mix.q": (qk, d), p + "mix.k": (qk, d),
                        p + "mix.v": (vo, d), p + "mix.g": (vo, d),
                        p + "mix.o": (d, vo), p + "mix.norm": (vo,),
                        p + "mix.i": (H, d), p + "mix.i.b": (H,),
                        p + "mix.f": (H, d), p + "mix.f.b": (H,)})
        else:
            a, b = m["left"], m["right"]
            vo, hd = a["heads"] * a["vdim"], b["heads"] * b["dim"]
            q = p + "mix.left."
            out.update({q + "q": (a["heads"] * a["dim"], d),
                        q + "k": (a["kv_heads"] * a["dim"], d),
                        q + "v": (a["kv_heads"] * a["vdim"], d),
                        q + "r1": (a["heads"],), q + "r2": (a["heads"],),
                        q + "o": (d, vo), q + "out": (d,)})
            q = p + "mix.right."
            out.update({q + "mu." + x: (d,) for x in "rkvgw"})
            out.update({q + x: (hd, d) for x in "rkvg"})
            out.update({q + "w1": (rank, d), q + "w2": (hd, rank),
                        q + "w0": (hd,), q + "u": (b["heads"], b["dim"]),
                        q + "norm": (hd,), q + "o": (d, hd),
                        q + "out": (d,)})
        if f is not None:
            out[p + "norm2"] = ()
            out.update({p + "mlp.gate": (f["ff"], d),
                        p + "mlp.up": (f["ff"], d),
                        p + "mlp.down": (d, f["ff"])})
    return out


def random_weights(config, seed=0, rank=8):
    """bfloat16 weights that keep every mechanism audible: unit-gain
    linears, norms a little off one, audible taps, decays from slow to
    fast, input gates of either sign, distance biases that matter.  Keys of
    the recurrences lean towards their queries: a sequence's first read-outs
    are normed, so a product near zero would decide their sign by rounding.
    """
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config, rank).items():
        t = torch.randn(shape, generator=g)
        u = torch.rand(shape, generator=g)
        leaf = name.split(".", 1)[-1]
        if leaf.endswith(("norm", "norm1", "norm2", ".out")):
            t = 1 + 0.2 * t
        elif leaf.endswith(".conv"):
            t = 0.7 * t
        elif leaf == "mix.A_log":
            t = -2.5 + 3 * u
        elif leaf == "mix.dt_bias":
            t = -1 + t
        elif leaf.endswith(("r1", "r2")):
            t = 0.1 + 0.9 * u
        elif ".mu." in leaf:
            t = u
        elif leaf.endswith("w0"):
            t = -5 + 5 * u
        elif leaf.endswith(".u"):
            t = 0.8 + 0.3 * t
        elif leaf == "mix.i.b":
            t = 1.5 * t
        elif leaf == "mix.f.b":
            t = 2.5 + 2 * t
        elif leaf in ("mix.i", "mix.f"):
            t = t * 2 / math.sqrt(shape[-1])
        elif leaf in ("mix.left.q", "mix.left.k"):
            t = t * 1.6 / math.sqrt(shape[-1])
        elif name == "pos":
            t = 0.5 * t
        elif name != "embed":
            t = t * 1.2 / math.sqrt(shape[-1])
        out[name] = t
    for name in list(out):
        q = name[:-1] + ("r" if name.endswith("right.k") else "q")
        if name.endswith((".mix.k", ".right.k")):
            out[name] = 0.6 * out[q] + 0.8 * out[name]
    return {name: t.to(torch.bfloat16) for name, t in out.items()}
