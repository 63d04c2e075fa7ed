"""Plain, slow Fimunex: the equations one by one, one function per
mechanism, one sequence at a time.

This is the yardstick of the Fimunex tests.  It shares no code with the
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


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


# ------------------------------------------------------ short convolution
def with_past(h, w):
    """h plus its causal depthwise convolution over time; w [width, taps],
    the last tap meets the present row, nothing comes before the first."""
    T, taps = h.shape[0], w.shape[1]
    out = h.clone()
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * h[s]
    return out


# --------------------------------------------------------------- rotation
def yarn_frequencies(dims, base, factor, original, fast, slow):
    """One frequency per pair: pairs that turn more than ``fast`` times
    over the original length keep theirs, those below ``slow`` turns are
    slowed down by ``factor``, a ramp lies between."""
    def pair_of(turns):
        return dims * math.log(original / (2 * math.pi * turns)) \
            / (2 * math.log(base))
    lo = max(math.floor(pair_of(fast)), 0)
    hi = min(math.ceil(pair_of(slow)), dims - 1)
    out = []
    for i in range(dims // 2):
        f = base ** (-2 * i / dims)
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1 - ramp))
    return out


def rotate_halves(x, pos, freqs, gain):
    """x [dim] at one position: dimension i turns with i + len(freqs); what
    is left over passes."""
    half = len(freqs)
    y = x.clone()
    for i, f in enumerate(freqs):
        c, s = gain * math.cos(pos * f), gain * math.sin(pos * f)
        y[i] = x[i] * c - x[half + i] * s
        y[half + i] = x[half + i] * c + x[i] * s
    return y


def rotate_all(x, freqs, gain):
    """rotate_halves of [T, ..., dim], position = first index."""
    half = len(freqs)
    f = torch.tensor(freqs, dtype=x.dtype)
    a = torch.arange(x.shape[0], dtype=x.dtype)[:, None] * f
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [half]
    c, s = (gain * a.cos()).view(shape), (gain * a.sin()).view(shape)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


# -------------------------------------------------------------- attention
def visible(T, chunk):
    """[T, T] which keys a query sees: its chunk's, up to its own."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    return (j <= i) & (i // chunk == j // chunk)


def softmax_map(q, k, v, scale, cap, chunk):
    """One map of one head: q [T, dim], k [T, dim], v [T, vdim]."""
    s = soft_cap(q @ k.T * scale, cap)
    s = s.masked_fill(~visible(q.shape[0], chunk), float("-inf"))
    return torch.softmax(s, -1) @ v


def lam(w, diff):
    return torch.exp((w["lq1"] * w["lk1"]).sum()) \
        - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def attention(h, w, m, eps):
    T, H, G, dim, vdim = (h.shape[0], m["heads"], m["kv_heads"], m["dim"],
                          m["vdim"])
    q = (h @ w["q"].T + w["q.b"]).view(T, H, 2, dim)
    k = (h @ w["k"].T + w["k.b"]).view(T, G, 2, dim)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, vdim)
    q, k = rms(q, eps) * w["q.norm"], rms(k, eps) * w["k.norm"]
    sc = m["rot"]["scaling"]
    freqs = yarn_frequencies(m["rot"]["dims"], m["rot"]["base"],
                             sc["factor"], sc["original"], sc["fast"],
                             sc["slow"])
    gain = 0.1 * math.log(sc["factor"]) + 1
    q, k = rotate_all(q, freqs, gain), rotate_all(k, freqs, gain)
    gate = torch.sigmoid(h @ w["g"].T)
    out = []
    for n in range(H):
        g = n // (H // G)
        a1, a2 = (softmax_map(q[:, n, i], k[:, g, i], v[:, g], m["scale"],
                              m["softcap"], m["mask"]["size"])
                  for i in range(2))
        o = rms(a1 - lam(w, m["diff"]) * a2, eps) * (1 - m["diff"])
        out.append(o * gate[:, n:n + 1])
    return torch.cat(out, -1) @ w["o"].T + w["o.b"]


# ---------------------------------------------------------------- experts
def choose(z, correction, top, count, keep):
    """Router of one token, logits z: chosen experts, best first, and their
    weights."""
    s = torch.softmax(z, -1)
    c = s + correction
    n = len(z) // count
    best = [float(c[g * n:(g + 1) * n].max()) for g in range(count)]
    groups = sorted(range(count), key=lambda g: (-best[g], g))[:keep]
    open_ = [e for g in groups for e in range(g * n, (g + 1) * n)]
    ids = sorted(open_, key=lambda e: (-float(c[e]), e))[:top]
    picked = s[ids]
    return ids, picked / (picked.sum() + 1e-20)


def expert(x, up, down):
    r = torch.clamp(x @ up.T, min=0)
    return (r * r) @ down.T


def experts(h, w, f):
    r = f["router"]
    z = h @ w["router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        ids, weights = choose(z[t], w["correction"], r["top"],
                              r["groups"]["count"], r["groups"]["keep"])
        for e, g in zip(ids, weights):
            y = h[t] if e >= r["experts"] else \
                expert(h[t], w[f"e{e}.up"], w[f"e{e}.down"])
            out[t] = out[t] + g * y
    return out


# ------------------------------------------------------------------ model
def layer_order(config):
    """The layers as they run, the loop unrolled."""
    n, loop = len(config["layers"]), config["loop"]
    a, b = loop["start"], loop["stop"]
    return [*range(a), *(list(range(a, b)) * loop["times"]), *range(b, n)]


def run(config, weights, tokens, dtype=torch.float64):
    """One sequence through the whole model.  Returns logits [T, vocab]
    and the residual after every layer that ran."""
    eps = config["norm"]["eps"]
    W = {k: v.to(dtype) for k, v in weights.items()}

    def under(prefix):
        return {k[len(prefix):]: v for k, v in W.items()
                if k.startswith(prefix)}

    x = W["embed"][torch.as_tensor(tokens)]
    after = []
    for i in layer_order(config):
        layer, p = config["layers"][i], f"l{i}."
        h = rms(x, eps) * (1 + W[p + "norm1"])
        h = with_past(h, W[p + "canon1"])
        x = x + attention(h, under(p + "mix."), layer["mixer"], eps)
        if layer["mlp"] is not None:
            h = rms(x, eps) * (1 + W[p + "norm2"])
            h = with_past(h, W[p + "canon2"])
            x = x + experts(h, under(p + "mlp."), layer["mlp"])
        after.append(x)
    h = rms(x, eps) * (1 + W["final.norm"])
    return soft_cap(h @ W["head"].T, config["logit_softcap"]), after


# ------------------------------------------------------------ test models
def make_config(layers, width=64, vocab=97, eps=1e-5, taps=3, softcap=9.0,
                loop=(0, 0, 1)):
    return {"architecture": "Fimunex", "canon": {"taps": taps},
            "layers": layers, "logit_softcap": softcap,
            "loop": dict(zip(("start", "stop", "times"), loop)),
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


def tensor_shapes(config):
    """Checkpoint names and shapes that a configuration implies."""
    d, taps = config["width"], config["canon"]["taps"]
    out = {"embed": (config["vocab"], d), "head": (config["vocab"], d),
           "final.norm": (d,)}
    for n, layer in enumerate(config["layers"]):
        m, f, p = layer["mixer"], layer["mlp"], f"l{n}."
        H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({p + "norm1": (d,), p + "canon1": (d, taps)})
        p += "mix."
        out.update({p + "q": (2 * H * dim, d), p + "q.b": (2 * H * dim,),
                    p + "k": (2 * G * dim, d), p + "k.b": (2 * G * dim,),
                    p + "v": (G * vdim, d), p + "v.b": (G * vdim,),
                    p + "o": (d, H * vdim), p + "o.b": (d,),
                    p + "g": (H, d)})
        out.update({p + x: (dim,) for x in (
            "q.norm", "k.norm", "lq1", "lk1", "lq2", "lk2")})
        if f is None:
            continue
        p, r, ff = f"l{n}.", f["router"], f["expert"]["ff"]
        out.update({p + "norm2": (d,), p + "canon2": (d, taps)})
        p += "mlp."
        routes = r["experts"] + r["identity"]
        out.update({p + "router": (routes, d), p + "correction": (routes,)})
        for e in range(r["experts"]):
            out[f"{p}e{e}.up"], out[f"{p}e{e}.down"] = (ff, d), (d, ff)
    return out


def random_weights(config, seed=0, decisive=False):
    """bfloat16 weights that keep every mechanism audible: unit-gain
    linears, biases and taps that matter, sharp queries and keys, routers
    that spread, corrections of either sign.  ``decisive``: corrections far
    apart, so that no rounding changes a choice."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config).items():
        t = torch.randn(shape, generator=g)
        leaf = name.split(".", 1)[-1]
        if leaf in ("mix.q.norm", "mix.k.norm"):
            t = 1.4 + 0.4 * t
        elif leaf.endswith(("norm", "norm1", "norm2")):
            t = 0.25 * t
        elif leaf.startswith("canon"):
            t = 0.4 * t
        elif leaf.endswith(".b"):
            t = 0.5 * t
        elif leaf.startswith("mix.l"):
            t = 0.3 * t
        elif leaf == "mlp.correction":
            t = -0.3 + 0.4 * t
            if decisive:
                t = -10 + 2.0 * torch.randperm(shape[0], generator=g).float()
        elif leaf == "mlp.router":
            t = t * 1.5 / math.sqrt(shape[-1])
        elif name != "embed":
            t = t * 1.2 / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    return out
