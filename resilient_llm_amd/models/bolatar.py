"""Bolatar: three kinds of token mixer in one residual stack, MI355X-first.

Per layer one of: a gated delta rule behind short convolutions; two mixers
side by side that read the same input, causal attention with a distance
bias beside an RWKV-style recurrence, each normed over the width and half
their sum taken; an mLSTM.  Per layer a clamped gated feed-forward, or none.
Norms have a single gain, positions are learned and added to the scaled
embedding, logits are soft-capped.  Sizes, constants and the order of
layers come from config.json.

Projections that share an input are one product.  The recurrence of a
parallel layer reads five mixes of a row with the one before it; mixing is a
two-tap convolution with five branches, for decoded tokens part of the pass
that writes the residual and norms it.  That pass also norms and merges a
parallel layer's two outputs.  Residual, norms, gates, decays and states
are 32-bit; product inputs, caches and convolution tails have the model
dtype, which may also be float32.
"""

from __future__ import annotations

import dataclasses

import torch
import torch.nn.functional as F

from .. import ops
from ..engine.kv_cache import (
    KVLayer, ScalarLayer, StateLayer, TailLayer, layer_parts,
)
from .llama import _linear
from .mixed import LayerSpec, MixedConfig, MixedModel


@dataclasses.dataclass(frozen=True)
class DeltaSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int

    @property
    def channels(self) -> int:
        """What the convolution sees: q, k and v."""
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


@dataclasses.dataclass(frozen=True)
class BiasedAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temp_coef: float
    temp_every: int


@dataclasses.dataclass(frozen=True)
class RwkvSpec:
    heads: int
    dim: int


@dataclasses.dataclass(frozen=True)
class ParallelSpec:
    left: BiasedAttentionSpec
    right: RwkvSpec


@dataclasses.dataclass(frozen=True)
class MlstmSpec:
    heads: int
    dim: int
    vdim: int
    cap: float


@dataclasses.dataclass(frozen=True)
class ClampedSpec:
    ff: int
    limit: float


def _mixer(kind: str, m: dict):
    if kind == "delta":
        return DeltaSpec(heads=m["heads"], kv_heads=m["kv_heads"],
                         dim=m["dim"], vdim=m["vdim"], taps=m["conv"])
    if kind == "parallel":
        a, b = m["left"], m["right"]
        return ParallelSpec(
            BiasedAttentionSpec(
                heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"],
                vdim=a["vdim"], scale=float(a["scale"]),
                temp_coef=float(a["q_temp"]["coef"]),
                temp_every=int(a["q_temp"]["every"])),
            RwkvSpec(heads=b["heads"], dim=b["dim"]))
    if kind == "mlstm":
        return MlstmSpec(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                         cap=float(m["gate_cap"]))
    raise ValueError(f"unknown mixer {kind!r}")


@dataclasses.dataclass
class BolatarConfig(MixedConfig):
    name: str
    hidden_size: int
    vocab_size: int
    rms_eps: float
    embed_scale: float
    logit_softcap: float
    max_position: int                # rows of the learned position table
    layers: tuple                    # LayerSpec
    decay_rank: int = 16             # random init; a checkpoint's own wins
    eos_ids: tuple = ()

    def __post_init__(self) -> None:
        if self.hidden_size > 16000:
            raise ValueError("width must be at most 16000")
        if self.logit_softcap <= 0:
            raise ValueError("the logits' cap must be positive")
        for i, spec in enumerate(self.layers):
            self._check(f"layer {i}", spec.mixer)

    @staticmethod
    def _check(where: str, m) -> None:
        def state(dim, columns):
            if dim > 256 or columns > 1024:
                raise ValueError(f"{where}: recurrent heads are at most "
                                 f"256 x 1024")

        def grouped(s):
            if s.heads % s.kv_heads:
                raise ValueError(f"{where}: heads % kv_heads")
        if isinstance(m, DeltaSpec):
            state(m.dim, m.vdim)
            grouped(m)
            if m.taps < 1:
                raise ValueError(f"{where}: a convolution has at least one "
                                 f"tap")
        elif isinstance(m, MlstmSpec):
            state(m.dim, m.vdim + 1)
            if m.cap <= 0:
                raise ValueError(f"{where}: gate_cap must be positive")
        else:
            state(m.right.dim, m.right.dim)
            grouped(m.left)
            if m.left.vdim > 512 or m.left.dim > 4096:
                raise ValueError(f"{where}: attention heads are at most "
                                 f"4096 wide, values 512")
            if m.left.temp_every < 1:
                raise ValueError(f"{where}: q_temp.every must be positive")

    @classmethod
    def from_dict(cls, d: dict, name: str = "bolatar", **kw):
        layers = []
        for i, e in enumerate(d["layers"]):
            f = e.get("mlp")
            if f is not None and f["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{f['kind']!r}")
            layers.append(LayerSpec(
                _mixer(e["type"], e["mixer"]),
                None if f is None else ClampedSpec(f["ff"],
                                                   float(f["limit"]))))
        return cls(name=name, hidden_size=d["width"], vocab_size=d["vocab"],
                   rms_eps=float(d["norm"]["eps"]),
                   embed_scale=float(d["embedding"]["scale"]),
                   logit_softcap=float(d["logit_softcap"]),
                   max_position=d["max_positions"], layers=tuple(layers),
                   **kw)

    def fit_positions(self, n: int) -> None:
        """The learned table is the limit, whatever the pool holds."""

    def cache_layers(self, tp_world: int = 1) -> list:
        """What each layer keeps per token and per sequence.  The delta
        rule's ring has a row more than its convolution looks back (see
        ops.delta_decode); the previous row of a parallel layer is whole on
        every rank."""
        out, n = [], tp_world
        for spec in self.layers:
            m = spec.mixer
            if isinstance(m, DeltaSpec):
                parts = [StateLayer(m.heads // n, m.dim, m.vdim)]
                if m.taps > 1:
                    parts.append(TailLayer(m.taps, m.channels // n))
            elif isinstance(m, MlstmSpec):
                # the last value column is the normalizer
                parts = [StateLayer(m.heads // n, m.dim, m.vdim + 1),
                         ScalarLayer(m.heads // n)]
            else:
                parts = [KVLayer(m.left.kv_heads // n, m.left.dim,
                                 m.left.vdim),
                         StateLayer(m.right.heads // n, m.right.dim,
                                    m.right.dim),
                         TailLayer(1, self.hidden_size)]
            out.append(tuple(parts))
        return out

    def kv_elems_per_token(self, tp_world: int = 1) -> int:
        return sum(s.n_kv_heads * (s.k_dim + s.v_dim)
                   for spec in self.cache_layers(tp_world)
                   for s in layer_parts(spec) if isinstance(s, KVLayer))


def hybrid_layers(n: int, parallel_every: int, parallel: dict, delta: dict,
                  mlstm: dict, mlp: dict) -> list:
    """config.json 'layers' of the usual shape: one parallel layer, then
    parallel_every - 1 recurrent ones that alternate, repeated."""
    out, k = [], 0
    for i in range(n):
        if i % parallel_every == 0:
            kind, mixer = "parallel", parallel
        else:
            kind, mixer = (("delta", delta), ("mlstm", mlstm))[k % 2]
            k += 1
        out.append({"type": kind, "mixer": dict(mixer), "mlp": dict(mlp)})
    return out


def _preset(name: str, width: int, vocab: int, layers: list,
            max_positions: int, **kw) -> BolatarConfig:
    return BolatarConfig.from_dict(
        {"layers": layers, "width": width, "vocab": vocab,
         "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
         "logit_softcap": 30.0, "max_positions": max_positions}, name=name,
        **kw)


def _parallel(heads, kv_heads, dim, rec_heads, rec_dim) -> dict:
    return {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": dim, "scale": dim ** -0.5,
                     "q_temp": {"coef": 0.1, "every": 4096}},
            "right": {"heads": rec_heads, "dim": rec_dim}}


BOLATAR_PRESETS = {
    # CPU-testable
    "bolatar-tiny": lambda: _preset(
        "bolatar-tiny", 128, 512, hybrid_layers(
            4, 3, _parallel(4, 2, 32, 2, 32),
            {"heads": 4, "kv_heads": 2, "dim": 32, "vdim": 32, "conv": 4},
            {"heads": 2, "dim": 32, "vdim": 48, "gate_cap": 15.0},
            {"kind": "dense", "ff": 192, "limit": 7.0}), 2048),
    # layers of a real model's size
    "bolatar-1b": lambda: _preset(
        "bolatar-1b", 2048, 65536, hybrid_layers(
            12, 3, _parallel(16, 4, 128, 16, 64),
            {"heads": 16, "kv_heads": 8, "dim": 128, "vdim": 128, "conv": 4},
            {"heads": 8, "dim": 128, "vdim": 256, "gate_cap": 15.0},
            {"kind": "dense", "ff": 4096, "limit": 7.0}), 32768,
        decay_rank=64),
}


class BolatarForCausalLM(MixedModel):
    """Inference-only Bolatar.  TP shards heads (attention and recurrent)
    with their convolutions and the feed-forward width column-wise, output
    projections row-wise, with an all-reduce per output; norms, token mixes
    and the residual are replicated."""

    EXTENSIONS = ("rlli_attn", "rlli_blk", "rlli_rec")

    def sharded_sizes(self) -> list:
        sizes = []
        for spec in self.config.layers:
            m = spec.mixer
            if isinstance(m, ParallelSpec):
                sizes += [m.left.heads, m.left.kv_heads, m.right.heads]
            else:
                sizes += [m.heads, getattr(m, "kv_heads", m.heads)]
            if spec.mlp is not None:
                sizes.append(spec.mlp.ff)
        return sizes

    # ------------------------------------------------------------ weights
    def tensor_shapes(self) -> dict:
        c = self.config
        d, rank = c.hidden_size, c.decay_rank
        out = {"embed": (c.vocab_size, d), "pos": (c.max_position, d)}
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            out[p + "norm1"] = ()
            if isinstance(m, DeltaSpec):
                qk, hv = m.kv_heads * m.dim, m.heads * m.vdim
                for x, rows in (("q", qk), ("k", qk), ("v", hv)):
                    out[f"{p}mix.{x}"] = (rows, d)
                    out[f"{p}mix.{x}.conv"] = (rows, m.taps)
                out[p + "mix.g"] = (hv, d)
                for x in "ba":
                    out[f"{p}mix.{x}"] = (m.heads, d)
                out[p + "mix.A_log"] = out[p + "mix.dt_bias"] = (m.heads,)
                out[p + "mix.norm"] = (m.vdim,)
                out[p + "mix.o"] = (d, hv)
            elif isinstance(m, MlstmSpec):
                qk, hv = m.heads * m.dim, m.heads * m.vdim
                for x, rows in (("q", qk), ("k", qk), ("v", hv), ("g", hv),
                                ("i", m.heads), ("f", m.heads)):
                    out[f"{p}mix.{x}"] = (rows, d)
                out[p + "mix.i.b"] = out[p + "mix.f.b"] = (m.heads,)
                out[p + "mix.norm"] = (hv,)
                out[p + "mix.o"] = (d, hv)
            else:
                a, q = m.left, p + "mix.left."
                out[q + "q"] = (a.heads * a.dim, d)
                out[q + "k"] = (a.kv_heads * a.dim, d)
                out[q + "v"] = (a.kv_heads * a.vdim, d)
                out[q + "r1"] = out[q + "r2"] = (a.heads,)
                out[q + "o"] = (d, a.heads * a.vdim)
                out[q + "out"] = (d,)
                b, q = m.right, p + "mix.right."
                n = b.heads * b.dim
                for x in "rkvgw":
                    out[f"{q}mu.{x}"] = (d,)
                for x in "rkvg":
                    out[q + x] = (n, d)
                out[q + "w1"] = (rank, d)
                out[q + "w2"] = (n, rank)
                out[q + "w0"] = (n,)
                out[q + "u"] = (b.heads, b.dim)
                out[q + "norm"] = (n,)
                out[q + "o"] = (d, n)
                out[q + "out"] = (d,)
            if f is not None:
                out[p + "norm2"] = ()
                out[p + "mlp.gate"] = (f.ff, d)
                out[p + "mlp.up"] = (f.ff, d)
                out[p + "mlp.down"] = (d, f.ff)
        out["final.norm"] = ()
        out["head"] = (c.vocab_size, d)
        return out

    def initial(self, leaf: str, shape: tuple):
        n = shape[0] if shape else 1
        if "norm" in leaf or leaf.endswith(".out"):
            return torch.ones(shape)
        if ".mu." in leaf:
            return torch.linspace(0.1, 0.9, n)
        if leaf.endswith(("r1", "r2")):
            return torch.linspace(0.1, 1.0, n)
        if leaf.endswith("w0"):
            return torch.linspace(-6.0, -0.5, n)
        if leaf == "mix.A_log":
            return torch.linspace(-2.0, 1.0, n)
        if leaf == "mix.dt_bias":
            return torch.full(shape, -2.0)
        if leaf == "mix.i.b":
            return torch.zeros(shape)
        if leaf == "mix.f.b":
            return torch.linspace(3.0, 6.0, n)
        return None

    def _checkpoint_shapes(self, shape_of, names) -> dict:
        # the decay rank is the one size that a tensor's shape gives
        shapes = self.tensor_shapes()
        for n, (_, d) in [(n, s) for n, s in shapes.items()
                          if n.endswith(".right.w1") and n in names]:
            rank = shape_of(n)[0]
            shapes[n] = (rank, d)
            w2 = n[:-1] + "2"
            shapes[w2] = (shapes[w2][0], rank)
        return shapes

    def _install(self, get) -> None:
        """Projections that share an input become one matrix (rows padded
        to eight, so that every activation row starts aligned), single
        gains become vectors, mixes with the previous row the taps of a
        convolution."""
        c, P = self.config, self.params

        def mat(name, **kw):
            return self._mat(get(name), **kw)

        def vec(name, **kw):
            return self._vec(get(name), **kw)

        def gain(name):
            return vec(name).reshape(1).expand(c.hidden_size).contiguous()

        def joint(p, names):
            w = torch.cat([mat(p + x, rows=True) for x in names])
            return F.pad(w, (0, 0, 0, -w.shape[0] % 8))
        P["embed"], P["pos"] = mat("embed"), mat("pos")
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            P[p + "norm1"] = gain(p + "norm1")
            q = p + "mix."
            if isinstance(m, DeltaSpec):
                P[p + "proj"] = joint(q, "qkvgba")
                P[p + "taps"] = torch.cat(
                    [vec(f"{q}{x}.conv", rows=True) for x in "qkv"]) \
                    .t().contiguous()
                P[p + "rate"] = torch.exp(vec(q + "A_log", rows=True))
                P[p + "dt_bias"] = vec(q + "dt_bias", rows=True)
                P[p + "head_norm"] = vec(q + "norm")
                P[p + "o"] = mat(q + "o", cols=True)
            elif isinstance(m, MlstmSpec):
                P[p + "proj"] = joint(q, "qkvgif")
                P[p + "i.b"] = vec(q + "i.b", rows=True)
                P[p + "f.b"] = vec(q + "f.b", rows=True)
                P[p + "head_norm"] = vec(q + "norm", rows=True)
                P[p + "o"] = mat(q + "o", cols=True)
            else:
                a, b = q + "left.", q + "right."
                P[p + "qkv"] = torch.cat([mat(a + x, rows=True)
                                          for x in "qkv"])
                P[p + "r1"] = vec(a + "r1", rows=True)
                P[p + "r2"] = vec(a + "r2", rows=True)
                P[p + "o_left"] = mat(a + "o", cols=True)
                P[p + "out_left"] = vec(a + "out")
                mu = torch.stack([vec(f"{b}mu.{x}") for x in "rkvgw"])
                P[p + "shift"] = torch.stack([mu, -mu], 1).contiguous()
                # [4, width, columns]: the right operand of a batched
                # product lies as it is read
                P[p + "rkvg"] = torch.stack(
                    [mat(b + x, rows=True).t() for x in "rkvg"]).contiguous()
                P[p + "w1"] = mat(b + "w1")
                P[p + "w2"] = mat(b + "w2", rows=True)
                P[p + "w0"] = vec(b + "w0", rows=True)
                P[p + "bonus"] = vec(b + "u", rows=True).flatten()
                P[p + "head_norm"] = vec(b + "norm", rows=True)
                P[p + "o_right"] = mat(b + "o", cols=True)
                P[p + "out_right"] = vec(b + "out")
            if f is not None:
                P[p + "norm2"] = gain(p + "norm2")
                P[p + "gate_up"] = torch.cat(
                    [mat(p + "mlp.gate", rows=True),
                     mat(p + "mlp.up", rows=True)])
                P[p + "down"] = mat(p + "mlp.down", cols=True)
        P["final.norm"] = gain("final.norm")
        P["head"] = mat("head")

    # ------------------------------------------------------------ compute
    def _empty(self, *shape):
        return torch.empty(shape, dtype=self.dtype, device=self.device)

    def _delta(self, i, m, h, kv_cache, step):
        P, p, nd = self.params, f"l{i}.", step.n_decode
        n, states, eps = self.tp_world, kv_cache.states, self.config.rms_eps
        proj = _linear(h, P[p + "proj"])
        out = self._empty(h.shape[0], m.heads // n * m.vdim)
        args = (P[p + "taps"], states.tail(i), P[p + "rate"],
                P[p + "dt_bias"], P[p + "head_norm"], states.layer(i))
        sizes = (m.kv_heads // n, m.vdim, eps)
        if nd:
            ops.delta_decode(proj[:nd], *args, step.state_slots,
                             step.positions[:nd], *sizes, out[:nd])
        if step.prompt is not None:
            ops.delta_prefill(proj[nd:], *args, step.prompt, *sizes, out[nd:])
        return _linear(out, P[p + "o"])

    def _mlstm(self, i, m, h, kv_cache, step):
        P, p, nd = self.params, f"l{i}.", step.n_decode
        states = kv_cache.states
        proj = _linear(h, P[p + "proj"])
        out = self._empty(h.shape[0], m.heads // self.tp_world * m.vdim)
        args = (P[p + "i.b"], P[p + "f.b"], P[p + "head_norm"],
                states.layer(i), states.scalar(i))
        sizes = (m.vdim, m.cap, self.config.rms_eps)
        if nd:
            ops.mlstm_decode(proj[:nd], *args, step.state_slots,
                             step.positions[:nd], *sizes, out[:nd])
        if step.prompt is not None:
            ops.mlstm_prefill(proj[nd:], *args, step.prompt, *sizes, out[nd:])
        return _linear(out, P[p + "o"])

    def _left(self, i, m, h, kv_cache, step):
        P, p, nd = self.params, f"l{i}.", step.n_decode
        qkv = _linear(h, P[p + "qkv"])
        score = (m.scale, m.heads // self.tp_world, P[p + "r1"], P[p + "r2"],
                 m.temp_coef, m.temp_every, self.config.rms_eps)
        k, v = kv_cache.layer(i)
        parts = []
        if nd:
            parts.append(ops.biased_decode(
                qkv[:nd], k, v, step.positions[:nd], step.slots[:nd],
                step.tables_dec, *score))
        if step.prompt is not None:
            parts.append(ops.biased_prefill(
                qkv[nd:], k, v, step.positions[nd:], step.slots[nd:],
                step.tables_pre, step.prompt, *score))
        out = parts[0] if len(parts) == 1 else torch.cat(parts)
        return _linear(out, P[p + "o_left"])

    def _right(self, i, m, mixes, kv_cache, step):
        P, p, nd = self.params, f"l{i}.", step.n_decode
        rkvg = torch.bmm(mixes[:4], P[p + "rkvg"])
        low = _linear(mixes[4], P[p + "w1"])
        out = self._empty(mixes.shape[1], rkvg.shape[2])
        args = (P[p + "w2"], P[p + "w0"], P[p + "bonus"], P[p + "head_norm"],
                kv_cache.states.layer(i))
        eps = self.config.rms_eps
        if nd:
            ops.rwkv_decode(rkvg[:, :nd], low[:nd], *args, step.state_slots,
                            step.positions[:nd], eps, out[:nd])
        if step.prompt is not None:
            ops.rwkv_prefill(rkvg[:, nd:], low[nd:], *args, step.prompt, eps,
                             out[nd:])
        return _linear(out, P[p + "o_right"])

    def _feed_forward(self, i, f, h):
        P, p = self.params, f"l{i}."
        act = self._empty(h.shape[0], f.ff // self.tp_world)
        ops.gate_act(_linear(h, P[p + "gate_up"]), act, "clamp_glu", f.limit)
        return _linear(act, P[p + "down"])

    def _forward(self, input_ids, kv_cache, step, sample_idx):
        P, c, nd = self.params, self.config, step.n_decode
        x = torch.empty((input_ids.shape[0], c.hidden_size),
                        dtype=torch.float32, device=self.device)

        def norm_args(i, which):
            """The norm ahead of a sublayer, and what it mixes in."""
            args = (P[f"l{i}.{which}"], 1, c.rms_eps)
            if which == "norm1" and isinstance(c.layers[i].mixer,
                                               ParallelSpec):
                return args, (P[f"l{i}.shift"], kv_cache.states.tail(i),
                              step.state_slots, nd)
            return args, ()

        norm, conv = norm_args(0, "norm1")
        h, mixes = ops.block_embed(
            input_ids, P["embed"], P["pos"], step.positions, x, *norm, *conv,
            scale=c.embed_scale)
        subs = [(i, w) for i, s in enumerate(c.layers)
                for w in (("norm1", "norm2") if s.mlp is not None
                          else ("norm1",))]
        for n, (i, which) in enumerate(subs):
            m, f, p = c.layers[i].mixer, c.layers[i].mlp, f"l{i}."
            both = {}
            if which == "norm2":
                y = self._reduce(self._feed_forward(i, f, h))
            elif isinstance(m, DeltaSpec):
                y = self._reduce(self._delta(i, m, h, kv_cache, step))
            elif isinstance(m, MlstmSpec):
                y = self._reduce(self._mlstm(i, m, h, kv_cache, step))
            else:
                if step.prompt is not None:
                    ops.conv_prompt(h[nd:], P[p + "shift"],
                                    kv_cache.states.tail(i), step.prompt,
                                    mixes[:, nd:])
                y, y2 = self._reduce(
                    self._left(i, m.left, h, kv_cache, step),
                    self._right(i, m.right, mixes, kv_cache, step))
                both = dict(y2=y2, gain1=P[p + "out_left"],
                            gain2=P[p + "out_right"])
            if n + 1 < len(subs):
                norm, conv = norm_args(*subs[n + 1])
                h, mixes = ops.block_step(x, y, *norm, step.positions, *conv,
                                          **both)
            else:
                h, _ = ops.block_step(
                    x, y, P["final.norm"], 1, c.rms_eps, step.positions,
                    rows=sample_idx, keep=False, **both)
        return ops.soft_cap(_linear(h, P["head"]), c.logit_softcap)
