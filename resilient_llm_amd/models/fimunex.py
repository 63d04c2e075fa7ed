"""Fimunex: differential attention and mixtures of experts in a looped stack,
MI355X-first.

Pre-norm layers; what a sublayer reads is first joined by a short causal
convolution of itself.  Attention is differential (two maps per head over the
same values), with normed queries and keys, YaRN rotation, capped scores, a
chunk of positions that a query sees, and one output gate per head.
Feed-forwards are squared-relu experts behind a softmax router with groups, a
correction of the choice and identity experts.  A range of layers may run
several times, each pass with a cache of its own.  Sizes, constants and the
order of layers come from config.json.

Projections that share an input are one product; its biases are added where
the product is read.  One pass sums a token's expert outputs, writes the
residual, norms it and, for decoded tokens, convolves.  Residual, norms,
angles, scores, router and convolution sums are 32-bit; product inputs,
caches and convolution tails have the model dtype, which may also be
float32.
"""

from __future__ import annotations

import dataclasses

import torch
import torch.nn.functional as F

from .. import ops
from ..engine.kv_cache import KVLayer, TailLayer, layer_parts
from .llama import _linear
from .mixed import LayerSpec, MixedConfig, MixedModel


@dataclasses.dataclass(frozen=True)
class YarnSpec:
    dims: int
    base: float
    factor: float
    original: float
    fast: float
    slow: float


@dataclasses.dataclass(frozen=True)
class DiffAttentionSpec:
    heads: int
    kv_heads: int
    dim: int                         # of one map
    vdim: int
    scale: float
    softcap: float
    chunk: int
    diff: float
    rot: YarnSpec


@dataclasses.dataclass(frozen=True)
class Relu2MoeSpec:
    experts: int
    identity: int
    top: int
    ff: int
    groups: int
    keep: int

    @property
    def routes(self) -> int:
        return self.experts + self.identity


def _mixer(kind: str, m: dict) -> DiffAttentionSpec:
    if kind != "attention":
        raise ValueError(f"unknown mixer {kind!r}")
    r, s = m["rot"], m["rot"]["scaling"]
    return DiffAttentionSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
        vdim=m["vdim"], scale=float(m["scale"]), softcap=float(m["softcap"]),
        chunk=int(m["mask"]["size"]), diff=float(m["diff"]),
        rot=YarnSpec(dims=r["dims"], base=float(r["base"]),
                     factor=float(s["factor"]),
                     original=float(s["original"]), fast=float(s["fast"]),
                     slow=float(s["slow"])))


def _feed_forward(f):
    if f is None:
        return None
    if f["kind"] != "moe":
        raise ValueError(f"unknown feed-forward {f['kind']!r}")
    r = f["router"]
    return Relu2MoeSpec(experts=r["experts"], identity=r["identity"],
                        top=r["top"], ff=f["expert"]["ff"],
                        groups=r["groups"]["count"],
                        keep=r["groups"]["keep"])


@dataclasses.dataclass
class FimunexConfig(MixedConfig):
    name: str
    hidden_size: int
    vocab_size: int
    rms_eps: float
    taps: int
    logit_softcap: float
    layers: tuple                    # LayerSpec
    loop: tuple = (0, 0, 1)          # first layer, one past the last, passes
    max_position: int = 32768        # serving limit, not a model constant
    eos_ids: tuple = ()

    def __post_init__(self) -> None:
        if self.hidden_size > 16000:
            raise ValueError("width must be at most 16000")
        if self.taps < 1:
            raise ValueError("a convolution has at least one tap")
        if self.logit_softcap <= 0:
            raise ValueError("the logits' cap must be positive")
        start, stop, times = self.loop
        if not (0 <= start <= stop <= len(self.layers) and times >= 1):
            raise ValueError("bad loop")
        for i, spec in enumerate(self.layers):
            m, f = spec.mixer, spec.mlp
            if m.heads % m.kv_heads:
                raise ValueError(f"layer {i}: heads % kv_heads")
            if m.rot.dims % 2 or m.rot.dims > m.dim:
                raise ValueError(f"layer {i}: bad rotation width")
            if m.vdim > 512 or m.dim > 2048:
                raise ValueError(f"layer {i}: attention maps are at most "
                                 f"2048 wide, values 512")
            if m.chunk < 1 or m.softcap <= 0:
                raise ValueError(f"layer {i}: chunk and softcap must be "
                                 f"positive")
            if f is None:
                continue
            if f.experts < 1 or f.routes > 256:
                raise ValueError(f"layer {i}: 1 to 256 experts, identities "
                                 f"included")
            if (f.groups < 1 or f.routes % f.groups
                    or not 1 <= f.keep <= f.groups
                    or not 1 <= f.top <= f.keep * (f.routes // f.groups)):
                raise ValueError(f"layer {i}: groups must divide the "
                                 f"experts, those kept hold the choice")

    @classmethod
    def from_dict(cls, d: dict, name: str = "fimunex", **kw):
        layers = []
        for i, e in enumerate(d["layers"]):
            try:
                layers.append(LayerSpec(_mixer(e["type"], e["mixer"]),
                                        _feed_forward(e.get("mlp"))))
            except ValueError as err:
                raise ValueError(f"layer {i}: {err}") from None
        loop = d.get("loop") or {"start": 0, "stop": 0, "times": 1}
        return cls(name=name, hidden_size=d["width"], vocab_size=d["vocab"],
                   rms_eps=float(d["norm"]["eps"]), taps=d["canon"]["taps"],
                   logit_softcap=float(d["logit_softcap"]),
                   layers=tuple(layers),
                   loop=(loop["start"], loop["stop"], loop["times"]), **kw)

    @property
    def order(self) -> list:
        """Layers as they run, the loop unrolled."""
        start, stop, times = self.loop
        n = list(range(len(self.layers)))
        return n[:start] + n[start:stop] * times + n[stop:]

    @property
    def sublayers(self) -> list:
        """(layer, 'mix' or 'mlp') as they run.  Each has a place of its own
        in the cache, also where layers run more than once."""
        return [(i, which) for i in self.order for which in ("mix", "mlp")
                if which == "mix" or self.layers[i].mlp is not None]

    def cache_layers(self, tp_world: int = 1) -> list:
        """What each sublayer that runs keeps per token and per sequence.
        Tails are whole on every rank."""
        tail = ((TailLayer(self.taps - 1, self.hidden_size),)
                if self.taps > 1 else ())
        out = []
        for i, which in self.sublayers:
            m = self.layers[i].mixer
            own = ((KVLayer(m.kv_heads // tp_world, 2 * m.dim, m.vdim),)
                   if which == "mix" else ())
            out.append((*own, *tail))
        return out

    def kv_elems_per_token(self, tp_world: int = 1) -> int:
        return sum(s.n_kv_heads * (s.k_dim + s.v_dim)
                   for spec in self.cache_layers(tp_world)
                   for s in layer_parts(spec) if isinstance(s, KVLayer))


def uniform_layers(n: int, attention: dict, mlp: dict) -> list:
    """config.json 'layers' of the usual shape: all alike."""
    return [{"type": "attention", "mixer": dict(attention),
             "mlp": dict(mlp)} for _ in range(n)]


def diff_attention(heads: int, kv_heads: int, dim: int, vdim: int,
                   chunk: int) -> dict:
    """config.json 'mixer' with the usual constants."""
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": dim ** -0.5, "softcap": 50.0, "diff": 0.5,
            "mask": {"size": chunk},
            "rot": {"dims": dim, "base": 1000000.0,
                    "scaling": {"factor": 8.0, "original": 4096,
                                "fast": 32.0, "slow": 1.0}}}


def relu2_moe(experts: int, identity: int, top: int, ff: int, groups: int,
              keep: int) -> dict:
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "identity": identity, "top": top,
                       "groups": {"count": groups, "keep": keep}}}


def _preset(name: str, width: int, vocab: int, layers: list, loop: tuple,
            **kw) -> FimunexConfig:
    return FimunexConfig.from_dict(
        {"layers": layers, "width": width, "vocab": vocab,
         "norm": {"eps": 1e-5}, "canon": {"taps": 4}, "logit_softcap": 30.0,
         "loop": dict(zip(("start", "stop", "times"), loop))}, name=name,
        **kw)


FIMUNEX_PRESETS = {
    # CPU-testable
    "fimunex-tiny": lambda: _preset(
        "fimunex-tiny", 128, 512, uniform_layers(
            3, diff_attention(4, 2, 16, 32, 48),
            relu2_moe(6, 2, 2, 64, 2, 1)), (1, 2, 2), max_position=2048),
    # layers of a real model's size
    "fimunex-2b": lambda: _preset(
        "fimunex-2b", 2048, 65536, uniform_layers(
            8, diff_attention(16, 4, 64, 128, 2048),
            relu2_moe(32, 8, 4, 1536, 8, 4)), (2, 6, 2)),
}


class FimunexForCausalLM(MixedModel):
    """Inference-only Fimunex.  TP shards heads and the expert width
    column-wise, output projections row-wise, with an all-reduce after each
    sublayer; router, convolutions, norms and the residual are replicated."""

    EXTENSIONS = ("rlli_attn", "rlli_blk", "rlli_mix")

    def sharded_sizes(self) -> list:
        sizes = []
        for spec in self.config.layers:
            sizes += [spec.mixer.heads, spec.mixer.kv_heads]
            if spec.mlp is not None:
                sizes.append(spec.mlp.ff)
        return sizes

    def _prepare(self) -> None:
        self._sublayers = self.config.sublayers
        self._rot = {
            r: ops.yarn_cos_sin(self.config.max_position, r.dims, r.base,
                                r.factor, r.original, r.fast, r.slow,
                                device=self.device).contiguous()
            for r in {spec.mixer.rot for spec in self.config.layers}}
        self._lambda: dict[int, float] = {}

    # ------------------------------------------------------------ weights
    def tensor_shapes(self) -> dict:
        c = self.config
        d = c.hidden_size
        out = {"embed": (c.vocab_size, d)}
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            out[p + "norm1"] = (d,)
            out[p + "canon1"] = (d, c.taps)
            q = p + "mix."
            for x, rows in (("q", m.heads * 2 * m.dim),
                            ("k", m.kv_heads * 2 * m.dim),
                            ("v", m.kv_heads * m.vdim)):
                out[q + x] = (rows, d)
                out[q + x + ".b"] = (rows,)
            for x in ("q.norm", "k.norm", "lq1", "lk1", "lq2", "lk2"):
                out[q + x] = (m.dim,)
            out[q + "g"] = (m.heads, d)
            out[q + "o"] = (d, m.heads * m.vdim)
            out[q + "o.b"] = (d,)
            if f is None:
                continue
            out[p + "norm2"] = (d,)
            out[p + "canon2"] = (d, c.taps)
            q = p + "mlp."
            out[q + "router"] = (f.routes, d)
            out[q + "correction"] = (f.routes,)
            for e in range(f.experts):
                out[f"{q}e{e}.up"] = (f.ff, d)
                out[f"{q}e{e}.down"] = (d, f.ff)
        out["final.norm"] = (d,)
        out["head"] = (c.vocab_size, d)
        return out

    def initial(self, leaf: str, shape: tuple):
        if leaf.endswith(("q.norm", "k.norm")):
            return torch.ones(shape)
        if "norm" in leaf or leaf.endswith((".b", ".correction")):
            return torch.zeros(shape)
        return None

    def _install(self, get) -> None:
        """Projections that share an input become one matrix (rows padded
        to eight, so that every activation row starts aligned), norm gains
        f32 multipliers (1 + w), an expert's width is zero-padded to 64 and
        the model's, where experts read it, to 8."""
        c, P = self.config, self.params
        d = c.hidden_size
        pad = -d % 8

        def mat(name, **kw):
            return self._mat(get(name), **kw)

        def vec(name, **kw):
            return self._vec(get(name), **kw)

        P["embed"] = mat("embed")
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            q = p + "mix."
            P[p + "norm.mix"] = 1 + vec(p + "norm1")
            P[p + "taps.mix"] = vec(p + "canon1").t().contiguous()
            w = torch.cat([mat(q + x, rows=True) for x in "qkvg"])
            P[p + "proj"] = F.pad(w, (0, 0, 0, -w.shape[0] % 8))
            P[p + "proj.b"] = torch.cat(
                [vec(f"{q}{x}.b", rows=True) for x in "qkv"])
            P[p + "q_norm"], P[p + "k_norm"] = (vec(q + "q.norm"),
                                                vec(q + "k.norm"))
            one, two = ((vec(q + "lq" + x) * vec(q + "lk" + x)).sum().exp()
                        for x in "12")
            self._lambda[i] = float(one - two) + m.diff
            P[p + "o"] = mat(q + "o", cols=True)
            P[p + "o.b"] = vec(q + "o.b")
            if f is None:
                continue
            q = p + "mlp."
            P[p + "norm.mlp"] = 1 + vec(p + "norm2")
            P[p + "taps.mlp"] = vec(p + "canon2").t().contiguous()
            P[p + "router"] = F.pad(mat(q + "router"), (0, pad))
            P[p + "correction"] = vec(q + "correction")
            ff = f.ff // self.tp_world
            ffp = -(-ff // 64) * 64
            up = torch.zeros((f.experts, ffp, d + pad), dtype=self.dtype,
                             device=self.device)
            down = torch.zeros((f.experts, d + pad, ffp), dtype=self.dtype,
                               device=self.device)
            for e in range(f.experts):
                up[e, :ff, :d] = mat(f"{q}e{e}.up", rows=True)
                down[e, :d, :ff] = mat(f"{q}e{e}.down", cols=True)
            P[p + "w_up"], P[p + "w_down"] = up, down
        P["final.norm"] = 1 + vec("final.norm")
        P["head"] = mat("head")

    # ------------------------------------------------------------ compute
    def _attention(self, i, place, h, kv_cache, step):
        """(output, what block_step needs to add it)."""
        P, p, nd = self.params, f"l{i}.", step.n_decode
        m, n = self.config.layers[i].mixer, self.tp_world
        qkv = _linear(h, P[p + "proj"])
        heads, kv = m.heads // n, m.kv_heads // n
        g0 = 2 * (heads + kv) * m.dim + kv * m.vdim
        gate = qkv[:, g0:g0 + heads]
        k, v = kv_cache.layer(place)
        score = (heads, P[p + "proj.b"], P[p + "q_norm"], P[p + "k_norm"],
                 m.scale, m.chunk, m.softcap, self._lambda[i], 1 - m.diff,
                 self.config.rms_eps)
        parts = []
        if nd:
            parts.append(ops.diff_decode(
                qkv[:nd], gate[:nd], k, v, step.positions[:nd],
                self._rot[m.rot], step.slots[:nd], step.tables_dec, *score))
        if step.prompt is not None:
            parts.append(ops.diff_prefill(
                qkv[nd:], gate[nd:], k, v, step.positions[nd:],
                self._rot[m.rot], step.slots[nd:], step.tables_pre,
                step.prompt, *score))
        out = parts[0] if len(parts) == 1 else torch.cat(parts)
        return (self._reduce(_linear(out, P[p + "o"])),
                dict(y_bias=P[p + "o.b"]))

    def _experts(self, i, h):
        """(output, what block_step needs to add it)."""
        P, f, p = self.params, self.config.layers[i].mlp, f"l{i}."
        W = h.shape[1]
        pad = -W % 8
        y, ids, w = ops.moe_relu2(
            F.pad(h, (0, pad)) if pad else h, P[p + "router"],
            P[p + "correction"], P[p + "w_up"], P[p + "w_down"], f.top,
            f.groups, f.keep)
        if pad:
            y = y[..., :W].contiguous()
        if self.tp_world == 1:
            return y, dict(part_ids=ids, part_w=w, part_h=h,
                           part_limit=f.experts)
        # experts are spread over the ranks, identities are whole on each
        same = (ids >= f.experts)[..., None]
        y = self._reduce(y.float().masked_fill(same, 0).sum(1)
                         .to(self.dtype))
        own = (w[..., None] * same).sum(1)
        return (y.float() + own * h.float()).to(self.dtype), {}

    def _forward(self, input_ids, kv_cache, step, sample_idx):
        P, c, nd = self.params, self.config, step.n_decode
        x = torch.empty((input_ids.shape[0], c.hidden_size),
                        dtype=torch.float32, device=self.device)

        def tail(n):
            return kv_cache.states.tail(n) if kv_cache.states else None

        def reads(n):
            """The norm and convolution ahead of sublayer n."""
            i, which = self._sublayers[n]
            return ((P[f"l{i}.norm.{which}"], 1, c.rms_eps),
                    (P[f"l{i}.taps.{which}"], tail(n), step.state_slots, nd))

        norm, conv = reads(0)
        h, hc = ops.block_embed(input_ids, P["embed"], None, step.positions,
                                x, *norm, *conv)
        for n, (i, which) in enumerate(self._sublayers):
            if step.prompt is not None:
                ops.conv_prompt(h[nd:], P[f"l{i}.taps.{which}"], tail(n),
                                step.prompt, hc[nd:])
            if which == "mix":
                y, more = self._attention(i, n, hc, kv_cache, step)
            else:
                y, more = self._experts(i, hc)
            if n + 1 < len(self._sublayers):
                norm, conv = reads(n + 1)
                h, hc = ops.block_step(x, y, *norm, step.positions, *conv,
                                       **more)
            else:
                h, _ = ops.block_step(
                    x, y, P["final.norm"], 1, c.rms_eps, step.positions,
                    rows=sample_idx, keep=False, **more)
        return ops.soft_cap(_linear(h, P["head"]), c.logit_softcap)
