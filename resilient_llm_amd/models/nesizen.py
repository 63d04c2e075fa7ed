"""Nesizen: a decoder whose layers differ, MI355X-first.

Residual streams (hyper-connections) instead of one residual; per layer
either windowed attention (kept first tokens, a learned sink, interleaved
partial rotation, optionally an earlier layer's keys and values) or gated
linear attention; per layer a squared-relu feed-forward, a mixture of
experts, or none.  Sizes, constants and the order of layers come from
config.json.

Same shape as models/llama.py: a flat parameter store and an explicit
forward over the serving ops.  Each layer is one projection GEMM, one
fused mixer op, one output GEMM, and between any two sublayers one
hyper_step op that writes the residual streams and norms the next input.
Streams, norms, routers, decays and recurrent states are 32-bit; GEMM
inputs and the KV cache have the model dtype, which may also be float32
throughout.
"""

from __future__ import annotations

import dataclasses
from typing import Optional

import torch
import torch.nn.functional as F

from .. import ops
from ..engine.kv_cache import KVLayer, StateLayer
from .llama import _linear
from .mixed import DenseSpec, LayerSpec, MixedConfig, MixedModel


@dataclasses.dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float
    window: int
    keep_first: int
    kv_from: Optional[int] = None


@dataclasses.dataclass(frozen=True)
class GlaSpec:
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclasses.dataclass(frozen=True)
class MoeSpec:
    experts: int
    top: int
    ff: int
    limit: float


@dataclasses.dataclass
class NesizenConfig(MixedConfig):
    name: str
    hidden_size: int
    vocab_size: int
    streams: int
    rms_eps: float
    layers: tuple
    decay_rank: int = 16             # random init; a checkpoint's own wins
    max_position: int = 32768        # serving limit, not a model constant
    eos_ids: tuple = ()

    def __post_init__(self) -> None:
        if self.hidden_size % 8 or self.hidden_size > 8192:
            raise ValueError("width must be a multiple of 8, at most 8192")
        if not 1 <= self.streams <= 8:
            raise ValueError("1 to 8 residual streams")
        for i, spec in enumerate(self.layers):
            m = spec.mixer
            if isinstance(m, AttentionSpec):
                if m.heads % m.kv_heads:
                    raise ValueError(f"layer {i}: heads % kv_heads")
                if m.rot_dims % 2 or m.rot_dims > m.dim:
                    raise ValueError(f"layer {i}: bad rotation width")
                if m.kv_from is not None:
                    src = (self.layers[m.kv_from].mixer
                           if 0 <= m.kv_from < i else None)
                    if (not isinstance(src, AttentionSpec)
                            or src.kv_from is not None
                            or (src.kv_heads, src.dim, src.vdim)
                            != (m.kv_heads, m.dim, m.vdim)):
                        raise ValueError(
                            f"layer {i}: kv_from must name an earlier "
                            f"attention layer with projections of its own "
                            f"and the same key/value sizes")

    @classmethod
    def from_dict(cls, d: dict, name: str = "nesizen", **kw):
        layers = []
        for i, e in enumerate(d["layers"]):
            m, f = e["mixer"], e.get("mlp")
            if e["type"] == "attention":
                mixer = AttentionSpec(
                    heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                    vdim=m["vdim"], scale=float(m["scale"]),
                    rot_dims=m["rot"]["dims"],
                    rot_base=float(m["rot"]["base"]),
                    window=m["mask"]["size"],
                    keep_first=m["mask"]["keep_first"],
                    kv_from=m.get("kv_from"))
            elif e["type"] == "gla":
                mixer = GlaSpec(heads=m["heads"], dim=m["dim"],
                                vdim=m["vdim"], tau=float(m["tau"]))
            else:
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            if f is None:
                mlp = None
            elif f["kind"] == "dense":
                mlp = DenseSpec(f["ff"])
            elif f["kind"] == "moe":
                mlp = MoeSpec(experts=f["router"]["experts"],
                              top=f["router"]["top"], ff=f["expert"]["ff"],
                              limit=float(f["expert"]["limit"]))
            else:
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{f['kind']!r}")
            layers.append(LayerSpec(mixer, mlp))
        return cls(name=name, hidden_size=d["width"], vocab_size=d["vocab"],
                   streams=d["streams"], rms_eps=float(d["norm"]["eps"]),
                   layers=tuple(layers), **kw)

    def cache_layers(self, tp_world: int = 1) -> list:
        """What each layer keeps per token or per sequence."""
        out = []
        for spec in self.layers:
            m = spec.mixer
            if isinstance(m, AttentionSpec):
                out.append(KVLayer(m.kv_heads // tp_world, m.dim, m.vdim,
                                   m.kv_from))
            else:
                out.append(StateLayer(m.heads // tp_world, m.dim, m.vdim))
        return out

    def kv_elems_per_token(self, tp_world: int = 1) -> int:
        return sum(s.n_kv_heads * (s.k_dim + s.v_dim)
                   for s in self.cache_layers(tp_world)
                   if isinstance(s, KVLayer) and s.share is None)


def hybrid_layers(n: int, attn_every: int, attention: dict, gla: dict,
                  mlp: dict, first_dense: Optional[dict] = None) -> list:
    """config.json 'layers' of the usual shape: one attention layer, then
    attn_every - 1 recurrent ones, repeated."""
    out = []
    for i in range(n):
        attn = i % attn_every == 0
        out.append({"type": "attention" if attn else "gla",
                    "mixer": dict(attention if attn else gla),
                    "mlp": dict(first_dense if i == 0 and first_dense
                                else mlp)})
    return out


def _preset(name: str, width: int, vocab: int, layers: list,
            **kw) -> NesizenConfig:
    return NesizenConfig.from_dict(
        {"layers": layers, "norm": {"eps": 1e-5}, "streams": 2,
         "vocab": vocab, "width": width}, name=name, **kw)


NESIZEN_PRESETS = {
    # CPU-testable
    "nesizen-tiny": lambda: _preset(
        "nesizen-tiny", 128, 512, hybrid_layers(
            4, 2,
            {"heads": 4, "kv_heads": 2, "dim": 32, "vdim": 32,
             "scale": 32 ** -0.5, "rot": {"dims": 16, "base": 10000.0},
             "mask": {"size": 48, "keep_first": 2}},
            {"heads": 2, "dim": 32, "vdim": 48, "tau": 8.0},
            {"kind": "moe", "expert": {"ff": 64, "limit": 2.0},
             "router": {"experts": 4, "top": 2}},
            {"kind": "dense", "ff": 192}), max_position=2048),
    # layers of a real model's size (bench.py --nesizen)
    "nesizen-3b": lambda: _preset(
        "nesizen-3b", 2048, 65536, hybrid_layers(
            12, 3,
            {"heads": 16, "kv_heads": 4, "dim": 128, "vdim": 128,
             "scale": 128 ** -0.5, "rot": {"dims": 64, "base": 1000000.0},
             "mask": {"size": 1024, "keep_first": 4}},
            {"heads": 8, "dim": 128, "vdim": 256, "tau": 16.0},
            {"kind": "moe", "expert": {"ff": 1024, "limit": 7.0},
             "router": {"experts": 32, "top": 4}},
            {"kind": "dense", "ff": 8192})),
}


class NesizenForCausalLM(MixedModel):
    """Inference-only Nesizen.  TP shards heads (attention and recurrent),
    the dense and expert widths column-wise, output projections row-wise,
    with an all-reduce after each sublayer; streams are replicated."""

    EXTENSIONS = ("rlli_attn", "rlli_mix", "rlli_rec")

    def sharded_sizes(self) -> list:
        sizes = []
        for spec in self.config.layers:
            m, f = spec.mixer, spec.mlp
            sizes.append(m.heads)
            if isinstance(m, AttentionSpec):
                sizes.append(m.kv_heads)
            if f is not None:
                sizes.append(f.ff)
        return sizes

    def _prepare(self) -> None:
        self._rot: dict[tuple, torch.Tensor] = {}
        for spec in self.config.layers:
            m = spec.mixer
            if isinstance(m, AttentionSpec):
                key = (m.rot_dims, m.rot_base)
                if key not in self._rot:
                    self._rot[key] = ops.build_cos_sin(
                        self.config.max_position, m.rot_dims, m.rot_base,
                        device=self.device).contiguous()

    # ------------------------------------------------------------ weights
    def tensor_shapes(self) -> dict:
        """Checkpoint names -> shapes (full, unsharded)."""
        c = self.config
        d, s, rank = c.hidden_size, c.streams, c.decay_rank
        out = {"embed": (c.vocab_size, d), "embed.norm": (d,)}
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            for q in (1, 2) if f is not None else (1,):
                out[f"{p}norm{q}"] = (d,)
                out[f"{p}hc{q}.in"] = (s,)
                out[f"{p}hc{q}.out"] = (s,)
                out[f"{p}hc{q}.mix"] = (s, s)
            out[p + "mix.q"] = (m.heads * m.dim, d)
            out[p + "mix.o"] = (d, m.heads * m.vdim)
            if isinstance(m, AttentionSpec):
                if m.kv_from is None:
                    out[p + "mix.k"] = (m.kv_heads * m.dim, d)
                    out[p + "mix.v"] = (m.kv_heads * m.vdim, d)
                out[p + "mix.sink"] = (m.heads,)
            else:
                out[p + "mix.k"] = (m.heads * m.dim, d)
                out[p + "mix.v"] = (m.heads * m.vdim, d)
                out[p + "mix.g"] = (m.heads * m.vdim, d)
                out[p + "mix.norm"] = (m.vdim,)
                out[p + "mix.a1"] = (rank, d)
                out[p + "mix.a2"] = (m.heads * m.dim, rank)
                out[p + "mix.a2.b"] = (m.heads * m.dim,)
            if isinstance(f, DenseSpec):
                out[p + "mlp.up"] = (f.ff, d)
                out[p + "mlp.down"] = (d, f.ff)
            elif isinstance(f, MoeSpec):
                out[p + "mlp.router"] = (f.experts, d)
                for e in range(f.experts):
                    out[f"{p}mlp.e{e}.gate"] = (f.ff, d)
                    out[f"{p}mlp.e{e}.up"] = (f.ff, d)
                    out[f"{p}mlp.e{e}.down"] = (d, f.ff)
        out["final.norm"] = (d,)
        out["head"] = (c.vocab_size, d)
        return out

    def initial(self, leaf: str, shape: tuple):
        s = self.config.streams
        if leaf == "mix.norm":
            return torch.ones(shape)
        if "norm" in leaf or leaf == "mix.sink":
            return torch.zeros(shape)
        if leaf.startswith("hc"):
            if leaf.endswith(".mix"):
                return torch.eye(s)
            return torch.full(shape, 1.0 / s if leaf.endswith(".in") else 1.0)
        if leaf == "mix.a2.b":
            return torch.full(shape, 2.0)
        return None

    def _checkpoint_shapes(self, shape_of, names) -> dict:
        # the decay rank is the one size that a tensor's shape gives
        shapes = self.tensor_shapes()
        for n, (_, d) in [(n, s) for n, s in shapes.items()
                          if n.endswith(".mix.a1") and n in names]:
            rank = shape_of(n)[0]
            shapes[n] = (rank, d)
            a2 = n[:-1] + "2"
            shapes[a2] = (shapes[a2][0], rank)
        return shapes

    def _install(self, get) -> None:
        """Pack full checkpoint tensors into this rank's parameters:
        projections that share an input become one matrix, norm gains are
        stored as f32 multipliers (1 + w), expert gate and up rows are
        interleaved in blocks of 16 (the grouped GEMM pairs them in its
        accumulators) with the expert width zero-padded to 64."""
        c, P = self.config, self.params
        n = self.tp_world

        def mat(name, **kw):
            return self._mat(get(name), **kw)

        def vec(name, **kw):
            return self._vec(get(name), **kw)

        P["embed"] = mat("embed")
        P["embed.norm"] = 1 + vec("embed.norm")
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            for q in (1, 2) if f is not None else (1,):
                P[f"{p}norm{q}"] = 1 + vec(f"{p}norm{q}")
                for leaf in ("in", "out", "mix"):
                    P[f"{p}hc{q}.{leaf}"] = vec(f"{p}hc{q}.{leaf}")
            if isinstance(m, AttentionSpec):
                names = ["q"] if m.kv_from is not None else ["q", "k", "v"]
                P[p + "proj"] = torch.cat(
                    [mat(f"{p}mix.{x}", rows=True) for x in names])
                P[p + "sink"] = vec(p + "mix.sink", rows=True)
            else:
                P[p + "proj"] = torch.cat(
                    [mat(f"{p}mix.{x}", rows=True) for x in "qkvg"]
                    + [mat(p + "mix.a1")])
                P[p + "a2"] = mat(p + "mix.a2", rows=True)
                P[p + "a2.b"] = vec(p + "mix.a2.b", rows=True)
                P[p + "gla_norm"] = vec(p + "mix.norm")
            P[p + "o"] = mat(p + "mix.o", cols=True)
            if isinstance(f, DenseSpec):
                P[p + "up"] = mat(p + "mlp.up", rows=True)
                P[p + "down"] = mat(p + "mlp.down", cols=True)
            elif isinstance(f, MoeSpec):
                P[p + "router"] = mat(p + "mlp.router")
                ff = f.ff // n
                ffp = -(-ff // 64) * 64
                d = c.hidden_size
                up = torch.zeros((f.experts, ffp // 16, 2, 16, d),
                                 dtype=self.dtype, device=self.device)
                down = torch.zeros((f.experts, d, ffp), dtype=self.dtype,
                                   device=self.device)
                for e in range(f.experts):
                    for g, x in enumerate(("gate", "up")):
                        t = mat(f"{p}mlp.e{e}.{x}", rows=True)
                        t = F.pad(t, (0, 0, 0, ffp - ff))
                        up[e, :, g] = t.view(ffp // 16, 16, d)
                    down[e, :, :ff] = mat(f"{p}mlp.e{e}.down", cols=True)
                P[p + "w_up"], P[p + "w_down"] = up, down
        P["final.norm"] = 1 + vec("final.norm")
        P["head"] = mat("head")

    # ------------------------------------------------------------ compute
    def _reduce(self, y: torch.Tensor) -> torch.Tensor:
        if self.tp_world > 1:
            import torch.distributed as dist
            if y.dim() == 3:
                y = y.float().sum(1).to(self.dtype)
            dist.all_reduce(y, group=self.tp_group)
        return y

    def _feed_forward(self, i: int, h: torch.Tensor) -> torch.Tensor:
        P, f, p = self.params, self.config.layers[i].mlp, f"l{i}."
        if isinstance(f, DenseSpec):
            return _linear(ops.relu2(_linear(h, P[p + "up"])), P[p + "down"])
        return ops.moe_experts(h, P[p + "router"], P[p + "w_up"],
                               P[p + "w_down"], f.top, f.limit)

    def _forward(self, input_ids, mixer, sample_idx) -> torch.Tensor:
        """``mixer(i, proj)``: the mixer of layer i on its projections."""
        P, c = self.params, self.config
        x = torch.empty((input_ids.shape[0], c.streams, c.hidden_size),
                        dtype=torch.float32, device=self.device)
        subs = [(i, q) for i, s in enumerate(c.layers)
                for q in ((1, 2) if s.mlp is not None else (1,))]
        h = ops.hyper_embed(input_ids, P["embed"], P["embed.norm"], x,
                            P["l0.hc1.in"], P["l0.norm1"], c.rms_eps)
        for n, (i, q) in enumerate(subs):
            p = f"l{i}."
            if q == 1:
                y = _linear(mixer(i, _linear(h, P[p + "proj"])), P[p + "o"])
            else:
                y = self._feed_forward(i, h)
            y = self._reduce(y)
            mix, out = P[f"{p}hc{q}.mix"], P[f"{p}hc{q}.out"]
            if n + 1 < len(subs):
                j, r = subs[n + 1]
                h = ops.hyper_step(x, y, mix, out, P[f"l{j}.hc{r}.in"],
                                   P[f"l{j}.norm{r}"], c.rms_eps)
            else:
                h = ops.hyper_step(x, y, mix, out, None, P["final.norm"],
                                   c.rms_eps, sample_idx, keep=False)
        return _linear(h, P["head"])

    def _attn_args(self, i: int, m: AttentionSpec):
        return (self.params[f"l{i}.sink"], m.scale, m.heads // self.tp_world,
                m.window, m.keep_first, m.kv_from is None)

    def _gla_args(self, i: int, kv_cache):
        P, p = self.params, f"l{i}."
        return (P[p + "a2"], P[p + "a2.b"], P[p + "gla_norm"],
                kv_cache.states.layer(i))

    def _decode_mixer(self, i, proj, positions, kv_cache, slots,
                      block_tables, state_slots):
        m = self.config.layers[i].mixer
        if isinstance(m, AttentionSpec):
            k, v = kv_cache.layer(i)
            return ops.window_decode(
                proj, k, v, positions, self._rot[m.rot_dims, m.rot_base],
                slots, block_tables, *self._attn_args(i, m))
        return ops.gla_decode(proj, *self._gla_args(i, kv_cache),
                              state_slots, positions, m.vdim, m.tau,
                              self.config.rms_eps)

    def _prompt_mixer(self, i, proj, positions, kv_cache, slots,
                      block_tables, prompt):
        m = self.config.layers[i].mixer
        if isinstance(m, AttentionSpec):
            k, v = kv_cache.layer(i)
            return ops.window_prefill(
                proj, k, v, positions, self._rot[m.rot_dims, m.rot_base],
                slots, block_tables, prompt, *self._attn_args(i, m))
        return ops.gla_prefill(proj, *self._gla_args(i, kv_cache), prompt,
                               m.vdim, m.tau, self.config.rms_eps)

    def forward_decode(self, input_ids, positions, kv_cache, slot_mapping,
                       block_tables, seq_lens, state_slots=None):
        """One token per sequence; returns [batch, vocab] logits."""
        return self._forward(
            input_ids,
            lambda i, proj: self._decode_mixer(
                i, proj, positions, kv_cache, slot_mapping, block_tables,
                state_slots),
            None)

    def forward_mixed(self, input_ids, positions, kv_cache, slot_mapping,
                      n_decode: int, block_tables_dec, seq_lens_dec,
                      block_tables_pre, prompt, sample_idx,
                      state_slots=None):
        """Rows [0, n_decode) decode one token per sequence, the rest are
        the portions of ``prompt`` (engine/batch.py).  Returns the logits
        of ``sample_idx`` rows."""
        nd = n_decode

        def mixer(i, proj):
            if not nd:
                return self._prompt_mixer(i, proj, positions, kv_cache,
                                          slot_mapping, block_tables_pre,
                                          prompt)
            return torch.cat([
                self._decode_mixer(i, proj[:nd], positions[:nd], kv_cache,
                                   slot_mapping[:nd], block_tables_dec,
                                   state_slots),
                self._prompt_mixer(i, proj[nd:], positions[nd:], kv_cache,
                                   slot_mapping[nd:], block_tables_pre,
                                   prompt)])
        return self._forward(input_ids, mixer, sample_idx)
