"""Riruzen: parallel blocks over latent attention and HGRN2, MI355X-first.

Every layer reads one grouped norm h of the residual; its mixer works on
h + conv(h), a short causal convolution, its feed-forward on h, and both
are added.  Mixers, in any order: latent attention without positions (one
normed latent per token is all it caches, queries through a latent of
their own, sigmoid output gate) and HGRN2 (a linear recurrence without keys:
a channel takes up as much as it lets go).  Learned positions are added to the
embedding; the output layer is the embedding.  Sizes, constants and the
order of layers come from config.json.

A layer is two input products (mixer, feed-forward), the mixer's ops, one
gated activation and ONE output product: mixer and feed-forward leave their
activations side by side, so W_o and W_down are one matrix and their sum is
formed in its accumulators.  Between layers one op writes the residual and
norms the next input; for decoded tokens it also convolves.  Residual,
norms, decays and states are 32-bit; product inputs, the cached latents and
the convolution tails have the model dtype, which may also be float32.
"""

from __future__ import annotations

import dataclasses

import torch

from .. import ops
from ..engine.kv_cache import LatentLayer, StateLayer, TailLayer, layer_parts
from .llama import _linear
from .mixed import DenseSpec, LayerSpec, MixedConfig, MixedModel


@dataclasses.dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float


@dataclasses.dataclass(frozen=True)
class Hgrn2Spec:
    heads: int
    dim: int
    vdim: int


@dataclasses.dataclass
class RiruzenConfig(MixedConfig):
    name: str
    hidden_size: int
    vocab_size: int
    norm_groups: int
    rms_eps: float
    taps: int
    logit_scale: float
    max_position: int                # rows of the learned position table
    layers: tuple                    # LayerSpec: LatentSpec | Hgrn2Spec
    eos_ids: tuple = ()

    def __post_init__(self) -> None:
        if self.norm_groups < 1 or self.hidden_size % self.norm_groups:
            raise ValueError("norm groups must divide the width")
        if self.hidden_size > 16000:
            raise ValueError("width must be at most 16000")
        if self.taps < 1:
            raise ValueError("a convolution has at least one tap")
        for i, spec in enumerate(self.layers):
            m = spec.mixer
            if isinstance(m, LatentSpec) and m.kv_rank > 1024:
                raise ValueError(f"layer {i}: kv_rank is at most 1024")
            if isinstance(m, Hgrn2Spec) and (m.dim > 256 or m.vdim > 1024):
                raise ValueError(f"layer {i}: recurrent heads are at most "
                                 f"256 x 1024")

    @classmethod
    def from_dict(cls, d: dict, name: str = "riruzen", **kw):
        layers = []
        for i, e in enumerate(d["layers"]):
            m, f = e["mixer"], e.get("mlp")
            if e["type"] == "latent_attention":
                mixer = LatentSpec(
                    heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                    q_rank=m["q_rank"], kv_rank=m["kv_rank"],
                    scale=float(m["scale"]))
            elif e["type"] == "hgrn2":
                mixer = Hgrn2Spec(heads=m["heads"], dim=m["dim"],
                                  vdim=m["vdim"])
            else:
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            if f is None:
                mlp = None
            elif f["kind"] == "dense":
                mlp = DenseSpec(f["ff"])
            else:
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{f['kind']!r}")
            layers.append(LayerSpec(mixer, mlp))
        return cls(name=name, hidden_size=d["width"], vocab_size=d["vocab"],
                   norm_groups=d["norm"]["groups"],
                   rms_eps=float(d["norm"]["eps"]), taps=d["canon"]["taps"],
                   logit_scale=float(d["logit_scale"]),
                   max_position=d["max_positions"], layers=tuple(layers),
                   **kw)

    def fit_positions(self, n: int) -> None:
        """The learned table is the limit, whatever the pool holds."""

    def cache_layers(self, tp_world: int = 1) -> list:
        """What each layer keeps per token and per sequence.  Latents
        serve all heads, so every rank holds them whole."""
        tail = ((TailLayer(self.taps - 1, self.hidden_size),)
                if self.taps > 1 else ())
        out = []
        for spec in self.layers:
            m = spec.mixer
            if isinstance(m, LatentSpec):
                own = LatentLayer(m.kv_rank)
            else:
                own = StateLayer(m.heads // tp_world, m.dim, m.vdim)
            out.append((own, *tail))
        return out

    def kv_elems_per_token(self, tp_world: int = 1) -> int:
        return sum(s.dim for spec in self.cache_layers(tp_world)
                   for s in layer_parts(spec) if isinstance(s, LatentLayer))


def hybrid_layers(n: int, attn_every: int, latent: dict, hgrn2: dict,
                  mlp: dict) -> list:
    """config.json 'layers' of the usual shape: one latent attention layer,
    then attn_every - 1 recurrent ones, repeated."""
    return [{"type": "hgrn2" if i % attn_every else "latent_attention",
             "mixer": dict(hgrn2 if i % attn_every else latent),
             "mlp": dict(mlp)} for i in range(n)]


def _preset(name: str, width: int, vocab: int, layers: list, groups: int,
            max_positions: int) -> RiruzenConfig:
    return RiruzenConfig.from_dict(
        {"layers": layers, "width": width, "vocab": vocab,
         "norm": {"eps": 1e-5, "groups": groups}, "canon": {"taps": 4},
         "logit_scale": 1.0, "max_positions": max_positions}, name=name)


RIRUZEN_PRESETS = {
    # CPU-testable
    "riruzen-tiny": lambda: _preset(
        "riruzen-tiny", 128, 512, hybrid_layers(
            4, 2,
            {"heads": 4, "dim": 32, "vdim": 32, "q_rank": 48, "kv_rank": 64,
             "scale": 32 ** -0.5},
            {"heads": 2, "dim": 32, "vdim": 48},
            {"kind": "dense", "ff": 256}), 4, 2048),
    # layers of a real model's size
    "riruzen-1b": lambda: _preset(
        "riruzen-1b", 2048, 65536, hybrid_layers(
            12, 3,
            {"heads": 16, "dim": 128, "vdim": 128, "q_rank": 768,
             "kv_rank": 512, "scale": 128 ** -0.5},
            {"heads": 16, "dim": 128, "vdim": 128},
            {"kind": "dense", "ff": 4096}), 4, 32768),
}


class RiruzenForCausalLM(MixedModel):
    """Inference-only Riruzen.  TP shards heads and the feed-forward width
    column-wise and the joint output product row-wise, with one all-reduce
    per layer; latents, norms, convolutions and the residual are
    replicated."""

    EXTENSIONS = ("rlli_attn", "rlli_blk", "rlli_rec", "rlli_lat")

    def sharded_sizes(self) -> list:
        return [s for spec in self.config.layers for s in
                (spec.mixer.heads, spec.mlp.ff if spec.mlp else 0)]

    # ------------------------------------------------------------ weights
    def tensor_shapes(self) -> dict:
        c = self.config
        d = c.hidden_size
        out = {"embed": (c.vocab_size, d), "pos": (c.max_position, d)}
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            out[p + "norm1"] = (d,)
            if isinstance(m, LatentSpec):
                out[p + "mix.dq"] = (m.q_rank, d)
                out[p + "mix.dq.norm"] = (m.q_rank,)
                out[p + "mix.uq"] = (m.heads * m.dim, m.q_rank)
                out[p + "mix.dkv"] = (m.kv_rank, d)
                out[p + "mix.dkv.norm"] = (m.kv_rank,)
                out[p + "mix.uk"] = (m.heads * m.dim, m.kv_rank)
                out[p + "mix.uv"] = (m.heads * m.vdim, m.kv_rank)
                out[p + "mix.g"] = (m.heads * m.vdim, d)
            else:
                out[p + "mix.q"] = (m.heads * m.dim, d)
                out[p + "mix.f"] = (m.heads * m.dim, d)
                out[p + "mix.f.b"] = (m.heads * m.dim,)
                out[p + "mix.lower"] = (m.heads * m.dim,)
                out[p + "mix.v"] = (m.heads * m.vdim, d)
                out[p + "mix.norm"] = (m.vdim,)
            out[p + "mix.o"] = (d, m.heads * m.vdim)
            if f is not None:
                out[p + "mlp.gate"] = (f.ff, d)
                out[p + "mlp.up"] = (f.ff, d)
                out[p + "mlp.down"] = (d, f.ff)
            out[p + "canon1"] = (d, c.taps)
        out["final.norm"] = (d,)
        return out

    def initial(self, leaf: str, shape: tuple):
        if leaf.endswith(("norm", "norm1")):
            return torch.ones(shape)
        if leaf == "mix.f.b":
            return torch.full(shape, 2.0)
        if leaf == "mix.lower":
            return torch.linspace(0.0, 0.9, shape[0])
        return None

    def _install(self, get) -> None:
        """Projections that share an input become one matrix, and so do the
        two output projections; key up-projections are also kept
        transposed, for absorbing them into queries; the output scale goes
        into the last norm's gain."""
        P = self.params

        def mat(name, **kw):
            return self._mat(get(name), **kw)

        def vec(name, **kw):
            return self._vec(get(name), **kw)

        P["embed"], P["pos"] = mat("embed"), mat("pos")
        for i, spec in enumerate(self.config.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            P[p + "norm"] = vec(p + "norm1")
            P[p + "taps"] = vec(p + "canon1").t().contiguous()
            if isinstance(m, LatentSpec):
                P[p + "proj"] = torch.cat(
                    [mat(p + "mix.dq"), mat(p + "mix.dkv"),
                     mat(p + "mix.g", rows=True)])
                P[p + "q_norm"] = vec(p + "mix.dq.norm")
                P[p + "kv_norm"] = vec(p + "mix.dkv.norm")
                P[p + "uq"] = mat(p + "mix.uq", rows=True)
                P[p + "uk"] = mat(p + "mix.uk", rows=True)
                P[p + "uk_t"] = P[p + "uk"].view(
                    -1, m.dim, m.kv_rank).transpose(1, 2).contiguous()
                P[p + "uv"] = mat(p + "mix.uv", rows=True)
            else:
                P[p + "proj"] = torch.cat(
                    [mat(f"{p}mix.{x}", rows=True) for x in "qfv"])
                P[p + "f.b"] = vec(p + "mix.f.b", rows=True)
                P[p + "lower"] = vec(p + "mix.lower", rows=True)
                P[p + "head_norm"] = vec(p + "mix.norm")
            out = [mat(p + "mix.o", cols=True)]
            if f is not None:
                P[p + "gate_up"] = torch.cat(
                    [mat(p + "mlp.gate", rows=True),
                     mat(p + "mlp.up", rows=True)])
                out.append(mat(p + "mlp.down", cols=True))
            P[p + "out"] = torch.cat(out, dim=1).contiguous()
        P["final.norm"] = vec("final.norm") * self.config.logit_scale

    # ------------------------------------------------------------ compute
    def _latent(self, i, m, proj, kv_cache, step, out) -> None:
        P, p, nd = self.params, f"l{i}.", step.n_decode
        cache, = kv_cache.layer(i)
        cq = ops.latent_prep(proj, P[p + "q_norm"], P[p + "kv_norm"],
                             self.config.rms_eps, cache, step.slots)
        q = _linear(cq, P[p + "uq"])
        gate = proj[:, m.q_rank + m.kv_rank:]
        uv = P[p + "uv"].view(-1, m.vdim, m.kv_rank)
        if nd:
            ops.latent_decode(q[:nd], gate[:nd], cache, step.positions[:nd],
                              step.tables_dec, m.scale, P[p + "uk_t"], uv,
                              out[:nd])
        if step.prompt is not None:
            ops.latent_prefill(q[nd:], gate[nd:], cache, step.tables_pre,
                               step.prompt, m.scale, P[p + "uk_t"], uv,
                               P[p + "uk"], P[p + "uv"], out[nd:])

    def _hgrn2(self, i, m, proj, kv_cache, step, out) -> None:
        P, p, nd = self.params, f"l{i}.", step.n_decode
        args = (P[p + "f.b"], P[p + "lower"], P[p + "head_norm"],
                kv_cache.states.layer(i))
        eps = self.config.rms_eps
        if nd:
            ops.hgrn2_decode(proj[:nd], *args, step.state_slots,
                             step.positions[:nd], m.vdim, eps, out[:nd])
        if step.prompt is not None:
            ops.hgrn2_prefill(proj[nd:], *args, step.prompt, m.vdim, eps,
                              out[nd:])

    def _forward(self, input_ids, kv_cache, step, sample_idx):
        P, c, nd = self.params, self.config, step.n_decode
        T = input_ids.shape[0]
        x = torch.empty((T, c.hidden_size), dtype=torch.float32,
                        device=self.device)

        def tail(i):
            return kv_cache.states.tail(i) if kv_cache.states else None

        def norm_args(i):
            return (P[f"l{i}.norm"], c.norm_groups, c.rms_eps)

        def conv_args(i):
            return (P[f"l{i}.taps"], tail(i), step.state_slots, nd)
        h, hm = ops.block_embed(input_ids, P["embed"], P["pos"],
                                step.positions, x, *norm_args(0),
                                *conv_args(0))
        for i, spec in enumerate(c.layers):
            m, f, p = spec.mixer, spec.mlp, f"l{i}."
            if step.prompt is not None:
                ops.conv_prompt(h[nd:], P[p + "taps"], tail(i), step.prompt,
                                hm[nd:])
            w_out = P[p + "out"]
            act = torch.empty((T, w_out.shape[1]), dtype=self.dtype,
                              device=self.device)
            hv = m.heads // self.tp_world * m.vdim
            mixer = self._latent if isinstance(m, LatentSpec) else self._hgrn2
            mixer(i, m, _linear(hm, P[p + "proj"]), kv_cache, step,
                  act[:, :hv])
            if f is not None:
                ops.gate_act(_linear(h, P[p + "gate_up"]), act[:, hv:],
                             "relu")
            y = self._reduce(_linear(act, w_out))
            if i + 1 < c.n_layers:
                h, hm = ops.block_step(x, y, *norm_args(i + 1),
                                       step.positions, *conv_args(i + 1))
            else:
                h, _ = ops.block_step(
                    x, y, P["final.norm"], c.norm_groups, c.rms_eps,
                    step.positions, rows=sample_idx, keep=False)
        return _linear(h, P["embed"])
