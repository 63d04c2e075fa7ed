"""What models share whose layers differ (a list of layers in config.json,
checkpoints under plain 'l<i>.' names): layer specifications, reading a
checkpoint directory, random initialisation, the decode and mixed-batch
entry points.

A model of this kind is a flat parameter store and an explicit forward over
the serving ops, like models/llama.py; it keeps no cache and runs no loop
of its own.
"""

from __future__ import annotations

import dataclasses
import json
import os
from typing import Optional

import torch


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    ff: int


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: object
    mlp: object                      # None: no feed-forward


class MixedConfig:
    """Mixed into configurations with ``layers``, ``from_dict`` and
    ``cache_layers``."""

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dir(cls, path: str, **kw):
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f), name=os.path.basename(
                os.path.normpath(path)), **kw)

    def fit_positions(self, n: int) -> None:
        """Serve sequences of up to ``n`` tokens, where nothing in the
        model limits them."""
        self.max_position = n


@dataclasses.dataclass
class Step:
    """What a step's mixers need besides their input rows."""
    positions: torch.Tensor
    slots: torch.Tensor              # cache slot of every row
    n_decode: int
    tables_dec: Optional[torch.Tensor]
    state_slots: Optional[torch.Tensor]
    tables_pre: Optional[torch.Tensor] = None
    prompt: object = None            # PromptRows


class MixedModel:
    # the engine hands prompt rows and state slots to such a model
    mixed_layers = True

    def __init__(self, config, device: str = "cpu",
                 dtype: torch.dtype = torch.bfloat16,
                 tp_rank: int = 0, tp_world: int = 1,
                 tp_group=None, seed: int = 0,
                 quant: Optional[str] = None,
                 weights: Optional[str] = None) -> None:
        if quant is not None:
            raise ValueError("quant is not available for this model")
        self.config = config
        self.device = torch.device(device)
        self.dtype = dtype
        self.quant = None
        self.tp_rank, self.tp_world, self.tp_group = tp_rank, tp_world, tp_group
        assert all(s % tp_world == 0 for s in self.sharded_sizes()), \
            f"TP={tp_world} must divide heads and feed-forward widths"
        self.params: dict[str, torch.Tensor] = {}
        self._prepare()
        if weights is not None:
            self.load_safetensors(weights)
        else:
            self._init_weights(seed)

    # ----------------------------------------------- what a model provides
    def sharded_sizes(self) -> list:
        """Sizes that tensor parallelism divides."""
        raise NotImplementedError

    def tensor_shapes(self) -> dict:
        """Checkpoint names -> shapes (full, unsharded)."""
        raise NotImplementedError

    def initial(self, leaf: str, shape: tuple) -> Optional[torch.Tensor]:
        """Random initialisation's value of tensors that are not drawn."""
        return None

    def _install(self, get) -> None:
        """Pack full checkpoint tensors ``get(name)`` into this rank's
        parameters."""
        raise NotImplementedError

    def _prepare(self) -> None:
        """Tables that do not come from a checkpoint."""

    # ------------------------------------------------------------ weights
    def _init_weights(self, seed: int) -> None:
        """Every rank draws the full tensors from one seed and keeps its
        shard, so TP=N computes the same function as TP=1."""
        gen = torch.Generator(device=self.device)
        shapes = self.tensor_shapes()
        std_o = 0.02 / (2 * max(1, self.config.n_layers)) ** 0.5
        order = {n: k for k, n in enumerate(shapes)}

        def draw(name):
            leaf = name.split(".", 1)[-1]
            t = self.initial(leaf, shapes[name])
            if t is not None:
                return t.to(self.device)
            gen.manual_seed(seed * 1000003 + order[name] * 1009 + 1)
            t = torch.empty(shapes[name], dtype=self.dtype,
                            device=self.device)
            return t.normal_(0.0, std_o if leaf.endswith((".o", ".down"))
                             else 0.02, generator=gen)
        self._install(draw)

    def load_safetensors(self, path: str) -> int:
        """Load a checkpoint directory, TP-sharded; returns the number of
        tensors consumed."""
        from safetensors import safe_open
        files = sorted(f for f in os.listdir(path)
                       if f.endswith(".safetensors"))
        if not files:
            raise FileNotFoundError(f"no .safetensors files under {path}")
        where = {}
        for f in files:
            h = safe_open(os.path.join(path, f), framework="pt")
            for k in h.keys():
                where[k] = h
        loaded: list[str] = []
        shapes = self._checkpoint_shapes(
            lambda n: tuple(where[n].get_slice(n).get_shape()), where)

        def take(name):
            if name not in where:
                raise KeyError(f"{path}: tensor {name!r} is missing")
            t = where[name].get_tensor(name)
            if tuple(t.shape) != tuple(shapes[name]):
                raise ValueError(f"{path}: {name} is {tuple(t.shape)}, "
                                 f"the configuration says "
                                 f"{tuple(shapes[name])}")
            loaded.append(name)
            return t
        self._install(take)
        return len(loaded)

    def _checkpoint_shapes(self, shape_of, names) -> dict:
        """tensor_shapes() for a checkpoint; ``shape_of(name)`` looks into
        it for sizes that only a tensor's shape gives."""
        return self.tensor_shapes()

    def _shard(self, t: torch.Tensor, dim: int) -> torch.Tensor:
        k = t.shape[dim] // self.tp_world
        return t.narrow(dim, self.tp_rank * k, k)

    def _mat(self, t: torch.Tensor, rows: bool = False,
             cols: bool = False) -> torch.Tensor:
        if rows:
            t = self._shard(t, 0)
        if cols:
            t = self._shard(t, 1)
        return t.to(self.device).to(self.dtype).contiguous()

    def _vec(self, t: torch.Tensor, rows: bool = False) -> torch.Tensor:
        if rows:
            t = self._shard(t, 0)
        return t.to(self.device).float().contiguous()

    def param_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.params.values())

    # ------------------------------------------------------------ compute
    def _forward(self, input_ids, kv_cache, step: Step, sample_idx):
        """Logits of ``sample_idx`` rows (None: all) of one step."""
        raise NotImplementedError

    def _reduce(self, *ys: torch.Tensor):
        """Sums of row-parallel products over the ranks."""
        if self.tp_world > 1:
            import torch.distributed as dist
            for y in ys:
                dist.all_reduce(y, group=self.tp_group)
        return ys if len(ys) > 1 else ys[0]

    def forward_decode(self, input_ids, positions, kv_cache, slot_mapping,
                       block_tables, seq_lens, state_slots=None):
        """One token per sequence; returns [batch, vocab] logits."""
        return self._forward(
            input_ids, kv_cache, Step(
                positions, slot_mapping, input_ids.shape[0], block_tables,
                state_slots), None)

    def forward_mixed(self, input_ids, positions, kv_cache, slot_mapping,
                      n_decode: int, block_tables_dec, seq_lens_dec,
                      block_tables_pre, prompt, sample_idx,
                      state_slots=None):
        """Rows [0, n_decode) decode one token per sequence, the rest are
        the portions of ``prompt`` (engine/batch.py).  Returns the logits
        of ``sample_idx`` rows."""
        return self._forward(
            input_ids, kv_cache, Step(
                positions, slot_mapping, n_decode, block_tables_dec,
                state_slots, block_tables_pre, prompt), sample_idx)
