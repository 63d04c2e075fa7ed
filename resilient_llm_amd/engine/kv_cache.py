"""Paged KV cache sized for 288 GB of HBM3E per GPU.

Layout [n_layers, num_blocks, n_kv_heads, block_size, head_dim] bf16 for
K and V — each (block, kv-head) row is a contiguous
[block_size, head_dim] tile, which is exactly what one lane-group of the
decode kernel streams (ops/csrc/decode_attn.hip).  Block size 16 tokens.

Allocation is refcounted with PREFIX CACHING: full prompt blocks are
content-addressed (sha1 chain over token ids), so a request whose prompt
shares a cached prefix acquires those blocks instead of recomputing them
— it simply enters the chunked-prefill path at the first uncached token.
Blocks whose refcount drops to zero stay indexed ("cached-free") and are
evicted FIFO only when a fresh allocation needs them.
"""

from __future__ import annotations

import collections
import dataclasses
import hashlib
import struct
from typing import Optional

import torch


class OutOfBlocks(RuntimeError):
    """KV budget exhausted — the worker surfaces this as Throttled (X13)."""


def block_hash_chain(token_ids, block_size: int) -> list[bytes]:
    """Content keys for each FULL block of a prompt: sha1(parent, tokens)."""
    keys = []
    parent = b"root"
    for i in range(len(token_ids) // block_size):
        blk = token_ids[i * block_size:(i + 1) * block_size]
        h = hashlib.sha1(parent + struct.pack(f"<{block_size}i", *blk)).digest()
        keys.append(h)
        parent = h
    return keys


@dataclasses.dataclass(frozen=True)
class KVLayer:
    """What one attention layer caches per token.  ``share`` names an
    earlier layer whose keys and values this layer reads instead."""
    n_kv_heads: int
    k_dim: int
    v_dim: int
    share: Optional[int] = None


@dataclasses.dataclass(frozen=True)
class LatentLayer:
    """What one latent attention layer caches per token: one vector that
    serves all heads as key and value."""
    dim: int


@dataclasses.dataclass(frozen=True)
class StateLayer:
    """What one recurrent layer carries per sequence (f32)."""
    heads: int
    dim: int
    vdim: int


@dataclasses.dataclass(frozen=True)
class ScalarLayer:
    """One number per head that a recurrent layer carries beside its state
    (f32), a running maximum say."""
    heads: int


@dataclasses.dataclass(frozen=True)
class TailLayer:
    """What a short causal convolution carries per sequence: its last
    ``rows`` inputs, a ring by position (activation dtype)."""
    rows: int
    width: int


def layer_parts(spec) -> tuple:
    """A layer may keep one thing or several."""
    return spec if isinstance(spec, tuple) else (spec,)


class RecurrentStates:
    """What live sequences carry from token to token: one slot per live
    sequence, and in each slot a [heads, dim, vdim] f32 state per recurrent
    layer (rows padded to 16 bytes), its scalars if it has any, and the tail
    of each convolution.  A
    slot is not cleared when it changes hands: what a sequence's first rows
    would read is zero by position."""

    def __init__(self, layers: list, n_slots: int, device,
                 dtype: torch.dtype = torch.bfloat16) -> None:
        self.n_slots = n_slots
        self._layers: dict[int, torch.Tensor] = {}
        self._scalars: dict[int, torch.Tensor] = {}
        self._tails: dict[int, torch.Tensor] = {}
        for i, spec in enumerate(layers):
            for s in layer_parts(spec):
                if isinstance(s, StateLayer):
                    self._layers[i] = torch.zeros(
                        (n_slots, s.heads, s.dim, -(-s.vdim // 4) * 4),
                        dtype=torch.float32, device=device)
                elif isinstance(s, ScalarLayer):
                    self._scalars[i] = torch.zeros(
                        (n_slots, s.heads), dtype=torch.float32,
                        device=device)
                elif isinstance(s, TailLayer):
                    self._tails[i] = torch.zeros(
                        (n_slots, s.rows, s.width), dtype=dtype,
                        device=device)
        self._free = list(range(n_slots - 1, -1, -1))

    @staticmethod
    def needed(layers: list) -> bool:
        return any(isinstance(s, (StateLayer, ScalarLayer, TailLayer))
                   for spec in layers for s in layer_parts(spec))

    def layer(self, i: int) -> torch.Tensor:
        return self._layers[i]

    def scalar(self, i: int) -> torch.Tensor:
        return self._scalars[i]

    def tail(self, i: int) -> Optional[torch.Tensor]:
        return self._tails.get(i)

    @property
    def free_slots(self) -> int:
        return len(self._free)

    def allocate(self) -> int:
        if not self._free:
            raise OutOfBlocks(f"all {self.n_slots} state slots are in use")
        return self._free.pop()

    def free(self, slot: int) -> None:
        self._free.append(slot)

    def cast(self, dtype: torch.dtype) -> None:
        self._tails = {i: t.to(dtype) for i, t in self._tails.items()}

    def _kinds(self) -> dict:
        return {"states": self._layers, "scalars": self._scalars,
                "tails": self._tails}

    def export(self, slot: int) -> dict:
        return {kind: {i: t[slot].cpu() for i, t in held.items()}
                for kind, held in self._kinds().items()}

    def import_(self, slot: int, payload: dict) -> None:
        for kind, held in self._kinds().items():
            for i, t in held.items():
                t[slot].copy_(payload[kind][i])

    def bytes_used(self) -> int:
        return sum(t.numel() * t.element_size()
                   for held in self._kinds().values() for t in held.values())


class PagedKVCache:
    states: Optional[RecurrentStates] = None

    def __init__(self, n_layers: int, num_blocks: int, n_kv_heads: int,
                 block_size: int, head_dim: int, device="cpu",
                 dtype: torch.dtype = torch.bfloat16) -> None:
        self.n_layers = n_layers
        self.n_kv_heads = n_kv_heads
        self.head_dim = head_dim
        shape = (n_layers, num_blocks, n_kv_heads, block_size, head_dim)
        self.k = torch.zeros(shape, dtype=dtype, device=device)
        self.v = torch.zeros(shape, dtype=dtype, device=device)
        self._init_blocks(num_blocks, block_size)

    def _init_blocks(self, num_blocks: int, block_size: int) -> None:
        self.num_blocks = num_blocks
        self.block_size = block_size
        self._free: list[int] = list(range(num_blocks - 1, -1, -1))
        self._ref = [0] * num_blocks
        # prefix cache state
        self._index: dict[bytes, int] = {}          # key -> block id
        self._block_key: dict[int, bytes] = {}      # block id -> key
        # evictable, still indexed
        self._cached_free: "collections.OrderedDict[int, None]" = \
            collections.OrderedDict()
        self.prefix_hits = 0
        self.prefix_lookups = 0

    @classmethod
    def for_model(cls, config, num_blocks: int, device="cpu",
                  block_size: int = 16, tp_world: int = 1,
                  kv_dtype: torch.dtype = torch.bfloat16,
                  state_slots: int = 65) -> "PagedKVCache":
        """``state_slots`` matters to models with recurrent layers: the
        most sequences that hold state at a time."""
        if hasattr(config, "cache_layers"):
            return LayeredKVCache(config.cache_layers(tp_world), num_blocks,
                                  block_size, device=device, dtype=kv_dtype,
                                  state_slots=state_slots)
        return cls(config.n_layers, num_blocks,
                   config.n_kv_heads // tp_world, block_size,
                   config.head_dim, device=device, dtype=kv_dtype)

    def layer(self, i: int) -> tuple[torch.Tensor, torch.Tensor]:
        return self.k[i], self.v[i]

    def cast(self, dtype: torch.dtype) -> None:
        self.k = self.k.to(dtype)
        self.v = self.v.to(dtype)

    # ------------------------------------------------ moving live sequences
    def export_blocks(self, blocks: list):
        """Host copies of ``blocks`` (every layer), for import_blocks."""
        idx = torch.tensor(blocks, dtype=torch.long, device=self.k.device)
        return (self.k.index_select(1, idx).to("cpu"),
                self.v.index_select(1, idx).to("cpu"))

    def import_blocks(self, blocks: list, payload) -> None:
        """Write an exported payload into the first of ``blocks``."""
        k_src, v_src = payload
        idx = torch.tensor(blocks[:k_src.shape[1]], dtype=torch.long,
                           device=self.k.device)
        self.k.index_copy_(1, idx, k_src.to(self.k.device, self.k.dtype))
        self.v.index_copy_(1, idx, v_src.to(self.v.device, self.v.dtype))

    @property
    def free_blocks(self) -> int:
        return len(self._free) + len(self._cached_free)

    def _drop_identity(self, b: int) -> None:
        key = self._block_key.pop(b, None)
        if key is not None and self._index.get(key) == b:
            del self._index[key]

    def allocate(self, n: int) -> list[int]:
        if n > self.free_blocks:
            raise OutOfBlocks(f"need {n} KV blocks, have {self.free_blocks}")
        out = []
        for _ in range(n):
            if self._free:
                b = self._free.pop()
            else:
                b, _ = self._cached_free.popitem(last=False)   # FIFO evict
                self._drop_identity(b)
            self._ref[b] = 1
            out.append(b)
        return out

    def free(self, blocks: list[int]) -> None:
        for b in blocks:
            self._ref[b] -= 1
            if self._ref[b] > 0:
                continue
            self._ref[b] = 0
            if b in self._block_key:
                self._cached_free[b] = None     # evictable but reusable
            else:
                self._free.append(b)

    # -------------------------------------------------------- prefix cache
    def lookup_prefix(self, keys: list[bytes]) -> list[int]:
        """Acquire (refcount) the longest cached chain matching ``keys``."""
        out: list[int] = []
        self.prefix_lookups += 1
        for key in keys:
            b = self._index.get(key)
            if b is None:
                break
            self._ref[b] += 1
            if self._ref[b] == 1:
                self._cached_free.pop(b, None)
            out.append(b)
        self.prefix_hits += len(out)
        return out

    def register_block(self, b: int, key: bytes) -> None:
        """Publish a fully-written prompt block under its content key."""
        if key in self._index or b in self._block_key:
            return
        self._index[key] = b
        self._block_key[b] = key

    def bytes_used(self) -> int:
        return self.k.numel() * self.k.element_size() * 2


class LayeredKVCache(PagedKVCache):
    """Paged cache of a model whose layers differ: every attention layer
    has its own [num_blocks, kv heads, block, width] K and V (widths may
    differ, layers may share), a latent attention layer one
    [num_blocks, 1, block, width] tensor, recurrent layers have none, and
    what layers carry per sequence lives in ``states``.  Blocks are
    allocated as in the uniform cache: one block id addresses a token range
    in every layer."""

    def __init__(self, layers: list, num_blocks: int, block_size: int,
                 device="cpu", dtype: torch.dtype = torch.bfloat16,
                 state_slots: int = 65) -> None:
        self.n_layers = len(layers)
        self._init_blocks(num_blocks, block_size)
        self._kv: dict[int, tuple] = {}
        self._own: list[int] = []
        self._share: dict[int, int] = {}

        def pages(heads, width):
            return torch.zeros((num_blocks, heads, block_size, width),
                               dtype=dtype, device=device)
        for i, spec in enumerate(layers):
            for s in layer_parts(spec):
                if isinstance(s, KVLayer) and s.share is not None:
                    self._kv[i] = self._kv[s.share]
                    self._share[i] = s.share
                elif isinstance(s, KVLayer):
                    self._own.append(i)
                    self._kv[i] = (pages(s.n_kv_heads, s.k_dim),
                                   pages(s.n_kv_heads, s.v_dim))
                elif isinstance(s, LatentLayer):
                    self._own.append(i)
                    self._kv[i] = (pages(1, s.dim),)
        if RecurrentStates.needed(layers):
            # tails hold activations, also where the cache is 8-bit
            self.states = RecurrentStates(
                layers, state_slots, device,
                dtype if dtype.itemsize > 1 else torch.bfloat16)

    def layer(self, i: int) -> tuple:
        return self._kv[i]

    def cast(self, dtype: torch.dtype) -> None:
        for i in self._own:
            self._kv[i] = tuple(t.to(dtype) for t in self._kv[i])
        for i, j in self._share.items():
            self._kv[i] = self._kv[j]
        if self.states is not None:
            self.states.cast(dtype)

    def export_blocks(self, blocks: list):
        return [tuple(t[torch.tensor(blocks, device=t.device)].to("cpu")
                      for t in self._kv[i]) for i in self._own]

    def import_blocks(self, blocks: list, payload) -> None:
        for i, own in zip(self._own, payload):
            for dst, src in zip(self._kv[i], own):
                idx = torch.tensor(blocks[:src.shape[0]], dtype=torch.long,
                                   device=dst.device)
                dst.index_copy_(0, idx, src.to(dst.device, dst.dtype))

    def bytes_used(self) -> int:
        return sum(t.numel() * t.element_size()
                   for i in self._own for t in self._kv[i])
