"""Prompt rows of one engine step, as the tiled kernels want them.

A step's prompt part is a list of portions (one per sequence): ``n`` rows
that start at batch row ``row0`` (counted from the first prompt row) and
at position ``pos0``.  Kernels that work in tiles of some height get a
table of tiles; different layers may use different heights, so the tables
are made on demand and kept for the step.
"""

from __future__ import annotations

import dataclasses

import torch


@dataclasses.dataclass(frozen=True)
class Portion:
    row0: int
    pos0: int
    n: int
    seq: int               # row of the step's prompt block tables
    slot: int = 0          # recurrent-state slot of the sequence


class PromptRows:
    def __init__(self, portions: list, device) -> None:
        self.portions = portions
        self.device = device
        self._made: dict[tuple, object] = {}

    def _once(self, key: tuple, make):
        if key not in self._made:
            self._made[key] = make()
        return self._made[key]

    def _table(self, rows: list) -> torch.Tensor:
        """Columns of ``rows`` as the rows of one int32 tensor."""
        return torch.tensor(rows, dtype=torch.int32).t().contiguous() \
            .to(self.device)

    def tiles(self, height: int) -> torch.Tensor:
        """int32 [4, n]: first row, its position, rows, sequence."""
        return self._once(("tiles", height), lambda: self._table(
            [(p.row0 + o, p.pos0 + o, min(height, p.n - o), p.seq)
             for p in self.portions for o in range(0, p.n, height)]))

    def seqs(self, height: int) -> torch.Tensor:
        """int32 [4, n]: first tile, tiles, first position, state slot."""
        def make():
            rows, first = [], 0
            for p in self.portions:
                k = -(-p.n // height)
                rows.append((first, k, p.pos0, p.slot))
                first += k
            return self._table(rows)
        return self._once(("seqs", height), make)

    def spans(self, height: int) -> torch.Tensor:
        """int32 [5, n]: first row, its position, rows, offset in the
        portion, state slot."""
        return self._once(("spans", height), lambda: self._table(
            [(p.row0 + o, p.pos0 + o, min(height, p.n - o), o, p.slot)
             for p in self.portions for o in range(0, p.n, height)]))

    def vectors(self, height: int, per_row: int) -> torch.Tensor:
        """int32 [4, n] over ``per_row`` vectors a row (its heads): first
        vector, offset in the portion, vectors, sequence."""
        return self._once(("vectors", height, per_row), lambda: self._table(
            [(p.row0 * per_row + o, o, min(height, p.n * per_row - o), p.seq)
             for p in self.portions
             for o in range(0, p.n * per_row, height)]))

    def pos0(self) -> torch.Tensor:
        """int32 [sequences]: first position of each one's portion."""
        def make():
            pos = [0] * (1 + max(p.seq for p in self.portions))
            for p in self.portions:
                pos[p.seq] = p.pos0
            return torch.tensor(pos, dtype=torch.int32).to(self.device)
        return self._once(("pos0",), make)

    def gathered(self, height: int, chunk: int = 0) -> tuple:
        """Every portion's sequence up to its last row, one after another,
        each padded to a multiple of ``height`` tokens: (int32 [4, n]
        blocks of that height: sequence, first token, tokens, output row;
        int32 [sequences] output row of position 0; output rows).  With
        ``chunk`` a sequence starts with the chunk of its first row (at a
        multiple of ``height``), so that row may be negative."""
        def make():
            rows, at = [], 0
            off = [0] * (1 + max(p.seq for p in self.portions))
            for p in self.portions:
                ctx = p.pos0 + p.n
                start = p.pos0 // chunk * chunk // height * height \
                    if chunk else 0
                off[p.seq] = at - start
                rows += [(p.seq, o, min(height, ctx - o), at - start + o)
                         for o in range(start, ctx, height)]
                at += -(-(ctx - start) // height) * height
            return (self._table(rows),
                    torch.tensor(off, dtype=torch.int32).to(self.device), at)
        return self._once(("gathered", height, chunk), make)
