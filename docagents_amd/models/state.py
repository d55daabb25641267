"""Per-sequence state of decoders that keep more than a KV cache: a pool of 64-token pages for what grows
with a sequence and fixed-size slots for what does not.

A layer declares what it keeps (``LayerState``): slot tensors (recurrent states, convolution inputs, the
token shift's previous row) are allocated [slots, ...], page tensors (keys, latents) [pages, ...]. A sequence owns one
slot and as many pages as its tokens need; ``table[slot, i]`` is the page of its tokens 64 i .. 64 i + 63,
shared by every layer. Nothing is cleared when a slot or page changes hands: the kernels start a sequence's
state at position 0 themselves, and read no key beyond a sequence's own tokens.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np
import torch

from ..ops import h2d
from ..ops.seq_batch import PAGE


@dataclass(frozen=True)
class RotaryTable:
    """cos and sin of position * base^(-2 i / dims), i < dims / 2, for every position a sequence can reach: fp32
    [positions, dims / 2, 2], from angles in double precision."""
    dims: int
    base: float

    def bytes(self, positions: int) -> int:
        return positions * self.dims * 4

    def build(self, positions: int, device) -> torch.Tensor:
        f = self.base ** (-2.0 * torch.arange(self.dims // 2, dtype=torch.float64) / self.dims)
        a = torch.arange(positions, dtype=torch.float64)[:, None] * f
        return torch.stack([a.cos(), a.sin()], -1).float().to(device)


@dataclass(frozen=True)
class LayerState:
    """Shapes (without the leading slot / page dimension) and dtypes by name; tables over positions by name, each
    built once for all layers that name an equal one."""
    slot: dict = field(default_factory=dict)
    page: dict = field(default_factory=dict)
    tables: dict = field(default_factory=dict)

    @staticmethod
    def _bytes(spec: dict) -> int:
        return sum(int(np.prod(shape)) * torch.empty((), dtype=dt).element_size() for shape, dt in spec.values())

    def bytes(self, slots: int, pages: int) -> int:
        return slots * self._bytes(self.slot) + pages * self._bytes(self.page)


def pages_for(tokens: int) -> int:
    return -(-tokens // PAGE)


class StateCache:
    """``slots`` sequences of at most ``max_seq`` tokens each, ``tokens`` tokens of pages in all (default:
    enough for every slot to reach max_seq)."""

    def __init__(self, layers: list[LayerState], slots: int, max_seq: int, device, tokens: int | None = None):
        self.slots, self.max_seq, self.device = slots, max_seq, torch.device(device)
        self.row_pages = pages_for(max_seq)
        self.pages = pages_for(tokens) if tokens else slots * self.row_pages
        make = lambda spec, n: {k: torch.zeros((n, *shape), dtype=dt, device=self.device)  # noqa: E731
                                for k, (shape, dt) in spec.items()}
        self.tables = {t: t.build(self.row_pages * PAGE, self.device) for s in layers for t in s.tables.values()}
        self.layers = [{**make(s.slot, slots), **make(s.page, self.pages), **{k: self.tables[t] for k, t in s.tables.items()}}
                       for s in layers]
        self.table = torch.zeros((slots, self.row_pages), dtype=torch.int32, device=self.device)
        self.free = list(range(slots - 1, -1, -1))
        self.free_pages = list(range(self.pages - 1, -1, -1))
        self.owned: dict[int, list[int]] = {}

    @staticmethod
    def bytes_for(layers: list[LayerState], slots: int, max_seq: int, tokens: int | None = None) -> int:
        pages = pages_for(tokens) if tokens else slots * pages_for(max_seq)
        tables = {t for s in layers for t in s.tables.values()}
        return sum(s.bytes(slots, pages) for s in layers) + sum(t.bytes(pages_for(max_seq) * PAGE) for t in tables)

    # ------------------------------------------------------------------ ownership
    def fits(self, tokens: list[int]) -> bool:
        """Whether sequences of these lengths can be admitted together now."""
        return len(tokens) <= len(self.free) and sum(pages_for(t) for t in tokens) <= len(self.free_pages)

    def capacity(self) -> int:
        """The longest sequence the whole pool could hold."""
        return min(self.max_seq, self.pages * PAGE)

    def acquire(self, n: int, tokens: list[int] | None = None) -> list[int]:
        """n slots, with the pages of ``tokens[i]`` tokens each (default: of max_seq)."""
        tokens = [self.max_seq] * n if tokens is None else list(tokens)
        if not self.fits(tokens):
            raise RuntimeError(f"state cache exhausted: want {n} slots and {sum(pages_for(t) for t in tokens)} pages, "
                               f"{len(self.free)} slots and {len(self.free_pages)} pages free")
        ids = [self.free.pop() for _ in range(n)]
        for i in ids:
            self.owned[i] = []
        self.extend(ids, tokens)
        return ids

    def extend(self, ids, tokens) -> None:
        """Pages for ``tokens[i]`` tokens in all for slot ``ids[i]`` (never fewer than it has)."""
        grown, rows = [], []
        for i, t in zip(ids, tokens):
            have = self.owned[i]
            need = pages_for(t) - len(have)
            if need <= 0:
                continue
            if t > self.max_seq:
                raise ValueError(f"{t} tokens exceed the context ({self.max_seq})")
            if need > len(self.free_pages):
                raise RuntimeError(f"state cache exhausted: want {need} pages, {len(self.free_pages)} free")
            have.extend(self.free_pages.pop() for _ in range(need))
            row = np.zeros(self.row_pages, dtype=np.int32)
            row[:len(have)] = have
            grown.append(i)
            rows.append(row)
        if grown:
            idx = h2d(np.asarray(grown, dtype=np.int64), self.device)
            self.table.index_copy_(0, idx, h2d(np.stack(rows), self.device))

    def release(self, ids) -> None:
        for i in ids:
            self.free_pages.extend(reversed(self.owned.pop(i)))
            self.free.append(i)
