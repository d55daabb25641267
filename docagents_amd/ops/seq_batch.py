"""The batch of one step: portions of sequences packed row after row, each against its own state slot."""
from __future__ import annotations

from dataclasses import dataclass, field, replace

import numpy as np
import torch

from . import h2d

CHUNK = 64  # a recurrence's chunks are multiples of this many tokens
PAGE = 64   # tokens per cache page (csrc/seq.h)


@dataclass
class SeqBatch:
    """Portion b is packed rows ``cu[b] .. cu[b + 1]``: the tokens at positions ``pos0[b]``, ... of the
    sequence in state slot ``slot[b]``; ``seq[t]`` is row t's portion (all int32, on the device)."""
    cu: torch.Tensor
    slot: torch.Tensor
    pos0: torch.Tensor
    seq: torch.Tensor
    T: int                 # packed rows
    B: int                 # portions
    max_len: int           # longest portion
    max_ctx: int           # bound on position + 1 over the batch (sets split counts: a host number)
    singles: bool = True   # a portion of one token may be in the batch
    table: torch.Tensor | None = None  # int32 [slots, pages of a slot]: the cache's page table
    lens: np.ndarray | None = None     # the portions' lengths (host); None: single tokens
    starts: np.ndarray | None = None   # pos0 on the host; what the device decides (decoded tokens) may differ
    _chunks: dict = field(default_factory=dict)  # lists derived from the lengths, made once for all layers

    def on(self, table) -> "SeqBatch":
        return replace(self, table=table)

    def split(self, n: int | None):
        """(portions of fewer than n tokens, the others), each None or (batch, its packed rows on the device: int64).
        The rows are None where all portions are on one side; n None: all are short."""
        if n is None or self.max_len < n:
            return (self, None), None
        if int(self.lens.min()) >= n:
            return None, (self, None)
        if ("split", n) not in self._chunks:
            dev, first = self.cu.device, np.cumsum(self.lens) - self.lens
            ends = self.starts + self.lens

            def side(pick):
                b = np.flatnonzero(pick)
                lens, at = self.lens[b], h2d(b, dev)
                rows = np.concatenate([np.arange(first[i], first[i] + self.lens[i]) for i in b])
                cu = np.zeros(len(b) + 1, dtype=np.int32)
                np.cumsum(lens, out=cu[1:])
                # single tokens' positions may be known to the device only
                ctx = self.max_ctx if lens.min() == 1 else int(ends[b].max())
                return SeqBatch(h2d(cu, dev), self.slot.index_select(0, at), self.pos0.index_select(0, at),
                                h2d(np.repeat(np.arange(len(b), dtype=np.int32), lens), dev), len(rows), len(b),
                                int(lens.max()), ctx, bool((lens == 1).any()), self.table, lens,
                                self.starts[b]), h2d(rows, dev)
            self._chunks["split", n] = side(self.lens < n), side(self.lens >= n)
        (short, srows), (long, lrows) = self._chunks["split", n]
        return (short, srows), (long, lrows)

    def context(self):
        """(int32 [B + 1]: offsets of the portions' whole contexts packed one after another, their sum)."""
        if "context" not in self._chunks:
            cu = np.zeros(self.B + 1, dtype=np.int32)
            np.cumsum(self.starts + self.lens, out=cu[1:])
            self._chunks["context"] = h2d(cu, self.cu.device), int(cu[-1])
        return self._chunks["context"]

    def chunk_len(self, waves: int, fill: int) -> int:
        """Tokens per chunk of a recurrence whose portions take ``waves`` waves each when walked from end to
        end: as long as the chip is filled (``fill`` waves); 0 when the portions alone do that, or are short."""
        if self.max_len <= CHUNK:
            return 0
        want = -(-fill * self.max_len // max(1, waves * self.T))  # chunks of the longest portion
        return 0 if want <= 1 else max(CHUNK, -(-self.max_len // (want * CHUNK)) * CHUNK)

    def chunks(self, n: int):
        """(int32 [chunks, 2]: portion and chunk of it, int32 [B]: chunks of the portions before b, chunks) of
        n tokens each."""
        if n not in self._chunks:
            per = -(-self.lens // n)
            base = np.cumsum(per) - per
            tot = int(per.sum())
            ck = np.stack([np.repeat(np.arange(self.B), per), np.arange(tot) - np.repeat(base, per)], axis=1)
            flat = h2d(np.concatenate([ck.ravel(), base]).astype(np.int32), self.cu.device)
            self._chunks[n] = (flat[:2 * tot].view(tot, 2), flat[2 * tot:], tot)
        return self._chunks[n]


def pack_batch(lens, slots, pos0, device, ids=None):
    """Host lists -> (SeqBatch, token ids on the device or None): one host-to-device copy."""
    lens = np.asarray(lens, dtype=np.int64)
    B, T = len(lens), int(lens.sum())
    if B == 0 or lens.min() < 1:
        raise ValueError("a batch needs portions of at least one token")
    cu = np.zeros(B + 1, dtype=np.int32)
    np.cumsum(lens, out=cu[1:])
    parts = [cu, np.asarray(slots, dtype=np.int32), np.asarray(pos0, dtype=np.int32),
             np.repeat(np.arange(B, dtype=np.int32), lens)]
    if ids is not None:
        parts.append(np.asarray(ids, dtype=np.int32))
    flat = h2d(np.concatenate(parts), device)
    out, at = [], 0
    for p in parts:
        out.append(flat[at:at + len(p)])
        at += len(p)
    m = SeqBatch(out[0], out[1], out[2], out[3], T, B, int(lens.max()), int((lens + parts[2]).max()),
                 bool((lens == 1).any()), lens=lens,
                 starts=np.asarray(pos0, dtype=np.int64))
    return m, (out[-1] if ids is not None else None)
