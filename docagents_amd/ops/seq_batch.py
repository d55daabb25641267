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
    _chunks: dict = field(default_factory=dict)

    def on(self, table) -> "SeqBatch":
        return replace(self, table=table)

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
                 bool((lens == 1).any()), lens=lens)
    return m, (out[-1] if ids is not None else None)
