"""Replay of a recorded request trace through a decoder's step: given token ids in, logits out, nothing sampled.

Steps are JSON objects, one a line: ``{"step": n, "entries": [{"id", "tokens", "want"}, ...], "end": [ids]}``.
A step is one batch: every entry brings its sequence's next tokens (a part of a prompt, or one decoded
token), run from the state earlier steps left; ``want`` lists the places among them whose logits are
written to ``<out>/<n>.f32`` (little-endian fp32, [wanted, vocab], in entry order). A sequence gets a slot of
the state cache at its first entry and its pages as it grows; ``end`` gives both back.
"""
from __future__ import annotations

import json
import os

import numpy as np
import torch

from ..ops import h2d
from ..ops.seq_batch import PAGE, pack_batch


class TraceReplay:
    SLOTS = 4  # live sequences

    def __init__(self, model, max_tokens: int):
        self.model = model
        tokens = -(-max_tokens // PAGE) * PAGE
        self.cache = model.alloc_cache(self.SLOTS, tokens, tokens=tokens)
        self.live: dict[str, list[int]] = {}  # id -> [slot, tokens so far]

    def step(self, entries, end=()) -> torch.Tensor | None:
        """Run one step's entries as one batch; logits fp32 [wanted, vocab] on the host, None if none are."""
        out = None
        if entries:
            lens, slots, pos0, ids, rows = [], [], [], [], []
            for e in entries:
                toks = e["tokens"]
                if not toks or min(toks) < 0 or max(toks) >= self.model.cfg.vocab:
                    raise ValueError(f"request {e['id']!r}: needs tokens within the vocabulary")
                if any(not 0 <= w < len(toks) for w in e["want"]):
                    raise ValueError(f"request {e['id']!r}: wants places outside its tokens")
                if e["id"] not in self.live:
                    self.live[e["id"]] = [self.cache.acquire(1, [0])[0], 0]
                slot, n = self.live[e["id"]]
                if slot in slots:
                    raise ValueError(f"request {e['id']!r} appears twice in a step")
                self.cache.extend([slot], [n + len(toks)])
                rows += [len(ids) + w for w in e["want"]]
                lens.append(len(toks)); slots.append(slot); pos0.append(n)
                ids += toks
                self.live[e["id"]][1] = n + len(toks)
            dev = self.model.device
            m, tok = pack_batch(lens, slots, pos0, dev, ids)
            logits = self.model.step(m, tok, h2d(np.asarray(rows, dtype=np.int64), dev) if rows else None)
            if logits is not None:
                out = logits.float().cpu()
        for i in end:
            self.cache.release([self.live.pop(i)[0]])
        return out


def replay(model, max_tokens: int, lines, out_dir: str, done) -> None:
    """Every step of ``lines``; ``done(step)`` after each, once its file is written."""
    r = TraceReplay(model, max_tokens)
    for line in lines:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = r.step(s["entries"], s.get("end", ()))
        if logits is not None:
            tmp = os.path.join(out_dir, f".{s['step']}.tmp")
            np.ascontiguousarray(logits.numpy(), dtype="<f4").tofile(tmp)
            os.replace(tmp, os.path.join(out_dir, f"{s['step']}.f32"))
        if model.device.type == "cuda":
            torch.cuda.synchronize(model.device)
        done(s["step"])
