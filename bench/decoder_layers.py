"""Prefill and decode throughput of decoders at full layer width (random weights), side by side: the workload of
``bench.py --decoders``. Prefill: one packed batch of prompts through ``prefill`` (all layers, last-token
logits). Decode: the captured decode step of B rows at a given context, sampler included."""
from __future__ import annotations

import os
import sys

import numpy as np
import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from docagents_amd.engine.generator import Generator  # noqa: E402
from docagents_amd.models import make_decoder  # noqa: E402
from docagents_amd.models.configs import decoder_config  # noqa: E402
from docagents_amd.ops import h2d  # noqa: E402


def _timed(fn, reps: int, warmup: int) -> float:
    """Mean ms of fn() on the device."""
    for _ in range(warmup):
        fn()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    torch.cuda.synchronize()
    a.record()
    for _ in range(reps):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / reps


def run(arch: str, prefills, decodes, context: int, steps: int, warmup: int, seed: int = 0) -> dict:
    """prefills: (prompts, tokens each); decodes: batch sizes."""
    cfg = decoder_config(arch)
    model = make_decoder(cfg, "cuda", seed=seed)
    B = max(max(decodes), max(n for n, _ in prefills))
    gen = Generator(model, max_batch=B, max_seq=max(context + 512, max(t for _, t in prefills)), temperature=0.0, seed=seed,
                    share_prefix=False)
    rng = np.random.default_rng(seed)
    out = {"model": arch, "params_g": round(cfg.param_count() / 1e9, 2), "prefill": [], "decode": []}
    dev = model.device

    def prefill_args(slots, n):
        lens = np.full(len(slots), n)
        cu = np.zeros(len(slots) + 1, dtype=np.int32)
        np.cumsum(lens, out=cu[1:])
        ids = rng.integers(0, cfg.vocab, int(cu[-1])).astype(np.int32)
        pos = np.tile(np.arange(n, dtype=np.int32), len(slots))
        args = [h2d(x, dev) for x in (ids, pos, np.repeat(np.asarray(slots, dtype=np.int32), n), cu)]
        return (*args, n, h2d((cu[1:] - 1).astype(np.int64), dev)), dict(local_logits=True, lens=lens.tolist())
    for n, t in prefills:
        slots = gen.cache.acquire(n, [t] * n)
        args, kw = prefill_args(slots, t)
        ms = _timed(lambda: model.prefill(*args, **kw), steps, warmup)
        gen.cache.release(slots)
        out["prefill"].append({"prompts": n, "tokens": t, "ms": round(ms, 3), "tokens_per_s": round(n * t / ms * 1e3)})
    for b in decodes:
        slots = gen.cache.acquire(b, [context + 512] * b)
        for s in range(0, b, 8):  # contexts that hold real keys and states
            args, kw = prefill_args(slots[s:s + 8], context)
            model.prefill(*args, **kw)
        st = gen._state(b, 480, lane=b)
        st.slot.copy_(torch.tensor(slots, dtype=torch.int32))
        st.pos.fill_(context)
        st.lens.fill_(context + 1)
        st.start.fill_(context)
        st.active.fill_(1)
        gen._capture(st)
        ms = _timed(st.graph.replay, min(16 * steps, 400), 8)
        gen.cache.release(slots)
        out["decode"].append({"rows": b, "context": context, "ms": round(ms, 4), "tokens_per_s": round(b / ms * 1e3)})
    gen.close()
    model.cache = None
    return out
