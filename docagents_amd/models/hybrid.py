"""Decoders that mix sequence mixers layer by layer, on the gfx950 kernels (Binupel, Zamitar).

Residual stream x in fp32. Per layer run, in a "postnorm" block (with alpha, the norm weights and the shift mu of the
configuration):

    h  = x + (x_previous - x) mu                token shift (x_previous: the previous token's row, state)
    x  = RMSNorm(alpha x + mixer(h)) w1
    x  = RMSNorm(alpha x + down(relu(gate x) * up x)) w2        where the layer has a feed-forward

and in a "parallel" block (learned column scales s1, s2; layers of the loop begin a pass by adding its vector and,
from the second pass on, the embedding output):

    h  = LayerNorm(x) w
    x  = x + s1 mixer(h) + s2 (down(silu(gate h + b) * (up h + b)) + b)

The sums of a line, the norm that follows them, the shift and the saving of its state are one launch
(``stream_step``, ``stream_add``). The mixers are in ``mixers``.

A step (``step``) runs any batch of portions of sequences (``SeqBatch``): whole prompts, parts of prompts and
single tokens side by side, each from the state its slot holds. Prefill and the graph-captured decode step
are that same step. ``dtype`` "fp32" runs everything in true fp32.
"""
from __future__ import annotations

import math

import torch

from ..ops import get_ops
from ..ops.reference import interleave_gate_up
from ..ops.seq_batch import PAGE, SeqBatch, pack_batch
from .configs import (ChannelDelta, GatedRecurrence, HybridConfig, LatentAttention, SelectiveScan, SigmoidAttention)
from .mixers import (MIXERS, AttentionMixer, DeltaMixer, LatentMixer, Linear, RecurrenceMixer, _pad, _up)
from .state import LayerState, StateCache

DTYPES = {"bf16": torch.bfloat16, "fp32": torch.float32}


def tensor_shapes(cfg: HybridConfig) -> dict[str, tuple]:
    """Name -> shape of every tensor of a checkpoint of this configuration."""
    h, parallel = cfg.hidden, cfg.block == "parallel"
    out = {"embed": (cfg.vocab, h)}
    if cfg.loop:
        out["loop.step"] = (cfg.loop.times, h)
    for i, s in enumerate(cfg.spec):
        if s.weights_of is not None:
            continue
        p = f"l{i}."
        out.update({p + "norm1": (h,), p + ("ls1" if parallel else "shift"): (h,)})
        out.update({f"{p}mix.{k}": v for k, v in MIXERS[type(s.mixer)].tensors(s.mixer, h).items()})
        if s.ff:
            out.update({p + ("ls2" if parallel else "norm2"): (h,), p + "mlp.gate": (s.ff, h), p + "mlp.up": (s.ff, h),
                        p + "mlp.down": (h, s.ff)})
            if parallel:
                out.update({p + "mlp.gate.b": (s.ff,), p + "mlp.up.b": (s.ff,), p + "mlp.down.b": (h,)})
    out["final.norm"] = (h,)
    if not parallel:
        out["head"] = (cfg.vocab, h)
    return out


def random_weights(cfg: HybridConfig, device="cpu", seed: int = 0) -> dict[str, torch.Tensor]:
    """Seeded random bf16 tensors that keep activations, decays and step sizes in their working ranges."""
    dev = torch.device(device)
    gen = torch.Generator(device=dev)
    gen.manual_seed(seed * 1_000_003 + 17)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        key = name.rsplit(".", 1)[-1] if not name.endswith((".b", ".norm")) else ".".join(name.split(".")[-2:])
        t = torch.empty(shape, dtype=torch.float32, device=dev)
        if key in ("norm1", "norm2", "final.norm", "q.norm", "k.norm", "D", "mix.norm", "dq.norm", "dkv.norm"):
            t.normal_(1.0, 0.1, generator=gen)
        elif key == "shift":
            t.uniform_(0.0, 0.6, generator=gen)
        elif key == "lam":
            t.uniform_(-5.0, -1.0, generator=gen)
        elif key == "A_log":
            t.uniform_(0.0, math.log(16.0), generator=gen)
        elif key in ("dt.b", "dt_bias"):
            t.uniform_(-5.0, -2.0, generator=gen)
        elif key in ("ls1", "ls2"):
            t.normal_(0.3, 0.05, generator=gen)
        elif key == "pb":
            t.normal_(-3.0, 0.5, generator=gen)
        elif key == "conv":
            t.normal_(0.0, shape[-1] ** -0.5, generator=gen)
        elif len(shape) > 1 and not key.endswith(".b"):
            t.normal_(0.0, shape[-1] ** -0.5, generator=gen)
        else:
            t.normal_(0.0, 0.1, generator=gen)
        out[name] = t.to(torch.bfloat16)
    return out


def layer_states(cfg: HybridConfig, act=torch.bfloat16) -> list[LayerState]:
    """What every layer run keeps per sequence: its mixer's state and, in postnorm blocks, the token shift's
    previous row."""
    per = [MIXERS[type(s.mixer)].state(s.mixer, act) for s in (cfg.spec[r.layer] for r in cfg.runs)]
    if cfg.block == "parallel":
        return per
    shift = {"shift": ((_up(cfg.hidden),), torch.float32)}
    return [LayerState({**p.slot, **shift}, p.page, p.tables) for p in per]


def cache_bytes(cfg: HybridConfig, slots: int, max_seq: int, act=torch.bfloat16) -> int:
    return StateCache.bytes_for(layer_states(cfg, act), slots, min(max_seq, cfg.max_pos))


def decode_workspace_bytes(cfg: HybridConfig, max_batch: int) -> int:
    """Split-K partials of the decode-sized products: up to 8 splits of the widest, or 256 tiles of 64 x 128."""
    widest = max(max(v[0] for v in tensor_shapes(cfg).values()), 2 * max(s.ff for s in cfg.spec))
    return max(64 << 20, 8 * max_batch * _up(widest) * 4)


def prefill_bytes_per_token(cfg: HybridConfig) -> int:
    """Activations of the widest layer while it runs: stream (fp32, two of it), its input and output, and the
    mixer's or the feed-forward's intermediates."""
    def mixer(m):
        if isinstance(m, GatedRecurrence):
            return RecurrenceMixer.padded(m)[1] * (2 * 2 + 2 + 2 * 4 + 2)
        if isinstance(m, SelectiveScan):
            return _up(m.inner) * (2 * 2 + 2 + 4 + 2) + 2 * _up(m.dt_rank + 2 * m.state)
        if isinstance(m, ChannelDelta):
            K, V = DeltaMixer.padded(m)
            return 2 * 2 * (2 * m.kv_heads * K + m.heads * V) + m.heads * (4 * K + 3 * 2 * V)
        if isinstance(m, LatentAttention):
            Q, L, R, D, V = LatentMixer.padded(m)
            return 2 * (2 * Q + 2 * (L + R) + m.heads * (2 * D + 3 * V))
        return AttentionMixer.padded(m) * 2 * (2 * m.heads + m.kv_heads)
    return 12 * _up(cfg.hidden) + max(mixer(s.mixer) + 2 * _up(s.ff) if cfg.block == "parallel" else
                                    max(mixer(s.mixer), 2 * _up(s.ff)) for s in cfg.spec)


class _Layer:
    """One layer's packed weights (shared by the runs that use them)."""

    def __init__(self, ops, cfg: HybridConfig, i: int, raw: dict, hp: int, act):
        s, pre = cfg.spec[i], f"l{i}."
        self.parallel = cfg.block == "parallel"
        mix = {k[len(pre) + 4:]: v for k, v in raw.items() if k.startswith(pre + "mix.")}
        self.mixer = MIXERS[type(s.mixer)](ops, s.mixer, mix, hp, cfg.eps, act)

        def vec(name):
            return _pad(raw[pre + name], hp).float()
        self.norm1 = vec("norm1")
        self.shift, self.scale1 = (None, vec("ls1")) if self.parallel else (vec("shift"), None)
        self.norm2 = self.scale2 = self.down_bias = self.gate_up = self.down = None
        if s.ff:
            f, bias = _up(s.ff), None
            if self.parallel:
                bias = interleave_gate_up(*(_pad(raw[pre + f"mlp.{k}.b"], f)[:, None] for k in ("gate", "up")))[:, 0]
                self.scale2, self.down_bias = vec("ls2"), vec("mlp.down.b")
            else:
                self.norm2 = vec("norm2")
            w = interleave_gate_up(_pad(raw[pre + "mlp.gate"], f, hp), _pad(raw[pre + "mlp.up"], f, hp))
            self.gate_up = Linear(ops, w, act, bias, gated="silu" if self.parallel else "relu")
            self.down = Linear(ops, _pad(raw[pre + "mlp.down"], hp, f), act)


class HybridDecoder:
    prefix_sharing = False  # a prompt head's recurrent state is not shared between sequences
    portion_steps = 8192    # a step runs any portions; prompts are cut at this many tokens by default
    stateful_step = True    # running a step twice advances a sequence twice (graph warm-up uses a spare slot)
    layer_hook = None       # prefill: called with the layer index before each layer (stream steering)

    def __init__(self, cfg: HybridConfig, device="cuda", seed: int = 0, tp=None, weights: dict | None = None,
                 dtype: str = "bf16"):
        from .llama import TPContext
        self.cfg = cfg
        self.device = torch.device(device)
        self.ops = get_ops(self.device)
        self.tp = tp or TPContext()
        if self.tp.size != 1:
            raise ValueError(f"{cfg.name}: tensor parallelism is not supported for decoders of mixed layers "
                             f"(TP={self.tp.size})")
        self.act = act = DTYPES[dtype]
        if weights is None:
            if cfg.path:
                from .checkpoint import load_weights
                weights = load_weights(cfg.path, self.device)
            else:
                weights = random_weights(cfg, self.device, seed)
        self._check(weights)
        raw = {k: v.to(self.device) for k, v in weights.items()}
        self.hp = hp = _up(cfg.hidden)
        own = {i: _Layer(self.ops, cfg, i, raw, hp, act) for i, s in enumerate(cfg.spec) if s.weights_of is None}
        self.layers = [own[r.weights] for r in cfg.runs]
        self.final_norm = _pad(raw["final.norm"], hp).float()
        self.pass_vec = _pad(raw["loop.step"], -1, hp).float() if cfg.loop else None
        if cfg.block == "parallel":
            self.head = Linear(self.ops, _pad(raw["embed"], _up(cfg.vocab), hp), act)
            self.embed = self.head.w[:cfg.vocab]
        else:
            self.embed = _pad(raw["embed"], -1, hp).to(act).contiguous()
            self.head = Linear(self.ops, _pad(raw["head"], _up(cfg.vocab), hp), act)
        self.cache: StateCache | None = None

    def _check(self, weights: dict) -> None:
        want = tensor_shapes(self.cfg)
        bad = [f"{k}: {tuple(weights[k].shape)}, want {v}" for k, v in want.items()
               if k in weights and tuple(weights[k].shape) != tuple(v)]
        missing = [k for k in want if k not in weights]
        if missing or bad:
            raise ValueError(f"{self.cfg.name}: missing tensors {missing[:4]}, wrong shapes {bad[:4]}")

    # ------------------------------------------------------------- state
    def alloc_cache(self, slots: int, max_seq: int, tokens: int | None = None) -> StateCache:
        self.cache = StateCache(layer_states(self.cfg, self.act), slots, min(max_seq, self.cfg.max_pos), self.device,
                                tokens)
        return self.cache

    def cache_bytes(self, slots: int, max_seq: int) -> int:
        return cache_bytes(self.cfg, slots, max_seq, self.act)

    def workspace_bytes(self, max_batch: int, max_seq: int) -> int:
        return decode_workspace_bytes(self.cfg, max_batch)

    # ------------------------------------------------------------- step
    def _forward(self, m: SeqBatch, ids) -> torch.Tensor:
        """The residual stream after the last layer [T, Dp] of a batch; updates pages and state."""
        m = m.on(self.cache.table)
        return self._parallel_blocks(m, ids) if self.cfg.block == "parallel" else self._postnorm_blocks(m, ids)

    def _postnorm_blocks(self, m: SeqBatch, ids) -> torch.Tensor:
        c, o, st, layers = self.cfg, self.ops, self.cache.layers, self.layers
        kw = dict(eps=c.eps, alpha=c.alpha, act=self.act)
        shift = [dict(mu=L.shift, prev=s["shift"]) for L, s in zip(layers, st)] + [dict(want_h=False)]
        x, h = o.stream_step(m, c.hidden, ids=ids, table=self.embed, act=self.act, **shift[0])
        for i, L in enumerate(layers):
            if self.layer_hook is not None:
                self.layer_hook(i)
            y = L.mixer(h, m, st[i])
            after = {} if L.gate_up else shift[i + 1]
            x, h = o.stream_step(m, c.hidden, x=x, y=y, w=L.norm1, save=st[i]["shift"], **after, **kw)
            if L.gate_up:
                x, h = o.stream_step(m, c.hidden, x=x, y=L.down(L.gate_up(h), partial=True), w=L.norm2, **shift[i + 1], **kw)
        return x

    def _parallel_blocks(self, m: SeqBatch, ids) -> torch.Tensor:
        c, o, st, layers, runs = self.cfg, self.ops, self.cache.layers, self.layers, self.cfg.runs
        emb = dict(ids=ids, table=self.embed, embed_scale=c.embed_scale)

        def before(i):  # what the stream gains ahead of run i, and the norm run i reads it through
            if i == len(runs):
                return {}
            t = runs[i].loop_pass
            return dict(w=layers[i].norm1, vec=None if t is None else self.pass_vec[t], **(emb if t else {}))
        x, h = o.stream_add(m.T, c.hidden, c.eps, self.act, **{**before(0), **emb})
        for i, L in enumerate(layers):
            if self.layer_hook is not None:
                self.layer_hook(i)
            parts = [(L.mixer(h, m, st[i], partial="own" if L.gate_up else True), L.scale1, None)]
            if L.gate_up:
                parts.append((L.down(L.gate_up(h), partial=True), L.scale2, L.down_bias))
            x, h = o.stream_add(m.T, c.hidden, c.eps, self.act, x=x, parts=parts, **before(i + 1))
        return x

    def _logits(self, x, rows=None, out=None):
        h = self.ops.stream_final(x, self.final_norm, self.cfg.eps, self.cfg.hidden, self.act, rows,
                                  center=self.cfg.block == "parallel")
        return self.head(h, out=out)[:, :self.cfg.vocab]

    def step(self, m: SeqBatch, ids, rows=None) -> torch.Tensor | None:
        """Run a batch of portions from their slots' state. rows (int64, device): packed rows whose logits
        [n, vocab] are returned, in the activation type (None: no logits)."""
        x = self._forward(m, ids)
        return None if rows is None else self._logits(x, rows)

    def prefill(self, ids, pos, slot_tok, cu, max_seqlen: int, last_idx, prefix=None, local_logits: bool = False,
                lens=None):
        """Packed prompts (LlamaDecoder.prefill's arguments; lens: the host's prompt lengths) -> logits of
        each one's last token."""
        if prefix is not None:
            raise ValueError("prompt heads cannot be shared between sequences of recurrent layers")
        lens = (cu[1:] - cu[:-1]).tolist() if lens is None else lens
        first = cu[:-1].long()
        m, _ = pack_batch(lens, [0] * len(lens), [0] * len(lens), self.device)
        m.slot, m.pos0 = slot_tok[first].contiguous(), pos[first].contiguous()
        m.max_ctx = self.cache.row_pages * PAGE
        return self.step(m, ids, last_idx)

    def decode_buffers(self, B: int) -> dict:
        """Static buffers of a decode state; tuples are shared as they are by views of fewer rows."""
        dev = self.device
        return {"rows_iota": (torch.arange(B + 1, dtype=torch.int32, device=dev),),
                "logits": torch.zeros(B, self.head.w.shape[0], dtype=self.act, device=dev)}

    def decode_step(self, st) -> torch.Tensor:
        """One token of every row of a decode state (graph-capturable), then the sampler's bookkeeping."""
        iota, = st.rows_iota
        m = SeqBatch(iota[:st.B + 1], st.slot, st.pos, iota[:st.B], st.B, st.B, 1, self.cache.row_pages * PAGE)
        logits = self._logits(self._forward(m, st.tokens), out=st.logits)
        self.sample(logits, st.temperature, st.seed, 0, out_tok=st.tokens, out_lp=st.lp, conf=st.conf, active=st.active,
                    ctr=st.pos, pos=st.pos, lens=st.lens, hist=st.hist, start=st.start, eos=st.eos)
        return st.tokens

    def sample(self, logits, temperature: float, seed: int, step: int = 0, **kw):
        return self.ops.sample(logits, temperature, seed, step, **kw)

    def prefill_flops(self, lens) -> float:
        c = self.cfg
        tot = 0.0
        for n in lens:
            for s in (c.spec[r.layer] for r in c.runs):
                tot += 2.0 * n * (s.mixer.param_count(c.hidden) + 3 * c.hidden * s.ff)
                if isinstance(s.mixer, SigmoidAttention):
                    tot += 2.0 * s.mixer.heads * s.mixer.dim * n * n
                elif isinstance(s.mixer, LatentAttention):
                    tot += s.mixer.heads * (s.mixer.dim + s.mixer.rot_dim + s.mixer.vdim) * n * n
                elif isinstance(s.mixer, ChannelDelta):
                    tot += 6.0 * n * s.mixer.heads * s.mixer.dim * s.mixer.vdim
            tot += 2.0 * c.hidden * c.vocab
        return tot
