"""Decoders that mix sequence mixers layer by layer, on the gfx950 kernels (Binupel).

Residual stream x in fp32; per layer, with alpha, the norm weights and the shift mu of the configuration:

    h  = x + (x_previous - x) mu                token shift (x_previous: the previous token's row, state)
    x  = RMSNorm(alpha x + mixer(h)) w1
    x  = RMSNorm(alpha x + down(relu(gate x) * up x)) w2        where the layer has a feed-forward

Each line's norm, the shift of the next layer's input and the saving of the shift's state are one launch
(``stream_step``). Mixers:

    gated recurrence   [gate | input] GEMM, causal conv, block-diagonal gates GEMM whose epilogue turns the
                       gates into decay and drive, scan (+ output gate, + conv state), output GEMM
    sigmoid attention  [q | k | gates] GEMM, query / key preparation + page write, attention over the paged
                       keys (values = keys, stored once), output GEMM
    selective scan     [x | z] GEMM, causal conv + silu, [dt | B | C] GEMM, step-size GEMM with a softplus
                       epilogue in fp32, scan (+ D x, silu(z), conv state), output GEMM

A step (``step``) runs any batch of portions of sequences (``SeqBatch``): whole prompts, parts of prompts and
single tokens side by side, each from the state its slot holds. Prefill and the graph-captured decode step
are that same step. Weights are packed once at load: projections that share an input are concatenated, and
every width is zero-padded to what the kernels tile by (norms divide by the true width), so any
configuration runs on the same kernels. ``dtype`` "fp32" runs everything in true fp32.
"""
from __future__ import annotations

import math

import torch

from ..ops import get_ops
from ..ops.reference import interleave_gate_up
from ..ops.seq_batch import PAGE, SeqBatch, pack_batch
from .configs import GatedRecurrence, HybridConfig, SelectiveScan, SigmoidAttention
from .state import LayerState, StateCache

EPI_NONE, EPI_BIAS, EPI_REGLU = 0, 1, 7
ANY_NONE, ANY_SOFTPLUS, ANY_REGLU = 0, 1, 2
DTYPES = {"bf16": torch.bfloat16, "fp32": torch.float32}
TILE = 64  # K of every product, N of the packed projections


def _up(n: int, m: int = TILE) -> int:
    return -(-n // m) * m


def _pad(t: torch.Tensor, *shape: int) -> torch.Tensor:
    """Zero-padded at the end of every dimension (-1: as it is)."""
    shape = [s if n < 0 else n for s, n in zip(t.shape, shape)]
    if list(t.shape) == shape:
        return t.contiguous()
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, s) for s in t.shape)] = t
    return out


class Linear:
    """x W^T (+ bias) in the activation type: gemm.hip's kernels in bf16, gemm_any in fp32."""

    def __init__(self, ops, w, act, bias=None, relu_gated: bool = False):
        self.ops, self.act = ops, act
        self.w = w.to(act).contiguous()
        self.bias = None if bias is None else bias.to(act).contiguous()
        self.gated = relu_gated

    def __call__(self, x, out=None, partial: bool = False):
        """partial: the consumer also takes fp32 split-K partials [splits, M, N]."""
        if self.act == torch.float32:
            y = self.ops.gemm_any(x, self.w, self.bias, ANY_REGLU if self.gated else ANY_NONE)
            return y if out is None else out.copy_(y)
        if partial and self.ops.partials_fit(x.shape[0], *self.w.shape):
            return self.ops.gemm_partials(x, self.w)
        epi = EPI_REGLU if self.gated else (EPI_NONE if self.bias is None else EPI_BIAS)
        return self.ops.gemm(x, self.w, bias=self.bias, epi=epi, out=out)


class RecurrenceMixer:
    @staticmethod
    def padded(s: GatedRecurrence) -> tuple[int, int]:
        """(channels of a block, of all blocks): a block a multiple of 16, all of them of 64."""
        bw = _up(s.width // s.blocks, max(16, TILE // math.gcd(s.blocks, TILE)))
        return bw, s.blocks * bw

    @classmethod
    def state(cls, s: GatedRecurrence, act) -> LayerState:
        _, C = cls.padded(s)
        return LayerState({"rec": ((C,), torch.float32), "conv": ((s.conv - 1, C), act)})

    @staticmethod
    def tensors(s: GatedRecurrence, h: int) -> dict:
        w, b = s.width, s.width // s.blocks
        return {"y": (w, h), "y.b": (w,), "x": (w, h), "x.b": (w,), "conv": (w, s.conv), "conv.b": (w,),
                "ra": (s.blocks, b, b), "ra.b": (s.blocks, b), "ri": (s.blocks, b, b), "ri.b": (s.blocks, b),
                "lam": (w,), "o": (h, w)}

    def __init__(self, ops, s: GatedRecurrence, w, hp: int, eps: float, act):
        self.ops, self.s = ops, s
        bw, C = self.padded(s)
        self.C = C
        b0 = s.width // s.blocks

        def chan(t):  # leading dimension: channels -> blocks of bw
            return _pad(t.reshape(s.blocks, b0, *t.shape[1:]), -1, bw, *[-1] * (t.dim() - 1)).reshape(C, *t.shape[1:])
        self.proj = Linear(ops, torch.cat([_pad(chan(w["y"]), -1, hp), _pad(chan(w["x"]), -1, hp)]), act,
                           torch.cat([chan(w["y.b"]), chan(w["x.b"])]))
        self.conv_w = chan(w["conv"]).float().t().contiguous()
        self.conv_b = chan(w["conv.b"]).float()
        ra, ri = (_pad(w[k], -1, bw, bw) for k in ("ra", "ri"))
        self.gate_w = torch.stack([interleave_gate_up(a, i) for a, i in zip(ra, ri)]).to(act).contiguous()
        rb, ib = (_pad(w[k], -1, bw).reshape(-1, 1) for k in ("ra.b", "ri.b"))
        self.gate_b = interleave_gate_up(rb, ib).reshape(s.blocks, 2 * bw).float().contiguous()
        lam = w["lam"].double()
        self.lam = chan((-8.0 * torch.nn.functional.softplus(lam, threshold=700.0)).float())
        self.out = Linear(ops, _pad(chan(w["o"].t()).t(), hp, -1), act)

    def __call__(self, h, m: SeqBatch, st: dict):
        o, C = self.ops, self.C
        yx = self.proj(h)
        gate, x = yx[:, :C], yx[:, C:]
        u = o.causal_conv(x, self.conv_w, self.conv_b, st["conv"], m, silu=False)
        decay, drive = o.rglru_gates(u, self.gate_w, self.gate_b, self.lam)
        return self.out(o.gated_scan(decay, drive, gate, st["rec"], x, st["conv"], m), partial=True)


class AttentionMixer:
    @staticmethod
    def padded(s: SigmoidAttention) -> int:
        d = _up(s.dim, 32 if s.heads % 2 == 0 else 64)
        return d if d <= 128 or d > 256 else _up(d, 64)

    @classmethod
    def state(cls, s: SigmoidAttention, act) -> LayerState:
        return LayerState(page={"k": ((s.kv_heads, PAGE, cls.padded(s)), act),
                                "k_rms": ((s.kv_heads, PAGE), torch.float32)})

    @staticmethod
    def tensors(s: SigmoidAttention, h: int) -> dict:
        return {"q": (s.heads * s.dim, h), "k": (s.kv_heads * s.dim, h), "q.norm": (s.dim,), "k.norm": (s.dim,),
                "pb": (s.heads,), "g": (s.heads, h), "o": (h, s.heads * s.dim)}

    def __init__(self, ops, s: SigmoidAttention, w, hp: int, eps: float, act):
        self.ops, self.s, self.eps = ops, s, eps
        D = self.padded(s)

        def heads(t, n):  # rows of n heads -> heads of D
            return _pad(t.reshape(n, s.dim, -1), -1, D, hp).reshape(n * D, hp)
        qkg = torch.cat([heads(w["q"], s.heads), heads(w["k"], s.kv_heads), _pad(w["g"], -1, hp)])
        self.proj = Linear(ops, _pad(qkg, _up(qkg.shape[0]), -1), act)
        self.qk_w = _pad(w["q.norm"].float() * w["k.norm"].float(), D)
        self.pb = w["pb"].float().contiguous()
        wo = w["o"].reshape(-1, s.heads, s.dim)
        self.out = Linear(ops, _pad(wo, hp, -1, D).reshape(hp, s.heads * D), act)

    def __call__(self, h, m: SeqBatch, st: dict):
        s = self.s
        a = self.ops.sigmoid_attn(self.proj(h), st["k"], st["k_rms"], self.pb, self.qk_w, m, s.heads, s.kv_heads, s.dim,
                                  s.scale, self.eps, s.q_temp)
        return self.out(a, partial=True)


class ScanMixer:
    @classmethod
    def state(cls, s: SelectiveScan, act) -> LayerState:
        C = _up(s.inner)
        return LayerState({"ssm": ((C, s.state), torch.float32), "conv": ((s.conv - 1, C), act)})

    @staticmethod
    def tensors(s: SelectiveScan, h: int) -> dict:
        n = s.inner
        return {"in": (2 * n, h), "conv": (n, s.conv), "conv.b": (n,), "x": (s.dt_rank + 2 * s.state, n),
                "dt": (n, s.dt_rank), "dt.b": (n,), "A_log": (n, s.state), "D": (n,), "o": (h, n)}

    def __init__(self, ops, s: SelectiveScan, w, hp: int, eps: float, act):
        self.ops, self.s = ops, s
        n, C = s.inner, _up(s.inner)
        self.C = C
        self.proj = Linear(ops, torch.cat([_pad(w["in"][:n], C, hp), _pad(w["in"][n:], C, hp)]), act)
        self.conv_w = _pad(w["conv"], C, -1).float().t().contiguous()
        self.conv_b = _pad(w["conv.b"], C).float()
        self.low = Linear(ops, _pad(w["x"], _up(s.dt_rank + 2 * s.state), C), act)
        # the step sizes' operand is the first columns of [dt | B | C]; zero weights meet the rest
        self.dt_k = _up(s.dt_rank)
        self.dt_w = _pad(w["dt"], C, self.dt_k).to(act).contiguous()
        self.dt_b = _pad(w["dt.b"], C).float()
        self.A = _pad((-torch.exp(w["A_log"].double()) * math.log2(math.e)).float(), C, -1)
        self.D = _pad(w["D"], C).float()
        self.out = Linear(ops, _pad(w["o"], hp, C), act)

    def __call__(self, h, m: SeqBatch, st: dict):
        o, C, s = self.ops, self.C, self.s
        xz = self.proj(h)
        x, z = xz[:, :C], xz[:, C:]
        xc = o.causal_conv(x, self.conv_w, self.conv_b, st["conv"], m, silu=True)
        low = self.low(xc)
        dt = o.gemm_any(low[:, :self.dt_k], self.dt_w, self.dt_b, ANY_SOFTPLUS)
        y = o.selective_scan(xc, dt, low, s.dt_rank, s.dt_rank + s.state, z, self.A, self.D, st["ssm"], x, st["conv"], m)
        return self.out(y, partial=True)


MIXERS = {GatedRecurrence: RecurrenceMixer, SigmoidAttention: AttentionMixer, SelectiveScan: ScanMixer}


def tensor_shapes(cfg: HybridConfig) -> dict[str, tuple]:
    """Name -> shape of every tensor of a checkpoint of this configuration."""
    h = cfg.hidden
    out = {"embed": (cfg.vocab, h)}
    for i, s in enumerate(cfg.spec):
        if s.weights_of is not None:
            continue
        out.update({f"l{i}.norm1": (h,), f"l{i}.shift": (h,)})
        out.update({f"l{i}.mix.{k}": v for k, v in MIXERS[type(s.mixer)].tensors(s.mixer, h).items()})
        if s.ff:
            out.update({f"l{i}.norm2": (h,), f"l{i}.mlp.gate": (s.ff, h), f"l{i}.mlp.up": (s.ff, h),
                        f"l{i}.mlp.down": (h, s.ff)})
    out.update({"final.norm": (h,), "head": (cfg.vocab, h)})
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
        if key in ("norm1", "norm2", "final.norm", "q.norm", "k.norm", "D"):
            t.normal_(1.0, 0.1, generator=gen)
        elif key == "shift":
            t.uniform_(0.0, 0.6, generator=gen)
        elif key == "lam":
            t.uniform_(-5.0, -1.0, generator=gen)
        elif key == "A_log":
            t.uniform_(0.0, math.log(16.0), generator=gen)
        elif key == "dt.b":
            t.uniform_(-5.0, -2.0, generator=gen)
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
    """What every layer keeps per sequence: its mixer's state and the token shift's previous row."""
    shift = {"shift": ((_up(cfg.hidden),), torch.float32)}
    per = [MIXERS[type(s.mixer)].state(s.mixer, act) for s in cfg.spec]
    return [LayerState({**p.slot, **shift}, p.page) for p in per]


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
        return AttentionMixer.padded(m) * 2 * (2 * m.heads + m.kv_heads)
    return 12 * _up(cfg.hidden) + max(max(mixer(s.mixer), 2 * _up(s.ff)) for s in cfg.spec)


class _Layer:
    """One layer's packed weights (shared by the layers that use them)."""

    def __init__(self, ops, cfg: HybridConfig, i: int, raw: dict, hp: int, act):
        s, pre = cfg.spec[i], f"l{i}."
        mix = {k[len(pre) + 4:]: v for k, v in raw.items() if k.startswith(pre + "mix.")}
        self.mixer = MIXERS[type(s.mixer)](ops, s.mixer, mix, hp, cfg.eps, act)
        self.norm1 = _pad(raw[pre + "norm1"], hp).float()
        self.shift = _pad(raw[pre + "shift"], hp).float()
        self.norm2 = self.gate_up = self.down = None
        if s.ff:
            f = _up(s.ff)
            self.norm2 = _pad(raw[pre + "norm2"], hp).float()
            self.gate_up = Linear(ops, interleave_gate_up(_pad(raw[pre + "mlp.gate"], f, hp),
                                                          _pad(raw[pre + "mlp.up"], f, hp)), act, relu_gated=True)
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
        self.layers = [own[i if s.weights_of is None else s.weights_of] for i, s in enumerate(cfg.spec)]
        self.embed = _pad(raw["embed"], -1, hp).to(act).contiguous()
        self.final_norm = _pad(raw["final.norm"], hp).float()
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
        c, o, st, layers = self.cfg, self.ops, self.cache.layers, self.layers
        kw = dict(eps=c.eps, alpha=c.alpha, act=self.act)
        shift = [dict(mu=L.shift, prev=s["shift"]) for L, s in zip(layers, st)] + [dict(want_h=False)]
        m = m.on(self.cache.table)
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

    def _logits(self, x, rows=None, out=None):
        h = self.ops.stream_final(x, self.final_norm, self.cfg.eps, self.cfg.hidden, self.act, rows)
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
            for s in c.spec:
                tot += 2.0 * n * (s.mixer.param_count(c.hidden) + 3 * c.hidden * s.ff)
                if isinstance(s.mixer, SigmoidAttention):
                    tot += 2.0 * s.mixer.heads * s.mixer.dim * n * n
            tot += 2.0 * c.hidden * c.vocab
        return tot
