"""Sequence mixers of the decoders of mixed layers: one class per kind, each with the tensors a checkpoint holds for
it, what it keeps per sequence (``LayerState``), its packed weights and its forward over a batch of portions.

    gated recurrence   [gate | input] GEMM, causal conv, block-diagonal gates GEMM whose epilogue turns the
                       gates into decay and drive, scan (+ output gate, + conv state), output GEMM
    sigmoid attention  [q | k | gates] GEMM, query / key preparation + page write, attention over the paged
                       keys (values = keys, stored once), output GEMM
    selective scan     [x | z] GEMM, causal conv + silu, [dt | B | C] GEMM, step-size GEMM with a softplus
                       epilogue in fp32, scan (+ D x, silu(z), conv state), output GEMM
    delta rule         [q | k | v | decay rank | gate rank | beta] GEMM, causal conv + silu, decay GEMM whose epilogue
                       leaves log decays in fp32, scan (+ unit norms, beta, conv state), gate GEMM, gated norm of
                       every head, output GEMM
    latent attention   [query rank | latent | rotated key | gates] GEMM, norms + rotation + page write, query GEMM;
                       short portions attend to the cached latents (queries taken into the latent space, results
                       out of it, head by head), long ones to keys and values expanded from them; output GEMM

Weights are packed once at load: projections that share an input are concatenated, and every width is
zero-padded to what the kernels tile by (means divide by the true width), so any configuration runs on the
same kernels.
"""
from __future__ import annotations

import math

import torch

from ..ops.reference import interleave_gate_up
from ..ops.seq_batch import PAGE, SeqBatch
from .configs import ChannelDelta, GatedRecurrence, LatentAttention, SelectiveScan, SigmoidAttention
from .state import LayerState, RotaryTable

EPI_NONE, EPI_BIAS = 0, 1
ANY_NONE, ANY_SOFTPLUS = 0, 1
GATED_EPI = {"silu": 3, "relu": 7}
GATED_ANY = {"silu": 4, "relu": 2}
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
    """x W^T (+ bias) in the activation type: gemm.hip's kernels in bf16, gemm_any in fp32. gated: rows interleaved
    by 16 (gate, up), result act(gate) * up with act "relu" or "silu"."""

    def __init__(self, ops, w, act, bias=None, gated: str | None = None):
        self.ops, self.act = ops, act
        self.w = w.to(act).contiguous()
        self.bias = None if bias is None else bias.to(act).contiguous()
        self.epi = GATED_EPI[gated] if gated else EPI_NONE if bias is None else EPI_BIAS
        self.any_epi = GATED_ANY[gated] if gated else ANY_NONE

    def __call__(self, x, out=None, partial: bool = False):
        """partial: the consumer also takes fp32 split-K partials [splits, M, N] (without the bias); "own": in a
        buffer of their own, valid past the next product."""
        if self.act == torch.float32:
            y = self.ops.gemm_any(x, self.w, self.bias, self.any_epi)
            return y if out is None else out.copy_(y)
        if partial and self.ops.partials_fit(x.shape[0], *self.w.shape):
            return self.ops.gemm_partials(x, self.w, own=partial == "own")
        return self.ops.gemm(x, self.w, bias=self.bias, epi=self.epi, out=out)


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

    def __call__(self, h, m: SeqBatch, st: dict, partial=True):
        o, C = self.ops, self.C
        yx = self.proj(h)
        gate, x = yx[:, :C], yx[:, C:]
        u = o.causal_conv(x, self.conv_w, self.conv_b, st["conv"], m, silu=False)
        decay, drive = o.rglru_gates(u, self.gate_w, self.gate_b, self.lam)
        return self.out(o.gated_scan(decay, drive, gate, st["rec"], x, st["conv"], m), partial=partial)


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

    def __call__(self, h, m: SeqBatch, st: dict, partial=True):
        s = self.s
        a = self.ops.sigmoid_attn(self.proj(h), st["k"], st["k_rms"], self.pb, self.qk_w, m, s.heads, s.kv_heads, s.dim,
                                  s.scale, self.eps, s.q_temp)
        return self.out(a, partial=partial)


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

    def __call__(self, h, m: SeqBatch, st: dict, partial=True):
        o, C, s = self.ops, self.C, self.s
        xz = self.proj(h)
        x, z = xz[:, :C], xz[:, C:]
        xc = o.causal_conv(x, self.conv_w, self.conv_b, st["conv"], m, silu=True)
        low = self.low(xc)
        dt = o.gemm_any(low[:, :self.dt_k], self.dt_w, self.dt_b, ANY_SOFTPLUS)
        y = o.selective_scan(xc, dt, low, s.dt_rank, s.dt_rank + s.state, z, self.A, self.D, st["ssm"], x, st["conv"], m)
        return self.out(y, partial=partial)


class DeltaMixer:
    UNIT_EPS = 1e-6  # of the unit norms of queries and keys

    @staticmethod
    def padded(s: ChannelDelta) -> tuple[int, int]:
        """(key channels, value channels) of a head: what the scan's lanes hold; all heads' values a multiple of 64."""
        K = _up(s.dim, 32) if s.dim <= 256 else _up(s.dim, 64) if s.dim <= 512 else _up(s.dim, 128)
        return K, _up(s.vdim, max(8, TILE // math.gcd(s.heads, TILE)))

    @classmethod
    def state(cls, s: ChannelDelta, act) -> LayerState:
        K, V = cls.padded(s)
        return LayerState({"delta": ((s.heads, V, K), torch.float32),
                           "conv": ((s.conv - 1, 2 * s.kv_heads * K + s.heads * V), act)})

    @staticmethod
    def tensors(s: ChannelDelta, h: int) -> dict:
        nk, nv, nd = s.kv_heads * s.dim, s.heads * s.vdim, s.heads * s.dim
        return {"q": (nk, h), "q.conv": (nk, s.conv), "k": (nk, h), "k.conv": (nk, s.conv), "v": (nv, h),
                "v.conv": (nv, s.conv), "b": (s.heads, h), "A_log": (s.heads,), "norm": (s.vdim,),
                "a1": (s.decay_rank, h), "a2": (nd, s.decay_rank), "dt_bias": (nd,), "g1": (s.gate_rank, h),
                "g2": (nv, s.gate_rank), "o": (h, nv)}

    def __init__(self, ops, s: ChannelDelta, w, hp: int, eps: float, act):
        self.ops, self.s, self.eps = ops, s, eps
        H, G = s.heads, s.kv_heads
        K, V = self.K, self.V = self.padded(s)

        def heads(t, n, to):  # rows of n heads -> heads of ``to`` rows
            return _pad(t.reshape(n, t.shape[0] // n, -1), -1, to, -1).reshape(n * to, -1)
        ra, rg = _up(s.decay_rank), _up(s.gate_rank)
        rows = [heads(w["q"], G, K), heads(w["k"], G, K), heads(w["v"], H, V), _pad(w["a1"], ra, -1), _pad(w["g1"], rg, -1),
                w["b"]]
        self.C = sum(r.shape[0] for r in rows[:3])
        self.at_decay, self.at_gate, self.at_beta = self.C, self.C + ra, self.C + ra + rg
        proj = torch.cat(rows)
        self.proj = Linear(ops, _pad(proj, _up(proj.shape[0]), hp), act)
        conv = torch.cat([heads(w["q.conv"], G, K), heads(w["k.conv"], G, K), heads(w["v.conv"], H, V)])
        self.conv_w = conv.float().t().contiguous()
        self.decay_w = _pad(heads(w["a2"], H, K), -1, ra).to(act).contiguous()
        self.dt_bias = _pad(w["dt_bias"].float().reshape(H, s.dim), -1, K).reshape(-1)
        # log2 of the decay per unit of softplus
        rate = (-torch.exp(w["A_log"].double()) * math.log2(math.e)).float()
        self.rate = rate[:, None].expand(H, K).reshape(-1).contiguous()
        self.gate = Linear(ops, _pad(heads(w["g2"], H, V), -1, rg), act)
        self.norm = _pad(w["norm"].float(), V)
        self.out = Linear(ops, _pad(heads(w["o"].t(), H, V).t(), hp, -1), act)

    def __call__(self, h, m: SeqBatch, st: dict, partial=True):
        o, s, C = self.ops, self.s, self.C
        y = self.proj(h)
        x = y[:, :C]
        qkv = o.causal_conv(x, self.conv_w, None, st["conv"], m, silu=True)
        decay = o.gemm_any(y[:, self.at_decay:self.at_gate], self.decay_w, self.dt_bias, ANY_SOFTPLUS, coef=self.rate)
        gate = self.gate(y[:, self.at_gate:self.at_beta])
        r = o.delta_rule(qkv, decay, y[:, self.at_beta:], st["delta"], x, st["conv"], m, s.heads, s.kv_heads,
                         s.dim ** -0.5, self.UNIT_EPS, norm=(self.norm, gate, s.vdim, self.eps))
        return self.out(r, partial=partial)


class LatentMixer:
    EXPAND_FROM = 128  # tokens from which a portion's keys and values are expanded from the latents

    @staticmethod
    def padded(s: LatentAttention, act=torch.bfloat16) -> tuple[int, int, int, int, int]:
        """(query rank, latent, rotated key, query / key head, value head) as the kernels tile them."""
        L = next((n for n in (64, 128, 256, 512) if s.kv_rank <= n), _up(s.kv_rank))
        R = next((n for n in (32, 64) if s.rot_dim <= n), _up(s.rot_dim))
        d = _up(s.dim, 8) + _up(s.rot_dim, 8)
        D = next((n for n in (64, 96, 128, 192, 256) if d <= n), _up(d))
        V = _up(s.vdim, max(32, TILE // math.gcd(s.heads, TILE)))
        return _up(s.q_rank), L, R, D, V

    @classmethod
    def state(cls, s: LatentAttention, act) -> LayerState:
        _, L, R, _, _ = cls.padded(s)
        return LayerState(page={"latent": ((PAGE, L + R), act)}, tables={"rot": RotaryTable(s.rot_dim, s.rot_base)})

    @staticmethod
    def tensors(s: LatentAttention, h: int) -> dict:
        H = s.heads
        return {"dq": (s.q_rank, h), "dq.norm": (s.q_rank,), "uq": (H * (s.dim + s.rot_dim), s.q_rank),
                "dkv": (s.kv_rank + s.rot_dim, h), "dkv.norm": (s.kv_rank,), "uk": (H * s.dim, s.kv_rank),
                "uv": (H * s.vdim, s.kv_rank), "sink": (H,), "g": (H * s.vdim, h), "o": (h, H * s.vdim)}

    def __init__(self, ops, s: LatentAttention, w, hp: int, eps: float, act):
        self.ops, self.s, self.eps, self.act = ops, s, eps, act
        H = s.heads
        Q, L, R, D, V = self.Q, self.L, self.R, self.D, self.V = self.padded(s)
        self.d = d = _up(s.dim, 8)  # unrotated columns of a head; the rotated ones follow
        g = _pad(w["g"].reshape(H, s.vdim, -1), -1, V, -1).reshape(H * V, -1)
        proj = torch.cat([_pad(w["dq"], Q, -1), _pad(w["dkv"][:s.kv_rank], L, -1), _pad(w["dkv"][s.kv_rank:], R, -1), g])
        self.proj = Linear(ops, _pad(proj, _up(proj.shape[0]), hp), act)
        self.at_gate = Q + L + R
        self.q_norm, self.c_norm = _pad(w["dq.norm"].float(), Q), _pad(w["dkv.norm"].float(), L)
        uq = w["uq"].reshape(H, s.dim + s.rot_dim, -1)
        uq = torch.cat([_pad(uq[:, :s.dim], -1, d, Q), _pad(uq[:, s.dim:], -1, D - d, Q)], 1)
        self.uq = Linear(ops, uq.reshape(H * D, Q), act)
        uk, uv = (w[k].reshape(H, n, -1) for k, n in (("uk", s.dim), ("uv", s.vdim)))
        # into and out of the latent space, head by head: [H, L, d] and [H, V, L]
        self.absorb = _pad(uk.transpose(1, 2), -1, L, d).to(act).contiguous()
        self.emit = _pad(uv, -1, V, L).to(act).contiguous()
        self.expand = None
        if act == torch.bfloat16 and ops.latent_flash_fits(D, V):
            kv = torch.cat([_pad(uk, -1, d, L), _pad(uv, -1, V, L)], 1)
            self.expand = Linear(ops, kv.reshape(H * (d + V), L), act)
        self.sink = w["sink"].float().contiguous()
        self.out = Linear(ops, _pad(_pad(w["o"].reshape(-1, H, s.vdim), -1, -1, V).reshape(-1, H * V), hp, -1), act)

    def __call__(self, h, m: SeqBatch, st: dict, partial=True):
        o, s = self.ops, self.s
        pages, rot = st["latent"], st["rot"]
        y = self.proj(h)
        cq = o.latent_prep(y, self.q_norm, s.q_rank, self.c_norm, s.kv_rank, s.rot_dim, self.eps, pages, rot, m)
        q, gate = self.uq(cq), y[:, self.at_gate:self.at_gate + s.heads * self.V]
        short, long = m.split(self.EXPAND_FROM if self.expand else None)
        if short is None or long is None:
            r = (self._absorbed if long is None else self._expanded)(m, q, gate, pages, rot)
        else:
            r = torch.empty((m.T, s.heads * self.V), dtype=q.dtype, device=q.device)
            for (part, rows), run in ((short, self._absorbed), (long, self._expanded)):
                r.index_copy_(0, rows, run(part, q.index_select(0, rows), gate.index_select(0, rows), pages, rot))
        return self.out(r, partial=partial)

    def _absorbed(self, m, q, gate, pages, rot):
        o, s = self.ops, self.s
        ql = o.gemm_heads(q, self.absorb, self.D)
        a = o.latent_attn(q, ql, pages, rot, self.sink, m, s.heads, self.d, s.rot_dim, self.L, s.scale)
        return o.gemm_heads(a, self.emit, self.L, gate=gate)

    def _expanded(self, m, q, gate, pages, rot):
        o, s = self.ops, self.s
        lat = o.latent_gather(pages, m)
        kv = self.expand(lat[:, :self.L])
        return o.latent_flash(q, lat, kv, gate, rot, self.sink, m, s.heads, self.d, s.rot_dim, self.L, self.V, s.scale)


MIXERS = {GatedRecurrence: RecurrenceMixer, SigmoidAttention: AttentionMixer, SelectiveScan: ScanMixer,
          ChannelDelta: DeltaMixer, LatentAttention: LatentMixer}
