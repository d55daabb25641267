"""The Zamitar decoder against its plain implementation (tests/zamitar_oracle.py): each mechanism alone, whole
models, portions of prompts, batches, slots and pages that change hands, and generation through the
framework's generator, scheduler and engine."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import zamitar_oracle as oracle
from docagents_amd.engine.generator import ContinuousScheduler, Generator
from docagents_amd.engine.replay import replay
from docagents_amd.models import make_decoder
from docagents_amd.models.configs import DECODERS, HybridConfig, checkpoint_config, decoder_config, zamitar_config
from docagents_amd.models.mixers import LatentMixer
from docagents_amd.models.state import LayerState, RotaryTable, StateCache
from docagents_amd.ops import get_ops
from docagents_amd.ops.reference import interleave_gate_up
from docagents_amd.ops.seq_batch import PAGE, pack_batch
from seq_cases import (ACT, CPU, GPU16, GPU32, WHERE, Portions, checkpoint, close, mixed_schedule, one_thread,  # noqa: F401
                       rand, row_errors, run, tokens)
from zamitar_cases import CONFIGS, TOL, build, check, config, delta, expect, latent, weights


# ---------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("dim,Dp", [(90, 128), (64, 64), (1030, 1088), (4700, 4736)])
def test_stream_sum_and_layer_norm(device, dtype, dim, Dp):
    """Every kind of term, alone and together; columns with a mean far from zero."""
    act, T, eps, ops = ACT[dtype], 7, 0.03, get_ops(device)
    pad = lambda t: torch.nn.functional.pad(t, (0, Dp - dim))  # noqa: E731
    f = lambda t: pad(t).float().to(device).contiguous()  # noqa: E731
    x, w, vec = rand(1, T, dim) + 5, rand(2, dim), rand(3, dim)
    ys = [pad(rand(4 + i, T, dim)).to(act) for i in range(2)]
    split = pad(rand(6, 11, T, dim, std=0.3))  # partials of a product
    s, b = [rand(7 + i, dim) for i in range(2)], [rand(9, dim), None]
    table, ids = pad(rand(10, 50, dim)).to(act), torch.tensor([3, 49, 0, 7, 7, 20, 1], dtype=torch.int32)
    yd = [y.double()[:, :dim] for y in ys]
    emb = table.double()[ids.long(), :dim] * 2.5
    part = lambda i, y=None: ((ys[i].to(device) if y is None else y), f(s[i]), None if b[i] is None else f(b[i]))  # noqa: E731
    lookup = dict(ids=ids.to(device), table=table.to(device), embed_scale=2.5)
    sums = {
        "embedding": (dict(lookup, vec=f(vec)), emb + vec),
        "one": (dict(x=f(x), parts=[part(1)]), x + yd[1] * s[1]),
        "two": (dict(x=f(x), parts=[part(0), part(1)]), x + (yd[0] + b[0]) * s[0] + yd[1] * s[1]),
        "pass": (dict(lookup, x=f(x), vec=f(vec), parts=[part(1), part(0, split.to(device))]),
                 x + yd[1] * s[1] + (split.double().sum(0)[:, :dim] + b[0]) * s[0] + emb + vec),
        "splits": (dict(x=f(x), parts=[part(0, split[:1].contiguous().to(device)), part(1, split[:9].contiguous().to(device))]),
                   x + (split[0].double()[:, :dim] + b[0]) * s[0] + split[:9].double().sum(0)[:, :dim] * s[1]),
    }
    for name, (kw, want) in sums.items():
        got, h = ops.stream_add(T, dim, eps, act, w=f(w), **kw)
        close(got[:, :dim], want, "fp32")
        assert not got[:, dim:].any() and not h[:, dim:].any(), name
        close(h[:, :dim], oracle.layer_norm(want, w.double(), eps), dtype)
        only, none = ops.stream_add(T, dim, eps, act, **kw)
        assert none is None and torch.equal(only, got)
    rows = torch.tensor([5, 0, 5])
    close(ops.stream_final(f(x), f(w), eps, dim, act, rows.to(device), center=True)[:, :dim],
          oracle.layer_norm(x.double(), w.double(), eps)[rows], dtype)
    close(ops.stream_final(f(x), f(w), eps, dim, act)[:, :dim], oracle.rms(x.double(), eps) * w, dtype)


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
@pytest.mark.parametrize("device,dtype", WHERE)
def test_causal_conv_without_bias(device, dtype, taps):
    """Its state is kept by the delta rule's launch in portions, by its own in single tokens."""
    P = Portions(device, dtype)
    H, G, K, V = 2, 1, 32, 16
    C, ops = 2 * G * K + H * V, get_ops(device)
    xs, w = [rand(i, n, C) for i, n in enumerate(P.lens)], rand(8, taps, C)
    state = P.state(taps - 1, C, dtype=P.act)
    for m, spans in P:
        x = P.pack(xs, spans)
        got = ops.causal_conv(x, w.to(device), None, state, m, True)
        z = torch.zeros(m.T, H * K, device=device)
        ops.delta_rule(x, z, x[:, :8], torch.zeros(4, H, V, K, device=device), x, state, m, H, G, 1.0, 1e-6,
                       (torch.ones(V, device=device), x[:, :H * V], V, 1e-6))
        row = 0
        for i, a, e in spans:
            close(got[row:row + e - a], oracle.silu(oracle.causal_conv(P.stored(xs)[i], w.double().t()))[a:e], dtype)
            row += e - a


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("M,N,K", [(1, 64, 64), (5, 96, 128), (23, 40, 64), (64, 72, 192), (130, 200, 64), (1500, 192, 128)])
def test_log_decays(device, dtype, M, N, K):
    """The low-rank projection's epilogue: softplus times a rate per column, in fp32 at every size of the decay."""
    a, w, b = rand(1, M, K).to(ACT[dtype]), rand(2, N, K, std=K ** -0.5).to(ACT[dtype]), rand(3, N) - 2
    rate = -torch.exp(rand(4, N) * 2)
    b[::7] = -25.0  # almost no decay
    want = oracle.softplus(a.double() @ w.double().t() + b.double()) * rate.double()
    got = get_ops(device).gemm_any(a.to(device), w.to(device), b.to(device), 1, coef=rate.to(device)).double().cpu()
    assert ((got - want).abs() / want.abs()).max() < 2e-5


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("M,H,N,K,stride", [(1, 3, 64, 40, 64), (16, 2, 44, 1160, 1160), (18, 2, 24, 520, 528), (37, 5, 40, 128, 128),
                                               (64, 2, 36, 640, 640), (200, 2, 128, 24, 32), (700, 16, 256, 64, 96)])
def test_products_per_head(device, dtype, M, H, N, K, stride):
    if M == 700 and device == "cpu":
        pytest.skip("the large tile, on the GPU")
    act = ACT[dtype]
    a, w, g = rand(1, M, H * stride).to(act), rand(2, H, N, K, std=K ** -0.5).to(act), rand(3, M, H * N + 8).to(act)
    want = torch.cat([a.double()[:, i * stride:i * stride + K] @ w[i].double().t() for i in range(H)], 1)
    o, gate = get_ops(device), g.to(device)[:, :H * N]
    close(o.gemm_heads(a.to(device), w.to(device), stride), want, dtype)
    close(o.gemm_heads(a.to(device), w.to(device), stride, gate=gate), want * torch.sigmoid(g.double()[:, :H * N]), dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("M", [1, 5, 40, 100, 300, 700, 2100])
@pytest.mark.parametrize("N,K", [(512, 512), (96, 192), (4096, 256)])
@pytest.mark.parametrize("epi", ["silu", "relu"])
def test_gated_epilogue_with_biases_of_every_product_route(M, N, K, epi):
    a, w, b = rand(1, M, K).bfloat16(), rand(2, N, K, std=K ** -0.5).bfloat16(), rand(3, N).bfloat16()
    act = {"silu": oracle.silu, "relu": torch.relu}[epi]
    yy = (a.double() @ w.double().t() + b.double()).view(M, N // 32, 2, 16)
    want = (act(yy[:, :, 0]) * yy[:, :, 1]).reshape(M, N // 2)
    code = {"silu": 3, "relu": 7}[epi]
    ops = get_ops("cuda")
    close(ops.gemm(a.cuda(), w.cuda(), bias=b.cuda(), epi=code), want, "bf16")
    if M >= 300:
        close(ops.gemm(a.cuda(), w.cuda(), bias=b.cuda(), epi=code, tile=13), want, "bf16")


@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
def test_gated_product_in_fp32(device, dtype):
    h, f, M = 64, 48, 9
    x, g, u, gb, ub = rand(1, M, h), rand(2, f, h), rand(3, f, h), rand(4, f), rand(5, f)
    w, b = interleave_gate_up(g, u), interleave_gate_up(gb[:, None], ub[:, None])[:, 0]
    got = get_ops(device).gemm_any(x.to(device), w.to(device).contiguous(), b.to(device).contiguous(), 4)
    want = oracle.silu(x.double() @ g.double().t() + gb) * (x.double() @ u.double().t() + ub)
    close(got, want, "fp32")


def delta_case(P, H, G, K, V, dim, vdim, seed=0):
    """(q | k | v sequences as stored, log2 decays, beta columns, gates), padding channels zero."""
    def heads(s, n, rows, true, to):
        return torch.nn.functional.pad(rand(s, n, rows, true), (0, to - true)).flatten(1)
    qkv, dec, beta, gate = [], [], [], []
    for i, n in enumerate(P.lens):
        s = seed + 100 * i
        qkv.append(torch.cat([heads(s + 1, n, G, dim, K), heads(s + 2, n, G, dim, K), heads(s + 3, n, H, vdim, V)], 1))
        dec.append(-torch.exp(rand(s + 4, n, H * K) * 2 - 3))
        beta.append(rand(s + 5, n, 8 * math.ceil(H / 8)) * 2)
        gate.append(rand(s + 6, n, H * V))
    return qkv, dec, beta, gate


def delta_want(qkv, dec, beta, gate, H, G, K, V, dim, vdim, weight, eps, scale):
    """-> (read-outs [T, H, vdim], states after every token [T, H, dim, vdim])"""
    T = len(qkv)
    q, k, v = (t.view(T, n, -1) for t, n in zip(qkv.split([G * K, G * K, H * V], 1), (G, G, H)))
    q, k = (oracle.unit(t[:, :, :dim]).repeat_interleave(H // G, 1) for t in (q, k))
    dec = dec.double().view(T, H, K)[:, :, :dim] * math.log(2)
    o, S = oracle.delta_scan(q * scale, k, v[:, :, :vdim], torch.sigmoid(beta[:, :H]), dec)
    return oracle.gated_head_norm(o, weight.double()[:vdim], gate.view(T, H, V)[:, :, :vdim], eps), S


DELTA = [(2, 2, 32, 32, 32, 32), (6, 2, 32, 40, 20, 33), (3, 1, 128, 128, 128, 128), (2, 1, 96, 72, 70, 70), (2, 2, 256, 64, 250, 64),
         (1, 1, 320, 16, 300, 9), (4, 4, 64, 200, 64, 200), (1, 1, 640, 64, 520, 64), (2, 1, 128, 48, 128, 48)]


@pytest.mark.parametrize("H,G,K,V,dim,vdim", DELTA)
@pytest.mark.parametrize("device,dtype", WHERE)
def test_delta_rule(device, dtype, H, G, K, V, dim, vdim):
    """One channel forgets within a token, one remembers everything; slots hold leftovers."""
    P = Portions(device, dtype)
    if device == "cpu":
        P = Portions(device, dtype, lens=(40, 3, 20), cuts=((2, 1, 30, 7), (1, 2), (16, 1, 3)))
    ops, eps, scale = get_ops(device), 1e-3, dim ** -0.5
    qkv, dec, beta, gate = delta_case(P, H, G, K, V, dim, vdim)
    for d in dec:
        d.view(-1, H, K)[:, 0, 0], d.view(-1, H, K)[:, -1, dim - 1] = -200.0, 0.0
    weight = torch.nn.functional.pad(1 + 0.3 * rand(9, vdim), (0, V - vdim))
    state, conv = P.state(H, V, K), P.state(0, 2 * G * K + H * V, dtype=P.act)
    want = [delta_want(P.stored(qkv)[i], dec[i], P.stored(beta)[i], P.stored(gate)[i], H, G, K, V, dim, vdim, weight, eps, scale)
            for i in range(len(P.lens))]
    for m, spans in P:
        x = P.pack(qkv, spans)
        d = torch.cat([dec[i][a:b] for i, a, b in spans]).to(device).contiguous()
        got = ops.delta_rule(x, d, P.pack(beta, spans), state, x, conv, m, H, G, scale, 1e-6,
                             (weight.to(device), P.pack(gate, spans), vdim, eps)).view(m.T, H, V)
        assert not got[:, :, vdim:].any()
        row = 0
        for i, a, b in spans:
            close(got[row:row + b - a, :, :vdim], want[i][0][a:b], dtype)
            row += b - a
    for i in range(len(P.lens)):
        s = state[P.slots[i]].double().cpu().transpose(1, 2)
        close(s[:, :dim, :vdim], want[i][1], "fp32", 2)
        assert not s[:, dim:].any() and not s[:, :, vdim:].any()


@pytest.mark.gpu
@pytest.mark.parametrize("act", ["fp32", "bf16"])
@pytest.mark.parametrize("strength", [-6.0, -1.0, 2.0, 5.0])
def test_delta_rule_over_long_portions(act, strength):
    """Decays from almost none to many powers of two per token, portions long enough for every way of walking them,
    starting from a stored state."""
    P = Portions("cuda", act, lens=(700, 333), cuts=((5, 641, 54), (300, 33)))
    H, G, K, V = 3, 1, 128, 128
    qkv, dec, beta, gate = delta_case(P, H, G, K, V, K, V)
    dec = [-torch.exp(rand(50 + i, len(d), H * K) + strength) for i, d in enumerate(dec)]
    weight, state = torch.ones(V), P.state(H, V, K)
    conv = P.state(0, 2 * G * K + H * V, dtype=P.act)
    want = [delta_want(P.stored(qkv)[i], dec[i], P.stored(beta)[i], P.stored(gate)[i], H, G, K, V, K, V, weight, 1e-4, 0.1)
            for i in range(2)]
    for m, spans in P:
        x = P.pack(qkv, spans)
        got = get_ops("cuda").delta_rule(x, torch.cat([dec[i][a:b] for i, a, b in spans]).cuda(), P.pack(beta, spans), state, x,
                                         conv, m, H, G, 0.1, 1e-6, (weight.cuda(), P.pack(gate, spans), V, 1e-4))
        row = 0
        for i, a, b in spans:
            close(got[row:row + b - a].view(-1, H, V), want[i][0][a:b], act)
            row += b - a
    for i in range(2):
        close(state[P.slots[i]].transpose(1, 2), want[i][1], "fp32", 5)


@pytest.mark.parametrize("device,dtype", WHERE)
def test_delta_state_keeps_what_was_written(device, dtype):
    """A value written under one key is read back hundreds of tokens later (in a portion and as single tokens),
    replaced when the key is written again, and forgotten where its channels decay."""
    H, K, V, n, act = 1, 32, 16, 300, ACT[dtype]
    basis = torch.eye(K)
    q, k, v = basis[2].repeat(n, 1), basis[5].repeat(n, 1), torch.zeros(n, V)
    k[0], v[0] = basis[2], torch.arange(V) / V + 0.5        # kept
    k[1], v[1] = basis[3], torch.ones(V)                     # on a channel that decays
    k[200], v[200] = basis[2], -torch.ones(V)                # replaces
    q[150] = basis[3]
    dec, beta = torch.zeros(n, K), torch.full((n, 8), 30.0)
    dec[:, 3] = -1.0
    x = torch.cat([q, k, v], 1).to(device, act)
    ops = get_ops(device)
    for cuts in ((n,), (1,) * n, (64, 1, 100, n - 165)):
        state = torch.full((2, H, V, K), 9.0, device=device)
        conv, at, out = torch.zeros(2, 0, 2 * K + V, dtype=act, device=device), 0, []
        for c in cuts:
            m, _ = pack_batch([c], [1], [at], device)
            s = slice(at, at + c)
            out.append(ops.delta_rule(x[s], dec[s].to(device), beta[s].to(device, act), state, x[s], conv, m, H, 1, 1.0, 1e-6,
                                      (torch.ones(V, device=device), torch.full((c, V), 30.0, device=device).to(act), V, 1e-8)))
            at += c
        o = torch.cat(out).float().cpu()
        for t in (0, 1, 63, 64, 130, 199):
            close(o[t], oracle.rms(v[0].double(), 1e-8), dtype)
        close(o[299], -torch.ones(V, dtype=torch.float64), dtype)
        close(state[1, 0, :, 2], -torch.ones(V, dtype=torch.float64), "fp32")
        assert o[150].abs().max() < 1e-3 and state[1, 0, :, 3].abs().max() < 1e-20


def latent_model(seed, H, dim, rot, vdim, L, base, scale, sink):
    """One attention layer's tensors (unit scale products) as the plain implementation takes them."""
    w = {"uk": rand(seed, H * dim, L, std=L ** -0.5), "uv": rand(seed + 1, H * vdim, L, std=L ** -0.5), "sink": sink}
    return w, dict(heads=H, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=L, rot={"base": base, "dims": rot}, scale=scale)


class LatentCase:
    """Sequences of (query, latent, key part, gate) run through the ops in portions on shuffled pages of leftovers."""

    def __init__(self, device, dtype, H, dim, rot, vdim, L, base=100.0, scale=None, sink=None, seed=0):
        from docagents_amd.models.configs import LatentAttention
        self.device, self.act, self.ops = device, ACT[dtype], get_ops(device)
        sink = rand(seed + 5, H) if sink is None else sink
        self.w, self.m = latent_model(seed + 60, H, dim, rot, vdim, L, base, scale or (dim + rot) ** -0.5, sink)
        self.w = {k: v if k == "sink" else v.to(self.act).float() for k, v in self.w.items()}
        self.spec = LatentAttention(H, dim, rot, vdim, 8, L, self.m["scale"], base)
        self.pad = LatentMixer.padded(self.spec)

    def want(self, q, c, kr, gate, c_w, eps):
        m, T = self.m, len(q)
        H, D, R, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
        q, c, kr, gate = (t.to(self.act).double() for t in (q, c, kr, gate))
        c = oracle.rms(c, eps) * c_w.double()
        kr = oracle.rotate(kr, range(T), m["rot"]["base"], R)
        qr = oracle.rotate(q[:, :, D:], range(T), m["rot"]["base"], R)
        k = torch.cat([(c @ self.w["uk"].double().t()).view(T, H, D), kr[:, None].expand(T, H, R)], -1)
        o = oracle.sink_attention(torch.cat([q[:, :, :D], qr], -1), k, (c @ self.w["uv"].double().t()).view(T, H, V), m["scale"],
                                  self.w["sink"].double())
        return o * torch.sigmoid(gate.view(T, H, V))

    def run(self, seqs, steps, c_w, eps, expand):
        o, m, dev, act = self.ops, self.m, self.device, self.act
        H, dim, rot, vdim, Lt = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        Q, L, R, D, V = self.pad
        d = 8 * math.ceil(dim / 8)
        pages = max(-(-len(s[0]) // PAGE) for s in seqs)
        order = np.random.default_rng(3).permutation(4 * pages).reshape(4, pages).astype(np.int32)
        pool, table = torch.full((4 * pages, PAGE, L + R), 5.0, dtype=act, device=dev), torch.from_numpy(order).to(dev)
        tab = RotaryTable(rot, m["rot"]["base"]).build(pages * PAGE, dev)
        pad = torch.nn.functional.pad
        out = [[] for _ in seqs]
        uk, uv = self.w["uk"].view(H, dim, Lt), self.w["uv"].view(H, vdim, Lt)
        absorb = pad(uk.transpose(1, 2), (0, d - dim, 0, L - Lt)).to(dev, act).contiguous()
        emit = pad(uv, (0, L - Lt, 0, V - vdim)).to(dev, act).contiguous()
        kv_w = torch.cat([pad(uk, (0, L - Lt, 0, d - dim)), pad(uv, (0, L - Lt, 0, V - vdim))], 1).reshape(H * (d + V), L)
        sink = self.w["sink"].float().to(dev)
        for spans in steps:
            mb, _ = pack_batch([b - a for _, a, b in spans], [i for i, _, _ in spans], [a for _, a, _ in spans], dev)
            mb = mb.on(table)
            cat = lambda k: torch.cat([seqs[i][k][a:b] for i, a, b in spans])  # noqa: E731
            q = torch.cat([pad(cat(0)[:, :, :dim], (0, d - dim)), pad(cat(0)[:, :, dim:], (0, D - d - rot))], -1)
            q = q.flatten(1).to(dev, act).contiguous()
            x = torch.cat([torch.zeros(mb.T, Q), pad(cat(1), (0, L - Lt)), pad(cat(2), (0, R - rot))], 1).to(dev, act)
            gate = pad(cat(3).view(-1, H, vdim), (0, V - vdim)).flatten(1).to(dev, act)
            o.latent_prep(x, torch.ones(Q, device=dev), Q, pad(c_w, (0, L - Lt)).to(dev), Lt, rot, eps, pool, tab, mb)
            if expand:
                lat = o.latent_gather(pool, mb)
                kv = o.gemm(lat[:, :L], kv_w.to(dev, act).contiguous())
                y = o.latent_flash(q, lat, kv, gate, tab, sink, mb, H, d, rot, L, V, m["scale"])
            else:
                a = o.latent_attn(q, o.gemm_heads(q, absorb, D), pool, tab, sink, mb, H, d, rot, L, m["scale"])
                y = o.gemm_heads(a, emit, L, gate=gate)
            y, row = y.float().cpu().view(-1, H, V), 0
            assert not y[:, :, vdim:].any()
            for i, a, b in spans:
                out[i].append(y[row:row + b - a, :, :vdim])
                row += b - a
        return [torch.cat(t) for t in out]

    def seq(self, n, seed):
        m = self.m
        H = m["heads"]
        return (rand(seed, n, H, m["dim"] + m["rot_dim"], std=1.5), rand(seed + 1, n, m["kv_rank"]), rand(seed + 2, n, m["rot_dim"]),
                rand(seed + 3, n, H * m["vdim"]))


PATHS = [pytest.param("cpu", "fp32", False, id="cpu-fp32"),
         pytest.param("cuda", "fp32", False, id="gpu-fp32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bf16", False, id="gpu-bf16", marks=pytest.mark.gpu),
         pytest.param("cuda", "bf16", True, id="gpu-bf16-expanded", marks=pytest.mark.gpu)]


@pytest.mark.parametrize("H,dim,rot,vdim,L", [(2, 32, 16, 32, 64), (5, 20, 6, 30, 100), (16, 64, 32, 64, 128), (20, 128, 64, 128, 512),
                                              (1, 8, 2, 16, 5), (33, 100, 40, 96, 250), (3, 130, 66, 40, 600), (4, 200, 64, 100, 300)])
@pytest.mark.parametrize("device,dtype,expand", PATHS)
def test_latent_attention(device, dtype, expand, H, dim, rot, vdim, L):
    if expand and not get_ops("cuda").latent_flash_fits(*LatentCase(device, dtype, H, dim, rot, vdim, L).pad[3:]):
        pytest.skip("this size is not expanded")
    c = LatentCase(device, dtype, H, dim, rot, vdim, L)
    lens = (200, 7, 131)
    seqs = [c.seq(n, 10 * i) for i, n in enumerate(lens)]
    c_w, eps = 1 + 0.3 * rand(77, L), 0.02
    steps = [[(0, 0, 63), (1, 0, 1), (2, 0, 131)], [(0, 63, 66), (1, 1, 7)], [(0, 66, 198)], [(0, 198, 199)], [(0, 199, 200)]]
    for s, got in zip(seqs, c.run(seqs, steps, c_w, eps, expand)):
        close(got, c.want(*s, c_w, eps), dtype)


@pytest.mark.parametrize("device,dtype,expand", PATHS)
@pytest.mark.parametrize("decoded", [False, True])
def test_one_key_stands_out(device, dtype, expand, decoded):
    """Queries that match one latent each (the first tokens, page borders, their own place, far away): the result is
    that token's value. Where the match lies one token ahead it must not be seen."""
    H, n, L = 2, 400, 64
    c = LatentCase(device, dtype, H, 32, 16, 32, L, scale=3.0, sink=torch.tensor([0.0, -4.0]), seed=4)
    pairs = {399: 0, 398: 1, 397: 63, 396: 64, 395: 127, 394: 128, 393: 393, 392: 391, 391: 319, 320: 320, 319: 0, 64: 63,
             63: 63, 127: 64, 128: 0, 192: 191, 0: 0, 1: 0}
    q, lat, kr, gate = c.seq(n, 30)
    q = q * 0.05
    ones = torch.ones(L)
    keys = (oracle.rms(lat, 1e-6) @ c.w["uk"].t()).view(n, H, 32)
    for i, j in {**pairs, 200: 201, 64 * 4 - 1: 64 * 4}.items():
        q[i, :, :32] = 6 * keys[j] / keys[j].norm(dim=-1, keepdim=True)
    cut = [0, *range(380, n + 1)] if decoded else [0, n]
    got, = c.run([(q, lat, kr, gate)], [[(0, a, b)] for a, b in zip(cut, cut[1:])], ones, 1e-6, expand)
    want = c.want(q, lat, kr, gate, ones, 1e-6)
    close(got, want, dtype, 2)
    v, g = (oracle.rms(lat, 1e-6) @ c.w["uv"].t()).view(n, H, 32), torch.sigmoid(gate.view(n, H, 32))
    for i, j in pairs.items():
        assert (got[i] - v[j] * g[i]).abs().max() < 0.05 * v.abs().max(), (i, j)


@pytest.mark.parametrize("device,dtype,expand", PATHS)
def test_rotation_counts_positions_from_the_start(device, dtype, expand):
    """Scores through the rotated parts alone: queries and keys that meet at one distance only, far into a sequence."""
    H, n, L, rot = 1, 330, 64, 32
    c = LatentCase(device, dtype, H, 16, rot, 32, L, base=2000.0, scale=1.0, sink=torch.tensor([-3.0]), seed=8)
    q, lat, kr, gate = c.seq(n, 40)
    q, kr = torch.zeros_like(q), torch.ones(n, rot)
    gap = 70
    turned = oracle.rotate(torch.ones(1, rot, dtype=torch.float64), [-gap], 2000.0, rot).float()  # looks back ``gap`` tokens
    q[:, 0, 16:] = 0.8 * turned
    cut = [0, 100, 101, 260, 300, *range(301, n + 1)]
    got, = c.run([(q, lat, kr, gate)], [[(0, a, b)] for a, b in zip(cut, cut[1:])], torch.ones(L), 1e-6, expand)
    close(got, c.want(q, lat, kr, gate, torch.ones(L), 1e-6), dtype, 2)


@pytest.mark.parametrize("device,dtype,expand", PATHS)
def test_sink_takes_its_share(device, dtype, expand):
    """All scores zero: the weights are 1 / (tokens + exp(sink)); a huge sink leaves nothing, a tiny one counts nothing."""
    H, n, L = 3, 130, 64
    c = LatentCase(device, dtype, H, 32, 16, 32, L, scale=0.7, sink=torch.tensor([3.0, 60.0, -60.0]), seed=9)
    q, lat, kr, gate = c.seq(n, 50)
    q, lat = torch.zeros_like(q), torch.ones(n, L)
    gate = torch.full_like(gate, 30.0)
    cut = [0, 1, 3, 128, 129, 130]
    got, = c.run([(q, lat, kr, gate)], [[(0, a, b)] for a, b in zip(cut, cut[1:])], torch.ones(L), 0.0, expand)
    v = c.w["uv"].sum(1).view(H, 32).double()
    t = torch.arange(1, n + 1, dtype=torch.float64)[:, None]
    close(got[:, 0], v[0] * t / (t + math.exp(3.0)), dtype)
    assert got[:, 1].abs().max() < 1e-6
    close(got[:, 2], v[2].expand(n, 32), dtype)


@pytest.mark.parametrize("Q,qd,L,cd", [(64, 40, 64, 50), (1664, 1650, 640, 630)])
@pytest.mark.parametrize("device,dtype", WHERE)
def test_latents_reach_their_pages(device, dtype, Q, qd, L, cd):
    """Norms and rotation of what is cached, page by page, and the normed query latent."""
    act, R, rot, n = ACT[dtype], 32, 10, 150
    ops = get_ops(device)
    x = rand(1, n, Q + L + R + 8).to(act)
    x[:, Q + cd:Q + L], x[:, Q + L + rot:Q + L + R] = 0, 0
    x[:, qd:Q] = 0
    qw, cw = torch.nn.functional.pad(rand(2, qd), (0, Q - qd)), torch.nn.functional.pad(rand(3, cd), (0, L - cd))
    table = torch.tensor([[5, 0, 3], [1, 4, 2]], dtype=torch.int32, device=device)
    pool = torch.zeros(6, PAGE, L + R, dtype=act, device=device)
    rt = RotaryTable(rot, 300.0).build(3 * PAGE, device)
    got = []
    for a, b in ((0, 65), (65, 66), (66, 150)):
        m, _ = pack_batch([b - a], [1], [a], device)
        got.append(ops.latent_prep(x[a:b].to(device), qw.to(device), qd, cw.to(device), cd, rot, 0.1, pool, rt, m.on(table)))
    xd = x.double()
    close(torch.cat(got)[:, :qd], oracle.rms(xd[:, :qd], 0.1) * qw[:qd].double(), dtype)
    rows = pool[[1, 4, 2]].flatten(0, 1)[:n].double().cpu()
    close(rows[:, :cd], oracle.rms(xd[:, Q:Q + cd], 0.1) * cw[:cd].double(), dtype)
    close(rows[:, L:L + rot], oracle.rotate(xd[:, Q + L:Q + L + rot], range(n), 300.0, rot), dtype)
    assert not rows[:, cd:L].any() and not rows[:, L + rot:].any() and not pool[[0, 3, 5]].any()


# ---------------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompts(tmp_path, name, device, dtype):
    model, cfg, w = build(tmp_path, name, device, dtype, seed=1)
    req = {n: tokens(cfg, n, n) for n in (1, 2, 65, 150)}
    got = run(model, req, [[(n, n)] for n in req])
    for n in req:
        check(got[n], expect(cfg, w, req[n]), dtype, f"{name}: prompt of {n}")


@pytest.mark.parametrize("device,dtype", WHERE)
def test_stream_after_every_layer(tmp_path, monkeypatch, device, dtype):
    model, cfg, w = build(tmp_path, "odd", device, dtype, seed=2)
    t = tokens(cfg, 70, 1)
    seen, real = [], model.ops.stream_add
    monkeypatch.setattr(model.ops, "stream_add", lambda *a, **k: seen.append(real(*a, **k)) or seen[-1])
    run(model, {"a": t}, [[("a", 70)]])
    _, want = oracle.forward(cfg, w, t)
    runs = oracle.layer_runs(cfg)
    assert len(seen) == len(runs) + 1 == model.cfg.layers + 1
    first = w["embed"][t].double() * cfg["embedding"]["scale"]
    for i, (x, _) in enumerate(seen):  # what comes ahead of the next layer run is part of the same sum
        x = x[:, :cfg["width"]].double().cpu()
        ref = first if i == 0 else want[i - 1]
        enter = runs[i][1] if i < len(runs) else None
        if enter is not None:
            ref = ref + w["loop.step"][enter].double() + (first if enter else 0)
        close(x, ref, dtype)


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("cuts", [(2,), (3, 64, 1, 29), (64, 65, 1), (63, 1, 2, 1, 130)])
def test_portions_equal_the_whole(tmp_path, name, device, dtype, cuts):
    model, cfg, w = build(tmp_path, name, device, dtype, seed=2)
    n = 40 if cuts == (2,) else 197
    req = {"a": tokens(cfg, n, 5)}
    sched, left, k = [], n, 0
    while left:
        c = min(left, cuts[k % len(cuts)])
        sched.append([("a", c)])
        left, k = left - c, k + 1
    check(run(model, req, sched)["a"], expect(cfg, w, req["a"]), dtype, f"{name} in {cuts}")


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_token_by_token_equals_the_prompt(tmp_path, name, device, dtype):
    model, cfg, w = build(tmp_path, name, device, dtype, seed=3)
    req = {"a": tokens(cfg, 140, 6)}
    check(run(model, req, [[("a", 1)]] * 140)["a"], expect(cfg, w, req["a"]), dtype, name)


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mixed_batches_reuse_slots_and_pages(tmp_path, name, device, dtype):
    """Nine requests through four slots and a pool that could not hold them all: every position equals the
    request alone."""
    model, cfg, w = build(tmp_path, name, device, dtype, seed=4)
    lens = {f"r{i}": n for i, n in enumerate((130, 5, 66, 1, 200, 64, 31, 90, 128))}
    req = {i: tokens(cfg, n, 50 + n) for i, n in lens.items()}
    got = run(model, req, mixed_schedule(lens, 7), max_seq=256, pool=4 * 200 + 64)
    for i in req:
        check(got[i], expect(cfg, w, req[i]), dtype, f"{name}: {i} of {lens[i]} tokens")


@pytest.mark.parametrize("device,dtype", [GPU16])
@pytest.mark.parametrize("at", [2, 33, 64, 1 << 20])
def test_expanded_and_absorbed_portions_agree(tmp_path, monkeypatch, device, dtype, at):
    """The same batches with keys and values expanded from 2, 33, 64 tokens on, or never."""
    monkeypatch.setattr(LatentMixer, "EXPAND_FROM", at)
    for name in ("odd", "wide"):
        model, cfg, w = build(tmp_path, name, device, dtype, seed=5)
        req = {"a": tokens(cfg, 330, 1), "b": tokens(cfg, 90, 2), "c": tokens(cfg, 2, 3)}
        got = run(model, req, [[("a", 130), ("b", 1)], [("b", 33), ("a", 1), ("c", 2)], [("b", 55), ("a", 198)], [("b", 1), ("a", 1)]])
        for i in req:
            check(got[i], expect(cfg, w, req[i]), dtype, f"{name}: {i}")


@pytest.mark.parametrize("device,dtype", WHERE)
def test_long_decoding_across_pages(tmp_path, device, dtype):
    model, cfg, w = build(tmp_path, "odd", device, dtype, seed=5)
    n = 160 if device == "cpu" else 330
    req = {"a": tokens(cfg, n, 8), "b": tokens(cfg, n - 30, 9)}
    sched = [[("a", 60), ("b", 31)]] + [[("a", 1), ("b", 1)]] * (n - 61) + [[("a", 1)]]
    got = run(model, req, sched)
    for i in req:
        check(got[i], expect(cfg, w, req[i]), dtype, i)


@pytest.mark.parametrize("device,dtype", WHERE)
def test_a_slots_earlier_owner_leaves_no_trace(tmp_path, device, dtype):
    """The same request before and after others used its slot and pages: equal to the last bit."""
    model, cfg, _ = build(tmp_path, "odd", device, dtype, seed=6)
    a, b = tokens(cfg, 90, 1), tokens(cfg, 90, 2)
    got = run(model, {"a": a, "b": b, "c": a}, [[("a", 90)], [("b", 90)], [("c", 90)]], slots=1)
    assert torch.equal(got["a"], got["c"]) and not torch.equal(got["a"], got["b"])


@pytest.mark.parametrize("loop", [(0, 3, 1), (0, 1, 4), (2, 3, 2), (1, 2, 2)])
def test_loops(tmp_path, loop):
    """At the start, at the end, of one pass: each pass has a state and a cache of its own, and one set of tensors."""
    cfg = config(40, 60, [(delta(2, 1, 16, 16), 24), (latent(2, 16, 8, 16, 24, 24), None), (delta(1, 1, 8, 24, 2), 32)], loop=loop)
    model, cfg, w = build(tmp_path, cfg, "cpu", "fp32", seed=7)
    assert [(r.weights, r.loop_pass) for r in model.cfg.runs] == oracle.layer_runs(cfg)
    assert len(model.alloc_cache(2, 64).layers) == model.cfg.layers == 3 + (loop[1] - loop[0]) * (loop[2] - 1)
    t = tokens(cfg, 50, 3)
    check(run(model, {"a": t}, [[("a", 23)], [("a", 27)]])["a"], expect(cfg, w, t), "fp32")


# ---------------------------------------------------------------------------------- generation
def greedy(cfg, w, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(oracle.forward(cfg, w, t)[0][-1].argmax()))
    return t[len(prompt):]


def sharp(w):
    w["final.norm"] = w["final.norm"] * 4  # far from ties


@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
def test_greedy_generation_through_generator_and_scheduler(tmp_path, device, dtype):
    """Generator waves and the continuous scheduler (its graphs on the GPU), both on a cache too small for all
    requests at once, and prompts in portions beside decoding rows, produce the plain implementation's tokens."""
    model, cfg, w = build(tmp_path, "odd", device, dtype, seed=8, edit=sharp)
    prompts = [tokens(cfg, n, 70 + n) for n in (3, 40, 70, 1, 66, 12, 29)]
    want = [greedy(cfg, w, p, 6) for p in prompts]
    model.alloc_cache(6, 128, tokens=6 * 64)
    g = Generator(model, max_batch=4, max_seq=128, temperature=0.0)
    assert [r.tokens for r in g.generate(prompts, 6)] == want
    sch = ContinuousScheduler(g, B=4, max_new_cap=16, chunk_steps=3)
    assert [r.tokens for r in sch.run_all(prompts, 6)] == want
    for chunk in (2, 16, 65):
        sch = ContinuousScheduler(g, B=4, max_new_cap=8, chunk_steps=2, prefill_chunk=chunk)
        assert [r.tokens for r in sch.run_all(prompts, 6)] == want
        assert sch.stats["mixed_steps"] > (70 // chunk) // 2 and not sch.filling
    g.close()
    assert len(model.cache.free) == 6 and len(model.cache.free_pages) == model.cache.pages


@pytest.mark.gpu
def test_decode_graphs_replay_the_eager_steps(tmp_path):
    """bf16: captured decode steps against eager ones over several waves with eager work in between."""
    model, cfg, _ = build(tmp_path, "wide", "cuda", "bf16", seed=9, edit=sharp)
    model.alloc_cache(10, 256)
    eager = Generator(model, max_batch=4, max_seq=256, temperature=0.0, use_graphs=False)
    graph = Generator(model, max_batch=4, max_seq=256, temperature=0.0, use_graphs=True)
    for wave in range(3):
        prompts = [tokens(cfg, n, 90 + n + wave) for n in (5, 150, 17, 64)]
        a = [r.tokens for r in eager.generate(prompts, 20)]
        torch.cuda.synchronize()
        assert a == [r.tokens for r in graph.generate(prompts, 20)]


def test_engine_serves_a_preset_and_a_checkpoint(tmp_path):
    from docagents_amd.engine.engine import Engine
    e = Engine("tiny-enc", "tiny-zamitar", "cpu", max_batch=4, max_seq=512, max_new_tokens=4, summary_max_new=4,
               use_graphs=False)
    assert isinstance(e.dec_cfg, HybridConfig) and e.describe()["decoder"] == "tiny-zamitar"
    (text, conf), = e.answer_many([("q?", [[10, 11, 12]], 0.9)], 4)
    assert isinstance(text, str) and 0 < conf <= 0.9
    out, busy = e.cb_tick([(1, ("q?", [[10, 11, 12]], 0.9))])
    while busy:
        o, busy = e.cb_tick([])
        out += o
    assert out[0][1] == text  # the scheduler and the wave path agree
    cfg = config(64, 1000, [(latent(2, 16, 8, 32, 40, 24), 64), (delta(2, 2, 16, 32), 64)])
    path = checkpoint(tmp_path, cfg, weights(cfg, 3))
    e = Engine("tiny-enc", path, "cpu", max_batch=2, max_seq=256, max_new_tokens=4, use_graphs=False, llm_dtype="fp32")
    r, = e.gen.generate([[5, 6, 7]], 4)
    assert r.n_tokens >= 1


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
def test_engine_on_the_gpu(dtype):
    from docagents_amd.engine.engine import Engine
    e = Engine("tiny-enc", "tiny-zamitar", "cuda", max_batch=4, max_seq=512, max_new_tokens=8, summary_max_new=8,
               temperature=0.0, llm_dtype=dtype)
    items = [(f"question {i}?", [list(range(10, 30 + 40 * i))], 0.9) for i in range(6)]
    wave = e.answer_many(items, 8)
    out, busy = e.cb_tick(list(enumerate(items)))
    while busy:
        o, busy = e.cb_tick([])
        out += o
    if dtype == "fp32":  # bf16: another batch size is another product kernel, near-ties may fall differently
        assert [t for _, t, _ in sorted(out)] == [t for t, _ in wave]
    assert len(out) == 6


# ---------------------------------------------------------------------------------- replay
def trace_steps(a, b):
    return [{"step": 0, "entries": [{"id": "a", "tokens": a[:70], "want": [0, 69]}, {"id": "b", "tokens": b, "want": [8]}],
             "end": ["b"]},
            {"step": 1, "entries": [{"id": "a", "tokens": a[70:71], "want": []}], "end": []},
            {"step": 2, "entries": [{"id": "a", "tokens": a[71:], "want": [8]}], "end": ["a"]}]


def check_trace(folder, cfg, w, a, b):
    ea, eb = expect(cfg, w, a), expect(cfg, w, b)
    read = lambda n: torch.from_numpy(np.fromfile(folder / f"{n}.f32", dtype="<f4")).view(-1, cfg["vocab"])  # noqa: E731
    check(read(0), torch.stack([ea[0], ea[69], eb[8]]), "fp32")
    assert not (folder / "1.f32").exists()
    check(read(2), ea[79:], "fp32")


def test_trace_replay_writes_the_wanted_rows(tmp_path):
    model, cfg, w = build(tmp_path, "odd", "cpu", "fp32", seed=11)
    a, b, done = tokens(cfg, 80, 1), tokens(cfg, 9, 2), []
    replay(model, 192, [json.dumps(s) for s in trace_steps(a, b)], str(tmp_path), done.append)
    assert done == [0, 1, 2]
    check_trace(tmp_path, cfg, w, a, b)


@pytest.mark.gpu
def test_trace_command(tmp_path):
    cfg = CONFIGS["deep"]
    w = weights(cfg, 12)
    (tmp_path / "m").mkdir(), (tmp_path / "o").mkdir()
    a, b = tokens(cfg, 80, 1), tokens(cfg, 9, 2)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model",
                        checkpoint(tmp_path / "m", cfg, w), "--dtype", "float32", "--out", str(tmp_path / "o"),
                        "--max-tokens", "192"], input="".join(json.dumps(s) + "\n" for s in trace_steps(a, b)), text=True,
                       capture_output=True, timeout=100)
    assert r.returncode == 0 and r.stdout.split() == "done 0 done 1 done 2".split(), r.stderr[-2000:]
    check_trace(tmp_path / "o", cfg, w, a, b)


# ---------------------------------------------------------------------------------- configuration, loading, state
def test_registry_and_configuration(tmp_path):
    assert isinstance(decoder_config("zamitar-8b"), HybridConfig)
    assert 8.2e9 < DECODERS["zamitar-8b"].param_count() < 8.4e9
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    c = decoder_config(checkpoint(tmp_path, cfg, w))
    assert c.layers == 8 and len(c.spec) == 4 and c.spec[0].ff == 0 and c.spec[1].ff == 100
    assert c.spec[1].mixer.decay_rank == w["l1.mix.a1"].shape[0] and c.spec[3].mixer.gate_rank == w["l3.mix.g1"].shape[0]
    assert c.param_count() == sum(v.numel() for v in w.values())
    assert c.kv_bytes_per_token() == 2 * (58 + 3 * 53)  # the looped layer keeps a cache per pass
    shapes = {k: tuple(v.shape) for k, v in w.items()}
    for change in (lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][1]["mlp"].update(kind="moe"),
                   lambda c: c["layers"][1]["mixer"].update(kv_heads=4), lambda c: c["loop"].update(stop=5),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=4), lambda c: c["loop"].update(start=3)):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises((ValueError, KeyError)):
            zamitar_config(bad, "bad", shapes=shapes)
    shapes.pop("l3.mix.a1")
    with pytest.raises(ValueError, match="l3.mix.a1"):
        zamitar_config(cfg, "bad", shapes=shapes)
    for name in ("loop.step", "l0.mix.sink", "l1.ls2", "l1.mlp.up.b"):
        bad = {k: v for k, v in w.items() if k != name}
        with pytest.raises(ValueError, match=name):
            make_decoder(checkpoint_config(str(tmp_path)), "cpu", weights=bad)


def test_layers_share_their_rotary_table():
    one, two = RotaryTable(8, 100.0), RotaryTable(8, 50.0)
    spec = [LayerState({"s": ((3,), torch.float32)}, {"k": ((PAGE, 4), torch.bfloat16)}, {"rot": t}) for t in (one, two, one)]
    c = StateCache(spec, 2, 100, "cpu")
    assert c.layers[0]["rot"] is c.layers[2]["rot"] and c.layers[1]["rot"].shape == (128, 4, 2)
    p, i = 77, 3
    assert np.allclose(c.layers[1]["rot"][p, i], [math.cos(p * 50.0 ** -0.75), math.sin(p * 50.0 ** -0.75)], atol=1e-6)
    held = {t.data_ptr(): t.numel() * t.element_size() for layer in c.layers for t in layer.values()}
    assert StateCache.bytes_for(spec, 2, 100) == sum(held.values())


def test_hbm_plan_prices_the_allocations():
    from docagents_amd.models.hybrid import HybridDecoder
    from docagents_amd.parallel import hbm_plan as HP
    cfg = decoder_config("tiny-zamitar")
    m = HybridDecoder(cfg, "cpu")
    c = m.alloc_cache(5, 300)
    held = {t.data_ptr(): t.numel() * t.element_size() for layer in c.layers for t in layer.values()}
    assert HP.kv_bytes(cfg, 5, 300) == sum(held.values()) == m.cache_bytes(5, 300)
    plan = HP.bench_plan(HP.BenchArgs(llm="zamitar-8b", batch=64), 1)
    assert HP.check(plan) == [] and plan["headline"]["decoder_weights"] == 2 * decoder_config("zamitar-8b").param_count()


def test_batches_split_by_the_portions_lengths():
    m, _ = pack_batch([1, 130, 64, 2], [2, 0, 1, 3], [9, 5, 0, 7], "cpu")
    assert m.split(None) == ((m, None), None) and m.split(200) == ((m, None), None) and m.split(1) == (None, (m, None))
    (s, sr), (g, gr) = m.split(64)
    assert sr.tolist() == [0, 195, 196] and s.cu.tolist() == [0, 1, 3] and s.slot.tolist() == [2, 3] and s.pos0.tolist() == [9, 7]
    assert gr.tolist() == list(range(1, 195)) and g.cu.tolist() == [0, 130, 194] and g.seq.tolist() == [0] * 130 + [1] * 64
    assert g.context()[0].tolist() == [0, 135, 199] and g.context()[1] == 199 and g.max_ctx == 135 and not g.singles
    assert s.max_ctx == m.max_ctx and s.singles and m.split(64)[0][0] is s  # (a single token's place may differ on the device)


def test_a_wrong_mechanism_shows():
    """The tolerance is sharp: small mistakes planted in the plain implementation exceed it by far."""
    cfg = CONFIGS["odd"]
    w = weights(cfg, 1)
    t = tokens(cfg, 100, 1)
    right = expect(cfg, w, t)
    swap = lambda a, b: {a: w[b], b: w[a]}  # noqa: E731
    plants = {"taps": {"l1.mix.q.conv": w["l1.mix.q.conv"].flip(1)}, "sink": {"l2.mix.sink": w["l2.mix.sink"] - 3},
              "decay": {"l1.mix.A_log": w["l1.mix.A_log"] + 1}, "passes": {"loop.step": w["loop.step"].flip(0)},
              "scales": swap("l1.ls1", "l1.ls2"), "bias": {"l2.mlp.gate.b": w["l2.mlp.gate.b"] * 0},
              "latent": {"l0.mix.dkv.norm": w["l0.mix.dkv.norm"].flip(0)}}
    for name, edit in plants.items():
        assert row_errors(expect(cfg, {**w, **edit}, t), right).max() > 3 * TOL["bf16"], name
    for change in (lambda c: c["layers"][2]["mixer"]["rot"].update(base=900.0), lambda c: c["loop"].update(times=2),
                   lambda c: c["embedding"].update(scale=2.0)):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        assert row_errors(expect(bad, w, t), right).max() > 100 * TOL["fp32"]
