"""Plain-PyTorch fp32 oracles of ``seq_kernels`` (same signatures, same in-place effects on caches and
state); the CPU execution path of the models that use them. Portions are walked one by one."""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F

from .seq_batch import PAGE, SeqBatch

ANY_NONE, ANY_SOFTPLUS, ANY_REGLU, ANY_RGLRU, ANY_SWIGLU = 0, 1, 2, 3, 4


def _portions(m: SeqBatch):
    cu, slot, pos0 = m.cu.tolist(), m.slot.tolist(), m.pos0.tolist()
    for b in range(m.B):
        yield cu[b], cu[b + 1], slot[b], pos0[b]


def _ungroup(y):
    """Columns interleaved by 16 -> the two halves."""
    yy = y.reshape(*y.shape[:-1], y.shape[-1] // 32, 2, 16)
    return yy[..., 0, :].flatten(-2), yy[..., 1, :].flatten(-2)


def gemm_any(a, w, bias=None, epi: int = ANY_NONE, coef=None):
    y = a.float() @ w.float().t()
    if bias is not None:
        y = y + bias
    if epi == ANY_SOFTPLUS:
        return F.softplus(y) if coef is None else F.softplus(y) * coef
    if epi in (ANY_REGLU, ANY_SWIGLU):
        g, u = _ungroup(y)
        return (F.relu(g) if epi == ANY_REGLU else F.silu(g)) * u
    return y


def gemm_heads(a, w, stride: int, gate=None):
    H, N, K = w.shape
    y = torch.cat([a[:, i * stride:i * stride + K].float() @ w[i].float().t() for i in range(H)], 1)
    return (y if gate is None else y * torch.sigmoid(gate.float())).to(a.dtype)


def partials_fit(M: int, N: int, K: int) -> bool:
    return False


def gemm_partials(a, w, own: bool = False):
    return (a.float() @ w.float().t())[None]


def rglru_gates(u, w, bias, lam):
    blocks, _, bw = w.shape
    ub = u.float().view(-1, blocks, bw)
    y = torch.stack([ub[:, b] @ w[b].float().t() + bias[b] for b in range(blocks)], 1)
    r, i = _ungroup(y)
    la = lam * torch.sigmoid(r.flatten(1))
    return la.exp(), torch.sqrt(-torch.expm1(2 * la)) * torch.sigmoid(i.flatten(1)) * u.float()


def stream_step(m: SeqBatch, dim: int, eps: float = 0.0, alpha: float = 1.0, ids=None, table=None, x=None, y=None,
                w=None, mu=None, prev=None, save=None, want_x: bool = True, want_h: bool = True, act=None):
    act = act or (table if ids is not None else y).dtype
    if y is not None and y.dim() == 3:
        y = y.sum(0)
    if ids is not None:
        xo = table[ids.long()].float()
    else:
        v = alpha * x + y.float()
        xo = v / torch.sqrt(v.pow(2).sum(-1, keepdim=True) / dim + eps) * w
    h = xo
    if mu is not None:
        before = torch.zeros_like(xo)
        before[1:] = xo[:-1]
        for t0, _, s, p in _portions(m):
            before[t0] = prev[s] if p > 0 else 0.0
        h = xo + (before - xo) * mu
    if save is not None:
        for _, t1, s, _ in _portions(m):
            save[s] = x[t1 - 1]
    return (xo if want_x else None), (h.to(act) if want_h else None)


def _layer_norm(x, w, eps: float, dim: int):
    v = x[:, :dim] - x[:, :dim].mean(-1, keepdim=True)
    out = torch.zeros_like(x)
    out[:, :dim] = v / torch.sqrt(v.pow(2).mean(-1, keepdim=True) + eps) * w[:dim]
    return out


def stream_add(T: int, dim: int, eps: float, act, x=None, parts=(), ids=None, table=None, embed_scale: float = 1.0,
               vec=None, w=None):
    out = None if x is None else x.clone()
    for y, scale, bias in parts:
        y = y.sum(0) if y.dim() == 3 else y.float()
        out = out + (y if bias is None else y + bias) * scale
    if ids is not None:
        e = table[ids.long()].float() * embed_scale
        out = e if out is None else out + e
    if vec is not None:
        out = out + vec
    return out, None if w is None else _layer_norm(out, w, eps, dim).to(act)


def stream_final(x, w, eps: float, dim: int, act, rows=None, center: bool = False):
    v = x if rows is None else x[rows]
    if center:
        return _layer_norm(v, w, eps, dim).to(act)
    return (v / torch.sqrt(v.pow(2).sum(-1, keepdim=True) / dim + eps) * w).to(act)


def causal_conv(x, w, bias, state, m: SeqBatch, silu: bool):
    taps = w.shape[0]
    y = torch.empty(x.shape, dtype=torch.float32)
    for t0, t1, s, p in _portions(m):
        old = state[s].float() if p > 0 else torch.zeros(taps - 1, x.shape[1])
        full = torch.cat([old, x[t0:t1].float()])
        y[t0:t1] = (0 if bias is None else bias) + sum(w[k] * full[k:k + t1 - t0] for k in range(taps))
    return (F.silu(y) if silu else y).to(x.dtype)


def _save_conv(conv_x, conv_state, t0, t1, s, p):
    keep = conv_state.shape[1]
    if keep:
        old = conv_state[s].clone() if p > 0 else torch.zeros_like(conv_state[s])
        conv_state[s] = torch.cat([old, conv_x[t0:t1]])[-keep:]


def selective_scan(x, dt, bc, off_b: int, off_c: int, z, A, D, state, conv_x, conv_state, m: SeqBatch):
    N = A.shape[1]
    y = torch.empty(x.shape, dtype=torch.float32)
    xf, B, C = x.float(), bc[:, off_b:off_b + N].float(), bc[:, off_c:off_c + N].float()
    for t0, t1, s, p in _portions(m):
        S = state[s].clone() if p > 0 else torch.zeros_like(state[s])
        for t in range(t0, t1):
            S = torch.exp2(dt[t, :, None] * A) * S + (dt[t] * xf[t])[:, None] * B[t]
            y[t] = S @ C[t] + D * xf[t]
        state[s] = S
        _save_conv(conv_x, conv_state, t0, t1, s, p)
    return (y * F.silu(z.float())).to(x.dtype)


def gated_scan(decay, drive, gate, state, conv_x, conv_state, m: SeqBatch):
    y = torch.empty(decay.shape, dtype=torch.float32)
    for t0, t1, s, p in _portions(m):
        S = state[s].clone() if p > 0 else torch.zeros_like(state[s])
        for t in range(t0, t1):
            S = decay[t] * S + drive[t]
            y[t] = S
        state[s] = S
        _save_conv(conv_x, conv_state, t0, t1, s, p)
    return (y * F.gelu(gate.float(), approximate="tanh")).to(gate.dtype)


def sigmoid_attn(qkg, kc, kr, pb, qk_w, m: SeqBatch, H: int, G: int, dim: int, scale: float, eps: float, temp=None):
    D, g = kc.shape[3], H // G
    out = torch.empty((m.T, H * D), dtype=qkg.dtype)
    table = m.table.tolist()
    for t0, t1, s, p in _portions(m):
        n = t1 - t0
        q = qkg[t0:t1, :H * D].float().view(n, H, D)
        k = qkg[t0:t1, H * D:(H + G) * D].reshape(n, G, D)
        gate = qkg[t0:t1, (H + G) * D:(H + G) * D + H].float()
        inv = lambda v: 1 / torch.sqrt(v.float().pow(2).sum(-1) / dim + eps)  # noqa: E731
        f = torch.full((n,), float(scale))
        if temp:
            f = torch.tensor([scale * (1 + temp[0] * math.log(math.floor((i + 1) / temp[1]) + 1)) for i in range(p, p + n)])
        q = (q * inv(q)[..., None] * qk_w * f[:, None, None]).to(qkg.dtype).float()
        kinv = inv(k)
        for i in range(n):
            page, r = table[s][(p + i) // PAGE], (p + i) % PAGE
            kc[page, :, r] = k[i]
            kr[page, :, r] = kinv[i]
        pages = table[s][:(p + n + PAGE - 1) // PAGE]
        ks = kc[pages].float().transpose(0, 1).reshape(G, -1, D)[:, :p + n].repeat_interleave(g, 0)
        ki = kr[pages].transpose(0, 1).reshape(G, -1)[:, :p + n].repeat_interleave(g, 0)
        sc = q.transpose(0, 1) @ ks.transpose(1, 2) * ki[:, None] + pb[:, None, None]
        wt = torch.sigmoid(sc) * torch.ones(n, p + n).tril(p)
        o = (wt @ ks).transpose(0, 1) * torch.sigmoid(gate)[..., None]
        out[t0:t1] = o.reshape(n, H * D).to(qkg.dtype)
    return out


def delta_rule(qkv, decay, beta, state, conv_x, conv_state, m: SeqBatch, H: int, G: int, q_scale: float, unit_eps: float,
               norm):
    weight, gate, dim, eps = norm
    _, _, V, K = state.shape
    g = H // G
    T = qkv.shape[0]
    unit = lambda x: x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + unit_eps)  # noqa: E731
    q = (unit(qkv[:, :G * K].float().view(T, G, K)) * q_scale).repeat_interleave(g, 1)
    k = unit(qkv[:, G * K:2 * G * K].float().reshape(T, G, K)).repeat_interleave(g, 1)
    v = qkv[:, 2 * G * K:].float().reshape(T, H, V)
    b, a = torch.sigmoid(beta[:, :H].float()), torch.exp2(decay.view(T, H, K))
    y = torch.empty(T, H, V)
    for t0, t1, s, p in _portions(m):
        S = state[s].clone() if p > 0 else torch.zeros_like(state[s])
        for t in range(t0, t1):
            S = S * a[t][:, None]
            u = b[t][:, None] * (v[t] - (S @ k[t][:, :, None])[..., 0])
            S = S + u[:, :, None] * k[t][:, None]
            y[t] = (S @ q[t][:, :, None])[..., 0]
        state[s] = S
        _save_conv(conv_x, conv_state, t0, t1, s, p)
    y = y.to(qkv.dtype).float()
    y = y / torch.sqrt(y.pow(2).sum(-1, keepdim=True) / dim + eps) * weight
    return (y.flatten(1) * torch.sigmoid(gate.float())).to(qkv.dtype)


def latent_flash_fits(D: int, V: int) -> bool:
    return False


def _turn(x, cs, R: int):
    """The first R columns of x [..., n] turned by the angles whose cos and sin are cs [..., R / 2, 2]."""
    h = R // 2
    u, v, c, s = x[..., :h], x[..., h:R], cs[..., 0], cs[..., 1]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., R:]], -1)


def latent_prep(x, q_w, q_dim: int, c_w, c_dim: int, rot_dim: int, eps: float, pages, rot, m: SeqBatch):
    Q, L, W = q_w.numel(), c_w.numel(), pages.shape[2]
    rms = lambda v, n: v / torch.sqrt(v.pow(2).sum(-1, keepdim=True) / n + eps)  # noqa: E731
    cq = rms(x[:, :Q].float(), q_dim) * q_w
    c = rms(x[:, Q:Q + L].float(), c_dim) * c_w
    kr = x[:, Q + L:Q + W].float()
    table = m.table.tolist()
    for t0, t1, s, p in _portions(m):
        row = torch.cat([c[t0:t1], _turn(kr[t0:t1], rot[p:p + t1 - t0], rot_dim)], 1).to(pages.dtype)
        for i in range(t1 - t0):
            pages[table[s][(p + i) // PAGE], (p + i) % PAGE] = row[i]
    return cq.to(x.dtype)


def latent_attn(q, ql, pages, rot, sink, m: SeqBatch, H: int, rot_at: int, rot_dim: int, L: int, scale: float):
    D = q.shape[1] // H
    out = torch.empty((m.T, H * L), dtype=q.dtype)
    table = m.table.tolist()
    for t0, t1, s, p in _portions(m):
        n = t1 - t0
        qr = q[t0:t1].float().view(n, H, D)[:, :, rot_at:rot_at + rot_dim]
        qr = _turn(qr, rot[p:p + n, None], rot_dim).to(q.dtype).float()
        c = pages[table[s][:(p + n + PAGE - 1) // PAGE]].float().flatten(0, 1)[:p + n]
        sc = ql[t0:t1].float().view(n, H, L) @ c[:, :L].t() + qr @ c[:, L:L + rot_dim].t()
        sc = (sc * scale).masked_fill(torch.ones(n, p + n).triu(p + 1)[:, None].bool(), -math.inf)
        w = torch.softmax(torch.cat([sc, sink[None, :, None].expand(n, H, 1)], -1), -1)[..., :-1]
        out[t0:t1] = (w @ c[:, :L]).reshape(n, H * L).to(q.dtype)
    return out
