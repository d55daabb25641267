"""Plain, slow implementation of the Zamitar decoder: one function per mechanism, float64 or float32 torch
on the CPU, no cache (a whole sequence at a time), no code shared with ``docagents_amd``.

Notation: a sequence is a matrix with one row per token; ``w`` is the dictionary of the model's tensors
(the names a checkpoint uses) and ``p`` the prefix of one layer's mixer, e.g. ``l3.mix.``.
"""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, weight, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def causal_conv(x, kernel):
    """y[t, c] = sum_k kernel[c, taps - 1 - k] * x[t - k, c], zeros before the start."""
    y = torch.zeros_like(x)
    taps = kernel.shape[1]
    for k in range(min(taps, x.shape[0])):
        y[k:] += x[:x.shape[0] - k] * kernel[:, taps - 1 - k]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def log_decay(z, A_log):
    """z [T, H, dim] (the low-rank projection with its bias) -> the logarithm of the decay."""
    return -torch.exp(A_log)[:, None] * softplus(z)


def delta_scan(q, k, v, beta, log_g, state=None):
    """q, k, log_g [T, H, K], v [T, H, V], beta [T, H] -> [T, H, V] and the state [H, K, V] after them.

    Per token and head: decay the rows of S, replace what S holds at k by a beta-weighted step towards v,
    read at q."""
    T, H, K = q.shape
    S = torch.zeros(H, K, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        S = torch.exp(log_g[t])[:, :, None] * S
        held = (S * k[t][:, :, None]).sum(1)
        u = beta[t][:, None] * (v[t] - held)
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def gated_head_norm(o, weight, gate, eps):
    """o, gate [T, H, V]; weight [V]."""
    return rms(o, eps) * weight * torch.sigmoid(gate)


def channel_delta(h, w, p, m, eps):
    T, H, G, K, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = (unit(q.view(T, G, K)) * K ** -0.5).repeat_interleave(H // G, 1)
    k = unit(k.view(T, G, K)).repeat_interleave(H // G, 1)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    o, _ = delta_scan(q, k, v.view(T, H, V), beta, log_decay(z.view(T, H, K), w[p + "A_log"]))
    gate = (h @ w[p + "g1"].T) @ w[p + "g2"].T
    return gated_head_norm(o, w[p + "norm"], gate.view(T, H, V), eps).reshape(T, -1) @ w[p + "o"].T


def rotate(x, positions, base, dims):
    """Columns i and i + dims / 2 of the first dims of x [T, ..., n] turned by position * base^(-2 i / dims)."""
    half = dims // 2
    i = torch.arange(half, dtype=torch.float64)
    a = torch.as_tensor(positions, dtype=torch.float64)[:, None] * base ** (-2 * i / dims)
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    c, s = (t.view(len(a), *[1] * (x.dim() - 2), half) for t in (c, s))
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def sink_attention(q, k, v, scale, sink):
    """q, k [T, H, d], v [T, H, dv]; the weights' denominator also holds exp(sink of the head)."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        s = (k[:t + 1] * q[t]).sum(-1) * scale            # [t + 1, H]
        top = torch.maximum(s.max(0).values, sink)
        e = torch.exp(s - top)
        out[t] = ((e / (e.sum(0) + torch.exp(sink - top)))[:, :, None] * v[:t + 1]).sum(0)
    return out


def latent_attention(h, w, p, m, eps):
    T, H, D, R, L, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"], m["vdim"]
    base, pos = m["rot"]["base"], range(T)
    cq = rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).view(T, H, D + R)
    dkv = h @ w[p + "dkv"].T
    c = rms(dkv[:, :L], eps) * w[p + "dkv.norm"]
    kr = rotate(dkv[:, L:], pos, base, m["rot"]["dims"])
    qr = rotate(q[:, :, D:], pos, base, m["rot"]["dims"])
    k = torch.cat([(c @ w[p + "uk"].T).view(T, H, D), kr[:, None].expand(T, H, R)], -1)
    o = sink_attention(torch.cat([q[:, :, :D], qr], -1), k, (c @ w[p + "uv"].T).view(T, H, V), m["scale"], w[p + "sink"])
    return (o.reshape(T, -1) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


MIXERS = {"channel_delta": channel_delta, "latent_attention": latent_attention}


def feed_forward(h, w, p):
    up = h @ w[p + "up"].T + w[p + "up.b"]
    return (silu(h @ w[p + "gate"].T + w[p + "gate.b"]) * up) @ w[p + "down"].T + w[p + "down.b"]


def layer_runs(cfg):
    """(layer, pass that starts with it or None) in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    body = [(i, t if i == loop["start"] else None) for t in range(loop["times"]) for i in range(loop["start"], loop["stop"])]
    return [(i, None) for i in range(loop["start"])] + body + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, w, tokens, dtype=torch.float64):
    """Logits [T, vocab] and the residual stream after every layer run [runs, T, width]."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    first = x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    stream = []
    for li, enter in layer_runs(cfg):
        layer, name = cfg["layers"][li], f"l{li}."
        if enter is not None:
            x = x + first if enter else x
            x = x + w["loop.step"][enter]
        h = layer_norm(x, w[name + "norm1"], eps)
        y = MIXERS[layer["type"]](h, w, name + "mix.", layer["mixer"], eps) * w[name + "ls1"]
        if layer.get("mlp"):
            y = y + feed_forward(h, w, name + "mlp.") * w[name + "ls2"]
        x = x + y
        stream.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["embed"].T, torch.stack(stream)
