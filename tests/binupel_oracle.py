"""Plain, slow implementation of the Binupel decoder: one function per mechanism, float64 or float32
torch on the CPU, no cache (a whole sequence at a time), no code shared with ``docagents_amd``.

Notation: a sequence is a matrix with one row per token; ``w`` is the dictionary of the model's
tensors (the names a checkpoint uses) and ``p`` the prefix of one layer's mixer, e.g. ``l3.mix.``.
"""
import math

import torch


def rms(x, weight, eps):
    """x / sqrt(mean(x^2) + eps), times a weight per column."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def previous_rows(x):
    """Row t holds row t - 1; row 0 holds zeros."""
    out = torch.zeros_like(x)
    out[1:] = x[:-1]
    return out


def token_shift(x, mu):
    return x + (previous_rows(x) - x) * mu


def causal_conv(x, kernel, bias):
    """y[t, c] = bias[c] + sum_k kernel[c, taps - 1 - k] * x[t - k, c], zeros before the start."""
    y = torch.zeros_like(x) + bias
    taps = kernel.shape[1]
    for k in range(min(taps, x.shape[0])):
        y[k:] += x[:x.shape[0] - k] * kernel[:, taps - 1 - k]
    return y


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def rglru_gates(u, w, p, blocks):
    """Block-diagonal gates: the recurrence gate r and the input gate i, both [T, width]."""
    bw = u.shape[1] // blocks
    r, i = torch.zeros_like(u), torch.zeros_like(u)
    for b in range(blocks):
        s = slice(b * bw, (b + 1) * bw)
        r[:, s] = torch.sigmoid(u[:, s] @ w[p + "ra"][b].T + w[p + "ra.b"][b])
        i[:, s] = torch.sigmoid(u[:, s] @ w[p + "ri"][b].T + w[p + "ri.b"][b])
    return r, i


def rglru_scan(u, r, i, lam):
    a = torch.exp(-8 * r * softplus(lam))
    drive = torch.sqrt(1 - a * a) * i * u
    s, out = torch.zeros_like(u[0]), []
    for t in range(u.shape[0]):
        s = a[t] * s + drive[t]
        out.append(s)
    return torch.stack(out)


def rglru(h, w, p, m):
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"])
    r, i = rglru_gates(u, w, p, m["blocks"])
    return (rglru_scan(u, r, i, w[p + "lam"]) * y) @ w[p + "o"].T


def query_temperature(positions, temp):
    if not temp:
        return torch.ones(len(positions), dtype=torch.float64)
    return torch.tensor([1 + temp["coef"] * math.log(math.floor((q + 1) / temp["every"]) + 1) for q in positions],
                        dtype=torch.float64)


def sigmoid_attention(q, k, v, scale, head_bias):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; key weights sigmoid(score + bias)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    seen = torch.ones(T, T, dtype=torch.bool).tril()
    for h in range(H):
        a = torch.sigmoid(q[:, h] @ k[:, h // per].T * scale + head_bias[h]) * seen
        out[:, h] = a @ v[:, h // per]
    return out


def attention(h, w, p, m, eps):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ w[p + "q"].T).view(T, H, m["dim"])
    k = (h @ w[p + "k"].T).view(T, G, m["dim"])
    v = k
    q = rms(q, w[p + "q.norm"], eps) * query_temperature(range(T), m.get("q_temp")).to(h.dtype)[:, None, None]
    k = rms(k, w[p + "k.norm"], eps)
    o = sigmoid_attention(q, k, v, m["scale"], w[p + "pb"])
    o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[p + "o"].T


def mamba1_scan(x, dt, B, C, A, D):
    """S <- exp(dt A) S + dt x B; y = S C + D x, channel by channel; A [inner, state]."""
    S, out = torch.zeros_like(A), []
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None]
        out.append(S @ C[t] + D * x[t])
    return torch.stack(out)


def mamba1(h, w, p, m):
    n, R, N = m["inner"], m["dt_rank"], m["state"]
    xz = h @ w[p + "in"].T
    x, z = xz[:, :n], xz[:, n:]
    x = causal_conv(x, w[p + "conv"], w[p + "conv.b"])
    x = x * torch.sigmoid(x)
    low = x @ w[p + "x"].T
    dt = softplus(low[:, :R] @ w[p + "dt"].T + w[p + "dt.b"])
    y = mamba1_scan(x, dt, low[:, R:R + N], low[:, R + N:], -torch.exp(w[p + "A_log"]), w[p + "D"])
    return (y * (z * torch.sigmoid(z))) @ w[p + "o"].T


def feed_forward(h, w, p):
    return (torch.relu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def forward(cfg, w, tokens, dtype=torch.float64):
    """Logits [T, vocab] and the residual stream after every layer [layers, T, width]."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"][torch.as_tensor(tokens)]
    stream = []
    for li, layer in enumerate(cfg["layers"]):
        src = layer.get("weights_of")
        name = f"l{li if src is None else src}."
        p, m = name + "mix.", layer["mixer"]
        h = token_shift(x, w[name + "shift"])
        if layer["type"] == "rglru":
            y = rglru(h, w, p, m)
        elif layer["type"] == "mamba1":
            y = mamba1(h, w, p, m)
        else:
            y = attention(h, w, p, m, eps)
        x = rms(alpha * x + y, w[name + "norm1"], eps)
        if layer.get("mlp"):
            x = rms(alpha * x + feed_forward(x, w, name + "mlp."), w[name + "norm2"], eps)
        stream.append(x)
    return rms(x, w["final.norm"], eps) @ w["head"].T, torch.stack(stream)
