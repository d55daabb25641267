"""Bindings of the batch-of-portions kernels (``csrc/stream_norm.hip``, ``recurrent.hip``, ``delta.hip``,
``paged_attn.hip``, ``latent_attn.hip``, ``gemm_any.hip``). Re-exported by ``kernels``; the fp32 oracles with the same
signatures are in ``seq_reference``. Activations are bf16, or fp32 in the fp32 precision; the residual
stream, recurrent state, decays, step sizes and attention weights are fp32 in both."""
from __future__ import annotations


import torch

from . import kernels as K
from .kernels import _check, _ptr, _req, _stream, c_float, c_int, c_longlong, c_void_p, lib
from .seq_batch import PAGE, SeqBatch

_META = [c_void_p] * 4 + [c_int] * 2
K._SIGS.update({
    "da_gemm_any": [c_void_p, c_int, c_void_p, c_void_p, c_int, c_void_p] + [c_int] * 6 + [c_longlong] * 4
                   + [c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_int, c_void_p],
    "da_gemm_partials": [c_void_p, c_int, c_void_p] + [c_int] * 5 + [c_void_p, c_void_p],
    "da_stream_step": [c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_int, c_void_p, c_float, c_float, c_int, c_int]
                      + [c_void_p] * 5 + _META + [c_int, c_int, c_void_p],
    "da_stream_final": [c_void_p, c_void_p, c_void_p, c_float, c_int, c_int, c_int, c_void_p, c_int, c_int, c_void_p],
    "da_stream_add": [c_void_p] + [c_void_p, c_int, c_void_p, c_void_p] * 2 + [c_void_p, c_void_p, c_int, c_float]
                     + [c_void_p, c_void_p, c_float, c_int, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p],
    "da_delta_rule": [c_void_p, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_int] + [c_int] * 4
                     + [c_float, c_float, c_void_p, c_void_p, c_int, c_int, c_float, c_void_p, c_int, c_void_p] + [c_int] * 4
                     + [c_void_p, c_void_p, c_int, c_void_p] + _META + [c_int, c_void_p],
    "da_latent_prep": [c_void_p, c_int, c_void_p, c_int, c_int, c_void_p, c_int, c_int, c_int, c_int, c_float, c_void_p,
                       c_void_p, c_int, c_void_p, c_int, c_void_p, c_int] + _META + [c_int, c_void_p],
    "da_latent_attn": [c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_void_p,
                       c_void_p, c_int] + [c_int] * 6 + [c_float, c_void_p, c_void_p, c_int, c_int, c_int] + _META
                      + [c_int, c_void_p],
    "da_causal_conv": [c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int] + _META
                      + [c_int, c_void_p],
    "da_selective_scan": [c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_int, c_int, c_void_p, c_int]
                         + [c_void_p] * 4 + [c_int] * 3 + [c_void_p, c_int, c_void_p, c_int]
                         + [c_void_p] * 4 + [c_int] * 3 + _META + [c_int, c_void_p],
    "da_gated_scan": [c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p, c_int, c_void_p,
                      c_int] + [c_void_p] * 4 + [c_int] * 2 + _META + [c_int, c_void_p],
    "da_latent_gather": [c_void_p, c_int, c_void_p, c_int, c_int, c_int, c_void_p, c_int, c_void_p] + _META + [c_void_p],
    "da_latent_flash": [c_void_p, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_void_p, c_void_p,
                        c_int] + [c_int] * 7 + [c_float, c_void_p, c_int] + _META + [c_void_p],
    "da_sigmoid_attn": [c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p, c_float,
                        c_float, c_float, K.ctypes.c_double] + [c_int] * 4 + [c_void_p, c_int, c_void_p] + [c_int] * 4
                       + _META + [c_int, c_void_p],
})
K._PART_OF.update({n: "hybrid" for n in ("da_gemm_any", "da_stream_step", "da_stream_final", "da_causal_conv",
                                         "da_selective_scan", "da_gated_scan", "da_sigmoid_attn", "da_stream_add", "da_delta_rule",
                                         "da_latent_prep", "da_latent_attn", "da_latent_gather", "da_latent_flash")})

ACTS = (torch.bfloat16, torch.float32)
DELTA_CHUNK = 32       # tokens of a chunk of the delta rule on the matrix cores (bf16)
DELTA_CHUNK_FROM = 33  # tokens from which a portion runs in chunks
LATENT_WGS, LATENT_MIN_PAGES = 512, 2  # of single tokens: about so many workgroups, so many pages each
LATENT_MFMA = (64, 128, 256, 512)  # latents the matrix-core attention takes (with a key part of 32 or 64 columns)
ANY_NONE, ANY_SOFTPLUS, ANY_REGLU, ANY_RGLRU, ANY_SWIGLU, ANY_ACT = 0, 1, 2, 3, 4, 5


def _act(t, name, dtype=None):
    _req(t.is_cuda and t.dtype in ACTS and (dtype is None or t.dtype == dtype), f"{name}: bf16 / fp32 on the GPU")
    _req(t.stride(-1) == 1 and t.data_ptr() % 16 == 0, f"{name} layout")
    return int(t.dtype == torch.float32)


def _f32(t, name, numel=None):
    _req(t.is_cuda and t.dtype == torch.float32 and t.is_contiguous(), f"{name} must be contiguous fp32 on GPU")
    _req(numel is None or t.numel() == numel, f"{name}: {t.numel()} elements, want {numel}")


def _meta(m: SeqBatch):
    for t, n, name in ((m.cu, m.B + 1, "cu"), (m.slot, m.B, "slot"), (m.pos0, m.B, "pos0"), (m.seq, m.T, "seq")):
        _req(t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.numel() >= n, f"batch {name}")
    return [_ptr(m.cu), _ptr(m.slot), _ptr(m.pos0), _ptr(m.seq), m.T, m.B]


def _scratch(m: SeqBatch, waves: int, fill: int, device, *shapes):
    """Arguments of a chunked recurrence: fp32 scratch [chunks + B, *shape] each, the chunk list, its length and
    the chunk length (no scratch and no chunks where the portions are walked from end to end)."""
    n = m.chunk_len(waves, fill)
    if n == 0:
        return [], [None] * len(shapes) + [None, None, 0, 0]
    ck, base, tot = m.chunks(n)
    ws = [torch.empty((tot + m.B, *s), dtype=torch.float32, device=device) for s in shapes]
    return ws, [*map(_ptr, ws), _ptr(ck), _ptr(base), tot, n]


def gemm_any(a, w, bias=None, epi: int = ANY_NONE, coef=None):
    """fp32 [M, N'] = epi(a[M, K] @ w[N, K]^T + bias), a and w both bf16 or both fp32, bias fp32; any M and
    N, K a multiple of 16 bytes. ANY_SOFTPLUS: softplus, times coef (fp32 [N]) if given; ANY_REGLU / ANY_SWIGLU: w
    rows interleaved by 16 (gate, up)."""
    f32 = _act(a, "a")
    _act(w, "w", a.dtype)
    M, Kd = a.shape
    N = w.shape[0]
    _req(w.is_contiguous() and Kd == w.shape[1] and epi in (ANY_NONE, ANY_SOFTPLUS, ANY_REGLU, ANY_SWIGLU), "gemm_any")
    if bias is not None:
        _f32(bias, "bias", N)
    if coef is not None:
        _f32(coef, "coef", N)
        _req(epi == ANY_SOFTPLUS, "coef goes with softplus")
    out = torch.empty((M, N // 2 if epi in (ANY_REGLU, ANY_SWIGLU) else N), dtype=torch.float32, device=a.device)
    _check(lib().da_gemm_any(_ptr(a), a.stride(0), _ptr(w), _ptr(out), out.stride(0), _ptr(bias), M, N, Kd, f32, epi, 1, 0,
                             0, 0, 0, None, 0, _ptr(coef), None, None, 0, _stream()), "gemm_any")
    return out


def gemm_heads(a, w, stride: int, gate=None):
    """Per head i: a[:, i * stride : + K] @ w[i]^T for w [H, N, K] -> [M, H * N] in the activation type, times
    sigmoid(gate [M, H * N]) if given."""
    f32 = _act(a, "a")
    _act(w, "w", a.dtype)
    (H, N, Kd), M = w.shape, a.shape[0]
    _req(w.is_contiguous() and a.shape[1] >= (H - 1) * stride + Kd and stride >= Kd and N % 4 == 0, "gemm_heads operands")
    out = torch.empty((M, H * N), dtype=a.dtype, device=a.device)
    if gate is not None:
        _act(gate, "gate", a.dtype)
        _req(gate.shape == out.shape and gate.stride(0) % 4 == 0, "gate")
    _check(lib().da_gemm_any(_ptr(a), a.stride(0), _ptr(w), _ptr(out), out.stride(0), None, M, N, Kd, f32, ANY_ACT, H, stride,
                             N * Kd, N, 0, _ptr(gate), 0 if gate is None else gate.stride(0), None, None, None, 0,
                             _stream()), "gemm_heads")
    return out


def partials_fit(M: int, N: int, Kd: int) -> bool:
    """Whether a decode-sized product would run as split-K partials + a reduce launch (see ``kernels.gemm``): then
    a consumer that sums the partials itself saves that launch and a rounding."""
    return 1 < M <= 128 and not (M <= K.DK_SPLITK_ABOVE and Kd % 256 == 0)


def gemm_partials(a, w, own: bool = False):
    """bf16 a[M, K] @ w[N, K]^T as fp32 partials [splits, M, N] (their sum is the product), in the shared workspace:
    valid until the next product (own: in a buffer of their own)."""
    K._bf16_cuda(a, "a"); K._bf16_cuda(w, "w")
    M, Kd = a.shape
    N = w.shape[0]
    _req(w.shape[1] == Kd and Kd % 64 == 0 and N % 8 == 0 and M <= 128 and w.is_contiguous() and a.stride(1) == 1
         and a.stride(0) % 8 == 0 and a.data_ptr() % 16 == 0 and w.data_ptr() % 16 == 0, "gemm_partials operands")
    tile = 9 if M > 64 else K._decode_tile(M)
    splits = K._auto_splits(M, N, Kd)
    n = splits * M * N * 4
    ws = torch.empty(n, dtype=torch.uint8, device=a.device) if own else K._workspace(n, a.device)
    _check(lib().da_gemm_partials(_ptr(a), a.stride(0), _ptr(w), M, N, Kd, tile, splits, _ptr(ws), _stream()),
           "gemm_partials")
    return ws[:splits * M * N * 4].view(torch.float32).view(splits, M, N)


def rglru_gates(u, w, bias, lam):
    """Gated linear recurrence, block-diagonal gates: u [T, blocks * bw], w [blocks, 2 bw, bw] (rows of the
    recurrence and input gates interleaved by 16), bias fp32 [blocks, 2 bw], lam fp32 [C] (the log decay at
    an open recurrence gate) -> (decay, drive) fp32 [T, C]: decay = exp(lam r), drive = sqrt(1 - decay^2) i u."""
    f32 = _act(u, "u")
    _act(w, "w", u.dtype)
    blocks, bw2, bw = w.shape
    T, C = u.shape
    _req(w.is_contiguous() and bw2 == 2 * bw and blocks * bw == C and bw % 16 == 0, "gate weights [blocks, 2 bw, bw]")
    _f32(bias, "bias", blocks * bw2)
    _f32(lam, "lam", C)
    decay = torch.empty((T, C), dtype=torch.float32, device=u.device)
    drive = torch.empty_like(decay)
    _check(lib().da_gemm_any(_ptr(u), u.stride(0), _ptr(w), None, 0, _ptr(bias), T, bw2, bw, f32, ANY_RGLRU, blocks, bw,
                             bw2 * bw, 0, bw2, _ptr(u), u.stride(0), _ptr(lam), _ptr(decay), _ptr(drive), C, _stream()),
           "rglru_gates")
    return decay, drive


def stream_step(m: SeqBatch, dim: int, eps: float = 0.0, alpha: float = 1.0, ids=None, table=None, x=None, y=None,
                w=None, mu=None, prev=None, save=None, want_x: bool = True, want_h: bool = True, act=None):
    """One update of the fp32 residual stream: x' = table[ids], or RMSNorm(alpha x + y) w over ``dim`` of the
    padded columns (y [T, Dp], or its fp32 partials
    [splits, T, Dp] from ``gemm_partials``); h = x' or, with mu / prev (state [slots, Dp]),
    x' + (x'_previous token - x') mu, in the activation type. save: state [slots, Dp] that receives each portion's last row of x. -> (x', h)."""
    src = table if ids is not None else y
    f32 = _act(src, "table / y", None if src.dim() == 3 else act)
    Dp = src.shape[-1]
    dev = src.device
    splits = src.shape[0] if src.dim() == 3 else 0
    if splits:
        f32 = int(act == torch.float32)
    _req(src.is_contiguous() and Dp % 4 == 0 and dim <= Dp <= 16384, "stream columns")
    if ids is not None:
        _req(ids.dtype == torch.int32 and ids.is_contiguous() and ids.numel() >= m.T and ids.is_cuda, "ids")
    else:
        _f32(x, "x", m.T * Dp)
        _f32(w, "w", Dp)
        _req(y.shape[-2] == m.T and (not splits or y.dtype == torch.float32), "y rows")
    if mu is not None:
        _f32(mu, "mu", Dp)
        _f32(prev, "prev")
    if save is not None:
        _f32(save, "save")
    xo = torch.empty((m.T, Dp), dtype=torch.float32, device=dev) if want_x else None
    ho = torch.empty((m.T, Dp), dtype=act or src.dtype, device=dev) if want_h else None
    rows = 1 if m.T <= 2048 or mu is None else 8
    _check(lib().da_stream_step(_ptr(ids), _ptr(table), 0 if table is None else table.shape[0], _ptr(x), _ptr(y), splits,
                                _ptr(w), float(alpha), float(eps), dim, Dp, _ptr(xo), _ptr(ho), _ptr(mu), _ptr(prev), _ptr(save),
                                *_meta(m), rows, f32, _stream()), "stream_step")
    return xo, ho


def stream_add(T: int, dim: int, eps: float, act, x=None, parts=(), ids=None, table=None, embed_scale: float = 1.0,
               vec=None, w=None):
    """One update of the fp32 residual stream [T, Dp]: x' = x + sum of scale (y + bias) over ``parts`` (at most two;
    y [T, Dp] in the activation type or fp32 partials [splits, T, Dp], scale and bias fp32 [Dp], bias or None)
    + table[ids] * embed_scale + vec; h = LayerNorm(x') w over ``dim`` of the padded columns, in the activation type
    (w None: none). -> (x', h)."""
    _req(len(parts) <= 2, "stream parts")
    ref = x if x is not None else table
    Dp, dev, f32 = ref.shape[-1], ref.device, int(act == torch.float32)
    _req(Dp % 4 == 0 and dim <= Dp <= 16384, "stream columns")
    if x is not None:
        _f32(x, "x", T * Dp)
    args = []
    for y, scale, bias in (*parts, *[(None, None, None)] * (2 - len(parts))):
        splits = 0
        if y is not None:
            splits = y.shape[0] if y.dim() == 3 else 0
            _act(y, "y", torch.float32 if splits else act)
            _req(y.is_contiguous() and y.shape[-2:] == (T, Dp), "y rows")
            _f32(scale, "scale", Dp)
            if bias is not None:
                _f32(bias, "bias", Dp)
        args += [_ptr(y), splits, _ptr(scale), _ptr(bias)]
    if ids is not None:
        _act(table, "table", act)
        _req(table.is_contiguous() and table.shape[1] == Dp, "table")
        _req(ids.dtype == torch.int32 and ids.is_contiguous() and ids.numel() >= T and ids.is_cuda, "ids")
    for t, name in ((vec, "vec"), (w, "w")):
        if t is not None:
            _f32(t, name, Dp)
    xo = torch.empty((T, Dp), dtype=torch.float32, device=dev)
    ho = None if w is None else torch.empty((T, Dp), dtype=act, device=dev)
    _check(lib().da_stream_add(_ptr(x), *args, _ptr(ids), _ptr(table) if ids is not None else None,
                               0 if ids is None else table.shape[0], float(embed_scale), _ptr(vec), _ptr(w), float(eps), T,
                               dim, Dp, _ptr(xo), _ptr(ho), f32, _stream()), "stream_add")
    return xo, ho


def stream_final(x, w, eps: float, dim: int, act, rows=None, center: bool = False):
    """RMSNorm (center: LayerNorm) of the (selected: rows int64) stream rows in the activation type."""
    _f32(x, "x")
    _f32(w, "w", x.shape[1])
    if rows is not None:
        _req(rows.dtype == torch.int64 and rows.is_contiguous() and rows.is_cuda, "rows int64")
    n = x.shape[0] if rows is None else rows.numel()
    y = torch.empty((n, x.shape[1]), dtype=act, device=x.device)
    _check(lib().da_stream_final(_ptr(x), _ptr(rows), _ptr(w), float(eps), dim, x.shape[1], int(center), _ptr(y), n,
                                 int(act == torch.float32), _stream()), "stream_final")
    return y


def causal_conv(x, w, bias, state, m: SeqBatch, silu: bool):
    """Per-channel causal convolution over each portion: x [T, C] (row view), w fp32 [taps, C] (last row: the
    current token), bias fp32 [C] or None, state [slots, taps - 1, C]: the inputs before the portion, replaced here in
    batches of single tokens and by the recurrence's op otherwise."""
    f32 = _act(x, "x")
    taps, C = w.shape
    _f32(w, "w")
    if bias is not None:
        _f32(bias, "bias", C)
    _req(x.shape == (m.T, C) and x.stride(0) % 4 == 0 and C % 4 == 0, "conv input")
    _req(state.dtype == x.dtype and state.is_contiguous() and state.shape[1:] == (taps - 1, C), "conv state")
    y = torch.empty((m.T, C), dtype=x.dtype, device=x.device)
    _check(lib().da_causal_conv(_ptr(x), x.stride(0), _ptr(w), _ptr(bias), _ptr(state), _ptr(y), C, C, taps, int(silu),
                                m.max_len, *_meta(m), f32, _stream()), "causal_conv")
    return y


def _conv_args(conv_x, conv_state, C, dtype, m: SeqBatch):
    """The recurrence replaces the convolution's state, except where the convolution did (single tokens)."""
    _act(conv_x, "conv_x", dtype)
    _req(conv_state.dtype == dtype and conv_state.is_contiguous() and conv_state.shape[2] == C, "conv state")
    keep = conv_state.shape[1]
    return [_ptr(conv_x), conv_x.stride(0), _ptr(conv_state) if keep and m.max_len > 1 else None, keep + 1]


def selective_scan(x, dt, bc, off_b: int, off_c: int, z, A, D, state, conv_x, conv_state, m: SeqBatch):
    """Mamba's recurrence: x, z [T, C]; dt fp32 [T, C]; B and C rows at columns off_b / off_c of bc; A fp32
    [C, N] = log2(e) * (negative rates); D fp32 [C]; state fp32 [slots, C, N], updated, as is conv_state (from
    the convolution's inputs conv_x). -> (S C + D x) silu(z) in the activation type."""
    f32 = _act(x, "x")
    _act(z, "z", x.dtype)
    _act(bc, "bc", x.dtype)
    C, N = A.shape
    for t, n, k in ((A, "A", C * N), (D, "D", C), (dt, "dt", m.T * C), (state, "state", None)):
        _f32(t, n, k)
    _req(x.shape == (m.T, C) and z.shape == (m.T, C) and state.shape[1:] == (C, N) and N <= 512
         and max(off_b, off_c) + N <= bc.shape[1] and bc.shape[0] == m.T, "selective_scan shapes")
    y = torch.empty((m.T, C), dtype=x.dtype, device=x.device)
    ws, chunk = _scratch(m, C * -(-N // 8) // 64, 2048, x.device, (C, N), (C,))
    _check(lib().da_selective_scan(_ptr(x), x.stride(0), _ptr(dt), C, _ptr(bc), bc.stride(0), off_b, off_c, _ptr(z),
                                   z.stride(0), _ptr(A), _ptr(D), _ptr(state), _ptr(y), C, C, N,
                                   *_conv_args(conv_x, conv_state, C, x.dtype, m), *chunk, m.max_len, *_meta(m), f32,
                                   _stream()), "selective_scan")
    del ws
    return y


def gated_scan(decay, drive, gate, state, conv_x, conv_state, m: SeqBatch):
    """S <- decay S + drive per channel (fp32 [T, C]), state fp32 [slots, C] updated (and conv_state, see
    ``selective_scan``) -> S gelu_tanh(gate) in gate's type."""
    f32 = _act(gate, "gate")
    C = state.shape[1]
    for t, n, k in ((decay, "decay", m.T * C), (drive, "drive", m.T * C), (state, "state", None)):
        _f32(t, n, k)
    _req(gate.shape == (m.T, C), "gate [T, C]")
    y = torch.empty((m.T, C), dtype=gate.dtype, device=gate.device)
    ws, chunk = _scratch(m, C // 64, 16384, gate.device, (C,), (C,))
    _check(lib().da_gated_scan(_ptr(decay), _ptr(drive), _ptr(gate), gate.stride(0), _ptr(state), _ptr(y), C, C,
                               *_conv_args(conv_x, conv_state, C, gate.dtype, m), *chunk, *_meta(m), f32, _stream()),
           "gated_scan")
    del ws
    return y


def _attn_split(B: int, G: int, qtiles: int, max_ctx: int):
    """(splits, pages per split) of the single-token kernel: ~1024 workgroups, >= 4 pages (one per wave) each."""
    pages = -(-max_ctx // PAGE)
    want = max(1, min(-(-1024 // (B * G * qtiles)), -(-pages // 4)))
    pps = -(-pages // want)
    return -(-pages // pps), pps


def sigmoid_attn(qkg, kc, kr, pb, qk_w, m: SeqBatch, H: int, G: int, dim: int, scale: float, eps: float, temp=None):
    """Attention with unnormalised sigmoid weights, values = keys: qkg [T, (H + G) D + >= H] (overwritten: the
    queries are prepared in place), pages kc [pages, G, 64, D] / kr fp32 [pages, G, 64] through m.table, pb fp32
    [H] added to the scores, qk_w fp32 [D] = query norm weight * key norm weight, temp = (coef, every) of the
    query temperature 1 + coef ln(floor((p + 1) / every) + 1). Every head's output is multiplied by the sigmoid
    of its gate column. -> [T, H D]."""
    f32 = _act(qkg, "qkg")
    D = kc.shape[3]
    _act(kc, "kc", qkg.dtype)
    _f32(kr, "kr")
    _f32(pb, "pb", H)
    _f32(qk_w, "qk_w", D)
    _req(qkg.shape[0] == m.T and qkg.shape[1] >= (H + G) * D + H and qkg.stride(0) % 8 == 0, "qkg columns")
    _req(kc.is_contiguous() and kc.shape[1:3] == (G, PAGE) and kr.shape == kc.shape[:3] and D % 32 == 0, "pages")
    t = m.table
    _req(t is not None and t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.dim() == 2, "page table")
    _req(m.max_ctx <= t.shape[1] * PAGE, f"context {m.max_ctx} exceeds the page table ({t.shape[1]} pages)")
    out = torch.empty((m.T, H * D), dtype=qkg.dtype, device=qkg.device)
    nsplit, pps = _attn_split(m.B, G, -(-(H // G) // 16), m.max_ctx)
    part = None
    if not f32 and m.singles and nsplit > 1:
        part = torch.empty((m.B, H, nsplit, D), dtype=torch.float32, device=qkg.device)
    coef, every = temp if temp else (0.0, 0.0)
    _check(lib().da_sigmoid_attn(_ptr(qkg), qkg.stride(0), _ptr(kc), _ptr(kr), _ptr(t), t.shape[1], kc.shape[0], _ptr(pb),
                                 _ptr(qk_w), float(scale), float(eps), float(coef), float(every), H, G, D, dim, _ptr(out),
                                 out.stride(0), _ptr(part), nsplit if part is not None else 1,
                                 pps if part is not None else -(-m.max_ctx // PAGE), m.max_len, int(m.singles), *_meta(m),
                                 f32, _stream()), "sigmoid_attn")
    return out


def delta_chunk_bytes(K: int) -> int:
    """Scratch of a chunk and head (fragments of 1 KB)."""
    return (3 * K // 8 + 9) * 1024


def delta_rule(qkv, decay, beta, state, conv_x, conv_state, m: SeqBatch, H: int, G: int, q_scale: float, unit_eps: float,
               norm):
    """Gated delta rule: qkv [T, 2 G K + H V] (after the convolution), decay fp32 [T, H K] (log2 of each key channel's
    decay), beta [T, >= H] before its sigmoid, state fp32 [slots, H, V, K], updated (and conv_state, see
    ``selective_scan``). norm = (weight fp32 [V], gate [T, H V], true channels of a value head, eps): every head's
    read-out is RMS-normed, weighted and gated. -> [T, H V] in the activation type."""
    weight, gate, dim, eps = norm
    f32 = _act(qkv, "qkv")
    _act(beta, "beta", qkv.dtype)
    _act(gate, "gate", qkv.dtype)
    _, H2, V, Kd = state.shape
    C = 2 * G * Kd + H * V
    _f32(state, "state")
    _f32(decay, "decay", m.T * H * Kd)
    _f32(weight, "weight", V)
    _req(H2 == H and qkv.shape == (m.T, C) and qkv.stride(0) % 4 == 0 and beta.shape[0] == m.T and beta.shape[1] >= H
         and gate.shape == (m.T, H * V) and gate.stride(0) % 4 == 0 and V % 4 == 0, "delta_rule shapes")
    o = torch.empty((m.T, H * V), dtype=qkv.dtype, device=qkv.device)
    ck = base = frags = None
    n = 0
    if not f32 and Kd <= 128 and m.max_len >= DELTA_CHUNK_FROM:
        ck, base, n = m.chunks(DELTA_CHUNK)
        frags = torch.empty(n * H * delta_chunk_bytes(Kd), dtype=torch.uint8, device=qkv.device)
    _check(lib().da_delta_rule(_ptr(qkv), qkv.stride(0), _ptr(decay), _ptr(beta), beta.stride(0), _ptr(state), _ptr(o), H * V,
                               H, G, Kd, V, float(q_scale), float(unit_eps), _ptr(weight), _ptr(gate), gate.stride(0), dim,
                               float(eps), *_conv_args(conv_x, conv_state, C, qkv.dtype, m), C,
                               1 if m.lens is None else int(m.lens.min()), DELTA_CHUNK_FROM, _ptr(ck), _ptr(base), n,
                               _ptr(frags), *_meta(m), f32, _stream()), "delta_rule")
    return o


def _latent_pages(pages, rot, m: SeqBatch, rot_dim: int):
    t = m.table
    _act(pages, "pages")
    _f32(rot, "rot")
    _req(pages.is_contiguous() and pages.dim() == 3 and pages.shape[1] == PAGE, "pages")
    _req(t is not None and t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.dim() == 2, "page table")
    _req(rot.shape[1:] == (rot_dim // 2, 2) and rot.shape[0] >= t.shape[1] * PAGE, "rotary table")
    _req(m.max_ctx <= t.shape[1] * PAGE, f"context {m.max_ctx} exceeds the page table ({t.shape[1]} pages)")
    return t


def latent_prep(x, q_w, q_dim: int, c_w, c_dim: int, rot_dim: int, eps: float, pages, rot, m: SeqBatch):
    """x [T, >= Q + L + R] = [query latent | latent | key part]: the query latent RMS-normed (weight q_w fp32 [Q], over
    q_dim columns) is returned; the latent, normed likewise, and the key part, rotated, go to the token's row of
    ``pages`` [pages, 64, L + R]. rot: fp32 [positions, rot_dim / 2, 2]."""
    f32 = _act(x, "x", pages.dtype)
    Q, L, W = q_w.numel(), c_w.numel(), pages.shape[2]
    _f32(q_w, "q_w")
    _f32(c_w, "c_w")
    t = _latent_pages(pages, rot, m, rot_dim)
    _req(x.shape[0] == m.T and x.shape[1] >= Q + W and x.stride(0) % 4 == 0 and Q % 4 == 0 and L % 4 == 0 and W > L, "x")
    cq = torch.empty((m.T, Q), dtype=x.dtype, device=x.device)
    _check(lib().da_latent_prep(_ptr(x), x.stride(0), _ptr(q_w), Q, q_dim, _ptr(c_w), L, c_dim, W - L, rot_dim, float(eps),
                                _ptr(cq), _ptr(pages), pages.shape[0], _ptr(t), t.shape[1], _ptr(rot), rot.shape[0],
                                *_meta(m), f32, _stream()), "latent_prep")
    return cq


def latent_attn(q, ql, pages, rot, sink, m: SeqBatch, H: int, rot_at: int, rot_dim: int, L: int, scale: float):
    """Attention in the latent space: ql [T, H L] queries against the latents, q [T, H D] the queries whose rotated part
    (before rotation) starts at column rot_at of a head; sink fp32 [H] -> sum of weight * latent, [T, H L]."""
    f32 = _act(q, "q", pages.dtype)
    _act(ql, "ql", pages.dtype)
    _f32(sink, "sink", H)
    t = _latent_pages(pages, rot, m, rot_dim)
    D, W = q.shape[1] // H, pages.shape[2]
    _req(q.shape == (m.T, H * D) and ql.shape == (m.T, H * L) and rot_at + rot_dim <= D and L + rot_dim <= W, "query columns")
    _req(L <= 1152 and W <= 1216, f"latents of {W} columns")
    out = torch.empty((m.T, H * L), dtype=q.dtype, device=q.device)
    part, ml, rows, pages_ctx = None, None, m.max_len * H, -(-m.max_ctx // PAGE)
    nsplit, pps = 1, pages_ctx
    if not f32 and L in LATENT_MFMA and W - L in (32, 64):
        want = max(1, min(-(-LATENT_WGS // (m.B * -(-rows // 16))), -(-pages_ctx // LATENT_MIN_PAGES)))
        pps = -(-pages_ctx // want)
        nsplit = -(-pages_ctx // pps)
    if nsplit > 1:
        part = torch.empty((m.B, rows, nsplit, L), dtype=torch.float32, device=q.device)
        ml = torch.empty((m.B, rows, nsplit, 2), dtype=torch.float32, device=q.device)
    _check(lib().da_latent_attn(_ptr(q), q.stride(0), _ptr(ql), ql.stride(0), _ptr(pages), pages.shape[0], _ptr(t), t.shape[1],
                                _ptr(rot), rot.shape[0], _ptr(sink), _ptr(out), out.stride(0), H, D, rot_at, rot_dim, L, W - L,
                                float(scale), _ptr(part), _ptr(ml), nsplit, pps, m.max_len, *_meta(m), f32, _stream()),
           "latent_attn")
    return out


def latent_flash_fits(D: int, V: int) -> bool:
    """Whether ``latent_flash`` takes (padded) query / key heads of D columns and value heads of V."""
    return D in (64, 96, 128, 192, 256) and V in (32, 64, 96, 128)


def latent_gather(pages, m: SeqBatch):
    """The cache rows of every portion's context (its tokens included), packed one portion after another."""
    t, (cctx, n) = m.table, m.context()
    _act(pages, "pages", torch.bfloat16)
    _req(pages.is_contiguous() and t is not None and t.dtype == torch.int32 and t.is_contiguous(), "pages")
    W = pages.shape[2]
    lat = torch.empty((n, W), dtype=pages.dtype, device=pages.device)
    _check(lib().da_latent_gather(_ptr(pages), pages.shape[0], _ptr(t), t.shape[1], W, 0, _ptr(cctx),
                                  int((m.starts + m.lens).max()), _ptr(lat), *_meta(m), _stream()), "latent_gather")
    return lat


def latent_flash(q, lat, kv, gate, rot, sink, m: SeqBatch, H: int, d: int, rot_dim: int, L: int, V: int, scale: float):
    """Attention over expanded keys and values (bf16): q [T, H D] (d plain columns of a head, then the rotated ones before
    rotation), lat from ``latent_gather`` (rotated key parts at column L), kv [contexts, H (d + V)], gate [T, H V]
    -> softmax(with sink) values * sigmoid(gate), [T, H V]."""
    for x, name in ((q, "q"), (lat, "lat"), (kv, "kv"), (gate, "gate")):
        _act(x, name, torch.bfloat16)
    cctx, n = m.context()
    D, W = q.shape[1] // H, lat.shape[1]
    _f32(rot, "rot")
    _f32(sink, "sink", H)
    _req(latent_flash_fits(D, V) and q.shape == (m.T, H * D) and d % 8 == 0 and d + rot_dim <= D, "query columns")
    _req(lat.shape[0] == n and lat.is_contiguous() and kv.shape == (n, H * (d + V)) and W - L >= rot_dim, "keys")
    _req(gate.shape == (m.T, H * V) and rot.shape[1:] == (rot_dim // 2, 2), "gate / rotary table")
    out = torch.empty((m.T, H * V), dtype=q.dtype, device=q.device)
    _check(lib().da_latent_flash(_ptr(q), q.stride(0), _ptr(lat), _ptr(kv), kv.stride(0), _ptr(gate), gate.stride(0),
                                 _ptr(rot), rot.shape[0], _ptr(sink), _ptr(out), out.stride(0), H, D, d, rot_dim, L, W - L,
                                 V, float(scale), _ptr(cctx), m.max_len, *_meta(m), _stream()), "latent_flash")
    return out
