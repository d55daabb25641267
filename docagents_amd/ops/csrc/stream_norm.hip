// The 32-bit residual stream.
//
// stream_add, for decoders with one norm ahead of parallel sublayers:
//   x' = x + sum_i s_i (y_i + b_i) (+ embedding rows, + a vector),  h = LayerNorm(x') * w
//
// stream_step, for decoders with the norm after the sum:
//   x' = RMSNorm(alpha * x + y) * w            (y: the sublayer's output)
// with, in the same pass, the next sublayer's input: x' itself, or x' mixed with the previous token's
// row of the same sequence (token shift), h = x' + (x'_prev - x') * mu. The previous row of a portion's
// first token comes from the sequence's state; the kernel that next replaces the stream saves the
// portion's last row there. The stream is never updated in place: a row's neighbour reads it too.
#include "seq.h"

struct StreamArgs {
  const int* ids; const void* table; int vocab;             // embedding: x' = table[ids]
  const float* x; const void* y; const float* w; float alpha, eps;
  int splits;                                               // y is the sum of `splits` fp32 [T][Dp] partials
  int D, Dp;                                                // columns, padded columns (row stride)
  float* x_out; void* h_out;
  const float* mu; const float* prev;                       // token shift: mu [Dp], state [slots][Dp]
  float* save;                                              // state that receives x's last row per portion
  SeqMeta m;
  int rows;                                                 // consecutive tokens per workgroup
};

enum StreamSrc : int { SRC_EMBED = 0, SRC_Y = 1, SRC_PARTIALS = 2 };

// A thread holds NCH 4-column pieces of a row. The next row's loads are issued before this row's sum.
template <typename T, int NCH, int SRC>
__global__ void __launch_bounds__(NCH == 1 ? 1024 : 256) stream_kernel(StreamArgs a) {
  __shared__ float red[16];
  const int nt = blockDim.x, nc = a.Dp / 4;
  f32x4_t nx[NCH], cur[NCH], prv[NCH];

  auto col = [&](int i) { return (int)threadIdx.x + i * nt; };  // this thread's i-th piece
  auto fetch = [&](int t) {  // alpha x + y of row t (embedding: the row itself) into nx
    const size_t src = SRC == SRC_EMBED ? min(max(a.ids[t], 0), a.vocab - 1) : t;
    if constexpr (SRC == SRC_PARTIALS) {
#pragma unroll
      for (int i = 0; i < NCH; ++i) nx[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      constexpr int U = NCH <= 2 ? 8 : 4;  // partials of every piece in flight together
      const size_t st = (size_t)a.m.T * a.Dp;
      for (int s0 = 0; s0 < a.splits; s0 += U) {
        f32x4_t v[U][NCH];
#pragma unroll
        for (int s = 0; s < U; ++s)
#pragma unroll
          for (int i = 0; i < NCH; ++i)
            v[s][i] = *(const f32x4_t*)((const float*)a.y + min(s0 + s, a.splits - 1) * st + src * a.Dp +
                                        min(col(i), nc - 1) * 4);
#pragma unroll
        for (int s = 0; s < U; ++s)
#pragma unroll
          for (int i = 0; i < NCH; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) nx[i][e] += s0 + s < a.splits ? v[s][i][e] : 0.f;
      }
    }
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const int c = min(col(i), nc - 1) * 4;
      if constexpr (SRC == SRC_EMBED) {
        nx[i] = Act<T>::load4((const T*)a.table + src * a.Dp + c);
      } else {
        const f32x4_t y = SRC == SRC_Y ? Act<T>::load4((const T*)a.y + src * a.Dp + c) : nx[i];
        const f32x4_t x = *(const f32x4_t*)(a.x + src * a.Dp + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) nx[i][e] = fmaf(a.alpha, x[e], y[e]);
      }
    }
  };
  auto normed = [&](f32x4_t (&v)[NCH]) {  // v = the fetched row, normalised; then nx is free
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      v[i] = nx[i];
      if (SRC != SRC_EMBED && col(i) < nc)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss = fmaf(v[i][e], v[i][e], ss);
    }
    return ss;
  };
  auto scale = [&](f32x4_t (&v)[NCH], float ss) {
    if constexpr (SRC == SRC_EMBED) return;
    const float inv = 1.f / sqrtf(block_sum(ss, red) / a.D + a.eps);
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const f32x4_t w = *(const f32x4_t*)(a.w + min(col(i), nc - 1) * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] *= inv * w[e];
    }
  };

  const int t0 = blockIdx.x * a.rows, t1 = min(t0 + a.rows, a.m.T);
  const bool redo = a.mu && t0 != a.m.cu[a.m.seq[t0]];  // the row before the first one is a neighbour's
  fetch(redo ? t0 - 1 : t0);
  if (redo) {
    const float ss = normed(prv);
    fetch(t0);
    scale(prv, ss);
  }
  for (int t = t0; t < t1; ++t) {
    const int b = a.m.seq[t];
    if (a.mu && t == a.m.cu[b]) {
      const bool start = a.m.pos0[b] == 0;
      const float* p = a.prev + (size_t)a.m.slot[b] * a.Dp;
#pragma unroll
      for (int i = 0; i < NCH; ++i) {
        prv[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (!start) prv[i] = *(const f32x4_t*)(p + min(col(i), nc - 1) * 4);
      }
    }
    const float ss = normed(cur);
    if (t + 1 < t1) fetch(t + 1);
    scale(cur, ss);
    const bool keep = a.save && t + 1 == a.m.cu[b + 1];
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const int c = col(i) * 4;
      if (c >= a.Dp) continue;
      if (a.x_out) *(f32x4_t*)(a.x_out + (size_t)t * a.Dp + c) = cur[i];
      if (a.h_out) {
        f32x4_t h = cur[i];
        if (a.mu) {
          const f32x4_t mu = *(const f32x4_t*)(a.mu + c);
#pragma unroll
          for (int e = 0; e < 4; ++e) h[e] = fmaf(prv[i][e] - cur[i][e], mu[e], cur[i][e]);
        }
        Act<T>::store4((T*)a.h_out + (size_t)t * a.Dp + c, h);
      }
      if (keep) *(f32x4_t*)(a.save + (size_t)a.m.slot[b] * a.Dp + c) = *(const f32x4_t*)(a.x + (size_t)t * a.Dp + c);
      prv[i] = cur[i];
    }
  }
}

// ------------------------------------------------------------------------------- parallel sublayers
struct AddPart {
  const void* y; int splits;            // [T][Dp] in the activation type, or `splits` fp32 partials of it
  const float* scale; const float* bias;  // [Dp], bias nullable
};
struct AddArgs {
  const float* x;                       // nullable
  AddPart part[2]; int nparts;
  const int* ids; const void* table; int vocab; float embed_scale;  // + table[ids] * embed_scale (ids nullable)
  const float* vec;                     // + vec [Dp] (nullable)
  const float* w; float eps;            // null: no norm
  int T, D, Dp;
  float* x_out; void* h_out;
};

// A row per workgroup, NCH 4-column pieces per thread; the row stays in registers through the norm's two sums.
template <typename T, int NCH>
__global__ void __launch_bounds__(NCH == 1 ? 1024 : 256) stream_add_kernel(AddArgs a) {
  __shared__ float red[16];
  const int nt = blockDim.x, nc = a.Dp / 4, t = blockIdx.x;
  f32x4_t v[NCH];
  auto col = [&](int i) { return (int)threadIdx.x + i * nt; };
  auto at = [&](int i) { return min(col(i), nc - 1) * 4; };
#pragma unroll
  for (int i = 0; i < NCH; ++i) {
    v[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (a.x) v[i] = *(const f32x4_t*)(a.x + (size_t)t * a.Dp + at(i));
  }
#pragma unroll
  for (int p = 0; p < 2; ++p) {
    if (p >= a.nparts) break;
    const AddPart& q = a.part[p];
    f32x4_t y[NCH];
    if (q.splits) {
#pragma unroll
      for (int i = 0; i < NCH; ++i) y[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      constexpr int U = NCH <= 2 ? 8 : 4;  // partials of every piece in flight together
      const size_t st = (size_t)a.T * a.Dp;
      for (int s0 = 0; s0 < q.splits; s0 += U) {
        f32x4_t u[U][NCH];
#pragma unroll
        for (int s = 0; s < U; ++s)
#pragma unroll
          for (int i = 0; i < NCH; ++i)
            u[s][i] = *(const f32x4_t*)((const float*)q.y + min(s0 + s, q.splits - 1) * st + (size_t)t * a.Dp + at(i));
#pragma unroll
        for (int s = 0; s < U; ++s)
#pragma unroll
          for (int i = 0; i < NCH; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) y[i][e] += s0 + s < q.splits ? u[s][i][e] : 0.f;
      }
    } else {
#pragma unroll
      for (int i = 0; i < NCH; ++i) y[i] = Act<T>::load4((const T*)q.y + (size_t)t * a.Dp + at(i));
    }
    if (q.bias) {
#pragma unroll
      for (int i = 0; i < NCH; ++i) y[i] += *(const f32x4_t*)(q.bias + at(i));
    }
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const f32x4_t s = *(const f32x4_t*)(q.scale + at(i));
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] = fmaf(y[i][e], s[e], v[i][e]);
    }
  }
  if (a.ids) {
    const T* row = (const T*)a.table + (size_t)min(max(a.ids[t], 0), a.vocab - 1) * a.Dp;
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const f32x4_t e4 = Act<T>::load4(row + at(i));
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] = fmaf(e4[e], a.embed_scale, v[i][e]);
    }
  }
  if (a.vec) {
#pragma unroll
    for (int i = 0; i < NCH; ++i) v[i] += *(const f32x4_t*)(a.vec + at(i));
  }
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < NCH; ++i) {
    if (col(i) >= nc) continue;
    *(f32x4_t*)(a.x_out + (size_t)t * a.Dp + at(i)) = v[i];
#pragma unroll
    for (int e = 0; e < 4; ++e) sum += v[i][e];  // padding columns hold zeros
  }
  if (!a.w) return;
  const float mean = block_sum(sum, red) / a.D;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NCH; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[i][e] = col(i) * 4 + e < a.D ? v[i][e] - mean : 0.f;
      ss = fmaf(v[i][e], v[i][e], ss);
    }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / a.D + a.eps);
#pragma unroll
  for (int i = 0; i < NCH; ++i) {
    if (col(i) >= nc) continue;
    const f32x4_t w = *(const f32x4_t*)(a.w + at(i));
#pragma unroll
    for (int e = 0; e < 4; ++e) v[i][e] *= inv * w[e];
    Act<T>::store4((T*)a.h_out + (size_t)t * a.Dp + at(i), v[i]);
  }
}

template <typename T>
static int launch_add(const AddArgs& a, hipStream_t s) {
  const int nc = a.Dp / 4;
  const int most = a.T <= 512 ? 1024 : 256, nt = nc >= most ? (nc > 1024 ? 256 : most) : (nc + 63) / 64 * 64;
  const int nch = (nc + nt - 1) / nt;
  if (nch <= 1) stream_add_kernel<T, 1><<<a.T, nt, 0, s>>>(a);
  else if (nch <= 2) stream_add_kernel<T, 2><<<a.T, nt, 0, s>>>(a);
  else if (nch <= 4) stream_add_kernel<T, 4><<<a.T, nt, 0, s>>>(a);
  else if (nch <= 8) stream_add_kernel<T, 8><<<a.T, nt, 0, s>>>(a);
  else if (nch <= 16) stream_add_kernel<T, 16><<<a.T, nt, 0, s>>>(a);
  else return (int)hipErrorInvalidValue;
  DA_LAUNCH_CHECK();
}

// x may be x_out (a row's reads precede its writes). D of Dp columns, Dp % 4 == 0; columns past D of every operand
// hold zeros.
DA_EXPORT int da_stream_add(const void* x, const void* y0, int splits0, const void* scale0, const void* bias0,
                            const void* y1, int splits1, const void* scale1, const void* bias1, const void* ids,
                            const void* table, int vocab, float embed_scale, const void* vec, const void* w, float eps,
                            int T, int D, int Dp, void* x_out, void* h_out, int f32, void* stream) {
  if (T < 1 || Dp % 4 || D < 1 || D > Dp || !x_out || (w && !h_out) || splits0 < 0 || splits1 < 0)
    return (int)hipErrorInvalidValue;
  if ((ids && (!table || vocab < 1)) || (y0 && !scale0) || (y1 && (!y0 || !scale1)) || (!x && !ids && !y0))
    return (int)hipErrorInvalidValue;
  AddArgs a{};
  a.x = (const float*)x;
  a.part[0] = AddPart{y0, splits0, (const float*)scale0, (const float*)bias0};
  a.part[1] = AddPart{y1, splits1, (const float*)scale1, (const float*)bias1};
  a.nparts = y1 ? 2 : y0 ? 1 : 0;
  a.ids = (const int*)ids; a.table = table; a.vocab = vocab; a.embed_scale = embed_scale;
  a.vec = (const float*)vec; a.w = (const float*)w; a.eps = eps;
  a.T = T; a.D = D; a.Dp = Dp;
  a.x_out = (float*)x_out; a.h_out = h_out;
  return f32 ? launch_add<float>(a, (hipStream_t)stream) : launch_add<bf16_t>(a, (hipStream_t)stream);
}

// y[i] = norm(x[rows ? rows[i] : i]) * w in the activation type (the stream's final norm): RMSNorm, or with
// `center` LayerNorm
template <typename T>
__global__ void __launch_bounds__(256)
stream_final_kernel(const float* __restrict__ x, const long long* __restrict__ rows, const float* __restrict__ w,
                    float eps, int D, int Dp, int center, T* __restrict__ y) {
  __shared__ float red[16];
  const float* r = x + (size_t)(rows ? rows[blockIdx.x] : blockIdx.x) * Dp;
  float mean = 0.f;
  if (center) {
    float sum = 0.f;
    for (int c = threadIdx.x; c < Dp / 4; c += blockDim.x) {
      const f32x4_t v = *(const f32x4_t*)(r + c * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) sum += v[e];
    }
    mean = block_sum(sum, red) / D;
  }
  float ss = 0.f;
  for (int c = threadIdx.x; c < Dp / 4; c += blockDim.x) {
    const f32x4_t v = *(const f32x4_t*)(r + c * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float d = c * 4 + e < D ? v[e] - mean : 0.f;
      ss = fmaf(d, d, ss);
    }
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / D + eps);
  for (int c = threadIdx.x; c < Dp / 4; c += blockDim.x) {
    f32x4_t v = *(const f32x4_t*)(r + c * 4);
    const f32x4_t g = *(const f32x4_t*)(w + c * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (v[e] - mean) * (inv * g[e]);  // padding: w is zero
    Act<T>::store4(y + (size_t)blockIdx.x * Dp + c * 4, v);
  }
}

template <typename T, int SRC>
static int launch_stream(const StreamArgs& a, hipStream_t s) {
  const int nc = a.Dp / 4;
  // few rows: a row over as many threads as it has pieces (latency); else 256 threads a row
  const int most = a.m.T <= 512 ? 1024 : 256, nt = nc >= most ? (nc > 1024 ? 256 : most) : (nc + 63) / 64 * 64;
  const int nch = (nc + nt - 1) / nt;
  const dim3 grid((a.m.T + a.rows - 1) / a.rows), block(nt);
  if (nch <= 1) stream_kernel<T, 1, SRC><<<grid, block, 0, s>>>(a);
  else if (nch <= 2) stream_kernel<T, 2, SRC><<<grid, block, 0, s>>>(a);
  else if (nch <= 4) stream_kernel<T, 4, SRC><<<grid, block, 0, s>>>(a);
  else if (nch <= 8) stream_kernel<T, 8, SRC><<<grid, block, 0, s>>>(a);
  else if (nch <= 16) stream_kernel<T, 16, SRC><<<grid, block, 0, s>>>(a);
  else return (int)hipErrorInvalidValue;
  DA_LAUNCH_CHECK();
}

// x' = norm(alpha x + y) (ids null) or table[ids] (embedding rows in the activation type); outputs
// and state as in StreamArgs, any of x_out / h_out / mu / save null. splits > 0: y holds that many fp32
// partials. D of Dp columns, Dp % 4 == 0.
DA_EXPORT int da_stream_step(const void* ids, const void* table, int vocab, const void* x, const void* y, int splits,
                             const void* w, float alpha, float eps, int D, int Dp, void* x_out, void* h_out,
                             const void* mu, const void* prev, void* save, const void* cu, const void* slot,
                             const void* pos0, const void* seq, int T, int B, int rows, int f32, void* stream) {
  if (T < 1 || B < 1 || rows < 1 || Dp % 4 || D < 1 || D > Dp || !cu || !slot || !pos0 || !seq || splits < 0)
    return (int)hipErrorInvalidValue;
  if (ids ? (!table || vocab < 1 || save) : (!x || !y || !w || x_out == x)) return (int)hipErrorInvalidValue;
  if (mu && (!prev || prev == save)) return (int)hipErrorInvalidValue;
  StreamArgs a{(const int*)ids, table, vocab, (const float*)x, y, (const float*)w, alpha, eps, splits, D, Dp,
               (float*)x_out, h_out, (const float*)mu, (const float*)prev, (float*)save,
               SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}, rows};
  hipStream_t s = (hipStream_t)stream;
  if (f32) return ids ? launch_stream<float, SRC_EMBED>(a, s)
                      : splits ? launch_stream<float, SRC_PARTIALS>(a, s) : launch_stream<float, SRC_Y>(a, s);
  return ids ? launch_stream<bf16_t, SRC_EMBED>(a, s)
             : splits ? launch_stream<bf16_t, SRC_PARTIALS>(a, s) : launch_stream<bf16_t, SRC_Y>(a, s);
}

DA_EXPORT int da_stream_final(const void* x, const void* rows, const void* w, float eps, int D, int Dp, int center,
                              void* y, int n, int f32, void* stream) {
  if (n < 1 || Dp % 4 || D < 1 || D > Dp) return (int)hipErrorInvalidValue;
  if (f32)
    stream_final_kernel<float><<<n, 256, 0, (hipStream_t)stream>>>((const float*)x, (const long long*)rows,
                                                                  (const float*)w, eps, D, Dp, center, (float*)y);
  else
    stream_final_kernel<bf16_t><<<n, 256, 0, (hipStream_t)stream>>>((const float*)x, (const long long*)rows,
                                                                    (const float*)w, eps, D, Dp, center, (bf16_t*)y);
  DA_LAUNCH_CHECK();
}
