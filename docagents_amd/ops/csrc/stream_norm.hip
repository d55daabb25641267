// The 32-bit residual stream of decoders with the norm after the sum:
//   x' = RMSNorm(alpha * x + y) * w            (y: the sublayer's output)
// with, in the same pass, the next sublayer's input: x' itself, or x' mixed with the previous token's
// row of the same sequence (token shift), h = x' + (x'_prev - x') * mu. The previous row of a portion's
// first token comes from the sequence's state; the kernel that next replaces the stream saves the
// portion's last row there. The stream is never updated in place: a row's neighbour reads it too.
#include "seq.h"

struct StreamArgs {
  const int* ids; const void* table; int vocab;             // EMBED: x' = table[ids]
  const float* x; const void* y; const float* w; float alpha, eps;
  int D, Dp;                                                // columns, padded columns (row stride)
  float* x_out; void* h_out;
  const float* mu; const float* prev;                       // token shift: mu [Dp], state [slots][Dp]
  float* save;                                              // state that receives x's last row per portion
  SeqMeta m;
  int rows;                                                 // consecutive tokens per workgroup
};

template <typename T, int NCH, bool EMBED>
__global__ void __launch_bounds__(256) stream_kernel(StreamArgs a) {
  __shared__ float red[16];
  const int nt = blockDim.x, nc = a.Dp / 4;
  f32x4_t cur[NCH], prv[NCH];

  auto row_of = [&](int t, f32x4_t (&v)[NCH]) {
    if constexpr (EMBED) {
      const int id = min(max(a.ids[t], 0), a.vocab - 1);
#pragma unroll
      for (int i = 0; i < NCH; ++i) {
        const int c = threadIdx.x + i * nt;
        v[i] = c < nc ? Act<T>::load4((const T*)a.table + (size_t)id * a.Dp + c * 4) : f32x4_t{0.f, 0.f, 0.f, 0.f};
      }
    } else {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < NCH; ++i) {
        const int c = threadIdx.x + i * nt;
        v[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (c < nc) {
          const f32x4_t x = *(const f32x4_t*)(a.x + (size_t)t * a.Dp + c * 4);
          const f32x4_t y = Act<T>::load4((const T*)a.y + (size_t)t * a.Dp + c * 4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            v[i][e] = fmaf(a.alpha, x[e], y[e]);
            ss = fmaf(v[i][e], v[i][e], ss);
          }
        }
      }
      const float inv = 1.f / sqrtf(block_sum(ss, red) / a.D + a.eps);
#pragma unroll
      for (int i = 0; i < NCH; ++i) {
        const int c = threadIdx.x + i * nt;
        if (c < nc) {
          const f32x4_t w = *(const f32x4_t*)(a.w + c * 4);
#pragma unroll
          for (int e = 0; e < 4; ++e) v[i][e] *= inv * w[e];
        }
      }
    }
  };

  const int t0 = blockIdx.x * a.rows;
  for (int t = t0; t < min(t0 + a.rows, a.m.T); ++t) {
    const int b = a.m.seq[t], s0 = a.m.cu[b];
    if (a.mu) {
      if (t == s0) {
        const bool start = a.m.pos0[b] == 0;
        const float* p = a.prev + (size_t)a.m.slot[b] * a.Dp;
#pragma unroll
        for (int i = 0; i < NCH; ++i) {
          const int c = threadIdx.x + i * nt;
          prv[i] = (!start && c < nc) ? *(const f32x4_t*)(p + c * 4) : f32x4_t{0.f, 0.f, 0.f, 0.f};
        }
      } else if (t == t0) {
        row_of(t - 1, prv);
      } else {
#pragma unroll
        for (int i = 0; i < NCH; ++i) prv[i] = cur[i];
      }
    }
    row_of(t, cur);
    const bool keep = a.save && t + 1 == a.m.cu[b + 1];
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const int c = threadIdx.x + i * nt;
      if (c >= nc) continue;
      if (a.x_out) *(f32x4_t*)(a.x_out + (size_t)t * a.Dp + c * 4) = cur[i];
      if (a.h_out) {
        f32x4_t h = cur[i];
        if (a.mu) {
          const f32x4_t mu = *(const f32x4_t*)(a.mu + c * 4);
#pragma unroll
          for (int e = 0; e < 4; ++e) h[e] = fmaf(prv[i][e] - cur[i][e], mu[e], cur[i][e]);
        }
        Act<T>::store4((T*)a.h_out + (size_t)t * a.Dp + c * 4, h);
      }
      if (keep)
        *(f32x4_t*)(a.save + (size_t)a.m.slot[b] * a.Dp + c * 4) = *(const f32x4_t*)(a.x + (size_t)t * a.Dp + c * 4);
    }
  }
}

// y[i] = RMSNorm(x[rows ? rows[i] : i]) * w in the activation type (the stream's final norm)
template <typename T>
__global__ void __launch_bounds__(256)
stream_final_kernel(const float* __restrict__ x, const long long* __restrict__ rows, const float* __restrict__ w,
                    float eps, int D, int Dp, T* __restrict__ y) {
  __shared__ float red[16];
  const float* r = x + (size_t)(rows ? rows[blockIdx.x] : blockIdx.x) * Dp;
  float ss = 0.f;
  for (int c = threadIdx.x; c < Dp / 4; c += blockDim.x) {
    const f32x4_t v = *(const f32x4_t*)(r + c * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss = fmaf(v[e], v[e], ss);
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / D + eps);
  for (int c = threadIdx.x; c < Dp / 4; c += blockDim.x) {
    f32x4_t v = *(const f32x4_t*)(r + c * 4);
    const f32x4_t g = *(const f32x4_t*)(w + c * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= inv * g[e];
    Act<T>::store4(y + (size_t)blockIdx.x * Dp + c * 4, v);
  }
}

template <typename T, bool EMBED>
static int launch_stream(const StreamArgs& a, hipStream_t s) {
  const int nc = a.Dp / 4;
  const int nt = nc >= 256 ? 256 : (nc + 63) / 64 * 64;
  const int nch = (nc + nt - 1) / nt;
  const dim3 grid((a.m.T + a.rows - 1) / a.rows), block(nt);
  if (nch <= 1) stream_kernel<T, 1, EMBED><<<grid, block, 0, s>>>(a);
  else if (nch <= 2) stream_kernel<T, 2, EMBED><<<grid, block, 0, s>>>(a);
  else if (nch <= 4) stream_kernel<T, 4, EMBED><<<grid, block, 0, s>>>(a);
  else if (nch <= 8) stream_kernel<T, 8, EMBED><<<grid, block, 0, s>>>(a);
  else if (nch <= 16) stream_kernel<T, 16, EMBED><<<grid, block, 0, s>>>(a);
  else return (int)hipErrorInvalidValue;
  DA_LAUNCH_CHECK();
}

// x' = norm(alpha x + y) (ids null) or table[ids] (embedding rows in the activation type); outputs
// and state as in StreamArgs, any of x_out / h_out / mu / save null. D % 4 == 0 columns of Dp.
DA_EXPORT int da_stream_step(const void* ids, const void* table, int vocab, const void* x, const void* y,
                             const void* w, float alpha, float eps, int D, int Dp, void* x_out, void* h_out,
                             const void* mu, const void* prev, void* save, const void* cu, const void* slot,
                             const void* pos0, const void* seq, int T, int B, int rows, int f32, void* stream) {
  if (T < 1 || B < 1 || rows < 1 || Dp % 4 || D < 1 || D > Dp || !cu || !slot || !pos0 || !seq || x_out == x)
    return (int)hipErrorInvalidValue;
  if (ids ? (!table || vocab < 1 || save) : (!x || !y || !w)) return (int)hipErrorInvalidValue;
  if (mu && (!prev || prev == save)) return (int)hipErrorInvalidValue;
  StreamArgs a{(const int*)ids, table, vocab, (const float*)x, y, (const float*)w, alpha, eps, D, Dp, (float*)x_out,
               h_out, (const float*)mu, (const float*)prev, (float*)save,
               SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}, rows};
  hipStream_t s = (hipStream_t)stream;
  if (f32) return ids ? launch_stream<float, true>(a, s) : launch_stream<float, false>(a, s);
  return ids ? launch_stream<bf16_t, true>(a, s) : launch_stream<bf16_t, false>(a, s);
}

DA_EXPORT int da_stream_final(const void* x, const void* rows, const void* w, float eps, int D, int Dp, void* y,
                              int n, int f32, void* stream) {
  if (n < 1 || Dp % 4 || D < 1 || D > Dp) return (int)hipErrorInvalidValue;
  if (f32)
    stream_final_kernel<float><<<n, 256, 0, (hipStream_t)stream>>>((const float*)x, (const long long*)rows,
                                                                  (const float*)w, eps, D, Dp, (float*)y);
  else
    stream_final_kernel<bf16_t><<<n, 256, 0, (hipStream_t)stream>>>((const float*)x, (const long long*)rows,
                                                                    (const float*)w, eps, D, Dp, (bf16_t*)y);
  DA_LAUNCH_CHECK();
}
