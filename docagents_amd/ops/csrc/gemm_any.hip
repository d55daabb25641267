// Matrix products of any M, N and K that keep fp32 results: C[M, N] = epi(A[M, K] . W[N, K]^T), with
// bf16 or fp32 operands (v_mfma_f32_16x16x32_bf16 / v_mfma_f32_16x16x4_f32: both accumulate in fp32, the
// fp32 form multiplies true fp32), batched over blockIdx.z. The serving precision uses it where a
// product feeds a recurrence (step sizes, gates), which must not be rounded to 16 bits; everything
// else runs on gemm.hip's kernels. The fp32 precision runs every product here.
//
// BT x BT tile (64, or 128 where the rows fill the chip), 4 waves of a quarter each, K in 128-byte slices through double-buffered LDS (rows padded to 144
// bytes: conflict-free 16-byte reads), the next slice's loads in flight while this one is multiplied.
#include "seq.h"

enum AnyEpi : int {
  ANY_NONE = 0,      // + bias
  ANY_SOFTPLUS = 1,  // softplus(x + bias), fp32 out
  ANY_REGLU = 2,     // W rows interleaved in 16-row (gate, up) groups: relu(g) * u
  ANY_RGLRU = 3,     // W rows interleaved in 16-row (recurrence, input) gate groups of one block
};

struct AnyArgs {
  const void* A; const void* W; void* C; const float* bias;
  int M, N, K, lda, ldc;
  long long sA, sW, sC, sBias;  // strides between the products of a batch, in elements
  // ANY_RGLRU: decay factors and driving terms of the recurrence, from the gates and its input u
  const void* u; const float* lam; float* decay; float* drive; int ldu, ldg;
};

constexpr int ANY_ROWB = 144;

template <typename T, int EPI, int BT>
__global__ void __launch_bounds__(256) gemm_any_kernel(AnyArgs p) {
  constexpr int TILEB = BT * ANY_ROWB, WT = BT / 2, F = BT / 32, LP = BT / 32;  // wave tile, its 16-blocks, pieces
  extern __shared__ __attribute__((aligned(16))) char sm[];
  constexpr int E16 = 16 / sizeof(T), KS = 128 / sizeof(T);  // elements per 16 bytes, per slice
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, wm = wv >> 1, wn = wv & 1;
  const int fr = lane & 15, fg = lane >> 4;
  const int n0 = blockIdx.x * BT, m0 = blockIdx.y * BT, z = blockIdx.z;
  const T* A = (const T*)p.A + z * p.sA;
  const T* W = (const T*)p.W + z * p.sW;

  // BT * 8 16-byte pieces per operand slice: thread tid carries pieces tid, tid + 256, ...
  u32x4_t ra[LP], rw[LP];
  auto load = [&](int k0) {
#pragma unroll
    for (int i = 0; i < LP; ++i) {
      const int pc = tid + 256 * i, row = pc >> 3, k = k0 + (pc & 7) * E16;
      const bool kin = k < p.K;
      const int kk = kin ? k : 0;
      const u32x4_t va = *(const u32x4_t*)(A + (size_t)min(m0 + row, p.M - 1) * p.lda + kk);
      const u32x4_t vw = *(const u32x4_t*)(W + (size_t)min(n0 + row, p.N - 1) * p.K + kk);
      ra[i] = (kin && m0 + row < p.M) ? va : u32x4_t{0, 0, 0, 0};
      rw[i] = (kin && n0 + row < p.N) ? vw : u32x4_t{0, 0, 0, 0};
    }
  };
  auto store = [&](int buf) {
#pragma unroll
    for (int i = 0; i < LP; ++i) {
      const int pc = tid + 256 * i, off = (pc >> 3) * ANY_ROWB + (pc & 7) * 16;
      *(u32x4_t*)(sm + buf * 2 * TILEB + off) = ra[i];
      *(u32x4_t*)(sm + buf * 2 * TILEB + TILEB + off) = rw[i];
    }
  };
  f32x4_t acc[F][F];
#pragma unroll
  for (int i = 0; i < F; ++i)
#pragma unroll
    for (int j = 0; j < F; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  const int nk = (p.K + KS - 1) / KS;
  load(0);
  store(0);
  __syncthreads();
  for (int s = 0; s < nk; ++s) {
    if (s + 1 < nk) load((s + 1) * KS);
    const char* sa = sm + (s & 1) * 2 * TILEB;
    const char* sw = sa + TILEB;
    if constexpr (sizeof(T) == 2) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        bf16x8_t fa[F], fw[F];
#pragma unroll
        for (int i = 0; i < F; ++i) {
          fa[i] = *(const bf16x8_t*)(sa + (wm * WT + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
          fw[i] = *(const bf16x8_t*)(sw + (wn * WT + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
        }
#pragma unroll
        for (int i = 0; i < F; ++i)
#pragma unroll
          for (int j = 0; j < F; ++j) acc[i][j] = mfma16(fw[j], fa[i], acc[i][j]);
      }
    } else {
      // a lane group's four consecutive k of a 16-k step go to four MFMAs (the same k of both operands)
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        f32x4_t fa[F], fw[F];
#pragma unroll
        for (int i = 0; i < F; ++i) {
          fa[i] = *(const f32x4_t*)(sa + (wm * WT + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
          fw[i] = *(const f32x4_t*)(sw + (wn * WT + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int i = 0; i < F; ++i)
#pragma unroll
            for (int j = 0; j < F; ++j)
              acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(fw[j][e], fa[i][e], acc[i][j], 0, 0, 0);
      }
    }
    if (s + 1 < nk) store((s + 1) & 1);
    __syncthreads();
  }

  // W is the MFMA's first operand: lane (fr, fg) holds row fr, columns 4 fg .. 4 fg + 3 of each 16 x 16 block
  const float* bias = p.bias ? p.bias + z * p.sBias : nullptr;
  const f32x4_t zero{0.f, 0.f, 0.f, 0.f};
  if constexpr (EPI == ANY_REGLU || EPI == ANY_RGLRU) {
#pragma unroll
    for (int jp = 0; jp < F / 2; ++jp) {
      const int nb = n0 + wn * WT + jp * 32;
      if (nb >= p.N) continue;
      const int col = nb / 2 + 4 * fg;
      const f32x4_t b0 = bias ? *(const f32x4_t*)(bias + nb + 4 * fg) : zero;
      const f32x4_t b1 = bias ? *(const f32x4_t*)(bias + nb + 16 + 4 * fg) : zero;
      const int ch = z * (p.N / 2) + col;
      const f32x4_t lam = EPI == ANY_RGLRU ? *(const f32x4_t*)(p.lam + ch) : zero;
#pragma unroll
      for (int i = 0; i < F; ++i) {
        const int m = m0 + wm * WT + i * 16 + fr;
        if (m >= p.M) continue;
        const f32x4_t x = acc[i][2 * jp] + b0, y = acc[i][2 * jp + 1] + b1;
        f32x4_t r, d;
        if constexpr (EPI == ANY_REGLU) {
#pragma unroll
          for (int e = 0; e < 4; ++e) r[e] = fmaxf(x[e], 0.f) * y[e];
          *(f32x4_t*)((float*)p.C + z * p.sC + (size_t)m * p.ldc + col) = r;
        } else {
          const f32x4_t u = Act<T>::load4((const T*)p.u + (size_t)m * p.ldu + ch);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float la = lam[e] * sigmoid32(x[e]);  // log of the decay, <= 0
            r[e] = exp32(la);
            d[e] = __builtin_amdgcn_sqrtf(one_minus_exp32(2.f * la)) * sigmoid32(y[e]) * u[e];
          }
          *(f32x4_t*)(p.decay + (size_t)m * p.ldg + ch) = r;
          *(f32x4_t*)(p.drive + (size_t)m * p.ldg + ch) = d;
        }
      }
    }
  } else {
    float* C = (float*)p.C + z * p.sC;
    const bool vec = (p.N & 3) == 0 && (p.ldc & 3) == 0;
#pragma unroll
    for (int j = 0; j < F; ++j) {
      const int n = n0 + wn * WT + j * 16 + 4 * fg;
      if (n >= p.N) continue;
      f32x4_t b = zero;
      if (bias)
#pragma unroll
        for (int e = 0; e < 4; ++e) b[e] = bias[min(n + e, p.N - 1)];
#pragma unroll
      for (int i = 0; i < F; ++i) {
        const int m = m0 + wm * WT + i * 16 + fr;
        if (m >= p.M) continue;
        f32x4_t v = acc[i][j] + b;
        if constexpr (EPI == ANY_SOFTPLUS)
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = softplus32(v[e]);
        float* o = C + (size_t)m * p.ldc + n;
        if (vec) {
          *(f32x4_t*)o = v;
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (n + e < p.N) o[e] = v[e];
        }
      }
    }
  }
}

template <typename T, int EPI, int BT>
static int launch_any(const AnyArgs& a, int batch, hipStream_t s) {
  constexpr int lds = 4 * BT * ANY_ROWB;
  if (lds > 65536) {
    static const hipError_t e = hipFuncSetAttribute((const void*)gemm_any_kernel<T, EPI, BT>,
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (e != hipSuccess) return (int)e;
  }
  gemm_any_kernel<T, EPI, BT><<<dim3((a.N + BT - 1) / BT, (a.M + BT - 1) / BT, batch), 256, lds, s>>>(a);
  DA_LAUNCH_CHECK();
}
template <typename T, int EPI>
static int launch_any_t(const AnyArgs& a, int batch, hipStream_t s) {
  const long tiles = (long)((a.N + 127) / 128) * ((a.M + 127) / 128) * batch;
  return a.N % 128 == 0 && tiles >= 512 ? launch_any<T, EPI, 128>(a, batch, s) : launch_any<T, EPI, 64>(a, batch, s);
}

// A [M, lda] and W [batch][N, K] of bf16 (f32 = 0) or fp32 (f32 = 1) elements with 16-byte aligned
// rows, K a multiple of 16 bytes. The result is fp32.
DA_EXPORT int da_gemm_any(const void* A, int lda, const void* W, void* C, int ldc, const void* bias, int M, int N,
                          int K, int f32, int epi, int batch, long long sA, long long sW, long long sC,
                          long long sBias, const void* u, int ldu, const void* lam, void* decay, void* drive, int ldg,
                          void* stream) {
  const int e16 = f32 ? 4 : 8;
  if (M < 1 || N < 1 || K < 1 || batch < 1 || K % e16 || lda % e16 || sA % e16 || sW % e16 || (M + 63) / 64 > 65535)
    return (int)hipErrorInvalidValue;
  if ((epi == ANY_REGLU || epi == ANY_RGLRU) && N % 32) return (int)hipErrorInvalidValue;
  if (epi == ANY_RGLRU && (!u || !lam || !decay || !drive || ldu % 4 || ldg % 4)) return (int)hipErrorInvalidValue;
  if (epi != ANY_RGLRU && !C) return (int)hipErrorInvalidValue;
  AnyArgs a{};
  a.A = A; a.W = W; a.C = C; a.bias = (const float*)bias;
  a.M = M; a.N = N; a.K = K; a.lda = lda; a.ldc = ldc;
  a.sA = sA; a.sW = sW; a.sC = sC; a.sBias = sBias;
  a.u = u; a.lam = (const float*)lam; a.decay = (float*)decay; a.drive = (float*)drive; a.ldu = ldu; a.ldg = ldg;
  hipStream_t s = (hipStream_t)stream;
#define ANY_CASE(E) \
  case E: return f32 ? launch_any_t<float, E>(a, batch, s) : launch_any_t<bf16_t, E>(a, batch, s);
  switch (epi) {
    ANY_CASE(ANY_NONE)
    ANY_CASE(ANY_SOFTPLUS)
    ANY_CASE(ANY_REGLU)
    ANY_CASE(ANY_RGLRU)
    default: return (int)hipErrorInvalidValue;
  }
#undef ANY_CASE
}
