// Matrix products of any M, N and K that keep fp32 results: C[M, N] = epi(A[M, K] . W[N, K]^T), with
// bf16 or fp32 operands (v_mfma_f32_16x16x32_bf16 / v_mfma_f32_16x16x4_f32: both accumulate in fp32, the
// fp32 form multiplies true fp32), batched over blockIdx.z. The serving precision uses it where a
// product feeds a recurrence (step sizes, gates), which must not be rounded to 16 bits; everything
// else runs on gemm.hip's kernels. The fp32 precision runs every product here.
//
// 64 x 64 tile, 4 waves x 32 x 32, K in 128-byte slices through double-buffered LDS (rows padded to 144
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

constexpr int ANY_ROWB = 144, ANY_TILEB = 64 * ANY_ROWB;

template <typename T, int EPI, typename OT>
__global__ void __launch_bounds__(256) gemm_any_kernel(AnyArgs p) {
  __shared__ __attribute__((aligned(16))) char sm[4 * ANY_TILEB];
  constexpr int E16 = 16 / sizeof(T), KS = 128 / sizeof(T);  // elements per 16 bytes, per slice
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, wm = wv >> 1, wn = wv & 1;
  const int fr = lane & 15, fg = lane >> 4;
  const int n0 = blockIdx.x * 64, m0 = blockIdx.y * 64, z = blockIdx.z;
  const T* A = (const T*)p.A + z * p.sA;
  const T* W = (const T*)p.W + z * p.sW;

  // 512 16-byte pieces per operand slice: thread tid carries pieces tid and tid + 256
  u32x4_t ra[2], rw[2];
  auto load = [&](int k0) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
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
    for (int i = 0; i < 2; ++i) {
      const int pc = tid + 256 * i, off = (pc >> 3) * ANY_ROWB + (pc & 7) * 16;
      *(u32x4_t*)(sm + buf * 2 * ANY_TILEB + off) = ra[i];
      *(u32x4_t*)(sm + buf * 2 * ANY_TILEB + ANY_TILEB + off) = rw[i];
    }
  };
  f32x4_t acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  const int nk = (p.K + KS - 1) / KS;
  load(0);
  store(0);
  __syncthreads();
  for (int s = 0; s < nk; ++s) {
    if (s + 1 < nk) load((s + 1) * KS);
    const char* sa = sm + (s & 1) * 2 * ANY_TILEB;
    const char* sw = sa + ANY_TILEB;
    if constexpr (sizeof(T) == 2) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        bf16x8_t fa[2], fw[2];
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          fa[i] = *(const bf16x8_t*)(sa + (wm * 32 + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
          fw[i] = *(const bf16x8_t*)(sw + (wn * 32 + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
        }
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int j = 0; j < 2; ++j) acc[i][j] = mfma16(fa[i], fw[j], acc[i][j]);
      }
    } else {
      // a lane group's four consecutive k of a 16-k step go to four MFMAs (the same k of both operands)
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        f32x4_t fa[2], fw[2];
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          fa[i] = *(const f32x4_t*)(sa + (wm * 32 + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
          fw[i] = *(const f32x4_t*)(sw + (wn * 32 + i * 16 + fr) * ANY_ROWB + ks * 64 + fg * 16);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int j = 0; j < 2; ++j)
              acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(fa[i][e], fw[j][e], acc[i][j], 0, 0, 0);
      }
    }
    if (s + 1 < nk) store((s + 1) & 1);
    __syncthreads();
  }

  // lane (fr, fg) holds rows 4 fg + q, column fr of each 16 x 16 block
  const float* bias = p.bias ? p.bias + z * p.sBias : nullptr;
  if constexpr (EPI == ANY_REGLU || EPI == ANY_RGLRU) {
    const int nb = n0 + wn * 32;
    if (nb >= p.N) return;
    const int col = nb / 2 + fr;
    const float b0 = bias ? bias[nb + fr] : 0.f, b1 = bias ? bias[nb + 16 + fr] : 0.f;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int m = m0 + wm * 32 + i * 16 + fg * 4 + q;
        if (m >= p.M) continue;
        const float x = acc[i][0][q] + b0, y = acc[i][1][q] + b1;
        if constexpr (EPI == ANY_REGLU) {
          ((OT*)p.C)[z * p.sC + (size_t)m * p.ldc + col] = Act<OT>::from_f(fmaxf(x, 0.f) * y);
        } else {
          const int ch = z * (p.N / 2) + col;
          const float la = p.lam[ch] * sigmoid32(x);  // log of the decay, <= 0
          const float u = Act<T>::to_f(((const T*)p.u)[(size_t)m * p.ldu + ch]);
          p.decay[(size_t)m * p.ldg + ch] = exp32(la);
          p.drive[(size_t)m * p.ldg + ch] = __builtin_amdgcn_sqrtf(one_minus_exp32(2.f * la)) * sigmoid32(y) * u;
        }
      }
  } else {
    OT* C = (OT*)p.C + z * p.sC;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int n = n0 + wn * 32 + j * 16 + fr;
      if (n >= p.N) continue;
      const float b = bias ? bias[n] : 0.f;
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const int m = m0 + wm * 32 + i * 16 + fg * 4 + q;
          if (m >= p.M) continue;
          float v = acc[i][j][q] + b;
          if constexpr (EPI == ANY_SOFTPLUS) v = softplus32(v);
          C[(size_t)m * p.ldc + n] = Act<OT>::from_f(v);
        }
    }
  }
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
  if (epi == ANY_RGLRU && (!u || !lam || !decay || !drive)) return (int)hipErrorInvalidValue;
  if (epi != ANY_RGLRU && !C) return (int)hipErrorInvalidValue;
  AnyArgs a{};
  a.A = A; a.W = W; a.C = C; a.bias = (const float*)bias;
  a.M = M; a.N = N; a.K = K; a.lda = lda; a.ldc = ldc;
  a.sA = sA; a.sW = sW; a.sC = sC; a.sBias = sBias;
  a.u = u; a.lam = (const float*)lam; a.decay = (float*)decay; a.drive = (float*)drive; a.ldu = ldu; a.ldg = ldg;
  const dim3 grid((N + 63) / 64, (M + 63) / 64, batch), block(256);
  hipStream_t s = (hipStream_t)stream;
#define ANY_CASE(E)                                                            \
  case E:                                                                      \
    if (f32) gemm_any_kernel<float, E, float><<<grid, block, 0, s>>>(a);       \
    else gemm_any_kernel<bf16_t, E, float><<<grid, block, 0, s>>>(a);          \
    break;
  switch (epi) {
    ANY_CASE(ANY_NONE)
    ANY_CASE(ANY_SOFTPLUS)
    ANY_CASE(ANY_REGLU)
    ANY_CASE(ANY_RGLRU)
    default: return (int)hipErrorInvalidValue;
  }
#undef ANY_CASE
  DA_LAUNCH_CHECK();
}
