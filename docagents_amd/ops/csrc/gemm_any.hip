// Matrix products of any M, N and K that keep fp32 results: C[M, N] = epi(A[M, K] . W[N, K]^T), with
// bf16 or fp32 operands (v_mfma_f32_16x16x32_bf16 / v_mfma_f32_16x16x4_f32: both accumulate in fp32, the
// fp32 form multiplies true fp32), batched over blockIdx.z. The serving precision uses it where a
// product feeds a recurrence (step sizes, gates), which must not be rounded to 16 bits; everything
// else runs on gemm.hip's kernels. The fp32 precision runs every product here.
//
// BT x BT tile (64, or 128 where the rows fill the chip), 4 waves of a quarter each, K in 128-byte slices through
// double-buffered LDS (rows padded to 144 bytes: conflict-free 16-byte reads), the next slice's loads in flight while this
// one is multiplied.
#include "seq.h"

enum AnyEpi : int {
  ANY_NONE = 0,      // + bias
  ANY_SOFTPLUS = 1,  // softplus(x + bias), times a coefficient per column where lam is given
  ANY_REGLU = 2,     // W rows interleaved in 16-row (gate, up) groups: relu(g) * u
  ANY_RGLRU = 3,     // W rows interleaved in 16-row (recurrence, input) gate groups of one block
  ANY_SWIGLU = 4,    // as ANY_REGLU: silu(g) * u
  ANY_ACT = 5,       // C in the operands' type, times sigmoid(u) where u is given
};
constexpr bool any_paired(int epi) { return epi == ANY_REGLU || epi == ANY_RGLRU || epi == ANY_SWIGLU; }

struct AnyArgs {
  const void* A; const void* W; void* C; const float* bias;
  int M, N, K, lda, ldc;
  long long sA, sW, sC, sBias;  // strides between the products of a batch, in elements
  // ANY_RGLRU: decay factors and driving terms of the recurrence, from the gates and its input u.
  // ANY_SOFTPLUS: lam [N] (nullable). ANY_ACT: u [M][ldu] (nullable), columns z N .. of product z
  const void* u; const float* lam; float* decay; float* drive; int ldu, ldg;
};

// Four neighbouring outputs of row m, columns n .. n + 3 (past N: not stored).
template <typename T, int EPI>
__device__ __forceinline__ void any_block(const AnyArgs& p, int z, int m, int n, f32x4_t v) {
  if (n >= p.N) return;
  if constexpr (EPI == ANY_ACT) {
    T* o = (T*)p.C + z * p.sC + (size_t)m * p.ldc + n;
    const T* g = p.u ? (const T*)p.u + (size_t)m * p.ldu + (size_t)z * p.N + n : nullptr;
    if ((p.N & 3) == 0 && (p.ldc & 3) == 0) {
      if (g) {
        const f32x4_t u = Act<T>::load4(g);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] *= sigmoid32(u[e]);
      }
      Act<T>::store4(o, v);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (n + e < p.N) o[e] = Act<T>::from_f(g ? v[e] * sigmoid32(Act<T>::to_f(g[e])) : v[e]);
    }
    return;
  }
  const float* bias = p.bias ? p.bias + z * p.sBias : nullptr;
  float* o = (float*)p.C + z * p.sC + (size_t)m * p.ldc + n;
  const bool vec = (p.N & 3) == 0 && (p.ldc & 3) == 0;
  if (bias) {
    if (vec) v += *(const f32x4_t*)(bias + n);
    else
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] += bias[min(n + e, p.N - 1)];
  }
  if constexpr (EPI == ANY_SOFTPLUS)
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = softplus32(v[e]) * (p.lam ? p.lam[min(n + e, p.N - 1)] : 1.f);
  if (vec) {
    *(f32x4_t*)o = v;
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (n + e < p.N) o[e] = v[e];
  }
}

// Gates of four neighbouring channels from ch on: decay and driving term of the recurrence.
__device__ __forceinline__ void any_gates(const float* lam4, const f32x4_t& x, const f32x4_t& y, const f32x4_t& u,
                                          f32x4_t& decay, f32x4_t& drive) {
  const f32x4_t lam = *(const f32x4_t*)lam4;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float la = lam[e] * sigmoid32(x[e]);  // log of the decay, <= 0
    decay[e] = exp32(la);
    drive[e] = __builtin_amdgcn_sqrtf(one_minus_square32(la, decay[e])) * sigmoid32(y[e]) * u[e];
  }
}

// Four neighbouring pairs of row m: columns nb + 4 fg .. of a 32-column group and the 16 after them (nb % 32 == 0).
template <int EPI>
__device__ __forceinline__ void any_pair(const AnyArgs& p, int z, int m, int nb, int fg, f32x4_t x, f32x4_t y,
                                         const f32x4_t& u) {
  if (p.bias) {
    const float* bias = p.bias + z * p.sBias + nb + 4 * fg;
    x += *(const f32x4_t*)bias;
    y += *(const f32x4_t*)(bias + 16);
  }
  const int col = nb / 2 + 4 * fg;
  f32x4_t r, d;
  if constexpr (EPI == ANY_REGLU || EPI == ANY_SWIGLU) {
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = (EPI == ANY_REGLU ? fmaxf(x[e], 0.f) : silu32(x[e])) * y[e];
    *(f32x4_t*)((float*)p.C + z * p.sC + (size_t)m * p.ldc + col) = r;
  } else {
    const int ch = z * (p.N / 2) + col;
    any_gates(p.lam + ch, x, y, u, r, d);
    *(f32x4_t*)(p.decay + (size_t)m * p.ldg + ch) = r;
    *(f32x4_t*)(p.drive + (size_t)m * p.ldg + ch) = d;
  }
}

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
#pragma unroll
  for (int i = 0; i < F; ++i) {
    const int m = m0 + wm * WT + i * 16 + fr;
    if (m >= p.M) continue;
    if constexpr (any_paired(EPI)) {
#pragma unroll
      for (int jp = 0; jp < F / 2; ++jp) {
        const int nb = n0 + wn * WT + jp * 32;
        if (nb >= p.N) continue;
        const int ch = z * (p.N / 2) + nb / 2 + 4 * fg;
        f32x4_t u{0.f, 0.f, 0.f, 0.f};
        if constexpr (EPI == ANY_RGLRU) u = Act<T>::load4((const T*)p.u + (size_t)m * p.ldu + ch);
        any_pair<EPI>(p, z, m, nb, fg, acc[i][2 * jp], acc[i][2 * jp + 1], u);
      }
    } else {
#pragma unroll
      for (int j = 0; j < F; ++j) any_block<T, EPI>(p, z, m, n0 + wn * WT + j * 16 + 4 * fg, acc[i][j]);
    }
  }
}

// K up to 256 and many rows (bf16): a workgroup keeps its 64 rows of W in LDS and walks row tiles of A, the
// next tile's loads in flight during this one's products and epilogue (which costs as much as they do). Results
// leave through LDS in whole lines (64-byte pieces of rows a power of two apart: 299 us, whole lines 240 us for
// 16384 x 8192 step sizes).
template <int EPI>
__global__ void __launch_bounds__(256) gemm_walk_kernel(AnyArgs p) {
  extern __shared__ __attribute__((aligned(16))) char sm[];
  const int rowb = p.K * 2 + 16, pieces = p.K / 8, lp = p.K / 32;  // bytes and 16-byte pieces of a row, per thread
  char* sW = sm;
  char* sA = sm + 64 * rowb;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, wm = wv >> 1, wn = wv & 1;
  const int fr = lane & 15, fg = lane >> 4;
  const int n0 = blockIdx.x * 64, z = blockIdx.z, mt = (p.M + 63) / 64;
  const bf16_t* A = (const bf16_t*)p.A + z * p.sA;
  const bf16_t* W = (const bf16_t*)p.W + z * p.sW;
  u32x4_t r[8];
  auto load = [&](const bf16_t* X, int row0, int rows, int ld) {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (i < lp) {
        const int pc = tid + 256 * i;
        r[i] = *(const u32x4_t*)(X + (size_t)min(row0 + pc / pieces, rows - 1) * ld + pc % pieces * 8);
      }
  };
  auto store = [&](char* s) {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (i < lp) {
        const int pc = tid + 256 * i;
        *(u32x4_t*)(s + pc / pieces * rowb + pc % pieces * 16) = r[i];
      }
  };
  load(W, n0, p.N, p.K);
  store(sW);
  load(A, blockIdx.y * 64, p.M, p.lda);
  store(sA);
  __syncthreads();
  for (int t = blockIdx.y; t < mt; t += gridDim.y) {
    if (t + (int)gridDim.y < mt) load(A, (t + gridDim.y) * 64, p.M, p.lda);
    f32x4_t acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < p.K; k += 32) {
      bf16x8_t fa[2], fw[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        fa[i] = *(const bf16x8_t*)(sA + (wm * 32 + i * 16 + fr) * rowb + k * 2 + fg * 16);
        fw[i] = *(const bf16x8_t*)(sW + (wn * 32 + i * 16 + fr) * rowb + k * 2 + fg * 16);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = mfma16(fw[j], fa[i], acc[i][j]);
    }
    // staged rows of 64 (gates: 32 decays, 32 driving terms) fp32, in place of the A tile
    constexpr int SW = 68;
    const int nb = n0 + wn * 32;
    f32x4_t v[2][2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int ml = wm * 32 + i * 16 + fr;
      f32x4_t b0{0.f, 0.f, 0.f, 0.f}, b1 = b0;
      if (p.bias && nb < p.N) {
        const float* bias = p.bias + z * p.sBias + nb + 4 * fg;
        b0 = *(const f32x4_t*)bias;
        if (nb + 16 < p.N) b1 = *(const f32x4_t*)(bias + 16);
      }
      v[i][0] = acc[i][0] + b0;
      v[i][1] = acc[i][1] + b1;
      if constexpr (EPI == ANY_RGLRU) {  // the gates' input is this tile of A
        if (nb < p.N)
          any_gates(p.lam + z * (p.N / 2) + nb / 2 + 4 * fg, v[i][0], v[i][1],
                    Act<bf16_t>::load4((const bf16_t*)(sA + ml * rowb) + nb / 2 + 4 * fg), v[i][0], v[i][1]);
      } else {
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          f32x4_t f{1.f, 1.f, 1.f, 1.f};
          if (p.lam && nb + 16 * j < p.N) f = *(const f32x4_t*)(p.lam + nb + 16 * j + 4 * fg);
#pragma unroll
          for (int e = 0; e < 4; ++e) v[i][j][e] = softplus32(v[i][j][e]) * f[e];
        }
      }
    }
    __syncthreads();  // the A tile has been read
    float* st = (float*)sA;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int col = EPI == ANY_RGLRU ? j * 32 + wn * 16 + 4 * fg : wn * 32 + j * 16 + 4 * fg;
        *(f32x4_t*)(st + (wm * 32 + i * 16 + fr) * SW + col) = v[i][j];
      }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = (tid >> 4) + 16 * i, c = (tid & 15) * 4, m = t * 64 + row;
      const f32x4_t o = *(const f32x4_t*)(st + row * SW + c);
      if (m >= p.M) continue;
      if constexpr (EPI == ANY_RGLRU) {
        const int cl = n0 / 2 + (c & 31);
        if (cl < p.N / 2) *(f32x4_t*)((c < 32 ? p.decay : p.drive) + (size_t)m * p.ldg + z * (p.N / 2) + cl) = o;
      } else {
        if (n0 + c < p.N) *(f32x4_t*)((float*)p.C + z * p.sC + (size_t)m * p.ldc + n0 + c) = o;
      }
    }
    __syncthreads();
    if (t + (int)gridDim.y < mt) store(sA);
    __syncthreads();
  }
}

// Few rows (16 RT at most), bf16: 32 columns per workgroup, its waves take turns at the 32-k steps, operands straight from
// memory to registers with U steps in flight, and their sums meet in LDS: one or two memory round trips in all.
template <int EPI, int RT>
__global__ void __launch_bounds__(256) gemm_rows_kernel(AnyArgs p) {
  constexpr int U = 4, SR = 36;  // steps in flight; floats of a staged row
  __shared__ __attribute__((aligned(16))) float part[4][RT * 16 * SR];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, fr = lane & 15, fg = lane >> 4;
  const int n0 = blockIdx.x * 32, z = blockIdx.z;
  const bf16_t* A = (const bf16_t*)p.A + z * p.sA;
  const bf16_t* W = (const bf16_t*)p.W + z * p.sW;
  f32x4_t acc[RT][2];
#pragma unroll
  for (int i = 0; i < RT; ++i) acc[i][0] = acc[i][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = wv * 32; k0 < p.K; k0 += 128 * U) {
    bf16x8_t fa[U][RT], fw[U][2];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = min(k0 + 128 * u + fg * 8, p.K - 8);
#pragma unroll
      for (int i = 0; i < RT; ++i) fa[u][i] = *(const bf16x8_t*)(A + (size_t)min(i * 16 + fr, p.M - 1) * p.lda + k);
#pragma unroll
      for (int j = 0; j < 2; ++j) fw[u][j] = *(const bf16x8_t*)(W + (size_t)min(n0 + j * 16 + fr, p.N - 1) * p.K + k);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const bool in = k0 + 128 * u + fg * 8 < p.K;
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const bf16x8_t w = in ? fw[u][j] : bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
        for (int i = 0; i < RT; ++i) acc[i][j] = mfma16(w, in ? fa[u][i] : bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0}, acc[i][j]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < RT; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) *(f32x4_t*)(part[wv] + (i * 16 + fr) * SR + j * 16 + 4 * fg) = acc[i][j];
  __syncthreads();
  for (int i = tid; i < RT * 16 * 8; i += 256) {
    const int m = i >> 3, c = (i & 7) * 4, at = m * SR + c;
    if (m >= p.M) continue;
    const f32x4_t v = (*(const f32x4_t*)(part[0] + at) + *(const f32x4_t*)(part[1] + at)) +
                      (*(const f32x4_t*)(part[2] + at) + *(const f32x4_t*)(part[3] + at));
    any_block<bf16_t, EPI>(p, z, m, n0 + c, v);
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
  if constexpr (sizeof(T) == 2 && (EPI == ANY_SOFTPLUS || EPI == ANY_RGLRU)) {
    if (a.M >= 1024 && a.K <= 256 && a.K % 32 == 0 && a.N % 16 == 0 && a.ldc % 4 == 0 &&
        (EPI != ANY_RGLRU || (a.A == a.u && a.sA == a.N / 2 && a.K == a.N / 2))) {
      const int row = a.K * 2 + 16 > 272 ? a.K * 2 + 16 : 272, lds = 64 * (a.K * 2 + 16 + row);
      const int nt = (a.N + 63) / 64 * batch, mt = (a.M + 63) / 64;
      static const hipError_t e = hipFuncSetAttribute((const void*)gemm_walk_kernel<EPI>,
                                                      hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 528);
      if (e != hipSuccess) return (int)e;
      const int walks = mt < (2048 + nt - 1) / nt ? mt : (2048 + nt - 1) / nt;  // ~2048 workgroups
      gemm_walk_kernel<EPI><<<dim3((a.N + 63) / 64, walks, batch), 256, lds, s>>>(a);
      DA_LAUNCH_CHECK();
    }
  }
  if constexpr (sizeof(T) == 2 && !any_paired(EPI) && EPI != ANY_NONE)
    if (a.M <= 64) {
      const dim3 grid((a.N + 31) / 32, 1, batch);
      if (a.M <= 16) gemm_rows_kernel<EPI, 1><<<grid, 256, 0, s>>>(a);
      else if (a.M <= 32) gemm_rows_kernel<EPI, 2><<<grid, 256, 0, s>>>(a);
      else gemm_rows_kernel<EPI, 4><<<grid, 256, 0, s>>>(a);
      DA_LAUNCH_CHECK();
    }
  const long tiles = (long)((a.N + 127) / 128) * ((a.M + 127) / 128) * batch;
  return a.N % 128 == 0 && tiles >= 512 ? launch_any<T, EPI, 128>(a, batch, s) : launch_any<T, EPI, 64>(a, batch, s);
}

// A [M, lda] and W [batch][N, K] of bf16 (f32 = 0) or fp32 (f32 = 1) elements with 16-byte aligned
// rows, K a multiple of 16 bytes. The result is fp32, with ANY_ACT of the operands' type.
DA_EXPORT int da_gemm_any(const void* A, int lda, const void* W, void* C, int ldc, const void* bias, int M, int N,
                          int K, int f32, int epi, int batch, long long sA, long long sW, long long sC,
                          long long sBias, const void* u, int ldu, const void* lam, void* decay, void* drive, int ldg,
                          void* stream) {
  const int e16 = f32 ? 4 : 8;
  if (M < 1 || N < 1 || K < 1 || batch < 1 || K % e16 || lda % e16 || sA % e16 || sW % e16 || (M + 63) / 64 > 65535)
    return (int)hipErrorInvalidValue;
  if (any_paired(epi) && N % 32) return (int)hipErrorInvalidValue;
  if (epi == ANY_RGLRU && (!u || !lam || !decay || !drive || ldu % 4 || ldg % 4)) return (int)hipErrorInvalidValue;
  if (epi != ANY_RGLRU && !C) return (int)hipErrorInvalidValue;
  if (epi == ANY_ACT && (sC % 4 || (u && ldu % 4))) return (int)hipErrorInvalidValue;
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
    ANY_CASE(ANY_SWIGLU)
    ANY_CASE(ANY_ACT)
    default: return (int)hipErrorInvalidValue;
  }
#undef ANY_CASE
}
