// Gated delta rule with a decay per key channel, over a batch of portions (SeqMeta), state per sequence slot.
//
// Per token and head, S [K][V] in fp32 (stored [V][K]), a = exp2(log decay) per key channel:
//   S <- a S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// with q and k made unit vectors (q scaled), then o / rms(o) * w * sigmoid(gate).
//
// The columns of S do not depend on each other: a group of LN lanes owns NC of them, 4 NS4 key channels
// of each per lane, so only the two products with S cross lanes. q, k and decays of a tile of tokens are staged
// in LDS as fp32 (unit norms taken on the way), the next tile's loads in flight meanwhile.
#include "seq.h"

struct DeltaArgs {
  const void* x; int ldx;             // [T][G K queries | G K keys | H V values]
  const float* decay;                 // log2 of the decays, [T][H K]
  const void* beta; int ldb;          // [T][ldb], H columns, before the sigmoid
  float* state;                       // [slots][H][V][K]
  void* o; int ldo;                   // [T][H V]
  int H, G, K, V;
  float q_scale, eps;                 // of the unit norms
  ConvState conv;
  SeqMeta m;
};

// Sum over groups of neighbouring lanes: 2, 4 (quad permutes), 8, 16 (mirrors of a row), then shuffles.
template <int CTRL> __device__ __forceinline__ float dpp_add(float v) {
  return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false));
}
template <int LANES> __device__ __forceinline__ float lanes_sum(float v) {
  v = dpp_add<0xb1>(v);                                // lane ^ 1
  v = dpp_add<0x4e>(v);                                // lane ^ 2
  v = dpp_add<0x141>(v);                               // mirror within 8
  if constexpr (LANES > 8) v = dpp_add<0x140>(v);      // mirror within 16
  if constexpr (LANES > 16) v += __shfl_xor(v, 16, 64);
  return v;
}

constexpr int DT = 8;  // tokens per tile: 32 lanes stage one

template <typename T, int LN, int NS4, int NC>
__global__ void __launch_bounds__(256) delta_scan_kernel(DeltaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int b = blockIdx.z, h = blockIdx.y, hk = h / (a.H / a.G);
  const int t0 = a.m.cu[b], t1 = a.m.cu[b + 1];
  if (t0 == t1) return;
  const int tid = threadIdx.x, g = tid % LN, grp = tid / LN;
  constexpr int ncol = 256 / LN * NC, K = LN * NS4 * 4, np = K / 4, nv = ncol / 4;
  const int c0 = blockIdx.x * ncol;
  float *sq = sm, *sk = sq + DT * K, *sa = sk + DT * K, *sv = sa + DT * K, *sb = sv + DT * ncol;

  f32x4_t S[NC][NS4];
  float* st[NC];
  bool live[NC];
  const bool stored = a.m.pos0[b] != 0;
#pragma unroll
  for (int j = 0; j < NC; ++j) {
    const int c = c0 + grp * NC + j;
    live[j] = c < a.V;
    st[j] = a.state + (((size_t)a.m.slot[b] * a.H + h) * a.V + min(c, a.V - 1)) * K + g * 4;
#pragma unroll
    for (int i = 0; i < NS4; ++i) {
      S[j][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (stored) S[j][i] = *(const f32x4_t*)(st[j] + i * LN * 4);
    }
  }

  // staging: token tid / 32 of the tile, lane tid % 32 takes every 32nd 4-channel piece
  constexpr int P = (np + 31) / 32;
  const int tt = tid >> 5, sl = tid & 31;
  f32x4_t rq[P], rk[P], ra[P], rv;
  float rb = 0.f;
  auto fetch = [&](int t) {
    const size_t row = min(t + tt, t1 - 1);
    const T* x = (const T*)a.x + row * a.ldx;
#pragma unroll
    for (int i = 0; i < P; ++i) {
      const int c = min(sl + 32 * i, np - 1) * 4;
      rq[i] = Act<T>::load4(x + hk * K + c);
      rk[i] = Act<T>::load4(x + (a.G + hk) * K + c);
      ra[i] = *(const f32x4_t*)(a.decay + row * a.H * K + (size_t)h * K + c);
    }
    if (sl < nv) rv = Act<T>::load4(x + 2 * a.G * K + h * a.V + min(c0 + sl * 4, a.V - 4));
    if (sl == 0) rb = Act<T>::to_f(((const T*)a.beta)[row * a.ldb + h]);
  };
  auto stage = [&]() {
    float qq = 0.f, kk = 0.f;
#pragma unroll
    for (int i = 0; i < P; ++i)
      if (sl + 32 * i < np)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          qq = fmaf(rq[i][e], rq[i][e], qq);
          kk = fmaf(rk[i][e], rk[i][e], kk);
        }
    qq = lanes_sum<32>(qq);
    kk = lanes_sum<32>(kk);
    const float fq = a.q_scale / sqrtf(qq + a.eps), fk = 1.f / sqrtf(kk + a.eps);
#pragma unroll
    for (int i = 0; i < P; ++i) {
      const int c = (sl + 32 * i) * 4;
      if (c >= K) continue;
      f32x4_t d;
#pragma unroll
      for (int e = 0; e < 4; ++e) d[e] = __builtin_amdgcn_exp2f(ra[i][e]);
      *(f32x4_t*)(sq + tt * K + c) = rq[i] * fq;
      *(f32x4_t*)(sk + tt * K + c) = rk[i] * fk;
      *(f32x4_t*)(sa + tt * K + c) = d;
    }
    if (sl < nv) *(f32x4_t*)(sv + tt * ncol + sl * 4) = rv;
    if (sl == 0) sb[tt] = sigmoid32(rb);
  };

  fetch(t0);
  for (int t = t0; t < t1; t += DT) {
    __syncthreads();
    stage();
    __syncthreads();
    if (t + DT < t1) fetch(t + DT);
    const int n = min(DT, t1 - t);
    for (int r = 0; r < n; ++r) {
      const float* pk = sk + r * K + g * 4;
      const float* pa = sa + r * K + g * 4;
      const float* pq = sq + r * K + g * 4;
      f32x4_t kv[NS4];
      float held[NC], o[NC];
#pragma unroll
      for (int j = 0; j < NC; ++j) held[j] = o[j] = 0.f;
#pragma unroll
      for (int i = 0; i < NS4; ++i) {
        kv[i] = *(const f32x4_t*)(pk + i * LN * 4);
        const f32x4_t d = *(const f32x4_t*)(pa + i * LN * 4);
#pragma unroll
        for (int j = 0; j < NC; ++j)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[j][i][e] *= d[e];
            held[j] = fmaf(S[j][i][e], kv[i][e], held[j]);
          }
      }
      const float beta = sb[r];
      float u[NC];
#pragma unroll
      for (int j = 0; j < NC; ++j) u[j] = beta * (sv[r * ncol + grp * NC + j] - lanes_sum<LN>(held[j]));
#pragma unroll
      for (int i = 0; i < NS4; ++i) {
        const f32x4_t q = *(const f32x4_t*)(pq + i * LN * 4);
#pragma unroll
        for (int j = 0; j < NC; ++j)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[j][i][e] = fmaf(kv[i][e], u[j], S[j][i][e]);
            o[j] = fmaf(S[j][i][e], q[e], o[j]);
          }
      }
#pragma unroll
      for (int j = 0; j < NC; ++j) {
        o[j] = lanes_sum<LN>(o[j]);
        if (g == 0 && live[j])
          ((T*)a.o)[(size_t)(t + r) * a.ldo + h * a.V + c0 + grp * NC + j] = Act<T>::from_f(o[j]);
      }
    }
  }
#pragma unroll
  for (int j = 0; j < NC; ++j)
    if (live[j])
#pragma unroll
      for (int i = 0; i < NS4; ++i) *(f32x4_t*)(st[j] + i * LN * 4) = S[j][i];
  // the convolution's state, shared out over the portion's workgroups
  const int wg = blockIdx.y * gridDim.x + blockIdx.x, step = gridDim.x * gridDim.y * 256;
  for (int c = wg * 256 + tid; c < a.conv.C; c += step) conv_state_store<T>(a.conv, a.m, b, c);
}

// o / rms(o) * w * sigmoid(gate), in place, per head: `lanes` lanes a head.
template <typename T>
__global__ void __launch_bounds__(256)
head_norm_kernel(T* o, int ldo, const T* gate, int ldg, const float* w, int T_, int H, int V, int dim, float eps, int lanes) {
  const int item = blockIdx.x * (256 / lanes) + threadIdx.x / lanes, l = threadIdx.x % lanes;
  const bool live = item < T_ * H;
  const int it = live ? item : T_ * H - 1, t = it / H, h = it % H;
  T* r = o + (size_t)t * ldo + (size_t)h * V;
  const T* gr = gate + (size_t)t * ldg + (size_t)h * V;
  constexpr int U = 4;
  f32x4_t v[U], g[U];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < U; ++i) {
    const int d = min((i * lanes + l) * 4, V - 4);
    v[i] = Act<T>::load4(r + d);
    g[i] = Act<T>::load4(gr + d);
    if ((i * lanes + l) * 4 < V)
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(v[i][e], v[i][e], ss);
  }
  for (int d = (U * lanes + l) * 4; d < V; d += lanes * 4) {
    const f32x4_t x = Act<T>::load4(r + d);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss = fmaf(x[e], x[e], ss);
  }
  for (int s = lanes >> 1; s > 0; s >>= 1) ss += __shfl_xor(ss, s, 64);
  if (!live) return;
  const float inv = 1.f / sqrtf(ss / dim + eps);
  auto put = [&](int d, const f32x4_t& x, const f32x4_t& gt) {
    const f32x4_t wv = *(const f32x4_t*)(w + d);
    f32x4_t y;
#pragma unroll
    for (int e = 0; e < 4; ++e) y[e] = x[e] * inv * wv[e] * sigmoid32(gt[e]);
    Act<T>::store4(r + d, y);
  };
#pragma unroll
  for (int i = 0; i < U; ++i)
    if ((i * lanes + l) * 4 < V) put((i * lanes + l) * 4, v[i], g[i]);
  for (int d = (U * lanes + l) * 4; d < V; d += lanes * 4) put(d, Act<T>::load4(r + d), Act<T>::load4(gr + d));
}

template <typename T, int LN, int NS4>
static int launch_delta(const DeltaArgs& a, hipStream_t s) {
  constexpr int NC = 2, ncol = 256 / LN * NC, lds = DT * (3 * LN * NS4 * 4 + ncol + 1) * 4;
  if (lds > 65536) {
    static const hipError_t e = hipFuncSetAttribute((const void*)delta_scan_kernel<T, LN, NS4, NC>,
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (e != hipSuccess) return (int)e;
  }
  delta_scan_kernel<T, LN, NS4, NC><<<dim3((a.V + ncol - 1) / ncol, a.H, a.m.B), 256, lds, s>>>(a);
  DA_LAUNCH_CHECK();
}

template <typename T>
static int launch_delta_t(const DeltaArgs& a, const void* w, const void* gate, int ldg, int dim, float eps, hipStream_t s) {
  int err;
  switch (a.K) {
#define DELTA_CASE(LN, N) \
  case LN * 4 * N: err = launch_delta<T, LN, N>(a, s); break;
    DELTA_CASE(8, 1) DELTA_CASE(8, 2) DELTA_CASE(8, 3) DELTA_CASE(8, 4)
    DELTA_CASE(8, 5) DELTA_CASE(8, 6) DELTA_CASE(8, 7) DELTA_CASE(8, 8)
    DELTA_CASE(16, 5) DELTA_CASE(16, 6) DELTA_CASE(16, 7) DELTA_CASE(16, 8)
    DELTA_CASE(32, 5) DELTA_CASE(32, 6) DELTA_CASE(32, 7) DELTA_CASE(32, 8)
#undef DELTA_CASE
    default: return (int)hipErrorInvalidValue;
  }
  if (err) return err;
  int lanes = 4;
  while (lanes < 64 && lanes * 4 < a.V) lanes *= 2;
  const int per = 256 / lanes;
  head_norm_kernel<T><<<(unsigned)(((size_t)a.m.T * a.H + per - 1) / per), 256, 0, s>>>(
      (T*)a.o, a.ldo, (const T*)gate, ldg, (const float*)w, a.m.T, a.H, a.V, dim, eps, lanes);
  DA_LAUNCH_CHECK();
}

// x [T][ldx] (activation type): G query heads, G key heads of K channels, H value heads of V; decay fp32 [T][H K];
// K = 32 n (n <= 8), 64 n (n <= 8) or 128 n (n <= 8); V % 4 == 0. norm weight w fp32 [V], gate [T][ldg]; dim: the
// channels a value head really has. conv: as the other recurrences' (state null: kept by the convolution's launch).
DA_EXPORT int da_delta_rule(const void* x, int ldx, const void* decay, const void* beta, int ldb, void* state, void* o,
                            int ldo, int H, int G, int K, int V, float q_scale, float unit_eps, const void* w,
                            const void* gate, int ldg, int dim, float eps, const void* conv_x, int ld_conv,
                            void* conv_state, int taps, int conv_c, const void* cu, const void* slot, const void* pos0,
                            const void* seq, int T, int B, int f32, void* stream) {
  if (T < 1 || B < 1 || B > 65535 || G < 1 || H % G || H > 65535 || V < 4 || V % 4 ||
      ldx % 4 || ldo % 4 || ldg % 4 || dim < 1 || dim > V || taps < 1 || (long long)T * H > 0x7fffffffll / 4)
    return (int)hipErrorInvalidValue;
  DeltaArgs a{x, ldx, (const float*)decay, beta, ldb, (float*)state, o, ldo, H, G, K, V, q_scale, unit_eps,
              ConvState{conv_x, ld_conv, conv_state, taps, conv_c},
              SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}};
  return f32 ? launch_delta_t<float>(a, w, gate, ldg, dim, eps, (hipStream_t)stream)
             : launch_delta_t<bf16_t>(a, w, gate, ldg, dim, eps, (hipStream_t)stream);
}
