// Gated delta rule with a decay per key channel, over a batch of portions (SeqMeta), state per sequence slot.
//
// Per token and head, S [K][V] in fp32 (stored [V][K]), D = diag(exp2(log decay)) over the key channels:
//   u = beta (v - k^T D S),  S' = D S + k u,  o = q^T S'      (v, u, o: rows of V)
// with q and k made unit vectors (q scaled), then o / rms(o) * w * sigmoid(gate).
//
// delta_scan: token by token on the vector ALUs, in fp32. The columns of S do not depend on each other: a group of LN
// lanes owns NC of them, 4 NS4 key channels of each per lane, so only the two products with S cross lanes. q, k and
// decays of a tile of tokens are staged in LDS as fp32 (unit norms taken on the way), the next tile's loads in flight
// meanwhile.
//
// delta_chunk: 32 tokens at a time on the matrix cores (below).
#include "seq.h"

struct DeltaArgs {
  const void* x; int ldx;             // [T][G K queries | G K keys | H V values]
  const float* decay;                 // log2 of the decays, [T][H K]
  const void* beta; int ldb;          // [T][ldb], H columns, before the sigmoid
  float* state;                       // [slots][H][V][K]
  void* o; int ldo;                   // [T][H V]
  int H, G, K, V;
  float q_scale, eps;                 // of the unit norms
  int below;                          // portions this launch runs: of fewer tokens (chunks: of as many or more)
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
  if (t0 == t1 || t1 - t0 >= a.below) return;
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
    lds_barrier();
    stage();
    lds_barrier();
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

// ------------------------------------------------------------------------------- matrix cores, chunks of 32 tokens
// With kappa, chi the keys and queries before their unit norms (norms rk, rq: k = rk kappa, q = rq chi), G_t the cumulative
// log2 decay of a channel from the chunk's start to token t, S the state before the chunk:
//   M_tj = sum_c kappa_t kappa_j 2^(G_t - G_j),  Q_tj likewise with chi_t,  b_t = beta_t rk_t^2
//   T  = (I + diag(b) tril(M, -1))^-1 diag(b)
//   U  = T (V / rk - (kappa 2^G) S)                                 rows u_t rk_t: what the tokens write
//   o  = rq ((chi 2^G) S + tril(Q) U)
//   S <- 2^G_end S + (kappa 2^(G_end - G))^T U
// delta_prep: a wave per chunk and head forms what does not depend on S (kappa 2^G, chi 2^G, kappa 2^(G_end - G), T, Q), as
// MFMA fragments in scratch memory. delta_apply: a wave walks its portion's chunks with 16 columns of V and S by itself,
// S staying in its accumulators; the waves of a workgroup share the fragments, which are on their way to LDS one and
// two chunks ahead.
//
// Every fp32 operand enters its product as two bf16 terms (its rounding and the remainder), three of their four
// products taken: about 16 bits, accumulated in fp32. The solve of T is in fp32.
//
// Products of 16-token blocks scale rows by 2^(G_t - m) and columns by 2^(m - G_j): m between the blocks off the
// diagonal (no factor above 1), the block's start on it. Where a channel decays by more than 2^100 within a block, rows go
// by 8 tokens with m in their middle and a token's decay limited to 2^-24 (a stronger one leaves less than the rounding
// of what it is added to), so that no factor leaves the range of an exponent.
constexpr int CT = 32;  // tokens of a chunk

struct ChunkArgs {
  DeltaArgs a;
  ChunkMeta ch;         // chunks of CT tokens of all portions
  char* frags;          // [chunks][H][NF KB]
};

struct Split { bf16x8_t hi, lo; };
__device__ __forceinline__ unsigned lo_of(unsigned hi, float a, float b) {
  return pack_bf2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}
__device__ __forceinline__ Split split8(const f32x4_t& a, const f32x4_t& b) {
  const u32x4_t h{pack_bf2(a[0], a[1]), pack_bf2(a[2], a[3]), pack_bf2(b[0], b[1]), pack_bf2(b[2], b[3])};
  const u32x4_t l{lo_of(h[0], a[0], a[1]), lo_of(h[1], a[2], a[3]), lo_of(h[2], b[0], b[1]), lo_of(h[3], b[2], b[3])};
  return {__builtin_bit_cast(bf16x8_t, h), __builtin_bit_cast(bf16x8_t, l)};
}
__device__ __forceinline__ f32x4_t mma3(const Split& a, const Split& b, f32x4_t c) {
  c = mfma16(a.lo, b.hi, c);
  c = mfma16(a.hi, b.lo, c);
  return mfma16(a.hi, b.hi, c);
}

// A fragment is 1 KB, lane l's 16 bytes at 16 l. Its lane (fr, fg) holds row fr and the 8 k values 16 u + 4 fg + e (u < 2,
// e < 4) of 32: the order in which an accumulator's rows become the other operand. An operand's two terms follow each other.
template <int KB> struct DC {  // K = 32 KB key channels; offsets in fragments
  static constexpr int K = 32 * KB;
  static constexpr int KP = 0, QP = 4 * KB;            // kappa 2^G, chi 2^G: [token block][32 channels]
  static constexpr int KM = 8 * KB;                    // (kappa 2^(G_end - G))^T: [16 channels][tokens]
  static constexpr int TF = 12 * KB, QF = TF + 4;      // T, Q: [token block][tokens]
  static constexpr int VEC = QF + 4;                   // fp32: 2^G_end [K], rk [32], rq [32]
  static constexpr int NF = VEC + 1;
  // delta_apply: what the state is multiplied by first, and the rest
  static constexpr int NA = KM, NB = NF - KM;
};

struct Vec8 { f32x4_t u[2]; };  // a lane's 8 channels (or tokens), 16 u + 4 fg + e
__device__ __forceinline__ Split split8(const Vec8& v) { return split8(v.u[0], v.u[1]); }
#define V8(expr)                                                                         \
  [&] {                                                                                  \
    Vec8 r_;                                                                             \
    _Pragma("unroll") for (int u = 0; u < 2; ++u)                                        \
        _Pragma("unroll") for (int e = 0; e < 4; ++e) r_.u[u][e] = (expr);                \
    return r_;                                                                           \
  }()

template <int D> __device__ __forceinline__ float row_shr(float v) {  // lane fr - D of the 16, 0 before the first
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x110 | D, 0xf, 0xf, true));
}
__device__ __forceinline__ float row_scan(float v) {  // inclusive sums over the 16 lanes
  v += row_shr<1>(v);
  v += row_shr<2>(v);
  v += row_shr<4>(v);
  return v + row_shr<8>(v);
}
template <int L> __device__ __forceinline__ float row_lane(float v) {  // lane L of the 16
  return __int_as_float(__builtin_amdgcn_ds_swizzle(__float_as_int(v), L << 5 | 0x10));
}

// LDS of a wave, used in turn: two terms of 32 tokens x 32 channels to be transposed; the solve.
struct PrepLds {
  static constexpr int ROW = 80;                                     // bytes of a token's 32 channels
  static constexpr int SM = 0, SQ = 32 * 36 * 4, SD = 2 * SQ;        // fp32 [32][36] twice, [3][16][17]
  static constexpr int TOK = SD + 3 * 16 * 17 * 4, BYTES = TOK + 32 * 4;  // b
};
static_assert(2 * 32 * PrepLds::ROW <= PrepLds::TOK, "the staged tile shares the solve's space");

template <int KB>
__global__ void __launch_bounds__(256, 2) delta_prep_kernel(ChunkArgs p) {
  using C = DC<KB>;
  const DeltaArgs& a = p.a;
  __shared__ __attribute__((aligned(16))) char smem[4 * PrepLds::BYTES];
  constexpr int K = C::K;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, fr = lane & 15, fg = lane >> 4;
  const int item = blockIdx.x * 4 + wv;
  if (item >= p.ch.n * a.H) return;  // the waves share nothing: no barriers below
  const int ci = item / a.H, h = item % a.H, hk = h / (a.H / a.G);
  const int b = p.ch.ck[2 * ci], s1 = a.m.cu[b + 1], t0 = a.m.cu[b] + p.ch.ck[2 * ci + 1] * CT;
  if (s1 - a.m.cu[b] < a.below) return;
  char* lds = smem + wv * PrepLds::BYTES;
  char* out = p.frags + (size_t)item * C::NF * 1024 + lane * 16;
  float* vec = (float*)(p.frags + ((size_t)item * C::NF + C::VEC) * 1024);
  auto wait_own = [] {  // this wave's LDS writes are read back by itself
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_wave_barrier();
  };
  auto put = [&](int f, const Split& v) {
    *(bf16x8_t*)(out + f * 1024) = v.hi;
    *(bf16x8_t*)(out + (f + 1) * 1024) = v.lo;
  };

  // rows of this lane's two tokens
  const bf16_t *xq[2], *xk[2];
  const float* xg[2];
  bool in[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int t = t0 + 16 * i + fr;
    in[i] = t < s1;
    const size_t row = min(t, s1 - 1);
    xq[i] = (const bf16_t*)a.x + row * a.ldx + hk * K + 4 * fg;
    xk[i] = xq[i] + a.G * K;
    xg[i] = a.decay + row * a.H * K + (size_t)h * K + 4 * fg;
  }
  struct Raw { u32x2_t q[2][2], k[2][2]; f32x4_t g[2][2]; };
  auto load = [&](int ks) {
    Raw r;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        r.q[i][u] = *(const u32x2_t*)(xq[i] + ks * 32 + 16 * u);
        r.k[i][u] = *(const u32x2_t*)(xk[i] + ks * 32 + 16 * u);
        r.g[i][u] = *(const f32x4_t*)(xg[i] + ks * 32 + 16 * u);
      }
    return r;
  };
  f32x4_t M[3], Q[3];  // blocks (0, 0), (1, 1), (1, 0)
#pragma unroll
  for (int i = 0; i < 3; ++i) M[i] = Q[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float nk[2] = {0.f, 0.f}, nq[2] = {0.f, 0.f};

  Raw next = load(0);
#pragma unroll 1
  for (int ks = 0; ks < KB; ++ks) {
    const Raw r = next;
    if (ks + 1 < KB) next = load(ks + 1);
    Vec8 k[2], q[2], g[2], L[2], P[2], E[2], eT[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      auto half = [&](const u32x2_t& w, int e) {
        return in[i] ? __uint_as_float(e & 1 ? w[e >> 1] & 0xffff0000u : w[e >> 1] << 16) : 0.f;
      };
      k[i] = V8(half(r.k[i][u], e));
      q[i] = V8(half(r.q[i][u], e));
      g[i] = V8(in[i] ? r.g[i][u][e] : 0.f);
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          nk[i] = fmaf(k[i].u[u][e], k[i].u[u][e], nk[i]);
          nq[i] = fmaf(q[i].u[u][e], q[i].u[u][e], nq[i]);
        }
      L[i] = V8(row_scan(g[i].u[u][e]));
      const Vec8 T = V8(row_lane<15>(L[i].u[u][e]));
      P[i] = V8(__builtin_amdgcn_exp2f(L[i].u[u][e]));                  // from the block's start
      E[i] = V8(k[i].u[u][e] * __builtin_amdgcn_exp2f(T.u[u][e] - L[i].u[u][e]));  // kappa to the block's end
      eT[i] = V8(row_lane<15>(P[i].u[u][e]));
      const Vec8 ka = V8(k[i].u[u][e] * P[i].u[u][e]), qa = V8(q[i].u[u][e] * P[i].u[u][e]);
      const Split sk = split8(ka), sq = split8(qa);
      if (i == 0) {
        put(C::KP + ks * 2, sk);
        put(C::QP + ks * 2, sq);
      } else {
        const Split B = split8(E[0]);
        M[2] = mma3(sk, B, M[2]);
        Q[2] = mma3(sq, B, Q[2]);
        put(C::KP + (KB + ks) * 2, split8(V8(ka.u[u][e] * eT[0].u[u][e])));
        put(C::QP + (KB + ks) * 2, split8(V8(qa.u[u][e] * eT[0].u[u][e])));
      }
      float lowest = 0.f;
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int e = 0; e < 4; ++e) lowest = fminf(lowest, T.u[u][e]);
      if (!__any(lowest < -100.f)) {
        const Split B = split8(V8(k[i].u[u][e] * __builtin_amdgcn_exp2f(-L[i].u[u][e])));
        M[i] = mma3(sk, B, M[i]);
        Q[i] = mma3(sq, B, Q[i]);
      } else {
        const Vec8 l = V8(row_scan(fmaxf(g[i].u[u][e], -24.f)));
        const Vec8 m0 = V8(row_lane<3>(l.u[u][e])), m1 = V8(row_lane<11>(l.u[u][e]));
        const bool up = fr >= 8;
        const Vec8 to = V8(__builtin_amdgcn_exp2f(l.u[u][e] - (up ? m1.u[u][e] : m0.u[u][e])));
        const Vec8 col = V8(k[i].u[u][e] * __builtin_amdgcn_exp2f((up ? m1.u[u][e] : m0.u[u][e]) - l.u[u][e]));
        // the step between the middles in two: the factor alone may underflow where the product does not
        const Vec8 half_step = V8(up ? 1.f : __builtin_amdgcn_exp2f(0.5f * (m1.u[u][e] - m0.u[u][e])));
        // rows 0 .. 7 against columns 0 .. 7, then rows 8 .. 15 against all
        Split B = split8(V8(up ? 0.f : col.u[u][e]));
        M[i] = mma3(split8(V8(up ? 0.f : k[i].u[u][e] * to.u[u][e])), B, M[i]);
        Q[i] = mma3(split8(V8(up ? 0.f : q[i].u[u][e] * to.u[u][e])), B, Q[i]);
        B = split8(V8(col.u[u][e] * half_step.u[u][e] * half_step.u[u][e]));
        M[i] = mma3(split8(V8(up ? k[i].u[u][e] * to.u[u][e] : 0.f)), B, M[i]);
        Q[i] = mma3(split8(V8(up ? q[i].u[u][e] * to.u[u][e] : 0.f)), B, Q[i]);
      }
    }
    if (fr == 0)
#pragma unroll
      for (int u = 0; u < 2; ++u) *(f32x4_t*)(vec + ks * 32 + 16 * u + 4 * fg) = eT[0].u[u] * eT[1].u[u];
    // kappa to the chunk's end, transposed: rows are channels
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const Split v = split8(i ? E[1] : V8(E[0].u[u][e] * eT[1].u[u][e]));
      char* w = lds + (16 * i + fr) * PrepLds::ROW + fg * 8;
      const u32x4_t hi = __builtin_bit_cast(u32x4_t, v.hi), lo = __builtin_bit_cast(u32x4_t, v.lo);
      *(u32x2_t*)w = u32x2_t{hi[0], hi[1]};
      *(u32x2_t*)(w + 32) = u32x2_t{hi[2], hi[3]};
      w += 32 * PrepLds::ROW;
      *(u32x2_t*)w = u32x2_t{lo[0], lo[1]};
      *(u32x2_t*)(w + 32) = u32x2_t{lo[2], lo[3]};
    }
    wait_own();
#pragma unroll
    for (int c = 0; c < 2; ++c)
#pragma unroll
      for (int part = 0; part < 2; ++part) {
        const char* v = lds + (part * 32 + 4 * fg + (fr >> 2)) * PrepLds::ROW + (c * 16 + 4 * (fr & 3)) * 2;
        const s16x4_t x = lds_read_tr16(v), y = lds_read_tr16(v + 16 * PrepLds::ROW);
        *(bf16x8_t*)(out + (C::KM + (2 * ks + c) * 2 + part) * 1024) =
            bf16x8_t{x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]};
      }
    wait_own();
  }

  // norms and write strengths of the tokens
  float* sM = (float*)(lds + PrepLds::SM);
  float* sQ = (float*)(lds + PrepLds::SQ);
  float* sD = (float*)(lds + PrepLds::SD);
  float* sB = (float*)(lds + PrepLds::TOK);
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    nk[i] += __shfl_xor(nk[i], 16, 64);
    nk[i] = sum_xhalf(nk[i]) + a.eps;
    nq[i] += __shfl_xor(nq[i], 16, 64);
    nq[i] = sum_xhalf(nq[i]) + a.eps;
    if (fg == 0) {
      vec[K + 16 * i + fr] = 1.f / sqrtf(nk[i]);
      vec[K + CT + 16 * i + fr] = a.q_scale / sqrtf(nq[i]);
      const float bt = bf2f(((const bf16_t*)a.beta)[(size_t)min(t0 + 16 * i + fr, s1 - 1) * a.ldb + h]);
      sB[16 * i + fr] = in[i] ? sigmoid32(bt) / nk[i] : 0.f;
    }
  }
  wait_own();
#pragma unroll
  for (int i = 0; i < 3; ++i) {
    const int r0 = i ? 16 : 0, c0 = i == 1 ? 16 : 0;
    const f32x4_t bt = *(const f32x4_t*)(sB + r0 + 4 * fg);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      sM[(r0 + 4 * fg + e) * 36 + c0 + fr] = M[i][e] * bt[e];
      sQ[(r0 + 4 * fg + e) * 36 + c0 + fr] = Q[i][e];
    }
  }
  wait_own();
  // the diagonal blocks' inverses by columns: lanes fg & 1 == blk take block blk, column fr
  const int blk = fg & 1;
  float x[16];
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    float v = r == fr ? 1.f : 0.f;
    const float* Lr = sM + (blk * 16 + r) * 36 + blk * 16;
#pragma unroll
    for (int i = 0; i < r; ++i) v = fmaf(-Lr[i], x[i], v);
    x[r] = v;
  }
  if (fg < 2)
#pragma unroll
    for (int r = 0; r < 16; ++r) sD[(blk * 16 + r) * 17 + fr] = x[r];
  // Q's lower triangle as fragments
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = 16 * i + fr;
    put(C::QF + i * 2, split8(V8(16 * u + 4 * fg + e <= r ? sQ[r * 36 + 16 * u + 4 * fg + e] : 0.f)));
  }
  wait_own();
  f32x4_t y{0.f, 0.f, 0.f, 0.f}, z = y;  // the block below the diagonal: -D1 (L10 D0)
#pragma unroll
  for (int i = 0; i < 4; ++i)
    y = __builtin_amdgcn_mfma_f32_16x16x4f32(sM[(16 + fr) * 36 + 4 * i + fg], sD[(4 * i + fg) * 17 + fr], y, 0, 0, 0);
#pragma unroll
  for (int e = 0; e < 4; ++e) sD[(32 + 4 * fg + e) * 17 + fr] = y[e];
  wait_own();
#pragma unroll
  for (int i = 0; i < 4; ++i)
    z = __builtin_amdgcn_mfma_f32_16x16x4f32(sD[(16 + fr) * 17 + 4 * i + fg], sD[(32 + 4 * i + fg) * 17 + fr], z, 0, 0, 0);
  const float bc = sB[fr], bd = sB[blk * 16 + fr];
#pragma unroll
  for (int e = 0; e < 4; ++e) sQ[(16 + 4 * fg + e) * 36 + fr] = -z[e] * bc;
  if (fg < 2)
#pragma unroll
    for (int r = 0; r < 16; ++r) sQ[(blk * 16 + r) * 36 + blk * 16 + fr] = x[r] * bd;
  wait_own();
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = 16 * i + fr;
    put(C::TF + i * 2, split8(V8(16 * u + 4 * fg + e <= r ? sQ[r * 36 + 16 * u + 4 * fg + e] : 0.f)));
  }
}

typedef __attribute__((address_space(1))) const void* frag_g_t;
typedef __attribute__((address_space(3))) void* frag_l_t;

template <int N> __device__ __forceinline__ void vm_wait() {  // all but this wave's last N memory operations are done
  asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory");
}

// LDS of NW waves: part A of three chunks (two with 8 waves, whose V takes the space), part B of two; V of the workgroup's
// columns of two.
template <int KB, int NW> struct DL {
  using C = DC<KB>;
  static constexpr int AHEAD = NW == 8 ? 1 : 2, B = (AHEAD + 1) * C::NA, VB = CT * 16 * NW * 2;  // chunks; fragments; bytes
  static constexpr int V = (B + 2 * C::NB) * 1024, BYTES = V + 2 * VB;
  static_assert(BYTES <= 160 * 1024, "LDS");
};

template <int KB, int NW>  // NW waves
__global__ void __launch_bounds__(64 * NW, NW == 8 ? 2 : 1) delta_apply_kernel(ChunkArgs p) {
  using C = DC<KB>;
  using D = DL<KB, NW>;
  const DeltaArgs& a = p.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int K = C::K;
  const int b = blockIdx.z, h = blockIdx.y;
  const int t0 = a.m.cu[b], t1 = a.m.cu[b + 1];
  if (t1 - t0 < a.below) return;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, fr = lane & 15, fg = lane >> 4;
  const int col = blockIdx.x * NW * 16 + wv * 16 + fr, colc = min(col, a.V - 1);
  const bool live = col < a.V;
  float* st = a.state + (((size_t)a.m.slot[b] * a.H + h) * a.V + colc) * K + 4 * fg;
  f32x4_t S[2 * KB];
  const bool stored = a.m.pos0[b] != 0;
#pragma unroll
  for (int i = 0; i < 2 * KB; ++i) {
    S[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (stored) S[i] = *(const f32x4_t*)(st + 16 * i);
  }
  const char* src = p.frags + ((size_t)p.ch.base[b] * a.H + h) * C::NF * 1024 + lane * 16;
  const size_t stride = (size_t)a.H * C::NF * 1024;
  const int nc = (t1 - t0 + CT - 1) / CT;
  // a chunk's two parts to LDS, PA and PB instructions a wave (chunks past the last one: that one again, unread)
  constexpr int PA = (C::NA + NW - 1) / NW, PB = (C::NB + NW - 1) / NW;
  auto issue_a = [&](int k) {
    const char* from = src + min(k, nc - 1) * stride;
    char* to = smem + k % (D::AHEAD + 1) * C::NA * 1024;
#pragma unroll
    for (int i = 0; i < PA; ++i) {
      const int f = min(wv + i * NW, C::NA - 1);
      __builtin_amdgcn_global_load_lds((frag_g_t)(from + f * 1024), (frag_l_t)(to + f * 1024), 16, 0, 0);
    }
  };
  auto issue_b = [&](int k) {
    const char* from = src + min(k, nc - 1) * stride + C::KM * 1024;
    char* to = smem + (D::B + (k & 1) * C::NB) * 1024;
#pragma unroll
    for (int i = 0; i < PB; ++i) {
      const int f = min(wv + i * NW, C::NB - 1);
      __builtin_amdgcn_global_load_lds((frag_g_t)(from + f * 1024), (frag_l_t)(to + f * 1024), 16, 0, 0);
    }
  };
  // V's tokens x columns, one instruction a wave: 16 bytes a lane, 2 NW lanes a token
  auto issue_v = [&](int k) {
    const int i = wv * 64 + lane, c = min(blockIdx.x * NW * 16 + i % (2 * NW) * 8, a.V - 8);
    const bf16_t* from = (const bf16_t*)a.x + (size_t)min(t0 + min(k, nc - 1) * CT + i / (2 * NW), t1 - 1) * a.ldx + 2 * a.G * K +
                         h * a.V + c;
    __builtin_amdgcn_global_load_lds((frag_g_t)from, (frag_l_t)(smem + D::V + (k & 1) * D::VB + wv * 1024), 16, 0, 0);
  };
  f32x4_t O[2];
  auto store_o = [&](int t) {
    if (!live) return;
    bf16_t* o = (bf16_t*)a.o + (size_t)(t + 4 * fg) * a.ldo + h * a.V + col;
    if (t + CT <= t1) {
#pragma unroll
      for (int i = 0; i < 8; ++i) o[(size_t)((i >> 2) * 16 + (i & 3)) * a.ldo] = f2bf(O[i >> 2][i & 3]);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (t + 4 * fg + (i >> 2) * 16 + (i & 3) < t1) o[(size_t)((i >> 2) * 16 + (i & 3)) * a.ldo] = f2bf(O[i >> 2][i & 3]);
    }
  };
  issue_a(0);
  issue_b(0);
  issue_v(0);
  if (D::AHEAD == 2) issue_a(1);
  // LDS reads run a step ahead of the products that use them; the scheduling barriers keep them there.
  for (int k = 0; k < nc; ++k) {
    const int t = t0 + k * CT;
    vm_wait<D::AHEAD == 2 ? PA : 0>();  // all but the next chunk's part A
    lds_barrier();  // this chunk's fragments are there; every wave is done with the last chunk's
    const char* bufa = smem + k % (D::AHEAD + 1) * C::NA * 1024;
    const char* bufb = smem + (D::B + (k & 1) * C::NB - C::KM) * 1024;
    const float* vec = (const float*)(bufb + C::VEC * 1024);
    auto frag = [&](int f) {
      const char* q = (f < C::NA ? bufa : bufb) + f * 1024 + lane * 16;
      return Split{*(const bf16x8_t*)q, *(const bf16x8_t*)(q + 1024)};
    };
    Split kp[2][2], qp[2][2], tf[2], qf[2], km[4];
    auto load_ks = [&](int ks) {
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        kp[ks & 1][i] = frag(C::KP + (i * KB + ks) * 2);
        qp[ks & 1][i] = frag(C::QP + (i * KB + ks) * 2);
      }
    };
    load_ks(0);
    f32x4_t rk[2], rq[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      rk[i] = *(const f32x4_t*)(vec + K + 16 * i + 4 * fg);
      rq[i] = *(const f32x4_t*)(vec + K + CT + 16 * i + 4 * fg);
    }
    if (k) store_o(t - CT);
    issue_b(k + 1);
    issue_v(k + 1);
    issue_a(k + D::AHEAD);
    f32x4_t R[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) R[i] = O[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KB; ++ks) {
      if (ks + 1 < KB) {
        load_ks(ks + 1);
      } else {
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          tf[i] = frag(C::TF + i * 2);
          qf[i] = frag(C::QF + i * 2);
        }
      }
      __builtin_amdgcn_sched_barrier(0);
      const Split B = split8(S[2 * ks], S[2 * ks + 1]);
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        R[i] = mma3(kp[ks & 1][i], B, R[i]);
        O[i] = mma3(qp[ks & 1][i], B, O[i]);
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    constexpr int PRE = 2 * KB < 4 ? 2 * KB : 4;
    f32x4_t end[2 * KB];
#pragma unroll
    for (int i = 0; i < PRE; ++i) km[i] = frag(C::KM + i * 2);
#pragma unroll
    for (int i = 0; i < 2 * KB; ++i) end[i] = *(const f32x4_t*)(vec + 16 * i + 4 * fg);
    const bf16_t* vl = (const bf16_t*)(smem + D::V + (k & 1) * D::VB) + 4 * fg * 16 * NW + wv * 16 + fr;
    unsigned rv[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) rv[i] = vl[((i >> 2) * 16 + (i & 3)) * 16 * NW];
    __builtin_amdgcn_sched_barrier(0);
    f32x4_t X[2], U[2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        X[i][e] = t + 16 * i + 4 * fg + e < t1
                      ? fmaf(__uint_as_float(rv[4 * i + e] << 16), __builtin_amdgcn_rcpf(rk[i][e]), -R[i][e]) : 0.f;
    Split B = split8(X[0], X[1]);
#pragma unroll
    for (int i = 0; i < 2; ++i) U[i] = mma3(tf[i], B, f32x4_t{0.f, 0.f, 0.f, 0.f});
    B = split8(U[0], U[1]);
#pragma unroll
    for (int i = 0; i < 2 * KB; ++i) S[i] *= end[i];
#pragma unroll
    for (int i = 0; i < 2; ++i) O[i] = mma3(qf[i], B, O[i]) * rq[i];
#pragma unroll
    for (int i = 0; i < 2 * KB; ++i) {
      S[i] = mma3(km[i % PRE], B, S[i]);
      if (i + PRE < 2 * KB) km[i % PRE] = frag(C::KM + (i + PRE) * 2);
    }
  }
  store_o(t0 + (nc - 1) * CT);
  if (live)
#pragma unroll
    for (int i = 0; i < 2 * KB; ++i) *(f32x4_t*)(st + 16 * i) = S[i];
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // no transfer to LDS outlives its workgroup
  const int wg = blockIdx.y * gridDim.x + blockIdx.x, step = gridDim.x * gridDim.y * 64 * NW;
  for (int c = wg * 64 * NW + threadIdx.x; c < a.conv.C; c += step) conv_state_store<bf16_t>(a.conv, a.m, b, c);
}

template <int KB, int NW>
static int launch_delta_apply(const ChunkArgs& p, hipStream_t s) {
  static const hipError_t e = hipFuncSetAttribute((const void*)delta_apply_kernel<KB, NW>,
                                                  hipFuncAttributeMaxDynamicSharedMemorySize, DL<KB, NW>::BYTES);
  if (e != hipSuccess) return (int)e;
  const DeltaArgs& a = p.a;
  delta_apply_kernel<KB, NW><<<dim3((a.V + 16 * NW - 1) / (16 * NW), a.H, a.m.B), 64 * NW, DL<KB, NW>::BYTES, s>>>(p);
  DA_LAUNCH_CHECK();
}
template <int KB>
static int launch_delta_chunk(const ChunkArgs& p, hipStream_t s) {
  const DeltaArgs& a = p.a;
  delta_prep_kernel<KB><<<(p.ch.n * a.H + 3) / 4, 256, 0, s>>>(p);
  // a head's columns on one CU where the heads fill the chip, else spread over more
  const long long heads = (long long)a.m.B * a.H;
  if (heads * ((a.V + 127) / 128) >= 256) return launch_delta_apply<KB, 8>(p, s);
  if (heads * ((a.V + 63) / 64) >= 256) return launch_delta_apply<KB, 4>(p, s);
  return launch_delta_apply<KB, 2>(p, s);
}

// o / rms(o) * w * sigmoid(gate), in place, per head: `lanes` lanes a head, U pieces of 4 columns of theirs in registers.
template <typename T, int U>
__global__ void __launch_bounds__(256)
head_norm_kernel(T* o, int ldo, const T* gate, int ldg, const float* w, int T_, int H, int V, int dim, float eps, int lanes) {
  const int item = blockIdx.x * (256 / lanes) + threadIdx.x / lanes, l = threadIdx.x % lanes;
  const bool live = item < T_ * H;
  const int it = live ? item : T_ * H - 1, t = it / H, h = it % H;
  T* r = o + (size_t)t * ldo + (size_t)h * V;
  const T* gr = gate + (size_t)t * ldg + (size_t)h * V;
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
static int launch_delta_t(const ChunkArgs& p0, int min_len, const void* w, const void* gate, int ldg, int dim, float eps,
                          hipStream_t s) {
  ChunkArgs p = p0;
  DeltaArgs& a = p.a;
  int err = 0;
  if (sizeof(T) == 2 && p.ch.n && a.V % 8 == 0 && a.ldx % 8 == 0) {
    switch (a.K) {
      case 32: err = launch_delta_chunk<1>(p, s); break;
      case 64: err = launch_delta_chunk<2>(p, s); break;
      case 96: err = launch_delta_chunk<3>(p, s); break;
      case 128: err = launch_delta_chunk<4>(p, s); break;
      default: return (int)hipErrorInvalidValue;
    }
    if (err) return err;
  } else {
    a.below = 0x7fffffff;
  }
  if (min_len < a.below) switch (a.K) {
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
  auto norm = a.V <= 4 * lanes ? head_norm_kernel<T, 1> : head_norm_kernel<T, 4>;
  norm<<<(unsigned)(((size_t)a.m.T * a.H + per - 1) / per), 256, 0, s>>>((T*)a.o, a.ldo, (const T*)gate, ldg, (const float*)w,
                                                                        a.m.T, a.H, a.V, dim, eps, lanes);
  DA_LAUNCH_CHECK();
}

// x [T][ldx] (activation type): G query heads, G key heads of K channels, H value heads of V; decay fp32 [T][H K];
// K = 32 n (n <= 8), 64 n (n <= 8) or 128 n (n <= 8); V % 4 == 0. norm weight w fp32 [V], gate [T][ldg]; dim: the
// channels a value head really has. conv: as the other recurrences' (state null: kept by the convolution's launch).
// min_len: shortest portion. Chunk list ck / base (n_chunks of them, 32 tokens each, of all portions) and scratch frags
// [n_chunks][H][(3 K / 8 + 9) KB]: bf16 portions of chunk_from tokens or more run in chunks (K 32, 64, 96 or 128).
DA_EXPORT int da_delta_rule(const void* x, int ldx, const void* decay, const void* beta, int ldb, void* state, void* o,
                            int ldo, int H, int G, int K, int V, float q_scale, float unit_eps, const void* w,
                            const void* gate, int ldg, int dim, float eps, const void* conv_x, int ld_conv,
                            void* conv_state, int taps, int conv_c, int min_len, int chunk_from, const void* ck,
                            const void* base, int n_chunks, void* frags, const void* cu,
                            const void* slot, const void* pos0, const void* seq, int T, int B, int f32, void* stream) {
  if (T < 1 || B < 1 || B > 65535 || G < 1 || H % G || H > 65535 || V < 4 || V % 4 ||
      ldx % 4 || ldo % 4 || ldg % 4 || dim < 1 || dim > V || taps < 1 || min_len < 1 || chunk_from < 1 || n_chunks < 0 ||
      (n_chunks && (!ck || !base || !frags)) || (long long)n_chunks * H > 0x7fffffffll / 4 ||
      (long long)T * H > 0x7fffffffll / 4)
    return (int)hipErrorInvalidValue;
  ChunkArgs p{DeltaArgs{x, ldx, (const float*)decay, beta, ldb, (float*)state, o, ldo, H, G, K, V, q_scale, unit_eps, chunk_from,
                        ConvState{conv_x, ld_conv, conv_state, taps, conv_c},
                        SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}},
              ChunkMeta{(const int*)ck, (const int*)base, n_chunks, CT}, (char*)frags};
  return f32 ? launch_delta_t<float>(p, min_len, w, gate, ldg, dim, eps, (hipStream_t)stream)
             : launch_delta_t<bf16_t>(p, min_len, w, gate, ldg, dim, eps, (hipStream_t)stream);
}
