// Gated delta rule with a decay per key channel, over a batch of portions (SeqMeta), state per sequence slot.
//
// Per token and head, S [K][V] in fp32 (stored [V][K]), a = exp2(log decay) per key channel:
//   S <- a S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
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

// ------------------------------------------------------------------------------- matrix cores, chunks of 32 tokens
// With kappa, chi the keys and queries before their unit norms (norms rk, rq: k = rk kappa, q = rq chi), G_t the cumulative
// log2 decay of a channel from the chunk's start to token t, S the state before the chunk:
//   M_tj = sum_c kappa_t kappa_j 2^(G_t - G_j),  Q_tj likewise with chi_t,  b_t = beta_t rk_t^2
//   T  = (I + diag(b) tril(M, -1))^-1 diag(b)
//   U  = T (V / rk - (kappa 2^G) S)                                 rows u_t rk_t: what the tokens write
//   o  = rq ((chi 2^G) S + tril(Q) U)
//   S <- 2^G_end S + (kappa 2^(G_end - G))^T U
// A workgroup of 8 waves walks a head's chunks; it forms the operands together (in LDS, as MFMA fragments), then each wave
// runs 16 columns of V and S by itself, S staying in its accumulators.
//
// Every fp32 operand enters its product as two bf16 terms (its rounding and the remainder), three of their four
// products taken: about 16 bits, accumulated in fp32. The solve of T's blocks is in fp32.
//
// M and Q: rows of an 8-token block are scaled by 2^(G_t - m) and columns by 2^(m - G_j), m the cumulative decay at the
// block's middle, so no factor leaves the range of an exponent as long as a token's decay is at least 2^-24; stronger ones
// count as that there (less than the rounding of what they are added to).
constexpr int CT = 32;                          // tokens of a chunk
constexpr int FG_B = 272, FRAG = 4 * FG_B;      // bytes: a fragment's four lane rows, padded apart; a fragment

// Operand with rows of 16 (lane fr) and 32 k values: k sits at lane row (k % 16) / 4, element (k / 16) * 4 + k % 4, the
// order in which an accumulator's rows become the other operand.
__device__ __forceinline__ int frag_at(int fr, int k) { return (k & 15) / 4 * FG_B + fr * 16 + ((k >> 4) * 4 + (k & 3)) * 2; }

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
__device__ __forceinline__ Split frag_load(const char* p, int lane) {
  p += (lane >> 4) * FG_B + (lane & 15) * 16;
  return {*(const bf16x8_t*)p, *(const bf16x8_t*)(p + FRAG)};
}

template <int KB> struct DC {                   // K = 32 KB key channels
  static constexpr int K = 32 * KB, OP = 4 * KB * FRAG;  // an operand of 32 tokens x K, both terms
  static constexpr int KP = 0, QP = OP, KM = 2 * OP, AK = 3 * OP, AQ = 4 * OP, BK = 5 * OP;
  static constexpr int TF = 6 * OP, QF = TF + 4 * FRAG;  // T and Q: 2 row blocks, both terms
  static constexpr int SM = QF + 4 * FRAG;               // diag(b) M: fp32 [32][36]
  static constexpr int SD = SM + 32 * 36 * 4;            // solve: fp32 [3][16][17]
  static constexpr int TOT = SD + 3 * 16 * 17 * 4;       // decay sums of 4 tokens: fp32 [2][8][K] (as they are, limited)
  static constexpr int MID = TOT + 2 * 8 * K * 4;        // fp32 [4][K]
  static constexpr int END = MID + 4 * K * 4;            // 2^G_end: fp32 [K]
  static constexpr int TOK = END + K * 4;                // per token, two chunks: rk, rq, b
  static constexpr int BYTES = TOK + 2 * 3 * CT * 4;
};

template <int KB>
__global__ void __launch_bounds__(512, 2) delta_chunk_kernel(DeltaArgs a) {
  using C = DC<KB>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int K = C::K, LP = KB == 1 ? 16 : KB == 2 ? 32 : 64;  // lanes of a token: a channel pair each
  const int b = blockIdx.z, h = blockIdx.y, hk = h / (a.H / a.G);
  const int t0 = a.m.cu[b], t1 = a.m.cu[b + 1];
  if (t1 - t0 < a.below) return;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, fr = lane & 15, fg = lane >> 4;
  const int pair = tid % LP, grp = tid / LP;                // staging: two channels of the chunk's tokens 4 grp ..
  const bool on = grp < 8 && 2 * pair < K;
  const int ch = min(2 * pair, K - 2);
  float* sM = (float*)(smem + C::SM);
  float* sD = (float*)(smem + C::SD);
  float* sT = (float*)(smem + C::TOT);
  float* sMid = (float*)(smem + C::MID);
  float* sEnd = (float*)(smem + C::END);

  for (int i = tid; i < 8 * FRAG / 16; i += 512) *(u32x4_t*)(smem + C::TF + i * 16) = u32x4_t{0, 0, 0, 0};

  // this wave's columns
  const int col = blockIdx.x * 128 + wv * 16 + fr, colc = min(col, a.V - 1);
  const bool live = col < a.V;
  float* st = a.state + (((size_t)a.m.slot[b] * a.H + h) * a.V + colc) * K + 4 * fg;
  f32x4_t S[2 * KB];
  const bool stored = a.m.pos0[b] != 0;
#pragma unroll
  for (int i = 0; i < 2 * KB; ++i) {
    S[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (stored) S[i] = *(const f32x4_t*)(st + 16 * i);
  }

  unsigned rk[4], rq[4];
  f32x2_t rg[4];
  bf16_t rv[8], rb = 0;
  auto fetch = [&](int t) {
    const bf16_t* x = (const bf16_t*)a.x;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const size_t row = min(t + 4 * min(grp, 7) + i, t1 - 1);
      rq[i] = *(const unsigned*)(x + row * a.ldx + hk * K + ch);
      rk[i] = *(const unsigned*)(x + row * a.ldx + (a.G + hk) * K + ch);
      rg[i] = *(const f32x2_t*)(a.decay + row * a.H * K + (size_t)h * K + ch);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i)
      rv[i] = x[(size_t)min(t + (i >> 2) * 16 + 4 * fg + (i & 3), t1 - 1) * a.ldx + 2 * a.G * K + h * a.V + colc];
    if (pair < 4) rb = ((const bf16_t*)a.beta)[(size_t)min(t + 4 * min(grp, 7) + pair, t1 - 1) * a.ldb + h];
  };

  fetch(t0);
  for (int t = t0, par = 0; t < t1; t += CT, par ^= 1) {
    float* tok_rk = (float*)(smem + C::TOK) + par * 3 * CT;
    float *tok_rq = tok_rk + CT, *tok_b = tok_rq + CT;
    // ---- sums of this thread's 4 tokens, norms of the tokens; tokens past the end are zero and decay nothing
    f32x2_t kap[4], chi[4], g[4], gl[4];
    f32x2_t vv[4];  // V / rk comes later: V of the wave's columns, rows 4 fg + (0..3) of both token blocks
    float nk[4], nq[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const bool in = on && t + 4 * grp + i < t1;
      kap[i] = in ? f32x2_t{__uint_as_float(rk[i] << 16), __uint_as_float(rk[i] & 0xffff0000u)} : f32x2_t{0.f, 0.f};
      chi[i] = in ? f32x2_t{__uint_as_float(rq[i] << 16), __uint_as_float(rq[i] & 0xffff0000u)} : f32x2_t{0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const float d = in ? rg[i][e] : 0.f;
        g[i][e] = (i ? g[i - 1][e] : 0.f) + d;
        gl[i][e] = (i ? gl[i - 1][e] : 0.f) + fmaxf(d, -24.f);
      }
      nk[i] = fmaf(kap[i][0], kap[i][0], kap[i][1] * kap[i][1]);
      nq[i] = fmaf(chi[i][0], chi[i][0], chi[i][1] * chi[i][1]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      vv[i] = f32x2_t{bf2f(rv[i]), bf2f(rv[4 + i])};
      nk[i] = lanes_sum<16>(nk[i]);
      nq[i] = lanes_sum<16>(nq[i]);
      if constexpr (LP > 16) {
        nk[i] += __shfl_xor(nk[i], 16, 64);
        nq[i] += __shfl_xor(nq[i], 16, 64);
      }
      if constexpr (LP > 32) {
        nk[i] = sum_xhalf(nk[i]);
        nq[i] = sum_xhalf(nq[i]);
      }
    }
    if (grp < 8) {
      if (on) {
        *(f32x2_t*)(sT + grp * K + ch) = g[3];
        *(f32x2_t*)(sT + (8 + grp) * K + ch) = gl[3];
      }
      if (pair < 4) {
        const float k2 = pair == 0 ? nk[0] : pair == 1 ? nk[1] : pair == 2 ? nk[2] : nk[3];
        const float q2 = pair == 0 ? nq[0] : pair == 1 ? nq[1] : pair == 2 ? nq[2] : nq[3];
        const int i = 4 * grp + pair;
        const float r2 = 1.f / (k2 + a.eps);
        tok_rk[i] = sqrtf(r2);
        tok_rq[i] = a.q_scale / sqrtf(q2 + a.eps);
        tok_b[i] = t + i < t1 ? sigmoid32(bf2f(rb)) * r2 : 0.f;
      }
    }
    __syncthreads();
    // ---- the operands
    if (on) {
      f32x2_t base{0.f, 0.f}, basel{0.f, 0.f}, mid{0.f, 0.f}, end{0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const f32x2_t v = *(const f32x2_t*)(sT + i * K + ch), vl = *(const f32x2_t*)(sT + (8 + i) * K + ch);
        end += v;
        if (i < grp) base += v, basel += vl;
        if (i <= (grp & ~1)) mid += vl;  // the first half of this thread's block of 8
      }
      if (!(grp & 1)) *(f32x2_t*)(sMid + grp / 2 * K + ch) = mid;
      if (grp == 0)
        *(f32x2_t*)(sEnd + ch) = f32x2_t{__builtin_amdgcn_exp2f(end[0]), __builtin_amdgcn_exp2f(end[1])};
      const int ks = ch >> 5, blk = grp >> 2;
      char* row = smem + ((blk * KB + ks) * 2) * FRAG;
      f32x2_t km[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        f32x2_t kp, qp, ak, aq, bk;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float G = base[e] + g[i][e], Gm = basel[e] + gl[i][e] - mid[e];
          const float P = __builtin_amdgcn_exp2f(G), E = __builtin_amdgcn_exp2f(Gm);
          kp[e] = kap[i][e] * P;
          qp[e] = chi[i][e] * P;
          ak[e] = kap[i][e] * E;
          aq[e] = chi[i][e] * E;
          bk[e] = kap[i][e] * __builtin_amdgcn_exp2f(-Gm);
          km[i][e] = kap[i][e] * __builtin_amdgcn_exp2f(end[e] - G);
        }
        const int at = frag_at((4 * grp + i) & 15, ch & 31);
        auto put = [&](int op, const f32x2_t& v) {
          const unsigned hi = pack_bf2(v[0], v[1]);
          *(unsigned*)(row + op + at) = hi;
          *(unsigned*)(row + op + FRAG + at) = lo_of(hi, v[0], v[1]);
        };
        put(C::KP, kp);
        put(C::QP, qp);
        put(C::AK, ak);
        put(C::AQ, aq);
        put(C::BK, bk);
      }
#pragma unroll
      for (int e = 0; e < 2; ++e) {  // rows: channels; k: tokens
        char* p = smem + C::KM + ((ch + e) >> 4) * 2 * FRAG + frag_at((ch + e) & 15, 4 * grp);
        const unsigned h0 = pack_bf2(km[0][e], km[1][e]), h1 = pack_bf2(km[2][e], km[3][e]);
        *(u32x2_t*)p = u32x2_t{h0, h1};
        *(u32x2_t*)(p + FRAG) = u32x2_t{lo_of(h0, km[0][e], km[1][e]), lo_of(h1, km[2][e], km[3][e])};
      }
    }
    if (t + CT < t1) fetch(t + CT);
    __syncthreads();
    // ---- M and Q, 8 x 8 blocks by the middle that their rows are scaled to. Waves 0, 1: blocks on the diagonal; 2, 3: below
    // it within 16 tokens; 4, 5: rows 16 .. 23 and 24 .. 31 against columns 0 .. 15
    if (wv < 6) {
      const int rblk = wv < 4 ? wv & 1 : 1, cblk = wv < 4 ? wv & 1 : 0;
      const int rsub = wv < 2 ? -1 : wv < 4 ? 2 * rblk + 1 : wv - 2;  // the rows' block of 8 that this wave fills
      f32x4_t m{0.f, 0.f, 0.f, 0.f}, q = m;
#pragma unroll
      for (int ks = 0; ks < KB; ++ks) {
        Split B = frag_load(smem + C::BK + (cblk * KB + ks) * 2 * FRAG, lane);
        if (rsub >= 0) {  // column fr is scaled to its own block's middle: to the rows'
          const int c = ks * 32 + 4 * fg;
          f32x4_t v[2];
#pragma unroll
          for (int u = 0; u < 2; ++u) {
            const f32x4_t to = *(const f32x4_t*)(sMid + rsub * K + c + 16 * u);
            const f32x4_t from = *(const f32x4_t*)(sMid + (cblk * 2 + (fr >> 3)) * K + c + 16 * u);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              // in two steps: the factor alone may underflow where the product does not
              const float f = __builtin_amdgcn_exp2f(0.5f * fminf(to[e] - from[e], 0.f));
              v[u][e] = (bf2f((bf16_t)B.hi[4 * u + e]) + bf2f((bf16_t)B.lo[4 * u + e])) * f * f;
            }
          }
          B = split8(v[0], v[1]);
        }
        m = mma3(frag_load(smem + C::AK + (rblk * KB + ks) * 2 * FRAG, lane), B, m);
        q = mma3(frag_load(smem + C::AQ + (rblk * KB + ks) * 2 * FRAG, lane), B, q);
      }
      const int j = cblk * 16 + fr;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int r = rblk * 16 + 4 * fg + e;
        const bool mine = rsub < 0 ? r / 8 == j / 8 : r / 8 == rsub && (wv >= 4 || j / 8 == rsub - 1);
        if (!mine) continue;
        sM[r * 36 + j] = j < r ? m[e] * tok_b[r] : 0.f;
        const float v = j <= r ? q[e] : 0.f;
        const bf16_t hi = f2bf(v);
        char* p = smem + C::QF + rblk * 2 * FRAG + frag_at(r & 15, j);
        *(bf16_t*)p = hi;
        *(bf16_t*)(p + FRAG) = f2bf(v - bf2f(hi));
      }
    }
    __syncthreads();
    // ---- T by wave 0, while the others begin with the products of the state
    if (wv == 0) {
      const int blk = fg & 1;
      const float* L = sM + blk * 16 * 36 + blk * 16;
      float x[16];
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        float v = r == fr ? 1.f : 0.f;
#pragma unroll
        for (int i = 0; i < r; ++i) v = fmaf(-L[r * 36 + i], x[i], v);
        x[r] = v;
      }
      auto put = [&](int r, int j, float v) {  // T[r][j]
        const bf16_t hi = f2bf(v);
        char* p = smem + C::TF + (r >> 4) * 2 * FRAG + frag_at(r & 15, j);
        *(bf16_t*)p = hi;
        *(bf16_t*)(p + FRAG) = f2bf(v - bf2f(hi));
      };
      if (fg < 2) {
        const float bj = tok_b[blk * 16 + fr];
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          sD[(blk * 16 + r) * 17 + fr] = x[r];
          put(blk * 16 + r, blk * 16 + fr, x[r] * bj);
        }
      }
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // this wave's own LDS writes are read back by it alone
      __builtin_amdgcn_wave_barrier();
      f32x4_t y{0.f, 0.f, 0.f, 0.f}, z = y;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(sM[(16 + fr) * 36 + 4 * i + fg], sD[(4 * i + fg) * 17 + fr], y, 0, 0, 0);
#pragma unroll
      for (int e = 0; e < 4; ++e) sD[(32 + 4 * fg + e) * 17 + fr] = y[e];
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int i = 0; i < 4; ++i)
        z = __builtin_amdgcn_mfma_f32_16x16x4f32(sD[(16 + fr) * 17 + 4 * i + fg], sD[(32 + 4 * i + fg) * 17 + fr], z, 0, 0, 0);
#pragma unroll
      for (int e = 0; e < 4; ++e) put(16 + 4 * fg + e, fr, -z[e] * tok_b[fr]);
    }
    f32x4_t R[2], O[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) R[i] = O[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KB; ++ks) {
      const Split B = split8(S[2 * ks], S[2 * ks + 1]);
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        R[i] = mma3(frag_load(smem + C::KP + (i * KB + ks) * 2 * FRAG, lane), B, R[i]);
        O[i] = mma3(frag_load(smem + C::QP + (i * KB + ks) * 2 * FRAG, lane), B, O[i]);
      }
    }
    __syncthreads();
    // ---- what the tokens write, what they read, the state after them
    f32x4_t X[2], U[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const f32x4_t r = *(const f32x4_t*)(tok_rk + 16 * i + 4 * fg);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        X[i][e] = t + 16 * i + 4 * fg + e < t1 ? vv[e][i] * __builtin_amdgcn_rcpf(r[e]) - R[i][e] : 0.f;
      U[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    Split B = split8(X[0], X[1]);
#pragma unroll
    for (int i = 0; i < 2; ++i) U[i] = mma3(frag_load(smem + C::TF + i * 2 * FRAG, lane), B, U[i]);
    B = split8(U[0], U[1]);
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      O[i] = mma3(frag_load(smem + C::QF + i * 2 * FRAG, lane), B, O[i]);
      const f32x4_t r = *(const f32x4_t*)(tok_rq + 16 * i + 4 * fg);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int tt = t + 16 * i + 4 * fg + e;
        if (live && tt < t1) ((bf16_t*)a.o)[(size_t)tt * a.ldo + h * a.V + col] = f2bf(O[i][e] * r[e]);
      }
    }
#pragma unroll
    for (int i = 0; i < 2 * KB; ++i) {
      S[i] *= *(const f32x4_t*)(sEnd + 16 * i + 4 * fg);
      S[i] = mma3(frag_load(smem + C::KM + i * 2 * FRAG, lane), B, S[i]);
    }
  }
  if (live)
#pragma unroll
    for (int i = 0; i < 2 * KB; ++i) *(f32x4_t*)(st + 16 * i) = S[i];
  const int wg = blockIdx.y * gridDim.x + blockIdx.x, step = gridDim.x * gridDim.y * 512;
  for (int c = wg * 512 + tid; c < a.conv.C; c += step) conv_state_store<bf16_t>(a.conv, a.m, b, c);
}

template <int KB>
static int launch_delta_chunk(const DeltaArgs& a, hipStream_t s) {
  static const hipError_t e = hipFuncSetAttribute((const void*)delta_chunk_kernel<KB>,
                                                  hipFuncAttributeMaxDynamicSharedMemorySize, DC<KB>::BYTES);
  if (e != hipSuccess) return (int)e;
  delta_chunk_kernel<KB><<<dim3((a.V + 127) / 128, a.H, a.m.B), 512, DC<KB>::BYTES, s>>>(a);
  DA_LAUNCH_CHECK();
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
static int launch_delta_t(const DeltaArgs& a0, int min_len, int max_len, int chunk_from, const void* w, const void* gate, int ldg, int dim,
                          float eps, hipStream_t s) {
  DeltaArgs a = a0;
  int err = 0;
  a.below = 0x7fffffff;
  if constexpr (sizeof(T) == 2) {
    if (max_len >= chunk_from && a.K <= 128) {
      a.below = chunk_from;
      switch (a.K) {
        case 32: err = launch_delta_chunk<1>(a, s); break;
        case 64: err = launch_delta_chunk<2>(a, s); break;
        case 96: err = launch_delta_chunk<3>(a, s); break;
        default: err = launch_delta_chunk<4>(a, s); break;
      }
      if (err) return err;
    }
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
  head_norm_kernel<T><<<(unsigned)(((size_t)a.m.T * a.H + per - 1) / per), 256, 0, s>>>(
      (T*)a.o, a.ldo, (const T*)gate, ldg, (const float*)w, a.m.T, a.H, a.V, dim, eps, lanes);
  DA_LAUNCH_CHECK();
}

// x [T][ldx] (activation type): G query heads, G key heads of K channels, H value heads of V; decay fp32 [T][H K];
// K = 32 n (n <= 8), 64 n (n <= 8) or 128 n (n <= 8); V % 4 == 0. norm weight w fp32 [V], gate [T][ldg]; dim: the
// channels a value head really has. conv: as the other recurrences' (state null: kept by the convolution's launch).
// min_len / max_len: shortest and longest portion; bf16 portions of chunk_from tokens or more run in chunks where K <= 128.
DA_EXPORT int da_delta_rule(const void* x, int ldx, const void* decay, const void* beta, int ldb, void* state, void* o,
                            int ldo, int H, int G, int K, int V, float q_scale, float unit_eps, const void* w,
                            const void* gate, int ldg, int dim, float eps, const void* conv_x, int ld_conv,
                            void* conv_state, int taps, int conv_c, int min_len, int max_len, int chunk_from, const void* cu,
                            const void* slot, const void* pos0, const void* seq, int T, int B, int f32, void* stream) {
  if (T < 1 || B < 1 || B > 65535 || G < 1 || H % G || H > 65535 || V < 4 || V % 4 ||
      ldx % 4 || ldo % 4 || ldg % 4 || dim < 1 || dim > V || taps < 1 || min_len < 1 || max_len < min_len || chunk_from < 1 || ldx % 2 || (long long)T * H > 0x7fffffffll / 4)
    return (int)hipErrorInvalidValue;
  DeltaArgs a{x, ldx, (const float*)decay, beta, ldb, (float*)state, o, ldo, H, G, K, V, q_scale, unit_eps, 0,
              ConvState{conv_x, ld_conv, conv_state, taps, conv_c},
              SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}};
  return f32 ? launch_delta_t<float>(a, min_len, max_len, chunk_from, w, gate, ldg, dim, eps, (hipStream_t)stream)
             : launch_delta_t<bf16_t>(a, min_len, max_len, chunk_from, w, gate, ldg, dim, eps, (hipStream_t)stream);
}
