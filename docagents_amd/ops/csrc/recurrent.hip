// Recurrent sequence mixers over a batch of portions (SeqMeta), state per sequence slot.
//
// 1) causal_conv: short per-channel convolution (the last taps - 1 inputs of a sequence are state).
// 2) selective scan (Mamba): S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;
//    y_c = (sum_n S[c, n] C_n + D_c x_c) * silu(z_c).
// 3) gated linear recurrence: S_c <- a_c S_c + d_c, y_c = S_c * gelu(g_c).
//
// Both recurrences run in fp32 in one of two ways. Short portions (decode, up to one chunk), and
// longer ones where the sequences alone fill the chip: one launch, a thread walks its channel's tokens from the
// stored state. Else the portions are cut into chunks: (a) every chunk but a portion's last runs from zero (the first: from the stored state)
// and leaves its end state and its total decay, (b) one pass over the chunks turns those into each
// chunk's start state, (c) every chunk runs again from its start state and writes its outputs. Chunks of
// all portions fill the chip, and a token's arithmetic differs between the two ways by rounding only.
// The convolution's state is replaced by the recurrence's launch, as its own launch still reads it (in
// batches of single tokens a thread's reads are its own: there the convolution replaces it).
#include "seq.h"

// ------------------------------------------------------------------------------- convolution
struct ConvArgs {
  const void* x; const float* w; const float* bias; void* state; void* y;  // w [taps][C], bias nullable
  int ldx, ldy, C, taps;
  int update;  // single tokens only: replace the state
  SeqMeta m;
};

template <typename T>
__device__ __forceinline__ f32x4_t conv_input(const ConvArgs& a, int t, int k, int c) {
  // the input k tokens before packed row t
  const int b = a.m.seq[t], j = t - a.m.cu[b];
  if (j >= k) return Act<T>::load4((const T*)a.x + (size_t)(t - k) * a.ldx + c);
  if (a.m.pos0[b] == 0) return f32x4_t{0.f, 0.f, 0.f, 0.f};
  return Act<T>::load4((const T*)a.state + ((size_t)a.m.slot[b] * (a.taps - 1) + (a.taps - 1 + j - k)) * a.C + c);
}

template <typename T, int TAPS, int SILU, int CONV_RUN>  // CONV_RUN: consecutive tokens of a thread
__global__ void __launch_bounds__(256) causal_conv_kernel(ConvArgs a) {
  const int c = (blockIdx.x * 64 + (threadIdx.x & 63)) * 4;
  const int t0 = (blockIdx.y * 4 + (threadIdx.x >> 6)) * CONV_RUN;
  if (c >= a.C || t0 >= a.m.T) return;
  const int t1 = min(t0 + CONV_RUN, a.m.T);
  f32x4_t bias{0.f, 0.f, 0.f, 0.f};
  if (a.bias) bias = *(const f32x4_t*)(a.bias + c);
  auto emit = [&](int t, f32x4_t v) {
    if constexpr (SILU) {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = act_silu<T>(v[e]);
    }
    Act<T>::store4((T*)a.y + (size_t)t * a.ldy + c, v);
  };
  if constexpr (TAPS > 0) {
    // the run's inputs and the taps - 1 before it, all loads issued together
    f32x4_t w[TAPS], x[CONV_RUN + TAPS - 1];
#pragma unroll
    for (int k = 0; k < TAPS; ++k) w[k] = *(const f32x4_t*)(a.w + (size_t)k * a.C + c);
    const int b0 = a.m.seq[t0], b1 = a.m.seq[t1 - 1];
    if (b0 == b1) {
      const int s0 = a.m.cu[b0];
      const T* st = (const T*)a.state + (size_t)a.m.slot[b0] * (TAPS - 1) * a.C + c;
      const bool stored = a.m.pos0[b0] != 0;
#pragma unroll
      for (int i = 0; i < CONV_RUN + TAPS - 1; ++i) {
        const int t = min(t0 + i - (TAPS - 1), t1 - 1);
        const T* in = (const T*)a.x + (size_t)max(t, s0) * a.ldx + c;
        x[i] = Act<T>::load4(t < s0 && stored ? st + (size_t)(TAPS - 1 + t - s0) * a.C : in);
      }
#pragma unroll
      for (int i = 0; i + 1 < TAPS; ++i)
        if (t0 + i - (TAPS - 1) < s0 && !stored) x[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < CONV_RUN; ++i) {
        if (t0 + i >= t1) break;
        f32x4_t v = bias;
#pragma unroll
        for (int k = 0; k < TAPS; ++k)
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = fmaf(w[k][e], x[i + k][e], v[e]);
        emit(t0 + i, v);
      }
      if (CONV_RUN == 1 && a.update) {
        T* w0 = (T*)a.state + (size_t)a.m.slot[b0] * (TAPS - 1) * a.C + c;
#pragma unroll
        for (int i = 0; i + 1 < TAPS; ++i) Act<T>::store4(w0 + (size_t)i * a.C, x[i + 1]);
      }
    } else {  // a portion ends inside the run
      for (int t = t0; t < t1; ++t) {
        f32x4_t v = bias;
#pragma unroll
        for (int k = 0; k < TAPS; ++k) {
          const f32x4_t xk = conv_input<T>(a, t, TAPS - 1 - k, c);
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = fmaf(w[k][e], xk[e], v[e]);
        }
        emit(t, v);
      }
    }
  } else {
    for (int t = t0; t < t1; ++t) {
      f32x4_t v = bias;
      for (int k = 0; k < a.taps; ++k) {
        const f32x4_t w = *(const f32x4_t*)(a.w + (size_t)(a.taps - 1 - k) * a.C + c);
        const f32x4_t x = conv_input<T>(a, t, k, c);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = fmaf(w[e], x[e], v[e]);
      }
      emit(t, v);
      if (a.update) {
        T* st = (T*)a.state + (size_t)a.m.slot[a.m.seq[t]] * (a.taps - 1) * a.C + c;
        for (int k = a.taps - 2; k >= 0; --k)  // oldest first
          Act<T>::store4(st + (size_t)(a.taps - 2 - k) * a.C, conv_input<T>(a, t, k, c));
      }
    }
  }
}

template <typename T, int CONV_RUN>
static int launch_conv(const ConvArgs& a, int silu, hipStream_t s) {
  const dim3 grid((a.C / 4 + 63) / 64, (a.m.T + 4 * CONV_RUN - 1) / (4 * CONV_RUN)), block(256);
#define CONV_CASE(K)                                                      \
  if (silu) causal_conv_kernel<T, K, 1, CONV_RUN><<<grid, block, 0, s>>>(a);        \
  else causal_conv_kernel<T, K, 0, CONV_RUN><<<grid, block, 0, s>>>(a);
  switch (a.taps) {
    case 2: CONV_CASE(2) break;
    case 3: CONV_CASE(3) break;
    case 4: CONV_CASE(4) break;
    default: CONV_CASE(0) break;
  }
#undef CONV_CASE
  DA_LAUNCH_CHECK();
}

// max_len: longest portion; batches of single tokens (max_len == 1) also replace the state.
DA_EXPORT int da_causal_conv(const void* x, int ldx, const void* w, const void* bias, void* state, void* y,
                             int ldy, int C, int taps, int silu, int max_len, const void* cu, const void* slot, const void* pos0,
                             const void* seq, int T, int B, int f32, void* stream) {
  if (T < 1 || B < 1 || C < 4 || C % 4 || ldx % 4 || ldy % 4 || taps < 1 || max_len < 1 ||
      (T + 3) / 4 > (max_len == 1 ? 65535 : 65535 * 8))
    return (int)hipErrorInvalidValue;
  ConvArgs a{x, (const float*)w, (const float*)bias, state, y, ldx, ldy, C, taps, max_len == 1,
             SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}};
  hipStream_t s = (hipStream_t)stream;
  if (max_len == 1) return f32 ? launch_conv<float, 1>(a, silu, s) : launch_conv<bf16_t, 1>(a, silu, s);
  return f32 ? launch_conv<float, 8>(a, silu, s) : launch_conv<bf16_t, 8>(a, silu, s);
}

// ------------------------------------------------------------------------------- phases
enum ScanPhase : int { SCAN_DIRECT = 0, SCAN_LOCAL = 1, SCAN_FINAL = 2 };

// The tokens a workgroup walks, its portion, and where its start / end states live.
struct ScanSpan {
  int b, t0, t1, k;     // portion, packed rows [t0, t1), chunk of the portion
  bool last, idle;      // the portion's last chunk; nothing to do
  __device__ bool only() const { return k == 0 && last; }  // the whole portion: runs from the stored state
};
template <int PHASE>
__device__ __forceinline__ ScanSpan scan_span(const SeqMeta& m, const ChunkMeta& ch, int g) {
  if constexpr (PHASE == SCAN_DIRECT) return ScanSpan{g, m.cu[g], m.cu[g + 1], 0, true, m.cu[g] == m.cu[g + 1]};
  const int b = ch.ck[2 * g], k = ch.ck[2 * g + 1];
  const int t0 = m.cu[b] + k * ch.len, t1 = min(t0 + ch.len, m.cu[b + 1]);
  const bool last = t1 == m.cu[b + 1];
  return ScanSpan{b, t0, t1, k, last, PHASE == SCAN_LOCAL && last};
}
// Chunk k of portion b starts from row base[b] + b + k of the chunk states (one more row than chunks).
__device__ __forceinline__ size_t chunk_row(const ChunkMeta& ch, int b, int k) { return (size_t)ch.base[b] + b + k; }

// ------------------------------------------------------------------------------- selective scan
struct SelArgs {
  const void* x; const float* dt; const void* bc; const void* z;  // x, z [T][ld], dt fp32 [T][C], B | C at bc
  const float* A; const float* D;                                 // A [C][N] = log2(e) * (negative rates)
  float* state; void* y;                                          // state [slots][C][N]
  float* chunk_state; float* chunk_dt;                            // [chunks + B][C][N], [chunks + B][C]
  int ldx, lddt, ldbc, ldz, ldy, offB, offC, C, N;
  int lanes, tile;                                                // lanes of a channel (power of two)
  ConvState conv;
  SeqMeta m;
  ChunkMeta ch;
};

// NS consecutive floats n0 .. of a row of N, zero past its end (vector accesses where rows are 16-byte aligned).
template <int NS>
__device__ __forceinline__ void row_load(float (&v)[NS], const float* p, int n0, int N) {
  if (N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < NS; i += 4) {
      const f32x4_t x = n0 + i < N ? *(const f32x4_t*)(p + n0 + i) : f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i + e] = x[e];
    }
  } else {
#pragma unroll
    for (int i = 0; i < NS; ++i) v[i] = n0 + i < N ? p[n0 + i] : 0.f;
  }
}
template <int NS>
__device__ __forceinline__ void row_store(float* p, const float (&v)[NS], int n0, int N) {
  if (N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < NS; i += 4)
      if (n0 + i < N) *(f32x4_t*)(p + n0 + i) = f32x4_t{v[i], v[i + 1], v[i + 2], v[i + 3]};
  } else {
#pragma unroll
    for (int i = 0; i < NS; ++i)
      if (n0 + i < N) p[n0 + i] = v[i];
  }
}

// A channel's N states live in `lanes` neighbouring lanes, NS each. B and C rows are staged `tile` tokens at a time in dynamic LDS
// ([tile][2][lanes * NS] fp32); the step sizes, inputs and gates of the next U tokens are in flight while
// the current ones are added.
template <typename T, int NS, int PHASE>
__global__ void __launch_bounds__(256) sel_scan_kernel(SelArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sbc[];
  const ScanSpan sp = scan_span<PHASE>(a.m, a.ch, blockIdx.y);
  if (sp.idle) return;
  const int G = a.lanes, NP = G * NS, cpb = 256 / G;
  const int c = blockIdx.x * cpb + threadIdx.x / G, g = threadIdx.x % G, n0 = g * NS;
  const bool live = c < a.C;
  const int cc = live ? c : a.C - 1;
  float S[NS], A[NS];
  float* st = a.state + ((size_t)a.m.slot[sp.b] * a.C + cc) * a.N;
  row_load<NS>(A, a.A + (size_t)cc * a.N, n0, a.N);
#pragma unroll
  for (int i = 0; i < NS; ++i) S[i] = 0.f;
  const bool stored = a.m.pos0[sp.b] != 0;
  if (PHASE == SCAN_FINAL && !sp.only()) {
    row_load<NS>(S, a.chunk_state + (chunk_row(a.ch, sp.b, sp.k) * a.C + cc) * a.N, n0, a.N);
  } else if (sp.k == 0) {
    if (stored) row_load<NS>(S, st, n0, a.N);
    if constexpr (PHASE == SCAN_LOCAL)
      if (live) row_store<NS>(a.chunk_state + (chunk_row(a.ch, sp.b, 0) * a.C + cc) * a.N, S, n0, a.N);
  }
  const float Dc = a.D[cc];
  float sdt = 0.f;
  const T* xp = (const T*)a.x + cc;
  const T* zp = (const T*)a.z + cc;
  const float* dp = a.dt + cc;
  constexpr int U = 4;
  float dt[U], x[U], z[U];
  auto fetch = [&](int t) {  // tokens past the span change nothing: step size and input 0
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const size_t tt = min(t + u, sp.t1 - 1);
      const float in = t + u < sp.t1 ? 1.f : 0.f;
      dt[u] = dp[tt * a.lddt] * in;
      x[u] = Act<T>::to_f(xp[tt * a.ldx]) * in;
      z[u] = PHASE == SCAN_LOCAL ? 0.f : Act<T>::to_f(zp[tt * a.ldz]);
    }
  };
  fetch(sp.t0);
  for (int tb = sp.t0; tb < sp.t1; tb += a.tile) {  // tile % U == 0
    const int nt = min(a.tile, (sp.t1 - tb + U - 1) / U * U);
    __syncthreads();
    for (int i = threadIdx.x; i < nt * 2 * NP; i += 256) {
      const int r = i / (2 * NP), q = i % (2 * NP), n = q % NP;
      const size_t t = min(tb + r, sp.t1 - 1);
      sbc[i] = n < a.N ? Act<T>::to_f(((const T*)a.bc)[t * a.ldbc + (q < NP ? a.offB : a.offC) + n]) : 0.f;
    }
    __syncthreads();
    for (int r0 = 0; r0 < nt; r0 += U) {
      float d_[U], x_[U], z_[U], y[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        d_[u] = dt[u];
        x_[u] = x[u];
        z_[u] = z[u];
      }
      fetch(tb + r0 + U);
      // straight-line over the U tokens: their exponentials and LDS reads overlap the states' chains
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float* br = sbc + (r0 + u) * 2 * NP + n0;
        const float dx = d_[u] * x_[u];
        y[u] = 0.f;
#pragma unroll
        for (int i = 0; i < NS; i += 4) {
          const f32x4_t B = *(const f32x4_t*)(br + i);
          f32x4_t C{0.f, 0.f, 0.f, 0.f};
          if constexpr (PHASE != SCAN_LOCAL) C = *(const f32x4_t*)(br + NP + i);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[i + e] = fmaf(__builtin_amdgcn_exp2f(d_[u] * A[i + e]), S[i + e], dx * B[e]);
            if constexpr (PHASE != SCAN_LOCAL) y[u] = fmaf(S[i + e], C[e], y[u]);
          }
        }
        sdt += d_[u];
      }
      if constexpr (PHASE != SCAN_LOCAL) {
        for (int o = 1; o < G; o <<= 1)
#pragma unroll
          for (int u = 0; u < U; ++u) y[u] += __shfl_xor(y[u], o, 64);
        if (live && g == 0)
#pragma unroll
          for (int u = 0; u < U; ++u)
            if (tb + r0 + u < sp.t1)
              ((T*)a.y)[(size_t)(tb + r0 + u) * a.ldy + c] = Act<T>::from_f(fmaf(Dc, x_[u], y[u]) * act_silu<T>(z_[u]));
      }
    }
  }
  if (!live) return;
  if constexpr (PHASE == SCAN_LOCAL) {
    const size_t row = chunk_row(a.ch, sp.b, sp.k + 1);
    row_store<NS>(a.chunk_state + (row * a.C + c) * a.N, S, n0, a.N);
    if (g == 0) a.chunk_dt[row * a.C + c] = sdt;
  } else if (sp.last) {
    row_store<NS>(st, S, n0, a.N);
    if (g == 0) conv_state_store<T>(a.conv, a.m, sp.b, c);
  }
}

// Start state of every chunk from the chunks' own end states: row k + 1 += decay(chunk k) * row k.
// One thread per (channel, state) of a portion; chunk 0 ran from the stored state.
__global__ void __launch_bounds__(256) sel_carry_kernel(SelArgs a) {
  const int i = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (i >= a.C * a.N) return;
  const int n = (a.m.cu[b + 1] - a.m.cu[b] + a.ch.len - 1) / a.ch.len;
  const int c = i / a.N;
  const size_t row = chunk_row(a.ch, b, 0), CN = (size_t)a.C * a.N;
  if (n < 3) return;  // rows 0 and 1 are final
  const float A = a.A[i];
  float s = a.chunk_state[(row + 1) * CN + i];
  for (int k0 = 2; k0 < n; k0 += 8) {
    float v[8], d[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const size_t r = row + min(k0 + u, n - 1);
      v[u] = a.chunk_state[r * CN + i];
      d[u] = a.chunk_dt[r * a.C + c];
    }
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (k0 + u < n) {
        s = fmaf(__builtin_amdgcn_exp2f(d[u] * A), s, v[u]);
        a.chunk_state[(row + k0 + u) * CN + i] = s;
      }
  }
}

template <typename T, int NS>
static int launch_sel(const SelArgs& a, hipStream_t s) {
  const int cpb = 256 / a.lanes;
  const unsigned gx = (a.C + cpb - 1) / cpb;
  const size_t lds = (size_t)a.tile * 2 * a.lanes * NS * 4;
  if (a.ch.n == 0) {
    sel_scan_kernel<T, NS, SCAN_DIRECT><<<dim3(gx, a.m.B), 256, lds, s>>>(a);
  } else {
    sel_scan_kernel<T, NS, SCAN_LOCAL><<<dim3(gx, a.ch.n), 256, lds, s>>>(a);
    sel_carry_kernel<<<dim3((a.C * a.N + 255) / 256, a.m.B), 256, 0, s>>>(a);
    sel_scan_kernel<T, NS, SCAN_FINAL><<<dim3(gx, a.ch.n), 256, lds, s>>>(a);
  }
  DA_LAUNCH_CHECK();
}

// n_chunks = 0: one launch (portions of a few tokens); else the chunk list ck / base and the scratch
// chunk_state [n_chunks + B][C][N], chunk_dt [n_chunks + B][C] (fp32). N <= 512.
DA_EXPORT int da_selective_scan(const void* x, int ldx, const void* dt, int lddt, const void* bc, int ldbc, int offB,
                                int offC, const void* z, int ldz, const void* A, const void* D, void* state, void* y,
                                int ldy, int C, int N, const void* conv_x, int ld_conv, void* conv_state, int taps,
                                void* chunk_state, void* chunk_dt, const void* ck, const void* base, int n_chunks,
                                int chunk, int max_len, const void* cu, const void* slot, const void* pos0, const void* seq, int T, int B,
                                int f32, void* stream) {
  if (T < 1 || B < 1 || B > 65535 || C < 1 || N < 1 || N > 512 || taps < 1 || n_chunks < 0 || n_chunks > 65535 || (n_chunks && chunk < 1))
    return (int)hipErrorInvalidValue;
  if (n_chunks && (!ck || !base || !chunk_state || !chunk_dt)) return (int)hipErrorInvalidValue;
  // single tokens: four states a lane, so the states' rows are read and written in whole lines
  const int ns = N <= 4 || (max_len <= 4 && N <= 256 && B < 16) ? 4 : 8;
  int lanes = 1;
  while (lanes * ns < N) lanes *= 2;
  const int tile = min(64, max(16, 2048 / (lanes * ns)));  // at most 64 KB of LDS
  SelArgs a{x, (const float*)dt, bc, z, (const float*)A, (const float*)D, (float*)state, y, (float*)chunk_state,
            (float*)chunk_dt, ldx, lddt, ldbc, ldz, ldy, offB, offC, C, N, lanes, tile,
            ConvState{conv_x, ld_conv, conv_state, taps, C},
            SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B},
            ChunkMeta{(const int*)ck, (const int*)base, n_chunks, chunk}};
  hipStream_t s = (hipStream_t)stream;
  if (f32) return ns == 4 ? launch_sel<float, 4>(a, s) : launch_sel<float, 8>(a, s);
  return ns == 4 ? launch_sel<bf16_t, 4>(a, s) : launch_sel<bf16_t, 8>(a, s);
}

// ------------------------------------------------------------------------------- gated recurrence
struct GruArgs {
  const float* decay; const float* drive; const void* gate;  // decay, drive fp32 [T][C], gate [T][ldg]
  float* state; void* y;                                     // state [slots][C]
  float* chunk_state; float* chunk_decay;                    // [chunks + B][C] each
  int ldg, ldy, C;
  ConvState conv;
  SeqMeta m;
  ChunkMeta ch;
};

template <typename T, int PHASE>
__global__ void __launch_bounds__(256) gru_scan_kernel(GruArgs a) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  const ScanSpan sp = scan_span<PHASE>(a.m, a.ch, blockIdx.y);
  if (c >= a.C || sp.idle) return;
  float* st = a.state + (size_t)a.m.slot[sp.b] * a.C + c;
  float s = 0.f, p = 1.f;
  if (PHASE == SCAN_FINAL && !sp.only()) {
    s = a.chunk_state[chunk_row(a.ch, sp.b, sp.k) * a.C + c];
  } else if (sp.k == 0) {
    if (a.m.pos0[sp.b] != 0) s = *st;
    if constexpr (PHASE == SCAN_LOCAL) a.chunk_state[chunk_row(a.ch, sp.b, 0) * a.C + c] = s;
  }
  constexpr int U = 8;
  float d[U], v[U], g[U];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const size_t t = min(t0 + u, sp.t1 - 1);
      d[u] = a.decay[t * a.C + c];
      v[u] = a.drive[t * a.C + c];
      g[u] = PHASE == SCAN_LOCAL ? 0.f : Act<T>::to_f(((const T*)a.gate)[t * a.ldg + c]);
    }
  };
  fetch(sp.t0);
  for (int t0 = sp.t0; t0 < sp.t1; t0 += U) {
    float o[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (t0 + u < sp.t1) {
        s = fmaf(d[u], s, v[u]);
        if constexpr (PHASE == SCAN_LOCAL) p *= d[u];
      }
      o[u] = s * act_gelu_tanh<T>(g[u]);
    }
    if (t0 + U < sp.t1) fetch(t0 + U);
    if constexpr (PHASE != SCAN_LOCAL)
#pragma unroll
      for (int u = 0; u < U; ++u)
        if (t0 + u < sp.t1) ((T*)a.y)[(size_t)(t0 + u) * a.ldy + c] = Act<T>::from_f(o[u]);
  }
  if constexpr (PHASE == SCAN_LOCAL) {
    const size_t row = chunk_row(a.ch, sp.b, sp.k + 1);
    a.chunk_state[row * a.C + c] = s;
    a.chunk_decay[row * a.C + c] = p;
  } else if (sp.last) {
    *st = s;
    conv_state_store<T>(a.conv, a.m, sp.b, c);
  }
}

__global__ void __launch_bounds__(256) gru_carry_kernel(GruArgs a) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  const int n = (a.m.cu[b + 1] - a.m.cu[b] + a.ch.len - 1) / a.ch.len;
  if (c >= a.C || n < 3) return;
  const size_t row = chunk_row(a.ch, b, 0);
  float s = a.chunk_state[(row + 1) * a.C + c];
  for (int k0 = 2; k0 < n; k0 += 8) {
    float v[8], d[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const size_t r = row + min(k0 + u, n - 1);
      v[u] = a.chunk_state[r * a.C + c];
      d[u] = a.chunk_decay[r * a.C + c];
    }
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (k0 + u < n) {
        s = fmaf(d[u], s, v[u]);
        a.chunk_state[(row + k0 + u) * a.C + c] = s;
      }
  }
}

template <typename T>
static int launch_gru(const GruArgs& a, hipStream_t s) {
  const unsigned gx = (a.C + 255) / 256;
  if (a.ch.n == 0) {
    gru_scan_kernel<T, SCAN_DIRECT><<<dim3(gx, a.m.B), 256, 0, s>>>(a);
  } else {
    gru_scan_kernel<T, SCAN_LOCAL><<<dim3(gx, a.ch.n), 256, 0, s>>>(a);
    gru_carry_kernel<<<dim3(gx, a.m.B), 256, 0, s>>>(a);
    gru_scan_kernel<T, SCAN_FINAL><<<dim3(gx, a.ch.n), 256, 0, s>>>(a);
  }
  DA_LAUNCH_CHECK();
}

DA_EXPORT int da_gated_scan(const void* decay, const void* drive, const void* gate, int ldg, void* state, void* y,
                            int ldy, int C, const void* conv_x, int ld_conv, void* conv_state, int taps,
                            void* chunk_state, void* chunk_decay, const void* ck, const void* base, int n_chunks,
                            int chunk, const void* cu, const void* slot, const void* pos0, const void* seq, int T, int B, int f32,
                            void* stream) {
  if (T < 1 || B < 1 || B > 65535 || C < 1 || taps < 1 || n_chunks < 0 || n_chunks > 65535 || (n_chunks && chunk < 1))
    return (int)hipErrorInvalidValue;
  if (n_chunks && (!ck || !base || !chunk_state || !chunk_decay)) return (int)hipErrorInvalidValue;
  GruArgs a{(const float*)decay, (const float*)drive, gate, (float*)state, y, (float*)chunk_state,
            (float*)chunk_decay, ldg, ldy, C, ConvState{conv_x, ld_conv, conv_state, taps, C},
            SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B},
            ChunkMeta{(const int*)ck, (const int*)base, n_chunks, chunk}};
  return f32 ? launch_gru<float>(a, (hipStream_t)stream) : launch_gru<bf16_t>(a, (hipStream_t)stream);
}
