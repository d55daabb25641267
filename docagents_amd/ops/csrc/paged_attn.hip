// Sigmoid attention over a paged cache in which the values are the keys.
//
//   w_ij = sigmoid(scale * temp_i * (norm(q_i) . norm(k_j)) + bias_h),  o_i = gate_i * sum_j w_ij k_j
//
// The weights are not normalised over the keys, so partial sums over key ranges just add.
//
// Cache: a pool of 64-token pages, page p of an attention layer holding, per key/value head, the keys
// as projected ([64][D], once: they are the values too) and 1 / rms of every key ([64], fp32). A key's
// norm is applied to its score; the norm weights, the query's temperature and the scale are folded into
// the query (attn_prep), so the score is (q' . k) * (1 / rms(k)) + bias. table[slot][i] is the page of
// tokens 64 i .. 64 i + 63 of the sequence in that slot.
//
// Query rows of one key/value head are packed token-major, row r = token r / g, head r % g of its g
// query heads, so every key staged serves all of them.
#include "seq.h"

struct AttnArgs {
  const void* qkg; int ld;                     // [T][q heads | k heads | gates], heads D columns wide
  void* kc; float* kr;                         // pages: keys [page][G][64][D], 1 / rms [page][G][64]
  const int* table; int max_pages, pages;
  const float* pb;                             // bias per query head
  void* out; int ldo;
  int H, G, D;
  SeqMeta m;
  float* part; int nsplit, pps;                // decode: partial sums [B][H][nsplit][D], pages per split
};

__device__ __forceinline__ int page_of(const AttnArgs& a, int slot, int i) {
  const int p = a.table[(size_t)slot * a.max_pages + min(i, a.max_pages - 1)];
  DA_ASSERT(p >= 0 && p < a.pages);
  return min(max(p, 0), a.pages - 1);
}
__device__ __forceinline__ float gate_of(float x) { return sigmoid32(x); }

// ------------------------------------------------------------------------------- query / key preparation
struct PrepArgs {
  AttnArgs a;
  const float* qk_w;            // [D] product of the query and key norm weights, zero in padding columns
  float scale, eps, temp_coef;
  double temp_every;            // <= 0: no temperature
  int dim;                      // columns a head really has
};

// A head per group of `lanes` lanes (a power of two >= D / 8, at most a wave), 8 columns per lane and
// step: queries are normalised and scaled in place, keys go to their page. STEPS * 8 * lanes >= D.
template <typename T, int STEPS>
__global__ void __launch_bounds__(256) attn_prep_kernel(PrepArgs p, int lanes) {
  const AttnArgs& a = p.a;
  const int per = 256 / lanes, heads = a.H + a.G;
  const int item = blockIdx.x * per + threadIdx.x / lanes, l = threadIdx.x % lanes;
  const bool live = item < a.m.T * heads;
  const int it = live ? item : a.m.T * heads - 1, t = it / heads, h = it % heads;
  const int b = a.m.seq[t], pos = a.m.pos0[b] + t - a.m.cu[b];
  T* row = (T*)a.qkg + (size_t)t * a.ld + (size_t)h * a.D;
  f32x4_t v[STEPS][2];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int d = (i * lanes + l) * 8;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      v[i][j] = d < a.D ? Act<T>::load4(row + d + 4 * j) : f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(v[i][j][e], v[i][j][e], ss);
    }
  }
  for (int o = lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  if (!live) return;
  const float inv = 1.f / sqrtf(ss / p.dim + p.eps);
  T* dst = row;
  float f = 1.f;
  if (h < a.H) {
    f = inv * p.scale;
    if (p.temp_every > 0.) f *= fmaf(p.temp_coef, logf((float)(floor((double)(pos + 1) / p.temp_every) + 1.)), 1.f);
  } else {
    const size_t kr = ((size_t)page_of(a, a.m.slot[b], pos / PAGE) * a.G + h - a.H) * PAGE + pos % PAGE;
    dst = (T*)a.kc + kr * a.D;
    if (l == 0) a.kr[kr] = inv;
  }
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int d = (i * lanes + l) * 8;
    if (d >= a.D) continue;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      f32x4_t x = v[i][j];
      if (h < a.H) {
        const f32x4_t w = *(const f32x4_t*)(p.qk_w + d + 4 * j);
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] *= f * w[e];
      }
      Act<T>::store4(dst + d + 4 * j, x);
    }
  }
}

template <typename T>
static void launch_prep(const PrepArgs& p, hipStream_t s) {
  int lanes = 4;
  while (lanes < 64 && lanes * 8 < p.a.D) lanes *= 2;
  const int per = 256 / lanes;
  const unsigned grid = ((size_t)p.a.m.T * (p.a.H + p.a.G) + per - 1) / per;
  if (p.a.D <= lanes * 8) attn_prep_kernel<T, 1><<<grid, 256, 0, s>>>(p, lanes);
  else attn_prep_kernel<T, 2><<<grid, 256, 0, s>>>(p, lanes);
}

// ------------------------------------------------------------------------------- any size, fp32 arithmetic
// 16 query rows per workgroup against 32-key tiles in LDS; scores and sums on the vector ALUs. The fp32
// precision runs here, and bf16 heads wider than the matrix-core kernels take.
template <typename T, int ND>  // ND: output columns per thread (16 threads a row)
__global__ void __launch_bounds__(256) attn_any_kernel(AttnArgs a) {
  extern __shared__ float sm[];
  constexpr int KT = 32;
  const int D = a.D, DS = D + 1, gs = a.H / a.G;
  const int b = blockIdx.z, g = blockIdx.y, s0 = a.m.cu[b], n = a.m.cu[b + 1] - s0;
  const int r0 = blockIdx.x * 16;
  if (r0 >= n * gs) return;
  float* sq = sm;              // [16][DS]
  float* sk = sq + 16 * DS;    // [KT][DS]
  float* sw = sk + KT * DS;    // [16][KT + 1]
  float* sr = sw + 16 * (KT + 1);  // [KT]
  const int tid = threadIdx.x, r = tid >> 4, j = tid & 15;
  const int pos0 = a.m.pos0[b], slot = a.m.slot[b];
  for (int i = tid; i < 16 * D; i += 256) {
    const int rr = min(r0 + i / D, n * gs - 1);
    sq[(i / D) * DS + i % D] =
        Act<T>::to_f(((const T*)a.qkg)[(size_t)(s0 + rr / gs) * a.ld + (size_t)(g * gs + rr % gs) * D + i % D]);
  }
  const int row = r0 + r, tok = min(row, n * gs - 1) / gs, hd = g * gs + min(row, n * gs - 1) % gs;
  const int qpos = pos0 + tok;
  const int kend = pos0 + min(r0 + 15, n * gs - 1) / gs + 1;  // keys the tile's last row sees
  const float pb = a.pb[hd];
  float acc[ND];
#pragma unroll
  for (int i = 0; i < ND; ++i) acc[i] = 0.f;
  for (int k0 = 0; k0 < kend; k0 += KT) {
    const size_t kr = ((size_t)page_of(a, slot, k0 / PAGE) * a.G + g) * PAGE + k0 % PAGE;
    const T* kp = (const T*)a.kc + kr * D;
    __syncthreads();
    for (int i = tid; i < KT * D; i += 256) sk[(i / D) * DS + i % D] = k0 + i / D < kend ? Act<T>::to_f(kp[i]) : 0.f;
    if (tid < KT) sr[tid] = k0 + tid < kend ? a.kr[kr + tid] : 0.f;
    __syncthreads();
    float d0 = 0.f, d1 = 0.f;
    const float* q = sq + r * DS;
    const float *x = sk + j * DS, *y = sk + (j + 16) * DS;
    for (int d = 0; d < D; ++d) {
      d0 = fmaf(q[d], x[d], d0);
      d1 = fmaf(q[d], y[d], d1);
    }
    sw[r * (KT + 1) + j] = k0 + j <= qpos ? sigmoid32(fmaf(d0, sr[j], pb)) : 0.f;
    sw[r * (KT + 1) + j + 16] = k0 + j + 16 <= qpos ? sigmoid32(fmaf(d1, sr[j + 16], pb)) : 0.f;
    __syncthreads();
    for (int k = 0; k < KT; ++k) {
      const float w = sw[r * (KT + 1) + k];
#pragma unroll
      for (int i = 0; i < ND; ++i)
        if (j + 16 * i < D) acc[i] = fmaf(w, sk[k * DS + j + 16 * i], acc[i]);
    }
  }
  if (row >= n * gs) return;
  const float gt = gate_of(Act<T>::to_f(((const T*)a.qkg)[(size_t)(s0 + tok) * a.ld + (size_t)(a.H + a.G) * D + hd]));
  T* o = (T*)a.out + (size_t)(s0 + tok) * a.ldo + (size_t)hd * D;
#pragma unroll
  for (int i = 0; i < ND; ++i)
    if (j + 16 * i < D) o[j + 16 * i] = Act<T>::from_f(acc[i] * gt);
}

// ------------------------------------------------------------------------------- matrix cores, portions
// 128 query rows per workgroup (4 waves x 32), one page of keys per step, double-buffered in LDS, as
// S^T = K . Q^T on 32x32x16 MFMAs: a lane owns one query row and 32 of the page's keys, its weights stay
// in registers and are the B operand of O^T += K^T . W^T. The page is loaded from HBM once and kept in
// LDS twice, with the row strides that the plain (scores) and the transposing (sums) reads each want. A
// weight enters the second product as the sum of two bf16 terms (its rounding and the remainder), so
// its fp32 value counts to about 16 bits.
template <int D> struct MA {
  static constexpr int KSTR = D * 2 + 16;
  static constexpr int VSTR = (D % 64 == 32) ? D * 2 : (D == 64 ? 192 : D * 2 + 64);
  static constexpr int KB = PAGE * KSTR, VB = PAGE * VSTR;
  static constexpr int BUF = KB + VB + PAGE * 4;
  static constexpr int LPT = D / 32;  // 16-byte pieces per thread
};

__device__ __forceinline__ unsigned split_lo(unsigned hi, float a, float b) {
  return pack_bf2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}

template <int D>
__global__ void __launch_bounds__(256, D <= 128 ? 2 : 1) sigmoid_attn_kernel(AttnArgs a, int skip_single) {
  using C = MA<D>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int NDS = D / 16, NDB = D / 32;
  const int b = blockIdx.z, g = blockIdx.y, gs = a.H / a.G;
  const int s0 = a.m.cu[b], n = a.m.cu[b + 1] - s0;
  const int qt = gridDim.x - 1 - blockIdx.x;  // the tiles with the most keys first
  if (qt * 128 >= n * gs || (skip_single && n == 1)) return;
  const int pos0 = a.m.pos0[b], slot = a.m.slot[b];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int qr = lane & 31, hi = lane >> 5;
  const int row = qt * 128 + wv * 32 + qr;
  const bool valid = row < n * gs;
  const int rc = valid ? row : n * gs - 1;
  const int tok = rc / gs, hd = g * gs + rc % gs;
  const int qpos = pos0 + tok;
  const int wfirst = pos0 + min(qt * 128 + wv * 32, n * gs - 1) / gs;       // this wave's first / last position
  const int wlast = pos0 + min(qt * 128 + wv * 32 + 31, n * gs - 1) / gs;
  const int klast = pos0 + min(qt * 128 + 127, n * gs - 1) / gs;            // last key of the workgroup
  const int ntiles = klast / PAGE + 1;

  bf16x8_t qf[NDS];
  const bf16_t* qp = (const bf16_t*)a.qkg + (size_t)(s0 + tok) * a.ld + (size_t)hd * D + hi * 8;
#pragma unroll
  for (int ds = 0; ds < NDS; ++ds) qf[ds] = *(const bf16x8_t*)(qp + ds * 16);
  const float pbn = -LOG2E * a.pb[hd];

  u32x4_t kreg[C::LPT];
  float rreg = 0.f;
  auto load_page = [&](int t) {
    const size_t pg = (size_t)page_of(a, slot, t) * a.G + g;
    const bf16_t* kp = (const bf16_t*)a.kc + pg * PAGE * D;
    const int keys = klast + 1 - t * PAGE;  // rows past it may hold anything: read as zero
#pragma unroll
    for (int i = 0; i < C::LPT; ++i) {
      const int pc = tid + 256 * i;
      const u32x4_t v = *(const u32x4_t*)(kp + (size_t)pc * 8);
      kreg[i] = pc / (D / 8) < keys ? v : u32x4_t{0, 0, 0, 0};
    }
    if (tid < PAGE) rreg = tid < keys ? -LOG2E * a.kr[pg * PAGE + tid] : 0.f;
  };
  auto store_page = [&](int buf) {
    char* base = smem + buf * C::BUF;
#pragma unroll
    for (int i = 0; i < C::LPT; ++i) {
      const int pc = tid + 256 * i, r = pc / (D / 8), c = pc % (D / 8);
      *(u32x4_t*)(base + r * C::KSTR + c * 16) = kreg[i];
      *(u32x4_t*)(base + C::KB + r * C::VSTR + c * 16) = kreg[i];
    }
    if (tid < PAGE) *(float*)(base + C::KB + C::VB + tid * 4) = rreg;
  };
  f32x16_t oacc[NDB];
#pragma unroll
  for (int i = 0; i < NDB; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) oacc[i][e] = 0.f;

  load_page(0);
  store_page(0);
  __syncthreads();
  for (int t = 0; t < ntiles; ++t) {
    if (t + 1 < ntiles) load_page(t + 1);
    const int kb = t * PAGE;
    if (kb <= wlast) {
      const char* sK = smem + (t & 1) * C::BUF;
      const char* sV = sK + C::KB;
      const float* sR = (const float*)(sV + C::VB);
      f32x16_t s[2];
#pragma unroll
      for (int hh = 0; hh < 2; ++hh) {
#pragma unroll
        for (int e = 0; e < 16; ++e) s[hh][e] = 0.f;
#pragma unroll
        for (int ds = 0; ds < NDS; ++ds) {
          const bf16x8_t kf = *(const bf16x8_t*)(sK + (hh * 32 + qr) * C::KSTR + ds * 32 + hi * 16);
          s[hh] = mfma32(kf, qf[ds], s[hh]);
        }
      }
      const bool edge = kb + PAGE - 1 > wfirst;
#pragma unroll
      for (int hh = 0; hh < 2; ++hh)
#pragma unroll
        for (int r4 = 0; r4 < 4; ++r4) {
          const int key = hh * 32 + 8 * r4 + 4 * hi;
          const f32x4_t rr = *(const f32x4_t*)(sR + key);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            float w = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(fmaf(s[hh][4 * r4 + e], rr[e], pbn)));
            if (edge && kb + key + e > qpos) w = 0.f;
            s[hh][4 * r4 + e] = w;
          }
        }
#pragma unroll
      for (int kc = 0; kc < 4; ++kc) {
        const int hh = kc >> 1, cb = (kc & 1) * 8;
        u32x4_t wh, wl;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float x = s[hh][cb + 2 * e], y = s[hh][cb + 2 * e + 1];
          wh[e] = pack_bf2(x, y);
          wl[e] = split_lo(wh[e], x, y);
        }
        const bf16x8_t bh = __builtin_bit_cast(bf16x8_t, wh), bl = __builtin_bit_cast(bf16x8_t, wl);
        const int g4 = lane >> 4, li = lane & 15;
        const int vrow = kc * 16 + 4 * (g4 >> 1) + (li >> 2);
#pragma unroll
        for (int db = 0; db < NDB; ++db) {
          const char* vp = sV + vrow * C::VSTR + (db * 32 + 16 * (g4 & 1) + 4 * (li & 3)) * 2;
          const s16x4_t lo = lds_read_tr16(vp), up = lds_read_tr16(vp + 8 * C::VSTR);
          const bf16x8_t va = bf16x8_t{lo[0], lo[1], lo[2], lo[3], up[0], up[1], up[2], up[3]};
          oacc[db] = mfma32(va, bh, oacc[db]);
          oacc[db] = mfma32(va, bl, oacc[db]);
        }
      }
    }
    if (t + 1 < ntiles) store_page((t + 1) & 1);
    __syncthreads();
  }
  if (!valid) return;
  const float gt = gate_of(bf2f(((const bf16_t*)a.qkg)[(size_t)(s0 + tok) * a.ld + (size_t)(a.H + a.G) * D + hd]));
  bf16_t* o = (bf16_t*)a.out + (size_t)(s0 + tok) * a.ldo + (size_t)hd * D;
#pragma unroll
  for (int db = 0; db < NDB; ++db)
#pragma unroll
    for (int q = 0; q < 4; ++q)
      *(u32x2_t*)(o + db * 32 + 8 * q + 4 * hi) =
          u32x2_t{pack_bf2(oacc[db][4 * q] * gt, oacc[db][4 * q + 1] * gt),
                  pack_bf2(oacc[db][4 * q + 2] * gt, oacc[db][4 * q + 3] * gt)};
}

// ------------------------------------------------------------------------------- matrix cores, single tokens
// Portions of one token: 16 of a key/value head's query heads per workgroup, its keys split over
// blockIdx.x; a wave takes every fourth page of the split. A page is loaded in the score product's operand
// layout straight to registers (every byte of the page once) and written to the wave's LDS tile only
// for the transposing reads of the sum; the next page's loads are in flight meanwhile.
template <int D> struct MD {
  static constexpr int VSTR = MA<D>::VSTR;
  static constexpr int WAVE = PAGE * VSTR > 16 * D * 4 ? PAGE * VSTR : 16 * D * 4;
};

template <int D>
__global__ void __launch_bounds__(256, D <= 128 ? 2 : 1) sigmoid_decode_kernel(AttnArgs a) {
  using C = MD<D>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int NDS = D / 32, NDB = D / 16;
  const int gs = a.H / a.G, qtiles = (gs + 15) / 16;
  const int split = blockIdx.x, g = blockIdx.y / qtiles, qt = blockIdx.y % qtiles, b = blockIdx.z;
  const int t = a.m.cu[b];
  if (a.m.cu[b + 1] - t != 1) return;
  const int len = a.m.pos0[b] + 1, slot = a.m.slot[b];
  const int npages = (len + PAGE - 1) / PAGE;
  const int p0 = split * a.pps, p1 = min(p0 + a.pps, npages);
  if (p0 >= p1) return;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, fr = lane & 15, fg = lane >> 4;
  char* sV = smem + wv * C::WAVE;
  const int qi = qt * 16 + fr;                      // this lane's query head of the group
  const int hd = g * gs + min(qi, gs - 1);
  bf16x8_t qf[NDS];
  const bf16_t* qp = (const bf16_t*)a.qkg + (size_t)t * a.ld + (size_t)hd * D + fg * 8;
#pragma unroll
  for (int ds = 0; ds < NDS; ++ds) qf[ds] = *(const bf16x8_t*)(qp + ds * 32);
  const float pbn = -LOG2E * a.pb[hd];
  f32x4_t oacc[NDB];
#pragma unroll
  for (int i = 0; i < NDB; ++i) oacc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  bf16x8_t kf[4][NDS];
  f32x4_t rr[4];
  auto load_page = [&](int p) {
    const size_t pg = (size_t)page_of(a, slot, p) * a.G + g;
    const bf16_t* kp = (const bf16_t*)a.kc + pg * PAGE * D;
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      const int key = kb * 16 + fr;
      const bool in = p * PAGE + key < len;
#pragma unroll
      for (int ds = 0; ds < NDS; ++ds) {
        const u32x4_t v = *(const u32x4_t*)(kp + (size_t)key * D + ds * 32 + fg * 8);
        kf[kb][ds] = __builtin_bit_cast(bf16x8_t, in ? v : u32x4_t{0, 0, 0, 0});
      }
      rr[kb] = *(const f32x4_t*)(a.kr + pg * PAGE + kb * 16 + fg * 4);
    }
  };
  int p = p0 + wv;
  if (p < p1) load_page(p);
  for (; p < p1; p += 4) {
    f32x4_t s[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      s[kb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ds = 0; ds < NDS; ++ds) s[kb] = mfma16(kf[kb][ds], qf[ds], s[kb]);
    }
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const bool in = p * PAGE + kb * 16 + fg * 4 + e < len;
        const float w = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(fmaf(s[kb][e], -LOG2E * rr[kb][e], pbn)));
        s[kb][e] = in ? w : 0.f;
      }
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int ds = 0; ds < NDS; ++ds)
        *(bf16x8_t*)(sV + (kb * 16 + fr) * C::VSTR + ds * 64 + fg * 16) = kf[kb][ds];
    if (p + 4 < p1) load_page(p + 4);
    // the tile belongs to this wave alone: its LDS accesses complete in order
    asm volatile("" ::: "memory");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      u32x4_t wh, wl;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float x = s[half * 2 + (e >> 1)][(e & 1) * 2], y = s[half * 2 + (e >> 1)][(e & 1) * 2 + 1];
        wh[e] = pack_bf2(x, y);
        wl[e] = split_lo(wh[e], x, y);
      }
      const bf16x8_t bh = __builtin_bit_cast(bf16x8_t, wh), bl = __builtin_bit_cast(bf16x8_t, wl);
      const int vrow = half * 32 + 4 * fg + (fr >> 2);
#pragma unroll
      for (int db = 0; db < NDB; ++db) {
        const char* vp = sV + vrow * C::VSTR + (db * 16 + 4 * (fr & 3)) * 2;
        const s16x4_t lo = lds_read_tr16(vp), up = lds_read_tr16(vp + 16 * C::VSTR);
        const bf16x8_t va = bf16x8_t{lo[0], lo[1], lo[2], lo[3], up[0], up[1], up[2], up[3]};
        oacc[db] = mfma16(va, bh, oacc[db]);
        oacc[db] = mfma16(va, bl, oacc[db]);
      }
    }
    asm volatile("" ::: "memory");
    __builtin_amdgcn_wave_barrier();
  }
  // sum of the four waves through LDS: [wave][16 rows][D]
  __syncthreads();
  float* sO = (float*)smem;
#pragma unroll
  for (int db = 0; db < NDB; ++db) *(f32x4_t*)(sO + (wv * 16 + fr) * D + db * 16 + fg * 4) = oacc[db];
  __syncthreads();
  const int rows = min(16, gs - qt * 16);
  for (int i = tid; i < rows * D / 4; i += 256) {
    const int r = i / (D / 4), c = (i % (D / 4)) * 4, h = g * gs + qt * 16 + r;
    f32x4_t v = *(const f32x4_t*)(sO + r * D + c);
#pragma unroll
    for (int w = 1; w < 4; ++w) v += *(const f32x4_t*)(sO + (w * 16 + r) * D + c);
    if (a.nsplit > 1) {
      *(f32x4_t*)(a.part + (((size_t)b * a.H + h) * a.nsplit + split) * D + c) = v;
    } else {
      const float gt = gate_of(bf2f(((const bf16_t*)a.qkg)[(size_t)t * a.ld + (size_t)(a.H + a.G) * D + h]));
      Act<bf16_t>::store4((bf16_t*)a.out + (size_t)t * a.ldo + (size_t)h * D + c, v * gt);
    }
  }
}

__global__ void __launch_bounds__(64) sigmoid_combine_kernel(AttnArgs a) {
  const int h = blockIdx.x, b = blockIdx.y, t = a.m.cu[b];
  if (a.m.cu[b + 1] - t != 1) return;
  const int used = min(a.nsplit, (a.m.pos0[b] / PAGE + a.pps) / a.pps);
  const float gt = gate_of(bf2f(((const bf16_t*)a.qkg)[(size_t)t * a.ld + (size_t)(a.H + a.G) * a.D + h]));
  const float* p = a.part + ((size_t)b * a.H + h) * a.nsplit * a.D;
  for (int c = threadIdx.x * 4; c < a.D; c += 256) {
    f32x4_t v{0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < used; s0 += 8) {
      f32x4_t x[8];
#pragma unroll
      for (int s = 0; s < 8; ++s) x[s] = *(const f32x4_t*)(p + (size_t)min(s0 + s, used - 1) * a.D + c);
#pragma unroll
      for (int s = 0; s < 8; ++s)
        if (s0 + s < used) v += x[s];
    }
    Act<bf16_t>::store4((bf16_t*)a.out + (size_t)t * a.ldo + (size_t)h * a.D + c, v * gt);
  }
}

// ------------------------------------------------------------------------------- launchers
template <typename T, int ND>
static int launch_any(const AttnArgs& a, int max_len, hipStream_t s) {
  const int gs = a.H / a.G;
  const size_t lds = (size_t)(48 * (a.D + 1) + 16 * 33 + 32) * 4;
  const void* fn = (const void*)attn_any_kernel<T, ND>;
  if (lds > 65536) {
    const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  attn_any_kernel<T, ND><<<dim3((max_len * gs + 15) / 16, a.G, a.m.B), 256, lds, s>>>(a);
  DA_LAUNCH_CHECK();
}
template <typename T>
static int launch_any_d(const AttnArgs& a, int max_len, hipStream_t s) {
  if (a.D <= 64) return launch_any<T, 4>(a, max_len, s);
  if (a.D <= 128) return launch_any<T, 8>(a, max_len, s);
  if (a.D <= 256) return launch_any<T, 16>(a, max_len, s);
  return launch_any<T, 48>(a, max_len, s);
}

template <int D>
static int launch_mfma(const AttnArgs& a, int max_len, int singles, hipStream_t s) {
  const int gs = a.H / a.G;
  if (max_len > 1) {
    constexpr int lds = 2 * MA<D>::BUF;
    static const hipError_t e = hipFuncSetAttribute((const void*)sigmoid_attn_kernel<D>,
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (e != hipSuccess) return (int)e;
    sigmoid_attn_kernel<D><<<dim3((max_len * gs + 127) / 128, a.G, a.m.B), 256, lds, s>>>(a, 1);
  }
  if (singles) {
    constexpr int lds = 4 * MD<D>::WAVE;
    static const hipError_t e = hipFuncSetAttribute((const void*)sigmoid_decode_kernel<D>,
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (e != hipSuccess) return (int)e;
    sigmoid_decode_kernel<D><<<dim3(a.nsplit, a.G * ((gs + 15) / 16), a.m.B), 256, lds, s>>>(a);
    if (a.nsplit > 1) sigmoid_combine_kernel<<<dim3(a.H, a.m.B), 64, 0, s>>>(a);
  }
  DA_LAUNCH_CHECK();
}

static bool mfma_dim(int D) { return D == 32 || D == 64 || D == 96 || D == 128 || D == 192 || D == 256; }

// qkg [T][ld]: H query heads, G key heads (D columns each, D % 32 == 0), then H gates. Keys are written
// to their pages, queries prepared in place, then attention of every token over positions 0 .. its own.
// max_len: longest portion; singles: whether a portion of one token may be in the batch (bf16: the
// split kernel, part [B][H][nsplit][D] fp32 where nsplit > 1, nsplit * pps pages >= the longest context).
DA_EXPORT int da_sigmoid_attn(void* qkg, int ld, void* kc, void* kr, const void* table, int max_pages, int pages,
                              const void* pb, const void* qk_w, float scale, float eps, float temp_coef,
                              double temp_every, int H, int G, int D, int dim, void* out, int ldo, void* part,
                              int nsplit, int pps, int max_len, int singles, const void* cu, const void* slot,
                              const void* pos0, const void* seq, int T, int B, int f32, void* stream) {
  if (T < 1 || B < 1 || B > 65535 || G < 1 || H % G || D < 32 || D % 32 || D > 768 || (long long)T * (H + G) > 0x7fffffffll || dim < 1 || dim > D || ld % 8 ||
      ldo % 8 || max_pages < 1 || pages < 1 || max_len < 1 || nsplit < 1 || pps < 1 || (nsplit > 1 && !part))
    return (int)hipErrorInvalidValue;
  AttnArgs a{qkg, ld, kc, (float*)kr, (const int*)table, max_pages, pages, (const float*)pb, out, ldo, H, G, D,
             SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}, (float*)part, nsplit,
             pps};
  PrepArgs p{a, (const float*)qk_w, scale, eps, temp_coef, temp_every, dim};
  hipStream_t s = (hipStream_t)stream;
  if (f32) {
    launch_prep<float>(p, s);
    return launch_any_d<float>(a, max_len, s);
  }
  launch_prep<bf16_t>(p, s);
  if (!mfma_dim(D)) return launch_any_d<bf16_t>(a, max_len, s);
  switch (D) {
    case 32: return launch_mfma<32>(a, max_len, singles, s);
    case 64: return launch_mfma<64>(a, max_len, singles, s);
    case 96: return launch_mfma<96>(a, max_len, singles, s);
    case 128: return launch_mfma<128>(a, max_len, singles, s);
    case 192: return launch_mfma<192>(a, max_len, singles, s);
    default: return launch_mfma<256>(a, max_len, singles, s);
  }
}
