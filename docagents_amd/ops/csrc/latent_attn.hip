// Softmax attention over a paged cache of low-rank latents.
//
// A token's cache row is [latent c (L columns) | rotated key part (R columns)], shared by all heads. A head's key is
// (W_uk c, rotated part) and its value W_uv c, so with the query's unrotated part taken into the latent space
// (q_lat = W_uk^T q), score = (q_lat . c + q_rot . k_rot) * scale, and the head's result is W_uv (sum_j p_j c_j): one row
// per token serves every head as key and as value ("absorbed": short portions). Long portions expand keys and values
// of their context from the latents once ("expanded").
//
// The softmax's denominator also holds exp(sink_h): the running maximum starts at the sink and the running sum at 1.
//
// Pages: [page][64][L + R]; table[slot][i] is the page of tokens 64 i .. 64 i + 63 of the sequence in that slot.
// Rotation: column i of the rotated part is paired with column i + rot / 2; cos / sin per position from a table.
// Query rows are packed token-major, row r = token r / H, head r % H.
#include "seq.h"

struct LatArgs {
  const void* q; int ldq;              // [T][H heads of D columns], rotated part at column ra of a head, before rotation
  const void* ql; int ldl;             // [T][H][L] queries in the latent space
  void* pages; const float* rot;       // rot [positions][rot / 2][2]
  const int* table; int max_pages, npages, npos;
  const float* sink;                   // [H]
  void* out; int ldo;                  // [T][H][L]
  int H, D, ra, rdim, L, R;            // heads, columns of a query head, rotated part's offset and true size
  float scale;
  SeqMeta m;
  float* part; float* part_ml; int nsplit, pps;  // splits over pages: [B][rows][nsplit][L], [B][rows][nsplit][2]
  int rows;                                      // rows (tokens x heads) of the longest portion
};

__device__ __forceinline__ int lat_entry(const LatArgs& a, int slot, int i) {
  return a.table[(size_t)slot * a.max_pages + min(i, a.max_pages - 1)];
}
__device__ __forceinline__ int lat_page_of(const LatArgs& a, int entry) {
  DA_ASSERT(entry >= 0 && entry < a.npages);
  return min(max(entry, 0), a.npages - 1);
}
__device__ __forceinline__ int lat_page(const LatArgs& a, int slot, int i) { return lat_page_of(a, lat_entry(a, slot, i)); }

// ------------------------------------------------------------------------------- norms, rotation, page write
struct LatPrepArgs {
  LatArgs a;
  const void* x; int ldx;              // [T][Q | L | R]
  const float* qw; const float* cw;    // norm weights, zero in padding columns
  void* cq; int Q, qdim, cdim;
  float eps;
};

template <int K> struct Pieces { static constexpr int N = K; };

// Two waves per token: one norms the query latent to its own matrix; the other norms the cached latent and rotates the
// key part, both to the token's page.
template <typename T>
__global__ void __launch_bounds__(256) latent_prep_kernel(LatPrepArgs p) {
  const LatArgs& a = p.a;
  const int item = blockIdx.x * 4 + (threadIdx.x >> 6), t = item >> 1, l = threadIdx.x & 63;
  if (t >= a.m.T) return;
  const T* x = (const T*)p.x + (size_t)t * p.ldx;
  auto norm = [&](auto pieces, const T* src, T* out, const float* w, int n, int dim) {
    constexpr int U = decltype(pieces)::N;  // pieces of 256 columns kept in registers
    f32x4_t v[U], g[U];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const int c = min((i * 64 + l) * 4, n - 4);
      v[i] = Act<T>::load4(src + c);
      g[i] = *(const f32x4_t*)(w + c);
    }
#pragma unroll
    for (int i = 0; i < U; ++i)
      if ((i * 64 + l) * 4 < n)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss = fmaf(v[i][e], v[i][e], ss);
    for (int c = (U * 64 + l) * 4; c < n; c += 256) {
      const f32x4_t y = Act<T>::load4(src + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(y[e], y[e], ss);
    }
    const float inv = 1.f / sqrtf(wave_sum(ss) / dim + p.eps);
#pragma unroll
    for (int i = 0; i < U; ++i)
      if ((i * 64 + l) * 4 < n) Act<T>::store4(out + (i * 64 + l) * 4, v[i] * inv * g[i]);
    for (int c = (U * 64 + l) * 4; c < n; c += 256)
      Act<T>::store4(out + c, Act<T>::load4(src + c) * inv * *(const f32x4_t*)(w + c));
  };
  if (!(item & 1)) {
    norm(Pieces<6>{}, x, (T*)p.cq + (size_t)t * p.Q, p.qw, p.Q, p.qdim);
    return;
  }
  const int b = a.m.seq[t], pos = a.m.pos0[b] + t - a.m.cu[b];
  const T* kr = x + p.Q + a.L;
  const int half = a.rdim / 2;
  const float* cs = a.rot + (size_t)min(pos, a.npos - 1) * a.rdim;
  auto turned = [&](int c) {  // loads first: column c, its partner, their angle
    const int i = min(c, a.rdim - 1), j = i < half ? i : i - half;
    const float v = Act<T>::to_f(kr[c]), w = Act<T>::to_f(kr[i < half ? i + half : j]), co = cs[2 * j], si = cs[2 * j + 1];
    return c >= a.rdim ? v : c < half ? v * co - w * si : v * co + w * si;
  };
  const float first = turned(min(l, a.R - 1));
  T* page = (T*)a.pages + ((size_t)lat_page(a, a.m.slot[b], pos / PAGE) * PAGE + pos % PAGE) * (a.L + a.R);
  if (l < a.R) page[a.L + l] = Act<T>::from_f(first);
  for (int c = l + 64; c < a.R; c += 64) page[a.L + c] = Act<T>::from_f(turned(c));
  norm(Pieces<2>{}, x + p.Q, page, p.cw, a.L, p.cdim);
}

// Element c of a query head's rotated part at position pos (zero past it). Rounded to the activation type, as the
// cached keys are.
template <typename T>
__device__ __forceinline__ float rotated(const T* qr, const float* cs, int rdim, int c) {
  const int half = rdim / 2;
  float v = 0.f;
  if (c < half) v = Act<T>::to_f(qr[c]) * cs[2 * c] - Act<T>::to_f(qr[c + half]) * cs[2 * c + 1];
  else if (c < rdim) v = Act<T>::to_f(qr[c]) * cs[2 * (c - half)] + Act<T>::to_f(qr[c - half]) * cs[2 * (c - half) + 1];
  return Act<T>::to_f(Act<T>::from_f(v));
}

// Elements c .. c + 7 (c a multiple of 8), with loads that do not wait for each other.
__device__ __forceinline__ bf16x8_t rotated8(const bf16_t* qr, const float* cs, int rdim, int c) {
  const int half = rdim / 2;
  float x[8], y[8], co[8], si[8];  // elements, what they are paired with, angles
  if (half % 8 == 0) {
    const int a = min(c, rdim - 8), j = a < half ? a : a - half;
    const bf16x8_t u = *(const bf16x8_t*)(qr + a), v = *(const bf16x8_t*)(qr + (a < half ? a + half : j));
    f32x4_t t[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) t[i] = *(const f32x4_t*)(cs + 2 * j + 4 * i);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      x[e] = bf2f((bf16_t)u[e]);
      y[e] = bf2f((bf16_t)v[e]);
      co[e] = t[e >> 1][2 * (e & 1)];
      si[e] = t[e >> 1][2 * (e & 1) + 1];
    }
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int a = min(c + e, rdim - 1), j = a < half ? a : a - half;
      x[e] = bf2f(qr[a]);
      y[e] = bf2f(qr[a < half ? a + half : j]);
      co[e] = cs[2 * j];
      si[e] = cs[2 * j + 1];
    }
  }
  bf16x8_t r;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float s = c + e < half ? -si[e] : si[e];
    r[e] = (short)f2bf(c + e < rdim ? fmaf(x[e], co[e], y[e] * s) : 0.f);
  }
  return r;
}

// ------------------------------------------------------------------------------- any size, fp32 arithmetic
// 16 query rows per workgroup against KT-key tiles in LDS; scores and sums on the vector ALUs. The fp32 precision
// runs here, and bf16 sizes that the matrix-core kernels do not take.
template <typename T, int KT, int ND>  // ND: output columns per thread (16 threads a row)
__global__ void __launch_bounds__(256) latent_any_kernel(LatArgs a) {
  extern __shared__ float sm[];
  const int W = a.L + a.R, WS = W + 1;
  const int b = blockIdx.y, s0 = a.m.cu[b], n = a.m.cu[b + 1] - s0, rows = n * a.H;
  const int r0 = blockIdx.x * 16;
  if (r0 >= rows) return;
  float* sq = sm;               // [16][WS]
  float* sk = sq + 16 * WS;     // [KT][WS]
  float* sw = sk + KT * WS;     // [16][KT + 1]
  const int tid = threadIdx.x, r = tid >> 4, j = tid & 15;
  const int pos0 = a.m.pos0[b], slot = a.m.slot[b];
  for (int i = tid; i < 16 * W; i += 256) {
    const int rr = min(r0 + i / W, rows - 1), c = i % W, tok = rr / a.H, h = rr % a.H;
    float v;
    if (c < a.L) v = Act<T>::to_f(((const T*)a.ql)[(size_t)(s0 + tok) * a.ldl + (size_t)h * a.L + c]);
    else v = rotated<T>((const T*)a.q + (size_t)(s0 + tok) * a.ldq + (size_t)h * a.D + a.ra,
                        a.rot + (size_t)min(pos0 + tok, a.npos - 1) * a.rdim, a.rdim, c - a.L);
    sq[(i / W) * WS + c] = v;
  }
  const int row = r0 + r, rc = min(row, rows - 1), tok = rc / a.H, hd = rc % a.H;
  const int qpos = pos0 + tok;
  const int kend = pos0 + min(r0 + 15, rows - 1) / a.H + 1;  // keys the tile's last row sees
  float mx = a.sink[hd], sum = 1.f, acc[ND];
#pragma unroll
  for (int i = 0; i < ND; ++i) acc[i] = 0.f;
  for (int k0 = 0; k0 < kend; k0 += KT) {
    const T* kp = (const T*)a.pages + ((size_t)lat_page(a, slot, k0 / PAGE) * PAGE + k0 % PAGE) * W;
    __syncthreads();
    for (int i = tid; i < KT * W; i += 256) sk[(i / W) * WS + i % W] = k0 + i / W < kend ? Act<T>::to_f(kp[i]) : 0.f;
    __syncthreads();
    const float* q = sq + r * WS;
    float s[KT / 16], top = mx;
#pragma unroll
    for (int u = 0; u < KT / 16; ++u) {
      const float* x = sk + (j + 16 * u) * WS;
      float d = 0.f;
      for (int c = 0; c < W; ++c) d = fmaf(q[c], x[c], d);
      s[u] = k0 + j + 16 * u <= qpos ? d * a.scale : -INFINITY;
      top = fmaxf(top, s[u]);
    }
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) top = fmaxf(top, __shfl_xor(top, o, 64));
    const float f = expf(mx - top);
    mx = top;
    float ps = 0.f;
#pragma unroll
    for (int u = 0; u < KT / 16; ++u) {
      const float w = expf(s[u] - top);
      sw[r * (KT + 1) + j + 16 * u] = w;
      ps += w;
    }
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) ps += __shfl_xor(ps, o, 64);
    sum = fmaf(sum, f, ps);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < ND; ++i) acc[i] *= f;
    for (int k = 0; k < KT; ++k) {
      const float w = sw[r * (KT + 1) + k];
#pragma unroll
      for (int i = 0; i < ND; ++i)
        if (j + 16 * i < a.L) acc[i] = fmaf(w, sk[k * WS + j + 16 * i], acc[i]);
    }
  }
  if (row >= rows) return;
  T* o = (T*)a.out + (size_t)(s0 + tok) * a.ldo + (size_t)hd * a.L;
#pragma unroll
  for (int i = 0; i < ND; ++i)
    if (j + 16 * i < a.L) o[j + 16 * i] = Act<T>::from_f(acc[i] / sum);
}

template <typename T, int KT, int ND>
static int launch_lat_any(const LatArgs& a, hipStream_t s) {
  const size_t lds = (size_t)((16 + KT) * (a.L + a.R + 1) + 16 * (KT + 1)) * 4;
  if (lds > 65536) {
    const hipError_t e = hipFuncSetAttribute((const void*)latent_any_kernel<T, KT, ND>,
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  latent_any_kernel<T, KT, ND><<<dim3((a.rows + 15) / 16, a.m.B), 256, lds, s>>>(a);
  DA_LAUNCH_CHECK();
}
template <typename T>
static int launch_lat_any_t(const LatArgs& a, hipStream_t s) {
  if (a.L <= 64) return launch_lat_any<T, 32, 4>(a, s);
  if (a.L <= 128) return launch_lat_any<T, 32, 8>(a, s);
  if (a.L <= 256) return launch_lat_any<T, 32, 16>(a, s);
  if (a.L + a.R <= 768) return launch_lat_any<T, 32, 48>(a, s);
  return launch_lat_any<T, 16, 72>(a, s);
}

// ------------------------------------------------------------------------------- matrix cores, absorbed
// 16 query rows per workgroup, 4 waves, one page per step. A wave loads its 16 keys of the page in the score
// product's operand layout straight to registers (S^T = K Q^T on 16x16x32 MFMAs), and leaves their latents in LDS for
// the transposing reads of the sum, O^T += C^T P^T, in which it owns a quarter of the latent's columns for all keys of the
// page. The next page's loads are in flight during the sum. A weight enters the second product as two bf16 terms (its
// rounding and the remainder), so its fp32 value counts to about 16 bits.
template <int L> struct LD {
  static constexpr int VSTR = L == 64 ? 192 : L * 2 + 64;  // bytes of a latent in LDS
  static constexpr int PSTR = PAGE * 2 + 16;               // bytes of a row's weights
  static constexpr int OFF_P = PAGE * VSTR, OFF_MX = OFF_P + 2 * 16 * PSTR, BYTES = OFF_MX + 4 * 16 * 4;
};

__device__ __forceinline__ unsigned split_lo(unsigned hi, float a, float b) {
  return pack_bf2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}

template <int L, int R>
__global__ void __launch_bounds__(256, 2) latent_mfma_kernel(LatArgs a, int rtiles, int ntiles) {
  using C = LD<L>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int W = L + R, NDS = W / 32, NLS = L / 32, NDB = L / 64;
  // the row tiles of one split of a portion follow each other on one XCD: its pages are read from HBM once
  const int id = xcd_remap(blockIdx.x, ntiles);
  const int rt = id % rtiles, split = id / rtiles % a.nsplit, b = id / rtiles / a.nsplit;
  const int s0 = a.m.cu[b], n = a.m.cu[b + 1] - s0, rows = n * a.H;
  if (rt * 16 >= rows) return;
  const int pos0 = a.m.pos0[b], slot = a.m.slot[b];
  const int klast = pos0 + min(rt * 16 + 15, rows - 1) / a.H;  // last key of the tile
  const int p0 = split * a.pps, p1 = min(p0 + a.pps, klast / PAGE + 1);
  if (p0 >= p1) return;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, fr = lane & 15, fg = lane >> 4;
  const int row = rt * 16 + fr, rc = min(row, rows - 1), tok = rc / a.H, hd = rc % a.H;
  const int qpos = pos0 + tok;
  char* sV = smem;
  char* sP = smem + C::OFF_P;
  float* sM = (float*)(smem + C::OFF_MX);

  bf16x8_t qf[NDS];
  const bf16_t* ql = (const bf16_t*)a.ql + (size_t)(s0 + tok) * a.ldl + (size_t)hd * L + fg * 8;
#pragma unroll
  for (int ds = 0; ds < NLS; ++ds) qf[ds] = *(const bf16x8_t*)(ql + ds * 32);
  const bf16_t* qr = (const bf16_t*)a.q + (size_t)(s0 + tok) * a.ldq + (size_t)hd * a.D + a.ra;
  const float* cs = a.rot + (size_t)min(qpos, a.npos - 1) * a.rdim;
#pragma unroll
  for (int ds = NLS; ds < NDS; ++ds) qf[ds] = rotated8(qr, cs, a.rdim, (ds - NLS) * 32 + fg * 8);
  const float c2 = a.scale * LOG2E;

  bf16x8_t kf[NDS];
  const int key = wv * 16 + fr;  // the key of a page this lane loads
  auto load_page = [&](int p, int entry) {
    // rows past the last key may hold anything: that key's instead (their weights are zero)
    const bf16_t* kp = (const bf16_t*)a.pages + ((size_t)lat_page_of(a, entry) * PAGE + min(key, klast - p * PAGE)) * W + fg * 8;
#pragma unroll
    for (int ds = 0; ds < NDS; ++ds) kf[ds] = *(const bf16x8_t*)(kp + ds * 32);
  };
  f32x4_t oacc[NDB];
#pragma unroll
  for (int i = 0; i < NDB; ++i) oacc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float mx = -1e30f, sum = 0.f;  // of row fr: common to the waves; over this lane's keys
  load_page(p0, lat_entry(a, slot, p0));
  int next = lat_entry(a, slot, p0 + 1);
  for (int p = p0; p < p1; ++p) {
    f32x4_t s{0.f, 0.f, 0.f, 0.f}, s1 = s;
#pragma unroll
    for (int ds = 0; ds < NDS; ds += 2) {
      s = mfma16(kf[ds], qf[ds], s);
      if (ds + 1 < NDS) s1 = mfma16(kf[ds + 1], qf[ds + 1], s1);
    }
    s += s1;
    float top = -1e30f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      s[e] = p * PAGE + wv * 16 + fg * 4 + e <= qpos ? s[e] * c2 : -INFINITY;
      top = fmaxf(top, s[e]);
    }
    top = fmaxf(top, __shfl_xor(top, 16, 64));
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    if (fg == 0) sM[wv * 16 + fr] = top;
    lds_barrier();  // maxima written; every wave is done with the last page's latents and weights
#pragma unroll
    for (int ds = 0; ds < NLS; ++ds) *(bf16x8_t*)(sV + key * C::VSTR + ds * 64 + fg * 16) = kf[ds];
    if (p + 1 < p1) {
      load_page(p + 1, next);
      next = lat_entry(a, slot, p + 2);
    }
    const float mnew = fmaxf(mx, fmaxf(fmaxf(sM[fr], sM[16 + fr]), fmaxf(sM[32 + fr], sM[48 + fr])));
    const float f = __builtin_amdgcn_exp2f(mx - mnew);
    mx = mnew;
    sum *= f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      s[e] = __builtin_amdgcn_exp2f(s[e] - mnew);
      sum += s[e];
    }
    const unsigned h0 = pack_bf2(s[0], s[1]), h1 = pack_bf2(s[2], s[3]);
    char* pp = sP + fr * C::PSTR + (wv * 16 + fg * 4) * 2;
    *(u32x2_t*)pp = u32x2_t{h0, h1};
    *(u32x2_t*)(pp + 16 * C::PSTR) = u32x2_t{split_lo(h0, s[0], s[1]), split_lo(h1, s[2], s[3])};
#pragma unroll
    for (int i = 0; i < NDB; ++i) oacc[i] *= f;
    lds_barrier();
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      // k slot 8 fg + j of the product holds key 32 half + 16 (j / 4) + 4 fg + j % 4
      const char* pr = sP + fr * C::PSTR + (half * 32 + fg * 4) * 2;
      const u32x2_t ha = *(const u32x2_t*)pr, hb = *(const u32x2_t*)(pr + 32);
      const u32x2_t la = *(const u32x2_t*)(pr + 16 * C::PSTR), lb = *(const u32x2_t*)(pr + 16 * C::PSTR + 32);
      const bf16x8_t bh = __builtin_bit_cast(bf16x8_t, u32x4_t{ha[0], ha[1], hb[0], hb[1]});
      const bf16x8_t bl = __builtin_bit_cast(bf16x8_t, u32x4_t{la[0], la[1], lb[0], lb[1]});
      const int vrow = half * 32 + 4 * fg + (fr >> 2);
#pragma unroll
      for (int db = 0; db < NDB; ++db) {
        const char* vp = sV + vrow * C::VSTR + ((wv * NDB + db) * 16 + 4 * (fr & 3)) * 2;
        const s16x4_t lo = lds_read_tr16(vp), up = lds_read_tr16(vp + 16 * C::VSTR);
        const bf16x8_t va = bf16x8_t{lo[0], lo[1], lo[2], lo[3], up[0], up[1], up[2], up[3]};
        oacc[db] = mfma16(va, bh, oacc[db]);
        oacc[db] = mfma16(va, bl, oacc[db]);
      }
    }
  }
  sum += __shfl_xor(sum, 16, 64);
  sum += __shfl_xor(sum, 32, 64);
  lds_barrier();
  if (fg == 0) sM[wv * 16 + fr] = sum;
  lds_barrier();
  sum = sM[fr] + sM[16 + fr] + sM[32 + fr] + sM[48 + fr];
  if (row >= rows) return;
  if (a.nsplit > 1) {
    const size_t at = ((size_t)b * a.rows + row) * a.nsplit + split;
    if (wv == 0 && fg == 0) *(f32x2_t*)(a.part_ml + at * 2) = f32x2_t{mx, sum};
#pragma unroll
    for (int db = 0; db < NDB; ++db) *(f32x4_t*)(a.part + at * L + (wv * NDB + db) * 16 + fg * 4) = oacc[db];
  } else {
    const float sink = a.sink[hd] * LOG2E, m2 = fmaxf(mx, sink);
    const float f = __builtin_amdgcn_exp2f(mx - m2), inv = f / fmaf(sum, f, __builtin_amdgcn_exp2f(sink - m2));
    bf16_t* o = (bf16_t*)a.out + (size_t)(s0 + tok) * a.ldo + (size_t)hd * L;
#pragma unroll
    for (int db = 0; db < NDB; ++db) Act<bf16_t>::store4(o + (wv * NDB + db) * 16 + fg * 4, oacc[db] * inv);
  }
}

// The splits of a row put together, and the sink. L / 4 threads (64 at least).
__global__ void latent_combine_kernel(LatArgs a) {
  const int row = blockIdx.x, b = blockIdx.y, s0 = a.m.cu[b], n = a.m.cu[b + 1] - s0;
  if (row >= n * a.H) return;
  const int tok = row / a.H, hd = row % a.H;
  const int used = min(a.nsplit, ((a.m.pos0[b] + tok) / PAGE + a.pps) / a.pps);  // splits that hold keys the row sees
  const size_t at = ((size_t)b * a.rows + row) * a.nsplit;
  const float sink = a.sink[hd] * LOG2E;
  float m = sink;
  for (int s = 0; s < used; ++s) m = fmaxf(m, a.part_ml[(at + s) * 2]);
  float sum = __builtin_amdgcn_exp2f(sink - m);
  const int c = threadIdx.x * 4;
  f32x4_t v{0.f, 0.f, 0.f, 0.f};
  for (int q = 0; q < used; q += 8) {
    f32x4_t x[8];
    f32x2_t ml[8];
#pragma unroll
    for (int s = 0; s < 8; ++s) {
      const size_t i = at + min(q + s, used - 1);
      x[s] = *(const f32x4_t*)(a.part + i * a.L + min(c, a.L - 4));
      ml[s] = *(const f32x2_t*)(a.part_ml + i * 2);
    }
#pragma unroll
    for (int s = 0; s < 8; ++s) {
      const float f = q + s < used ? __builtin_amdgcn_exp2f(ml[s][0] - m) : 0.f;
      sum = fmaf(ml[s][1], f, sum);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = fmaf(x[s][e], f, v[e]);
    }
  }
  if (c < a.L) Act<bf16_t>::store4((bf16_t*)a.out + (size_t)(s0 + tok) * a.ldo + (size_t)hd * a.L + c, v * (1.f / sum));
}

template <int L, int R>
static int launch_lat_mfma(const LatArgs& a, hipStream_t s) {
  static const hipError_t e = hipFuncSetAttribute((const void*)latent_mfma_kernel<L, R>,
                                                  hipFuncAttributeMaxDynamicSharedMemorySize, LD<L>::BYTES);
  if (e != hipSuccess) return (int)e;
  const int rtiles = (a.rows + 15) / 16;
  const long long tiles = (long long)rtiles * a.nsplit * a.m.B;
  if (tiles > 0x7fffffffll) return (int)hipErrorInvalidValue;
  latent_mfma_kernel<L, R><<<(int)tiles, 256, LD<L>::BYTES, s>>>(a, rtiles, (int)tiles);
  if (a.nsplit > 1) latent_combine_kernel<<<dim3(a.rows, a.m.B), L < 256 ? 64 : L / 4, 0, s>>>(a);
  DA_LAUNCH_CHECK();
}
static bool lat_mfma_dims(int L, int R) { return (L == 64 || L == 128 || L == 256 || L == 512) && (R == 32 || R == 64); }
static int launch_lat_mfma_t(const LatArgs& a, hipStream_t s) {
#define LAT_CASE(LL, RR) \
  if (a.L == LL && a.R == RR) return launch_lat_mfma<LL, RR>(a, s);
  LAT_CASE(64, 32) LAT_CASE(64, 64) LAT_CASE(128, 32) LAT_CASE(128, 64)
  LAT_CASE(256, 32) LAT_CASE(256, 64) LAT_CASE(512, 32) LAT_CASE(512, 64)
#undef LAT_CASE
  return (int)hipErrorInvalidValue;
}

// ------------------------------------------------------------------------------- matrix cores, expanded
// A page of a portion's context per workgroup: its cache rows to row cctx[b] + position of a packed matrix.
__global__ void __launch_bounds__(256) latent_gather_kernel(LatArgs a, const int* cctx, bf16_t* lat) {
  const int b = blockIdx.y, p = blockIdx.x, W = a.L + a.R, c0 = cctx[b];
  const int n = min(PAGE, cctx[b + 1] - c0 - p * PAGE);
  if (n <= 0) return;
  const u32x4_t* src = (const u32x4_t*)((const bf16_t*)a.pages + (size_t)lat_page(a, a.m.slot[b], p) * PAGE * W);
  u32x4_t* dst = (u32x4_t*)(lat + (size_t)(c0 + p * PAGE) * W);
  const int pieces = n * W / 8;
  constexpr int U = 6;
  for (int i0 = threadIdx.x; i0 < pieces; i0 += 256 * U) {
    u32x4_t v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) v[u] = src[min(i0 + 256 * u, pieces - 1)];
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (i0 + 256 * u < pieces) dst[i0 + 256 * u] = v[u];
  }
}

struct FlashArgs {
  LatArgs a;                  // q, rot, sink, out [T][H V], m
  const int* cctx;            // rows of portion b's context in lat / kv: cctx[b] + position
  const bf16_t* lat;          // [contexts][L + R]
  const bf16_t* kv; int ldkv; // [contexts][H][d keys | V values]
  const bf16_t* gate; int ldg;
  int qtiles;
};

// 128 query rows (tokens) of one head per workgroup (4 waves x 32), 64 keys per step: S^T = K Q^T on 32x32x16 MFMAs, a
// lane owns one query and 32 of the step's keys; its weights stay in registers as the B operand of O^T += V^T P^T. The
// next step's keys are in flight while this one's are used.
template <int D, int V> struct LF {
  static constexpr int KSTR = D * 2 + 16;
  static constexpr int VSTR = (V % 64 == 32) ? V * 2 : (V == 64 ? 192 : V * 2 + 64);
  static constexpr int KB = PAGE * KSTR, BYTES = KB + PAGE * VSTR;
};

template <int D, int V>
__global__ void __launch_bounds__(256, D + V > 320 ? 1 : 2) latent_flash_kernel(FlashArgs p, int ntiles) {
  using C = LF<D, V>;
  const LatArgs& a = p.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int NDS = D / 16, NDB = V / 32, KP = D / 32, VP = V / 32;  // MFMA steps, blocks; 16-byte pieces per thread
  // a head's tiles follow each other on one XCD (they read the same keys), the longest first
  const int id = xcd_remap(blockIdx.x, ntiles);
  const int qt = p.qtiles - 1 - id % p.qtiles, hd = id / p.qtiles % a.H, b = id / p.qtiles / a.H;
  const int s0 = a.m.cu[b], n = a.m.cu[b + 1] - s0;
  if (qt * 128 >= n) return;
  const int pos0 = a.m.pos0[b], c0 = p.cctx[b], nctx = p.cctx[b + 1] - c0;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, qr = lane & 31, hi = lane >> 5;
  const int tok = qt * 128 + wv * 32 + qr, tc = min(tok, n - 1), qpos = pos0 + tc;
  const int wfirst = pos0 + min(qt * 128 + wv * 32, n - 1), wlast = pos0 + min(qt * 128 + wv * 32 + 31, n - 1);
  const int klast = min(pos0 + min(qt * 128 + 127, n - 1), nctx - 1), nt = klast / PAGE + 1;
  const int d = a.ra, W = a.L + a.R;

  bf16x8_t qf[NDS];
  const bf16_t* qp = (const bf16_t*)a.q + (size_t)(s0 + tc) * a.ldq + (size_t)hd * a.D;
  const float* cs = a.rot + (size_t)min(qpos, a.npos - 1) * a.rdim;
#pragma unroll
  for (int ds = 0; ds < NDS; ++ds) {
    const int c = ds * 16 + hi * 8;
    if (ds * 16 < d) qf[ds] = *(const bf16x8_t*)(qp + min(c, d - 8));
    if (ds * 16 + 8 >= d) {
      const bf16x8_t r = rotated8(qp + d, cs, a.rdim, max(c - d, 0));
      qf[ds] = c < d ? qf[ds] : r;
    }
  }
  const float c2 = a.scale * LOG2E;

  u32x4_t kreg[KP], vreg[VP];
  auto load = [&](int t) {
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int pc = tid + 256 * i, r = pc / (D / 8), c = pc % (D / 8) * 8;
      const int k = min(t * PAGE + r, klast);
      const bf16_t* src = c < d ? p.kv + (size_t)(c0 + k) * p.ldkv + (size_t)hd * (d + V) + c
                                : p.lat + (size_t)(c0 + k) * W + a.L + min(c - d, a.R - 8);
      kreg[i] = *(const u32x4_t*)src;  // past d + R: any key's columns, the queries are zero there
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int pc = tid + 256 * i, r = pc / (V / 8), c = pc % (V / 8) * 8;
      vreg[i] = *(const u32x4_t*)(p.kv + (size_t)(c0 + min(t * PAGE + r, klast)) * p.ldkv + (size_t)hd * (d + V) + d + c);
    }
  };
  auto store = [&]() {
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int pc = tid + 256 * i;
      *(u32x4_t*)(smem + pc / (D / 8) * C::KSTR + pc % (D / 8) * 16) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int pc = tid + 256 * i;
      *(u32x4_t*)(smem + C::KB + pc / (V / 8) * C::VSTR + pc % (V / 8) * 16) = vreg[i];
    }
  };
  f32x16_t oacc[NDB];
#pragma unroll
  for (int i = 0; i < NDB; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) oacc[i][e] = 0.f;
  float mx = a.sink[hd] * LOG2E, sum = 1.f;

  load(0);
  for (int t = 0; t < nt; ++t) {
    lds_barrier();
    store();
    lds_barrier();
    if (t + 1 < nt) load(t + 1);
    const int kb = t * PAGE;
    if (kb > wlast) continue;
    f32x16_t s[2];
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
#pragma unroll
      for (int e = 0; e < 16; ++e) s[hh][e] = 0.f;
#pragma unroll
      for (int ds = 0; ds < NDS; ++ds) {
        const bf16x8_t kf = *(const bf16x8_t*)(smem + (hh * 32 + qr) * C::KSTR + ds * 32 + hi * 16);
        s[hh] = mfma32(kf, qf[ds], s[hh]);
      }
    }
    if (kb + PAGE - 1 > wfirst) {
#pragma unroll
      for (int hh = 0; hh < 2; ++hh)
#pragma unroll
        for (int e = 0; e < 16; ++e)
          if (kb + hh * 32 + 8 * (e >> 2) + 4 * hi + (e & 3) > qpos) s[hh][e] = -INFINITY;
    }
    float top = s[0][0];
#pragma unroll
    for (int e = 1; e < 16; ++e) top = fmaxf(top, s[0][e]);
#pragma unroll
    for (int e = 0; e < 16; ++e) top = fmaxf(top, s[1][e]);
    top = max_xhalf(top) * c2;
    if (__any(top > mx)) {
      const float mnew = fmaxf(mx, top), f = __builtin_amdgcn_exp2f(mx - mnew);
      mx = mnew;
      sum *= f;
#pragma unroll
      for (int i = 0; i < NDB; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e) oacc[i][e] *= f;
    }
    float ps = 0.f;
#pragma unroll
    for (int hh = 0; hh < 2; ++hh)
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        s[hh][e] = __builtin_amdgcn_exp2f(fmaf(s[hh][e], c2, -mx));
        ps += s[hh][e];
      }
    sum += sum_xhalf(ps);
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
        const char* vp = smem + C::KB + vrow * C::VSTR + (db * 32 + 16 * (g4 & 1) + 4 * (li & 3)) * 2;
        const s16x4_t lo = lds_read_tr16(vp), up = lds_read_tr16(vp + 8 * C::VSTR);
        const bf16x8_t va = bf16x8_t{lo[0], lo[1], lo[2], lo[3], up[0], up[1], up[2], up[3]};
        oacc[db] = mfma32(va, bh, oacc[db]);
        oacc[db] = mfma32(va, bl, oacc[db]);
      }
    }
  }
  if (tok >= n) return;
  const float inv = 1.f / sum;
  const bf16_t* g = p.gate + (size_t)(s0 + tok) * p.ldg + (size_t)hd * V;
  bf16_t* o = (bf16_t*)a.out + (size_t)(s0 + tok) * a.ldo + (size_t)hd * V;
  u32x2_t gates[NDB][4];  // loaded ahead of the stores, which they might alias
#pragma unroll
  for (int db = 0; db < NDB; ++db)
#pragma unroll
    for (int q = 0; q < 4; ++q) gates[db][q] = *(const u32x2_t*)(g + db * 32 + 8 * q + 4 * hi);
#pragma unroll
  for (int db = 0; db < NDB; ++db)
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int c = db * 32 + 8 * q + 4 * hi;
      const f32x4_t gt = Act<bf16_t>::load4((const bf16_t*)&gates[db][q]);
      f32x4_t y;
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] = oacc[db][4 * q + e] * inv * sigmoid32(gt[e]);
      Act<bf16_t>::store4(o + c, y);
    }
}

template <int D, int V>
static int launch_lat_flash(const FlashArgs& p, hipStream_t s) {
  static const hipError_t e = hipFuncSetAttribute((const void*)latent_flash_kernel<D, V>,
                                                  hipFuncAttributeMaxDynamicSharedMemorySize, LF<D, V>::BYTES);
  if (e != hipSuccess) return (int)e;
  const long long tiles = (long long)p.qtiles * p.a.H * p.a.m.B;
  if (tiles > 0x7fffffffll) return (int)hipErrorInvalidValue;
  latent_flash_kernel<D, V><<<(int)tiles, 256, LF<D, V>::BYTES, s>>>(p, (int)tiles);
  DA_LAUNCH_CHECK();
}
template <int D>
static int launch_lat_flash_v(const FlashArgs& p, int V, hipStream_t s) {
  switch (V) {
    case 32: return launch_lat_flash<D, 32>(p, s);
    case 64: return launch_lat_flash<D, 64>(p, s);
    case 96: return launch_lat_flash<D, 96>(p, s);
    case 128: return launch_lat_flash<D, 128>(p, s);
    default: return (int)hipErrorInvalidValue;
  }
}

// lat [contexts][L + R] <- the cache rows of every portion's context (positions 0 .. its last token), packed at cctx.
DA_EXPORT int da_latent_gather(void* pages, int npages, const void* table, int max_pages, int L, int R, const void* cctx,
                               int max_ctx, void* lat, const void* cu, const void* slot, const void* pos0, const void* seq,
                               int T, int B, void* stream) {
  if (T < 1 || B < 1 || B > 65535 || max_ctx < 1 || (L + R) % 8 || npages < 1 || max_pages < 1 ||
      (max_ctx + PAGE - 1) / PAGE > max_pages)
    return (int)hipErrorInvalidValue;
  LatArgs a{};
  a.pages = pages; a.table = (const int*)table; a.max_pages = max_pages; a.npages = npages; a.L = L; a.R = R;
  a.m = SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B};
  latent_gather_kernel<<<dim3((max_ctx + PAGE - 1) / PAGE, B), 256, 0, (hipStream_t)stream>>>(a, (const int*)cctx,
                                                                                             (bf16_t*)lat);
  DA_LAUNCH_CHECK();
}

// Attention (bf16) over keys and values expanded from the latents: kv [contexts][H][d | V], rotated key parts at column L
// of lat; times sigmoid(gate). D in {64, 96, 128, 192, 256} >= d + the rotated part, V in {32, 64, 96, 128}.
DA_EXPORT int da_latent_flash(const void* q, int ldq, const void* lat, const void* kv, int ldkv, const void* gate, int ldg,
                              const void* rot, int npos, const void* sink, void* out, int ldo, int H, int D, int d, int rdim,
                              int L, int R, int V, float scale, const void* cctx, int max_len, const void* cu,
                              const void* slot, const void* pos0, const void* seq, int T, int B, void* stream) {
  if (T < 1 || B < 1 || H < 1 || d < 8 || d % 8 || rdim < 2 || rdim % 2 || rdim > R || d + rdim > D || L % 8 || R < 8 || R % 8 ||
      ldq % 8 || ldkv % 8 || ldkv < H * (d + V) || ldg % 4 || ldo % 4 || npos < 1 || max_len < 1)
    return (int)hipErrorInvalidValue;
  FlashArgs p{};
  p.a.q = q; p.a.ldq = ldq; p.a.rot = (const float*)rot; p.a.npos = npos; p.a.sink = (const float*)sink;
  p.a.out = out; p.a.ldo = ldo; p.a.H = H; p.a.D = D; p.a.ra = d; p.a.rdim = rdim; p.a.L = L; p.a.R = R; p.a.scale = scale;
  p.a.m = SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B};
  p.cctx = (const int*)cctx; p.lat = (const bf16_t*)lat; p.kv = (const bf16_t*)kv; p.ldkv = ldkv;
  p.gate = (const bf16_t*)gate; p.ldg = ldg; p.qtiles = (max_len + 127) / 128;
  hipStream_t s = (hipStream_t)stream;
  switch (D) {
    case 64: return launch_lat_flash_v<64>(p, V, s);
    case 96: return launch_lat_flash_v<96>(p, V, s);
    case 128: return launch_lat_flash_v<128>(p, V, s);
    case 192: return launch_lat_flash_v<192>(p, V, s);
    case 256: return launch_lat_flash_v<256>(p, V, s);
    default: return (int)hipErrorInvalidValue;
  }
}

// x [T][ldx] = [query latent Q | latent L | key part R] before their norms and rotation -> cq [T][Q], and the token's
// cache row. rot fp32 [npos][rdim / 2][2]. Every count of columns a multiple of 4.
DA_EXPORT int da_latent_prep(const void* x, int ldx, const void* qw, int Q, int qdim, const void* cw, int L, int cdim, int R,
                             int rdim, float eps, void* cq, void* pages, int npages, const void* table, int max_pages,
                             const void* rot, int npos, const void* cu, const void* slot, const void* pos0,
                             const void* seq, int T, int B, int f32, void* stream) {
  if (T < 1 || B < 1 || Q < 4 || Q % 4 || L < 4 || L % 4 || R < 4 || R % 4 || rdim < 2 || rdim % 2 || rdim > R || qdim < 1 ||
      qdim > Q || cdim < 1 || cdim > L || ldx % 4 || npages < 1 || max_pages < 1 || npos < 1)
    return (int)hipErrorInvalidValue;
  LatPrepArgs p{};
  p.a.pages = pages; p.a.rot = (const float*)rot; p.a.table = (const int*)table;
  p.a.max_pages = max_pages; p.a.npages = npages; p.a.npos = npos;
  p.a.rdim = rdim; p.a.L = L; p.a.R = R;
  p.a.m = SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B};
  p.x = x; p.ldx = ldx; p.qw = (const float*)qw; p.cw = (const float*)cw; p.cq = cq;
  p.Q = Q; p.qdim = qdim; p.cdim = cdim; p.eps = eps;
  hipStream_t s = (hipStream_t)stream;
  if (f32) latent_prep_kernel<float><<<(T + 1) / 2, 256, 0, s>>>(p);
  else latent_prep_kernel<bf16_t><<<(T + 1) / 2, 256, 0, s>>>(p);
  DA_LAUNCH_CHECK();
}

// Attention of every token over positions 0 .. its own of its sequence, in the latent space (absorbed).
// max_len: longest portion. part / part_ml: scratch where nsplit > 1 (nsplit * pps pages >= the longest context).
DA_EXPORT int da_latent_attn(const void* q, int ldq, const void* ql, int ldl, void* pages, int npages, const void* table,
                             int max_pages, const void* rot, int npos, const void* sink, void* out, int ldo, int H, int D,
                             int ra, int rdim, int L, int R, float scale, void* part, void* part_ml, int nsplit, int pps,
                             int max_len, const void* cu, const void* slot, const void* pos0, const void* seq, int T,
                             int B, int f32, void* stream) {
  if (T < 1 || B < 1 || B > 65535 || H < 1 || ra < 0 || rdim < 2 || rdim % 2 || rdim > R || ra + rdim > D || L < 4 || L % 4 ||
      R % 4 || L > 1152 || L + R > 1216 || npages < 1 || max_pages < 1 || npos < 1 || max_len < 1 || nsplit < 1 || pps < 1 ||
      (nsplit > 1 && (!part || !part_ml)) || (long long)max_len * H > 0x7fffffffll)
    return (int)hipErrorInvalidValue;
  LatArgs a{q, ldq, ql, ldl, pages, (const float*)rot, (const int*)table, max_pages, npages, npos, (const float*)sink, out,
            ldo, H, D, ra, rdim, L, R, scale,
            SeqMeta{(const int*)cu, (const int*)slot, (const int*)pos0, (const int*)seq, T, B}, (float*)part,
            (float*)part_ml, nsplit, pps, max_len * H};
  hipStream_t s = (hipStream_t)stream;
  if (f32) return launch_lat_any_t<float>(a, s);
  return lat_mfma_dims(L, R) ? launch_lat_mfma_t(a, s) : launch_lat_any_t<bf16_t>(a, s);
}
