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

__device__ __forceinline__ int lat_page(const LatArgs& a, int slot, int i) {
  const int p = a.table[(size_t)slot * a.max_pages + min(i, a.max_pages - 1)];
  DA_ASSERT(p >= 0 && p < a.npages);
  return min(max(p, 0), a.npages - 1);
}

// ------------------------------------------------------------------------------- norms, rotation, page write
struct LatPrepArgs {
  LatArgs a;
  const void* x; int ldx;              // [T][Q | L | R]
  const float* qw; const float* cw;    // norm weights, zero in padding columns
  void* cq; int Q, qdim, cdim;
  float eps;
};

// A wave per token: the query latent normed to its own matrix, the cached latent normed and the key part rotated to
// the token's page.
template <typename T>
__global__ void __launch_bounds__(256) latent_prep_kernel(LatPrepArgs p) {
  const LatArgs& a = p.a;
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), l = threadIdx.x & 63;
  if (t >= a.m.T) return;
  const int b = a.m.seq[t], pos = a.m.pos0[b] + t - a.m.cu[b];
  const T* x = (const T*)p.x + (size_t)t * p.ldx;
  const int W = a.L + a.R;
  T* page = (T*)a.pages + ((size_t)lat_page(a, a.m.slot[b], pos / PAGE) * PAGE + pos % PAGE) * W;
  auto norm = [&](const T* src, T* dst, const float* w, int n, int dim) {
    float ss = 0.f;
    for (int c = l * 4; c < n; c += 256) {
      const f32x4_t v = Act<T>::load4(src + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(v[e], v[e], ss);
    }
    const float inv = 1.f / sqrtf(wave_sum(ss) / dim + p.eps);
    for (int c = l * 4; c < n; c += 256) {
      f32x4_t v = Act<T>::load4(src + c);
      const f32x4_t g = *(const f32x4_t*)(w + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= inv * g[e];
      Act<T>::store4(dst + c, v);
    }
  };
  norm(x, (T*)p.cq + (size_t)t * p.Q, p.qw, p.Q, p.qdim);
  norm(x + p.Q, page, p.cw, a.L, p.cdim);
  const T* kr = x + p.Q + a.L;
  const int half = a.rdim / 2;
  const float* cs = a.rot + (size_t)min(pos, a.npos - 1) * a.rdim;
  for (int c = l; c < a.R; c += 64) {
    float v = Act<T>::to_f(kr[c]);
    if (c < half) v = v * cs[2 * c] - Act<T>::to_f(kr[c + half]) * cs[2 * c + 1];
    else if (c < a.rdim) v = v * cs[2 * (c - half)] + Act<T>::to_f(kr[c - half]) * cs[2 * (c - half) + 1];
    page[a.L + c] = Act<T>::from_f(v);
  }
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
  if (f32) latent_prep_kernel<float><<<(T + 3) / 4, 256, 0, s>>>(p);
  else latent_prep_kernel<bf16_t><<<(T + 3) / 4, 256, 0, s>>>(p);
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
  return f32 ? launch_lat_any_t<float>(a, s) : launch_lat_any_t<bf16_t>(a, s);
}
