// Shared pieces of the kernels that run a batch of sequence portions against per-sequence state.
#pragma once
#include "common.h"

// A step's batch: B portions packed row after row. Portion b is rows cu[b] .. cu[b + 1] - 1 of the
// packed matrices, the tokens at positions pos0[b], pos0[b] + 1, ... of the sequence that owns state
// slot slot[b]; seq[t] is the portion of packed row t. A portion at position 0 starts its sequence:
// whatever its slot holds from an earlier owner is not read.
struct SeqMeta {
  const int* cu; const int* slot; const int* pos0; const int* seq;
  int T, B;
};

// Chunks of `len` tokens for the recurrences: chunk i is tokens [len * ck[2i+1], + len) of portion ck[2i];
// base[b] is the number of chunks of the portions before b.
struct ChunkMeta {
  const int* ck; const int* base;
  int n, len;
};
constexpr int PAGE = 64;  // tokens per cache page

// Activation storage: bf16 (the serving precision) or fp32; arithmetic is fp32 either way.
template <typename T> struct Act;
template <> struct Act<bf16_t> {
  __device__ static __forceinline__ float to_f(bf16_t v) { return bf2f(v); }
  __device__ static __forceinline__ bf16_t from_f(float v) { return f2bf(v); }
  __device__ static __forceinline__ f32x4_t load4(const bf16_t* p) {
    const u32x2_t u = *(const u32x2_t*)p;
    return f32x4_t{__uint_as_float(u[0] << 16), __uint_as_float(u[0] & 0xffff0000u), __uint_as_float(u[1] << 16),
                   __uint_as_float(u[1] & 0xffff0000u)};
  }
  __device__ static __forceinline__ void store4(bf16_t* p, const f32x4_t& v) {
    *(u32x2_t*)p = u32x2_t{pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3])};
  }
  __device__ static __forceinline__ f32x2_t load2(const bf16_t* p) {
    const unsigned u = *(const unsigned*)p;
    return f32x2_t{__uint_as_float(u << 16), __uint_as_float(u & 0xffff0000u)};
  }
  __device__ static __forceinline__ void store2(bf16_t* p, float a, float b) { *(unsigned*)p = pack_bf2(a, b); }
};
template <> struct Act<float> {
  __device__ static __forceinline__ float to_f(float v) { return v; }
  __device__ static __forceinline__ float from_f(float v) { return v; }
  __device__ static __forceinline__ f32x4_t load4(const float* p) { return *(const f32x4_t*)p; }
  __device__ static __forceinline__ void store4(float* p, const f32x4_t& v) { *(f32x4_t*)p = v; }
  __device__ static __forceinline__ f32x2_t load2(const float* p) { return *(const f32x2_t*)p; }
  __device__ static __forceinline__ void store2(float* p, float a, float b) { *(f32x2_t*)p = f32x2_t{a, b}; }
};

// Workgroup barrier for LDS alone: this wave's LDS accesses are done, its global loads stay in flight
// (__syncthreads() waits for those too).
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// Elementary functions good to a few fp32 ulp on the hardware's 1-ulp exp2 / log2 / rcp / sqrt (the library
// forms spend most of their instructions on cases that cannot occur here: the epilogues and scans that
// use these run at their instruction count).
constexpr float LOG2E = 1.4426950408889634f;
// e^x: relative error |x| * 2^-24 from the product's rounding, 1 ulp from the exponential
__device__ __forceinline__ float exp32(float x) { return __builtin_amdgcn_exp2f(x * LOG2E); }
__device__ __forceinline__ float sigmoid32(float x) { return __builtin_amdgcn_rcpf(1.f + exp32(-x)); }
// log(1 + e^x) = max(x, 0) + log1p(e), e = e^-|x|; log1p(e) = log(u) e / (u - 1) with u = fl(1 + e), which
// cancels the rounding of u (Goldberg, "What every computer scientist should know about floating-point
// arithmetic", 1991, theorem 4).
__device__ __forceinline__ float softplus32(float x) {
  const float e = exp32(-fabsf(x)), u = 1.f + e, d = u - 1.f;
  const float l = __builtin_amdgcn_logf(u) * 0.6931471805599453f;
  return fmaxf(x, 0.f) + (d == 0.f ? e : l * e * __builtin_amdgcn_rcpf(d));
}
// 1 - e^(2 y) for y <= 0, given a = e^y: the series of the exponential where the difference would cancel.
__device__ __forceinline__ float one_minus_square32(float y, float a) {
  const float x = 2.f * y;
  float p = fmaf(x, 1.f / 8.f, 1.f);
  p = fmaf(p * x, 1.f / 7.f, 1.f);
  p = fmaf(p * x, 1.f / 6.f, 1.f);
  p = fmaf(p * x, 1.f / 5.f, 1.f);
  p = fmaf(p * x, 1.f / 4.f, 1.f);
  p = fmaf(p * x, 1.f / 3.f, 1.f);
  p = fmaf(p * x, 1.f / 2.f, 1.f);
  return x > -0.4f ? -x * p : fmaf(-a, a, 1.f);
}
__device__ __forceinline__ float silu32(float x) { return x * sigmoid32(x); }
// The same for outputs that are rounded to the activation type anyway: bf16 takes the short forms.
template <typename T> __device__ __forceinline__ float act_silu(float x) {
  if constexpr (sizeof(T) == 2) return silu(x);
  else return silu32(x);
}
__device__ __forceinline__ float gelu_tanh32(float x) {
  // 0.5 (1 + tanh(z)) = sigmoid(2 z)
  return x * sigmoid32(1.5957691216057308f * (x + 0.044715f * x * x * x));
}
template <typename T> __device__ __forceinline__ float act_gelu_tanh(float x) {
  if constexpr (sizeof(T) == 4) return gelu_tanh32(x);
  return x * __builtin_amdgcn_rcpf(1.f + __expf(-1.5957691216057308f * (x + 0.044715f * x * x * x)));
}

// The state of a short causal convolution, replaced by the launch of the recurrence behind it.
struct ConvState {
  const void* x; int ldx;   // the convolution's inputs
  void* state; int taps, C; // [slots][taps - 1][C], oldest first
};

// The last taps - 1 inputs of portion b's channel c, after its n tokens (the slot's older ones where the
// portion is shorter; one thread per channel, old entries are read before they are overwritten).
template <typename T>
__device__ __forceinline__ void conv_state_store(const ConvState& s, const SeqMeta& m, int b, int c) {
  if (!s.state) return;
  const int s0 = m.cu[b], n = m.cu[b + 1] - s0, keep = s.taps - 1;
  const bool start = m.pos0[b] == 0;
  T* st = (T*)s.state + (size_t)m.slot[b] * keep * s.C + c;
  const T* x = (const T*)s.x + c;
  constexpr int U = 4;
  for (int i0 = 0; i0 < keep; i0 += U) {
    T v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int i = min(i0 + u, keep - 1), j = n - keep + i;
      v[u] = j >= 0 ? x[(size_t)(s0 + j) * s.ldx] : (start ? Act<T>::from_f(0.f) : st[(size_t)(i + n) * s.C]);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (i0 + u < keep) st[(size_t)(i0 + u) * s.C] = v[u];
  }
}
