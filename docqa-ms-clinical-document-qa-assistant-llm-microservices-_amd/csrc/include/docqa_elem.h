// docqa_elem.h -- element access for kernels templated over bf16 and fp32 operands: vectors
// of V elements as floats, and sums over split-K slabs.
#pragma once
#include "docqa_common.h"

namespace docqa {

// element type tags are the storage types: uint16_t (bf16 bits) and float
__device__ __forceinline__ float ld1(const float* p) { return *p; }
__device__ __forceinline__ float ld1(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ void st1(float* p, float v) { *p = v; }
__device__ __forceinline__ void st1(uint16_t* p, float v) { *p = f2bf(v); }
// v as the storage type holds it
__device__ __forceinline__ float rnd(const float*, float v) { return v; }
__device__ __forceinline__ float rnd(const uint16_t*, float v) { return bf2f(f2bf(v)); }

template <int V>
__device__ __forceinline__ void ldv(const float* p, float* f) {
  if constexpr (V % 4 == 0) {
#pragma unroll
    for (int i = 0; i < V; i += 4) {
      const float4 v = *reinterpret_cast<const float4*>(p + i);
      f[i] = v.x; f[i + 1] = v.y; f[i + 2] = v.z; f[i + 3] = v.w;
    }
  } else if constexpr (V == 2) {
    const float2 v = *reinterpret_cast<const float2*>(p);
    f[0] = v.x; f[1] = v.y;
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) f[i] = p[i];
  }
}
template <int V>
__device__ __forceinline__ void ldv(const uint16_t* p, float* f) {
  if constexpr (V % 8 == 0) {
#pragma unroll
    for (int i = 0; i < V; i += 8) unpack8(*reinterpret_cast<const uint4*>(p + i), f + i);
  } else if constexpr (V == 4) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
    f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
  } else if constexpr (V == 2) {
    const uint32_t v = *reinterpret_cast<const uint32_t*>(p);
    f[0] = __uint_as_float(v << 16); f[1] = __uint_as_float(v & 0xffff0000u);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) f[i] = bf2f(p[i]);
  }
}
template <int V>
__device__ __forceinline__ void stv(float* p, const float* f) {
  if constexpr (V % 4 == 0) {
#pragma unroll
    for (int i = 0; i < V; i += 4) *reinterpret_cast<float4*>(p + i) = make_float4(f[i], f[i + 1], f[i + 2], f[i + 3]);
  } else if constexpr (V == 2) {
    *reinterpret_cast<float2*>(p) = make_float2(f[0], f[1]);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) p[i] = f[i];
  }
}
template <int V>
__device__ __forceinline__ void stv(uint16_t* p, const float* f) {
  if constexpr (V % 8 == 0) {
#pragma unroll
    for (int i = 0; i < V; i += 8) *reinterpret_cast<uint4*>(p + i) = pack8(f + i);
  } else if constexpr (V == 4) {
    uint2 v;
    v.x = pack2(f[0], f[1]); v.y = pack2(f[2], f[3]);
    *reinterpret_cast<uint2*>(p) = v;
  } else if constexpr (V == 2) {
    *reinterpret_cast<uint32_t*>(p) = pack2(f[0], f[1]);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) p[i] = f2bf(f[i]);
  }
}
// sum over S slabs of V consecutive elements at p (slab stride in elements), fp32
template <int V, typename PT>
__device__ __forceinline__ void ld_slabs(const PT* p, int S, size_t slab, float* f) {
  ldv<V>(p, f);
  int s = 1;
  for (; s + 1 < S; s += 2) {
    float g[V], h[V];
    ldv<V>(p + (size_t)s * slab, g);
    ldv<V>(p + (size_t)(s + 1) * slab, h);
#pragma unroll
    for (int i = 0; i < V; ++i) f[i] = (f[i] + g[i]) + h[i];
  }
  if (s < S) {
    float g[V];
    ldv<V>(p + (size_t)s * slab, g);
#pragma unroll
    for (int i = 0; i < V; ++i) f[i] += g[i];
  }
}

__device__ __forceinline__ float silu_fast(float x) { return x * __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
// log(1 + e^x) = max(x, 0) + log1p(e), e = e^-|x|; log1p(e) = log(u) e / (u - 1) with u = 1 + e
// rounded (Kahan's correction of the rounding in u), e itself once u rounds to 1
__device__ __forceinline__ float softplus_f(float x) {
  const float e = __expf(-fabsf(x)), u = 1.f + e, v = u - 1.f;
  const float l = v > 0.f ? __logf(u) * e * __builtin_amdgcn_rcpf(v) : e;
  return fmaxf(x, 0.f) + l;
}

}  // namespace docqa
