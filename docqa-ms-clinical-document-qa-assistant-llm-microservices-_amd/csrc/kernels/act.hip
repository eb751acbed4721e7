// act.hip -- element-wise activations that sit between library GEMMs:
//   * silu_mul  : SwiGLU  out[t, i] = silu(gu[t, i]) * gu[t, I + i]   (Llama MLP; the
//                 gate and up projections are one fused [H, 2I] GEMM whose output rows
//                 are [gate | up])
//   * bias_gelu : out = gelu_erf(x + bias)  (BERT FFN, when the bias is not fused into
//                 the MFMA GEMM epilogue)
//   * add_bias  : out = x + bias [+ residual]
// All are 16-byte vectorised and grid-strided (cdna_hip_programming.md Guideline 13,
// Guideline 11 grid sizing: <= 2048 blocks, grid-stride the rest).
#include "docqa_common.h"
#include "docqa_elem.h"
#include "docqa_gate.h"

using namespace docqa;

__device__ __forceinline__ float silu(float x) { return x / (1.f + __expf(-x)); }
__device__ __forceinline__ float gelu_erf(float x) { return 0.5f * x * (1.f + erff(x * 0.70710678118654752f)); }

// IL: gate|up rows interleaved in blocks of 8 (the layout the decode GEMM's fused SwiGLU
// epilogue reads): output chunk c = silu(chunk 2c) * chunk 2c+1 of the row.
template <bool IL>
__global__ __launch_bounds__(256) void silu_mul_kernel(const uint16_t* __restrict__ gu,
                                                       uint16_t* __restrict__ out, int T, int I) {
  // 32-bit index math (T * I / 8 < 2^31 is checked by the launcher): 64-bit integer
  // division is a ~100-instruction software sequence on CDNA.
  const int cpr = I >> 3;  // chunks per row
  const int total = T * cpr;
  for (int idx = blockIdx.x * blockDim.x + threadIdx.x; idx < total;
       idx += gridDim.x * blockDim.x) {
    const int t = idx / cpr;
    const int c = idx - t * cpr;
    const uint4* row = reinterpret_cast<const uint4*>(gu + t * (size_t)(2 * I));
    float g[8], u[8], o[8];
    unpack8(row[IL ? 2 * c : c], g);
    unpack8(row[IL ? 2 * c + 1 : cpr + c], u);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = silu(g[j]) * u[j];
    reinterpret_cast<uint4*>(out + t * (size_t)I)[c] = pack8(o);
  }
}

// split-K SwiGLU consumer: P [S, T, 2I] fp32 slabs of an 8-interleaved gate|up GEMM ->
// out [T, I] = silu(bf16(sum gate)) * bf16(sum up), slabs summed in slab order (the rounding
// of the fused-epilogue GEMMs: the gate / up values as the bf16 GEMM output).  The gate|up
// projection at prefill sizes whose 256 x 256 tiles cannot fill the chip (the 70B TP-8
// shard: 56 tiles at 512 rows) is split over K into these slabs (pgemm.hip EPI_PARTIAL).
__global__ __launch_bounds__(256) void silu_mul_splitk_kernel(const float* __restrict__ P,
                                                              uint16_t* __restrict__ out, int S, int T, int I) {
  const int cpr = I >> 3;
  const int total = T * cpr;
  const size_t slab4 = (size_t)T * (size_t)(2 * I) / 4;   // one slab in float4
  for (int idx = blockIdx.x * blockDim.x + threadIdx.x; idx < total; idx += gridDim.x * blockDim.x) {
    const int t = idx / cpr;
    const int c = idx - t * cpr;
    const float4* p = reinterpret_cast<const float4*>(P + (size_t)t * (size_t)(2 * I)) + 4 * c;
    float4 v[4] = {p[0], p[1], p[2], p[3]};
    for (int sl = 1; sl < S; ++sl) {
      const float4* q = p + sl * slab4;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float4 w = q[j];
        v[j].x += w.x; v[j].y += w.y; v[j].z += w.z; v[j].w += w.w;
      }
    }
    const float g[8] = {v[0].x, v[0].y, v[0].z, v[0].w, v[1].x, v[1].y, v[1].z, v[1].w};
    const float u[8] = {v[2].x, v[2].y, v[2].z, v[2].w, v[3].x, v[3].y, v[3].z, v[3].w};
    float o[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = silu(bf2f(f2bf(g[j]))) * bf2f(f2bf(u[j]));
    reinterpret_cast<uint4*>(out + (size_t)t * I)[c] = pack8(o);
  }
}

// the same from bf16 slabs (mgemm.hip EPI_PARTIAL16: the batch-256 decode gate|up on 256-wide
// tiles split over K, X re-read half as often as the fused-SwiGLU 128-wide tiles).  NS > 0:
// S known at compile time, every slab load in flight before the first add; sum in fp32 in
// slab order.
template <int NS>
__global__ __launch_bounds__(256) void silu_mul_splitk16_kernel(const uint16_t* __restrict__ P,
                                                                uint16_t* __restrict__ out, int S, int T, int I) {
  const int cpr = I >> 3;
  const int total = T * cpr;
  const size_t slab8 = (size_t)T * (size_t)(2 * I) / 8;   // one slab in uint4
  for (int idx = blockIdx.x * blockDim.x + threadIdx.x; idx < total; idx += gridDim.x * blockDim.x) {
    const int t = idx / cpr;
    const int c = idx - t * cpr;
    const uint4* p = reinterpret_cast<const uint4*>(P + (size_t)t * (size_t)(2 * I)) + 2 * c;
    float g[8], u[8];
    if constexpr (NS > 0) {
      uint4 a[NS], b[NS];
#pragma unroll
      for (int sl = 0; sl < NS; ++sl) {
        a[sl] = p[sl * slab8];
        b[sl] = p[sl * slab8 + 1];
      }
      unpack8(a[0], g);
      unpack8(b[0], u);
#pragma unroll
      for (int sl = 1; sl < NS; ++sl) {
        float g2[8], u2[8];
        unpack8(a[sl], g2);
        unpack8(b[sl], u2);
#pragma unroll
        for (int j = 0; j < 8; ++j) { g[j] += g2[j]; u[j] += u2[j]; }
      }
    } else {
      unpack8(p[0], g);
      unpack8(p[1], u);
      for (int sl = 1; sl < S; ++sl) {
        float g2[8], u2[8];
        unpack8(p[sl * slab8], g2);
        unpack8(p[sl * slab8 + 1], u2);
#pragma unroll
        for (int j = 0; j < 8; ++j) { g[j] += g2[j]; u[j] += u2[j]; }
      }
    }
    float o[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = silu(bf2f(f2bf(g[j]))) * bf2f(f2bf(u[j]));
    reinterpret_cast<uint4*>(out + (size_t)t * I)[c] = pack8(o);
  }
}

template <bool GELU, bool RES>
__global__ __launch_bounds__(256) void bias_act_kernel(const uint16_t* __restrict__ x,
                                                       const uint16_t* __restrict__ bias,
                                                       const uint16_t* __restrict__ res,
                                                       uint16_t* __restrict__ out, int T, int N) {
  const int cpr = N >> 3;
  const int total = T * cpr;
  for (int idx = blockIdx.x * blockDim.x + threadIdx.x; idx < total;
       idx += gridDim.x * blockDim.x) {
    const int c = idx % cpr;
    float v[8], b[8];
    unpack8(reinterpret_cast<const uint4*>(x)[idx], v);
    unpack8(reinterpret_cast<const uint4*>(bias)[c], b);
    if constexpr (RES) {
      float r[8];
      unpack8(reinterpret_cast<const uint4*>(res)[idx], r);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] += r[j];
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = GELU ? gelu_erf(v[j] + b[j]) : v[j] + b[j];
    reinterpret_cast<uint4*>(out)[idx] = pack8(v);
  }
}

static inline int grid_for(size_t work) {
  size_t g = (work + 255) / 256;
  return (int)(g > 2048 ? 2048 : (g == 0 ? 1 : g));
}

int docqa_silu_mul(const void* gu, void* out, int T, int I, int interleaved, hipStream_t s) {
  if (I % 8 != 0 || (long long)T * (I / 8) >= (1LL << 31)) return -1;
  if (T == 0) return 0;
  if (interleaved)
    silu_mul_kernel<true><<<grid_for((size_t)T * (I / 8)), 256, 0, s>>>((const uint16_t*)gu,
                                                                       (uint16_t*)out, T, I);
  else
    silu_mul_kernel<false><<<grid_for((size_t)T * (I / 8)), 256, 0, s>>>((const uint16_t*)gu,
                                                                        (uint16_t*)out, T, I);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_silu_mul_splitk(const float* P, void* out, int S, int T, int I, hipStream_t s) {
  if (I % 8 != 0 || S < 1 || (long long)T * (I / 8) >= (1LL << 31)) return -1;
  if (T == 0) return 0;
  if (!docqa_aligned16(P) || !docqa_aligned16(out)) return -1;
  silu_mul_splitk_kernel<<<grid_for((size_t)T * (I / 8)), 256, 0, s>>>(P, (uint16_t*)out, S, T, I);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_silu_mul_splitk16(const void* P, void* out, int S, int T, int I, hipStream_t s) {
  if (I % 8 != 0 || S < 1 || (long long)T * (I / 8) >= (1LL << 31)) return -1;
  if (T == 0) return 0;
  if (!docqa_aligned16(P) || !docqa_aligned16(out)) return -1;
  const uint16_t* p = (const uint16_t*)P;
  uint16_t* o = (uint16_t*)out;
  const dim3 g = grid_for((size_t)T * (I / 8));
  switch (S) {
    case 2: silu_mul_splitk16_kernel<2><<<g, 256, 0, s>>>(p, o, S, T, I); break;
    case 4: silu_mul_splitk16_kernel<4><<<g, 256, 0, s>>>(p, o, S, T, I); break;
    default: silu_mul_splitk16_kernel<0><<<g, 256, 0, s>>>(p, o, S, T, I); break;
  }
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_bias_act(const void* x, const void* bias, const void* res, void* out, int T, int N,
                   int gelu, hipStream_t s) {
  if (N % 8 != 0 || (long long)T * (N / 8) >= (1LL << 31)) return -1;
  if (T == 0) return 0;
  const int g = grid_for((size_t)T * (N / 8));
  const uint16_t *xp = (const uint16_t*)x, *bp = (const uint16_t*)bias, *rp = (const uint16_t*)res;
  uint16_t* op = (uint16_t*)out;
  if (gelu) {
    if (res) bias_act_kernel<true, true><<<g, 256, 0, s>>>(xp, bp, rp, op, T, N);
    else bias_act_kernel<true, false><<<g, 256, 0, s>>>(xp, bp, rp, op, T, N);
  } else {
    if (res) bias_act_kernel<false, true><<<g, 256, 0, s>>>(xp, bp, rp, op, T, N);
    else bias_act_kernel<false, false><<<g, 256, 0, s>>>(xp, bp, rp, op, T, N);
  }
  DOCQA_CHECK_LAUNCH();
  return 0;
}

// activation of a projection given as S split-K slabs (or its one [n] product), fp32 or
// bf16 in, fp32 or bf16 out: out = act(sum_s P[s])
template <int ACT, int V, typename PT, typename OT>
__global__ __launch_bounds__(256) void slab_activation_kernel(const PT* __restrict__ P, int S, size_t n,
                                                           OT* __restrict__ out) {
  const size_t step = (size_t)gridDim.x * 256 * V;
  for (size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * V; i < n; i += step) {
    float f[V];
    ld_slabs<V>(P + i, S, n, f);
#pragma unroll
    for (int j = 0; j < V; ++j) f[j] = act_f<ACT>(f[j]);
    stv<V>(out + i, f);
  }
}

// cap tanh(x / cap), fp32 out
template <typename T>
__global__ __launch_bounds__(256) void soft_cap_kernel(const T* __restrict__ x, float* __restrict__ out, size_t n,
                                                       float cap) {
  const float inv = 1.f / cap;
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256)
    out[i] = cap * tanhf(ld1(x + i) * inv);
}

// columns [0, n0) and [n0, n0 + n1) of a projection given as S split-K slabs [S, T, ld] (or its
// product), as two matrices of their own: out0 [T, n0], out1 [T, n1] (V | n0, n1, ld)
template <int V, typename PT, typename OT>
__global__ __launch_bounds__(256) void slab_columns_kernel(const PT* __restrict__ P, int S, size_t slab, int T, int ld,
                                                           OT* __restrict__ out0, int n0, OT* __restrict__ out1,
                                                           int n1) {
  const int cpr = (n0 + n1) / V, total = T * cpr;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < total; i += gridDim.x * 256) {
    const int t = i / cpr, c = (i - t * cpr) * V;
    float f[V];
    ld_slabs<V>(P + (size_t)t * ld + c, S, slab, f);
    if (c < n0) stv<V>(out0 + (size_t)t * n0 + c, f);
    else stv<V>(out1 + (size_t)t * n1 + (c - n0), f);
  }
}

template <typename PT, typename OT>
static int launch_slab_columns(const PT* P, int S, int T, int ld, OT* out0, int n0, OT* out1, int n1, hipStream_t s) {
  const long long total = (long long)T * ((n0 + n1) / 4);
  if (total >= (1ll << 31)) return -1;
  const long long g = (total + 255) / 256;
  slab_columns_kernel<4, PT, OT><<<(int)(g < 4096 ? g : 4096), 256, 0, s>>>(P, S, (size_t)T * ld, T, ld, out0, n0, out1, n1);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_slab_columns(const void* P, int p_f32, int S, int T, int ld, void* out0, int n0, void* out1, int n1,
                       int out_f32, hipStream_t s) {
  if (T == 0) return 0;
  if (S < 1 || n0 % 4 || n1 % 4 || ld % 4 || n0 + n1 > ld) return -1;
  if (p_f32)
    return out_f32 ? launch_slab_columns((const float*)P, S, T, ld, (float*)out0, n0, (float*)out1, n1, s)
                   : launch_slab_columns((const float*)P, S, T, ld, (uint16_t*)out0, n0, (uint16_t*)out1, n1, s);
  return out_f32 ? launch_slab_columns((const uint16_t*)P, S, T, ld, (float*)out0, n0, (float*)out1, n1, s)
                 : launch_slab_columns((const uint16_t*)P, S, T, ld, (uint16_t*)out0, n0, (uint16_t*)out1, n1, s);
}

template <int ACT, typename PT, typename OT>
static int launch_activation(const PT* P, int S, size_t n, OT* out, hipStream_t s) {
  if (n % 8 == 0) {
    const size_t g = (n / 8 + 255) / 256;
    slab_activation_kernel<ACT, 8, PT, OT><<<(int)(g < 4096 ? g : 4096), 256, 0, s>>>(P, S, n, out);
  } else {
    const size_t g = (n + 255) / 256;
    slab_activation_kernel<ACT, 1, PT, OT><<<(int)(g < 4096 ? g : 4096), 256, 0, s>>>(P, S, n, out);
  }
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <int ACT>
static int activation_types(const void* P, int p_f32, int S, size_t n, void* out, int out_f32, hipStream_t s) {
  if (p_f32)
    return out_f32 ? launch_activation<ACT>((const float*)P, S, n, (float*)out, s)
                   : launch_activation<ACT>((const float*)P, S, n, (uint16_t*)out, s);
  return out_f32 ? launch_activation<ACT>((const uint16_t*)P, S, n, (float*)out, s)
                 : launch_activation<ACT>((const uint16_t*)P, S, n, (uint16_t*)out, s);
}

int docqa_slab_activation(const void* P, int p_f32, int S, size_t n, int act, void* out, int out_f32, hipStream_t s) {
  if (n == 0) return 0;
  if (S < 1) return -1;
  if (act == ACT_RELU2) return activation_types<ACT_RELU2>(P, p_f32, S, n, out, out_f32, s);
  if (act == ACT_GELU_TANH) return activation_types<ACT_GELU_TANH>(P, p_f32, S, n, out, out_f32, s);
  return -1;
}

int docqa_soft_cap(const void* x, int f32, float* out, size_t n, float cap, hipStream_t s) {
  if (n == 0) return 0;
  const size_t g = (n + 255) / 256;
  const int grid = (int)(g < 8192 ? g : 8192);
  if (f32) soft_cap_kernel<<<grid, 256, 0, s>>>((const float*)x, out, n, cap);
  else soft_cap_kernel<<<grid, 256, 0, s>>>((const uint16_t*)x, out, n, cap);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

// silu(gate) * up of columns [col, col + n) and [col + n, col + 2 n), rows times scale [T]
template <int V, typename PT, typename OT>
__global__ __launch_bounds__(256) void slab_glu_kernel(const PT* __restrict__ P, int S, size_t slab, int ld, int col, int n,
                                                       const float* __restrict__ scale, OT* __restrict__ out, int T) {
  const int per = n / V;
  const size_t total = (size_t)T * per;
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
    const size_t t = i / per;
    const int c = (int)(i - t * per) * V;
    float g[V], u[V];
    docqa::ld_slabs<V>(P + t * ld + col + c, S, slab, g);
    docqa::ld_slabs<V>(P + t * ld + col + n + c, S, slab, u);
    const float s = scale ? scale[t] : 1.f;
#pragma unroll
    for (int j = 0; j < V; ++j) g[j] = g[j] / (1.f + __expf(-g[j])) * u[j] * s;
    docqa::stv<V>(out + t * n + c, g);
  }
}

template <typename PT, typename OT>
static int launch_slab_glu(const PT* P, int S, size_t slab, int ld, int col, int n, const float* scale, OT* out, int T,
                           hipStream_t s) {
  const bool vec = n % 4 == 0 && ld % 4 == 0 && col % 4 == 0;
  const size_t g = ((size_t)T * n / (vec ? 4 : 1) + 255) / 256;
  const int grid = (int)(g < 8192 ? (g ? g : 1) : 8192);
  if (vec) slab_glu_kernel<4, PT, OT><<<grid, 256, 0, s>>>(P, S, slab, ld, col, n, scale, out, T);
  else slab_glu_kernel<1, PT, OT><<<grid, 256, 0, s>>>(P, S, slab, ld, col, n, scale, out, T);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_slab_glu(const void* P, int p_f32, int S, size_t slab, int ld, int col, int n, const float* scale, void* out,
                   int out_f32, int T, hipStream_t s) {
  if (T == 0) return 0;
  if (S < 1 || n < 1 || col < 0 || col + 2 * n > ld) return -1;
  if (p_f32)
    return out_f32 ? launch_slab_glu((const float*)P, S, slab, ld, col, n, scale, (float*)out, T, s)
                   : launch_slab_glu((const float*)P, S, slab, ld, col, n, scale, (uint16_t*)out, T, s);
  return out_f32 ? launch_slab_glu((const uint16_t*)P, S, slab, ld, col, n, scale, (float*)out, T, s)
                 : launch_slab_glu((const uint16_t*)P, S, slab, ld, col, n, scale, (uint16_t*)out, T, s);
}

// PolyNorm of z = P + bias over a row of n: a N(z) + b N(z^2) + c N(z^3) + e with N(v) = v / sqrt(mean(v^2) + eps),
// (a, b, c, e) = act.  One workgroup of NT threads a row, the row in registers
template <int NT, int NV, int V, typename PT, typename OT>
__global__ __launch_bounds__(NT) void poly_norm_kernel(const PT* __restrict__ P, int S, size_t slab, int ld,
                                                       const float* __restrict__ bias, const float* __restrict__ act,
                                                       OT* __restrict__ out, int n, int n_out, float eps) {
  __shared__ float red[3][NT / 64];
  const size_t t = blockIdx.x;
  const int tid = threadIdx.x;
  float z[NV][V], s2 = 0.f, s4 = 0.f, s6 = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (tid + NT * i) * V;
#pragma unroll
    for (int j = 0; j < V; ++j) z[i][j] = 0.f;
    if (c < n) {
      float b[V];
      docqa::ld_slabs<V>(P + t * ld + c, S, slab, z[i]);
      docqa::ldv<V>(bias + c, b);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        z[i][j] += b[j];
        const float q = z[i][j] * z[i][j];
        s2 += q;
        s4 += q * q;
        s6 += q * q * q;
      }
    }
  }
  s2 = wave_sum(s2);
  s4 = wave_sum(s4);
  s6 = wave_sum(s6);
  if ((tid & 63) == 0) {
    red[0][tid >> 6] = s2;
    red[1][tid >> 6] = s4;
    red[2][tid >> 6] = s6;
  }
  __syncthreads();
  s2 = s4 = s6 = 0.f;
#pragma unroll
  for (int w = 0; w < NT / 64; ++w) {
    s2 += red[0][w];
    s4 += red[1][w];
    s6 += red[2][w];
  }
  const float rn = 1.f / (float)n;
  const float a = act[0] / sqrtf(s2 * rn + eps), b = act[1] / sqrtf(s4 * rn + eps), c3 = act[2] / sqrtf(s6 * rn + eps), e = act[3];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (tid + NT * i) * V;
    if (c >= n_out) continue;
    float y[V];
#pragma unroll
    for (int j = 0; j < V; ++j) y[j] = c < n ? z[i][j] * (a + z[i][j] * (b + z[i][j] * c3)) + e : 0.f;
    docqa::stv<V>(out + t * n_out + c, y);
  }
}

template <int NT, int V, typename PT, typename OT>
static int launch_poly_norm(const PT* P, int S, size_t slab, int ld, const float* bias, const float* act, OT* out, int T, int n,
                            int n_out, float eps, hipStream_t s) {
  constexpr int MAX = V == 1 ? 32 : 64 / V;      // most pieces a thread
  const int nv = (n_out / V + NT - 1) / NT;
#define GO(NV)                                                                                                          \
  do {                                                                                                                  \
    constexpr int M = NV < MAX ? NV : MAX;                                                                              \
    poly_norm_kernel<NT, M, V, PT, OT><<<T, NT, 0, s>>>(P, S, slab, ld, bias, act, out, n, n_out, eps);                 \
  } while (0)
  if (nv > MAX) return -1;
  switch (nv) {
    case 1: GO(1); break;
    case 2: GO(2); break;
    case 3: GO(3); break;
    case 4: GO(4); break;
    case 5: GO(5); break;
    case 6: GO(6); break;
    case 7: case 8: GO(8); break;
    default: GO(32);                             // (MAX pieces)
  }
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <typename PT, typename OT>
static int poly_norm_vec(const void* P, int S, size_t slab, int ld, const float* bias, const float* act, void* out, int T, int n,
                         int n_out, float eps, hipStream_t s) {
#define GO(NT, V) return launch_poly_norm<NT, V, PT, OT>((const PT*)P, S, slab, ld, bias, act, (OT*)out, T, n, n_out, eps, s)
  if (n % 4 || n_out % 4 || ld % 4) {
    if (n_out <= 8192) GO(256, 1);
    GO(1024, 1);
  }
  if (n_out <= 4096) GO(256, 4);
  if (n % 8 == 0 && n_out % 8 == 0 && ld % 8 == 0) {
    if (T <= 512 || n_out > 32768) GO(1024, 8);
    GO(512, 8);
  }
  GO(1024, 4);
#undef GO
}

int docqa_poly_norm(const void* P, int p_f32, int S, size_t slab, int ld, const float* bias, const float* act, void* out,
                    int out_f32, int T, int n, int n_out, float eps, hipStream_t s) {
  if (T == 0) return 0;
  if (S < 1 || n < 1 || n > ld || n_out < n) return -1;
#define ARGS P, S, slab, ld, bias, act, out, T, n, n_out, eps, s
  if (p_f32) return out_f32 ? poly_norm_vec<float, float>(ARGS) : poly_norm_vec<float, uint16_t>(ARGS);
  return out_f32 ? poly_norm_vec<uint16_t, float>(ARGS) : poly_norm_vec<uint16_t, uint16_t>(ARGS);
#undef ARGS
}

// heads times their output gate, where no kernel that writes them takes it (docqa_gate.h)
template <int V, typename T>
__global__ __launch_bounds__(256) void head_gate_kernel(const T* __restrict__ x, DocqaGate gate, T* __restrict__ y, int rows, int n) {
  const int m = n / V;
  const size_t total = (size_t)rows * m;
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
    const size_t t = i / m;
    const int c = (int)(i - t * m) * V;
    float f[V];
    docqa::ldv<V>(x + t * n + c, f);
    docqa::apply_gate<V>(gate, t, c, f);
    docqa::stv<V>(y + t * n + c, f);
  }
}

int docqa_head_gate(const void* x, int f32, const DocqaGate& gate, void* y, int T, int n, hipStream_t s) {
  if (T == 0) return 0;
  if (!gate.P || gate.S < 1 || n < 1 || gate.per < 1 || n % gate.per || gate.col < 0 || gate.col + n / gate.per > gate.ld) return -1;
  const bool vec = n % 4 == 0 && docqa_gate_vec(gate, 4);
  const size_t g = ((size_t)T * (n / (vec ? 4 : 1)) + 255) / 256;
  const int grid = (int)(g < 8192 ? g : 8192);
  if (f32) {
    if (vec) head_gate_kernel<4, float><<<grid, 256, 0, s>>>((const float*)x, gate, (float*)y, T, n);
    else head_gate_kernel<1, float><<<grid, 256, 0, s>>>((const float*)x, gate, (float*)y, T, n);
  } else {
    if (vec) head_gate_kernel<4, uint16_t><<<grid, 256, 0, s>>>((const uint16_t*)x, gate, (uint16_t*)y, T, n);
    else head_gate_kernel<1, uint16_t><<<grid, 256, 0, s>>>((const uint16_t*)x, gate, (uint16_t*)y, T, n);
  }
  DOCQA_CHECK_LAUNCH();
  return 0;
}
