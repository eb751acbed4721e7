// attn_window.hip -- causal attention over a sliding window with an optional per-head sink,
// read from the paged cache; head-wise query / key RMS norm; keys shared as values.
//
//   s_j = scale * k_scale_j * (q . K_j)   for  pos - window < j <= pos
//   out = sum_j exp(s_j) V_j / (sum_j exp(s_j) + exp(sink_h))
//
// * qk_norm_store: q <- rms(q) * w over each head, K rows stored as projected with their
//   inverse root mean square beside them (k_scale).  With the key norm's weight folded into
//   w the normalised key is never materialised: one cached row serves as key and as value,
//   half the bytes of a K / V pair.
// * window <= 0: no window; sink null: none; k_scale null: 1; V may be the K cache itself.
// * prefill (several query tokens a sequence) and decode (one) share the kernels.
#include "docqa_common.h"
#include "docqa_elem.h"
#include <float.h>

using namespace docqa;

namespace {
constexpr float kLog2e = 1.4426950408889634f;

// one wave per (token, head); heads [0, H) are queries, [H, H + G) keys
template <int V, int NI, typename PT, typename T>
__global__ __launch_bounds__(256) void qk_norm_store_kernel(const PT* __restrict__ P, int S, size_t slab, int ld,
                                                            const float* __restrict__ wq,
                                                            const int* __restrict__ slot_mapping, T* __restrict__ q,
                                                            T* __restrict__ kc, float* __restrict__ ks, int tokens,
                                                            int H, int G, int D, int BS, float eps) {
  const int u = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int t = u / (H + G), h = u % (H + G);
  if (t >= tokens) return;
  const PT* p = P + (size_t)t * ld + (size_t)h * D;
  float x[NI][V];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (lane + 64 * i) * V;
    if (c < D) {
      ld_slabs<V>(p + c, S, slab, x[i]);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        if (h >= H) x[i][j] = rnd((const T*)nullptr, x[i][j]);   // the scale belongs to the stored row
        ss += x[i][j] * x[i][j];
      }
    }
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / (float)D + eps);
  if (h < H) {
    T* o = q + ((size_t)t * H + h) * D;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (lane + 64 * i) * V;
      if (c < D) {
        float w[V];
        ldv<V>(wq + c, w);
#pragma unroll
        for (int j = 0; j < V; ++j) x[i][j] *= inv * w[j];
        stv<V>(o + c, x[i]);
      }
    }
  } else {
    const int slot = slot_mapping[t];
    if (slot < 0) return;
    const size_t row = ((size_t)(slot / BS) * G + (h - H)) * BS + slot % BS;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (lane + 64 * i) * V;
      if (c < D) stv<V>(kc + row * D + c, x[i]);
    }
    if (lane == 0) ks[row] = inv;
  }
}

struct WindowArgs {
  const int* block_tables;
  int maxb;
  const int* cu;          // [B + 1] query offsets; null: one query token per sequence (decode)
  const int* ctx;         // prefill: first position of each sequence's query tokens; decode:
                          // context length including the new token
  const float* k_scale;   // [blocks, G, BS] or null
  const float* sink;      // [H] or null
  int H, G, D, BS;
  float scale;
  int window;
};

// LDS written by some lanes of a wave and read by others: in order in hardware, so only the
// compiler has to be held back
__device__ __forceinline__ void wave_lds_sync() { asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); }

// tokens [q0, q0 + L) of sequence b and the position of the first
__device__ __forceinline__ bool seq_range(const WindowArgs& a, int b, int& q0, int& L, int& p0) {
  if (a.cu) {
    q0 = a.cu[b];
    L = a.cu[b + 1] - q0;
    p0 = a.ctx[b];
  } else {
    q0 = b;
    L = 1;
    p0 = a.ctx[b] - 1;
  }
  return L > 0 && p0 >= 0;
}

// Any head size and element type: one wave per (token, head).  64 keys at a time, one per
// lane for the scores, then the lanes run over the value's elements.
template <typename T, int NI>
__global__ __launch_bounds__(256) void window_attn_kernel(const T* __restrict__ q, const T* __restrict__ kc,
                                                          const T* __restrict__ vc, T* __restrict__ out,
                                                          WindowArgs a) {
  __shared__ float sq[4][512];
  __shared__ float sp[4][64];
  __shared__ int srow[4][64];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int b = blockIdx.y, u = blockIdx.x * 4 + wave;
  const int tok = u / a.H, h = u % a.H;
  int q0 = 0, L = 0, p0 = 0;
  const bool live = seq_range(a, b, q0, L, p0);
  if (tok >= (a.cu ? L : 1)) return;       // whole waves; no workgroup barrier below
  const int D = a.D;
  T* o = out + ((size_t)(q0 + tok) * a.H + h) * D;
  if (!live) {                             // a padded decode row
    for (int c = lane; c < D; c += 64) st1(o + c, 0.f);
    return;
  }
  const int g = h / (a.H / a.G), pos = p0 + tok;
  const T* qp = q + ((size_t)(q0 + tok) * a.H + h) * D;
  for (int c = lane; c < D; c += 64) sq[wave][c] = ld1(qp + c);
  wave_lds_sync();
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  float m = a.sink ? a.sink[h] * kLog2e : -INFINITY, l = a.sink ? 1.f : 0.f;
  float acc[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) acc[i] = 0.f;
  const float sl2 = a.scale * kLog2e;
  for (int k0 = lo; k0 <= pos; k0 += 64) {
    const int key = k0 + lane;
    float s = -INFINITY;
    int row = 0;
    if (key <= pos) {
      const int blk = a.block_tables[(size_t)b * a.maxb + key / a.BS];
      row = (blk * a.G + g) * a.BS + key % a.BS;
      const T* kp = kc + (size_t)row * D;
      float d0 = 0.f, d1 = 0.f;
      int c = 0;
      if (D % 8 == 0) {
        for (; c < D; c += 8) {
          float f[8];
          ldv<8>(kp + c, f);
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            d0 += f[j] * sq[wave][c + j];
            d1 += f[4 + j] * sq[wave][c + 4 + j];
          }
        }
      } else {
        for (; c < D; ++c) d0 += ld1(kp + c) * sq[wave][c];
      }
      s = (d0 + d1) * sl2 * (a.k_scale ? a.k_scale[row] : 1.f);
    }
    const float mn = fmaxf(m, wave_max(s));
    const float alpha = exp2f(m - mn);
    const float p = key <= pos ? exp2f(s - mn) : 0.f;
    l = l * alpha + wave_sum(p);
    m = mn;
    sp[wave][lane] = p;
    srow[wave][lane] = row;
    wave_lds_sync();
    const int n = min(64, pos - k0 + 1);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = lane + 64 * i;
      if (c < D) {
        float v = acc[i] * alpha;
        for (int j = 0; j < n; ++j) v += sp[wave][j] * ld1(vc + (size_t)srow[wave][j] * D + c);
        acc[i] = v;
      }
    }
    wave_lds_sync();
  }
  const float inv = 1.f / l;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = lane + 64 * i;
    if (c < D) st1(o + c, acc[i] * inv);
  }
}

template <typename PT, typename T>
int qk_store(const PT* P, int S, size_t slab, int ld, const float* wq, const int* sm, T* q, T* kc, float* ks,
             int tokens, int H, int G, int D, int BS, float eps, hipStream_t s) {
  const int grid = (int)(((long long)tokens * (H + G) + 3) / 4);
#define GO(V, N) qk_norm_store_kernel<V, N, PT, T><<<grid, 256, 0, s>>>(P, S, slab, ld, wq, sm, q, kc, ks, tokens, H, G, D, BS, eps)
  if (D % 2 == 0 && ld % 2 == 0) {
    if (D <= 128) GO(2, 1);
    else if (D <= 256) GO(2, 2);
    else GO(2, 4);
  } else {
    if (D <= 64) GO(1, 1);
    else if (D <= 128) GO(1, 2);
    else GO(1, 8);
  }
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}
}  // namespace

int docqa_qk_norm_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* wq, const int* slots,
                        void* q, void* kc, float* ks, int f32, int tokens, int H, int G, int D, int BS, float eps,
                        hipStream_t s) {
  if (tokens == 0) return 0;
  if (S < 1 || D < 1 || D > 512 || H < 1 || G < 1 || ld < (H + G) * D) return -1;
  if (f32) {
    if (!p_f32) return -1;
    return qk_store((const float*)P, S, slab, ld, wq, slots, (float*)q, (float*)kc, ks, tokens, H, G, D, BS, eps, s);
  }
  if (p_f32)
    return qk_store((const float*)P, S, slab, ld, wq, slots, (uint16_t*)q, (uint16_t*)kc, ks, tokens, H, G, D, BS, eps, s);
  return qk_store((const uint16_t*)P, S, slab, ld, wq, slots, (uint16_t*)q, (uint16_t*)kc, ks, tokens, H, G, D, BS, eps, s);
}

int docqa_window_attn(const void* q, const void* kc, const void* vc, const float* k_scale, const int* block_tables,
                      int maxb, const int* cu, const int* ctx, const float* sink, void* out, int f32, int B,
                      int max_q, int H, int G, int D, int BS, float scale, int window, hipStream_t s) {
  if (B == 0 || max_q == 0) return 0;
  if (H % G != 0 || D < 1 || D > 512 || (BS & (BS - 1)) != 0) return -1;
  const WindowArgs a{block_tables, maxb, cu, ctx, k_scale, sink, H, G, D, BS, scale, window};
  dim3 grid((max_q * H + 3) / 4, B);
#define GO(T, N) window_attn_kernel<T, N><<<grid, 256, 0, s>>>((const T*)q, (const T*)kc, (const T*)vc, (T*)out, a)
  if (f32) {
    if (D <= 64) GO(float, 1);
    else if (D <= 128) GO(float, 2);
    else if (D <= 256) GO(float, 4);
    else GO(float, 8);
  } else {
    if (D <= 64) GO(uint16_t, 1);
    else if (D <= 128) GO(uint16_t, 2);
    else if (D <= 256) GO(uint16_t, 4);
    else GO(uint16_t, 8);
  }
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}
