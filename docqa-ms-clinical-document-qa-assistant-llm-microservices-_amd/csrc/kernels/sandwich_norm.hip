// sandwich_norm.hip -- norms of decoders that keep the residual stream in fp32 and normalise
// both a sublayer's input and its output:
//   x <- x + rms(y) * w_post (+ add);   h = rms(x) * w_next
// One launch between two projections does all of it: it sums the split-K slabs of the
// sublayer's last projection, normalises that output, updates the fp32 residual, and emits
// the next projection's input in the compute dtype.  One 256-thread workgroup per row; each
// thread keeps its elements of x in registers between the two reductions, so the residual is
// read and written once.
#include "docqa_common.h"
#include "docqa_elem.h"

using namespace docqa;

namespace {
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

template <int NV, int V, typename PT, typename OT>
__global__ __launch_bounds__(256) void sandwich_rmsnorm_kernel(const PT* __restrict__ P, int S, size_t slab,
                                                               float* __restrict__ res,
                                                               const float* __restrict__ w_post,
                                                               const float* __restrict__ add,
                                                               const float* __restrict__ w_next,
                                                               OT* __restrict__ out, int H, float eps) {
  __shared__ float red[2][4];
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x, n = H / V;
  float y[NV][V], x[NV][V];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + 256 * i;
    if (c < n) {
      ld_slabs<V>(P + row * H + c * V, S, slab, y[i]);
      ldv<V>(res + row * H + c * V, x[i]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += y[i][j] * y[i][j];
    }
  }
  const float iy = 1.f / sqrtf(block_sum(ss, red[0]) / (float)H + eps);
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + 256 * i;
    if (c < n) {
      float g[V], a[V];
      ldv<V>(w_post + c * V, g);
      if (add) ldv<V>(add + row * H + c * V, a);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        x[i][j] += y[i][j] * iy * g[j];
        if (add) x[i][j] += a[j];
        ss += x[i][j] * x[i][j];
      }
      stv<V>(res + row * H + c * V, x[i]);
    }
  }
  const float ix = 1.f / sqrtf(block_sum(ss, red[1]) / (float)H + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + 256 * i;
    if (c < n) {
      float g[V], o[V];
      ldv<V>(w_next + c * V, g);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = x[i][j] * ix * g[j];
      stv<V>(out + row * H + c * V, o);
    }
  }
}

// h = table[id] * scale (fp32 residual, and a second copy when ``emb``), out = rms(h) * w
template <int NV, int V, typename T>
__global__ __launch_bounds__(256) void embed_scale_rmsnorm_kernel(const int* __restrict__ ids,
                                                                  const T* __restrict__ table, float scale,
                                                                  const float* __restrict__ w,
                                                                  float* __restrict__ res, float* __restrict__ emb,
                                                                  T* __restrict__ out, int H, int vocab, float eps) {
  __shared__ float red[4];
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x, n = H / V;
  const int id = min(max(ids[row], 0), vocab - 1);
  float x[NV][V];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + 256 * i;
    if (c < n) {
      ldv<V>(table + (size_t)id * H + c * V, x[i]);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        x[i][j] *= scale;
        ss += x[i][j] * x[i][j];
      }
      stv<V>(res + row * H + c * V, x[i]);
      if (emb) stv<V>(emb + row * H + c * V, x[i]);
    }
  }
  const float ix = 1.f / sqrtf(block_sum(ss, red) / (float)H + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + 256 * i;
    if (c < n) {
      float g[V], o[V];
      ldv<V>(w + c * V, g);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = x[i][j] * ix * g[j];
      stv<V>(out + row * H + c * V, o);
    }
  }
}

// res += m (P + Q) of two projections (Q null: one), each a product or split-K slabs, and a copy
// in the compute dtype: the stream update between sublayers without a norm of their own
template <int V, typename PT, typename QT>
__global__ __launch_bounds__(256) void add_scaled_kernel(const PT* __restrict__ P, int SP, const QT* __restrict__ Q,
                                                         int SQ, float* __restrict__ res, float m,
                                                         uint16_t* __restrict__ out, size_t n) {
  const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= n) return;
  float x[V], y[V];
  ldv<V>(res + i, x);
  ld_slabs<V>(P + i, SP, n, y);
  if (Q) {
    float z[V];
    ld_slabs<V>(Q + i, SQ, n, z);
#pragma unroll
    for (int j = 0; j < V; ++j) y[j] += z[j];
  }
#pragma unroll
  for (int j = 0; j < V; ++j) x[j] += m * y[j];
  stv<V>(res + i, x);
  if (out) stv<V>(out + i, x);
}

template <typename PT, typename QT>
int launch_add_scaled(const void* P, int SP, const void* Q, int SQ, float* res, float m, void* out, size_t n,
                      hipStream_t s) {
  if (n % 4 == 0)
    add_scaled_kernel<4, PT, QT><<<(unsigned)((n / 4 + 255) / 256), 256, 0, s>>>((const PT*)P, SP, (const QT*)Q, SQ, res,
                                                                                 m, (uint16_t*)out, n);
  else
    add_scaled_kernel<1, PT, QT><<<(unsigned)((n + 255) / 256), 256, 0, s>>>((const PT*)P, SP, (const QT*)Q, SQ, res, m,
                                                                             (uint16_t*)out, n);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <int V, typename PT, typename OT>
int launch_sandwich(const PT* P, int S, float* res, const float* w_post, const float* add, const float* w_next,
                    OT* out, int rows, int H, float eps, hipStream_t s) {
  const size_t slab = (size_t)rows * H;
  const int nv = (H / V + 255) / 256;
#define GO(N) sandwich_rmsnorm_kernel<N, V, PT, OT><<<rows, 256, 0, s>>>(P, S, slab, res, w_post, add, w_next, out, H, eps)
  if (nv <= 1) GO(1);
  else if (nv <= 2) GO(2);
  else if (nv <= 4) GO(4);
  else if (nv <= 8) GO(8);
  else if (nv <= 16) GO(16);
  else return -1;
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <typename PT>
int sandwich_out(const PT* P, int S, float* res, const float* w_post, const float* add, const float* w_next,
                 void* out, int out_f32, int rows, int H, float eps, hipStream_t s) {
  if (out_f32)
    return H % 4 == 0 ? launch_sandwich<4>(P, S, res, w_post, add, w_next, (float*)out, rows, H, eps, s)
                      : launch_sandwich<1>(P, S, res, w_post, add, w_next, (float*)out, rows, H, eps, s);
  return H % 4 == 0 ? launch_sandwich<4>(P, S, res, w_post, add, w_next, (uint16_t*)out, rows, H, eps, s)
                    : launch_sandwich<1>(P, S, res, w_post, add, w_next, (uint16_t*)out, rows, H, eps, s);
}

template <int V, typename T>
int launch_embed(const int* ids, const T* table, float scale, const float* w, float* res, float* emb, T* out,
                 int rows, int H, int vocab, float eps, hipStream_t s) {
  const int nv = (H / V + 255) / 256;
#define GO(N) embed_scale_rmsnorm_kernel<N, V, T><<<rows, 256, 0, s>>>(ids, table, scale, w, res, emb, out, H, vocab, eps)
  if (nv <= 1) GO(1);
  else if (nv <= 2) GO(2);
  else if (nv <= 4) GO(4);
  else if (nv <= 8) GO(8);
  else if (nv <= 16) GO(16);
  else return -1;
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}
}  // namespace

int docqa_sandwich_rmsnorm(const void* P, int p_f32, int S, float* res, const float* w_post, const float* add,
                           const float* w_next, void* out, int out_f32, int rows, int H, float eps, hipStream_t s) {
  if (rows == 0) return 0;
  if (S < 1 || H < 1) return -1;
  return p_f32 ? sandwich_out((const float*)P, S, res, w_post, add, w_next, out, out_f32, rows, H, eps, s)
               : sandwich_out((const uint16_t*)P, S, res, w_post, add, w_next, out, out_f32, rows, H, eps, s);
}

int docqa_embed_scale_rmsnorm(const int* ids, const void* table, int f32, float scale, const float* w, float* res,
                              float* emb, void* out, int rows, int H, int vocab, float eps, hipStream_t s) {
  if (rows == 0) return 0;
  if (f32)
    return H % 4 == 0 ? launch_embed<4>(ids, (const float*)table, scale, w, res, emb, (float*)out, rows, H, vocab, eps, s)
                      : launch_embed<1>(ids, (const float*)table, scale, w, res, emb, (float*)out, rows, H, vocab, eps, s);
  return H % 4 == 0
             ? launch_embed<4>(ids, (const uint16_t*)table, scale, w, res, emb, (uint16_t*)out, rows, H, vocab, eps, s)
             : launch_embed<1>(ids, (const uint16_t*)table, scale, w, res, emb, (uint16_t*)out, rows, H, vocab, eps, s);
}

int docqa_add_scaled(const void* P, int p_f32, int SP, const void* Q, int q_f32, int SQ, float* res, float m, void* out,
                     size_t n, hipStream_t s) {
  if (n == 0) return 0;
  if (SP < 1 || (Q && SQ < 1) || n >= ((size_t)1 << 38)) return -1;
  if (p_f32)
    return q_f32 ? launch_add_scaled<float, float>(P, SP, Q, SQ, res, m, out, n, s)
                 : launch_add_scaled<float, uint16_t>(P, SP, Q, SQ, res, m, out, n, s);
  return q_f32 ? launch_add_scaled<uint16_t, float>(P, SP, Q, SQ, res, m, out, n, s)
               : launch_add_scaled<uint16_t, uint16_t>(P, SP, Q, SQ, res, m, out, n, s);
}
