// sandwich_norm.hip -- norms of decoders that keep the residual stream in fp32 and normalise
// both a sublayer's input and its output:
//   x <- x + rms(y) * w_post (+ add);   h = rms(x) * w_next
// One launch between two projections does all of it: it sums the split-K slabs of the
// sublayer's last projection, normalises that output, updates the fp32 residual, and emits
// the next projection's input in the compute dtype.  One 256-thread workgroup per row; each
// thread keeps its elements of x in registers between the two reductions, so the residual is
// read and written once.
//
// post_norm: norms after the sum, over equal parts of the row, behind a gated residual:
//   x <- groupnorm(alpha x + sigmoid(gate + b) * y) * w
// scaled_rmsnorm: a norm ahead of every sublayer alone, results scaled per channel, y a product with
// its bias or the weighted sum of the chosen experts' outputs:
//   x <- x + scale * y;   h = rms(x) * w_next
#include "docqa_common.h"
#include "docqa_elem.h"
#include "docqa_hybrid.h"
#include <type_traits>

using namespace docqa;

namespace {
// over a workgroup of NT threads
template <int NT = 256>
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) s += red[i];
  return s;
}

// one new token a row, an input convolution behind the norm: out2 = h + conv(h), the identity in
// w's last tap; state holds the last taps - 1 rows h of each slot (slot -1: none, position 0: zeros)
template <typename OT>
struct ConvArgs {
  const float* w;         // [taps, H]
  int taps;
  OT* state;              // [slots, taps - 1, H]
  const int* slots;
  const int* positions;
  OT* out2;
};

// CONV: 0 none, taps of 2 to 4 with the state's rows loaded ahead of the reductions, -1 any taps
// NT threads a row: 256, or 1024 where rows are few and wide
template <int NT, int NV, int V, typename PT, typename OT, int CONV = 0>
__global__ __launch_bounds__(NT) void sandwich_rmsnorm_kernel(const PT* __restrict__ P, int S, size_t slab,
                                                               float* __restrict__ res,
                                                               const float* __restrict__ w_post,
                                                               const float* __restrict__ add,
                                                               const float* __restrict__ w_next,
                                                               OT* __restrict__ out, int H, float eps,
                                                               ConvArgs<OT> cv) {
  __shared__ float red[2][NT / 64];
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x, n = H / V;
  float y[NV][V], x[NV][V];
  constexpr int NS = CONV > 0 ? CONV - 1 : 1;
  float st[CONV > 0 ? NV : 1][NS][V];                    // the slot's rows (zeros at position 0)
  if constexpr (CONV > 0) {
    const int slot = cv.slots[row];
    const bool carry = slot >= 0 && cv.positions[row] > 0;
    const OT* sp = cv.state + (size_t)max(slot, 0) * NS * H;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int k = 0; k < NS; ++k) {
        const int c = min(tid + NT * i, n - 1);
        ldv<V>(sp + (size_t)k * H + c * V, st[i][k]);
#pragma unroll
        for (int j = 0; j < V; ++j) st[i][k][j] = carry ? st[i][k][j] : 0.f;
      }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + NT * i;
    if (c < n) {
      ld_slabs<V>(P + row * H + c * V, S, slab, y[i]);
      ldv<V>(res + row * H + c * V, x[i]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += y[i][j] * y[i][j];
    }
  }
  const float iy = 1.f / sqrtf(block_sum<NT>(ss, red[0]) / (float)H + eps);
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + NT * i;
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
  const float ix = 1.f / sqrtf(block_sum<NT>(ss, red[1]) / (float)H + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + NT * i;
    if (c < n) {
      float g[V], o[V];
      ldv<V>(w_next + c * V, g);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = x[i][j] * ix * g[j];
      stv<V>(out + row * H + c * V, o);
      if constexpr (CONV > 0) {
        float s[V], wk[V];
        ldv<V>(cv.w + (size_t)NS * H + c * V, wk);
#pragma unroll
        for (int j = 0; j < V; ++j) {
          o[j] = rnd((const OT*)nullptr, o[j]);
          s[j] = wk[j] * o[j];
        }
        const int slot = cv.slots[row];
#pragma unroll
        for (int k = 0; k < NS; ++k) {
          ldv<V>(cv.w + (size_t)k * H + c * V, wk);
#pragma unroll
          for (int j = 0; j < V; ++j) s[j] += wk[j] * st[i][k][j];
          if (slot >= 0)
            stv<V>(cv.state + ((size_t)slot * NS + k) * H + c * V, k + 1 < NS ? st[i][k + 1 < NS ? k + 1 : 0] : o);
        }
        stv<V>(cv.out2 + row * H + c * V, s);
      } else if constexpr (CONV < 0) {
        const int slot = cv.slots[row], last = cv.taps - 1;
        const bool carry = slot >= 0 && cv.positions[row] > 0;
        OT* st = cv.state + (size_t)max(slot, 0) * last * H + c * V;
        float s[V], wk[V];
        ldv<V>(cv.w + (size_t)last * H + c * V, wk);
#pragma unroll
        for (int j = 0; j < V; ++j) {
          o[j] = rnd((const OT*)nullptr, o[j]);
          s[j] = wk[j] * o[j];
        }
        for (int k = 0; k < last; ++k) {               // row k <- row k + 1, the last <- h
          float f[V], nx[V];
#pragma unroll
          for (int j = 0; j < V; ++j) f[j] = 0.f, nx[j] = k + 1 == last ? o[j] : 0.f;
          if (carry) {
            ldv<V>(st + (size_t)k * H, f);
            if (k + 1 < last) ldv<V>(st + (size_t)(k + 1) * H, nx);
          }
          ldv<V>(cv.w + (size_t)k * H + c * V, wk);
#pragma unroll
          for (int j = 0; j < V; ++j) s[j] += wk[j] * f[j];
          if (slot >= 0) stv<V>(st + (size_t)k * H, nx);
        }
        stv<V>(cv.out2 + row * H + c * V, s);
      }
    }
  }
}

// h = table[id] * scale (fp32 residual, and a second copy when ``emb``), out = rms(h) * w (w null: h)
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
  const float ix = w ? 1.f / sqrtf(block_sum(ss, red) / (float)H + eps) : 1.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + 256 * i;
    if (c < n) {
      float g[V], o[V];
#pragma unroll
      for (int j = 0; j < V; ++j) g[j] = 1.f;
      if (w) ldv<V>(w + c * V, g);
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
                    OT* out, int rows, int H, float eps, const std::common_type_t<ConvArgs<OT>>* cv, hipStream_t s) {
  const size_t slab = (size_t)rows * H;
  const int nv = (H / V + 255) / 256;
  const ConvArgs<OT> none{};
#define LAUNCH(N, C)                                                                                                   \
  do {                                                                                                                 \
    if (V > 1 && rows <= 512 && N >= 4) {                                                                              \
      constexpr int NW = N >= 4 ? N / 4 : 1;                                                                           \
      sandwich_rmsnorm_kernel<1024, NW, V, PT, OT, (C)><<<rows, 1024, 0, s>>>(P, S, slab, res, w_post, add, w_next,    \
                                                                              out, H, eps, cv ? *cv : none);           \
    } else {                                                                                                           \
      sandwich_rmsnorm_kernel<256, N, V, PT, OT, (C)><<<rows, 256, 0, s>>>(P, S, slab, res, w_post, add, w_next, out,  \
                                                                           H, eps, cv ? *cv : none);                   \
    }                                                                                                                  \
  } while (0)
#define GO(N)                                                      \
  do {                                                             \
    const int taps = cv ? cv->taps : 0;                            \
    if (!cv) LAUNCH(N, 0);                                         \
    else if (V > 1 && N <= 8 && taps == 2) LAUNCH(N, V > 1 && N <= 8 ? 2 : -1); \
    else if (V > 1 && N <= 8 && taps == 3) LAUNCH(N, V > 1 && N <= 8 ? 3 : -1); \
    else if (V > 1 && N <= 8 && taps == 4) LAUNCH(N, V > 1 && N <= 8 ? 4 : -1); \
    else LAUNCH(N, -1);                                            \
  } while (0)
  if (nv <= 1) GO(1);
  else if (nv <= 2) GO(2);
  else if (nv <= 4) GO(4);
  else if (nv <= 8) GO(8);
  else if (nv <= 16) GO(16);
  else return -1;
#undef GO
#undef LAUNCH
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <typename PT>
int sandwich_out(const PT* P, int S, float* res, const float* w_post, const float* add, const float* w_next,
                 void* out, int out_f32, int rows, int H, float eps, hipStream_t s) {
  if (out_f32)
    return H % 4 == 0 ? launch_sandwich<4>(P, S, res, w_post, add, w_next, (float*)out, rows, H, eps, nullptr, s)
                      : launch_sandwich<1>(P, S, res, w_post, add, w_next, (float*)out, rows, H, eps, nullptr, s);
  return H % 4 == 0 ? launch_sandwich<4>(P, S, res, w_post, add, w_next, (uint16_t*)out, rows, H, eps, nullptr, s)
                    : launch_sandwich<1>(P, S, res, w_post, add, w_next, (uint16_t*)out, rows, H, eps, nullptr, s);
}

template <typename PT, typename OT>
int sandwich_conv(const PT* P, int S, float* res, const float* w_post, const float* w_next, const float* cw, int taps,
                  void* state, const int* slots, const int* positions, void* out, void* out2, int rows, int H, float eps,
                  hipStream_t s) {
  const ConvArgs<OT> cv{cw, taps, (OT*)state, slots, positions, (OT*)out2};
  return H % 4 == 0 ? launch_sandwich<4>(P, S, res, w_post, (const float*)nullptr, w_next, (OT*)out, rows, H, eps, &cv, s)
                    : launch_sandwich<1>(P, S, res, w_post, (const float*)nullptr, w_next, (OT*)out, rows, H, eps, &cv, s);
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
template <int V>
__device__ __forceinline__ void ld_any(const void* p, int f32, int S, size_t slab, size_t off, float* f) {
  if (f32) ld_slabs<V>((const float*)p + off, S, slab, f);
  else ld_slabs<V>((const uint16_t*)p + off, S, slab, f);
}

// one workgroup of NT threads a row, V consecutive elements of NV pieces a thread.  A piece lies in one
// group; where groups are whole multiples of a wave's piece (GW) the wave's sum is one LDS word, else
// every piece's is, and a wave sums each group's.  Sums are in a fixed order either way.
template <int NT, int NV, int V, bool GW>
__global__ __launch_bounds__(NT) void post_norm_kernel(DocqaPostNorm a) {
  extern __shared__ float part[];                       // GW: [NV * NT / 64], else [W / V + groups]
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x, W = a.W, n = W / V, gn = n / a.groups;      // pieces of a row, of a group
  const size_t pslab = (size_t)a.rows * W;
  float x[NV][V];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + NT * i;
    float ss = 0.f;
    if (c < n) {
      ldv<V>(a.res + row * W + c * V, x[i]);
#pragma unroll
      for (int j = 0; j < V; ++j) x[i][j] *= a.alpha;
      if (a.P) {
        float y[V], g[V], b[V];
        ld_any<V>(a.P, a.pf32, a.SP, pslab, row * W + c * V, y);
        ld_any<V>(a.gate, a.gf32, a.SG, a.gslab, row * a.ldg + a.col + c * V, g);
        ldv<V>(a.gb + c * V, b);
        if (a.Q) {
          float z[V];
          ld_any<V>(a.Q, a.qf32, a.SQ, pslab, row * W + c * V, z);
#pragma unroll
          for (int j = 0; j < V; ++j) y[j] += z[j];
        }
#pragma unroll
        for (int j = 0; j < V; ++j) x[i][j] += y[j] / (1.f + __expf(-(g[j] + b[j])));
      }
#pragma unroll
      for (int j = 0; j < V; ++j) ss += x[i][j] * x[i][j];
      if constexpr (!GW) part[c] = ss;
    }
    if constexpr (GW) {
      ss = wave_sum(ss);
      if ((tid & 63) == 0) part[i * (NT / 64) + (tid >> 6)] = ss;
    }
  }
  __syncthreads();
  if constexpr (!GW) {
    for (int g = tid >> 6; g < a.groups; g += NT / 64) {
      float s = 0.f;
      for (int e = tid & 63; e < gn; e += 64) s += part[g * gn + e];
      s = wave_sum(s);
      if ((tid & 63) == 0) part[n + g] = s;
    }
    __syncthreads();
  }
  const float rg = 1.f / ((float)gn * V);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + NT * i;
    if (c >= n) continue;
    float s = 0.f;
    const int g = c / gn;
    if constexpr (GW) {
      const int m = gn / 64;                            // waves' pieces of the group
      for (int e = 0; e < m; ++e) s += part[g * m + e];
    } else {
      s = part[n + g];
    }
    const float inv = 1.f / sqrtf(s * rg + a.eps);
    float w[V];
    ldv<V>(a.w + c * V, w);
#pragma unroll
    for (int j = 0; j < V; ++j) x[i][j] *= inv * w[j];
    stv<V>(a.res + row * W + c * V, x[i]);
    if (a.out) stv<V>((uint16_t*)a.out + row * W + c * V, x[i]);
  }
}

// one workgroup of NT threads a row, V consecutive elements of NV pieces a thread.  MIX: P (of type PT, as x)
// holds the chosen experts' outputs
template <int NT, int NV, int V, typename PT, bool MIX>
__global__ __launch_bounds__(NT) void scaled_rmsnorm_kernel(DocqaScaledNorm a) {
  __shared__ float red[NT / 64];
  const size_t row = blockIdx.x, slab = (size_t)a.rows * a.W;
  const int tid = threadIdx.x, W = a.W, n = W / V;
  const PT *P = (const PT*)a.P + row * W, *xr = (const PT*)a.x + row * W;
  float x[NV][V], y[NV][V];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = min(tid + NT * i, n - 1);
    ldv<V>(a.res + row * W + c * V, x[i]);
    if constexpr (!MIX) ld_slabs<V>(P + c * V, a.SP, slab, y[i]);
  }
  if constexpr (MIX) {
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int j = 0; j < V; ++j) y[i][j] = 0.f;
    for (int k0 = 0; k0 < a.SP; k0 += 4) {               // four at a time: past the last, weight 0
      const PT* p[4];
      float w[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int k = min(k0 + u, a.SP - 1);
        p[u] = a.ids[row * a.SP + k] < a.experts ? P + k * slab : xr;
        w[u] = k0 + u < a.SP ? a.wts[row * a.SP + k] : 0.f;
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = min(tid + NT * i, n - 1);
        float f[4][V];
#pragma unroll
        for (int u = 0; u < 4; ++u) ldv<V>(p[u] + c * V, f[u]);
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int j = 0; j < V; ++j) y[i][j] += w[u] * f[u][j];
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + NT * i;
    if (c < n) {
      float g[V], b[V];
      ldv<V>(a.scale + c * V, g);
#pragma unroll
      for (int j = 0; j < V; ++j) b[j] = 0.f;
      if (a.bias) ldv<V>(a.bias + c * V, b);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        x[i][j] += g[j] * (y[i][j] + b[j]);
        ss += x[i][j] * x[i][j];
      }
      stv<V>(a.res + row * W + c * V, x[i]);
    }
  }
  const float inv = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)W + a.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + NT * i;
    if (c < n) {
      float g[V];
      ldv<V>(a.w + c * V, g);
#pragma unroll
      for (int j = 0; j < V; ++j) g[j] *= x[i][j] * inv;
      if (a.of32) stv<V>((float*)a.out + row * W + c * V, g);
      else stv<V>((uint16_t*)a.out + row * W + c * V, g);
    }
  }
}

template <int V, typename PT, bool MIX>
int launch_scaled(const DocqaScaledNorm& a, hipStream_t s) {
  const int nv = (a.W / V + 255) / 256;
#define GO(NV)                                                                                                  \
  do {                                                                                                          \
    if (V > 1 && NV >= 4 && a.rows <= 512)                                                                      \
      scaled_rmsnorm_kernel<1024, (NV >= 4 ? NV / 4 : 1), V, PT, MIX><<<a.rows, 1024, 0, s>>>(a);               \
    else                                                                                                        \
      scaled_rmsnorm_kernel<256, NV, V, PT, MIX><<<a.rows, 256, 0, s>>>(a);                                     \
  } while (0)
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
int scaled_mix(const DocqaScaledNorm& a, hipStream_t s) {
  if (a.ids) return a.W % 4 == 0 ? launch_scaled<4, PT, true>(a, s) : launch_scaled<1, PT, true>(a, s);
  return a.W % 4 == 0 ? launch_scaled<4, PT, false>(a, s) : launch_scaled<1, PT, false>(a, s);
}

template <int V>
int launch_post_norm(const DocqaPostNorm& a, hipStream_t s) {
  const int n = a.W / V, gn = n / a.groups;
  const bool gw = gn % 64 == 0;
#define RUN(NT, NV, GW) \
  post_norm_kernel<NT, NV, V, GW><<<a.rows, NT, (GW ? NV * NT / 64 : n + a.groups) * sizeof(float), s>>>(a)
#define GO(NV)                                                                \
  do {                                                                        \
    if (!gw) RUN(256, NV, false);                                             \
    else if (NV >= 4 && a.rows <= 512) RUN(1024, (NV >= 4 ? NV / 4 : 1), true); \
    else RUN(256, NV, true);                                                  \
  } while (0)
  const int nv = (n + 255) / 256;
  if (nv <= 1) GO(1);
  else if (nv <= 2) GO(2);
  else if (nv <= 4) GO(4);
  else if (nv <= 8) GO(8);
  else if (nv <= 16) GO(16);
  else return -1;
#undef GO
#undef RUN
  DOCQA_CHECK_LAUNCH();
  return 0;
}
}  // namespace

int docqa_scaled_rmsnorm(const DocqaScaledNorm& a, hipStream_t s) {
  if (a.rows == 0) return 0;
  if (a.W < 1 || a.SP < 1 || !a.scale || (a.ids && (!a.wts || !a.x))) return -1;
  return a.pf32 ? scaled_mix<float>(a, s) : scaled_mix<uint16_t>(a, s);
}

int docqa_post_norm(const DocqaPostNorm& a, hipStream_t s) {
  if (a.rows == 0) return 0;
  if (a.W < 1 || a.groups < 1 || a.W % a.groups || a.SP < 1 || a.SQ < 1 || a.SG < 1 || (a.P && (!a.gate || !a.gb))) return -1;
  const bool vec = a.W / a.groups % 4 == 0 && a.col % 4 == 0 && (!a.P || a.ldg % 4 == 0);
  return vec ? launch_post_norm<4>(a, s) : launch_post_norm<1>(a, s);
}

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

int docqa_sandwich_rmsnorm_conv(const void* P, int p_f32, int S, float* res, const float* w_post, const float* w_next,
                                const float* cw, int taps, void* state, const int* slots, const int* positions, void* out,
                                void* out2, int out_f32, int rows, int H, float eps, hipStream_t s) {
  if (rows == 0) return 0;
  if (S < 1 || H < 1 || taps < 1 || (out_f32 && !p_f32)) return -1;
#define ARGS S, res, w_post, w_next, cw, taps, state, slots, positions, out, out2, rows, H, eps, s
  if (out_f32) return sandwich_conv<float, float>((const float*)P, ARGS);
  return p_f32 ? sandwich_conv<float, uint16_t>((const float*)P, ARGS) : sandwich_conv<uint16_t, uint16_t>((const uint16_t*)P, ARGS);
#undef ARGS
}
