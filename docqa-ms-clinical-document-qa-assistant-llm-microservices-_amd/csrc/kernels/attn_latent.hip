// attn_latent.hip -- latent attention: per-head keys and values are linear in one normed latent
// row a token, plus a rotated key part all heads share, so the paged cache holds a single row
//   [latent: R | rotated part: r]       (each padded with zeros to 8 elements: R8, r8)
// for all heads.  A query head is [unrotated: d | rotated: r], padded alike (d8, r8).
//
//   * rope_table:    [cos | sin] rows of a forward's positions, angles in fp64, once for all layers;
//   * latent_store:  consumer of the [q | latent | key part] projection: sums the split-K slabs,
//                    rotates the query heads, normalises the latent, rotates the key part, stores
//                    the cache row;
//   * absorbed form (decode, short portions): head_project takes the query heads into the latent
//     space, every head attends the cached rows themselves -- key and value at once -- and
//     head_project takes the attended latents to values (summing the key splits on the way);
//   * expanded form (prompts): latent_gather packs the visible rows, a GEMM makes every head's
//     keys and values of them, attn_window.hip's packed form attends.
//
// latent_attn: query rows are (token, head) pairs, 16 QT to a workgroup.  A 64-key tile in LDS
// serves both products: the waves take 16 keys each for S^T = K Q^T, exchange row maxima and the
// bf16 scores through LDS, and take a slice of the latent's columns each for O^T += V^T P^T (V^T by
// transposing LDS reads of the same tile).  So a tile is read twice per workgroup however many rows
// it serves, and a wave's accumulators are a slice of a row, not the 512-wide row itself.  Few
// sequences: the keys are split over workgroups (partials in fp32, merged by latent_merge).
#include "docqa_common.h"
#include "docqa_elem.h"
#include "docqa_hybrid.h"

using namespace docqa;

namespace {
constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

__global__ __launch_bounds__(256) void rope_table_kernel(const int* __restrict__ pos, const double* __restrict__ freq,
                                                         float* __restrict__ out, int T, int half) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= T * half) return;
  const int t = i / half, k = i - t * half;
  double s, c;
  sincos((double)pos[t] * freq[k], &s, &c);
  out[(size_t)t * 2 * half + k] = (float)c;
  out[(size_t)t * 2 * half + half + k] = (float)s;
}

struct StoreArgs {
  int S, ld;
  size_t slab;
  const float* cs;        // [T, r]
  const int* slots;
  const float* wn;        // [R] or null: no latent in the projection
  int H, d, r, R, d8, r8, R8, D, log2BS;
  float eps;
};

// grid (token, y): y < ny: 256 V-element items of the query heads; y == ny: the latent row
template <int V, int NI, typename PT, typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(const PT* __restrict__ P, T* __restrict__ q,
                                                           T* __restrict__ cache, int ny, StoreArgs a) {
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x, half = a.r / 2;
  const PT* p = P + (size_t)t * a.ld;
  const float* cs = a.cs + (size_t)t * a.r;
  auto rotate = [&](const PT* x, T* o, int i) {          // V pairs from pair i on
    float u[V], v[V], c[V], s[V], x0[V], x1[V];
    ld_slabs<V>(x + i, a.S, a.slab, u);
    ld_slabs<V>(x + half + i, a.S, a.slab, v);
    ldv<V>(cs + i, c);
    ldv<V>(cs + half + i, s);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      x0[j] = u[j] * c[j] - v[j] * s[j];
      x1[j] = v[j] * c[j] + u[j] * s[j];
    }
    stv<V>(o + i, x0);
    stv<V>(o + half + i, x1);
  };
  if ((int)blockIdx.y < ny) {
    // a head's items: d / V copies, half / V rotations, then (V = 1) the zero padding
    const int nc = a.d / V, nr = half / V, zd = a.d8 - a.d, nz = V == 1 ? zd + a.r8 - a.r : 0, per = nc + nr + nz;
    const int i = blockIdx.y * 256 + tid;
    if (i >= a.H * per) return;
    const int h = i / per, k = i - h * per;
    const PT* x = p + h * (a.d + a.r);
    T* o = q + ((size_t)t * a.H + h) * (a.d8 + a.r8);
    if (k < nc) {
      float f[V];
      ld_slabs<V>(x + k * V, a.S, a.slab, f);
      stv<V>(o + k * V, f);
    } else if (k < nc + nr) {
      rotate(x + a.d, o + a.d8, (k - nc) * V);
    } else {
      const int z = k - nc - nr;
      st1(o + (z < zd ? a.d + z : a.d8 + a.r + z - zd), 0.f);
    }
    return;
  }
  const int slot = a.slots[t];
  if (slot < 0) return;                                  // the whole workgroup
  // one KV head: row = slot of the paged cache
  T* o = cache + (size_t)slot * a.D;
  const PT* x = p + a.H * (a.d + a.r);
  float f[NI][V];
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < NI; ++n) {
    const int c = (tid + 256 * n) * V;
    if (c < a.R) {
      ld_slabs<V>(x + c, a.S, a.slab, f[n]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += f[n][j] * f[n][j];
    }
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.R + a.eps);
#pragma unroll
  for (int n = 0; n < NI; ++n) {
    const int c = (tid + 256 * n) * V;
    if (c < a.R) {
      float w[V];
      ldv<V>(a.wn + c, w);
#pragma unroll
      for (int j = 0; j < V; ++j) f[n][j] *= inv * w[j];
      stv<V>(o + c, f[n]);
    }
  }
  for (int i = tid; i < half / V; i += 256) rotate(x + a.R, o + a.R8, i * V);
  if (V == 1) {
    for (int i = tid; i < a.R8 - a.R; i += 256) st1(o + a.R + i, 0.f);
    for (int i = tid; i < a.r8 - a.r; i += 256) st1(o + a.R8 + a.r + i, 0.f);
  }
}

// ------------------------------------------------------------------ per-head products
// y[t, h, :N] = x[t, h, :K] . w[h]^T; y[t, h, N : N + E] = x[t, h, K : K + E].  One workgroup:
// 16 MT rows of one head, 128 outputs; x rows staged in LDS, w straight to registers.
template <int MT>
__global__ __launch_bounds__(256) void head_project_kernel(const uint16_t* __restrict__ x,
                                                           const uint16_t* __restrict__ w, uint16_t* __restrict__ y,
                                                           int T, int H, int K, int N, int E) {
  extern __shared__ __attribute__((aligned(16))) uint16_t sx[];       // [16 MT][pitch]
  const int kp = (K + 31) / 32 * 32, pitch = kp + 8;
  const int h = blockIdx.x, m0 = blockIdx.y * 16 * MT, tid = threadIdx.x;
  const int ldx = H * (K + E), ldy = H * (N + E);
  const uint16_t* xh = x + (size_t)h * (K + E);
  uint16_t* yh = y + (size_t)h * (N + E);
  const int per = kp / 8;
  for (int i = tid; i < 16 * MT * per; i += 256) {
    const int r = i / per, c = (i - r * per) * 8;
    uint4 v = make_uint4(0, 0, 0, 0);
    if (m0 + r < T && c < K) v = *reinterpret_cast<const uint4*>(xh + (size_t)(m0 + r) * ldx + c);
    *reinterpret_cast<uint4*>(sx + r * pitch + c) = v;
  }
  if (blockIdx.z == 0 && E > 0) {
    const int pe = E / 8;
    for (int i = tid; i < 16 * MT * pe; i += 256) {
      const int r = i / pe, c = (i - r * pe) * 8;
      if (m0 + r < T)
        *reinterpret_cast<uint4*>(yh + (size_t)(m0 + r) * ldy + N + c) =
            *reinterpret_cast<const uint4*>(xh + (size_t)(m0 + r) * ldx + K + c);
    }
  }
  __syncthreads();
  const int lane = tid & 63, wave = tid >> 6, fr = lane & 15, g4 = lane >> 4;
  const int n0 = blockIdx.z * 128 + wave * 32;                        // this wave's outputs n0 .. n0 + 31
  if (n0 >= N) return;
  f32x4 acc[MT][2];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const uint16_t* wh = w + (size_t)h * N * K;
#pragma unroll 4
  for (int k = 0; k < kp; k += 32) {
    const int kk = k + g4 * 8;
    bf16x8 wf[2], xf[MT];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int n = n0 + 16 * j + fr;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (n < N && kk < K) v = *reinterpret_cast<const uint4*>(wh + (size_t)n * K + kk);
      wf[j] = *reinterpret_cast<bf16x8*>(&v);
    }
#pragma unroll
    for (int i = 0; i < MT; ++i) xf[i] = *reinterpret_cast<const bf16x8*>(sx + (i * 16 + fr) * pitch + kk);
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[j], xf[i], acc[i][j], 0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int row = m0 + i * 16 + fr;
    if (row >= T) continue;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int n = n0 + 16 * j + g4 * 4;
      uint16_t* op = yh + (size_t)row * ldy + n;
      if (N % 4 == 0) {
        if (n < N) {
          const float f[4] = {acc[i][j][0], acc[i][j][1], acc[i][j][2], acc[i][j][3]};
          stv<4>(op, f);
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (n + r < N) op[r] = f2bf(acc[i][j][r]);
      }
    }
  }
}

// packed copies of the cached rows of positions [first[b], first[b] + n_b): c [total, R8], kr [total, r8]
__global__ __launch_bounds__(256) void latent_gather_kernel(const uint16_t* __restrict__ cache,
                                                            const int* __restrict__ bt, int maxb,
                                                            const int* __restrict__ first, const int* __restrict__ cu_k,
                                                            uint16_t* __restrict__ c, uint16_t* __restrict__ kr, int R8,
                                                            int r8, int log2BS) {
  const int b = blockIdx.y, n = cu_k[b + 1] - cu_k[b], D = R8 + r8, per = D / 8;
  const int i = blockIdx.x * 256 + threadIdx.x, j = i / per, e = (i - j * per) * 8;
  if (j >= n) return;
  const int key = first[b] + j;
  const size_t row = ((size_t)bt[(size_t)b * maxb + (key >> log2BS)] << log2BS) + (key & ((1 << log2BS) - 1));
  const uint4 v = *reinterpret_cast<const uint4*>(cache + row * D + e);
  const size_t dst = (size_t)cu_k[b] + j;
  if (e < R8) *reinterpret_cast<uint4*>(c + dst * R8 + e) = v;
  else *reinterpret_cast<uint4*>(kr + dst * r8 + (e - R8)) = v;
}

template <typename PT, typename T>
int store_types(const void* P, void* q, void* cache, int T_, const StoreArgs& a, hipStream_t s) {
  const bool v4 = a.d % 8 == 0 && a.r % 8 == 0 && a.R % 8 == 0 && a.ld % 4 == 0;
  const int V = v4 ? 4 : 1;
  const int per = a.d / V + a.r / 2 / V + (v4 ? 0 : a.d8 - a.d + a.r8 - a.r);
  const int ny = (a.H * per + 255) / 256;
  dim3 grid(T_, ny + (a.wn ? 1 : 0));
  if (v4) latent_store_kernel<4, 2, PT, T><<<grid, 256, 0, s>>>((const PT*)P, (T*)q, (T*)cache, ny, a);
  else latent_store_kernel<1, 8, PT, T><<<grid, 256, 0, s>>>((const PT*)P, (T*)q, (T*)cache, ny, a);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int log2_of(int n) {
  int l = 0;
  while ((1 << l) < n) ++l;
  return l;
}
}  // namespace

int docqa_rope_table(const int* positions, const double* freq, float* out, int T, int half, hipStream_t s) {
  if (T == 0) return 0;
  if (half < 1 || (long long)T * half >= (1ll << 31)) return -1;
  rope_table_kernel<<<(T * half + 255) / 256, 256, 0, s>>>(positions, freq, out, T, half);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_latent_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* cs, const int* slots,
                       const float* c_norm, void* q, void* cache, int f32, int T, int H, int d, int r, int R, int BS,
                       float eps, hipStream_t s) {
  if (T == 0) return 0;
  if (S < 1 || H < 1 || d < 1 || r < 2 || r % 2 || R < 1 || R > 2048 || (BS & (BS - 1)) != 0) return -1;
  if (ld < H * (d + r) + (c_norm ? R + r : 0) || (f32 && !p_f32)) return -1;
  StoreArgs a{S, ld, slab, cs, slots, c_norm, H, d, r, R, (d + 7) / 8 * 8, (r + 7) / 8 * 8, (R + 7) / 8 * 8, 0,
              log2_of(BS), eps};
  a.D = a.R8 + a.r8;
  if (f32) return store_types<float, float>(P, q, cache, T, a, s);
  return p_f32 ? store_types<float, uint16_t>(P, q, cache, T, a, s)
               : store_types<uint16_t, uint16_t>(P, q, cache, T, a, s);
}

int docqa_head_project(const void* x, const void* w, void* y, int T, int H, int K, int N, int E, hipStream_t s) {
  if (T == 0) return 0;
  if (H < 1 || K < 8 || K % 8 || K > 2048 || N < 1 || E < 0 || E % 8 || (E > 0 && N % 8)) return -1;
  if (!docqa_aligned16(x) || !docqa_aligned16(w) || !docqa_aligned16(y)) return -1;
  const int pitch = (K + 31) / 32 * 32 + 8;
#define GO(MT)                                                                                                        \
  do {                                                                                                                \
    const size_t lds = (size_t)16 * MT * pitch * 2;                                                                   \
    auto kern = head_project_kernel<MT>;                                                                              \
    if (lds > 64 * 1024) {                                                                                            \
      static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern),                            \
                                                      hipFuncAttributeMaxDynamicSharedMemorySize, 80 * 1024);         \
      if (e != hipSuccess) return (int)e;                                                                             \
    }                                                                                                                 \
    kern<<<dim3(H, (T + 16 * MT - 1) / (16 * MT), (N + 127) / 128), 256, lds, s>>>((const uint16_t*)x,                \
        (const uint16_t*)w, (uint16_t*)y, T, H, K, N, E);                                                             \
  } while (0)
  if (T > 32 && K <= 256) GO(4);
  else if (T > 16 && K <= 1024) GO(2);
  else GO(1);
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_latent_gather(const void* cache, const int* block_tables, int maxb, const int* first, const int* cu_k, void* c,
                        void* kr, int B, int max_keys, int R8, int r8, int BS, hipStream_t s) {
  if (B == 0 || max_keys == 0) return 0;
  if (R8 < 8 || R8 % 8 || r8 < 8 || r8 % 8 || B > 65535 || (BS & (BS - 1)) != 0) return -1;
  const long long items = (long long)max_keys * ((R8 + r8) / 8);
  if (items >= (1ll << 31)) return -1;
  latent_gather_kernel<<<dim3((unsigned)((items + 255) / 256), B), 256, 0, s>>>(
      (const uint16_t*)cache, block_tables, maxb, first, cu_k, (uint16_t*)c, (uint16_t*)kr, R8, r8, log2_of(BS));
  DOCQA_CHECK_LAUNCH();
  return 0;
}
