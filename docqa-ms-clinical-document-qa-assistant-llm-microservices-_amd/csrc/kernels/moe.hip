// moe.hip -- routed experts: E SwiGLU feed-forwards, `top` of them a token, each reading the token
// times its score:  y_k[t] = down_e (silu(s g) * (s u)),  g = gate_e x_t, u = up_e x_t, e = ids[t, k];
// or, clamped, the token itself:  down_e (g sigmoid(1.702 g) (u + 1)),  g from above, u on both sides.
// Ids from E on have no expert: their pairs are left out.
//
// * route: scores sigmoid(x w^T) in fp32 (bf16 operands: MFMA, K split over 16 waves), the largest
//   `top` of the first E, and the scores of the remaining columns.  Groups: softmax scores, the largest
//   by score + correction within the best groups, weights normed over the chosen.
// * a (token, choice) pair p = t top + k is a row of the grouped products; gate and up rows meet in
//   the same lane's accumulators, so the activation is the first product's epilogue.
//   Few pairs (decode): a workgroup takes one expert and 16 (or 32) output columns, finds the expert's
//   pairs itself, streams its weight rows once into registers, K split over 4 or 8 waves.
//   Many (prompts): pairs sorted by expert in one small launch, then 128 x 128 tiles as in gemm.hip,
//   A rows gathered by the LDS-DMA's per-lane source addresses.
//   fp32 and odd sizes: a wave an output element.
#include "docqa_common.h"
#include "docqa_elem.h"
#include "docqa_hybrid.h"

using namespace docqa;

namespace {
constexpr int kSkinnyPairs = 512;       // pairs up to which a launch finds its rows itself
constexpr int BM = 128, BK = 64, kGroup = 8;

__device__ __forceinline__ float sigmoid_x(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float glu_f(float g, float u, float s, float limit) {
  if (limit > 0.f) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.f + __expf(-1.702f * g)) * (u + 1.f);
  }
  g *= s;
  return g / (1.f + __expf(-g)) * (u * s);
}

// ------------------------------------------------------------------ routing
// the largest `top` of sc[0, E) by one wave, ties to the lower index
__device__ __forceinline__ void pick(const float* sc, int E, int top, int* ids, float* wts) {
  const int lane = threadIdx.x & 63;
  float v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = lane + 64 * i < E ? sc[lane + 64 * i] : -1.f;
  for (int k = 0; k < top; ++k) {
    float m = -1.f;
    int at = 0;
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (v[i] > m) m = v[i], at = lane + 64 * i;
    const float best = wave_max(m);
    int idx = m == best ? at : 1 << 30;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) idx = min(idx, __shfl_xor(idx, o, 64));
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (lane + 64 * i == idx) v[i] = -2.f;
    if (lane == 0) {
      ids[k] = min(idx, E - 1);
      wts[k] = best;
    }
  }
}

struct RouteArgs {
  int* ids;
  float *wts, *rest;       // rest: scores of columns [E, N)
  int K, N, E, top;
  const float* corr;       // groups: [N]
  int groups, keep;
  float scale;
};

// between a wave's own writes to LDS and its reads of other lanes' parts
__device__ __forceinline__ void wave_lds_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

// one wave's token: logits sc[0, N) (N <= 512) -> choice; sc[N, 2 N) is scratch
__device__ __forceinline__ void pick_groups(float* sc, const RouteArgs& a, int* ids, float* wts) {
  const int lane = threadIdx.x & 63, N = a.N, gs = N / a.groups;
  float s[8], c[8], m = -INFINITY, sum = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    s[i] = lane + 64 * i < N ? sc[lane + 64 * i] : -INFINITY;
    m = fmaxf(m, s[i]);
  }
  m = wave_max(m);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    s[i] = expf(s[i] - m);
    sum += s[i];
  }
  sum = 1.f / wave_sum(sum);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int n = lane + 64 * i;
    s[i] *= sum;
    c[i] = n < N ? s[i] + a.corr[n] : -INFINITY;
  }
  if (a.keep < a.groups) {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (lane + 64 * i < N) sc[lane + 64 * i] = c[i];
    wave_lds_sync();
    float* best = sc + N;                     // a group's largest choice score
    for (int g = lane; g < a.groups; g += 64) {
      float b = sc[g * gs];
      for (int j = 1; j < gs; ++j) b = fmaxf(b, sc[g * gs + j]);
      best[g] = b;
    }
    wave_lds_sync();
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int n = lane + 64 * i;
      if (n >= N) continue;
      const int g = n / gs;
      const float b = best[g];
      int ahead = 0;
      for (int h = 0; h < a.groups; ++h) ahead += best[h] > b || (best[h] == b && h < g);
      if (ahead >= a.keep) c[i] = -INFINITY;
    }
  }
  float own = 0.f, total = 0.f;
  int id = 0;
  for (int k = 0; k < a.top; ++k) {
    float b = -INFINITY, w = 0.f;
    int at = 1 << 30;
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (c[i] > b) b = c[i], at = lane + 64 * i;
    int idx = b == wave_max(b) ? at : 1 << 30;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) idx = min(idx, __shfl_xor(idx, o, 64));
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (lane + 64 * i == idx) w = s[i], c[i] = -INFINITY;
    w = wave_sum(w);
    total += w;
    if (lane == k) own = w, id = min(idx, N - 1);
  }
  if (lane < a.top) {
    ids[lane] = id;
    wts[lane] = own / (total + 1e-20f) * a.scale;
  }
}

// 16 tokens a workgroup of 16 waves that split K, 32 columns a pass; x [T, K], w [N, K], K % 32 == 0
template <bool GROUPS>
__global__ __launch_bounds__(1024) void moe_route_mfma_kernel(const uint16_t* __restrict__ x, const uint16_t* __restrict__ w,
                                                              RouteArgs a, int T) {
  extern __shared__ float sc[];              // [16][N] scores (groups: [16][2 N])
  const int K = a.K, N = a.N, E = a.E, top = a.top, ld = GROUPS ? 2 * N : N;
  __shared__ float red[16][2][16][17];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, fr = lane & 15, g4 = lane >> 4;
  const int t0 = blockIdx.x * 16;
  const uint16_t* xp = x + (size_t)min(t0 + fr, T - 1) * K + g4 * 8;
  for (int n0 = 0; n0 < N; n0 += 32) {
    const uint16_t *w0 = w + (size_t)min(n0 + fr, N - 1) * K + g4 * 8, *w1 = w + (size_t)min(n0 + 16 + fr, N - 1) * K + g4 * 8;
    f32x4 a0 = f32x4{0.f, 0.f, 0.f, 0.f}, a1 = a0;
#pragma unroll 4
    for (int k = wave * 32; k < K; k += 512) {
      const bf16x8 v = *reinterpret_cast<const bf16x8*>(xp + k);
      a0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, *reinterpret_cast<const bf16x8*>(w0 + k), a0, 0, 0, 0);
      a1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, *reinterpret_cast<const bf16x8*>(w1 + k), a1, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      red[wave][0][g4 * 4 + r][fr] = a0[r];
      red[wave][1][g4 * 4 + r][fr] = a1[r];
    }
    __syncthreads();
    if (tid < 512) {
      const int t = tid >> 5, c = tid & 31;
      float z = 0.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) z += red[i][c >> 4][t][c & 15];
      if (n0 + c < N) sc[t * ld + n0 + c] = GROUPS ? z : sigmoid_x(z);
    }
    __syncthreads();
  }
  if (t0 + wave < T) {
    const size_t t = t0 + wave;
    if constexpr (GROUPS) {
      pick_groups(sc + wave * ld, a, a.ids + t * top, a.wts + t * top);
    } else {
      pick(sc + wave * N, E, top, a.ids + t * top, a.wts + t * top);
      for (int c = E + lane; c < N; c += 64) a.rest[t * (N - E) + c - E] = sc[wave * N + c];
    }
  }
}

// any size and element type: a workgroup a token, a wave a score at a time
template <typename T, bool GROUPS>
__global__ __launch_bounds__(256) void moe_route_kernel(const T* __restrict__ x, const T* __restrict__ w, RouteArgs a) {
  extern __shared__ float sc[];              // [N] (groups: [2 N])
  const int K = a.K, N = a.N, E = a.E, top = a.top;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const size_t t = blockIdx.x;
  for (int n = wave; n < N; n += 4) {
    float z = 0.f;
    for (int k = lane; k < K; k += 64) z += ld1(x + t * K + k) * ld1(w + (size_t)n * K + k);
    z = wave_sum(z);
    if (lane == 0) sc[n] = GROUPS ? z : sigmoid_x(z);
  }
  __syncthreads();
  if constexpr (GROUPS) {
    if (wave == 0) pick_groups(sc, a, a.ids + t * top, a.wts + t * top);
  } else {
    if (wave == 0) pick(sc, E, top, a.ids + t * top, a.wts + t * top);
    for (int c = E + threadIdx.x; c < N; c += 256) a.rest[t * (N - E) + c - E] = sc[c];
  }
}

// ------------------------------------------------------------------ any size: a wave an element
template <typename T, bool UP>
__global__ __launch_bounds__(256) void moe_plain_kernel(const T* __restrict__ x, const int* __restrict__ ids,
                                                        const float* __restrict__ wts, const T* __restrict__ w, T* __restrict__ y,
                                                        int Tn, int top, int E, int K, int N, float limit) {
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const size_t p = blockIdx.y + (size_t)blockIdx.z * 65535;
  if (n >= N || p >= (size_t)Tn * top || ids[p] >= E) return;
  const T* xp = x + (UP ? p / top : p) * K;
  const T* wp = w + ((size_t)ids[p] * (UP ? 2 : 1) * N + n) * K;
  float a = 0.f, b = 0.f;
  for (int k = lane; k < K; k += 64) {
    const float v = ld1(xp + k);
    a += v * ld1(wp + k);
    if constexpr (UP) b += v * ld1(wp + (size_t)N * K + k);
  }
  a = wave_sum(a);
  if constexpr (UP) b = wave_sum(b);
  if (lane) return;
  if constexpr (UP) st1(y + p * N + n, glu_f(a, b, wts[p], limit));
  else st1(y + ((p % top) * Tn + p / top) * N + n, a);
}

// ------------------------------------------------------------------ few pairs
// blockIdx.y: the expert, or (E > pairs) a pair whose expert no earlier pair has.  MT row tiles of 16 at
// a time against two column tiles of 16: gate and up rows n0.. (UP), or rows n0.. and n0 + 16.. (down)
template <int MT, int NW, bool UP>
__global__ __launch_bounds__(64 * NW) void moe_skinny_kernel(const uint16_t* __restrict__ x, const int* __restrict__ ids,
                                                         const float* __restrict__ wts, const uint16_t* __restrict__ w,
                                                         uint16_t* __restrict__ y, int Tn, int top, int E, int K, int N,
                                                         float limit) {
  __shared__ int rows[kSkinnyPairs];
  __shared__ int count;
  __shared__ float red[NW][MT][2][16][17];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, fr = lane & 15, g4 = lane >> 4;
  const int P = Tn * top, n0 = blockIdx.x * (UP ? 16 : 32);
  int e = blockIdx.y;
  if (E > P) {
    const int p = e;
    e = ids[p];
    if (e >= E) return;
    for (int i = 0; i < p; ++i)
      if (ids[i] == e) return;
  }
  if (tid == 0) count = 0;
  __syncthreads();
  for (int p = tid; p < P; p += 64 * NW)
    if (ids[p] == e) rows[atomicAdd(&count, 1)] = p;
  __syncthreads();
  const int m = count;
  const uint16_t* w0 = w + ((size_t)e * (UP ? 2 : 1) * N + min(n0 + fr, N - 1)) * K + g4 * 8;
  const uint16_t* w1 = UP ? w0 + (size_t)N * K : w + ((size_t)e * N + min(n0 + 16 + fr, N - 1)) * K + g4 * 8;
  for (int r0 = 0; r0 < m; r0 += 16 * MT) {
    const uint16_t* xp[MT];
    f32x4 acc[MT][2];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int p = rows[min(r0 + i * 16 + fr, m - 1)];
      xp[i] = x + (size_t)(UP ? p / top : p) * K + g4 * 8;
      acc[i][0] = acc[i][1] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll 4
    for (int k = wave * 32; k < K; k += 32 * NW) {
      const bf16x8 b0 = *reinterpret_cast<const bf16x8*>(w0 + k), b1 = *reinterpret_cast<const bf16x8*>(w1 + k);
#pragma unroll
      for (int i = 0; i < MT; ++i) {
        const bf16x8 av = *reinterpret_cast<const bf16x8*>(xp[i] + k);
        acc[i][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av, b0, acc[i][0], 0, 0, 0);
        acc[i][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av, b1, acc[i][1], 0, 0, 0);
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int c = 0; c < 2; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) red[wave][i][c][g4 * 4 + r][fr] = acc[i][c][r];
    __syncthreads();
    const int c = tid & 15, r = tid >> 4;
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int row = r0 + i * 16 + r;
      if (r >= 16 || row >= m) continue;
      const int p = rows[row];
      float a = 0.f, b = 0.f;
#pragma unroll
      for (int q = 0; q < NW; ++q) {
        a += red[q][i][0][r][c];
        b += red[q][i][1][r][c];
      }
      if constexpr (UP) {
        if (n0 + c < N) y[(size_t)p * N + n0 + c] = f2bf(glu_f(a, b, wts[p], limit));
      } else {
        uint16_t* o = y + ((size_t)(p % top) * Tn + p / top) * N + n0;
        if (n0 + c < N) o[c] = f2bf(a);
        if (n0 + 16 + c < N) o[16 + c] = f2bf(b);
      }
    }
  }
}

// ------------------------------------------------------------------ many pairs
// scratch: rows [P] sorted by expert | tile expert [tiles] | tile first row [tiles] | tile last row + 1 [tiles]
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int* __restrict__ ids, int* __restrict__ scratch, int P, int E,
                                                        int tiles) {
  __shared__ int cnt[512], start[513];
  const int tid = threadIdx.x;
  for (int i = tid; i < E; i += 1024) cnt[i] = 0;
  __syncthreads();
  for (int p = tid; p < P; p += 1024)
    if (ids[p] < E) atomicAdd(&cnt[ids[p]], 1);
  __syncthreads();
  int *te = scratch + P, *tb = te + tiles, *tn = tb + tiles;
  if (tid == 0) {
    int s = 0;
    for (int e = 0; e < E; ++e) {
      start[e] = s;
      s += cnt[e];
    }
    start[E] = s;
  }
  for (int i = tid; i < tiles; i += 1024) te[i] = -1;
  __syncthreads();
  if (tid < E) {
    int t = 0;                                 // tiles ahead of this expert's
    for (int e = 0; e < tid; ++e) t += (cnt[e] + BM - 1) / BM;
    for (int r = start[tid]; r < start[tid + 1]; r += BM, ++t) {
      te[t] = tid;
      tb[t] = r;
      tn[t] = min(start[tid + 1], r + BM);
    }
  }
  __syncthreads();
  for (int i = tid; i < E; i += 1024) cnt[i] = start[i];
  __syncthreads();
  for (int p = tid; p < P; p += 1024)
    if (ids[p] < E) scratch[atomicAdd(&cnt[ids[p]], 1)] = p;
}

__device__ __forceinline__ int sw_off(int row, int ch) { return row * BK + ((ch ^ ((row >> 1) & 7)) << 3); }

// the tile and pipeline of gemm.hip.  UP: a tile's 128 weight rows are 64 gate and 64 up rows, arranged so
// that a wave's column tiles 0, 1 are gate and 2, 3 the matching up columns
template <bool UP>
__global__ __launch_bounds__(256) void moe_gemm_kernel(const uint16_t* __restrict__ x, const float* __restrict__ wts,
                                                       const uint16_t* __restrict__ w, uint16_t* __restrict__ y,
                                                       const int* __restrict__ scratch, int Tn, int top, int K, int N, int tiles,
                                                       float limit) {
  __shared__ __attribute__((aligned(16))) uint16_t smem[4 * 64 * 65 * 2];
  __shared__ int srow[BM];
  const int nbn = (N + (UP ? 63 : 127)) / (UP ? 64 : 128);
  const int wg = xcd_remap(blockIdx.x, gridDim.x);
  // row tiles in groups of kGroup, column after column: a group's tiles, mostly of one expert, share the
  // weight rows they read at about the same time
  const int g0 = wg / (kGroup * nbn) * kGroup, gs = min(kGroup, tiles - g0), gi = wg - g0 * nbn;
  const int bm = g0 + gi % gs, bn = gi / gs, P = Tn * top;
  const int *te = scratch + P, *tb = te + tiles, *tn = tb + tiles;
  const int e = te[bm];
  if (e < 0) return;
  const int r0 = tb[bm], m = tn[bm] - r0;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int wr = wave >> 1, wc = wave & 1, fr = lane & 15, fk = lane >> 4;
  if (tid < BM) srow[tid] = scratch[r0 + min(tid, m - 1)];
  __syncthreads();
  const uint16_t* we = w + (size_t)e * (UP ? 2 : 1) * N * K;
  const uint16_t *ap[4], *wp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int p = (i * 4 + wave) * 64 + lane, r = p >> 3, ch = (p & 7) ^ ((r >> 1) & 7);
    const int pair = srow[r];
    ap[i] = x + (size_t)(UP ? pair / top : pair) * K + ch * 8;
    int col;
    if constexpr (UP) {
      const int f = bn * 64 + (r >> 6) * 32 + ((r >> 4) & 1) * 16 + (r & 15);
      col = (((r >> 5) & 1) ? N : 0) + min(f, N - 1);
    } else {
      col = min(bn * 128 + r, N - 1);
    }
    wp[i] = we + (size_t)col * K + ch * 8;
  }
  f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  typedef __attribute__((address_space(3))) void lds_void;
  auto stage = [&](int kt, int buf) {
    uint16_t* sa = smem + buf * (2 * BM * BK);
    uint16_t* sw = sa + BM * BK;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int p0 = (i * 4 + wave) * 64;
      __builtin_amdgcn_global_load_lds(ap[i] + kt * BK, (lds_void*)(sa + p0 * 8), 16, 0, 0);
      __builtin_amdgcn_global_load_lds(wp[i] + kt * BK, (lds_void*)(sw + p0 * 8), 16, 0, 0);
    }
  };
  const int nk = K / BK;
  stage(0, 0);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  for (int kt = 0; kt < nk; ++kt) {
    const int buf = kt & 1;
    if (kt + 1 < nk) stage(kt + 1, buf ^ 1);
    const uint16_t* sa = smem + buf * (2 * BM * BK);
    const uint16_t* sw = sa + BM * BK;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 af[4], bf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        af[i] = *reinterpret_cast<const bf16x8*>(sa + sw_off(wr * 64 + i * 16 + fr, ks * 4 + fk));
        bf[i] = *reinterpret_cast<const bf16x8*>(sw + sw_off(wc * 64 + i * 16 + fr, ks * 4 + fk));
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af[i], bf[j], acc[i][j], 0, 0, 0);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
  }
  // epilogue: the wave's tile through its own LDS, then 16-byte stores
  float* st = reinterpret_cast<float*>(smem) + wave * (64 * 65);
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = i * 16 + fk * 4 + r;
      if constexpr (UP) {
        const float s = wts[srow[wr * 64 + row]];
#pragma unroll
        for (int j = 0; j < 2; ++j) st[row * 65 + j * 16 + fr] = glu_f(acc[i][j][r], acc[i][2 + j][r], s, limit);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) st[row * 65 + j * 16 + fr] = acc[i][j][r];
      }
    }
  __syncthreads();
  constexpr int CH = UP ? 4 : 8;               // 8-column pieces of the wave's tile
  for (int it = 0; it < CH; ++it) {
    const int row = it * (64 / CH) + lane / CH, c = (lane % CH) * 8, lr = wr * 64 + row;
    const int gc = UP ? bn * 64 + wc * 32 + c : bn * 128 + wc * 64 + c;
    if (lr >= m || gc >= N) continue;
    const int pair = srow[lr];
    float v[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = st[row * 65 + c + j];
    uint16_t* o = UP ? y + (size_t)pair * N : y + ((size_t)(pair % top) * Tn + pair / top) * N;
    *reinterpret_cast<uint4*>(o + gc) = pack8(v);
  }
}

bool skinny_ok(int K, int N) { return K % 32 == 0 && N >= 1; }
bool tile_ok(int K, int N) { return K % 64 == 0 && N % 8 == 0; }
int tile_count(int P, int E) { return P / BM + E; }

template <typename T>
int plain(const void* x, const int* ids, const float* wts, const void* up, const void* down, void* act, void* out, int Tn, int top,
          int E, int K, int F, int W, float limit, hipStream_t s) {
  const long long P = (long long)Tn * top;
  const unsigned gy = (unsigned)(P < 65535 ? P : 65535), gz = (unsigned)((P + 65534) / 65535);
  moe_plain_kernel<T, true><<<dim3((F + 3) / 4, gy, gz), 256, 0, s>>>((const T*)x, ids, wts, (const T*)up, (T*)act, Tn, top, E, K, F, limit);
  DOCQA_CHECK_LAUNCH();
  moe_plain_kernel<T, false><<<dim3((W + 3) / 4, gy, gz), 256, 0, s>>>((const T*)act, ids, wts, (const T*)down, (T*)out, Tn, top, E, F, W, limit);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <bool GROUPS>
int route(const void* x, const void* w, int f32, const RouteArgs& a, int T, hipStream_t s) {
  const size_t row = (size_t)a.N * (GROUPS ? 8 : 4);
  if (!f32 && a.K % 32 == 0 && 16 * row <= 64 * 1024 - 36 * 1024)
    moe_route_mfma_kernel<GROUPS><<<(T + 15) / 16, 1024, 16 * row, s>>>((const uint16_t*)x, (const uint16_t*)w, a, T);
  else if (f32)
    moe_route_kernel<float, GROUPS><<<T, 256, row, s>>>((const float*)x, (const float*)w, a);
  else
    moe_route_kernel<uint16_t, GROUPS><<<T, 256, row, s>>>((const uint16_t*)x, (const uint16_t*)w, a);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <int MT>
int skinny(const uint16_t* x, const int* ids, const float* wts, const uint16_t* up, const uint16_t* down, uint16_t* act,
           uint16_t* out, int Tn, int top, int E, int K, int F, int W, float limit, hipStream_t s) {
  const int gy = E < Tn * top ? E : Tn * top;
  constexpr int NW = MT == 1 ? 8 : 4;
  moe_skinny_kernel<MT, NW, true><<<dim3((F + 15) / 16, gy), 64 * NW, 0, s>>>(x, ids, wts, up, act, Tn, top, E, K, F, limit);
  DOCQA_CHECK_LAUNCH();
  moe_skinny_kernel<MT, NW, false><<<dim3((W + 31) / 32, gy), 64 * NW, 0, s>>>(act, ids, wts, down, out, Tn, top, E, F, W, limit);
  DOCQA_CHECK_LAUNCH();
  return 0;
}
}  // namespace

int docqa_moe_route(const void* x, const void* w, int f32, int* ids, float* wts, float* rest, int T, int K, int N, int E,
                    int top, hipStream_t s) {
  if (T == 0) return 0;
  if (E < 1 || E > 512 || N < E || N > 1024 || top < 1 || top > E || K < 1) return -1;
  return route<false>(x, w, f32, RouteArgs{ids, wts, rest, K, N, E, top, nullptr, 1, 1, 1.f}, T, s);
}

int docqa_moe_route_groups(const void* x, const void* w, int f32, const float* corr, int* ids, float* wts, int T, int K, int N,
                           int top, int groups, int keep, float scale, hipStream_t s) {
  if (T == 0) return 0;
  if (N < 1 || N > 512 || K < 1 || !corr || groups < 1 || N % groups || keep < 1 || keep > groups || top < 1 || top > 64 ||
      top > keep * (N / groups))
    return -1;
  return route<true>(x, w, f32, RouteArgs{ids, wts, nullptr, K, N, N, top, corr, groups, keep, scale}, T, s);
}

int docqa_moe_scratch(int f32, int T, int top, int E, int K, int F, int W) {
  const long long P = (long long)T * top;
  if (f32 || P <= kSkinnyPairs || !tile_ok(K, F) || !tile_ok(F, W)) return 0;
  return (int)(P + 3 * tile_count((int)P, E));
}

int docqa_moe_experts(const void* x, const int* ids, const float* wts, const void* up, const void* down, void* act, void* out,
                      int* scratch, int f32, int T, int top, int E, int K, int F, int W, float limit, hipStream_t s) {
  const long long P = (long long)T * top;
  if (P == 0) return 0;
  if (E < 1 || E > 512 || top < 1 || K < 1 || F < 1 || W < 1 || P >= (1ll << 30)) return -1;
  if (f32) return plain<float>(x, ids, wts, up, down, act, out, T, top, E, K, F, W, limit, s);
  const uint16_t *xp = (const uint16_t*)x, *u = (const uint16_t*)up, *d = (const uint16_t*)down;
  uint16_t *a = (uint16_t*)act, *o = (uint16_t*)out;
  if (scratch) {
    if (!tile_ok(K, F) || !tile_ok(F, W)) return -1;
    const int tiles = tile_count((int)P, E);
    moe_sort_kernel<<<1, 1024, 0, s>>>(ids, scratch, (int)P, E, tiles);
    DOCQA_CHECK_LAUNCH();
    moe_gemm_kernel<true><<<tiles * ((F + 63) / 64), 256, 0, s>>>(xp, wts, u, a, scratch, T, top, K, F, tiles, limit);
    DOCQA_CHECK_LAUNCH();
    moe_gemm_kernel<false><<<tiles * ((W + 127) / 128), 256, 0, s>>>(a, wts, d, o, scratch, T, top, F, W, tiles, limit);
    DOCQA_CHECK_LAUNCH();
    return 0;
  }
  if (P <= kSkinnyPairs && skinny_ok(K, F) && skinny_ok(F, W)) {
    if (P <= 16 * E || P <= 16) return skinny<1>(xp, ids, wts, u, d, a, o, T, top, E, K, F, W, limit, s);
    if (P <= 32 * E) return skinny<2>(xp, ids, wts, u, d, a, o, T, top, E, K, F, W, limit, s);
    return skinny<4>(xp, ids, wts, u, d, a, o, T, top, E, K, F, W, limit, s);
  }
  return plain<uint16_t>(x, ids, wts, up, down, act, out, T, top, E, K, F, W, limit, s);
}
