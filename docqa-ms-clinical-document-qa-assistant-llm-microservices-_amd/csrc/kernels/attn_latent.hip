// attn_latent.hip -- latent attention: per-head keys and values are linear in one normed latent
// row a token, plus a rotated key part all heads share, so the paged cache holds a single row
//   [latent: R | rotated part: r]       (each padded with zeros to 8 elements: R8, r8)
// for all heads.  A query head is [unrotated: d | rotated: r], padded alike (d8, r8).
//
//   * rope_table:    [cos | sin] rows of a forward's positions, angles in fp64, once for all layers;
//   * latent_store:  consumer of the [q | latent | key part] projection: sums the split-K slabs,
//                    rotates the query heads, normalises the latent, rotates the key part, stores
//                    the cache row; with a query latent (latent_norm_store) that is normed in the same
//                    launch, and a second one rotates the heads its projection makes;
//   * absorbed form (decode, short portions): head_project takes the query heads into the latent
//     space, every head attends the cached rows themselves -- key and value at once -- and
//     head_project takes the attended latents to values (summing the key splits on the way, an
//     output gate in its epilogue);
//   * expanded form (prompts): latent_gather packs the visible rows, a GEMM makes every head's
//     keys and values of them, attn_window.hip's packed form attends.
//
// latent_attn: query rows are (token, head) pairs, 16 QT to a workgroup.  A 64-key tile in LDS
// serves both products: the waves take 16 keys each for S^T = K Q^T, exchange row maxima and the
// bf16 scores through LDS, and take a slice of the latent's columns each for O^T += V^T P^T (V^T by
// transposing LDS reads of the same tile).  So a tile is read twice per workgroup however many rows
// it serves, and a wave's accumulators are a slice of a row, not the 512-wide row itself.  Few
// sequences: the keys are split over workgroups; the value projection sums the splits' outputs.
#include "docqa_common.h"
#include "docqa_elem.h"
#include "docqa_gate.h"
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

// LDS-only workgroup barrier: __syncthreads() also drains the global loads in flight, and the
// next tiles' are meant to stay there
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

__global__ __launch_bounds__(256) void rope_table_kernel(const int* __restrict__ pos, const double* __restrict__ freq,
                                                         float* __restrict__ out, int T, int half, double mult) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= T * half) return;
  const int t = i / half, k = i - t * half;
  double s, c;
  sincos((double)pos[t] * freq[k], &s, &c);
  out[(size_t)t * 2 * half + k] = (float)(c * mult);
  out[(size_t)t * 2 * half + half + k] = (float)(s * mult);
}

struct StoreArgs {
  int S, ld;
  size_t slab;
  const float* cs;        // [T, r]
  const int* slots;
  const float* wn;        // [R] or null: no latent in the projection
  int H, d, r, R, d8, r8, R8, D, log2BS;
  float eps;
  const float* wq;        // [Rq] or null: a query latent ahead of the latent, H = 0
  int Rq;
};

// grid (token, y): y < ny: 256 V-element items of the query heads; y == ny: the latent row; y > ny: the
// query latent, normed, to q
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
  auto normed = [&](const PT* x, int R, const float* wn, T* o) {
    float f[NI][V];
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < NI; ++n) {
      const int c = (tid + 256 * n) * V;
      if (c < R) {
        ld_slabs<V>(x + c, a.S, a.slab, f[n]);
#pragma unroll
        for (int j = 0; j < V; ++j) ss += f[n][j] * f[n][j];
      }
    }
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)R + a.eps);
#pragma unroll
    for (int n = 0; n < NI; ++n) {
      const int c = (tid + 256 * n) * V;
      if (c < R) {
        float w[V];
        ldv<V>(wn + c, w);
#pragma unroll
        for (int j = 0; j < V; ++j) f[n][j] *= inv * w[j];
        stv<V>(o + c, f[n]);
      }
    }
  };
  if ((int)blockIdx.y > ny) {
    normed(p, a.Rq, a.wq, q + (size_t)t * a.Rq);
    return;
  }
  const int slot = a.slots[t];
  if (slot < 0) return;                                  // the whole workgroup
  // one KV head: row = slot of the paged cache
  T* o = cache + (size_t)slot * a.D;
  const PT* x = p + a.H * (a.d + a.r) + a.Rq;
  normed(x, a.R, a.wn, o);
  for (int i = tid; i < half / V; i += 256) rotate(x + a.R, o + a.R8, i * V);
  if (V == 1) {
    for (int i = tid; i < a.R8 - a.R; i += 256) st1(o + a.R + i, 0.f);
    for (int i = tid; i < a.r8 - a.r; i += 256) st1(o + a.R8 + a.r + i, 0.f);
  }
}

// ------------------------------------------------------------------ per-head products
// y[t, h, :N] = x[t, h, :K] . w[h]^T; y[t, h, N : N + E] = x[t, h, K : K + E].  One workgroup:
// 16 MT rows of one head, 64 NJ outputs; x rows staged in LDS, w straight to registers.  MERGE: the
// rows are attended latents as key splits' outputs, x = sum_s w_s part_s, w_s = e^(m_s - m) l_s / sum.
constexpr int kMaxSplit = 32;

template <int MT, int NJ, bool MERGE, bool GATE>
__global__ __launch_bounds__(256) void head_project_kernel(const uint16_t* __restrict__ x,
                                                           const uint16_t* __restrict__ part,
                                                           const float2* __restrict__ ml, int nsplit,
                                                           const uint16_t* __restrict__ w, uint16_t* __restrict__ y,
                                                           int T, int H, int K, int N, int E, DocqaGate gate) {
  extern __shared__ __attribute__((aligned(16))) uint16_t sx[];       // [16 MT][pitch]
  __shared__ float sw[MERGE ? 16 * MT : 1][kMaxSplit];                // a row's weight of each split
  const int kp = (K + 31) / 32 * 32, pitch = kp + 8;
  const int h = blockIdx.x, m0 = blockIdx.y * 16 * MT, tid = threadIdx.x;
  const int ldx = H * (K + E), ldy = H * (N + E);
  const uint16_t* xh = x + (size_t)h * (K + E);
  uint16_t* yh = y + (size_t)h * (N + E);
  const int per = kp / 8;
  if constexpr (MERGE) {
    const size_t all = (size_t)T * H;
    static_assert(kMaxSplit == 32, "a row's splits in 32 lanes");
    for (int i = tid >> 5; i < 16 * MT; i += 8) {
      const size_t row = (size_t)min(m0 + i, T - 1) * H + h;
      const int s = tid & 31;
      const float2 v = s < nsplit ? ml[s * all + row] : make_float2(-1e30f, 0.f);
      const float m = group_max<32>(v.x);
      const float e = v.y > 0.f ? __builtin_amdgcn_exp2f(v.x - m) * v.y : 0.f;       // 0: nothing seen, nothing written
      const float l = group_sum<32>(e);
      sw[i][s] = l > 0.f ? e / l : 0.f;
    }
    __syncthreads();
    for (int i = tid; i < 16 * MT * per; i += 256) {
      const int r = i / per, c = (i - r * per) * 8;
      float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (m0 + r < T && c < K) {
        const uint16_t* p = part + ((size_t)(m0 + r) * H + h) * K + c;
        for (int s0 = 0; s0 < nsplit; s0 += 4) {         // four at a time: past the last, weight 0
          float g[4][8];
#pragma unroll
          for (int u = 0; u < 4; ++u) ldv<8>(p + min(s0 + u, nsplit - 1) * all * K, g[u]);
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            const float e = sw[r][s0 + u];
#pragma unroll
            for (int j = 0; j < 8; ++j) f[j] += e > 0.f ? e * g[u][j] : 0.f;   // (not written: any bits)
          }
        }
      }
      stv<8>(sx + r * pitch + c, f);
    }
  } else {
    for (int i = tid; i < 16 * MT * per; i += 256) {
      const int r = i / per, c = (i - r * per) * 8;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (m0 + r < T && c < K) v = *reinterpret_cast<const uint4*>(xh + (size_t)(m0 + r) * ldx + c);
      *reinterpret_cast<uint4*>(sx + r * pitch + c) = v;
    }
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
  const int n0 = (blockIdx.z * 4 + wave) * 16 * NJ;                   // this wave's first output
  if (n0 >= N) return;
  f32x4 acc[MT][NJ];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NJ; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const uint16_t* wh = w + (size_t)h * N * K;
#pragma unroll 8
  for (int k = 0; k < kp; k += 32) {
    const int kk = k + g4 * 8;
    bf16x8 wf[NJ], xf[MT];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
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
      for (int j = 0; j < NJ; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[j], xf[i], acc[i][j], 0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int row = m0 + i * 16 + fr;
    if (row >= T) continue;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int n = n0 + 16 * j + g4 * 4;
      uint16_t* op = yh + (size_t)row * ldy + n;
      if (N % 4 == 0) {
        if (n < N) {
          float f[4] = {acc[i][j][0], acc[i][j][1], acc[i][j][2], acc[i][j][3]};
          if constexpr (GATE) apply_gate<4>(gate, row, h * N + n, f);
          stv<4>(op, f);
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (n + r < N) {
            float f = acc[i][j][r];
            if constexpr (GATE) apply_gate<1>(gate, row, h * N + n + r, &f);
            op[r] = f2bf(f);
          }
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

// ------------------------------------------------------------------ attention, latent space
typedef __attribute__((address_space(3))) i16x4 lds_i16x4;
constexpr int KB = 64;        // keys of a tile: 16 per wave of S^T
constexpr int kMaxBT = 256;   // block ids staged in LDS at a time

struct LatentArgs {
  const uint16_t* q;      // [tokens, H, D]
  const uint16_t* kc;     // paged rows [slots, D]
  uint16_t* out;          // [tokens, H, DV]
  const int* bt;
  int maxb;
  const int* cu;          // null: decode
  const int* ctx;
  const float* sink;
  uint16_t* part;         // [nsplit, tokens H, DV] each split's output, null: one split
  float2* ml;             // [nsplit, tokens H] (row maximum, row sum)
  int tokens, H, D, DV, log2BS, nsplit, window;
  float scale;
};

// grid (row tiles, sequences, key splits)
template <int DPV, int DPK, int QT, int NW>
__global__ __launch_bounds__(64 * NW) void latent_attn_kernel(LatentArgs a) {
  constexpr int PITCH = DPK + 8, NKS = DPK / 32, RW = 16 * QT, PP = KB + 8;
  // a tile's 16-byte pieces: the first DPV columns a wave takes RPI rows at a time, the other 64
  // eight rows at a time
  static_assert(DPK == DPV + 64, "row layout");
  constexpr int LPR = DPV / 8, RPI = 64 / LPR, NL = KB / RPI / NW, NE = KB / 8 / NW;
  constexpr int QTW = QT / (NW / 4);           // row tiles whose scores this wave makes
  constexpr int NDT = DPV / 16 / NW;           // 16-column tiles of its slice of the output
  static_assert(NW % 4 == 0 && QTW >= 1 && NDT >= 1 && LPR <= 64 && NL >= 1 && NE >= 1, "wave roles");
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* tiles = reinterpret_cast<uint16_t*>(smem);                  // [2][KB][PITCH]
  uint16_t* sp = tiles + 2 * KB * PITCH;                                // [RW][PP]
  float* smax = reinterpret_cast<float*>(sp + RW * PP);                 // [4][RW]
  __shared__ int s_bt[kMaxBT];

  const int b = blockIdx.y, split = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, fr = lane & 15, g4 = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  int q0, L, p0;
  if (a.cu) {
    q0 = a.cu[b];
    L = a.cu[b + 1] - q0;
    p0 = a.ctx[b];
  } else {
    q0 = b;
    L = 1;
    p0 = a.ctx[b] - 1;
  }
  const int row0 = (gridDim.x - 1 - blockIdx.x) * RW, rows = L * a.H;   // longest windows first
  if (row0 >= rows) return;
  const size_t grow0 = (size_t)q0 * a.H;                                // first row of the sequence
  const size_t all = (size_t)a.tokens * a.H;
  const int nrow = min(RW, rows - row0);
  if (p0 < 0) {                                                         // a padded decode row
    if (a.nsplit == 1) {
      for (int e = tid; e < nrow * a.DV; e += 64 * NW) a.out[(grow0 + row0) * a.DV + e] = 0;
    } else {
      for (int r = tid; r < nrow; r += 64 * NW) a.ml[split * all + grow0 + row0 + r] = make_float2(-1e30f, 0.f);
    }
    return;
  }
  const int pos_lo = p0 + row0 / a.H, pos_hi = p0 + (row0 + nrow - 1) / a.H;
  const int key0 = a.window > 0 ? max(0, pos_lo - a.window + 1) : 0;
  const int ntiles = (pos_hi - key0) / KB + 1, per = (ntiles + a.nsplit - 1) / a.nsplit;
  const int t0 = split * per, t1 = min(ntiles, t0 + per);
  if (t0 >= t1) {                                                       // more splits than tiles
    for (int r = tid; r < nrow; r += 64 * NW) a.ml[split * all + grow0 + row0 + r] = make_float2(-1e30f, 0.f);
    return;
  }
  const int last = min(pos_hi, key0 + t1 * KB - 1);
  int blk0 = (key0 + t0 * KB) >> a.log2BS;               // first staged block id
  auto stage_blocks = [&]() {
    const int n = min(kMaxBT, (last >> a.log2BS) - blk0 + 1);
    for (int i = tid; i < n; i += 64 * NW) s_bt[i] = a.bt[(size_t)b * a.maxb + blk0 + i];
    __syncthreads();
  };
  stage_blocks();

  // Every load of a tile issues without a branch: keys past the end repeat the last one (their
  // scores are masked), columns past the row repeat its first (the query is zero there, the
  // output is dropped).
  const int lrow = lane / LPR, c0 = (lane % LPR) * 8, cl = c0 < a.D ? c0 : 0;       // first columns
  const int erow = lane >> 3, e0 = DPV + (lane & 7) * 8, ce = e0 < a.D ? e0 : 0;    // the others
  auto cached = [&](int key) {                           // element offset of a key's row
    const int blk = s_bt[(key >> a.log2BS) - blk0];
    return (((size_t)blk << a.log2BS) + (key & ((1 << a.log2BS) - 1))) * a.D;
  };
  auto load = [&](int t, u32x4 (&rk)[NL + NE]) {
    const int kb = key0 + t * KB;
    if ((min(kb + KB - 1, last) >> a.log2BS) - blk0 >= kMaxBT) {       // the whole workgroup
      lds_barrier();
      blk0 = kb >> a.log2BS;
      stage_blocks();
    }
#pragma unroll
    for (int i = 0; i < NL; ++i)
      rk[i] = *reinterpret_cast<const u32x4*>(a.kc + cached(min(kb + (i * NW + wave) * RPI + lrow, last)) + cl);
#pragma unroll
    for (int i = 0; i < NE; ++i)
      rk[NL + i] = *reinterpret_cast<const u32x4*>(a.kc + cached(min(kb + (i * NW + wave) * 8 + erow, last)) + ce);
  };
  auto store = [&](int buf, const u32x4 (&rk)[NL + NE]) {
    uint16_t* k = tiles + buf * KB * PITCH;
#pragma unroll
    for (int i = 0; i < NL; ++i)
      *reinterpret_cast<u32x4*>(k + ((i * NW + wave) * RPI + lrow) * PITCH + c0) = rk[i];
#pragma unroll
    for (int i = 0; i < NE; ++i)
      *reinterpret_cast<u32x4*>(k + ((i * NW + wave) * 8 + erow) * PITCH + e0) = rk[NL + i];
  };
  // the query rows come through LDS (a wave's fragments are 16 rows wide: read directly, every wave
  // of a row tile would fetch 16 cache lines an instruction)
  constexpr int QL = (RW + RPI * NW - 1) / (RPI * NW), QE = (RW + 8 * NW - 1) / (8 * NW);
  u32x4 rq[QL + QE], rk[NL + NE], rk2[NL + NE];
  const u32x4 zero = {0, 0, 0, 0};
#pragma unroll
  for (int i = 0; i < QL; ++i) {
    const int r = min(row0 + (i * NW + wave) * RPI + lrow, rows - 1);
    rq[i] = *reinterpret_cast<const u32x4*>(a.q + (grow0 + r) * a.D + cl);
  }
#pragma unroll
  for (int i = 0; i < QE; ++i) {
    const int r = min(row0 + (i * NW + wave) * 8 + erow, rows - 1);
    rq[QL + i] = *reinterpret_cast<const u32x4*>(a.q + (grow0 + r) * a.D + ce);
  }
  load(t0, rk);
  if (t0 + 1 < t1) load(t0 + 1, rk2);
  uint16_t* sq = tiles + KB * PITCH;                     // [RW][PITCH], where tile t0 + 1 goes next
#pragma unroll
  for (int i = 0; i < QL; ++i) {
    const int r = (i * NW + wave) * RPI + lrow;
    if (r < RW) *reinterpret_cast<u32x4*>(sq + r * PITCH + c0) = c0 < a.D ? rq[i] : zero;
  }
#pragma unroll
  for (int i = 0; i < QE; ++i) {
    const int r = (i * NW + wave) * 8 + erow;
    if (r < RW) *reinterpret_cast<u32x4*>(sq + r * PITCH + e0) = e0 < a.D ? rq[QL + i] : zero;
  }
  lds_barrier();

  const int ksub = wave & 3, rg = (wave >> 2) * QTW;     // this wave's keys of a tile / first row tile
  bf16x8 qf[QTW][NKS];
  int pos[QTW], below[QTW];                              // a row sees keys in (below, pos]
#pragma unroll
  for (int t = 0; t < QTW; ++t) {
    const int r = min(row0 + (rg + t) * 16 + fr, rows - 1);
    pos[t] = p0 + r / a.H;
    below[t] = a.window > 0 ? pos[t] - a.window : -1;
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks)
      qf[t][ks] = *reinterpret_cast<const bf16x8*>(sq + ((rg + t) * 16 + fr) * PITCH + ks * 32 + g4 * 8);
  }
  lds_barrier();
  // the sink is the sum's first term: the maximum starts there in every wave, the sum in one
  float m[QT], l[QTW];
  f32x4 o[QT][NDT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int r = min(row0 + t * 16 + fr, rows - 1);
    m[t] = a.sink && split == 0 ? a.sink[r % a.H] * kLog2e : -1e30f;
#pragma unroll
    for (int i = 0; i < NDT; ++i) o[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll
  for (int t = 0; t < QTW; ++t) l[t] = a.sink && split == 0 && ksub == 0 && g4 == 0 ? 1.f : 0.f;
  const float sl2 = a.scale * kLog2e;
  const int tq = fr >> 2, tp = fr & 3;

  store(0, rk);
  if (t0 + 1 < t1) store(1, rk2);
  u32x4 rn[NL + NE];                                     // the tile after next, in flight for a tile's work
  if (t0 + 2 < t1) load(t0 + 2, rn);
  lds_barrier();
  for (int t = t0; t < t1; ++t) {
    const int buf = (t - t0) & 1, kb = key0 + t * KB;
    const uint16_t* sk = tiles + buf * KB * PITCH;
    f32x4 x[QTW];
#pragma unroll
    for (int i = 0; i < QTW; ++i) x[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks) {
      const bf16x8 kf = *reinterpret_cast<const bf16x8*>(sk + (ksub * 16 + fr) * PITCH + ks * 32 + g4 * 8);
#pragma unroll
      for (int i = 0; i < QTW; ++i) x[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[i][ks], x[i], 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < QTW; ++i) {
      float mx = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = kb + ksub * 16 + g4 * 4 + r;
        const float v = ((key <= pos[i]) & (key > below[i])) ? x[i][r] * sl2 : -INFINITY;
        x[i][r] = v;
        mx = fmaxf(mx, v);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (g4 == 0) smax[ksub * RW + (rg + i) * 16 + fr] = mx;
    }
    lds_barrier();                                       // maxima; every wave is past the last tile
    float alpha[QT];
#pragma unroll
    for (int i = 0; i < QT; ++i) {
      float mn = m[i];
#pragma unroll
      for (int k = 0; k < 4; ++k) mn = fmaxf(mn, smax[k * RW + i * 16 + fr]);
      alpha[i] = __builtin_amdgcn_exp2f(m[i] - mn);
      m[i] = mn;
    }
#pragma unroll
    for (int i = 0; i < QTW; ++i) {
      const float mn = NW == 4 ? m[i] : (rg == 0 ? m[i] : m[(QTW + i) % QT]);
      const float al = NW == 4 ? alpha[i] : (rg == 0 ? alpha[i] : alpha[(QTW + i) % QT]);
      float p[4], rs = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        p[r] = __builtin_amdgcn_exp2f(x[i][r] - mn);
        rs += p[r];
      }
      l[i] = l[i] * al + rs;
      stv<4>(sp + ((rg + i) * 16 + fr) * PP + ksub * 16 + g4 * 4, p);
    }
    if (t > t0 && t + 1 < t1) store(buf ^ 1, rn);
    if (t > t0 && t + 2 < t1) load(t + 2, rn);
    lds_barrier();                                       // scores, next tile
#pragma unroll
    for (int i = 0; i < QT; ++i)
#pragma unroll
      for (int n = 0; n < NDT; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[i][n][r] *= alpha[i];
#pragma unroll
    for (int s = 0; s < KB / 32; ++s) {
      bf16x8 pb[QT];
#pragma unroll
      for (int i = 0; i < QT; ++i) {
        const uint16_t* pr = sp + (i * 16 + fr) * PP + s * 32 + g4 * 4;
        uint2 lo = *reinterpret_cast<const uint2*>(pr), hi = *reinterpret_cast<const uint2*>(pr + 16);
        uint4 v = make_uint4(lo.x, lo.y, hi.x, hi.y);
        pb[i] = *reinterpret_cast<bf16x8*>(&v);
      }
      const uint16_t* vr = sk + (s * 32 + g4 * 4 + tq) * PITCH + wave * NDT * 16 + 4 * tp;
#pragma unroll
      for (int n = 0; n < NDT; ++n) {
        const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + n * 16));
        const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + 16 * PITCH + n * 16));
        bf16x8 vf;
        const __bf16* lp = reinterpret_cast<const __bf16*>(&lo);
        const __bf16* hp = reinterpret_cast<const __bf16*>(&hi);
#pragma unroll
        for (int j = 0; j < 4; ++j) { vf[j] = lp[j]; vf[4 + j] = hp[j]; }
#pragma unroll
        for (int i = 0; i < QT; ++i) o[i][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pb[i], o[i][n], 0, 0, 0);
      }
    }
  }
  // row sums: over a wave's key groups, then over the four key waves of the row
#pragma unroll
  for (int i = 0; i < QTW; ++i) {
    l[i] += __shfl_xor(l[i], 16, 64);
    l[i] += __shfl_xor(l[i], 32, 64);
    if (g4 == 0) smax[ksub * RW + (rg + i) * 16 + fr] = l[i];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < QT; ++i) {
    const int r = i * 16 + fr;
    if (r >= nrow) continue;
    const float sum = (smax[r] + smax[RW + r]) + (smax[2 * RW + r] + smax[3 * RW + r]);
    const size_t row = grow0 + row0 + r;
    const float inv = sum > 0.f ? 1.f / sum : 0.f;
    if (a.nsplit > 1 && wave == 0 && g4 == 0) a.ml[split * all + row] = make_float2(m[i], sum);
#pragma unroll
    for (int n = 0; n < NDT; ++n) {
      const int c = wave * NDT * 16 + n * 16 + g4 * 4;
      if (c >= a.DV) continue;
      const float f[4] = {o[i][n][0] * inv, o[i][n][1] * inv, o[i][n][2] * inv, o[i][n][3] * inv};
      stv<4>(a.nsplit > 1 ? a.part + (split * all + row) * a.DV + c : a.out + row * a.DV + c, f);
    }
  }
}

template <int DPV, int QT, int NW>
int launch_latent(const LatentArgs& a, int B, int max_q, hipStream_t s) {
  constexpr int DPK = DPV + 64, RW = 16 * QT;
  constexpr size_t lds = (size_t)2 * KB * (DPK + 8) * 2 + (size_t)RW * (KB + 8) * 2 + (size_t)4 * RW * 4;
  static_assert(lds + kMaxBT * 4 <= 160 * 1024 && RW <= KB, "LDS");
  const long long nz = ((long long)max_q * a.H + RW - 1) / RW;
  if (nz >= (1ll << 31) || B > 65535) return -1;
  auto kern = latent_attn_kernel<DPV, DPK, QT, NW>;
  if constexpr (lds > 64 * 1024) {
    static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  kern<<<dim3((unsigned)nz, B, a.nsplit), 64 * NW, lds, s>>>(a);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

// row tiles of a workgroup by the rows a sequence has
template <int DPV>
int dispatch_latent(const LatentArgs& a, int B, int max_q, hipStream_t s) {
  const long long rows = (long long)max_q * a.H;
  constexpr int NW = DPV >= 128 ? 8 : 4;
  if (rows <= 16) return launch_latent<DPV, 1, 4>(a, B, max_q, s);
  if (DPV > 256 || rows <= 32) return launch_latent<DPV, 2, NW>(a, B, max_q, s);
  if constexpr (DPV <= 256) return launch_latent<DPV, 4, NW>(a, B, max_q, s);
  return -1;
}

template <typename PT, typename T>
int store_types(const void* P, void* q, void* cache, int T_, const StoreArgs& a, hipStream_t s) {
  const bool v4 = a.d % 8 == 0 && a.r % 8 == 0 && a.R % 8 == 0 && a.Rq % 8 == 0 && a.ld % 4 == 0;
  // many tokens: 16-byte pieces of bf16 rows
  const bool v8 = v4 && T_ >= 256 && sizeof(T) == 2 && a.r % 16 == 0 && a.ld % 8 == 0;
  const int V = v8 ? 8 : v4 ? 4 : 1;
  const int per = a.d / V + a.r / 2 / V + (v4 ? 0 : a.d8 - a.d + a.r8 - a.r);
  const int ny = (a.H * per + 255) / 256;
  dim3 grid(T_, ny + (a.wn ? 1 : 0) + (a.wq ? 1 : 0));
  if (v8) latent_store_kernel<8, 1, PT, T><<<grid, 256, 0, s>>>((const PT*)P, (T*)q, (T*)cache, ny, a);
  else if (v4) latent_store_kernel<4, 2, PT, T><<<grid, 256, 0, s>>>((const PT*)P, (T*)q, (T*)cache, ny, a);
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

int docqa_rope_table(const int* positions, const double* freq, float* out, int T, int half, double mult, hipStream_t s) {
  if (T == 0) return 0;
  if (half < 1 || (long long)T * half >= (1ll << 31)) return -1;
  rope_table_kernel<<<(T * half + 255) / 256, 256, 0, s>>>(positions, freq, out, T, half, mult);
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
              log2_of(BS), eps, nullptr, 0};
  a.D = a.R8 + a.r8;
  if (f32) return store_types<float, float>(P, q, cache, T, a, s);
  return p_f32 ? store_types<float, uint16_t>(P, q, cache, T, a, s)
               : store_types<uint16_t, uint16_t>(P, q, cache, T, a, s);
}

int docqa_latent_norm_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* cs, const int* slots,
                            const float* q_norm, const float* c_norm, void* cq, void* cache, int f32, int T, int Rq, int r,
                            int R, int BS, float eps, hipStream_t s) {
  if (T == 0) return 0;
  if (S < 1 || r < 2 || r % 2 || R < 1 || R > 2048 || Rq < 1 || Rq > 2048 || !q_norm || !c_norm || (BS & (BS - 1)) != 0) return -1;
  if (ld < Rq + R + r || (f32 && !p_f32)) return -1;
  StoreArgs a{S, ld, slab, cs, slots, c_norm, 0, 0, r, R, 0, (r + 7) / 8 * 8, (R + 7) / 8 * 8, 0, log2_of(BS), eps, q_norm, Rq};
  a.D = a.R8 + a.r8;
  if (f32) return store_types<float, float>(P, cq, cache, T, a, s);
  return p_f32 ? store_types<float, uint16_t>(P, cq, cache, T, a, s)
               : store_types<uint16_t, uint16_t>(P, cq, cache, T, a, s);
}

int docqa_head_project(const void* x, const void* part, const void* ml, int nsplit, const void* w, void* y, int T, int H,
                       int K, int N, int E, const DocqaGate& gate, hipStream_t s) {
  if (T == 0) return 0;
  if (gate.P && (E > 0 || (N % 4 == 0 && !docqa_gate_vec(gate, 4)))) return -1;
  if (H < 1 || K < 8 || K % 8 || K > 2048 || N < 1 || E < 0 || E % 8 || (E > 0 && N % 8)) return -1;
  if (!docqa_aligned16(w) || !docqa_aligned16(y) || !docqa_aligned16(part ? part : x)) return -1;
  if (part && (!ml || nsplit < 1 || nsplit > kMaxSplit || E > 0)) return -1;
  const int pitch = (K + 31) / 32 * 32 + 8;
#define LAUNCH(MT, NJ, MERGE, GATE)                                                                                         \
  do {                                                                                                                \
    const size_t lds = (size_t)16 * MT * pitch * 2;                                                                   \
    auto kern = head_project_kernel<MT, NJ, MERGE, GATE>;                                                                   \
    if (lds > 56 * 1024) {                                                                                            \
      static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern),                            \
                                                      hipFuncAttributeMaxDynamicSharedMemorySize, 80 * 1024);         \
      if (e != hipSuccess) return (int)e;                                                                             \
    }                                                                                                                 \
    kern<<<dim3(H, (T + 16 * MT - 1) / (16 * MT), (N + 64 * NJ - 1) / (64 * NJ)), 256, lds, s>>>(                     \
        (const uint16_t*)x, (const uint16_t*)part, (const float2*)ml, nsplit, (const uint16_t*)w, (uint16_t*)y, T, H, K, N, E, gate);  \
  } while (0)
#define GO(MT, NJ)                       \
  do {                                   \
    if (part && gate.P) LAUNCH(MT, NJ, true, true);  \
    else if (part) LAUNCH(MT, NJ, true, false);      \
    else if (gate.P) LAUNCH(MT, NJ, false, true);    \
    else LAUNCH(MT, NJ, false, false);               \
  } while (0)
  if (T > 64 && K <= 256) GO(4, 2);
  else if (T > 64 && K <= 1024) GO(2, 2);
  else GO(1, 1);
#undef GO
#undef LAUNCH
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

int docqa_latent_attn_ok(int D, int DV) { return D % 8 == 0 && DV % 8 == 0 && DV <= 512 && D > DV && D <= (DV <= 64 ? 128 : DV <= 128 ? 192 : DV <= 256 ? 320 : 576); }

// Key splits: enough workgroups for every CU; two tiles each unless there are few sequences
int docqa_latent_splits(int B, int max_q, int H, int DV, int max_keys) {
  const long long rows = (long long)max_q * H;
  const int rw = rows <= 16 ? 16 : (DV > 256 || rows <= 32) ? 32 : 64;
  const long long wgs = (long long)B * ((rows + rw - 1) / rw);
  const int tiles = (max_keys + KB - 1) / KB + 1;
  const long long n = wgs > 0 ? 256 / wgs : 1;
  int most = n >= 8 ? tiles : tiles / 2;
  if (most > kMaxSplit) most = kMaxSplit;
  return n < 1 || most < 1 ? 1 : (int)(n < most ? n : most);
}

int docqa_latent_attn(const void* q, const void* kc, const int* block_tables, int maxb, const int* cu, const int* ctx,
                      const float* sink, void* out, void* part, void* ml, int nsplit, int B, int max_q, int tokens, int H,
                      int D, int DV, int BS, float scale, int window, hipStream_t s) {
  if (B == 0 || max_q == 0 || tokens == 0) return 0;
  if (!docqa_latent_attn_ok(D, DV) || H < 1 || (BS & (BS - 1)) != 0 || nsplit < 1 || nsplit > 65535) return -1;
  if (nsplit > 1 && (!part || !ml)) return -1;
  if (!docqa_aligned16(q) || !docqa_aligned16(kc) || !docqa_aligned16(out)) return -1;
  const LatentArgs a{(const uint16_t*)q, (const uint16_t*)kc, (uint16_t*)out, block_tables, maxb, cu, ctx, sink, (uint16_t*)part,
                     (float2*)ml, tokens, H, D, DV, log2_of(BS), nsplit, window, scale};
  if (DV <= 64) return dispatch_latent<64>(a, B, max_q, s);
  if (DV <= 128) return dispatch_latent<128>(a, B, max_q, s);
  if (DV <= 256) return dispatch_latent<256>(a, B, max_q, s);
  return dispatch_latent<512>(a, B, max_q, s);
}
