// attn_window.hip -- causal attention over a sliding window with an optional per-head sink,
// read from the paged cache; head-wise query / key RMS norm; keys shared as values.
//
//   s_j = cap(scale * k_scale_j * (q . K_j))   for  pos - window < j <= pos,  cap(s) = c tanh(s / c)
//   out = out_scale * sum_j exp(s_j) V_j / (sum_j exp(s_j) + exp(sink_h))
//
// * qkv_rope_store: [q | k | v] projection -> query heads (bias, norm, rotation of the first r
//   dimensions), keys alike and values into the paged cache; key and value rows may differ in size.
// * qk_norm_store: q <- rms(q) * w over each head, K rows stored as projected with their
//   inverse root mean square beside them (k_scale).  With the key norm's weight folded into
//   w the normalised key is never materialised: one cached row serves as key and as value,
//   half the bytes of a K / V pair.
// * window <= 0: no window; sink null: none; k_scale null: 1; V may be the K cache itself, or the
//   first DV elements of its rows (latent attention; its MFMA form is attn_latent.hip).
// * packed keys (latent attention over prompts): per-head keys and values of the visible rows in
//   one matrix, a key part all heads share in another, instead of the paged cache.
// * prefill (several query tokens a sequence) and decode (one) share the kernels: bf16 heads of
//   up to 256 elements run on MFMA, fp32 and odd head sizes on a wave-per-row kernel.
#include "docqa_common.h"
#include "docqa_elem.h"
#include "docqa_gate.h"
#include <float.h>
#include <type_traits>

using namespace docqa;

namespace {
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kMaxBT = 256;   // block ids of a row tile's keys staged in LDS (else read per tile)

// LPH lanes per (token, head), V elements a lane at a time; heads [0, H) are queries,
// [H, H + G) keys
template <int V, int NI, int LPH, typename PT, typename T>
__global__ __launch_bounds__(256) void qk_norm_store_kernel(const PT* __restrict__ P, int S, size_t slab, int ld,
                                                            const float* __restrict__ wq,
                                                            const int* __restrict__ slot_mapping, T* __restrict__ q,
                                                            T* __restrict__ kc, float* __restrict__ ks, int tokens,
                                                            int H, int G, int D, int log2BS, float eps) {
  const int heads = H + G;
  const unsigned u = blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  const int lane = threadIdx.x % LPH, t = u / heads, h = u - t * heads;
  if (t >= tokens) return;                 // whole lane groups
  const PT* p = P + (size_t)t * ld + (size_t)h * D;
  float x[NI][V];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (lane + LPH * i) * V;
    if (c < D) {
      ld_slabs<V>(p + c, S, slab, x[i]);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        if (h >= H) x[i][j] = rnd((const T*)nullptr, x[i][j]);   // the scale belongs to the stored row
        ss += x[i][j] * x[i][j];
      }
    }
  }
  const float inv = 1.f / sqrtf(group_sum<LPH>(ss) / (float)D + eps);
  if (h < H) {
    T* o = q + ((size_t)t * H + h) * D;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (lane + LPH * i) * V;
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
    const size_t row = ((((size_t)(slot >> log2BS)) * G + (h - H)) << log2BS) + (slot & ((1 << log2BS) - 1));
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (lane + LPH * i) * V;
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
  int H, G, D, BS, log2BS;
  float scale;
  int window;
  int DV;                 // value elements of a head
  int ldv;                // elements of a cached value row (D where the keys are the values)
  float cap;              // 0: none
  float out_scale;
  int ldo;                // elements of an output row
  // packed keys: row j of sequence b at cu_k[b] + j holds [H x kd | H x vd ..] (ld elements), the
  // other D - kd key elements at kr; the last query token is at the last key
  const int* cu_k;
  const uint16_t* kr;
  int ld, kd, vd;
  DocqaGate gate;         // packed form
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

// the same over packed keys: positions count from the sequence's first visible key
__device__ __forceinline__ bool packed_range(const WindowArgs& a, int b, int& q0, int& L, int& p0) {
  q0 = a.cu[b];
  L = a.cu[b + 1] - q0;
  p0 = a.cu_k[b + 1] - a.cu_k[b] - L;
  return L > 0 && p0 >= 0;
}

// Any head size and element type: one wave per (token, head).  64 keys at a time, one per
// lane for the scores, then the lanes run over the value's elements.
template <typename T, int NI>
__global__ __launch_bounds__(256) void window_attn_kernel(const T* __restrict__ q, const T* __restrict__ kc,
                                                          const T* __restrict__ vc, T* __restrict__ out,
                                                          WindowArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sq_all[];      // [4][D]
  __shared__ float sp[4][64];
  __shared__ int srow[4][64];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int b = blockIdx.y, u = blockIdx.x * 4 + wave;
  const int tok = u / a.H, h = u % a.H;
  int q0 = 0, L = 0, p0 = 0;
  const bool live = seq_range(a, b, q0, L, p0);
  if (tok >= (a.cu ? L : 1)) return;       // whole waves; no workgroup barrier below
  const int D = a.D, DV = a.DV;
  T* o = out + (size_t)(q0 + tok) * a.ldo + h * DV;
  if (!live) {                             // a padded decode row
    for (int c = lane; c < DV; c += 64) st1(o + c, 0.f);
    return;
  }
  float* sq = sq_all + wave * D;
  const int g = h / (a.H / a.G), pos = p0 + tok;
  const T* qp = q + ((size_t)(q0 + tok) * a.H + h) * D;
  for (int c = lane; c < D; c += 64) sq[c] = ld1(qp + c);
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
      const int blk = a.block_tables[(size_t)b * a.maxb + (key >> a.log2BS)];
      row = ((blk * a.G + g) << a.log2BS) + (key & (a.BS - 1));
      const T* kp = kc + (size_t)row * D;
      float d0 = 0.f, d1 = 0.f;
      int c = 0;
      if (D % 8 == 0) {
        for (; c < D; c += 8) {
          float f[8];
          ldv<8>(kp + c, f);
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            d0 += f[j] * sq[c + j];
            d1 += f[4 + j] * sq[c + 4 + j];
          }
        }
      } else {
        for (; c < D; ++c) d0 += ld1(kp + c) * sq[c];
      }
      s = (d0 + d1) * sl2 * (a.k_scale ? a.k_scale[row] : 1.f);
      if (a.cap > 0.f) s = a.cap * kLog2e * tanhf(s / (a.cap * kLog2e));
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
      if (c < DV) {
        float v = acc[i] * alpha;
        for (int j = 0; j < n; ++j) v += sp[wave][j] * ld1(vc + (size_t)srow[wave][j] * a.ldv + c);
        acc[i] = v;
      }
    }
    wave_lds_sync();
  }
  const float inv = a.out_scale / l;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = lane + 64 * i;
    if (c < DV) st1(o + c, acc[i] * inv);
  }
}

// ---- MFMA form (bf16, head sizes that are multiples of 8) ---------------------------------
// Query rows are (token, head of the GQA group) pairs, so any group size fills the 16-row MFMA
// tiles.  S^T = K Q^T on v_mfma_f32_16x16x32_bf16: a lane holds one query row's scores of
// 4 keys per 16-key sub-tile, so the online softmax is in-lane plus two cross-group shuffles,
// and the scores turned bf16 are the B operand of O^T += V^T P^T as they are (the key order of
// a k-step is the accumulators': keys 4g..4g+3 of two sub-tiles for lane group g).  V^T comes
// from the row-major tile by transposing LDS reads -- from the K tile itself when the keys are
// the values.  Tile rows are padded by 16 bytes: conflict-free for both read patterns.
//   SPLIT = false: 4 waves, each 16 QT rows of its own, one double-buffered K (V) tile for all;
//   SPLIT = true (few rows, decode): NW waves take every NW-th key tile of the same rows, each
//   with a private LDS tile, and merge at the end.
typedef __attribute__((address_space(3))) i16x4 lds_i16x4;

// PACKED: keys and values from packed matrices (WindowArgs::cu_k) instead of the paged cache.
template <int DP, int DPV, int QT, int KB, int NW, bool SHARED, bool SPLIT, bool PACKED = false>
__global__ __launch_bounds__(64 * NW, NW == 4 ? 2 : 1) void window_attn_mfma_kernel(const uint16_t* __restrict__ q,
                                                                   const uint16_t* __restrict__ kc,
                                                                   const uint16_t* __restrict__ vc,
                                                                   uint16_t* __restrict__ out, WindowArgs a) {
  static_assert(!SHARED || DP == DPV, "shared rows");
  static_assert(!PACKED || ((KB * DP / 8) % (64 * NW) == 0 && (KB * DPV / 8) % (64 * NW) == 0), "packed loads");
  constexpr int PITCH = DP + 8, PITCHV = DPV + 8, NCH = DP / 8, NCV = DPV / 8, NKT = KB / 16, NKS = DP / 32,
                NDT = DPV / 16;
  constexpr int TILES = SPLIT ? NW : 2;
  constexpr int KTILE = KB * PITCH, TILE = KTILE + (SHARED ? 0 : KB * PITCHV);    // elements of one buffer
  constexpr int LOADERS = SPLIT ? 64 : 64 * NW;                     // threads staging one tile
  constexpr int CPT = (KB * NCH + LOADERS - 1) / LOADERS, CPV = (KB * NCV + LOADERS - 1) / LOADERS;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* tiles = reinterpret_cast<uint16_t*>(smem);
  float* scales = reinterpret_cast<float*>(tiles + TILES * TILE);   // [TILES][KB]
  __shared__ int s_bt[kMaxBT];              // block ids of the keys the rows see

  const int kvh = blockIdx.x, b = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int fr = lane & 15, g4 = lane >> 4;
  int q0 = 0, L = 0, p0 = 0;
  const bool live = PACKED ? packed_range(a, b, q0, L, p0) : seq_range(a, b, q0, L, p0);
  const int Gs = PACKED ? 1 : a.H / a.G, D = a.D, DV = a.DV;
  constexpr int RW = 16 * QT;
  const int tile_rows = SPLIT ? RW : RW * NW;
  const int row0 = (gridDim.z - 1 - blockIdx.z) * tile_rows;         // longest windows first
  if (!live) {                                                       // a padded decode row
    if (!a.cu)
      for (int e = tid; e < Gs * DV; e += 64 * NW) out[(size_t)b * a.ldo + kvh * Gs * DV + e] = 0;
    return;
  }
  const int rows = L * Gs;
  if (row0 >= rows) return;
  const int wrow = row0 + (SPLIT ? 0 : wave * RW);                   // first row of this wave
  // positions the workgroup's rows / this wave's rows span
  const int pos_lo = p0 + row0 / Gs, pos_hi = p0 + (min(row0 + tile_rows, rows) - 1) / Gs;
  const int wpos_lo = p0 + min(wrow, rows - 1) / Gs, wpos_hi = p0 + (min(wrow + RW, rows) - 1) / Gs;
  const bool wlive = wrow < rows;
  const int key0 = a.window > 0 ? max(0, pos_lo - a.window + 1) : 0;
  const int ntiles = (pos_hi - key0) / KB + 1;

  const int blk0 = key0 >> a.log2BS, nblk = (pos_hi >> a.log2BS) - blk0 + 1;
  const bool bt_lds = nblk <= kMaxBT;
  const int kbase = PACKED ? a.cu_k[b] : 0;
  if (!PACKED && bt_lds) {
    for (int i = tid; i < nblk; i += 64 * NW) s_bt[i] = a.block_tables[(size_t)b * a.maxb + blk0 + i];
    __syncthreads();
  }

  bf16x8 qf[QT][NKS];
  int pos[QT], below[QT];                  // a row sees keys in (below, pos]
  float m[QT], l[QT];
  f32x4 o[QT][NDT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int r = wrow + t * 16 + fr, rc = min(r, rows - 1);
    const int tok = rc / Gs, h = kvh * Gs + rc % Gs;
    pos[t] = p0 + tok;
    below[t] = a.window > 0 ? pos[t] - a.window : -1;
    const uint16_t* qp = q + ((size_t)(q0 + tok) * a.H + h) * D;
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks) {
      const int c = ks * 32 + g4 * 8;
      uint4 v = c < D ? *reinterpret_cast<const uint4*>(qp + c) : make_uint4(0, 0, 0, 0);
      qf[t][ks] = *reinterpret_cast<bf16x8*>(&v);
    }
    // the sink: one more exponential in the denominator (in one wave only when they split)
    const bool sk = a.sink && (!SPLIT || wave == 0);
    m[t] = sk ? a.sink[h] * kLog2e : -1e30f;
    l[t] = sk ? 1.f : 0.f;
#pragma unroll
    for (int i = 0; i < NDT; ++i) o[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float sl2 = a.scale * kLog2e;

  const int ltid = SPLIT ? lane : tid;
  // packed: every thread's pieces of a tile start at fixed pointers, a row apart by a fixed stride, and
  // load without a branch: keys past the end repeat the last one (masked), columns past a row its first
  const uint16_t *kp[PACKED ? CPT : 1], *vp[PACKED ? CPV : 1];
  size_t kst[PACKED ? CPT : 1];
  if constexpr (PACKED) {
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c0 = ((ltid + LOADERS * i) % NCH) * 8, c = c0 < D ? c0 : 0;
      kp[i] = c < a.kd ? kc + (size_t)kvh * a.kd + c : a.kr + (c - a.kd);
      kst[i] = c < a.kd ? a.ld : D - a.kd;
    }
#pragma unroll
    for (int i = 0; i < CPV; ++i) {
      const int c = ((ltid + LOADERS * i) % NCV) * 8;
      vp[i] = vc + (size_t)kvh * a.vd + (c < a.vd ? c : 0);
    }
  }
  u32x4 rk[CPT], rv[SHARED ? 1 : CPV];
  float rs_ = 1.f;
  auto cache_row = [&](int key) {
    const int kblk = key >> a.log2BS;
    const int blk = bt_lds ? s_bt[kblk - blk0] : a.block_tables[(size_t)b * a.maxb + kblk];
    return (size_t)((((blk * a.G + kvh) << a.log2BS)) + (key & (a.BS - 1)));
  };
  auto load = [&](int t) {
    const int kb = key0 + t * KB;
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int e = ltid + LOADERS * i, row = e / NCH, c = (e % NCH) * 8;
      if constexpr (PACKED) {
        rk[i] = *reinterpret_cast<const u32x4*>(kp[i] + (kbase + min(kb + row, pos_hi)) * kst[i]);
      } else {
        rk[i] = u32x4{0, 0, 0, 0};
        if (e < KB * NCH && kb + row <= pos_hi && c < D)
          rk[i] = *reinterpret_cast<const u32x4*>(kc + cache_row(kb + row) * D + c);
      }
    }
    if constexpr (!SHARED) {
#pragma unroll
      for (int i = 0; i < CPV; ++i) {
        const int e = ltid + LOADERS * i, row = e / NCV, c = (e % NCV) * 8;
        if constexpr (PACKED) {
          rv[i] = *reinterpret_cast<const u32x4*>(vp[i] + (size_t)(kbase + min(kb + row, pos_hi)) * a.ld);
        } else {
          rv[i] = u32x4{0, 0, 0, 0};
          if (e < KB * NCV && kb + row <= pos_hi && c < DV)
            rv[i] = *reinterpret_cast<const u32x4*>(vc + cache_row(kb + row) * DV + c);
        }
      }
    }
    if (ltid < KB) {
      const int key = kb + ltid;
      rs_ = (a.k_scale && key <= pos_hi) ? a.k_scale[cache_row(key)] * sl2 : sl2;
    }
  };
  auto store = [&](int buf) {
    uint16_t* k = tiles + buf * TILE;
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int e = ltid + LOADERS * i, row = e / NCH, c = (e % NCH) * 8;
      if (e < KB * NCH) {
        *reinterpret_cast<u32x4*>(k + row * PITCH + c) = rk[i];
      }
    }
    if constexpr (!SHARED) {
#pragma unroll
      for (int i = 0; i < CPV; ++i) {
        const int e = ltid + LOADERS * i, row = e / NCV, c = (e % NCV) * 8;
        if (e < KB * NCV) *reinterpret_cast<u32x4*>(k + KTILE + row * PITCHV + c) = rv[i];
      }
    }
    if (ltid < KB) scales[buf * KB + ltid] = rs_;
  };
  // one key tile against this wave's rows; `part`: some of its keys are hidden from some rows
  auto compute_tile = [&](int kb, int buf, auto part) {
    constexpr bool PART = decltype(part)::value;
    const uint16_t* sk = tiles + buf * TILE;
    const uint16_t* sv = SHARED ? sk : sk + KTILE;
    const float* sc = scales + buf * KB;
    f32x4 x[QT][NKT];
#pragma unroll
    for (int kt = 0; kt < NKT; ++kt) {
#pragma unroll
      for (int t2 = 0; t2 < QT; ++t2) x[t2][kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NKS; ++ks) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(sk + (kt * 16 + fr) * PITCH + ks * 32 + g4 * 8);
#pragma unroll
        for (int t2 = 0; t2 < QT; ++t2)
          x[t2][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[t2][ks], x[t2][kt], 0, 0, 0);
      }
    }
    const float cap2 = a.cap * kLog2e;
#pragma unroll
    for (int t2 = 0; t2 < QT; ++t2) {
      float mx = -INFINITY;
#pragma unroll
      for (int kt = 0; kt < NKT; ++kt) {
        const float4 ks4 = *reinterpret_cast<const float4*>(sc + kt * 16 + g4 * 4);
        const float kss[4] = {ks4.x, ks4.y, ks4.z, ks4.w};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float v = x[t2][kt][r] * kss[r];
          // cap tanh(v / cap), tanh y = 1 - 2 / (e^2y + 1)
          if (cap2 > 0.f) v = cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(v * (2.f * kLog2e / cap2)) + 1.f);
          if constexpr (PART) {
            const int key = kb + kt * 16 + g4 * 4 + r;
            v = ((key <= pos[t2]) & (key > below[t2])) ? v : -INFINITY;
          }
          x[t2][kt][r] = v;
          mx = fmaxf(mx, v);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m[t2], mx);
      const float alpha = __builtin_amdgcn_exp2f(m[t2] - mn);
      float rs = 0.f;
#pragma unroll
      for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = __builtin_amdgcn_exp2f(x[t2][kt][r] - mn);
          x[t2][kt][r] = p;
          rs += p;
        }
      rs += __shfl_xor(rs, 16, 64);
      rs += __shfl_xor(rs, 32, 64);
      l[t2] = l[t2] * alpha + rs;
      m[t2] = mn;
#pragma unroll
      for (int i = 0; i < NDT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[t2][i][r] *= alpha;
    }
    const int tq = fr >> 2, tp = fr & 3;
#pragma unroll
    for (int s = 0; s < NKT / 2; ++s) {
      bf16x8 pb[QT];
#pragma unroll
      for (int t2 = 0; t2 < QT; ++t2)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          pb[t2][j] = (__bf16)x[t2][2 * s][j];
          pb[t2][4 + j] = (__bf16)x[t2][2 * s + 1][j];
        }
      const uint16_t* vr = sv + (s * 32 + g4 * 4 + tq) * PITCHV + 4 * tp;
#pragma unroll
      for (int i = 0; i < NDT; ++i) {
        const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + i * 16));
        const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + 16 * PITCHV + i * 16));
        bf16x8 vf;
        const __bf16* lp = reinterpret_cast<const __bf16*>(&lo);
        const __bf16* hp = reinterpret_cast<const __bf16*>(&hi);
#pragma unroll
        for (int j = 0; j < 4; ++j) { vf[j] = lp[j]; vf[4 + j] = hp[j]; }
#pragma unroll
        for (int t2 = 0; t2 < QT; ++t2)
          o[t2][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pb[t2], o[t2][i], 0, 0, 0);
      }
    }
  };

  auto compute = [&](int t, int buf) {
    const int kb = key0 + t * KB;
    if (!wlive || kb > wpos_hi || (a.window > 0 && kb + KB - 1 <= wpos_lo - a.window)) return;
    if (kb + KB - 1 <= wpos_lo && (a.window <= 0 || kb > wpos_hi - a.window))
      compute_tile(kb, buf, std::false_type{});
    else
      compute_tile(kb, buf, std::true_type{});
  };

  if constexpr (!SPLIT) {
    load(0);
    store(0);
    __syncthreads();
    for (int t = 0; t < ntiles; ++t) {
      if (t + 1 < ntiles) load(t + 1);
      compute(t, t & 1);
      if (t + 1 < ntiles) store((t + 1) & 1);    // last read one iteration (one barrier) ago
      __syncthreads();
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      const int r = wrow + t * 16 + fr;
      if (r >= rows) continue;
      uint16_t* op = out + (size_t)(q0 + r / Gs) * a.ldo + (kvh * Gs + r % Gs) * DV;
      const float inv = a.out_scale / l[t];
#pragma unroll
      for (int i = 0; i < NDT; ++i) {
        const int c = i * 16 + g4 * 4;
        if (c < DV) {
          float f[4] = {o[t][i][0] * inv, o[t][i][1] * inv, o[t][i][2] * inv, o[t][i][3] * inv};
          if constexpr (PACKED) {
            if (a.gate.P) apply_gate<4>(a.gate, q0 + r, kvh * DV + c, f);
          }
          stv<4>(op + c, f);
        }
      }
    }
  } else {
    static_assert(QT == 1 || !SPLIT, "split rows: one 16-row tile");
    if (wave < ntiles) load(wave);
    for (int t = wave; t < ntiles; t += NW) {
      wave_lds_sync();                           // this wave's reads of the tile are done
      store(wave);
      wave_lds_sync();
      if (t + NW < ntiles) load(t + NW);
      compute(t, wave);
    }
    __syncthreads();                             // tiles dead: partials [NW][16][DPV] + (m, l)
    constexpr int OP = DPV + 4;
    float* po = reinterpret_cast<float*>(smem);
    float2* pml = reinterpret_cast<float2*>(po + NW * 16 * OP);
#pragma unroll
    for (int i = 0; i < NDT; ++i)
      *reinterpret_cast<float4*>(po + (wave * 16 + fr) * OP + i * 16 + g4 * 4) =
          make_float4(o[0][i][0], o[0][i][1], o[0][i][2], o[0][i][3]);
    if (g4 == 0) pml[wave * 16 + fr] = make_float2(m[0], l[0]);
    __syncthreads();
    const int n = min(16, rows - row0);
    for (int e = tid; e < n * (DPV / 4); e += 64 * NW) {
      const int r = e / (DPV / 4), c = (e % (DPV / 4)) * 4;
      if (c >= DV) continue;
      float mm = -1e30f;
#pragma unroll
      for (int w = 0; w < NW; ++w) mm = fmaxf(mm, pml[w * 16 + r].x);
      float ll = 0.f;
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        const float2 ml = pml[w * 16 + r];
        const float f = __builtin_amdgcn_exp2f(ml.x - mm);
        const float4 p = *reinterpret_cast<const float4*>(po + (w * 16 + r) * OP + c);
        ll += ml.y * f;
        v.x += p.x * f; v.y += p.y * f; v.z += p.z * f; v.w += p.w * f;
      }
      const float inv = a.out_scale / ll;
      uint2 w2;
      w2.x = pack2(v.x * inv, v.y * inv);
      w2.y = pack2(v.z * inv, v.w * inv);
      const int row = row0 + r;
      *reinterpret_cast<uint2*>(out + (size_t)(q0 + row / Gs) * a.ldo + (kvh * Gs + row % Gs) * DV + c) = w2;
    }
  }
}

template <int DP, int DPV, int QT, int KB, int NW, bool SHARED, bool SPLIT, bool PACKED = false>
int launch_mfma(const void* q, const void* kc, const void* vc, void* out, const WindowArgs& a, int B, int max_q,
                hipStream_t s) {
  constexpr int TILES = SPLIT ? NW : 2;
  constexpr size_t tile_b = (size_t)TILES * KB * (DP + 8 + (SHARED ? 0 : DPV + 8)) * 2 + (size_t)TILES * KB * 4;
  constexpr size_t merge_b = SPLIT ? (size_t)NW * 16 * (DPV + 4) * 4 + (size_t)NW * 16 * 8 : 0;
  constexpr size_t lds = tile_b > merge_b ? tile_b : merge_b;
  static_assert(lds <= 160 * 1024, "LDS");
  const int tile_rows = 16 * QT * (SPLIT ? 1 : NW), Gs = PACKED ? 1 : a.H / a.G;
  const long long nz = ((long long)max_q * Gs + tile_rows - 1) / tile_rows;
  if (nz > 65535) return -1;
  auto kern = window_attn_mfma_kernel<DP, DPV, QT, KB, NW, SHARED, SPLIT, PACKED>;
  if constexpr (lds > 64 * 1024) {
    static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  kern<<<dim3(PACKED ? a.H : a.G, B, (int)nz), 64 * NW, lds, s>>>((const uint16_t*)q, (const uint16_t*)kc, (const uint16_t*)vc,
                                                   (uint16_t*)out, a);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

// decode-like launches (the rows of one sequence fit one 16-row tile): waves split the keys, as
// many to a workgroup as give a CU 16 of them
template <int DP, int DPV, bool SHARED>
int dispatch_mfma(const void* q, const void* kc, const void* vc, void* out, const WindowArgs& a, int B, int max_q,
                  hipStream_t s) {
  constexpr int QT = DP <= 128 && DPV <= 128 ? 2 : 1;
  if (max_q * (a.H / a.G) <= 16) {
    if constexpr (DP <= 128 && DPV <= 128) {
      const long long wgs = (long long)B * a.G;
      if constexpr (SHARED) {
        if (wgs <= 256) return launch_mfma<DP, DPV, 1, 32, 16, SHARED, true>(q, kc, vc, out, a, B, max_q, s);
      }
      if (wgs <= 512) return launch_mfma<DP, DPV, 1, 32, 8, SHARED, true>(q, kc, vc, out, a, B, max_q, s);
    }
    return launch_mfma<DP, DPV, 1, 32, 4, SHARED, true>(q, kc, vc, out, a, B, max_q, s);
  }
  return launch_mfma<DP, DPV, QT, 64, 4, SHARED, false>(q, kc, vc, out, a, B, max_q, s);
}

int dispatch_shared(const void* q, const void* kc, void* out, const WindowArgs& a, int B, int max_q, hipStream_t s) {
#define GO(N) return dispatch_mfma<N, N, true>(q, kc, kc, out, a, B, max_q, s)
  if (a.D <= 32) GO(32);
  if (a.D <= 64) GO(64);
  if (a.D <= 96) GO(96);
  if (a.D <= 128) GO(128);
  if (a.D <= 192) GO(192);
  GO(256);
#undef GO
}
// key and value rows of their own
template <int DP>
int dispatch_values(const void* q, const void* kc, const void* vc, void* out, const WindowArgs& a, int B, int max_q,
                    hipStream_t s) {
  if (a.DV <= 64) return dispatch_mfma<DP, 64, false>(q, kc, vc, out, a, B, max_q, s);
  if (a.DV <= 128) return dispatch_mfma<DP, 128, false>(q, kc, vc, out, a, B, max_q, s);
  return dispatch_mfma<DP, 256, false>(q, kc, vc, out, a, B, max_q, s);
}
int dispatch_pair(const void* q, const void* kc, const void* vc, void* out, const WindowArgs& a, int B, int max_q,
                  hipStream_t s) {
  if (a.D <= 64) return dispatch_values<64>(q, kc, vc, out, a, B, max_q, s);
  if (a.D <= 128) return dispatch_values<128>(q, kc, vc, out, a, B, max_q, s);
  return dispatch_values<256>(q, kc, vc, out, a, B, max_q, s);
}

// heads of a [q: H D | k: G D | v: G DV] projection, LPH lanes each: bias, RMS norm and rotation of
// query and key heads, V items of two kinds -- V pairs (i, i + r / 2) of the rotated dimensions, V
// unrotated ones -- then the stores; value heads are copied
struct QkvArgs {
  int S, ld;
  size_t slab;
  const float* bias;      // [H D + G D + G DV] or null
  const float *qw, *kw;   // [D] or null: no norm
  const float* cs;        // [tokens, r]: cosines, sines
  const int* slots;
  int tokens, H, G, D, DV, r, log2BS;
  float eps;
};
template <int V, int NI, int LPH, typename PT, typename T>
__global__ __launch_bounds__(256) void qkv_rope_store_kernel(const PT* __restrict__ P, T* __restrict__ q,
                                                             T* __restrict__ kc, T* __restrict__ vc, QkvArgs a) {
  const int heads = a.H + 2 * a.G;
  const unsigned u = blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  const int lane = threadIdx.x % LPH, t = u / heads, h = u - t * heads;
  if (t >= a.tokens) return;                 // whole lane groups
  const PT* row = P + (size_t)t * a.ld;
  const int D = a.D, r2 = a.r / 2, slot = h < a.H ? 0 : a.slots[t];
  if (slot < 0) return;
  const int BS = 1 << a.log2BS;
  auto cache_row = [&](int g) { return ((((size_t)(slot >> a.log2BS)) * a.G + g) << a.log2BS) + (slot & (BS - 1)); };
  auto get = [&](int c, float* f) {
    ld_slabs<V>(row + c, a.S, a.slab, f);
    if (a.bias) {
      float b[V];
      ldv<V>(a.bias + c, b);
#pragma unroll
      for (int j = 0; j < V; ++j) f[j] += b[j];
    }
  };
  if (h >= a.H + a.G) {
    const int g = h - a.H - a.G, c0 = (a.H + a.G) * D + g * a.DV;
    T* o = vc + cache_row(g) * a.DV;
    for (int c = lane * V; c < a.DV; c += LPH * V) {
      float f[V];
      get(c0 + c, f);
      stv<V>(o + c, f);
    }
    return;
  }
  const int items = (D - r2) / V, npair = r2 / V;
  float x[NI][V], y[NI][V], ss = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int e = lane + LPH * i;
    if (e < items) {
      const int c = e < npair ? e * V : e * V + r2;
      get(h * D + c, x[i]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += x[i][j] * x[i][j];
      if (e < npair) {
        get(h * D + c + r2, y[i]);
#pragma unroll
        for (int j = 0; j < V; ++j) ss += y[i][j] * y[i][j];
      }
    }
  }
  const float* w = h < a.H ? a.qw : a.kw;
  const float inv = w ? 1.f / sqrtf(group_sum<LPH>(ss) / (float)D + a.eps) : 1.f;
  T* o = h < a.H ? q + ((size_t)t * a.H + h) * D : kc + cache_row(h - a.H) * D;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int e = lane + LPH * i;
    if (e >= items) continue;
    const int c = e < npair ? e * V : e * V + r2;
    float f[V];
    if (w) {
      ldv<V>(w + c, f);
#pragma unroll
      for (int j = 0; j < V; ++j) x[i][j] *= inv * f[j];
    }
    if (e < npair) {
      float co[V], si[V];
      if (w) {
        ldv<V>(w + c + r2, f);
#pragma unroll
        for (int j = 0; j < V; ++j) y[i][j] *= inv * f[j];
      }
      ldv<V>(a.cs + (size_t)t * a.r + c, co);
      ldv<V>(a.cs + (size_t)t * a.r + r2 + c, si);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float xu = x[i][j], xv = y[i][j];
        x[i][j] = xu * co[j] - xv * si[j];
        y[i][j] = xv * co[j] + xu * si[j];
      }
      stv<V>(o + c + r2, y[i]);
    }
    stv<V>(o + c, x[i]);
  }
}

template <typename PT, typename T>
int qkv_store(const PT* P, T* q, T* kc, T* vc, const QkvArgs& a, hipStream_t s) {
  const long long units = (long long)a.tokens * (a.H + 2 * a.G);
#define GO(V, N, L) qkv_rope_store_kernel<V, N, L, PT, T><<<(int)((units + 256 / L - 1) / (256 / L)), 256, 0, s>>>(P, q, kc, vc, a)
  const int items = a.D - a.r / 2;
  if (a.D % 4 == 0 && a.DV % 4 == 0 && a.r % 8 == 0 && a.ld % 4 == 0) {
    if (items <= 32) GO(4, 1, 8);
    else if (items <= 64) GO(4, 1, 16);
    else if (items <= 128) GO(4, 1, 32);
    else GO(4, 2, 64);
  } else {
    if (items <= 64) GO(1, 1, 64);
    else if (items <= 128) GO(1, 2, 64);
    else GO(1, 8, 64);
  }
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <typename PT, typename T>
int qk_store(const PT* P, int S, size_t slab, int ld, const float* wq, const int* sm, T* q, T* kc, float* ks,
             int tokens, int H, int G, int D, int BS, float eps, hipStream_t s) {
  int log2BS = 0;
  while ((1 << log2BS) < BS) ++log2BS;
#define GO(V, N, L)                                                                                        \
  qk_norm_store_kernel<V, N, L, PT, T><<<(int)(((long long)tokens * (H + G) + 256 / L - 1) / (256 / L)), 256, 0, s>>>( \
      P, S, slab, ld, wq, sm, q, kc, ks, tokens, H, G, D, log2BS, eps)
  if (D % 8 == 0 && ld % 8 == 0) {
    if (D <= 64) GO(8, 1, 8);
    else if (D <= 128) GO(8, 1, 16);
    else if (D <= 256) GO(8, 1, 32);
    else GO(8, 1, 64);
  } else {
    if (D <= 64) GO(1, 1, 64);
    else if (D <= 128) GO(1, 2, 64);
    else GO(1, 8, 64);
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
  if (S < 1 || D < 1 || D > 512 || H < 1 || G < 1 || ld < (H + G) * D || (BS & (BS - 1)) != 0) return -1;
  if ((long long)tokens * (H + G) >= (1ll << 31)) return -1;
  if (f32) {
    if (!p_f32) return -1;
    return qk_store((const float*)P, S, slab, ld, wq, slots, (float*)q, (float*)kc, ks, tokens, H, G, D, BS, eps, s);
  }
  if (p_f32)
    return qk_store((const float*)P, S, slab, ld, wq, slots, (uint16_t*)q, (uint16_t*)kc, ks, tokens, H, G, D, BS, eps, s);
  return qk_store((const uint16_t*)P, S, slab, ld, wq, slots, (uint16_t*)q, (uint16_t*)kc, ks, tokens, H, G, D, BS, eps, s);
}

int docqa_qkv_rope_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* bias, const float* qw,
                         const float* kw, const float* cs, int r, const int* slots, void* q, void* kc, void* vc, int f32,
                         int tokens, int H, int G, int D, int DV, int BS, float eps, hipStream_t s) {
  if (tokens == 0) return 0;
  if (S < 1 || D < 1 || D > 512 || DV < 1 || H < 1 || G < 1 || r < 0 || r % 2 || r > D || (BS & (BS - 1)) != 0) return -1;
  if (ld < (H + G) * D + G * DV || (long long)tokens * (H + 2 * G) >= (1ll << 31) || (f32 && !p_f32)) return -1;
  QkvArgs a{S, ld, slab, bias, qw, kw, cs, slots, tokens, H, G, D, DV, r, 0, eps};
  while ((1 << a.log2BS) < BS) ++a.log2BS;
  if (f32) return qkv_store((const float*)P, (float*)q, (float*)kc, (float*)vc, a, s);
  if (p_f32) return qkv_store((const float*)P, (uint16_t*)q, (uint16_t*)kc, (uint16_t*)vc, a, s);
  return qkv_store((const uint16_t*)P, (uint16_t*)q, (uint16_t*)kc, (uint16_t*)vc, a, s);
}

int docqa_window_attn(const void* q, const void* kc, const void* vc, const float* k_scale, const int* block_tables,
                      int maxb, const int* cu, const int* ctx, const float* sink, void* out, int ldo, int f32, int B,
                      int max_q, int H, int G, int D, int DV, int BS, float scale, int window, float cap, float out_scale,
                      hipStream_t s) {
  if (B == 0 || max_q == 0) return 0;
  const bool shared = kc == vc;
  if (H % G != 0 || D < 1 || D > 2560 || DV < 1 || (shared && DV > D) || DV > 2048 || (BS & (BS - 1)) != 0) return -1;
  if (ldo < H * DV || cap < 0.f) return -1;
  int log2BS = 0;
  while ((1 << log2BS) < BS) ++log2BS;
  const WindowArgs a{block_tables, maxb, cu, ctx, k_scale, sink, H, G, D, BS, log2BS, scale, window, DV,
                     shared ? D : DV, cap, out_scale, ldo, nullptr, nullptr, 0, 0, 0, {}};
  // rows are stored 8 bytes at a time
  const bool stores = ldo % 4 == 0 && DV % 4 == 0 && (reinterpret_cast<uintptr_t>(out) & 7) == 0;
  if (!f32 && D % 8 == 0 && DV % 8 == 0 && D <= 256 && DV <= 256 && (!shared || DV == D) && docqa_aligned16(q) && stores)
    return shared ? dispatch_shared(q, kc, out, a, B, max_q, s) : dispatch_pair(q, kc, vc, out, a, B, max_q, s);
  dim3 grid((max_q * H + 3) / 4, B);
#define GO(T, N) window_attn_kernel<T, N><<<grid, 256, (size_t)D * 16, s>>>((const T*)q, (const T*)kc, (const T*)vc, (T*)out, a)
  if (f32) {
    if (DV <= 64) GO(float, 1);
    else if (DV <= 128) GO(float, 2);
    else if (DV <= 256) GO(float, 4);
    else if (DV <= 512) GO(float, 8);
    else GO(float, 32);
  } else {
    if (DV <= 64) GO(uint16_t, 1);
    else if (DV <= 128) GO(uint16_t, 2);
    else if (DV <= 256) GO(uint16_t, 4);
    else if (DV <= 512) GO(uint16_t, 8);
    else GO(uint16_t, 32);
  }
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_packed_window_attn(const void* q, const void* kv, const void* kr, const int* cu, const int* cu_k,
                             const float* sink, void* out, int B, int max_q, int H, int d8, int r8, int vdim, int ld,
                             float scale, int window, const DocqaGate& gate, hipStream_t s) {
  if (B == 0 || max_q == 0) return 0;
  if (gate.P && !docqa_gate_vec(gate, 4)) return -1;
  const int D = d8 + r8, v8 = (vdim + 7) / 8 * 8;
  if (H < 1 || d8 < 8 || d8 % 8 || r8 < 0 || r8 % 8 || D > 256 || vdim < 4 || vdim % 4 || vdim > 256) return -1;
  if (ld % 8 || ld < H * (d8 + v8) || B > 65535) return -1;
  if (!docqa_aligned16(q) || !docqa_aligned16(kv) || !docqa_aligned16(kr) || !docqa_aligned16(out)) return -1;
  const WindowArgs a{nullptr, 0, cu, nullptr, nullptr, sink, H, H, D, 64, 6, scale, window, vdim, 0, 0.f, 1.f, H * vdim,
                     cu_k, (const uint16_t*)kr, ld, d8, v8, gate};
  const uint16_t* v = (const uint16_t*)kv + (size_t)H * d8;
  // 128 query rows a workgroup, 64 where that leaves CUs without one, or (no window: the last rows see
  // all keys, the first few) without a second one to even out their work
  const bool few = (long long)B * H * ((max_q + 127) / 128) < (window > 0 ? 384 : 640);
#define RUN(DP, DPV, QT, KB) return launch_mfma<DP, DPV, QT, KB, 4, false, false, true>(q, kv, v, out, a, B, max_q, s)
#define GO(DP, DPV, KB)               \
  do {                                \
    if (few) RUN(DP, DPV, 1, KB);     \
    RUN(DP, DPV, 2, KB);              \
  } while (0)
  if (D <= 64 && vdim <= 64) GO(64, 64, 64);
  if (D <= 96 && vdim <= 64) GO(96, 64, 64);
  if (D <= 128 && vdim <= 128) GO(128, 128, 64);
  if (D <= 192 && vdim <= 128) GO(192, 128, 32);
  RUN(256, 256, 1, 32);
#undef GO
#undef RUN
}
