// side_input.hip -- a layer's input from the token's side embedding:
//   g = gelu_tanh(P) * e,  e = table[id][col, col + n)   and, fused, y = g . w^T
// P is the gate projection [M, N] (a product or split-K slabs), N >= n with padded columns zero.
//
//   * side_gate: g alone (prompts: g feeds a prefill GEMM);
//   * side_project: one workgroup per 16 MT rows x 64 NC outputs builds g of its rows in LDS (the
//     slab sum, the activation and the embedding row never reach HBM) and multiplies it with
//     w [W, N] on MFMA.  N is small, so the weight goes straight to registers.
#include "docqa_common.h"
#include "docqa_elem.h"

using namespace docqa;

namespace {
template <int V, typename PT, typename ET>
__device__ __forceinline__ void gate(const PT* P, int S, size_t slab, int M, int N, int t, int c,
                                     const int* __restrict__ ids, const ET* __restrict__ table, int ld, int vocab,
                                     int col, int n, float* g) {
  float e[V];
  const ET* ep = table + (size_t)min(max(ids[t], 0), vocab - 1) * ld + col;
  if (V > 1 && c + V <= n) {
    ldv<V>(ep + c, e);
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) e[j] = c + j < n ? ld1(ep + c + j) : 0.f;
  }
  ld_slabs<V>(P + (size_t)t * N + c, S, slab, g);
#pragma unroll
  for (int j = 0; j < V; ++j) g[j] = gelu_tanh(g[j]) * e[j];
}

template <int V, typename PT, typename T>
__global__ __launch_bounds__(256) void side_gate_kernel(const PT* __restrict__ P, int S, int M, int N,
                                                        const int* __restrict__ ids, const T* __restrict__ table,
                                                        int ld, int vocab, int col, int n, T* __restrict__ out) {
  const int per = N / V;
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long long)M * per) return;
  const int t = (int)(i / per), c = (int)(i - (long long)t * per) * V;
  float g[V];
  gate<V>(P, S, (size_t)M * N, M, N, t, c, ids, table, ld, vocab, col, n, g);
  stv<V>(out + (size_t)t * N + c, g);
}

template <int V, int MT, int NC, typename PT>
__global__ __launch_bounds__(256) void side_project_kernel(const PT* __restrict__ P, int S, int M, int N,
                                                           const int* __restrict__ ids,
                                                           const uint16_t* __restrict__ table, int ld, int vocab,
                                                           int col, int n, const uint16_t* __restrict__ w, int W,
                                                           uint16_t* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) uint16_t sg[];       // [16 MT][pitch]
  const int kp = (N + 31) / 32 * 32, pitch = kp + 8;
  const int m0 = blockIdx.y * 16 * MT, tid = threadIdx.x;
  const int per = kp / V;
  for (int i = tid; i < 16 * MT * per; i += 256) {
    const int r = i / per, c = (i - r * per) * V;
    float g[V];
    if (m0 + r < M && c < N) {
      gate<V>(P, S, (size_t)M * N, M, N, m0 + r, c, ids, table, ld, vocab, col, n, g);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) g[j] = 0.f;
    }
    stv<V>(sg + r * pitch + c, g);
  }
  __syncthreads();
  const int lane = tid & 63, wave = tid >> 6, fr = lane & 15, g4 = lane >> 4;
  f32x4 acc[MT][NC];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NC; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int o0 = blockIdx.x * 64 * NC + wave * 16;                    // this wave's columns: o0 + 64 j + fr
  for (int k = 0; k < kp; k += 32) {
    const int kk = k + g4 * 8;
    bf16x8 wf[NC], xf[MT];
#pragma unroll
    for (int j = 0; j < NC; ++j) {
      const int o = o0 + 64 * j + fr;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (o < W && kk < N) v = *reinterpret_cast<const uint4*>(w + (size_t)o * N + kk);
      wf[j] = *reinterpret_cast<bf16x8*>(&v);
    }
#pragma unroll
    for (int i = 0; i < MT; ++i) xf[i] = *reinterpret_cast<const bf16x8*>(sg + (i * 16 + fr) * pitch + kk);
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < NC; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[j], xf[i], acc[i][j], 0, 0, 0);
  }
  // lane: row fr of the tile, outputs 4 g4 .. 4 g4 + 3
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int row = m0 + i * 16 + fr;
    if (row >= M) continue;
#pragma unroll
    for (int j = 0; j < NC; ++j) {
      const int o = o0 + 64 * j + g4 * 4;
      uint16_t* op = out + (size_t)row * W + o;
      if (W % 4 == 0) {
        if (o < W) {
          const float f[4] = {acc[i][j][0], acc[i][j][1], acc[i][j][2], acc[i][j][3]};
          stv<4>(op, f);
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (o + r < W) op[r] = f2bf(acc[i][j][r]);
      }
    }
  }
}

template <typename PT, typename T>
int gate_types(const void* P, int S, int M, int N, const int* ids, const void* table, int ld, int vocab, int col, int n,
               void* out, hipStream_t s) {
  const bool v4 = N % 4 == 0 && ld % 4 == 0 && col % 4 == 0;
  const long long items = (long long)M * (v4 ? N / 4 : N);
  if ((items + 255) / 256 >= (1ll << 31)) return -1;
  const int grid = (int)((items + 255) / 256);
  if (v4)
    side_gate_kernel<4, PT, T><<<grid, 256, 0, s>>>((const PT*)P, S, M, N, ids, (const T*)table, ld, vocab, col, n, (T*)out);
  else
    side_gate_kernel<1, PT, T><<<grid, 256, 0, s>>>((const PT*)P, S, M, N, ids, (const T*)table, ld, vocab, col, n, (T*)out);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <int V, typename PT>
int launch_project(const PT* P, int S, int M, int N, const int* ids, const uint16_t* table, int ld, int vocab, int col,
                   int n, const uint16_t* w, int W, uint16_t* out, hipStream_t s) {
  const int pitch = (N + 31) / 32 * 32 + 8;
  constexpr int MT = 1, NC = 2;
  side_project_kernel<V, MT, NC, PT><<<dim3((W + 64 * NC - 1) / (64 * NC), (M + 16 * MT - 1) / (16 * MT)), 256,
                                       (size_t)16 * MT * pitch * 2, s>>>(P, S, M, N, ids, table, ld, vocab, col, n, w, W, out);
  DOCQA_CHECK_LAUNCH();
  return 0;
}
}  // namespace

int docqa_side_gate(const void* P, int p_f32, int S, int M, int N, const int* ids, const void* table, int f32, int ld,
                    int vocab, int col, int n, void* out, hipStream_t s) {
  if (M == 0 || N == 0) return 0;
  if (S < 1 || n < 0 || n > N || col < 0 || col + n > ld || vocab < 1 || (f32 && !p_f32)) return -1;
  if (f32) return gate_types<float, float>(P, S, M, N, ids, table, ld, vocab, col, n, out, s);
  return p_f32 ? gate_types<float, uint16_t>(P, S, M, N, ids, table, ld, vocab, col, n, out, s)
               : gate_types<uint16_t, uint16_t>(P, S, M, N, ids, table, ld, vocab, col, n, out, s);
}

int docqa_side_project(const void* P, int p_f32, int S, int M, int N, const int* ids, const void* table, int ld,
                       int vocab, int col, int n, const void* w, int W, void* out, hipStream_t s) {
  if (M == 0 || W == 0) return 0;
  if (S < 1 || N < 8 || N % 8 || N > 1024 || n < 0 || n > N || col < 0 || col + n > ld || vocab < 1) return -1;
  if (!docqa_aligned16(w) || !docqa_aligned16(P) || !docqa_aligned16(out)) return -1;
  const bool v4 = ld % 4 == 0 && col % 4 == 0;
  const uint16_t *t = (const uint16_t*)table, *wp = (const uint16_t*)w;
  uint16_t* o = (uint16_t*)out;
  if (p_f32)
    return v4 ? launch_project<4>((const float*)P, S, M, N, ids, t, ld, vocab, col, n, wp, W, o, s)
              : launch_project<1>((const float*)P, S, M, N, ids, t, ld, vocab, col, n, wp, W, o, s);
  return v4 ? launch_project<4>((const uint16_t*)P, S, M, N, ids, t, ld, vocab, col, n, wp, W, o, s)
            : launch_project<1>((const uint16_t*)P, S, M, N, ids, t, ld, vocab, col, n, wp, W, o, s);
}
