// ssm.hip -- recurrent mixers: a short causal convolution per channel and the selective scan
// (Mamba, Gu & Dao 2023), each as a prefill kernel over packed sequences and a decode step.
//
//   conv:  y[t, c] = act(b[c] + sum_k w[k, c] x[t - (taps - 1) + k, c]), act silu or none
//   scan:  dt = softplus(dt_pre + dt_b);  S[c, n] <- 2^(dt A2[c, n]) S[c, n] + dt x B[n]
//          y = (sum_n S[c, n] C[n] + D x) silu(z)           A2 = -exp(A_log) log2(e)
//
// Per sequence the state pool holds (slot = one live request):
//   conv state [slots, taps - 1, C]  the last inputs, oldest first, in the compute dtype
//   scan state [slots, C, Np]        fp32, Np = N rounded up to 4 (padding stays zero)
// A sequence whose first token is position 0 starts from zero whatever its slot held, so a
// slot needs no clearing when it changes hands.
//
// MI355X mapping of the scan: one lane owns one or two channels with all their states in registers
// (LPC lanes a channel when there are more than 32 states), so the recurrence never leaves
// the lane; B / C of 16 tokens at a time are widened into LDS once a workgroup and broadcast;
// x, dt and z are loaded 8 tokens ahead.  A long prompt
// is cut into chunks that run side by side -- chunk states from zero, a carry pass over the
// chunks, then the scan proper from each chunk's true entry state -- because one sequence's
// channels alone (8192 = 128 waves) leave most of the 1024 SIMDs idle.
#include "docqa_common.h"
#include "docqa_elem.h"

using namespace docqa;

namespace {
constexpr int TB = 16;   // tokens whose B / C are staged in LDS at a time
constexpr int UB = 8;    // tokens whose x / dt / z are loaded ahead of their use

// ------------------------------------------------------------------ convolution, prefill
// thread: V channels x TT consecutive tokens, a window of the last K inputs in registers
template <typename T, int V, int K, int TT>
__global__ __launch_bounds__(256) void causal_conv_kernel(const T* __restrict__ x, int ldx,
                                                          const float* __restrict__ w, const float* __restrict__ bias,
                                                          T* __restrict__ state, const int* __restrict__ slots,
                                                          const int* __restrict__ cu, const int* __restrict__ ctx,
                                                          T* __restrict__ y, int C, int taps, int silu) {
  const int b = blockIdx.z, q0 = cu[b], L = cu[b + 1] - q0;
  const int nt = K > 0 ? K : taps;
  // a thread's tokens: at least the carried inputs, so the thread of token 0 alone reads (and
  // then replaces) a sequence's state
  static_assert(K <= 0 || TT >= K - 1, "tokens per thread");
  const int tt = K > 0 ? TT : max(TT, nt - 1);
  const int t0 = (blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6)) * tt;
  const int c0 = (blockIdx.x * 64 + (threadIdx.x & 63)) * V;
  if (t0 >= L || c0 >= C) return;
  const bool carry = ctx[b] > 0 && slots[b] >= 0;
  const T* st = carry ? state + (size_t)slots[b] * (nt - 1) * C + c0 : nullptr;
  float bv[V];
#pragma unroll
  for (int j = 0; j < V; ++j) bv[j] = 0.f;
  if (bias) ldv<V>(bias + c0, bv);
  auto input = [&](int t, float* f) {       // input at token t of this portion (t < 0: carried)
    if (t >= 0) {
      ldv<V>(x + (size_t)(q0 + t) * ldx + c0, f);
    } else if (carry) {
      ldv<V>(st + (size_t)(nt - 1 + t) * C, f);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) f[j] = 0.f;
    }
  };
  if constexpr (K > 0) {
    float wv[K][V], in[TT + K - 1][V];      // inputs t0 - (K - 1) .. t0 + TT - 1, all in flight at once
    if (t0 >= K - 1) {                      // whole waves: nothing carried, no branch between the loads
#pragma unroll
      for (int i = 0; i < TT + K - 1; ++i) ldv<V>(x + (size_t)(q0 + min(t0 + i - (K - 1), L - 1)) * ldx + c0, in[i]);
    } else {
#pragma unroll
      for (int i = 0; i < TT + K - 1; ++i) input(min(t0 + i - (K - 1), L - 1), in[i]);
    }
#pragma unroll
    for (int k = 0; k < K; ++k) ldv<V>(w + (size_t)k * C + c0, wv[k]);
#pragma unroll
    for (int i = 0; i < TT; ++i) {
      float o[V];
#pragma unroll
      for (int j = 0; j < V; ++j) {
        float s = bv[j];
#pragma unroll
        for (int k = 0; k < K; ++k) s += wv[k][j] * in[i + k][j];
        o[j] = silu ? silu_fast(s) : s;
      }
      if (t0 + i < L) stv<V>(y + (size_t)(q0 + t0 + i) * C + c0, o);
    }
  } else {
    for (int i = 0; i < tt && t0 + i < L; ++i) {
      float s[V], f[V], wk[V];
#pragma unroll
      for (int j = 0; j < V; ++j) s[j] = bv[j];
      for (int k = 0; k < nt; ++k) {
        input(t0 + i - (nt - 1) + k, f);
        ldv<V>(w + (size_t)k * C + c0, wk);
#pragma unroll
        for (int j = 0; j < V; ++j) s[j] += wk[j] * f[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) s[j] = silu ? silu_fast(s[j]) : s[j];
      stv<V>(y + (size_t)(q0 + t0 + i) * C + c0, s);
    }
  }
  // The last taps - 1 inputs into the state, by the one thread that read it (t0 = 0): row r
  // takes the input of portion token L - (taps - 1) + r, or old row r + L (> r, so ascending r
  // reads before it writes), or zero ahead of the sequence.
  if (t0 == 0 && slots[b] >= 0) {
    T* so = state + (size_t)slots[b] * (nt - 1) * C + c0;
    for (int r = 0; r < nt - 1; ++r) {
      float f[V];
      input(L - (nt - 1) + r, f);
      stv<V>(so + (size_t)r * C, f);
    }
  }
}

// ------------------------------------------------------------------ convolution, decode
// one new token a row; P [S, B, ld]: the input projection [x: C | z: C] as split-K slabs (or
// its product).  Writes silu(conv) and, when z_out, the next NZ columns summed; advances the state.
template <typename PT, typename T, int V, int K>
__global__ __launch_bounds__(256) void conv_step_kernel(const PT* __restrict__ P, int S, size_t slab, int ld,
                                                        const float* __restrict__ w, const float* __restrict__ bias,
                                                        T* __restrict__ state, const int* __restrict__ slots,
                                                        const int* __restrict__ positions, T* __restrict__ y,
                                                        T* __restrict__ z_out, int C, int NZ, int taps, int silu) {
  const int b = blockIdx.y, c0 = (blockIdx.x * 256 + threadIdx.x) * V;
  const int nt = K > 0 ? K : taps;
  if (c0 >= C + NZ) return;
  const PT* p = P + (size_t)b * ld + c0;
  float xn[V];
  ld_slabs<V>(p, S, slab, xn);
  if (c0 >= C) {
    stv<V>(z_out + (size_t)b * NZ + (c0 - C), xn);
    return;
  }
  const int slot = slots[b];
  const bool carry = slot >= 0 && positions[b] > 0;
  T* st = state + (size_t)max(slot, 0) * (nt - 1) * C + c0;
  float s[V], wk[V];
#pragma unroll
  for (int j = 0; j < V; ++j) s[j] = 0.f;
  if (bias) ldv<V>(bias + c0, s);
#pragma unroll
  for (int j = 0; j < V; ++j) xn[j] = rnd((const T*)nullptr, xn[j]);
  ldv<V>(w + (size_t)(nt - 1) * C + c0, wk);
#pragma unroll
  for (int j = 0; j < V; ++j) s[j] += wk[j] * xn[j];
  if constexpr (K > 0) {
    float h[K][V];
#pragma unroll
    for (int k = 0; k < K - 1; ++k) {
      if (carry) {
        ldv<V>(st + (size_t)k * C, h[k]);
      } else {
#pragma unroll
        for (int j = 0; j < V; ++j) h[k][j] = 0.f;
      }
    }
#pragma unroll
    for (int j = 0; j < V; ++j) h[K - 1][j] = xn[j];
#pragma unroll
    for (int k = 0; k < K - 1; ++k) {
      ldv<V>(w + (size_t)k * C + c0, wk);
#pragma unroll
      for (int j = 0; j < V; ++j) s[j] += wk[j] * h[k][j];
      if (slot >= 0) stv<V>(st + (size_t)k * C, h[k + 1]);
    }
  } else {
    for (int k = 0; k < nt - 1; ++k) {
      float h[V], nx[V];
#pragma unroll
      for (int j = 0; j < V; ++j) h[j] = 0.f, nx[j] = k == nt - 2 ? xn[j] : 0.f;
      if (carry) {
        ldv<V>(st + (size_t)k * C, h);
        if (k < nt - 2) ldv<V>(st + (size_t)(k + 1) * C, nx);
      }
      ldv<V>(w + (size_t)k * C + c0, wk);
#pragma unroll
      for (int j = 0; j < V; ++j) s[j] += wk[j] * h[j];
      if (slot >= 0) stv<V>(st + (size_t)k * C, nx);
    }
  }
#pragma unroll
  for (int j = 0; j < V; ++j) s[j] = silu ? silu_fast(s[j]) : s[j];
  stv<V>(y + (size_t)b * C + c0, s);
}

// ------------------------------------------------------------------ selective scan, prefill
struct ScanArgs {
  const void* x;       // [tokens, C] convolved input
  const void* dt;      // [tokens, C] step projection ahead of bias and softplus
  const void* bc;      // [tokens, ld_bc] B at bc_off, C at bc_off + c_off
  const void* z;       // [tokens, ld_z] gate
  void* y;             // [tokens, C]
  int ld_bc, b_off, c_off, ld_z;
  const float* A2;     // [C, Np]
  const float* D;      // [C]
  const float* dt_b;   // [C]
  float* state;        // [slots, C, Np]
  const int* slots;
  const int* cu;
  const int* ctx;
  float* cstate;       // [B, nchunk, C, Np] chunk states (chunked prompts)
  float* csum;         // [B, nchunk, C] sum of dt of each chunk
  int C, N, Np, chunk, nchunk;
};

// LOCAL: the chunk's state from zero and its sum of dt (all chunks but a sequence's last).
// Otherwise the scan proper, entering from the carried state (chunk 0) or the carry pass.
// CPL: channels per lane -- two share a token's loads, address arithmetic and B / C reads.
template <typename T, int NS, int LPC, int CPL, bool LOCAL>
__global__ __launch_bounds__(256) void selective_scan_kernel(ScanArgs a) {
  constexpr int NSP = NS * LPC, CB = 256 / LPC * CPL;
  __shared__ __attribute__((aligned(16))) float sbc[2][TB][2 * NSP];
  const int b = blockIdx.z, ck = blockIdx.y;
  const int q0 = a.cu[b], L = a.cu[b + 1] - q0;
  const int t_beg = ck * a.chunk, t_end = min(L, t_beg + a.chunk);
  if (t_beg >= L || (LOCAL && t_end >= L)) return;
  const int tid = threadIdx.x;
  const int c = blockIdx.x * CB + tid / LPC * CPL, l = tid % LPC;
  const bool ok = c < a.C;
  const int cc = ok ? c : a.C - CPL;
  const int slot = a.slots[b];
  const T *X = (const T*)a.x, *DT = (const T*)a.dt, *bc = (const T*)a.bc, *Z = (const T*)a.z;

  float A[CPL][NS], S[CPL][NS], Dc[CPL], db[CPL], sum[CPL];
#pragma unroll
  for (int j = 0; j < CPL; ++j) {
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const int n = l * NS + i;
      A[j][i] = n < a.N ? a.A2[(size_t)(cc + j) * a.Np + n] : 0.f;
      S[j][i] = 0.f;
    }
    Dc[j] = a.D[cc + j];
    db[j] = a.dt_b[cc + j];
    sum[j] = 0.f;
  }
  if constexpr (!LOCAL) {
    const float* s0 = nullptr;
    if (ck > 0) s0 = a.cstate + (((size_t)b * a.nchunk + ck) * a.C + cc) * a.Np;
    else if (a.ctx[b] > 0 && slot >= 0) s0 = a.state + ((size_t)slot * a.C + cc) * a.Np;
    if (s0) {
#pragma unroll
      for (int j = 0; j < CPL; ++j)
#pragma unroll
        for (int i = 0; i < NS; ++i)
          if (l * NS + i < a.N) S[j][i] = s0[(size_t)j * a.Np + l * NS + i];
    }
  }

  auto stage = [&](int t0, int buf) {
    for (int e = tid; e < TB * 2 * NSP; e += 256) {
      const int t = e / (2 * NSP), j = e % (2 * NSP), n = j < NSP ? j : j - NSP;
      float v = 0.f;
      if (t0 + t < t_end && n < a.N)
        v = ld1(bc + (size_t)(q0 + t0 + t) * a.ld_bc + (j < NSP ? a.b_off : a.c_off) + n);
      sbc[buf][t][j] = v;
    }
  };
  // x, dt, z of UB tokens from t (clamped: a token past the end is computed with dt = 0, which
  // leaves the state alone, and stores nothing); row pointers are uniform, lanes add a column
  float xn[UB][CPL], dn[UB][CPL], zn[UB][CPL];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < UB; ++i) {
      const size_t r = q0 + min(t0 + i, t_end - 1);
      ldv<CPL>(X + r * a.C + (unsigned)cc, xn[i]);
      ldv<CPL>(DT + r * a.C + (unsigned)cc, dn[i]);
      if constexpr (!LOCAL) ldv<CPL>(Z + r * a.ld_z + (unsigned)cc, zn[i]);
    }
  };
  stage(t_beg, 0);
  fetch(t_beg);
  int buf = 0;
  for (int t0 = t_beg; t0 < t_end; t0 += TB, buf ^= 1) {
    __syncthreads();
    if (t0 + TB < t_end) stage(t0 + TB, buf ^ 1);
#pragma unroll 1
    for (int u = 0; u < TB; u += UB) {
      float xv[UB][CPL], dv[UB][CPL], zv[UB][CPL];
#pragma unroll
      for (int i = 0; i < UB; ++i)
#pragma unroll
        for (int j = 0; j < CPL; ++j) {
          xv[i][j] = xn[i][j];
          dv[i][j] = t0 + u + i < t_end ? softplus_f(dn[i][j] + db[j]) : 0.f;
          if constexpr (!LOCAL) zv[i][j] = silu_fast(zn[i][j]);
        }
      fetch(t0 + u + UB);
#pragma unroll
      for (int i = 0; i < UB; ++i) {
        const float* Bt = &sbc[buf][u + i][l * NS];
        const float* Ct = &sbc[buf][u + i][NSP + l * NS];
        float y[CPL];
#pragma unroll
        for (int j = 0; j < CPL; ++j) {
          const float d = dv[i][j], dx = d * xv[i][j];
          y[j] = 0.f;
#pragma unroll
          for (int n = 0; n < NS; ++n) {
            S[j][n] = __builtin_amdgcn_exp2f(d * A[j][n]) * S[j][n] + dx * Bt[n];
            if constexpr (!LOCAL) y[j] += S[j][n] * Ct[n];
          }
          sum[j] += d;
        }
        if constexpr (!LOCAL) {
#pragma unroll
          for (int j = 0; j < CPL; ++j) {
#pragma unroll
            for (int o = 1; o < LPC; o <<= 1) y[j] += __shfl_xor(y[j], o, 64);
            y[j] = (y[j] + Dc[j] * xv[i][j]) * zv[i][j];
          }
          if (l == 0 && ok && t0 + u + i < t_end)
            stv<CPL>((T*)a.y + (size_t)(q0 + t0 + u + i) * a.C + (unsigned)c, y);
        }
      }
    }
  }
  if (!ok) return;
  float* o = nullptr;
  if constexpr (LOCAL) o = a.cstate + (((size_t)b * a.nchunk + ck + 1) * a.C + c) * a.Np;   // enters chunk ck + 1
  else if (t_end == L && slot >= 0) o = a.state + ((size_t)slot * a.C + c) * a.Np;
  if (!o) return;
#pragma unroll
  for (int j = 0; j < CPL; ++j) {
#pragma unroll
    for (int i = 0; i < NS; ++i)
      if (l * NS + i < a.N) o[(size_t)j * a.Np + l * NS + i] = S[j][i];
    if (LOCAL && l == 0) a.csum[((size_t)b * a.nchunk + ck + 1) * a.C + c + j] = sum[j];
  }
}

// chunk k's entry state: decay over chunk k - 1 times its own entry state, plus the local one
__global__ __launch_bounds__(256) void scan_carry_kernel(ScanArgs a) {
  const int b = blockIdx.y, L = a.cu[b + 1] - a.cu[b];
  const int e = blockIdx.x * 256 + threadIdx.x;
  const int c = e / a.Np, n = e % a.Np;
  if (c >= a.C || n >= a.N || L <= a.chunk) return;
  const float A = a.A2[e];
  const int slot = a.slots[b];
  float s = (a.ctx[b] > 0 && slot >= 0) ? a.state[(size_t)slot * a.C * a.Np + e] : 0.f;
  for (int k = 1; k * a.chunk < L; ++k) {
    const size_t o = ((size_t)b * a.nchunk + k) * a.C;
    s = __builtin_amdgcn_exp2f(A * a.csum[o + c]) * s + a.cstate[o * a.Np + e];
    a.cstate[o * a.Np + e] = s;
  }
}

// ------------------------------------------------------------------ selective scan, decode
// One token a row.  A lane holds 4 states of a channel (16-byte state accesses, the launch's
// HBM traffic), a workgroup 256 / lq channels of RB rows, so A is read once for all of them;
// every row's state is in flight before anything is computed.  The rows' step sizes, inputs,
// gates, B and C go through LDS.  w_dt given: the step projection runs here too, on MFMA
// (the RB rows against the workgroup's channels, K = R), instead of a GEMM launch of its own.
struct StepDt {
  const uint16_t* w;    // [C, R] bf16, R % 32 == 0; null: ScanArgs::dt holds the product
  const uint16_t* in;   // [B, R]
  int R;
};
template <typename T, int RB>
__global__ __launch_bounds__(256) void selective_step_kernel(ScanArgs a, StepDt sd, const int* __restrict__ positions,
                                                             int B, int lq) {
  __shared__ float sdt[RB][256], sx[RB][256], sg[RB][256];
  __shared__ __attribute__((aligned(16))) float sb[RB][256], sc[RB][256];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int CB = 256 / lq;                              // channels of this workgroup
  const int cb = blockIdx.x * CB, cl = tid / lq, c = cb + cl, g = tid % lq, n0 = g * 4;
  const int r0 = blockIdx.y * RB;
  const bool ok = c < a.C && n0 < a.Np;
  float4 A = make_float4(0.f, 0.f, 0.f, 0.f), S[RB];
  int slot[RB];
#pragma unroll
  for (int i = 0; i < RB; ++i) {
    const int r = min(r0 + i, B - 1);
    slot[i] = r0 + i < B ? a.slots[r] : -1;
    S[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (ok && slot[i] >= 0 && positions[r] > 0)
      S[i] = *reinterpret_cast<const float4*>(a.state + ((size_t)slot[i] * a.C + c) * a.Np + n0);
  }
  if (ok) A = *reinterpret_cast<const float4*>(a.A2 + (size_t)c * a.Np + n0);
  const float Dc = a.D[min(c, a.C - 1)];

  for (int e = tid; e < RB * CB; e += 256) {
    const int i = e / CB, j = e % CB, cc = min(cb + j, a.C - 1);
    const size_t r = min(r0 + i, B - 1);
    sx[i][j] = ld1((const T*)a.x + r * a.C + cc);
    sg[i][j] = silu_fast(ld1((const T*)a.z + r * a.ld_z + cc));
    if (!sd.w) sdt[i][j] = softplus_f(ld1((const T*)a.dt + r * a.C + cc) + a.dt_b[cc]);
  }
  for (int e = tid; e < RB * a.Np; e += 256) {
    const int i = e / a.Np, n = e % a.Np;
    const T* bc = (const T*)a.bc + (size_t)min(r0 + i, B - 1) * a.ld_bc;
    sb[i][n] = n < a.N ? ld1(bc + a.b_off + n) : 0.f;
    sc[i][n] = n < a.N ? ld1(bc + a.c_off + n) : 0.f;
  }
  if (sd.w) {
    // 16-channel tiles: A rows = token rows, B rows = channels; D: lane & 15 the channel,
    // 4 (lane >> 4) + r the row
    const int fr = lane & 15, g4 = lane >> 4;
    const uint16_t* ip = sd.in + (size_t)min(r0 + min(fr, RB - 1), B - 1) * sd.R + g4 * 8;
    for (int t = wave; t < (CB + 15) / 16; t += 4) {
      const int ch = min(cb + t * 16 + fr, a.C - 1);
      const uint16_t* wp = sd.w + (size_t)ch * sd.R + g4 * 8;
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
      for (int k = 0; k < sd.R; k += 32)
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(ip + k),
                                                      *reinterpret_cast<const bf16x8*>(wp + k), acc, 0, 0, 0);
      const float db = a.dt_b[ch];
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (g4 * 4 + r < RB && t * 16 + fr < CB) sdt[g4 * 4 + r][t * 16 + fr] = softplus_f(acc[r] + db);
    }
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < RB; ++i) {
    const float d = sdt[i][cl], x = sx[i][cl], dx = d * x;
    float4 s = S[i];
    float y = 0.f;
    if (ok) {
      const float4 bv = *reinterpret_cast<const float4*>(&sb[i][n0]), cv = *reinterpret_cast<const float4*>(&sc[i][n0]);
      s.x = __builtin_amdgcn_exp2f(d * A.x) * s.x + dx * bv.x;
      s.y = __builtin_amdgcn_exp2f(d * A.y) * s.y + dx * bv.y;
      s.z = __builtin_amdgcn_exp2f(d * A.z) * s.z + dx * bv.z;
      s.w = __builtin_amdgcn_exp2f(d * A.w) * s.w + dx * bv.w;
      y = (s.x * cv.x + s.y * cv.y) + (s.z * cv.z + s.w * cv.w);
      if (slot[i] >= 0) *reinterpret_cast<float4*>(a.state + ((size_t)slot[i] * a.C + c) * a.Np + n0) = s;
    }
    for (int o = 1; o < lq; o <<= 1) y += __shfl_xor(y, o, 64);
    // a channel's lanes are one wave's: they have all read sx[i][cl] above
    if (g == 0) sx[i][cl] = (y + Dc * x) * sg[i][cl];
  }
  __syncthreads();
  for (int e = tid; e < RB * CB; e += 256) {
    const int i = e / CB, j = e % CB;
    if (r0 + i < B && cb + j < a.C) st1((T*)a.y + (size_t)(r0 + i) * a.C + cb + j, sx[i][j]);
  }
}

template <typename T, int V>
int launch_conv(const void* x, int ldx, const float* w, const float* b, void* state, const int* slots, const int* cu,
                const int* ctx, void* y, int B, int max_len, int C, int taps, int silu, hipStream_t s) {
  const int gx = (C + 64 * V - 1) / (64 * V);
  // 8 tokens a thread; fewer where that leaves most of the chip without a workgroup
  const bool few = (long long)gx * ((max_len + 31) / 32) * B < 512;
#define LAUNCH(K, TT, tt)                                                                                   \
  causal_conv_kernel<T, V, K, TT><<<dim3(gx, (max_len + 4 * (tt)-1) / (4 * (tt)), B), 256, 0, s>>>(         \
      (const T*)x, ldx, w, b, (T*)state, slots, cu, ctx, (T*)y, C, taps, silu)
#define GO(K)                                        \
  do {                                               \
    constexpr int TF = K == 4 ? 3 : 2;               \
    if (few) LAUNCH(K, TF, K > 0 ? TF : (TF > taps - 1 ? TF : taps - 1)); \
    else LAUNCH(K, 8, K > 0 ? 8 : (8 > taps - 1 ? 8 : taps - 1));        \
  } while (0)
  switch (taps) {
    case 2: GO(2); break;
    case 3: GO(3); break;
    case 4: GO(4); break;
    default: GO(0); break;
  }
#undef GO
#undef LAUNCH
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <typename PT, typename T, int V>
int launch_conv_step(const void* P, int S, size_t slab, int ld, const float* w, const float* b, void* state,
                     const int* slots, const int* pos, void* y, void* z, int B, int C, int NZ, int taps, int silu,
                     hipStream_t s) {
  const int n = (C + NZ) / V;
  dim3 grid((n + 255) / 256, B);
#define GO(K) conv_step_kernel<PT, T, V, K><<<grid, 256, 0, s>>>((const PT*)P, S, slab, ld, w, b, (T*)state, slots, pos, (T*)y, (T*)z, C, NZ, taps, silu)
  switch (taps) {
    case 2: GO(2); break;
    case 3: GO(3); break;
    case 4: GO(4); break;
    default: GO(0); break;
  }
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <typename T, int NS, int LPC, int CPL>
int launch_scan(const ScanArgs& a, int B, hipStream_t s) {
  constexpr int CB = 256 / LPC * CPL;
  dim3 grid((a.C + CB - 1) / CB, a.nchunk, B);
  if (a.nchunk > 1) {
    selective_scan_kernel<T, NS, LPC, CPL, true><<<grid, 256, 0, s>>>(a);
    DOCQA_CHECK_LAUNCH();
    scan_carry_kernel<<<dim3((a.C * a.Np + 255) / 256, B), 256, 0, s>>>(a);
    DOCQA_CHECK_LAUNCH();
  }
  selective_scan_kernel<T, NS, LPC, CPL, false><<<grid, 256, 0, s>>>(a);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

template <typename T>
int dispatch_scan(const ScanArgs& a, int B, hipStream_t s) {
  const bool pair = a.C % 2 == 0 && a.ld_z % 2 == 0 && docqa_aligned16(a.x) && docqa_aligned16(a.dt) &&
                    (reinterpret_cast<uintptr_t>(a.z) & 7) == 0 && docqa_aligned16(a.y);
  if (a.N <= 8) return pair ? launch_scan<T, 8, 1, 2>(a, B, s) : launch_scan<T, 8, 1, 1>(a, B, s);
  if (a.N <= 16) return pair ? launch_scan<T, 16, 1, 2>(a, B, s) : launch_scan<T, 16, 1, 1>(a, B, s);
  if (a.N <= 24) return launch_scan<T, 24, 1, 1>(a, B, s);
  if (a.N <= 32) return launch_scan<T, 32, 1, 1>(a, B, s);
  if (a.N <= 64) return launch_scan<T, 32, 2, 1>(a, B, s);
  if (a.N <= 128) return launch_scan<T, 32, 4, 1>(a, B, s);
  if (a.N <= 256) return launch_scan<T, 32, 8, 1>(a, B, s);
  return -1;
}
}  // namespace

int docqa_causal_conv(const void* x, int ldx, const float* w, const float* b, void* state, const int* slots,
                      const int* cu, const int* ctx, void* y, int f32, int B, int max_len, int C, int taps,
                      int silu, hipStream_t s) {
  if (B == 0 || max_len == 0) return 0;
  if (taps < 1 || C < 1 || ldx < C) return -1;
  const bool vec = C % 8 == 0 && ldx % 8 == 0 && docqa_aligned16(x) && docqa_aligned16(state) && docqa_aligned16(y);
  if (f32)
    return vec ? launch_conv<float, 4>(x, ldx, w, b, state, slots, cu, ctx, y, B, max_len, C, taps, silu, s)
               : launch_conv<float, 1>(x, ldx, w, b, state, slots, cu, ctx, y, B, max_len, C, taps, silu, s);
  return vec ? launch_conv<uint16_t, 8>(x, ldx, w, b, state, slots, cu, ctx, y, B, max_len, C, taps, silu, s)
             : launch_conv<uint16_t, 1>(x, ldx, w, b, state, slots, cu, ctx, y, B, max_len, C, taps, silu, s);
}

int docqa_conv_step(const void* P, int p_f32, int S, size_t slab, int ld, const float* w, const float* b, void* state,
                    const int* slots, const int* positions, void* y, void* z, int f32, int B, int C, int NZ, int taps,
                    int silu, hipStream_t s) {
  if (B == 0) return 0;
  if (taps < 1 || C < 1 || S < 1 || NZ < 0 || (NZ > 0 && !z) || ld < C + NZ || (f32 && !p_f32)) return -1;
  const bool vec = C % 4 == 0 && NZ % 4 == 0 && ld % 4 == 0 && docqa_aligned16(P) && docqa_aligned16(state) && docqa_aligned16(y);
#define ARGS P, S, slab, ld, w, b, state, slots, positions, y, z, B, C, NZ, taps, silu, s
  if (f32) return vec ? launch_conv_step<float, float, 4>(ARGS) : launch_conv_step<float, float, 1>(ARGS);
  if (p_f32) return vec ? launch_conv_step<float, uint16_t, 4>(ARGS) : launch_conv_step<float, uint16_t, 1>(ARGS);
  return vec ? launch_conv_step<uint16_t, uint16_t, 4>(ARGS) : launch_conv_step<uint16_t, uint16_t, 1>(ARGS);
#undef ARGS
}

int docqa_selective_scan(const void* x, const void* dt, const void* bc, int ld_bc, int b_off, int c_off,
                         const void* z, int ld_z, const float* A2, const float* D, const float* dt_b, float* state,
                         const int* slots, const int* cu, const int* ctx, void* y, float* cstate, float* csum,
                         int f32, int B, int C, int N, int Np, int chunk, int nchunk, hipStream_t s) {
  if (B == 0 || nchunk == 0) return 0;
  if (N < 1 || Np < N || Np % 4 || chunk < 1 || (nchunk > 1 && (!cstate || !csum))) return -1;
  const ScanArgs a{x, dt, bc, z, y, ld_bc, b_off, c_off, ld_z, A2, D, dt_b, state, slots, cu, ctx, cstate, csum,
                   C, N, Np, chunk, nchunk};
  return f32 ? dispatch_scan<float>(a, B, s) : dispatch_scan<uint16_t>(a, B, s);
}

int docqa_selective_step(const void* x, const void* dt, const void* dt_in, const void* w_dt, int R, const void* bc,
                         int ld_bc, int b_off, int c_off, const void* z, int ld_z, const float* A2, const float* D,
                         const float* dt_b, float* state, const int* slots, const int* positions, void* y, int f32,
                         int B, int C, int N, int Np, hipStream_t s) {
  if (B == 0) return 0;
  if (N < 1 || Np < N || Np % 4 || Np > 256) return -1;
  if (w_dt ? (f32 || !dt_in || R < 32 || R % 32 || !docqa_aligned16(w_dt) || !docqa_aligned16(dt_in)) : !dt) return -1;
  const ScanArgs a{x, dt, bc, z, y, ld_bc, b_off, c_off, ld_z, A2, D, dt_b, state, slots, nullptr, nullptr, nullptr,
                   nullptr, C, N, Np, 0, 0};
  const StepDt sd{(const uint16_t*)w_dt, (const uint16_t*)dt_in, R};
  int lq = 1;
  while (lq * 4 < Np) lq *= 2;
  const int gx = (C + 256 / lq - 1) / (256 / lq);
#define GO(T, RB) selective_step_kernel<T, RB><<<dim3(gx, (B + RB - 1) / RB), 256, 0, s>>>(a, sd, positions, B, lq)
  if (f32) {
    if (B >= 4) GO(float, 4);
    else GO(float, 1);
  } else if (B >= 32) {
    GO(uint16_t, 8);
  } else if (B >= 4) {
    GO(uint16_t, 4);
  } else {
    GO(uint16_t, 1);
  }
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}
