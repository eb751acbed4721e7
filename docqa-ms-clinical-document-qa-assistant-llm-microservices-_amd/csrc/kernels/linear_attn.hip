// linear_attn.hip -- linear-attention recurrences with one [dk, dv] matrix S a head:
//   S_t = diag(a_t) S_{t-1} + k_t u_t^T,  o_t = S_t^T q_t,  y = rms(o) w silu(g)   (or sigmoid(g))
//   channel: a = sigmoid(z)^(1/tau) per key channel, z = w1 . w2 + b of a low-rank projection; u = v
//   fixed:   a constant per head; q, k rotated by position; u = v
//   delta:   a = exp(A softplus(z + b)) per head; unit q, k; u = sigmoid(beta) (v - (a S_{t-1})^T k)
//   channel delta: the delta rule with a per key channel, A per head
// The state pool holds [slots, H, dk, dvp] fp32 (dvp: dv rounded up to 4, padding zero).  A sequence
// whose first token is position 0 starts from zero whatever its slot held.
//
// Everything between the projections and the gated heads is fp32, matrix products included
// (v_mfma_f32_16x16x4_f32).
//
// step (one token a row): a workgroup a head; a wave holds 32 columns of S in registers (8 lanes of
//   4 columns x 8 row groups; heads of more than 128 rows: 4 lanes x 16 row groups), so the state is
//   read and written once in 128-byte pieces.
// scan (prompts), chunks of C tokens, b_t the log decays summed inside the chunk:
//   prep   per (chunk, head), all side by side:  Q' = q e^{b_t},  K' = k e^{b_C - b_t} (transposed),
//          A[t, s] = q_t . k_s e^{b_t - b_s} (s <= t); delta: M[t, s] = beta_t e^{b_t - b_s} k_t . k_s
//          (s < t) and, by forward substitution over blocks of 16 tokens with the diagonal blocks
//          inverted ahead, U = (1 + M)^-1 beta v, W = (1 + M)^-1 beta e^{b_t} k.
//          Where decays differ by channel, a 16 x 16 block of A (and M) below the diagonal takes both
//          factors relative to the last token ahead of its rows, so no exponent is positive.  One on
//          the diagonal takes them relative to its middle token while no channel decays by more than
//          e^-kMaxDrop within the block, and is summed directly, exponent by exponent, otherwise.
//   chunk  per (sequence, head, dv tile), chunk after chunk, S in accumulators:
//          u = v or U - W S;  o = Q' S + A u;  S = e^{b_C} S + K'^T u
//   gate   y = rms(o) w silu(g) per (token, head)
#include "docqa_common.h"
#include "docqa_elem.h"
#include "docqa_hybrid.h"

using namespace docqa;

namespace {
// V columns of a product or of slabs, element type by a uniform flag
template <int V>
__device__ __forceinline__ void ldx(const void* p, int f32, int S, size_t slab, size_t off, float* f) {
  if (f32) ld_slabs<V>((const float*)p + off, S, slab, f);
  else ld_slabs<V>((const uint16_t*)p + off, S, slab, f);
}
__device__ __forceinline__ float ldx1(const void* p, int f32, int S, size_t slab, size_t off) {
  float f;
  ldx<1>(p, f32, S, slab, off, &f);
  return f;
}
__device__ __forceinline__ void stx(void* p, int f32, size_t off, float v) {
  if (f32) ((float*)p)[off] = v;
  else ((uint16_t*)p)[off] = f2bf(v);
}
__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
// log(1 + e^x)
__device__ __forceinline__ float softplus_x(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ f32x4 mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// ------------------------------------------------------------------ one token a row
// CG: lanes of 4 columns each; NR: rows of S a lane holds, NR 64 / CG >= dk; MT: most threads.
// NR stays at 16: with 32 rows a lane, registers ran out and the compiler copied live row numbers
// under a narrowed EXEC mask, which lost those of the other lanes.
template <int CG, int NR, int MT>
__global__ __launch_bounds__(MT) void linear_step_kernel(DocqaLinear a, const int* __restrict__ positions) {
  constexpr int RG = 64 / CG, RP = RG * NR;
  extern __shared__ float lds[];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, nt = blockDim.x, lane = tid & 63, wave = tid >> 6;
  const int dk = a.dk, dv = a.dv, dvp = (dv + 3) & ~3, kh = h / (a.H / a.G);
  float *sq = lds, *sk = sq + RP, *sa = sk + RP, *sv = sa + RP, *sg = sv + dvp;   // q, k, decays (zero past dk), v, gates
  float *sr = sg + dvp, *red = sr + a.rank;                                       // low-rank inputs; [waves]
  const int slot = a.slots[b];
  const int cg = lane % CG, rg = lane / CG, c0 = (wave * CG + cg) * 4;
  const bool carry = slot >= 0 && positions[b] > 0, cok = c0 < dvp;
  char* sp = reinterpret_cast<char*>(a.state + ((size_t)max(slot, 0) * a.H + h) * dk * dvp);
  float4 S[NR];                              // rows past the last repeat it: their k and q are zero
#pragma unroll
  for (int i = 0; i < NR; ++i) S[i] = make_float4(0.f, 0.f, 0.f, 0.f);
  if (carry && cok) {
#pragma unroll
    for (int i = 0; i < NR; ++i) S[i] = *reinterpret_cast<const float4*>(sp + (unsigned)(min(i * RG + rg, dk - 1) * dvp + c0) * 4u);
  }
  const size_t xr = (size_t)b * a.ldx, zr = (size_t)b * a.ldz;
  for (int i = tid; i < RP; i += nt) {
    sq[i] = i < dk ? ldx1(a.X, a.xf32, a.Sx, a.xslab, xr + a.qo + kh * dk + i) : 0.f;
    sk[i] = i < dk ? ldx1(a.X, a.xf32, a.Sx, a.xslab, xr + a.ko + kh * dk + i) : 0.f;
    sa[i] = 0.f;
  }
  for (int i = tid; i < dvp; i += nt) {
    sv[i] = i < dv ? ldx1(a.X, a.xf32, a.Sx, a.xslab, xr + a.vo + h * dv + i) : 0.f;
    sg[i] = i < dv ? ldx1(a.Z, a.zf32, a.Sz, a.zslab, zr + a.go + h * dv + i) : 0.f;
  }
  float qs = a.qs, ks = a.ks, beta = 1.f, al = 1.f;
  const bool chan = a.kind == LIN_CHANNEL || a.kind == LIN_CHANNEL_DELTA, delta = a.kind >= LIN_DELTA;
  if (a.kind == LIN_CHANNEL) {
    for (int i = tid; i < a.rank; i += nt) sr[i] = ldx1(a.Z, a.zf32, a.Sz, a.zslab, zr + a.ao + i);
  } else if (a.kind == LIN_FIXED) {
    al = expf(a.w_gate[h]);
  } else if (a.kind == LIN_DELTA) {
    al = expf(a.w_gate[h] * softplus_x(ldx1(a.Z, a.zf32, a.Sz, a.zslab, zr + a.ao + h) + a.b_gate[h]));
  } else {
    // (a thread's own i: it zeroed this element above)
    for (int i = tid; i < dk; i += nt)
      sa[i] = expf(a.w_gate[h] * softplus_x(ldx1(a.Z, a.zf32, a.Sz, a.zslab, zr + a.ao + h * dk + i) + a.b_gate[h * dk + i]));
  }
  if (delta) beta = sigmoid_f(ldx1(a.Z, a.zf32, a.Sz, a.zslab, zr + a.bo + h));
  __syncthreads();
  if (a.kind == LIN_CHANNEL) {
    for (int i = tid; i < dk; i += nt) {
      const float* w = a.w_gate + ((size_t)h * dk + i) * a.rank;
      float z = a.b_gate[h * dk + i];
      for (int r = 0; r < a.rank; ++r) z += sr[r] * w[r];
      sa[i] = expf(-softplus_x(-z) * a.inv_tau);
    }
    __syncthreads();
  } else if (a.kind == LIN_FIXED && a.r > 0) {
    const int r2 = a.r / 2;
    for (int e = tid; e < a.r; e += nt) {
      float* s = e < r2 ? sq : sk;
      const int i = e < r2 ? e : e - r2;
      const float c = a.cs[(size_t)b * a.r + i], si = a.cs[(size_t)b * a.r + r2 + i], x = s[i], y = s[i + r2];
      s[i] = x * c - y * si;
      s[i + r2] = y * c + x * si;
    }
    __syncthreads();
  } else if (delta) {
    float nq = 0.f, nk = 0.f;
    for (int i = lane; i < dk; i += 64) {
      nq += sq[i] * sq[i];
      nk += sk[i] * sk[i];
    }
    qs *= 1.f / sqrtf(wave_sum(nq) + 1e-6f);
    ks *= 1.f / sqrtf(wave_sum(nk) + 1e-6f);
  }
  auto rows_sum = [](float x) {              // over the row groups of a column
#pragma unroll
    for (int m = CG; m < 64; m <<= 1) x += __shfl_xor(x, m, 64);
    return x;
  };
  float v[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = cok ? sv[c0 + j] : 0.f;
  float p[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int r = i * RG + rg;
    const float d = chan ? sa[r] : al, k = sk[r] * ks;
    S[i].x *= d; S[i].y *= d; S[i].z *= d; S[i].w *= d;
    p[0] += S[i].x * k; p[1] += S[i].y * k; p[2] += S[i].z * k; p[3] += S[i].w * k;
  }
  if (delta) {
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = beta * (v[j] - rows_sum(p[j]));
  }
  float o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int r = i * RG + rg;
    const float k = sk[r] * ks, q = sq[r] * qs;
    S[i].x += k * v[0]; S[i].y += k * v[1]; S[i].z += k * v[2]; S[i].w += k * v[3];
    o[0] += S[i].x * q; o[1] += S[i].y * q; o[2] += S[i].z * q; o[3] += S[i].w * q;
    if (slot >= 0 && cok && r < dk) *reinterpret_cast<float4*>(sp + (unsigned)(r * dvp + c0) * 4u) = S[i];
  }
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    o[j] = rows_sum(o[j]);
    if (rg == 0 && c0 + j < dv) ss += o[j] * o[j];
  }
  ss = wave_sum(ss);
  if (lane == 0) red[wave] = ss;
  __syncthreads();
  float tot = 0.f;
  for (int w = 0; w < (nt >> 6); ++w) tot += red[w];
  const float inv = 1.f / sqrtf(tot / (float)dv + a.eps);
  if (rg == 0) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (c0 + j < dv) {
        const float g = sg[c0 + j];
        stx(a.out, a.of32, (size_t)b * a.ldo + h * dv + c0 + j, o[j] * inv * a.norm[c0 + j] * (a.sig ? 1.f : g) * sigmoid_f(g));
      }
  }
}

// ------------------------------------------------------------------ prompts
struct ScanArgs {
  DocqaLinear a;
  const int *cu, *ctx;
  int nchunk;                            // most chunks of a sequence
  float *Q, *K, *A, *G, *W, *U, *O;      // per (chunk, head): [C, dkp], [dkp, C], [C, C], [dkp], [C, dkp], [C, dvq]; O [T, H, dvq]
};
// chunk ids: sequence b's follow those of the sequences ahead of it, whatever their lengths
__device__ __forceinline__ size_t chunk_id(const ScanArgs& s, int b, int ck, int C) { return (size_t)(s.cu[b] / C) + b + ck; }

// between a wave's own writes to LDS and its reads of other lanes' parts
__device__ __forceinline__ void wave_lds_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

constexpr float kMaxDrop = 30.f;
constexpr int NTP = 512, NWP = NTP / 64, PT = 20;
constexpr int prep_q(int C, int DKP, bool delta) { return delta && NWP * C * PT > C * (DKP + 4) ? NWP * C * PT : C * (DKP + 4); }
// pitch of the low-rank inputs: the rank in whole MFMA steps
__host__ __device__ __forceinline__ int rank_pitch(int rank) { return ((rank + 15) & ~15) + 4; }
template <int C, int DKP, int KIND, int V>
__global__ __launch_bounds__(NTP) void linear_prep_kernel(ScanArgs sc) {
  constexpr int PK = DKP + 4, NB = C / 16, PM = C + 4;
  constexpr bool CH = KIND == LIN_CHANNEL || KIND == LIN_CHANNEL_DELTA, DELTA = KIND >= LIN_DELTA;
  __shared__ int s_direct[NB];                               // diagonal blocks to be summed directly
  extern __shared__ __attribute__((aligned(16))) float lds[];
  // delta: sQ's place later holds the waves' parts of the solution, [NWP, C, PT]
  float *sQ = lds, *sK = sQ + prep_q(C, DKP, DELTA), *sB = sK + C * PK;   // sB: [C, PK] (channel) or [C] log decays, summed
  float* sM = sB + (CH ? C * PK : C);                        // delta: [C, PM]; channel: low-rank inputs [C, rank_pitch]
  float *sT = sM + C * PM, *sbeta = sT + C * PT;             // delta: inverses of 1 + M's diagonal blocks; [C]
  const DocqaLinear& a = sc.a;
  const int h = blockIdx.x, ck = blockIdx.y, b = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int q0 = sc.cu[b], L = sc.cu[b + 1] - q0, t0 = ck * C;
  if (t0 >= L) return;
  const int n = min(C, L - t0), dk = a.dk, dv = a.dv, kh = h / (a.H / a.G), dvq = (dv + 15) & ~15;
  const size_t cid = chunk_id(sc, b, ck, C) * a.H + h, row0 = q0 + t0;

  for (int e = tid; e < C * (DKP / V); e += NTP) {
    const int t = e / (DKP / V), d = (e % (DKP / V)) * V;
    float q[V], k[V];
#pragma unroll
    for (int j = 0; j < V; ++j) q[j] = k[j] = 0.f;
    if (t < n && d < dk) {
      const size_t r = (row0 + t) * a.ldx + kh * dk + d;
      ldx<V>(a.X, a.xf32, a.Sx, a.xslab, r + a.qo, q);
      ldx<V>(a.X, a.xf32, a.Sx, a.xslab, r + a.ko, k);
    }
#pragma unroll
    for (int j = 0; j < V; ++j) {
      sQ[t * PK + d + j] = q[j];
      sK[t * PK + d + j] = k[j];
    }
  }
  if (DELTA && wave == 1) {
    if (lane < C) sbeta[lane] = lane < n ? sigmoid_f(ldx1(a.Z, a.zf32, a.Sz, a.zslab, (row0 + lane) * a.ldz + a.bo + h)) : 0.f;
  }
  if constexpr (KIND == LIN_CHANNEL_DELTA) {
    const float A = a.w_gate[h];
    for (int e = tid; e < C * (DKP / V); e += NTP) {
      const int t = e / (DKP / V), d = (e % (DKP / V)) * V;
      float z[V];
#pragma unroll
      for (int j = 0; j < V; ++j) z[j] = 0.f;
      if (t < n && d < dk) {
        float bias[V];
        ldx<V>(a.Z, a.zf32, a.Sz, a.zslab, (row0 + t) * a.ldz + a.ao + h * dk + d, z);
        ldv<V>(a.b_gate + h * dk + d, bias);
#pragma unroll
        for (int j = 0; j < V; ++j) z[j] = A * softplus_x(z[j] + bias[j]);
      }
      stv<V>(sB + t * PK + d, z);
    }
  } else if constexpr (CH) {
    const int rp = rank_pitch(a.rank);
    for (int e = tid; e < C * rp; e += NTP) {
      const int t = e / rp, r = e % rp;
      sM[e] = t < n && r < a.rank ? ldx1(a.Z, a.zf32, a.Sz, a.zslab, (row0 + t) * a.ldz + a.ao + r) : 0.f;
    }
  } else if (wave == 0) {
    float la = 0.f;
    if (lane < n) {
      la = a.w_gate[h];
      if constexpr (DELTA) la *= softplus_x(ldx1(a.Z, a.zf32, a.Sz, a.zslab, (row0 + lane) * a.ldz + a.ao + h) + a.b_gate[h]);
    }
#pragma unroll
    for (int o = 1; o < C; o <<= 1) {
      const float u = __shfl_up(la, o, 64);
      if (lane >= o) la += u;
    }
    if (lane < C) sB[lane] = la;
  }
  __syncthreads();

  if constexpr (KIND == LIN_FIXED) {
    const int r2 = a.r / 2;
    for (int e = tid; e < n * a.r; e += NTP) {
      const int t = e / a.r, i = e % a.r, p = i % (r2 > 0 ? r2 : 1);
      float* s = (i < r2 ? sQ : sK) + t * PK;
      const float c = a.cs[(row0 + t) * a.r + p], si = a.cs[(row0 + t) * a.r + r2 + p], x = s[p], y = s[p + r2];
      s[p] = x * c - y * si;
      s[p + r2] = y * c + x * si;
    }
    __syncthreads();
  }
  // scales (and unit norms) in place
  for (int t = wave; t < C; t += NWP) {
    float qs = a.qs, ks = a.ks;
    if constexpr (DELTA) {
      float nq = 0.f, nk = 0.f;
      for (int d = lane; d < DKP; d += 64) {
        nq += sQ[t * PK + d] * sQ[t * PK + d];
        nk += sK[t * PK + d] * sK[t * PK + d];
      }
      qs *= 1.f / sqrtf(wave_sum(nq) + 1e-6f);
      ks *= 1.f / sqrtf(wave_sum(nk) + 1e-6f);
    }
    for (int d = lane; d < DKP; d += 64) {
      sQ[t * PK + d] *= qs;
      sK[t * PK + d] *= ks;
    }
  }
  if constexpr (KIND == LIN_CHANNEL) {
    // log decays: z of 16 tokens x 16 channels a wave
    const int fr = lane & 15, g4 = lane >> 4, rp = rank_pitch(a.rank);
    for (int it = wave; it < NB * (DKP / 16); it += NWP) {
      const int t = it % NB * 16, d = it / NB * 16 + fr;
      const float* w = a.w_gate + ((size_t)h * dk + min(d, dk - 1)) * a.rank;
      f32x4 z = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int k0 = 0; k0 < a.rank; k0 += 16) {
        const int k = k0 + 4 * g4;
        const float4 x = *reinterpret_cast<const float4*>(sM + (t + fr) * rp + k);     // zero past the rank
        const int last = a.rank - 1;
        z = mfma(x.x, w[min(k, last)], z);
        z = mfma(x.y, w[min(k + 1, last)], z);
        z = mfma(x.z, w[min(k + 2, last)], z);
        z = mfma(x.w, w[min(k + 3, last)], z);
      }
      const float bias = d < dk ? a.b_gate[h * dk + d] : 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tt = t + 4 * g4 + r;
        sB[tt * PK + d] = d < dk && tt < n ? -softplus_x(-(z[r] + bias)) * a.inv_tau : 0.f;
      }
    }
    __syncthreads();
  }
  if constexpr (CH) {
    // their sums: a thread a channel and a stretch of tokens
    constexpr int NS = NTP / DKP >= 4 ? 4 : NTP / DKP >= 2 ? 2 : 1, TS = C / NS;
    for (int e = tid; e < DKP * NS; e += NTP) {
      const int d = e % DKP, s = e / DKP;
      float sum = 0.f;
#pragma unroll 8
      for (int i = 0; i < TS; ++i) {
        sum += sB[(s * TS + i) * PK + d];
        sB[(s * TS + i) * PK + d] = sum;
      }
    }
    __syncthreads();
    if constexpr (NS > 1) {
      // every stretch's total ahead of it, then added: totals are read before any of them changes
      static_assert(DKP * NS <= NTP, "a thread a stretch");
      const int d = tid % DKP, st = tid / DKP;
      float base = 0.f;
      if (st < NS)
        for (int p = 0; p < st; ++p) base += sB[((p + 1) * TS - 1) * PK + d];
      __syncthreads();
      if (st < NS)
        for (int i = 0; i < TS; ++i) sB[(st * TS + i) * PK + d] += base;
    }
  }
  __syncthreads();

  // blocks of A (and M) on or below the diagonal
  const int fr = lane & 15, g4 = lane >> 4;
  float *gA = sc.A + cid * C * C, *gU = sc.U + cid * C * dvq;
  int item = 0;
  for (int i = 0; i < NB; ++i)
    for (int j = 0; j <= i; ++j) {
      if (item++ % NWP != wave) continue;
      if (CH && i == j) {
        float drop = 0.f;
        for (int d = lane; d < DKP; d += 64) drop = fmaxf(drop, sB[i * 16 * PK + d] - sB[(i * 16 + 15) * PK + d]);
        drop = wave_max(drop);
        if (lane == 0) s_direct[i] = drop > kMaxDrop;
        if (drop > kMaxDrop) continue;
      }
      f32x4 qa = f32x4{0.f, 0.f, 0.f, 0.f}, ka = qa;
      const int tr = i * 16 + fr, sr = j * 16 + fr, ref = i == j ? i * 16 + 7 : i * 16 - 1;
#pragma unroll 4
      for (int k0 = 0; k0 < DKP; k0 += 16) {
        const int k = k0 + 4 * g4;
        float4 q = *reinterpret_cast<const float4*>(sQ + tr * PK + k);
        float4 ks = *reinterpret_cast<const float4*>(sK + sr * PK + k), kt;
        if constexpr (DELTA) kt = *reinterpret_cast<const float4*>(sK + tr * PK + k);
        if constexpr (CH) {
          const float4 bt = *reinterpret_cast<const float4*>(sB + tr * PK + k), bs = *reinterpret_cast<const float4*>(sB + sr * PK + k);
          const float4 br = *reinterpret_cast<const float4*>(sB + ref * PK + k);
          const float4 f = make_float4(__expf(bt.x - br.x), __expf(bt.y - br.y), __expf(bt.z - br.z), __expf(bt.w - br.w));
          q.x *= f.x; q.y *= f.y; q.z *= f.z; q.w *= f.w;
          if constexpr (DELTA) {
            kt.x *= f.x; kt.y *= f.y; kt.z *= f.z; kt.w *= f.w;
          }
          ks.x *= __expf(br.x - bs.x); ks.y *= __expf(br.y - bs.y); ks.z *= __expf(br.z - bs.z); ks.w *= __expf(br.w - bs.w);
        }
        qa = mfma(q.x, ks.x, qa); qa = mfma(q.y, ks.y, qa); qa = mfma(q.z, ks.z, qa); qa = mfma(q.w, ks.w, qa);
        if constexpr (DELTA) {
          ka = mfma(kt.x, ks.x, ka); ka = mfma(kt.y, ks.y, ka); ka = mfma(kt.z, ks.z, ka); ka = mfma(kt.w, ks.w, ka);
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = i * 16 + 4 * g4 + r, s = j * 16 + fr;
        float f = 1.f;
        if constexpr (!CH) f = s <= t ? expf(sB[t] - sB[s]) : 0.f;
        gA[t * C + s] = s <= t ? qa[r] * f : 0.f;
        if constexpr (DELTA) sM[t * PM + s] = s < t ? sbeta[t] * ka[r] * f : 0.f;
      }
    }
  if constexpr (CH) {
    __syncthreads();
    const int t16 = (tid >> 4) & 15, s16 = tid & 15;
    for (int i = tid >> 8; i < NB; i += NTP / 256) {
      if (!s_direct[i]) continue;
      const int t = i * 16 + t16, s = i * 16 + s16;
      float acc = 0.f, kk = 0.f;
      if (s <= t) {
        for (int d = 0; d < DKP; d += 4) {
          const float4 q = *reinterpret_cast<const float4*>(sQ + t * PK + d);
          float4 k = *reinterpret_cast<const float4*>(sK + s * PK + d);
          const float4 bt = *reinterpret_cast<const float4*>(sB + t * PK + d), bs = *reinterpret_cast<const float4*>(sB + s * PK + d);
          k.x *= __expf(bt.x - bs.x); k.y *= __expf(bt.y - bs.y); k.z *= __expf(bt.z - bs.z); k.w *= __expf(bt.w - bs.w);
          acc += q.x * k.x + q.y * k.y + q.z * k.z + q.w * k.w;
          if constexpr (DELTA) {
            const float4 kt = *reinterpret_cast<const float4*>(sK + t * PK + d);
            kk += kt.x * k.x + kt.y * k.y + kt.z * k.z + kt.w * k.w;
          }
        }
      }
      gA[t * C + s] = acc;
      if constexpr (DELTA) sM[t * PM + s] = s < t ? sbeta[t] * kk : 0.f;
    }
  }
  if constexpr (DELTA) __syncthreads();

  // Q' and K' (transposed), the chunk's decay
  float *gQ = sc.Q + cid * C * DKP, *gK = sc.K + cid * C * DKP;
  for (int e = tid; e < C * (DKP / 4); e += NTP) {
    const int t = e / (DKP / 4), d = (e % (DKP / 4)) * 4;
    float4 q = *reinterpret_cast<const float4*>(sQ + t * PK + d);
    float4 f;
    if constexpr (CH) {
      const float4 bt = *reinterpret_cast<const float4*>(sB + t * PK + d);
      f = make_float4(__expf(bt.x), __expf(bt.y), __expf(bt.z), __expf(bt.w));
    } else {
      const float x = expf(sB[t]);
      f = make_float4(x, x, x, x);
    }
    *reinterpret_cast<float4*>(gQ + t * DKP + d) = make_float4(q.x * f.x, q.y * f.y, q.z * f.z, q.w * f.w);
  }
  for (int e = tid; e < C * DKP; e += NTP) {
    const int d = e / C, t = e % C;
    const float f = CH ? __expf(sB[(C - 1) * PK + d] - sB[t * PK + d]) : expf(sB[C - 1] - sB[t]);
    gK[e] = sK[t * PK + d] * f;
  }
  for (int d = tid; d < DKP; d += NTP) sc.G[cid * DKP + d] = CH ? expf(sB[(C - 1) * PK + d]) : expf(sB[C - 1]);

  if constexpr (!DELTA) {
    for (int e = tid; e < C * (dvq / V); e += NTP) {
      const int t = e / (dvq / V), c = (e % (dvq / V)) * V;
      float v[V];
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = 0.f;
      if (t < n && c < dv) ldx<V>(a.X, a.xf32, a.Sx, a.xslab, (row0 + t) * a.ldx + a.vo + h * dv + c, v);
      stv<V>(gU + t * dvq + c, v);
    }
  }
  if constexpr (DELTA) {
    if (tid < C) {                              // a thread a column of a diagonal block's inverse
      const int i0 = tid & ~15, c = tid & 15;
      float x[16];
#pragma unroll
      for (int t = 0; t < 16; ++t) {
        float acc = t == c ? 1.f : 0.f;
#pragma unroll
        for (int s = 0; s < t; ++s) acc -= sM[(i0 + t) * PM + i0 + s] * x[s];
        x[t] = acc;
        sT[(i0 + t) * PT + c] = acc;
      }
    }
    __syncthreads();
    // a wave 16 columns of [beta v | beta e^b k], block of tokens after block
    float *gW = sc.W + cid * C * DKP, *buf = sQ + wave * C * PT;
    for (int ct = wave; ct < (dvq + DKP) / 16; ct += NWP) {
      const bool val = ct * 16 < dvq;
      const int c = ct * 16 - (val ? 0 : dvq) + fr;
      float y[NB][4];
      if (val) {
        const size_t col = (size_t)a.vo + h * dv + min(c, dv - 1);
        if (a.Sx == 1 && !a.xf32) {             // all of them in flight together
          const uint16_t* X = (const uint16_t*)a.X + col;
#pragma unroll
          for (int i = 0; i < NB; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) y[i][r] = ld1(X + (row0 + min(i * 16 + 4 * g4 + r, n - 1)) * a.ldx);
        } else {
#pragma unroll
          for (int i = 0; i < NB; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r)
              y[i][r] = ldx1(a.X, a.xf32, a.Sx, a.xslab, (row0 + min(i * 16 + 4 * g4 + r, n - 1)) * a.ldx + col);
        }
      }
#pragma unroll
      for (int i = 0; i < NB; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = i * 16 + 4 * g4 + r;
          y[i][r] = sbeta[t] * (val ? (t < n && c < dv ? y[i][r] : 0.f) : expf(sB[CH ? t * PK + c : t]) * sK[t * PK + c]);
        }
#pragma unroll
      for (int i = 0; i < NB; ++i) {
        f32x4 x = f32x4{0.f, 0.f, 0.f, 0.f}, acc = x;
#pragma unroll
        for (int j = 0; j < i; ++j) {
          const float4 m = *reinterpret_cast<const float4*>(sM + (i * 16 + fr) * PM + j * 16 + 4 * g4);
          const float* p = buf + (j * 16 + 4 * g4) * PT + fr;
          acc = mfma(m.x, p[0], acc); acc = mfma(m.y, p[PT], acc); acc = mfma(m.z, p[2 * PT], acc); acc = mfma(m.w, p[3 * PT], acc);
        }
        float* p = buf + (i * 16 + 4 * g4) * PT + fr;
#pragma unroll
        for (int r = 0; r < 4; ++r) p[r * PT] = y[i][r] - acc[r];
        wave_lds_sync();
        const float4 m = *reinterpret_cast<const float4*>(sT + (i * 16 + fr) * PT + 4 * g4);
        x = mfma(m.x, p[0], x); x = mfma(m.y, p[PT], x); x = mfma(m.z, p[2 * PT], x); x = mfma(m.w, p[3 * PT], x);
        wave_lds_sync();
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = i * 16 + 4 * g4 + r;
          p[r * PT] = x[r];
          if (val) gU[t * dvq + c] = x[r];
          else gW[t * DKP + c] = x[r];
        }
        wave_lds_sync();
      }
    }
  }
}

// LDS reads and writes of every wave before it are done; loads from memory stay in flight
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// 4 waves; S rows in 16-row tiles dealt to the waves, token rows 16 to a wave.  A chunk's operands are in
// registers when its turn comes: each is loaded for the next chunk right after its use.
template <int C, int DKP, int NT, bool DELTA>
__global__ __launch_bounds__(256) void linear_chunk_kernel(ScanArgs sc) {
  constexpr int DVT = 16 * NT, PS = DVT + 4, RT = DKP / 16, RPW = (RT + 3) / 4, NTT = C / 16;
  __shared__ float sS[DKP * PS];
  __shared__ float sV[C * PS];
  const DocqaLinear& a = sc.a;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, fr = lane & 15, g4 = lane >> 4;
  const int dv = a.dv, dvp = (dv + 3) & ~3, dvq = (dv + 15) & ~15, tiles = (dvq + DVT - 1) / DVT;
  const int u = xcd_remap(blockIdx.x, gridDim.x);              // a head's tiles share an L2
  const int ct = u % tiles, h = u / tiles % a.H, b = u / (tiles * a.H);
  const int q0 = sc.cu[b], L = sc.cu[b + 1] - q0, c0 = ct * DVT, slot = a.slots[b];
  if (L <= 0) return;
  const bool carry = sc.ctx[b] > 0 && slot >= 0;
  float* st = a.state + ((size_t)max(slot, 0) * a.H + h) * a.dk * dvp;
  f32x4 S[RPW][NT];
#pragma unroll
  for (int q = 0; q < RPW; ++q) {
    const int rt = wave + 4 * q;
#pragma unroll
    for (int c = 0; c < NT; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = rt * 16 + 4 * g4 + r, col = c0 + c * 16 + fr;
        S[q][c][r] = carry && rt < RT && d < a.dk && col < dv ? st[(size_t)d * dvp + col] : 0.f;
      }
  }
  auto publish = [&]() {
#pragma unroll
    for (int q = 0; q < RPW; ++q) {
      const int rt = wave + 4 * q;
      if (rt < RT)
#pragma unroll
        for (int c = 0; c < NT; ++c)
#pragma unroll
          for (int r = 0; r < 4; ++r) sS[(rt * 16 + 4 * g4 + r) * PS + c * 16 + fr] = S[q][c][r];
    }
  };
  // k runs in steps of 16, lane group g4 taking 4 consecutive k (any order will do if both operands share it)
  auto step = [&](const float4& x, const float* B, int k0, f32x4* acc) {
    const float* br = B + (k0 + 4 * g4) * PS + fr;
#pragma unroll
    for (int c = 0; c < NT; ++c) {
      acc[c] = mfma(x.x, br[c * 16], acc[c]);
      acc[c] = mfma(x.y, br[PS + c * 16], acc[c]);
      acc[c] = mfma(x.z, br[2 * PS + c * 16], acc[c]);
      acc[c] = mfma(x.w, br[3 * PS + c * 16], acc[c]);
    }
  };
  const int wt = min(wave, NTT - 1);                           // the wave's token tile (the last one's loads are idle copies)
  float4 rW[DELTA ? RT : 1], rQ[RT], rA[NTT], rK[RPW][NTT], rG[RPW];
  float rV[4 * NT];
  auto row16 = [&](const float* p, int ld) { return reinterpret_cast<const float4*>(p + (size_t)fr * ld + 4 * g4); };
  auto load_w = [&](size_t cid) {
    if constexpr (DELTA) {
      const float4* p = row16(sc.W + (cid * C + wt * 16) * DKP, DKP);
#pragma unroll
      for (int k = 0; k < RT; ++k) rW[k] = p[k * 4];
    }
  };
  auto load_v = [&](size_t cid) {
#pragma unroll
    for (int c = 0; c < NT; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        rV[c * 4 + r] = sc.U[(cid * C + wt * 16 + 4 * g4 + r) * dvq + min(c0 + c * 16 + fr, dvq - 1)];
  };
  auto load_qa = [&](size_t cid) {
    const float4 *p = row16(sc.Q + (cid * C + wt * 16) * DKP, DKP), *q = row16(sc.A + (cid * C + wt * 16) * C, C);
#pragma unroll
    for (int k = 0; k < RT; ++k) rQ[k] = p[k * 4];
#pragma unroll
    for (int k = 0; k < NTT; ++k) rA[k] = q[k * 4];
  };
  auto load_k = [&](size_t cid) {
#pragma unroll
    for (int q = 0; q < RPW; ++q) {
      const int rt = min(wave + 4 * q, RT - 1);
      const float4* p = row16(sc.K + (cid * DKP + rt * 16) * C, C);
#pragma unroll
      for (int k = 0; k < NTT; ++k) rK[q][k] = p[k * 4];
      rG[q] = *reinterpret_cast<const float4*>(sc.G + cid * DKP + rt * 16 + 4 * g4);
    }
  };
  const int chunks = (L + C - 1) / C;
  const size_t id0 = chunk_id(sc, b, 0, C) * a.H + h;          // chunk ck's: id0 + ck H
  load_w(id0);
  load_v(id0);
  load_qa(id0);
  load_k(id0);
  publish();
#pragma unroll 1
  for (int ck = 0; ck < chunks; ++ck) {
    const int n = min(C, L - ck * C), nx = min(ck + 1, chunks - 1);
    const size_t row0 = q0 + ck * C, nid = id0 + (size_t)nx * a.H;
    lds_barrier();                                     // sS is written, sV free
    f32x4 w[NT], acc[NT];
#pragma unroll
    for (int c = 0; c < NT; ++c) w[c] = acc[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (wave < NTT) {
      if constexpr (DELTA) {
#pragma unroll
        for (int k = 0; k < RT; ++k) step(rW[k], sS, k * 16, w);
      }
#pragma unroll
      for (int c = 0; c < NT; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          sV[(wave * 16 + 4 * g4 + r) * PS + c * 16 + fr] = c0 + c * 16 + fr < dvq ? rV[c * 4 + r] - w[c][r] : 0.f;
    }
    load_w(nid);
    load_v(nid);
    lds_barrier();
    if (wave < NTT && wave * 16 < n) {
#pragma unroll
      for (int k = 0; k < RT; ++k) step(rQ[k], sS, k * 16, acc);
#pragma unroll
      for (int k = 0; k < NTT; ++k)
        if (k <= wave) step(rA[k], sV, k * 16, acc);
    }
    load_qa(nid);
    if (wave < NTT) {
#pragma unroll
      for (int c = 0; c < NT; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = wave * 16 + 4 * g4 + r, col = c0 + c * 16 + fr;
          if (t < n && col < dvq) sc.O[((row0 + t) * a.H + h) * dvq + col] = acc[c][r];
        }
    }
#pragma unroll
    for (int q = 0; q < RPW; ++q) {
#pragma unroll
      for (int c = 0; c < NT; ++c) {
        S[q][c][0] *= rG[q].x; S[q][c][1] *= rG[q].y; S[q][c][2] *= rG[q].z; S[q][c][3] *= rG[q].w;
      }
#pragma unroll
      for (int k = 0; k < NTT; ++k) step(rK[q][k], sV, k * 16, S[q]);
    }
    load_k(nid);
    lds_barrier();                                     // everyone has read sS
    publish();
  }
  if (slot < 0) return;
#pragma unroll
  for (int q = 0; q < RPW; ++q) {
    const int rt = wave + 4 * q;
#pragma unroll
    for (int c = 0; c < NT; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = rt * 16 + 4 * g4 + r, col = c0 + c * 16 + fr;
        if (rt < RT && d < a.dk && col < dv) st[(size_t)d * dvp + col] = S[q][c][r];
      }
  }
}

// LR lanes a (token, head), V columns at a time each, NI times
template <int LR, int V, int NI>
__global__ __launch_bounds__(256) void linear_gate_kernel(DocqaLinear a, const float* __restrict__ O, int tokens) {
  const int u = blockIdx.x * (256 / LR) + threadIdx.x / LR, lane = threadIdx.x % LR;
  const int t = u / a.H, h = u % a.H, dv = a.dv, dvq = (dv + 15) & ~15;
  const bool ok = t < tokens;
  const float* o = O + ((size_t)(ok ? t : 0) * a.H + h) * dvq;
  float x[NI][V], ss = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (lane + LR * i) * V;
#pragma unroll
    for (int j = 0; j < V; ++j) x[i][j] = 0.f;
    if (c < dv) ldv<V>(o + c, x[i]);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += x[i][j] * x[i][j];
  }
  const float inv = 1.f / sqrtf(group_sum<LR>(ss) / (float)dv + a.eps);
  if (!ok) return;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (lane + LR * i) * V;
    if (c >= dv) continue;
    float g[V], w[V];
    ldx<V>(a.Z, a.zf32, a.Sz, a.zslab, (size_t)t * a.ldz + a.go + h * dv + c, g);
    ldv<V>(a.norm + c, w);
#pragma unroll
    for (int j = 0; j < V; ++j) g[j] = x[i][j] * inv * w[j] * (a.sig ? 1.f : g[j]) * sigmoid_f(g[j]);
    const size_t at = (size_t)t * a.ldo + h * dv + c;
    if (a.of32) stv<V>((float*)a.out + at, g);
    else stv<V>((uint16_t*)a.out + at, g);
  }
}

template <int LR, int V, int NI>
void launch_gate(const DocqaLinear& a, const float* O, int tokens, hipStream_t s) {
  const long long rows = (long long)tokens * a.H;
  linear_gate_kernel<LR, V, NI><<<(unsigned)((rows + 256 / LR - 1) / (256 / LR)), 256, 0, s>>>(a, O, tokens);
}

template <int C, int DKP, int KIND>
int launch_scan(const ScanArgs& sc, int tokens, int B, hipStream_t s) {
  constexpr int PK = DKP + 4;
  constexpr bool CH = KIND == LIN_CHANNEL || KIND == LIN_CHANNEL_DELTA, DELTA = KIND >= LIN_DELTA;
  const DocqaLinear& a = sc.a;
  const size_t low = KIND == LIN_CHANNEL ? (size_t)C * rank_pitch(a.rank) : DELTA ? (size_t)C * (C + 4 + PT + 1) : 0;
  const size_t lds = (prep_q(C, DKP, DELTA) + C * PK + (CH ? C * PK : C) + low) * 4;
  if (lds > 160 * 1024 - 64) return -1;
  const bool vec = (KIND != LIN_CHANNEL_DELTA || (docqa_aligned16(a.Z) && docqa_aligned16(a.b_gate) && a.ao % 4 == 0 && a.ldz % 4 == 0)) &&
                   docqa_aligned16(a.X) && a.dk % 4 == 0 && a.qo % 4 == 0 && a.ko % 4 == 0 && a.ldx % 4 == 0 && a.dv % 4 == 0 &&
                   a.vo % 4 == 0;
  dim3 grid(a.H, sc.nchunk, B);
  auto prep = vec ? linear_prep_kernel<C, DKP, KIND, 4> : linear_prep_kernel<C, DKP, KIND, 1>;
  if (lds > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(prep), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  prep<<<grid, NTP, lds, s>>>(sc);
  DOCQA_CHECK_LAUNCH();
  const int dvq = (a.dv + 15) & ~15;
  const long long one = (long long)B * a.H * (dvq / 16);
  // narrow tiles while they leave CUs without a workgroup
  if (one <= 512 || dvq == 16) linear_chunk_kernel<C, DKP, 1, DELTA><<<(unsigned)one, 256, 0, s>>>(sc);
  else linear_chunk_kernel<C, DKP, 2, DELTA><<<(unsigned)((long long)B * a.H * ((dvq + 31) / 32)), 256, 0, s>>>(sc);
  DOCQA_CHECK_LAUNCH();
  const bool v4 = a.dv % 4 == 0 && a.go % 4 == 0 && a.ldz % 4 == 0 && a.ldo % 4 == 0 && docqa_aligned16(a.Z) &&
                  docqa_aligned16(a.out) && docqa_aligned16(a.norm);
  if (!v4) launch_gate<64, 1, 8>(a, sc.O, tokens, s);
  else if (a.dv <= 64) launch_gate<16, 4, 1>(a, sc.O, tokens, s);
  else if (a.dv <= 128) launch_gate<32, 4, 1>(a, sc.O, tokens, s);
  else launch_gate<64, 4, 2>(a, sc.O, tokens, s);
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int dk_pad(int dk) { return dk <= 64 ? 64 : dk <= 128 ? 128 : 256; }

template <int KIND>
int dispatch_scan(const ScanArgs& sc, int tokens, int B, hipStream_t s) {
  switch (dk_pad(sc.a.dk)) {
    case 64: return launch_scan<64, 64, KIND>(sc, tokens, B, s);
    case 128: return launch_scan<64, 128, KIND>(sc, tokens, B, s);
    default: return launch_scan<32, 256, KIND>(sc, tokens, B, s);
  }
}
}  // namespace

int docqa_linear_step(const DocqaLinear& a, const int* positions, int B, hipStream_t s) {
  if (B == 0) return 0;
  if (a.dk < 1 || a.dk > 256 || a.dv < 1 || a.dv > 512 || B > 65535 || !docqa_aligned16(a.state)) return -1;
  const bool tall = a.dk > 128;
  if (tall && a.dv > 256) return -1;
  const int waves = tall ? (a.dv + 15) / 16 : (a.dv + 31) / 32, dvp = (a.dv + 3) & ~3;
  const size_t lds = (size_t)(3 * (tall ? 256 : a.dk <= 64 ? 64 : 128) + 2 * dvp + a.rank + waves) * 4;
  dim3 grid(a.H, B);
#define RUN(CG, NR, MT) linear_step_kernel<CG, NR, MT><<<grid, 64 * waves, lds, s>>>(a, positions)
#define GO(CG, NR)                        \
  do {                                    \
    if (waves <= 4) RUN(CG, NR, 256);     \
    else if (waves <= 8) RUN(CG, NR, 512); \
    else RUN(CG, NR, 1024);               \
  } while (0)
  if (tall) GO(4, 16);
  else if (a.dk <= 64) GO(8, 8);
  else GO(8, 16);
#undef GO
#undef RUN
  DOCQA_CHECK_LAUNCH();
  return 0;
}

int docqa_linear_chunk(int dk) { return dk <= 128 ? 64 : 32; }

namespace {
struct Sizes {
  size_t Q, A, G, W, U, O, total;
};
Sizes scratch_sizes(int kind, int tokens, int B, int H, int dk, int dv) {
  const size_t C = docqa_linear_chunk(dk), dkp = dk_pad(dk), dvq = (dv + 15) & ~15;
  const size_t n = (tokens / C + B + 1) * H;          // chunk ids are below tokens / C + B
  const bool delta = kind >= LIN_DELTA;
  Sizes z{n * C * dkp, n * C * C, n * dkp, delta ? n * C * dkp : 0, n * C * dvq, (size_t)tokens * H * dvq, 0};
  z.total = 2 * z.Q + z.A + z.G + z.W + z.U + z.O;
  return z;
}
}  // namespace

size_t docqa_linear_scratch(int kind, int tokens, int B, int H, int dk, int dv) {
  return scratch_sizes(kind, tokens, B, H, dk, dv).total;
}

int docqa_linear_scan(const DocqaLinear& a, const int* cu, const int* ctx, float* scratch, int tokens, int B, int max_len,
                      hipStream_t s) {
  if (B == 0 || max_len == 0) return 0;
  if (a.dk < 1 || a.dk > 256 || a.dv < 1 || a.dv > 512 || B > 65535) return -1;
  const int C = docqa_linear_chunk(a.dk);
  const Sizes z = scratch_sizes(a.kind, tokens, B, a.H, a.dk, a.dv);
  ScanArgs sc{a, cu, ctx, (max_len + C - 1) / C, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr};
  if (sc.nchunk > 65535) return -1;
  sc.Q = scratch; sc.K = sc.Q + z.Q; sc.A = sc.K + z.Q; sc.W = sc.A + z.A; sc.U = sc.W + z.W; sc.O = sc.U + z.U; sc.G = sc.O + z.O;
  if (a.kind == LIN_CHANNEL) return dispatch_scan<LIN_CHANNEL>(sc, tokens, B, s);
  if (a.kind == LIN_FIXED) return dispatch_scan<LIN_FIXED>(sc, tokens, B, s);
  if (a.kind == LIN_DELTA) return dispatch_scan<LIN_DELTA>(sc, tokens, B, s);
  return dispatch_scan<LIN_CHANNEL_DELTA>(sc, tokens, B, s);
}

// ------------------------------------------------------------------ projections through few elements
namespace {
struct LowRank {
  const uint16_t* z;              // [T, ldz]: columns [Ka | Kg | n] from `at` on
  int ldz, at;
  const uint16_t *wa, *wg;        // [Na, Ka], [Ng, Kg]
  int Na, Ka, Ng, Kg, n;
  float* y;                       // [T, Na + Ng + n]
  int T;
};
// 16 MT rows x 64 NJ outputs of one of the two products, rows staged in LDS; the first workgroup of a
// row tile carries the other columns
template <int MT, int NJ>
__global__ __launch_bounds__(256) void low_rank_kernel(LowRank a) {
  extern __shared__ __attribute__((aligned(16))) uint16_t sx[];       // [16 MT][pitch]
  const int ta = (a.Na + 64 * NJ - 1) / (64 * NJ);
  const bool gate = (int)blockIdx.x >= ta;
  const int K = gate ? a.Kg : a.Ka, N = gate ? a.Ng : a.Na, off = gate ? a.Ka : 0, yo = gate ? a.Na : 0, ldy = a.Na + a.Ng + a.n;
  const int kp = (K + 31) / 32 * 32, pitch = kp + 8, m0 = blockIdx.y * 16 * MT, tid = threadIdx.x;
  const uint16_t *x = a.z + a.at + off, *w = gate ? a.wg : a.wa;
  const bool vec = ((reinterpret_cast<uintptr_t>(x) | (size_t)a.ldz * 2) & 15) == 0;
  const int per = kp / 8;
  for (int i = tid; i < 16 * MT * per; i += 256) {
    const int r = i / per, c = (i - r * per) * 8;
    union {
      uint4 v;
      uint16_t e[8];
    } u;
    u.v = make_uint4(0, 0, 0, 0);
    if (m0 + r < a.T && c < K) {
      const uint16_t* p = x + (size_t)(m0 + r) * a.ldz + c;
      if (vec) u.v = *reinterpret_cast<const uint4*>(p);
      else
#pragma unroll
        for (int j = 0; j < 8; ++j) u.e[j] = p[j];
    }
    *reinterpret_cast<uint4*>(sx + r * pitch + c) = u.v;
  }
  if (blockIdx.x == 0)
    for (int i = tid; i < 16 * MT * a.n; i += 256) {
      const int r = i / a.n, c = i - r * a.n;
      if (m0 + r < a.T) a.y[(size_t)(m0 + r) * ldy + a.Na + a.Ng + c] = bf2f(a.z[(size_t)(m0 + r) * a.ldz + a.at + a.Ka + a.Kg + c]);
    }
  __syncthreads();
  const int lane = tid & 63, wave = tid >> 6, fr = lane & 15, g4 = lane >> 4;
  const int n0 = (((int)blockIdx.x - (gate ? ta : 0)) * 4 + wave) * 16 * NJ;
  if (n0 >= N) return;
  f32x4 acc[MT][NJ];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NJ; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 0; k < kp; k += 32) {
    const int kk = k + g4 * 8;
    bf16x8 wf[NJ], xf[MT];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int n = n0 + 16 * j + fr;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (n < N && kk < K) v = *reinterpret_cast<const uint4*>(w + (size_t)n * K + kk);
      wf[j] = *reinterpret_cast<bf16x8*>(&v);
    }
#pragma unroll
    for (int i = 0; i < MT; ++i) xf[i] = *reinterpret_cast<const bf16x8*>(sx + (i * 16 + fr) * pitch + kk);
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < NJ; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[j], xf[i], acc[i][j], 0, 0, 0);
  }
  const bool v4 = ((ldy | N | yo) & 3) == 0;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int row = m0 + i * 16 + fr;
    if (row >= a.T) continue;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int n = n0 + 16 * j + g4 * 4;
      float* o = a.y + (size_t)row * ldy + yo + n;
      const float f[4] = {acc[i][j][0], acc[i][j][1], acc[i][j][2], acc[i][j][3]};
      if (v4) {
        if (n < N) stv<4>(o, f);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (n + r < N) o[r] = f[r];
      }
    }
  }
}
}  // namespace

int docqa_low_rank(const void* z, int ldz, int at, const void* wa, int Na, int Ka, const void* wg, int Ng, int Kg, int n,
                   float* y, int T, hipStream_t s) {
  if (T == 0) return 0;
  if (Na < 1 || Ng < 1 || n < 0 || Ka < 8 || Ka % 8 || Kg < 8 || Kg % 8 || Ka > 1024 || Kg > 1024 || at < 0 || at + Ka + Kg + n > ldz)
    return -1;
  if (!docqa_aligned16(wa) || !docqa_aligned16(wg) || !docqa_aligned16(y)) return -1;
  const LowRank a{(const uint16_t*)z, ldz, at, (const uint16_t*)wa, (const uint16_t*)wg, Na, Ka, Ng, Kg, n, y, T};
  const int K = Ka > Kg ? Ka : Kg, pitch = (K + 31) / 32 * 32 + 8;
#define GO(MT, NJ)                                                                                                          \
  low_rank_kernel<MT, NJ><<<dim3((Na + 64 * NJ - 1) / (64 * NJ) + (Ng + 64 * NJ - 1) / (64 * NJ), (T + 16 * MT - 1) / (16 * MT)), \
                            256, (size_t)16 * MT * pitch * 2, s>>>(a)
  if (T > 64 && K <= 256) GO(4, 2);
  else GO(1, 1);
#undef GO
  DOCQA_CHECK_LAUNCH();
  return 0;
}
