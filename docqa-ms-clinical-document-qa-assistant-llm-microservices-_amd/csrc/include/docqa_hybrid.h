// docqa_hybrid.h -- host launchers of the kernels behind hybrid recurrent / windowed- and latent-
// attention decoders (sandwich_norm.hip, attn_window.hip, attn_latent.hip, side_input.hip, ssm.hip,
// act.hip).  Same rules as
// docqa_kernels.h: 0 on success, negative for an unsupported shape, else a hipError_t; nothing
// is allocated and nothing synchronises.  "f32" flags pick fp32 over bf16 storage; P operands
// are S split-K slabs (S = 1: the product itself).
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

int docqa_sandwich_rmsnorm(const void* P, int p_f32, int S, float* res, const float* w_post, const float* add,
                           const float* w_next, void* out, int out_f32, int rows, int H, float eps, hipStream_t s);
int docqa_embed_scale_rmsnorm(const int* ids, const void* table, int f32, float scale, const float* w, float* res,
                              float* emb, void* out, int rows, int H, int vocab, float eps, hipStream_t s);
// sandwich_rmsnorm of one token a row, and h + conv(h): w [taps, H] with the identity in its last tap,
// state [slots, taps - 1, H] of out's type; out2 [rows, H]
int docqa_sandwich_rmsnorm_conv(const void* P, int p_f32, int S, float* res, const float* w_post, const float* w_next,
                                const float* cw, int taps, void* state, const int* slots, const int* positions, void* out,
                                void* out2, int out_f32, int rows, int H, float eps, hipStream_t s);
// res += scale (P + bias) per channel, out = rms(res) w
struct DocqaScaledNorm {
  const void* P;                  // [SP, rows, W]: slabs, or (ids) the SP chosen experts' outputs, of x's type
  int pf32, SP;
  const float *scale, *bias;      // [W]; bias null: none
  const int* ids;                 // [rows, SP] or null; from `experts` on: x itself
  const float* wts;               // [rows, SP]
  const void* x;                  // [rows, W]
  int experts;
  float* res;
  const float* w;
  void* out;
  int of32, rows, W;
  float eps;
};
int docqa_scaled_rmsnorm(const DocqaScaledNorm& a, hipStream_t s);
// z = P + bias [n]: out [T, n_out] = a N(z) + b N(z^2) + c N(z^3) + e, N over the row's RMS, zero past n
int docqa_poly_norm(const void* P, int p_f32, int S, size_t slab, int ld, const float* bias, const float* act, void* out,
                    int out_f32, int T, int n, int n_out, float eps, hipStream_t s);
// res [n] += m (P + Q) (Q null: P alone), each with its own slab count; out null or bf16 [n]: a copy of res
int docqa_add_scaled(const void* P, int p_f32, int SP, const void* Q, int q_f32, int SQ, float* res, float m, void* out,
                     size_t n, hipStream_t s);
// Y [M, N] = act(X [M, K] . W [N, K]^T), bf16, act: docqa_common.h ACT_* (dgemm.hip: M <= 192, N % 64,
// K % 512; mgemm.hip: N % 128, K % 128)
int docqa_gemv_act(const void* X, const void* W, void* Y, int act, int N, int K, hipStream_t s);   // M = 1
int docqa_dgemm_act(const void* X, const void* W, void* Y, int act, int M, int N, int K, hipStream_t s);
int docqa_mgemm_act(const void* X, const void* W, void* Y, int act, int M, int N, int K, hipStream_t s);
int docqa_slab_columns(const void* P, int p_f32, int S, int T, int ld, void* out0, int n0, void* out1, int n1,
                       int out_f32, hipStream_t s);
int docqa_slab_activation(const void* P, int p_f32, int S, size_t n, int act, void* out, int out_f32, hipStream_t s);
int docqa_soft_cap(const void* x, int f32, float* out, size_t n, float cap, hipStream_t s);
// g [M, N] = gelu_tanh(P) * table[ids][col + c] (c < n, else 0); side_project: y [M, W] = g . w [W, N]^T (bf16)
int docqa_side_gate(const void* P, int p_f32, int S, int M, int N, const int* ids, const void* table, int f32, int ld,
                    int vocab, int col, int n, void* out, hipStream_t s);
int docqa_side_project(const void* P, int p_f32, int S, int M, int N, const int* ids, const void* table, int ld,
                       int vocab, int col, int n, const void* w, int W, void* out, hipStream_t s);

int docqa_qk_norm_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* wq, const int* slots,
                        void* q, void* kc, float* ks, int f32, int tokens, int H, int G, int D, int BS, float eps,
                        hipStream_t s);
// cu null: decode (one query token a row, ctx = context length including it); DV: value elements of a row
// (vc == kc: the first DV of the key's D); ldo: elements of an output row; cap 0: scores as they are
int docqa_window_attn(const void* q, const void* kc, const void* vc, const float* k_scale, const int* block_tables,
                      int maxb, const int* cu, const int* ctx, const float* sink, void* out, int ldo, int f32, int B,
                      int max_q, int H, int G, int D, int DV, int BS, float scale, int window, float cap, float out_scale,
                      hipStream_t s);
// P [T, ld]: [q: H D | k: G D | v: G DV | ..]; bias, norm weights qw / kw [D] may be null; cs [T, r]
int docqa_qkv_rope_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* bias, const float* qw,
                         const float* kw, const float* cs, int r, const int* slots, void* q, void* kc, void* vc, int f32,
                         int tokens, int H, int G, int D, int DV, int BS, float eps, hipStream_t s);
// an output gate: row t's head elements i times sigmoid(P[row0 + t, col + i / per])
struct DocqaGate {
  const void* P;            // product or slabs; null: no gate
  int f32, S;
  size_t slab;
  int ld, col, per, row0;
};
// kv [keys, ld] rows [H x d8 keys | H x v8 values], kr [keys, r8]; bf16
int docqa_packed_window_attn(const void* q, const void* kv, const void* kr, const int* cu, const int* cu_k,
                             const float* sink, void* out, int B, int max_q, int H, int d8, int r8, int vdim, int ld,
                             float scale, int window, const DocqaGate& gate, hipStream_t s);

int docqa_rope_table(const int* positions, const double* freq, float* out, int T, int half, double mult, hipStream_t s);
// c_norm null: the projection holds query heads only
int docqa_latent_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* cs, const int* slots,
                       const float* c_norm, void* q, void* cache, int f32, int T, int H, int d, int r, int R, int BS,
                       float eps, hipStream_t s);
// part null: rows x; else the rows are docqa_latent_attn's nsplit partials (E = 0)
int docqa_head_project(const void* x, const void* part, const void* ml, int nsplit, const void* w, void* y, int T, int H,
                       int K, int N, int E, const DocqaGate& gate, hipStream_t s);
// attention in the latent space, bf16, one KV head, values = the first DV elements of a row (sizes:
// latent_attn_ok).  nsplit > 1 (latent_splits): partials for docqa_head_project instead of out -- part
// bf16 [nsplit, tokens H, DV] each split's output, ml float2 [nsplit, tokens H] (maximum, sum)
int docqa_latent_attn_ok(int D, int DV);
int docqa_latent_splits(int B, int max_q, int H, int DV, int max_keys);
int docqa_latent_attn(const void* q, const void* kc, const int* block_tables, int maxb, const int* cu, const int* ctx,
                      const float* sink, void* out, void* part, void* ml, int nsplit, int B, int max_q, int tokens, int H,
                      int D, int DV, int BS, float scale, int window, hipStream_t s);
// P [T, ld]: [query latent Rq | latent R | key part r | ..]: the normed query latent, the cache row
int docqa_latent_norm_store(const void* P, int p_f32, int S, size_t slab, int ld, const float* cs, const int* slots,
                            const float* q_norm, const float* c_norm, void* cq, void* cache, int f32, int T, int Rq, int r,
                            int R, int BS, float eps, hipStream_t s);
int docqa_head_gate(const void* x, int f32, const DocqaGate& gate, void* y, int T, int n, hipStream_t s);   // [T, n]
int docqa_latent_gather(const void* cache, const int* block_tables, int maxb, const int* first, const int* cu_k, void* c,
                        void* kr, int B, int max_keys, int R8, int r8, int BS, hipStream_t s);

int docqa_causal_conv(const void* x, int ldx, const float* w, const float* b, void* state, const int* slots,
                      const int* cu, const int* ctx, void* y, int f32, int B, int max_len, int C, int taps,
                      int silu, hipStream_t s);
int docqa_conv_step(const void* P, int p_f32, int S, size_t slab, int ld, const float* w, const float* b, void* state,
                    const int* slots, const int* positions, void* y, void* z, int f32, int B, int C, int NZ, int taps,
                    int silu, hipStream_t s);
int docqa_selective_scan(const void* x, const void* dt, const void* bc, int ld_bc, int b_off, int c_off,
                         const void* z, int ld_z, const float* A2, const float* D, const float* dt_b, float* state,
                         const int* slots, const int* cu, const int* ctx, void* y, float* cstate, float* csum,
                         int f32, int B, int C, int N, int Np, int chunk, int nchunk, hipStream_t s);
// w_dt (bf16 [C, R], R % 32): the step projection of dt_in [B, R] inside the launch, else dt [B, C]
int docqa_selective_step(const void* x, const void* dt, const void* dt_in, const void* w_dt, int R, const void* bc,
                         int ld_bc, int b_off, int c_off, const void* z, int ld_z, const float* A2, const float* D,
                         const float* dt_b, float* state, const int* slots, const int* positions, void* y, int f32,
                         int B, int C, int N, int Np, hipStream_t s);

// ---- linear attention (linear_attn.hip)
enum { LIN_CHANNEL = 0, LIN_FIXED = 1, LIN_DELTA = 2, LIN_CHANNEL_DELTA = 3 };
struct DocqaLinear {
  const void *X, *Z;        // [tokens, ldx], [tokens, ldz]: products or slabs
  int xf32, Sx, ldx, zf32, Sz, ldz;
  size_t xslab, zslab;
  int kind, H, G, dk, dv, qo, ko, vo, go, ao, bo, rank, r;   // column offsets; rotated dimensions
  int sig;                  // output gate: sigmoid(g), else silu(g)
  float qs, ks, inv_tau, eps;
  const float *w_gate, *b_gate;   // channel: [H dk, rank], [H dk]; fixed: log decay [H], -; delta: -exp(A) [H], [H];
                                  // channel delta: -exp(A) [H], [H dk]
  const float* cs;          // [tokens, r]
  const float* norm;        // [dv]
  float* state;             // [slots, H, dk, dvp], dvp = dv rounded up to 4
  const int* slots;
  void* out;                // [tokens, ldo]
  int of32, ldo;
};
int docqa_linear_step(const DocqaLinear& a, const int* positions, int B, hipStream_t s);
// chunk of a scan and the fp32 scratch (elements) it needs
int docqa_linear_chunk(int dk);
size_t docqa_linear_scratch(int kind, int tokens, int B, int H, int dk, int dv);
int docqa_linear_scan(const DocqaLinear& a, const int* cu, const int* ctx, float* scratch, int tokens, int B, int max_len,
                      hipStream_t s);

// y fp32 [T, Na + Ng + n] of columns [Ka | Kg | n] of z [T, ldz] from `at` on: .. wa [Na, Ka]^T, .. wg [Ng, Kg]^T, as
// they are
int docqa_low_rank(const void* z, int ldz, int at, const void* wa, int Na, int Ka, const void* wg, int Ng, int Kg, int n,
                   float* y, int T, hipStream_t s);

// ---- norms after the sum (sandwich_norm.hip): res <- groupnorm(alpha res + sigmoid(gate[:, col:] + gb) (P + Q)) w
struct DocqaPostNorm {
  const void *P, *Q, *gate;       // null: left out (gate with P)
  int pf32, SP, qf32, SQ, gf32, SG, ldg, col;
  size_t gslab;
  const float* gb;
  float* res;
  const float* w;
  void* out;                      // null: none
  int of32, rows, W, groups;
  float alpha, eps;
};
int docqa_post_norm(const DocqaPostNorm& a, hipStream_t s);

// ---- experts (moe.hip)
int docqa_moe_route(const void* x, const void* w, int f32, int* ids, float* wts, float* rest, int T, int K, int N, int E,
                    int top, hipStream_t s);
// softmax scores, choice by score + corr [N] within the best `keep` of `groups`, weights over their sum times scale
int docqa_moe_route_groups(const void* x, const void* w, int f32, const float* corr, int* ids, float* wts, int T, int K, int N,
                           int top, int groups, int keep, float scale, hipStream_t s);
int docqa_slab_glu(const void* P, int p_f32, int S, size_t slab, int ld, int col, int n, const float* scale, void* out,
                   int out_f32, int T, hipStream_t s);
// int32 scratch of a sorted launch; 0: the rows are found in the launch
int docqa_moe_scratch(int f32, int T, int top, int E, int K, int F, int W);
// limit > 0: clamped experts on x itself (wts unused); ids from E on have no expert, nothing is written for them
int docqa_moe_experts(const void* x, const int* ids, const float* wts, const void* up, const void* down, void* act,
                      void* out, int* scratch, int f32, int T, int top, int E, int K, int F, int W, float limit, hipStream_t s);
