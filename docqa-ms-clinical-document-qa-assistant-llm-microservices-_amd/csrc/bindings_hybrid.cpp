// bindings_hybrid.cpp -- torch operators of the hybrid recurrent / windowed-attention decoder
// kernels (docqa_hybrid.h).  Every shape the kernels index by is checked here against the
// tensors' sizes before a launch.
#include <tuple>

#include "docqa_bind.h"
#include "docqa_hybrid.h"

namespace {

using at::Tensor;
using OptT = c10::optional<Tensor>;

#define CHECK_F32(t) TORCH_CHECK((t).scalar_type() == at::kFloat, #t " must be float32")
#define CHECK_ACT(t)                                                                                  \
  TORCH_CHECK((t).is_cuda() && ((t).scalar_type() == at::kFloat || (t).scalar_type() == at::kBFloat16), \
              #t " must be a bf16 or fp32 GPU tensor")

bool is_f32(const Tensor& t) { return t.scalar_type() == at::kFloat; }

// P [M, N] (a product) or [S, M, N] (split-K slabs), contiguous
struct Slabs {
  int S, M, N;
  size_t slab;
};
Slabs slabs_of(const Tensor& P) {
  CHECK_ACT(P); CHECK_CONTIG(P);
  TORCH_CHECK(P.dim() == 2 || P.dim() == 3, "P must be [M, N] or [S, M, N]");
  const int d = P.dim() - 2;
  const int S = d ? P.size(0) : 1;
  TORCH_CHECK(S >= 1, "P needs at least one slab");
  return {S, (int)P.size(d), (int)P.size(d + 1), (size_t)P.size(d) * P.size(d + 1)};
}
void check_vec(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == n, name,
              ": fp32 vector of ", n, " expected");
}
void check_i32(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() >= n, name,
              ": int32 vector of >= ", n, " expected");
}
// a [rows, cols] view whose rows are contiguous
void check_rows(const Tensor& t, int64_t rows, int64_t cols, const Tensor& like, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == like.scalar_type() && t.dim() == 2 && t.size(0) == rows &&
                  t.size(1) >= cols && t.stride(1) == 1 && (rows <= 1 || t.stride(0) >= cols),
              name, ": rows [", rows, ", >= ", cols, "] of the activations' dtype expected");
}

// gates of `rows` rows of `n` head elements: columns [col, col + n / per) of P from row row0 on
DocqaGate gate_args(const OptT& P, int64_t col, int64_t per, int64_t row0, int64_t rows, int64_t n) {
  DocqaGate g{};
  if (!P.has_value()) return g;
  const Slabs p = slabs_of(*P);
  TORCH_CHECK(per >= 1 && n % per == 0 && col >= 0 && col + n / per <= p.N && row0 >= 0 && row0 + rows <= p.M, "output gate: columns");
  g.P = P->data_ptr(); g.f32 = is_f32(*P); g.S = p.S; g.slab = p.slab; g.ld = p.N; g.col = (int)col; g.per = (int)per; g.row0 = (int)row0;
  return g;
}

Tensor sandwich_rmsnorm(const Tensor& P, Tensor residual, const Tensor& w_post, const OptT& add, const Tensor& w_next,
                        double eps, bool out_f32) {
  const Slabs p = slabs_of(P);
  CHECK_GPU(residual); CHECK_F32(residual); CHECK_CONTIG(residual);
  TORCH_CHECK(residual.dim() == 2 && residual.size(0) == p.M && residual.size(1) == p.N, "residual shape mismatch");
  check_vec(w_post, p.N, "w_post");
  check_vec(w_next, p.N, "w_next");
  const float* ap = nullptr;
  if (add.has_value()) {
    check_vec(*add, residual.numel(), "add");
    ap = add->data_ptr<float>();
  }
  c10::DeviceGuard g(P.device());
  auto out = at::empty({p.M, p.N}, P.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  CHECK_ALIGN16(P); CHECK_ALIGN16(residual); CHECK_ALIGN16(w_post); CHECK_ALIGN16(w_next);
  CHECK_RC(docqa_sandwich_rmsnorm(P.data_ptr(), is_f32(P), p.S, residual.data_ptr<float>(), w_post.data_ptr<float>(),
                                  ap, w_next.data_ptr<float>(), out.data_ptr(), out_f32, p.M, p.N, (float)eps,
                                  stream()),
           "sandwich_rmsnorm");
  return out;
}

std::tuple<Tensor, Tensor, Tensor> embed_scale_rmsnorm(const Tensor& ids, const Tensor& table, double scale,
                                                       const OptT& w, double eps, bool keep) {
  CHECK_ACT(table); CHECK_CONTIG(table); CHECK_ALIGN16(table);
  TORCH_CHECK(table.dim() == 2, "table must be [vocab, width]");
  const int T = ids.numel(), H = table.size(1);
  check_i32(ids, T, "ids");
  if (w.has_value()) {
    check_vec(*w, H, "w");
    CHECK_ALIGN16(*w);
  }
  c10::DeviceGuard g(table.device());
  auto f32 = table.options().dtype(at::kFloat);
  auto res = at::empty({T, H}, f32);
  auto emb = keep ? at::empty({T, H}, f32) : at::empty({0}, f32);
  auto out = at::empty({T, H}, table.options());
  CHECK_RC(docqa_embed_scale_rmsnorm(ids.data_ptr<int>(), table.data_ptr(), is_f32(table), (float)scale,
                                     w.has_value() ? w->data_ptr<float>() : nullptr, res.data_ptr<float>(),
                                     keep ? emb.data_ptr<float>() : nullptr, out.data_ptr(), T, H,
                                     (int)table.size(0), (float)eps, stream()),
           "embed_scale_rmsnorm");
  return {res, emb, out};
}

// residual += m (P + Q); the bf16 copy of it (empty when out_f32)
Tensor add_scaled(const Tensor& P, const OptT& Q, Tensor residual, double m, bool out_f32) {
  const Slabs p = slabs_of(P);
  CHECK_GPU(residual); CHECK_F32(residual); CHECK_CONTIG(residual);
  TORCH_CHECK(residual.dim() == 2 && residual.size(0) == p.M && residual.size(1) == p.N, "residual shape mismatch");
  CHECK_ALIGN16(P); CHECK_ALIGN16(residual);
  Slabs q{1, p.M, p.N, 0};
  if (Q.has_value()) {
    q = slabs_of(*Q);
    TORCH_CHECK(q.M == p.M && q.N == p.N, "Q shape mismatch");
    CHECK_ALIGN16(*Q);
  }
  c10::DeviceGuard g(P.device());
  auto out = at::empty(out_f32 ? at::IntArrayRef({0}) : residual.sizes(), P.options().dtype(at::kBFloat16));
  CHECK_RC(docqa_add_scaled(P.data_ptr(), is_f32(P), p.S, Q.has_value() ? Q->data_ptr() : nullptr,
                            Q.has_value() && is_f32(*Q), q.S, residual.data_ptr<float>(), (float)m,
                            out_f32 ? nullptr : out.data_ptr(), (size_t)p.M * p.N, stream()),
           "add_scaled");
  return out;
}

// residual += scale (P + bias), or scale times the weighted sum of the chosen experts' outputs P; rms(residual) w
Tensor scaled_rmsnorm(const Tensor& P, Tensor residual, const Tensor& scale, const OptT& bias, const OptT& ids, const OptT& wts,
                      int64_t experts, const OptT& x, const Tensor& w, double eps, bool out_f32) {
  const Slabs p = slabs_of(P);
  CHECK_GPU(residual); CHECK_F32(residual); CHECK_CONTIG(residual); CHECK_ALIGN16(residual); CHECK_ALIGN16(P);
  TORCH_CHECK(residual.dim() == 2 && residual.size(0) == p.M && residual.size(1) == p.N, "residual shape mismatch");
  check_vec(scale, p.N, "scale"); check_vec(w, p.N, "w");
  CHECK_ALIGN16(scale); CHECK_ALIGN16(w);
  DocqaScaledNorm a{};
  a.P = P.data_ptr(); a.pf32 = is_f32(P); a.SP = p.S; a.rows = p.M; a.W = p.N;
  if (bias.has_value()) {
    check_vec(*bias, p.N, "bias");
    CHECK_ALIGN16(*bias);
    a.bias = bias->data_ptr<float>();
  }
  if (ids.has_value()) {
    TORCH_CHECK(wts.has_value() && x.has_value() && P.dim() == 3, "scaled_rmsnorm: weights and the experts' input");
    TORCH_CHECK(ids->dim() == 2 && ids->size(0) == p.M && ids->size(1) == p.S, "scaled_rmsnorm: ids [rows, chosen]");
    check_i32(*ids, (int64_t)p.M * p.S, "ids");
    check_vec(*wts, (int64_t)p.M * p.S, "wts");
    CHECK_ACT(*x); CHECK_CONTIG(*x); CHECK_ALIGN16(*x);
    TORCH_CHECK(x->scalar_type() == P.scalar_type() && x->dim() == 2 && x->size(0) == p.M && x->size(1) == p.N, "scaled_rmsnorm: x");
    a.ids = ids->data_ptr<int>(); a.wts = wts->data_ptr<float>(); a.x = x->data_ptr(); a.experts = (int)experts;
  }
  c10::DeviceGuard g(P.device());
  auto out = at::empty({p.M, p.N}, P.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  a.scale = scale.data_ptr<float>(); a.res = residual.data_ptr<float>(); a.w = w.data_ptr<float>(); a.out = out.data_ptr();
  a.of32 = out_f32; a.eps = (float)eps;
  CHECK_RC(docqa_scaled_rmsnorm(a, stream()), "scaled_rmsnorm");
  return out;
}

Tensor poly_norm(const Tensor& P, const Tensor& bias, const Tensor& act, int64_t n_out, double eps, bool out_f32) {
  const Slabs p = slabs_of(P);
  const int n = bias.numel();
  check_vec(bias, n, "bias"); check_vec(act, 4, "act");
  CHECK_ALIGN16(P); CHECK_ALIGN16(bias);
  TORCH_CHECK(n >= 1 && n <= p.N && n_out >= n && n_out <= (1 << 20), "poly_norm: columns");
  c10::DeviceGuard g(P.device());
  auto out = at::empty({p.M, n_out}, P.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  CHECK_RC(docqa_poly_norm(P.data_ptr(), is_f32(P), p.S, p.slab, p.N, bias.data_ptr<float>(), act.data_ptr<float>(),
                           out.data_ptr(), out_f32, p.M, n, (int)n_out, (float)eps, stream()),
           "poly_norm");
  return out;
}

Tensor head_gate(const Tensor& x, const Tensor& P, int64_t col, int64_t per, int64_t row0) {
  CHECK_ACT(x); CHECK_CONTIG(x); CHECK_ALIGN16(x);
  TORCH_CHECK(x.dim() == 2, "head_gate: x must be [rows, heads * dim]");
  const DocqaGate gate = gate_args(P, col, per, row0, x.size(0), x.size(1));
  c10::DeviceGuard g(x.device());
  auto y = at::empty_like(x);
  CHECK_RC(docqa_head_gate(x.data_ptr(), is_f32(x), gate, y.data_ptr(), (int)x.size(0), (int)x.size(1), stream()), "head_gate");
  return y;
}

Tensor soft_cap(const Tensor& x, double cap) {
  CHECK_ACT(x); CHECK_CONTIG(x);
  TORCH_CHECK(cap > 0, "cap");
  c10::DeviceGuard g(x.device());
  auto out = at::empty(x.sizes(), x.options().dtype(at::kFloat));
  CHECK_RC(docqa_soft_cap(x.data_ptr(), is_f32(x), out.data_ptr<float>(), x.numel(), (float)cap, stream()), "soft_cap");
  return out;
}

void check_side(const Slabs& p, const Tensor& ids, const Tensor& table, int64_t col, int64_t n) {
  CHECK_ACT(table); CHECK_CONTIG(table); CHECK_ALIGN16(table);
  TORCH_CHECK(table.dim() == 2 && col >= 0 && n >= 0 && n <= p.N && col + n <= table.size(1), "side columns");
  check_i32(ids, p.M, "ids");
}

Tensor side_gate(const Tensor& P, const Tensor& ids, const Tensor& table, int64_t col, int64_t n, bool out_f32) {
  const Slabs p = slabs_of(P);
  check_side(p, ids, table, col, n);
  CHECK_ALIGN16(P);
  TORCH_CHECK(out_f32 == is_f32(table), "side_gate: the output has the table's dtype");
  c10::DeviceGuard g(P.device());
  auto out = at::empty({p.M, p.N}, table.options());
  CHECK_RC(docqa_side_gate(P.data_ptr(), is_f32(P), p.S, p.M, p.N, ids.data_ptr<int>(), table.data_ptr(), out_f32,
                           (int)table.size(1), (int)table.size(0), (int)col, (int)n, out.data_ptr(), stream()),
           "side_gate");
  return out;
}

Tensor side_project(const Tensor& P, const Tensor& ids, const Tensor& table, int64_t col, int64_t n, const Tensor& w) {
  const Slabs p = slabs_of(P);
  check_side(p, ids, table, col, n);
  CHECK_BF16(table); CHECK_BF16(w); CHECK_GPU(w); CHECK_CONTIG(w);
  TORCH_CHECK(w.dim() == 2 && w.size(1) == p.N, "side_project: w must be [width, N]");
  c10::DeviceGuard g(P.device());
  auto out = at::empty({p.M, w.size(0)}, table.options());
  CHECK_RC(docqa_side_project(P.data_ptr(), is_f32(P), p.S, p.M, p.N, ids.data_ptr<int>(), table.data_ptr(),
                              (int)table.size(1), (int)table.size(0), (int)col, (int)n, w.data_ptr(), (int)w.size(0),
                              out.data_ptr(), stream()),
           "side_project");
  return out;
}

Tensor slab_activation(const Tensor& P, int64_t act, bool out_f32) {
  const Slabs p = slabs_of(P);
  CHECK_ALIGN16(P);
  c10::DeviceGuard g(P.device());
  auto out = at::empty({p.M, p.N}, P.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  CHECK_RC(docqa_slab_activation(P.data_ptr(), is_f32(P), p.S, p.slab, (int)act, out.data_ptr(), out_f32, stream()),
           "slab_activation");
  return out;
}

// act(x . w^T) on the decode GEMMs: the GEMV for one row, skinny up to 192, the mid-M kernel beyond
Tensor decode_act(const Tensor& x, const Tensor& w, int64_t act) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(w); CHECK_CONTIG(x); CHECK_CONTIG(w); CHECK_ALIGN16(x); CHECK_ALIGN16(w);
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && w.size(1) == x.size(1), "decode_act: shapes");
  const int M = x.size(0), N = w.size(0), K = x.size(1);
  c10::DeviceGuard g(x.device());
  auto out = at::empty({M, N}, x.options());
  CHECK_RC(M == 1 && N % 8 == 0 && (K == 2048 || K == 4096)
               ? docqa_gemv_act(x.data_ptr(), w.data_ptr(), out.data_ptr(), (int)act, N, K, stream())
           : M <= 192 && N % 64 == 0 && K % 512 == 0
               ? docqa_dgemm_act(x.data_ptr(), w.data_ptr(), out.data_ptr(), (int)act, M, N, K, stream())
               : docqa_mgemm_act(x.data_ptr(), w.data_ptr(), out.data_ptr(), (int)act, M, N, K, stream()),
           "decode_act");
  return out;
}

// columns [0, n0) and [n0, n0 + n1) of a projection (product or slabs) as two tensors
std::tuple<Tensor, Tensor> slab_columns(const Tensor& P, int64_t n0, int64_t n1, bool out_f32) {
  const Slabs p = slabs_of(P);
  CHECK_ALIGN16(P);
  TORCH_CHECK(n0 >= 0 && n1 >= 0 && n0 % 4 == 0 && n1 % 4 == 0 && p.N % 4 == 0 && n0 + n1 <= p.N, "slab_columns: columns");
  c10::DeviceGuard g(P.device());
  auto opt = P.options().dtype(out_f32 ? at::kFloat : at::kBFloat16);
  auto a = at::empty({p.M, n0}, opt), b = at::empty({p.M, n1}, opt);
  CHECK_RC(docqa_slab_columns(P.data_ptr(), is_f32(P), p.S, p.M, p.N, a.data_ptr(), (int)n0, b.data_ptr(), (int)n1,
                              out_f32, stream()),
           "slab_columns");
  return {a, b};
}

Tensor qk_norm_store(const Tensor& P, const Tensor& w, const Tensor& slots, Tensor k_cache, Tensor k_scale, int64_t H,
                     double eps) {
  const Slabs p = slabs_of(P);
  CHECK_ACT(k_cache); CHECK_CONTIG(k_cache); CHECK_CONTIG(k_scale); CHECK_F32(k_scale);
  TORCH_CHECK(k_cache.dim() == 4, "k_cache must be [blocks, kv heads, block, dim]");
  const int G = k_cache.size(1), BS = k_cache.size(2), D = k_cache.size(3);
  TORCH_CHECK(p.N >= (H + G) * D, "qk_norm_store: projection width");
  TORCH_CHECK(k_scale.numel() == k_cache.numel() / D, "k_scale must be [blocks, kv heads, block]");
  check_vec(w, D, "w");
  check_i32(slots, p.M, "slots");
  c10::DeviceGuard g(P.device());
  CHECK_ALIGN16(P); CHECK_ALIGN16(k_cache); CHECK_ALIGN16(w);
  auto q = at::empty({p.M, H * D}, k_cache.options());
  CHECK_RC(docqa_qk_norm_store(P.data_ptr(), is_f32(P), p.S, p.slab, p.N, w.data_ptr<float>(), slots.data_ptr<int>(),
                               q.data_ptr(), k_cache.data_ptr(), k_scale.data_ptr<float>(), is_f32(k_cache), p.M,
                               (int)H, G, D, BS, (float)eps, stream()),
           "qk_norm_store");
  return q;
}

// cu: [B + 1] query offsets with ctx the first positions (prefill), or null: one query token a
// row with ctx the context lengths (decode)
void window_attn(const Tensor& q, const Tensor& k_cache, const OptT& v_cache, const OptT& k_scale,
                 const Tensor& block_tables, const OptT& cu, const Tensor& ctx, int64_t max_q, double scale,
                 int64_t window, const OptT& sink, int64_t v_dim, double cap, double out_scale, Tensor out) {
  CHECK_ACT(q); CHECK_CONTIG(q); CHECK_CONTIG(k_cache);
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.scalar_type() == q.scalar_type(), "k_cache dtype / shape");
  const int G = k_cache.size(1), BS = k_cache.size(2), D = k_cache.size(3);
  TORCH_CHECK(q.dim() == 2 && q.size(1) % D == 0, "q must be [rows, H * dim]");
  const int H = q.size(1) / D, B = block_tables.size(0);
  const int DV = v_cache.has_value() ? v_cache->size(3) : v_dim ? v_dim : D;
  TORCH_CHECK(DV >= 1 && (v_cache.has_value() ? !v_dim || v_dim == DV : DV <= D), "v_dim: part of the shared row");
  CHECK_GPU(block_tables); CHECK_I32(block_tables); CHECK_CONTIG(block_tables);
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.size(1) >= 1, "block_tables must be [B, blocks]");
  check_i32(ctx, B, "ctx");
  if (cu.has_value()) check_i32(*cu, B + 1, "cu");
  else TORCH_CHECK(q.size(0) == B && max_q == 1, "decode: one query row a sequence");
  TORCH_CHECK(k_cache.numel() / D < (1ll << 31), "cache rows must fit 31 bits");
  if (v_cache.has_value())
    TORCH_CHECK(v_cache->is_cuda() && v_cache->dim() == 4 && v_cache->sizes().slice(0, 3) == k_cache.sizes().slice(0, 3) &&
                    v_cache->scalar_type() == q.scalar_type() && v_cache->is_contiguous() &&
                    (reinterpret_cast<uintptr_t>(v_cache->data_ptr()) & 15u) == 0, "v_cache must match k_cache");
  if (k_scale.has_value()) check_vec(*k_scale, k_cache.numel() / D, "k_scale");
  if (sink.has_value()) check_vec(*sink, H, "sink");
  c10::DeviceGuard g(q.device());
  CHECK_ALIGN16(k_cache);     // cached rows are read in 16-byte pieces, q row by row
  TORCH_CHECK(out.size(1) == (int64_t)H * DV, "window_attn: output width");
  check_rows(out, q.size(0), (int64_t)H * DV, q, "out");
  CHECK_RC(docqa_window_attn(q.data_ptr(), k_cache.data_ptr(), v_cache.has_value() ? v_cache->data_ptr() : k_cache.data_ptr(),
                             k_scale.has_value() ? k_scale->data_ptr<float>() : nullptr, block_tables.data_ptr<int>(),
                             (int)block_tables.size(1), cu.has_value() ? cu->data_ptr<int>() : nullptr,
                             ctx.data_ptr<int>(), sink.has_value() ? sink->data_ptr<float>() : nullptr,
                             out.data_ptr(), (int)out.stride(0), is_f32(q), B, (int)max_q, H, G, D, DV, BS, (float)scale,
                             (int)window, (float)cap, (float)out_scale, stream()),
           "window_attn");
}

Tensor qkv_rope_store(const Tensor& P, const OptT& bias, const OptT& qw, const OptT& kw, const Tensor& cs, const Tensor& slots,
                      Tensor k_cache, Tensor v_cache, int64_t H, double eps) {
  const Slabs p = slabs_of(P);
  CHECK_ACT(k_cache); CHECK_CONTIG(k_cache); CHECK_CONTIG(v_cache); CHECK_ALIGN16(k_cache); CHECK_ALIGN16(v_cache);
  CHECK_ALIGN16(P); CHECK_ALIGN16(cs);
  TORCH_CHECK(k_cache.dim() == 4 && v_cache.dim() == 4 && v_cache.is_cuda() && v_cache.scalar_type() == k_cache.scalar_type() &&
                  v_cache.sizes().slice(0, 3) == k_cache.sizes().slice(0, 3), "caches must be [blocks, kv heads, block, dim]");
  const int G = k_cache.size(1), BS = k_cache.size(2), D = k_cache.size(3), DV = v_cache.size(3);
  TORCH_CHECK(H >= 1 && p.N >= (H + G) * D + (int64_t)G * DV, "qkv_rope_store: projection width");
  auto vec = [](const OptT& t, int64_t n, const char* name) -> const float* {
    if (!t.has_value()) return nullptr;
    check_vec(*t, n, name);
    CHECK_ALIGN16(*t);
    return t->data_ptr<float>();
  };
  TORCH_CHECK(cs.dim() == 2 && cs.size(1) <= D, "cs must be [tokens, r]");
  check_vec(cs, (int64_t)p.M * cs.size(1), "cs");
  check_i32(slots, p.M, "slots");
  c10::DeviceGuard g(P.device());
  auto q = at::empty({p.M, H * D}, k_cache.options());
  CHECK_RC(docqa_qkv_rope_store(P.data_ptr(), is_f32(P), p.S, p.slab, p.N, vec(bias, (H + G) * D + (int64_t)G * DV, "bias"),
                                vec(qw, D, "q norm"), vec(kw, D, "k norm"), cs.data_ptr<float>(), (int)cs.size(1),
                                slots.data_ptr<int>(), q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), is_f32(k_cache),
                                p.M, (int)H, G, D, DV, BS, (float)eps, stream()),
           "qkv_rope_store");
  return q;
}

// window_attn in the latent space (one KV head, values = the first K elements of a cached row, K =
// w.size(2)) followed by head_project with w [H, N, K]; bf16, sizes by docqa_latent_attn_ok
Tensor latent_attn(const Tensor& q, const Tensor& cache, const Tensor& block_tables, const OptT& cu, const Tensor& ctx,
                   int64_t max_q, double scale, int64_t window, const OptT& sink, const Tensor& w, const OptT& gp, int64_t gcol,
                   int64_t gper, int64_t grow) {
  CHECK_GPU(q); CHECK_BF16(q); CHECK_CONTIG(q); CHECK_GPU(cache); CHECK_BF16(cache); CHECK_CONTIG(cache);
  CHECK_GPU(w); CHECK_BF16(w); CHECK_CONTIG(w);
  TORCH_CHECK(cache.dim() == 4 && cache.size(1) == 1 && w.dim() == 3, "latent_attn: cache [blocks, 1, block, D], w [H, N, K]");
  const int BS = cache.size(2), D = cache.size(3), H = w.size(0), N = w.size(1), DV = w.size(2);
  TORCH_CHECK(q.dim() == 2 && q.size(1) == (int64_t)H * D && docqa_latent_attn_ok(D, DV), "latent_attn: sizes");
  const int T = q.size(0), B = block_tables.size(0);
  CHECK_GPU(block_tables); CHECK_I32(block_tables); CHECK_CONTIG(block_tables);
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.size(1) >= 1, "block_tables must be [B, blocks]");
  check_i32(ctx, B, "ctx");
  if (cu.has_value()) check_i32(*cu, B + 1, "cu");
  else TORCH_CHECK(T == B && max_q == 1, "decode: one query row a sequence");
  TORCH_CHECK(cache.numel() / D < (1ll << 31), "cache rows must fit 31 bits");
  if (sink.has_value()) check_vec(*sink, H, "sink");
  CHECK_ALIGN16(cache); CHECK_ALIGN16(q); CHECK_ALIGN16(w);
  c10::DeviceGuard g(q.device());
  const int64_t table = block_tables.size(1) * (int64_t)BS;
  const int keys = (int)(window > 0 ? std::min<int64_t>(window + max_q - 1, table) : table);
  const int ns = docqa_latent_splits(B, (int)max_q, H, DV, keys);
  auto f32 = q.options().dtype(at::kFloat);
  auto x = at::empty({ns > 1 ? 0 : T, (int64_t)H * DV}, q.options());
  auto part = at::empty({ns > 1 ? ns : 0, T, (int64_t)H * DV}, q.options()), ml = at::empty({ns > 1 ? ns : 0, T, H, 2}, f32);
  void* pp = ns > 1 ? part.data_ptr() : nullptr;
  void* mp = ns > 1 ? ml.data_ptr() : nullptr;
  CHECK_RC(docqa_latent_attn(q.data_ptr(), cache.data_ptr(), block_tables.data_ptr<int>(), (int)block_tables.size(1),
                             cu.has_value() ? cu->data_ptr<int>() : nullptr, ctx.data_ptr<int>(),
                             sink.has_value() ? sink->data_ptr<float>() : nullptr, x.data_ptr(), pp, mp, ns, B,
                             (int)max_q, T, H, D, DV, BS, (float)scale, (int)window, stream()),
           "latent_attn");
  auto y = at::empty({T, (int64_t)H * N}, q.options());
  const DocqaGate gate = gate_args(gp, gcol, gper, grow, T, (int64_t)H * N);
  CHECK_RC(docqa_head_project(x.data_ptr(), pp, mp, ns, w.data_ptr(), y.data_ptr(), T, H, DV, N, 0, gate, stream()),
           "latent_attn values");
  return y;
}

Tensor packed_window_attn(const Tensor& q, const Tensor& kv, const Tensor& kr, int64_t H, int64_t dim, int64_t vdim,
                          const Tensor& cu, const Tensor& cu_k, int64_t max_q, double scale, int64_t window,
                          const OptT& sink, const OptT& gp, int64_t gcol, int64_t gper, int64_t grow) {
  CHECK_GPU(q); CHECK_BF16(q); CHECK_BF16(kv); CHECK_BF16(kr); CHECK_CONTIG(q); CHECK_CONTIG(kv); CHECK_CONTIG(kr);
  CHECK_GPU(kv); CHECK_GPU(kr);
  TORCH_CHECK(q.dim() == 2 && kv.dim() == 2 && kr.dim() == 2 && kr.size(0) == kv.size(0) && H >= 1, "packed_window_attn: shapes");
  const int64_t r8 = kr.size(1), d8 = (dim + 7) / 8 * 8;
  TORCH_CHECK(q.size(1) == H * (d8 + r8), "packed_window_attn: query width");
  const int B = cu.numel() - 1;
  check_i32(cu, B + 1, "cu"); check_i32(cu_k, B + 1, "cu_k");
  if (sink.has_value()) check_vec(*sink, H, "sink");
  c10::DeviceGuard g(q.device());
  auto out = at::empty({q.size(0), H * vdim}, q.options());
  CHECK_RC(docqa_packed_window_attn(q.data_ptr(), kv.data_ptr(), kr.data_ptr(), cu.data_ptr<int>(), cu_k.data_ptr<int>(),
                                    sink.has_value() ? sink->data_ptr<float>() : nullptr, out.data_ptr(), B, (int)max_q,
                                    (int)H, (int)d8, (int)r8, (int)vdim, (int)kv.size(1), (float)scale, (int)window,
                                    gate_args(gp, gcol, gper, grow, q.size(0), H * vdim), stream()),
           "packed_window_attn");
  return out;
}

Tensor rope_table(const Tensor& positions, const Tensor& freq, double mult) {
  const int T = positions.numel(), half = freq.numel();
  check_i32(positions, T, "positions");
  TORCH_CHECK(freq.is_cuda() && freq.scalar_type() == at::kDouble && freq.is_contiguous(), "freq: fp64 vector expected");
  c10::DeviceGuard g(positions.device());
  auto out = at::empty({T, 2 * half}, positions.options().dtype(at::kFloat));
  CHECK_RC(docqa_rope_table(positions.data_ptr<int>(), freq.data_ptr<double>(), out.data_ptr<float>(), T, half, mult, stream()),
           "rope_table");
  return out;
}

// P: [q: H (dim + r) | latent: rank | r] (c_norm) or the query heads only -> rotated query heads
Tensor latent_store(const Tensor& P, const Tensor& cs, const Tensor& slots, Tensor cache, const OptT& c_norm, int64_t H,
                    int64_t dim, int64_t rank, double eps) {
  const Slabs p = slabs_of(P);
  CHECK_ACT(cache); CHECK_CONTIG(cache); CHECK_ALIGN16(cache); CHECK_ALIGN16(P); CHECK_ALIGN16(cs);
  TORCH_CHECK(cs.dim() == 2, "cs must be [tokens, r]");
  const int64_t r = cs.size(1), d8 = (dim + 7) / 8 * 8, r8 = (r + 7) / 8 * 8;
  check_vec(cs, p.M * r, "cs");
  check_i32(slots, p.M, "slots");
  TORCH_CHECK(cache.dim() == 4 && cache.size(1) == 1 && cache.size(3) == (rank + 7) / 8 * 8 + r8,
              "cache must be [blocks, 1, block, latent + rotated part]");
  TORCH_CHECK(p.N >= H * (dim + r) + (c_norm.has_value() ? rank + r : 0), "latent_store: projection width");
  if (c_norm.has_value()) {
    check_vec(*c_norm, rank, "c_norm");
    CHECK_ALIGN16(*c_norm);
  }
  c10::DeviceGuard g(P.device());
  auto q = at::empty({p.M, H * (d8 + r8)}, cache.options());
  CHECK_RC(docqa_latent_store(P.data_ptr(), is_f32(P), p.S, p.slab, p.N, cs.data_ptr<float>(), slots.data_ptr<int>(),
                              c_norm.has_value() ? c_norm->data_ptr<float>() : nullptr, q.data_ptr(), cache.data_ptr(),
                              is_f32(cache), p.M, (int)H, (int)dim, (int)r, (int)rank, (int)cache.size(2), (float)eps,
                              stream()),
           "latent_store");
  return q;
}

// P: [query latent | latent: rank | r | ..] -> the normed query latent; the cache row is stored
Tensor latent_norm_store(const Tensor& P, const Tensor& cs, const Tensor& slots, Tensor cache, const Tensor& q_norm,
                         const Tensor& c_norm, double eps) {
  const Slabs p = slabs_of(P);
  CHECK_ACT(cache); CHECK_CONTIG(cache); CHECK_ALIGN16(cache); CHECK_ALIGN16(P); CHECK_ALIGN16(cs);
  TORCH_CHECK(cs.dim() == 2, "cs must be [tokens, r]");
  const int64_t r = cs.size(1), Rq = q_norm.numel(), R = c_norm.numel();
  check_vec(cs, p.M * r, "cs"); check_vec(q_norm, Rq, "q_norm"); check_vec(c_norm, R, "c_norm");
  CHECK_ALIGN16(q_norm); CHECK_ALIGN16(c_norm);
  check_i32(slots, p.M, "slots");
  TORCH_CHECK(cache.dim() == 4 && cache.size(1) == 1 && cache.size(3) == (R + 7) / 8 * 8 + (r + 7) / 8 * 8,
              "cache must be [blocks, 1, block, latent + rotated part]");
  TORCH_CHECK(p.N >= Rq + R + r, "latent_norm_store: projection width");
  c10::DeviceGuard g(P.device());
  auto cq = at::empty({p.M, Rq}, cache.options());
  CHECK_RC(docqa_latent_norm_store(P.data_ptr(), is_f32(P), p.S, p.slab, p.N, cs.data_ptr<float>(), slots.data_ptr<int>(),
                                   q_norm.data_ptr<float>(), c_norm.data_ptr<float>(), cq.data_ptr(), cache.data_ptr(),
                                   is_f32(cache), p.M, (int)Rq, (int)r, (int)R, (int)cache.size(2), (float)eps, stream()),
           "latent_norm_store");
  return cq;
}

Tensor head_project(const Tensor& x, const Tensor& w, int64_t carry) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(w); CHECK_GPU(w); CHECK_CONTIG(x); CHECK_CONTIG(w);
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && carry >= 0 && x.size(1) == w.size(0) * (w.size(2) + carry), "head_project: shapes");
  c10::DeviceGuard g(x.device());
  auto y = at::empty({x.size(0), w.size(0) * (w.size(1) + carry)}, x.options());
  CHECK_RC(docqa_head_project(x.data_ptr(), nullptr, nullptr, 1, w.data_ptr(), y.data_ptr(), (int)x.size(0), (int)w.size(0), (int)w.size(2),
                              (int)w.size(1), (int)carry, DocqaGate{}, stream()),
           "head_project");
  return y;
}

std::tuple<Tensor, Tensor> latent_gather(const Tensor& cache, const Tensor& block_tables, const Tensor& first,
                                         const Tensor& cu_k, int64_t total, int64_t rank) {
  CHECK_GPU(cache); CHECK_BF16(cache); CHECK_CONTIG(cache); CHECK_ALIGN16(cache);
  TORCH_CHECK(cache.dim() == 4 && cache.size(1) == 1 && rank >= 8 && rank < cache.size(3), "latent_gather: cache");
  const int B = block_tables.size(0);
  CHECK_GPU(block_tables); CHECK_I32(block_tables); CHECK_CONTIG(block_tables);
  check_i32(first, B, "first"); check_i32(cu_k, B + 1, "cu_k");
  c10::DeviceGuard g(cache.device());
  const int64_t r8 = cache.size(3) - rank;
  auto c = at::empty({total, rank}, cache.options()), kr = at::empty({total, r8}, cache.options());
  // a sequence's keys are at most the table's blocks, and at most all of them
  const int64_t most = std::min<int64_t>(total, block_tables.size(1) * cache.size(2));
  CHECK_RC(docqa_latent_gather(cache.data_ptr(), block_tables.data_ptr<int>(), (int)block_tables.size(1),
                               first.data_ptr<int>(), cu_k.data_ptr<int>(), c.data_ptr(), kr.data_ptr(), B, (int)most,
                               (int)rank, (int)r8, (int)cache.size(2), stream()),
           "latent_gather");
  return {c, kr};
}

void check_conv(const Tensor& w, const OptT& bias, const Tensor& state, int C, int& taps) {
  TORCH_CHECK(w.dim() == 2 && w.size(1) == C, "conv weight must be [taps, channels]");
  taps = w.size(0);
  check_vec(w, (int64_t)taps * C, "conv weight");
  if (bias.has_value()) check_vec(*bias, C, "conv bias");
  CHECK_CONTIG(state);
  TORCH_CHECK(state.dim() == 3 && state.size(1) == taps - 1 && state.size(2) == C, "conv state must be [slots, taps - 1, channels]");
}

// x: [tokens, >= C] rows (the first C columns are convolved); advances the sequences' state
Tensor causal_conv(const Tensor& x, const Tensor& w, const OptT& bias, Tensor state, const Tensor& slots,
                   const Tensor& cu, const Tensor& ctx, int64_t max_len, bool silu) {
  CHECK_ACT(x);
  const int C = w.size(1), T = x.size(0), B = cu.numel() - 1;
  int taps;
  check_conv(w, bias, state, C, taps);
  check_rows(x, T, C, x, "x");
  TORCH_CHECK(state.scalar_type() == x.scalar_type(), "conv state dtype");
  check_i32(slots, B, "slots"); check_i32(cu, B + 1, "cu"); check_i32(ctx, B, "ctx");
  c10::DeviceGuard g(x.device());
  auto y = at::empty({T, C}, x.options());
  CHECK_RC(docqa_causal_conv(x.data_ptr(), (int)x.stride(0), w.data_ptr<float>(),
                             bias.has_value() ? bias->data_ptr<float>() : nullptr, state.data_ptr(), slots.data_ptr<int>(), cu.data_ptr<int>(), ctx.data_ptr<int>(),
                             y.data_ptr(), is_f32(x), B, (int)max_len, C, taps, silu, stream()),
           "causal_conv");
  return y;
}

// sandwich_rmsnorm of one token a row and its input convolution: (h, h + conv(h)) in the state's dtype
std::tuple<Tensor, Tensor> sandwich_rmsnorm_conv(const Tensor& P, Tensor residual, const Tensor& w_post,
                                                 const Tensor& w_next, const Tensor& cw, Tensor state,
                                                 const Tensor& slots, const Tensor& positions, double eps) {
  const Slabs p = slabs_of(P);
  CHECK_GPU(residual); CHECK_F32(residual); CHECK_CONTIG(residual);
  TORCH_CHECK(residual.dim() == 2 && residual.size(0) == p.M && residual.size(1) == p.N, "residual shape mismatch");
  check_vec(w_post, p.N, "w_post");
  check_vec(w_next, p.N, "w_next");
  int taps;
  check_conv(cw, c10::nullopt, state, p.N, taps);
  CHECK_ACT(state);
  check_i32(slots, p.M, "slots"); check_i32(positions, p.M, "positions");
  CHECK_ALIGN16(P); CHECK_ALIGN16(residual); CHECK_ALIGN16(w_post); CHECK_ALIGN16(w_next); CHECK_ALIGN16(cw); CHECK_ALIGN16(state);
  c10::DeviceGuard g(P.device());
  auto h = at::empty({p.M, p.N}, state.options()), hc = at::empty({p.M, p.N}, state.options());
  CHECK_RC(docqa_sandwich_rmsnorm_conv(P.data_ptr(), is_f32(P), p.S, residual.data_ptr<float>(), w_post.data_ptr<float>(),
                                       w_next.data_ptr<float>(), cw.data_ptr<float>(), taps, state.data_ptr(),
                                       slots.data_ptr<int>(), positions.data_ptr<int>(), h.data_ptr(), hc.data_ptr(),
                                       is_f32(state), p.M, p.N, (float)eps, stream()),
           "sandwich_rmsnorm_conv");
  return {h, hc};
}

// P: [x: C | z: rest | ..] input projection of one token a row -> (conv x, z); rest -1: all of the columns
std::tuple<Tensor, Tensor> conv_step(const Tensor& P, const Tensor& w, const OptT& bias, Tensor state,
                                     const Tensor& slots, const Tensor& positions, bool silu, int64_t rest) {
  const Slabs p = slabs_of(P);
  const int C = w.size(1);
  int taps;
  check_conv(w, bias, state, C, taps);
  CHECK_ACT(state);
  const int64_t nz = rest < 0 ? p.N - C : rest;
  TORCH_CHECK(nz >= 0 && C + nz <= p.N, "conv_step: columns of P");
  TORCH_CHECK(is_f32(P) || !is_f32(state), "conv_step: fp32 state needs fp32 projections");
  check_i32(slots, p.M, "slots"); check_i32(positions, p.M, "positions");
  c10::DeviceGuard g(P.device());
  auto y = at::empty({p.M, C}, state.options()), z = at::empty({nz ? p.M : 0, nz}, state.options());
  CHECK_RC(docqa_conv_step(P.data_ptr(), is_f32(P), p.S, p.slab, p.N, w.data_ptr<float>(),
                           bias.has_value() ? bias->data_ptr<float>() : nullptr,
                           state.data_ptr(), slots.data_ptr<int>(), positions.data_ptr<int>(), y.data_ptr(),
                           nz ? z.data_ptr() : nullptr, is_f32(state), p.M, C, (int)nz, taps, silu, stream()),
           "conv_step");
  return {y, z};
}

int check_scan(const Tensor& x, const OptT& dt, const Tensor& bc, const Tensor& z, const Tensor& A2, const Tensor& D,
               const Tensor& dt_b, const Tensor& state, int64_t N, int64_t b_off, int64_t c_off) {
  CHECK_ACT(x); CHECK_CONTIG(x);
  TORCH_CHECK(x.dim() == 2, "x must be [tokens, channels]");
  const int T = x.size(0), C = x.size(1);
  if (dt.has_value())
    TORCH_CHECK(dt->is_contiguous() && dt->sizes() == x.sizes() && dt->scalar_type() == x.scalar_type(), "dt must match x");
  TORCH_CHECK(A2.dim() == 2 && A2.size(0) == C && A2.size(1) >= N && A2.size(1) % 4 == 0, "A2 must be [channels, N padded to 4]");
  const int Np = A2.size(1);
  check_vec(A2, (int64_t)C * Np, "A2");
  check_vec(D, C, "D"); check_vec(dt_b, C, "dt_b");
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 3 &&
                  state.size(1) == C && state.size(2) == Np, "scan state must be fp32 [slots, channels, Np]");
  TORCH_CHECK(b_off >= 0 && c_off >= 0, "B / C offsets");
  check_rows(bc, T, std::max(b_off, c_off) + N, x, "bc");
  check_rows(z, T, C, x, "z");
  CHECK_ALIGN16(A2); CHECK_ALIGN16(state);
  return Np;
}

Tensor selective_scan(const Tensor& x, const Tensor& dt, const Tensor& bc, int64_t b_off, int64_t c_off, int64_t N,
                      const Tensor& z, const Tensor& A2, const Tensor& D, const Tensor& dt_b, Tensor state,
                      const Tensor& slots, const Tensor& cu, const Tensor& ctx, int64_t max_len, int64_t chunk) {
  const int Np = check_scan(x, dt, bc, z, A2, D, dt_b, state, N, b_off, c_off);
  const int B = cu.numel() - 1, C = x.size(1);
  check_i32(slots, B, "slots"); check_i32(cu, B + 1, "cu"); check_i32(ctx, B, "ctx");
  TORCH_CHECK(chunk >= 1 && max_len >= 0, "chunk");
  const int nchunk = (int)((max_len + chunk - 1) / chunk);
  TORCH_CHECK(nchunk <= 65535 && B <= 65535, "scan grid");
  c10::DeviceGuard g(x.device());
  auto y = at::empty_like(x);
  Tensor cs, sum;
  if (nchunk > 1) {
    cs = at::empty({B, nchunk, C, Np}, state.options());
    sum = at::empty({B, nchunk, C}, state.options());
  }
  CHECK_RC(docqa_selective_scan(x.data_ptr(), dt.data_ptr(), bc.data_ptr(), (int)bc.stride(0), (int)b_off, (int)c_off,
                                z.data_ptr(), (int)z.stride(0), A2.data_ptr<float>(), D.data_ptr<float>(),
                                dt_b.data_ptr<float>(), state.data_ptr<float>(), slots.data_ptr<int>(),
                                cu.data_ptr<int>(), ctx.data_ptr<int>(), y.data_ptr(),
                                nchunk > 1 ? cs.data_ptr<float>() : nullptr, nchunk > 1 ? sum.data_ptr<float>() : nullptr,
                                is_f32(x), B, C, (int)N, Np, (int)chunk, nchunk, stream()),
           "selective_scan");
  return y;
}

// dt: the step projection [B, C], or (dt_in [B, R], w_dt [C, R]) to run it inside the launch
Tensor selective_step(const Tensor& x, const OptT& dt, const OptT& dt_in, const OptT& w_dt, const Tensor& bc,
                      int64_t b_off, int64_t c_off, int64_t N, const Tensor& z, const Tensor& A2, const Tensor& D,
                      const Tensor& dt_b, Tensor state, const Tensor& slots, const Tensor& positions) {
  const int Np = check_scan(x, dt, bc, z, A2, D, dt_b, state, N, b_off, c_off);
  const int B = x.size(0), C = x.size(1);
  check_i32(slots, B, "slots"); check_i32(positions, B, "positions");
  TORCH_CHECK(dt.has_value() != w_dt.has_value() && dt_in.has_value() == w_dt.has_value(), "dt, or dt_in and w_dt");
  int R = 0;
  if (w_dt.has_value()) {
    CHECK_BF16(*w_dt); CHECK_BF16(*dt_in); CHECK_BF16(x); CHECK_CONTIG(*w_dt); CHECK_CONTIG(*dt_in);
    CHECK_GPU(*w_dt); CHECK_GPU(*dt_in);
    R = w_dt->size(1);
    TORCH_CHECK(w_dt->dim() == 2 && w_dt->size(0) == C && dt_in->dim() == 2 && dt_in->size(0) == B && dt_in->size(1) == R,
                "w_dt [C, R], dt_in [B, R]");
  }
  c10::DeviceGuard g(x.device());
  auto y = at::empty_like(x);
  CHECK_RC(docqa_selective_step(x.data_ptr(), dt.has_value() ? dt->data_ptr() : nullptr,
                                w_dt.has_value() ? dt_in->data_ptr() : nullptr, w_dt.has_value() ? w_dt->data_ptr() : nullptr,
                                R, bc.data_ptr(), (int)bc.stride(0), (int)b_off, (int)c_off, z.data_ptr(),
                                (int)z.stride(0), A2.data_ptr<float>(), D.data_ptr<float>(), dt_b.data_ptr<float>(),
                                state.data_ptr<float>(), slots.data_ptr<int>(), positions.data_ptr<int>(), y.data_ptr(),
                                is_f32(x), B, C, (int)N, Np, stream()),
           "selective_step");
  return y;
}

// the recurrence's operands: dims / consts are ops.LinearMix.native()
DocqaLinear linear_args(const Tensor& X, const Tensor& Z, at::IntArrayRef d, at::ArrayRef<double> f, const Tensor& w_gate,
                        const OptT& b_gate, const OptT& cs, const Tensor& norm, const Tensor& state, Tensor& out) {
  const Slabs x = slabs_of(X), z = slabs_of(Z);
  CHECK_ALIGN16(state);
  TORCH_CHECK(d.size() == 13 && f.size() == 4, "linear attention: arguments");
  DocqaLinear a{};
  int* const to[13] = {&a.kind, &a.H, &a.G, &a.dk, &a.dv, &a.qo, &a.ko, &a.vo, &a.go, &a.ao, &a.bo, &a.rank, &a.sig};
  for (int i = 0; i < 13; ++i) {
    TORCH_CHECK(d[i] >= 0 && d[i] < (1 << 24), "linear attention: sizes");
    *to[i] = (int)d[i];
  }
  a.X = X.data_ptr(); a.Z = Z.data_ptr();
  a.xf32 = is_f32(X); a.Sx = x.S; a.ldx = x.N; a.xslab = x.slab;
  a.zf32 = is_f32(Z); a.Sz = z.S; a.ldz = z.N; a.zslab = z.slab;
  a.qs = (float)f[0]; a.ks = (float)f[1]; a.inv_tau = (float)f[2]; a.eps = (float)f[3];
  TORCH_CHECK(a.kind <= LIN_CHANNEL_DELTA && a.H >= 1 && a.G >= 1 && a.H % a.G == 0 && a.dk >= 1 && a.dk <= 256 && a.dv >= 1 && a.dv <= 512,
              "linear attention: heads up to [256, 512]");
  TORCH_CHECK(a.qo + a.G * a.dk <= x.N && a.ko + a.G * a.dk <= x.N && a.vo + a.H * a.dv <= x.N && a.go + a.H * a.dv <= z.N &&
                  x.M == z.M, "linear attention: columns");
  const int64_t n = (int64_t)a.H * a.dk;
  if (a.kind == LIN_CHANNEL) {
    TORCH_CHECK(a.rank >= 1 && a.rank <= 1024 && a.ao + a.rank <= z.N && b_gate.has_value(), "linear attention: decay projection");
    check_vec(w_gate, n * a.rank, "w_gate");
    check_vec(*b_gate, n, "b_gate");
  } else {
    check_vec(w_gate, a.H, "w_gate");
    if (a.kind >= LIN_DELTA) {
      const int64_t na = a.kind == LIN_DELTA ? a.H : n;
      TORCH_CHECK(a.ao + na <= z.N && a.bo + a.H <= z.N && b_gate.has_value(), "linear attention: decay columns");
      check_vec(*b_gate, na, "b_gate");
    }
  }
  if (a.kind == LIN_FIXED) {
    TORCH_CHECK(cs.has_value() && cs->dim() == 2 && cs->size(1) <= a.dk && cs->size(1) % 2 == 0, "linear attention: rotation rows");
    a.r = cs->size(1);
    check_vec(*cs, (int64_t)x.M * a.r, "cs");
    a.cs = cs->data_ptr<float>();
  }
  a.w_gate = w_gate.data_ptr<float>();
  a.b_gate = b_gate.has_value() ? b_gate->data_ptr<float>() : nullptr;
  check_vec(norm, a.dv, "norm");
  a.norm = norm.data_ptr<float>();
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 4 &&
                  state.size(1) == a.H && state.size(2) == a.dk && state.size(3) == (a.dv + 3) / 4 * 4,
              "linear attention: state must be fp32 [slots, H, dk, dv padded to 4]");
  a.state = state.data_ptr<float>();
  CHECK_ACT(out);
  TORCH_CHECK(out.size(1) == (int64_t)a.H * a.dv, "linear attention: output width");
  check_rows(out, x.M, (int64_t)a.H * a.dv, out, "out");
  a.out = out.data_ptr(); a.of32 = is_f32(out); a.ldo = (int)out.stride(0);
  return a;
}

void linear_step(const Tensor& X, const Tensor& Z, at::IntArrayRef dims, at::ArrayRef<double> consts, const Tensor& w_gate,
                 const OptT& b_gate, const OptT& cs, const Tensor& norm, Tensor state, const Tensor& slots,
                 const Tensor& positions, Tensor out) {
  DocqaLinear a = linear_args(X, Z, dims, consts, w_gate, b_gate, cs, norm, state, out);
  const int B = out.size(0);
  check_i32(slots, B, "slots"); check_i32(positions, B, "positions");
  a.slots = slots.data_ptr<int>();
  c10::DeviceGuard g(X.device());
  CHECK_RC(docqa_linear_step(a, positions.data_ptr<int>(), B, stream()), "linear_step");
}

void linear_scan(const Tensor& X, const Tensor& Z, at::IntArrayRef dims, at::ArrayRef<double> consts, const Tensor& w_gate,
                 const OptT& b_gate, const OptT& cs, const Tensor& norm, Tensor state, const Tensor& slots, const Tensor& cu,
                 const Tensor& ctx, int64_t max_len, Tensor out) {
  DocqaLinear a = linear_args(X, Z, dims, consts, w_gate, b_gate, cs, norm, state, out);
  const int T = out.size(0), B = cu.numel() - 1;
  check_i32(slots, B, "slots"); check_i32(cu, B + 1, "cu"); check_i32(ctx, B, "ctx");
  TORCH_CHECK(max_len >= 0 && max_len <= T && B <= 65535, "linear_scan: lengths");
  a.slots = slots.data_ptr<int>();
  c10::DeviceGuard g(X.device());
  auto scratch = at::empty({(int64_t)docqa_linear_scratch(a.kind, T, B, a.H, a.dk, a.dv)}, X.options().dtype(at::kFloat));
  CHECK_RC(docqa_linear_scan(a, cu.data_ptr<int>(), ctx.data_ptr<int>(), scratch.data_ptr<float>(), T, B, (int)max_len,
                             stream()),
           "linear_scan");
}

Tensor low_rank(const Tensor& z, int64_t at_, const Tensor& wa, const Tensor& wg, int64_t n) {
  CHECK_GPU(z); CHECK_BF16(z); CHECK_BF16(wa); CHECK_BF16(wg); CHECK_GPU(wa); CHECK_GPU(wg); CHECK_CONTIG(wa); CHECK_CONTIG(wg);
  CHECK_ALIGN16(wa); CHECK_ALIGN16(wg);
  TORCH_CHECK(wa.dim() == 2 && wg.dim() == 2 && n >= 0 && at_ >= 0, "low_rank: weights [out, in]");
  const int64_t T = z.size(0), Na = wa.size(0), Ka = wa.size(1), Ng = wg.size(0), Kg = wg.size(1);
  check_rows(z, T, at_ + Ka + Kg + n, z, "z");
  c10::DeviceGuard g(z.device());
  auto y = at::empty({T, Na + Ng + n}, z.options().dtype(at::kFloat));
  // (a row of one: its stride may be anything)
  CHECK_RC(docqa_low_rank(z.data_ptr(), T > 1 ? (int)z.stride(0) : (int)z.size(1), (int)at_, wa.data_ptr(), (int)Na, (int)Ka,
                          wg.data_ptr(), (int)Ng, (int)Kg, (int)n, y.data_ptr<float>(), (int)T, stream()),
           "low_rank");
  return y;
}

Tensor post_norm(const OptT& P, const OptT& Q, const OptT& gate, int64_t col, const OptT& gate_b, Tensor residual,
                 double alpha, const Tensor& w, int64_t groups, double eps, bool out_f32) {
  CHECK_GPU(residual); CHECK_F32(residual); CHECK_CONTIG(residual); CHECK_ALIGN16(residual);
  TORCH_CHECK(residual.dim() == 2, "residual must be [rows, width]");
  DocqaPostNorm a{};
  a.rows = residual.size(0); a.W = residual.size(1); a.groups = (int)groups;
  a.SP = a.SQ = a.SG = 1;
  check_vec(w, a.W, "w");
  CHECK_ALIGN16(w);
  if (P.has_value()) {
    const Slabs p = slabs_of(*P);
    TORCH_CHECK(p.M == a.rows && p.N == a.W && gate.has_value() && gate_b.has_value(), "post_norm: P, gate");
    CHECK_ALIGN16(*P);
    const Slabs s = slabs_of(*gate);
    TORCH_CHECK(s.M == a.rows && col >= 0 && col + a.W <= s.N, "post_norm: gate columns");
    CHECK_ALIGN16(*gate);
    check_vec(*gate_b, a.W, "gate_b");
    CHECK_ALIGN16(*gate_b);
    a.P = P->data_ptr(); a.pf32 = is_f32(*P); a.SP = p.S;
    a.gate = gate->data_ptr(); a.gf32 = is_f32(*gate); a.SG = s.S; a.ldg = s.N; a.gslab = s.slab; a.col = (int)col;
    a.gb = gate_b->data_ptr<float>();
  }
  if (Q.has_value()) {
    const Slabs q = slabs_of(*Q);
    TORCH_CHECK(P.has_value() && q.M == a.rows && q.N == a.W, "post_norm: Q");
    CHECK_ALIGN16(*Q);
    a.Q = Q->data_ptr(); a.qf32 = is_f32(*Q); a.SQ = q.S;
  }
  c10::DeviceGuard g(residual.device());
  auto out = at::empty({out_f32 ? 0 : a.rows, a.W}, residual.options().dtype(at::kBFloat16));
  a.res = residual.data_ptr<float>(); a.w = w.data_ptr<float>(); a.out = out_f32 ? nullptr : out.data_ptr();
  a.alpha = (float)alpha; a.eps = (float)eps;
  CHECK_RC(docqa_post_norm(a, stream()), "post_norm");
  return out;
}

std::tuple<Tensor, Tensor, Tensor> moe_route(const Tensor& x, const Tensor& w, int64_t experts, int64_t top) {
  CHECK_ACT(x); CHECK_CONTIG(x); CHECK_CONTIG(w); CHECK_GPU(w); CHECK_ALIGN16(x); CHECK_ALIGN16(w);
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && w.size(1) == x.size(1) && w.scalar_type() == x.scalar_type(), "moe_route: shapes");
  const int64_t T = x.size(0), N = w.size(0);
  TORCH_CHECK(top >= 1 && top <= experts && experts <= N, "moe_route: experts");
  c10::DeviceGuard g(x.device());
  auto f32 = x.options().dtype(at::kFloat);
  auto ids = at::empty({T, top}, x.options().dtype(at::kInt)), wts = at::empty({T, top}, f32), rest = at::empty({T, N - experts}, f32);
  CHECK_RC(docqa_moe_route(x.data_ptr(), w.data_ptr(), is_f32(x), ids.data_ptr<int>(), wts.data_ptr<float>(),
                           rest.data_ptr<float>(), (int)T, (int)x.size(1), (int)N, (int)experts, (int)top, stream()),
           "moe_route");
  return {ids, wts, rest};
}

std::tuple<Tensor, Tensor> moe_route_groups(const Tensor& x, const Tensor& w, const Tensor& corr, int64_t top, int64_t groups,
                                            int64_t keep, double scale) {
  CHECK_ACT(x); CHECK_CONTIG(x); CHECK_CONTIG(w); CHECK_GPU(w); CHECK_ALIGN16(x); CHECK_ALIGN16(w);
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && w.size(1) == x.size(1) && w.scalar_type() == x.scalar_type(), "moe_route_groups: shapes");
  const int64_t T = x.size(0), N = w.size(0);
  check_vec(corr, N, "correction");
  TORCH_CHECK(groups >= 1 && N % groups == 0 && keep >= 1 && keep <= groups && top >= 1 && top <= keep * (N / groups),
              "moe_route_groups: groups");
  c10::DeviceGuard g(x.device());
  auto ids = at::empty({T, top}, x.options().dtype(at::kInt)), wts = at::empty({T, top}, x.options().dtype(at::kFloat));
  CHECK_RC(docqa_moe_route_groups(x.data_ptr(), w.data_ptr(), is_f32(x), corr.data_ptr<float>(), ids.data_ptr<int>(),
                                  wts.data_ptr<float>(), (int)T, (int)x.size(1), (int)N, (int)top, (int)groups, (int)keep,
                                  (float)scale, stream()),
           "moe_route_groups");
  return {ids, wts};
}

Tensor slab_glu(const Tensor& P, int64_t col, int64_t n, const OptT& scale, bool out_f32) {
  const Slabs p = slabs_of(P);
  CHECK_ALIGN16(P);
  TORCH_CHECK(col >= 0 && n >= 1 && col + 2 * n <= p.N, "slab_glu: columns");
  if (scale.has_value()) check_vec(*scale, p.M, "scale");
  c10::DeviceGuard g(P.device());
  auto out = at::empty({p.M, n}, P.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  CHECK_RC(docqa_slab_glu(P.data_ptr(), is_f32(P), p.S, p.slab, p.N, (int)col, (int)n,
                          scale.has_value() ? scale->data_ptr<float>() : nullptr, out.data_ptr(), out_f32, p.M, stream()),
           "slab_glu");
  return out;
}

Tensor moe_experts(const Tensor& x, const Tensor& ids, const Tensor& wts, const Tensor& up, const Tensor& down, double limit) {
  CHECK_ACT(x); CHECK_CONTIG(x); CHECK_CONTIG(up); CHECK_CONTIG(down); CHECK_GPU(up); CHECK_GPU(down);
  CHECK_ALIGN16(x); CHECK_ALIGN16(up); CHECK_ALIGN16(down);
  TORCH_CHECK(x.dim() == 2 && up.dim() == 4 && up.size(1) == 2 && down.dim() == 3 && ids.dim() == 2 && ids.size(0) == x.size(0),
              "moe_experts: shapes");
  const int64_t T = x.size(0), K = x.size(1), E = up.size(0), F = up.size(2), W = down.size(1), top = ids.size(1);
  TORCH_CHECK(up.size(3) == K && down.size(0) == E && down.size(2) == F && up.scalar_type() == x.scalar_type() &&
                  down.scalar_type() == x.scalar_type(), "moe_experts: weights");
  check_i32(ids, T * top, "ids");
  check_vec(wts, T * top, "wts");
  c10::DeviceGuard g(x.device());
  auto act = at::empty({T * top, F}, x.options()), out = at::empty({top, T, W}, x.options());
  const int n = docqa_moe_scratch(is_f32(x), (int)T, (int)top, (int)E, (int)K, (int)F, (int)W);
  auto scratch = at::empty({n}, ids.options());
  CHECK_RC(docqa_moe_experts(x.data_ptr(), ids.data_ptr<int>(), wts.data_ptr<float>(), up.data_ptr(), down.data_ptr(),
                             act.data_ptr(), out.data_ptr(), n ? scratch.data_ptr<int>() : nullptr, is_f32(x), (int)T,
                             (int)top, (int)E, (int)K, (int)F, (int)W, (float)limit, stream()),
           "moe_experts");
  return out;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(docqa, m) {
  m.def("sandwich_rmsnorm(Tensor P, Tensor(a!) residual, Tensor w_post, Tensor? add, Tensor w_next, float eps, "
        "bool out_f32) -> Tensor");
  m.def("embed_scale_rmsnorm(Tensor ids, Tensor table, float scale, Tensor? w, float eps, bool keep) "
        "-> (Tensor, Tensor, Tensor)");
  m.def("decode_act(Tensor x, Tensor w, int act) -> Tensor");
  m.def("add_scaled(Tensor P, Tensor? Q, Tensor(a!) residual, float m, bool out_f32) -> Tensor");
  m.def("scaled_rmsnorm(Tensor P, Tensor(a!) residual, Tensor scale, Tensor? bias, Tensor? ids, Tensor? wts, int experts, "
        "Tensor? x, Tensor w, float eps, bool out_f32) -> Tensor");
  m.def("poly_norm(Tensor P, Tensor bias, Tensor act, int n_out, float eps, bool out_f32) -> Tensor");
  m.def("head_gate(Tensor x, Tensor P, int col, int per, int row0) -> Tensor");
  m.def("latent_norm_store(Tensor P, Tensor cs, Tensor slots, Tensor(a!) cache, Tensor q_norm, Tensor c_norm, float eps) -> Tensor");
  m.def("low_rank(Tensor z, int at, Tensor wa, Tensor wg, int n) -> Tensor");
  m.def("moe_route_groups(Tensor x, Tensor w, Tensor corr, int top, int groups, int keep, float scale) -> (Tensor, Tensor)");
  m.def("soft_cap(Tensor x, float cap) -> Tensor");
  m.def("side_gate(Tensor P, Tensor ids, Tensor table, int col, int n, bool out_f32) -> Tensor");
  m.def("side_project(Tensor P, Tensor ids, Tensor table, int col, int n, Tensor w) -> Tensor");
  m.def("latent_attn(Tensor q, Tensor cache, Tensor block_tables, Tensor? cu, Tensor ctx, int max_q, float scale, "
        "int window, Tensor? sink, Tensor w, Tensor? gp, int gcol, int gper, int grow) -> Tensor");
  m.def("sandwich_rmsnorm_conv(Tensor P, Tensor(a!) residual, Tensor w_post, Tensor w_next, Tensor cw, "
        "Tensor(b!) state, Tensor slots, Tensor positions, float eps) -> (Tensor, Tensor)");
  m.def("packed_window_attn(Tensor q, Tensor kv, Tensor kr, int H, int dim, int vdim, Tensor cu, Tensor cu_k, int max_q, "
        "float scale, int window, Tensor? sink, Tensor? gp, int gcol, int gper, int grow) -> Tensor");
  m.def("rope_table(Tensor positions, Tensor freq, float mult) -> Tensor");
  m.def("latent_store(Tensor P, Tensor cs, Tensor slots, Tensor(a!) cache, Tensor? c_norm, int H, int dim, int rank, "
        "float eps) -> Tensor");
  m.def("head_project(Tensor x, Tensor w, int carry) -> Tensor");
  m.def("latent_gather(Tensor cache, Tensor block_tables, Tensor first, Tensor cu_k, int total, int rank) "
        "-> (Tensor, Tensor)");
  m.def("slab_columns(Tensor P, int n0, int n1, bool out_f32) -> (Tensor, Tensor)");
  m.def("slab_activation(Tensor P, int act, bool out_f32) -> Tensor");
  m.def("qk_norm_store(Tensor P, Tensor w, Tensor slots, Tensor(a!) k_cache, Tensor(b!) k_scale, int H, float eps) "
        "-> Tensor");
  m.def("window_attn(Tensor q, Tensor k_cache, Tensor? v_cache, Tensor? k_scale, Tensor block_tables, Tensor? cu, "
        "Tensor ctx, int max_q, float scale, int window, Tensor? sink, int v_dim, float cap, float out_scale, Tensor(a!) out) -> ()");
  m.def("qkv_rope_store(Tensor P, Tensor? bias, Tensor? qw, Tensor? kw, Tensor cs, Tensor slots, Tensor(a!) k_cache, "
        "Tensor(b!) v_cache, int H, float eps) -> Tensor");
  m.def("linear_step(Tensor X, Tensor Z, int[] dims, float[] consts, Tensor w_gate, Tensor? b_gate, Tensor? cs, Tensor norm, "
        "Tensor(a!) state, Tensor slots, Tensor positions, Tensor(b!) out) -> ()");
  m.def("linear_scan(Tensor X, Tensor Z, int[] dims, float[] consts, Tensor w_gate, Tensor? b_gate, Tensor? cs, Tensor norm, "
        "Tensor(a!) state, Tensor slots, Tensor cu, Tensor ctx, int max_len, Tensor(b!) out) -> ()");
  m.def("post_norm(Tensor? P, Tensor? Q, Tensor? gate, int col, Tensor? gate_b, Tensor(a!) residual, float alpha, Tensor w, "
        "int groups, float eps, bool out_f32) -> Tensor");
  m.def("moe_route(Tensor x, Tensor w, int experts, int top) -> (Tensor, Tensor, Tensor)");
  m.def("slab_glu(Tensor P, int col, int n, Tensor? scale, bool out_f32) -> Tensor");
  m.def("moe_experts(Tensor x, Tensor ids, Tensor wts, Tensor up, Tensor down, float limit) -> Tensor");
  m.def("causal_conv(Tensor x, Tensor w, Tensor? bias, Tensor(a!) state, Tensor slots, Tensor cu, Tensor ctx, "
        "int max_len, bool silu) -> Tensor");
  m.def("conv_step(Tensor P, Tensor w, Tensor? bias, Tensor(a!) state, Tensor slots, Tensor positions, bool silu, "
        "int rest) -> (Tensor, Tensor)");
  m.def("selective_scan(Tensor x, Tensor dt, Tensor bc, int b_off, int c_off, int N, Tensor z, Tensor A2, Tensor D, "
        "Tensor dt_b, Tensor(a!) state, Tensor slots, Tensor cu, Tensor ctx, int max_len, int chunk) -> Tensor");
  m.def("selective_step(Tensor x, Tensor? dt, Tensor? dt_in, Tensor? w_dt, Tensor bc, int b_off, int c_off, int N, Tensor z, Tensor A2, Tensor D, "
        "Tensor dt_b, Tensor(a!) state, Tensor slots, Tensor positions) -> Tensor");
}

TORCH_LIBRARY_IMPL(docqa, CUDA, m) {
  m.impl("sandwich_rmsnorm", &sandwich_rmsnorm);
  m.impl("embed_scale_rmsnorm", &embed_scale_rmsnorm);
  m.impl("decode_act", &decode_act);
  m.impl("add_scaled", &add_scaled);
  m.impl("scaled_rmsnorm", &scaled_rmsnorm);
  m.impl("poly_norm", &poly_norm);
  m.impl("head_gate", &head_gate);
  m.impl("latent_norm_store", &latent_norm_store);
  m.impl("low_rank", &low_rank);
  m.impl("moe_route_groups", &moe_route_groups);
  m.impl("soft_cap", &soft_cap);
  m.impl("side_gate", &side_gate);
  m.impl("side_project", &side_project);
  m.impl("latent_attn", &latent_attn);
  m.impl("sandwich_rmsnorm_conv", &sandwich_rmsnorm_conv);
  m.impl("packed_window_attn", &packed_window_attn);
  m.impl("rope_table", &rope_table);
  m.impl("latent_store", &latent_store);
  m.impl("head_project", &head_project);
  m.impl("latent_gather", &latent_gather);
  m.impl("slab_columns", &slab_columns);
  m.impl("slab_activation", &slab_activation);
  m.impl("qk_norm_store", &qk_norm_store);
  m.impl("window_attn", &window_attn);
  m.impl("qkv_rope_store", &qkv_rope_store);
  m.impl("linear_step", &linear_step);
  m.impl("linear_scan", &linear_scan);
  m.impl("post_norm", &post_norm);
  m.impl("moe_route", &moe_route);
  m.impl("slab_glu", &slab_glu);
  m.impl("moe_experts", &moe_experts);
  m.impl("causal_conv", &causal_conv);
  m.impl("conv_step", &conv_step);
  m.impl("selective_scan", &selective_scan);
  m.impl("selective_step", &selective_step);
}
