// Python bindings for gated linear attention (scan and chunk form) and for
// the routed experts (selection, pair sort, grouped products, combine).
// Host-side glue and shape checks only; registered into the main module by
// register_gla_ops().

#include <torch/extension.h>

#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

extern "C" {
int tl_gla_chunks_ok(int D, int R, int C);
int tl_gla_chunks(const void* proj, int ld, int q_off, int k_off, int v_off,
                  int r_off, const void* a2t, const void* bias, int R,
                  float inv_tau, float qscale, void* S, const void* cu_c,
                  int NC, const void* base, const void* cnt, const void* slots,
                  const void* pos0, int B, void* U, void* dec, void* out,
                  int H, int D, int V, int C, int is_f32, hipStream_t stream);
int tl_gla_scan(const void* proj, int ld, int q_off, int k_off, int v_off,
                int r_off, const void* a2t, const void* bias, int R,
                float inv_tau, float qscale, void* S, const void* cu,
                const void* slots, const void* pos0, void* out, int B, int H,
                int D, int V, int is_f32, hipStream_t stream);
int tl_moe_max_experts();
int tl_moe_max_top();
void tl_moe_route(const void* h, const void* w, const void* z, void* wt,
                  void* idx, int64_t T, int W, int E, int top, int is_f32,
                  hipStream_t stream);
void tl_moe_route_scores(const void* z, int64_t ldz, const void* corr,
                         void* wt, void* idx, int64_t T, int E, int top,
                         hipStream_t stream);
int tl_moe_sort_blocks(int P);
void tl_moe_sort(const void* idx, int P, int E, int top, void* seg,
                 void* pair_tok, void* rank, void* hist, hipStream_t stream);
void tl_grouped_any(const void* x, const void* tok_idx, const void* seg,
                    const void* w, void* out, int P, int E, int N, int K,
                    int is_f32, hipStream_t stream);
void tl_moe_gemm_stacked(const void* x, const void* tok_idx,
                         const void* seg_off, const void* w, void* out, int E,
                         int N, int K, hipStream_t stream);
void tl_moe_tiles(const void* x, const void* tok, const void* seg,
                  const void* w, void* out, int P, int E, int N, int K,
                  hipStream_t stream);
void tl_moe_rows(const void* x, const void* tok, const void* seg,
                 const void* w, void* out, int P, int E, int N, int K,
                 hipStream_t stream);
void tl_act_gate(const void* p, int64_t ld, int aligned, void* out,
                 int64_t rows, int N, int act, float lim, float alpha,
                 int is_f32, hipStream_t stream);
void tl_moe_combine(const void* y, const void* rank, const void* wt,
                    const void* shared, const void* sg, int ldg, int sg_col,
                    const void* ident, const void* n_real, void* out,
                    int64_t T, int W, int top, int is_f32,
                    hipStream_t stream);
}

namespace {

using torch::Tensor;

hipStream_t gla_stream() { return c10::hip::getCurrentHIPStream().stream(); }

#define GLA_IN(t)                                    \
  TORCH_CHECK((t).is_cuda(), #t " must be on GPU");  \
  TORCH_CHECK((t).is_contiguous(), #t " must be contiguous")
#define GLA_F32(t) \
  GLA_IN(t);       \
  TORCH_CHECK((t).scalar_type() == torch::kFloat, #t " must be fp32")
#define GLA_I32(t) \
  GLA_IN(t);       \
  TORCH_CHECK((t).scalar_type() == torch::kInt, #t " must be int32")

int gla_is_f32(const Tensor& t) {
  TORCH_CHECK(t.scalar_type() == torch::kFloat ||
                  t.scalar_type() == torch::kBFloat16,
              "activations must be fp32 or bf16");
  return t.scalar_type() == torch::kFloat ? 1 : 0;
}

void check_gla(const Tensor& proj, int64_t q_off, int64_t k_off,
               int64_t v_off, int64_t r_off, const Tensor& a2t,
               const Tensor& bias, double tau, const Tensor& S,
               const Tensor& slots, const Tensor& pos0, int64_t H, int64_t D,
               int64_t V) {
  GLA_IN(proj);
  GLA_F32(a2t);
  GLA_F32(bias);
  GLA_F32(S);
  GLA_I32(slots);
  GLA_I32(pos0);
  TORCH_CHECK(proj.dim() == 2 && a2t.dim() == 2, "proj [T, L], a2t [R, H*D]");
  const int64_t ld = proj.size(1);
  TORCH_CHECK(H >= 1 && D >= 1 && V >= 1 && tau > 0, "sizes");
  TORCH_CHECK(q_off >= 0 && k_off >= 0 && v_off >= 0 && r_off >= 0 &&
                  q_off + H * D <= ld && k_off + H * D <= ld &&
                  v_off + H * V <= ld && r_off + a2t.size(0) <= ld,
              "projection columns out of range");
  TORCH_CHECK(a2t.size(0) >= 1 && a2t.size(1) == H * D &&
                  bias.numel() == H * D,
              "decay weights must be [R, H*D] and [H*D]");
  TORCH_CHECK(S.dim() == 4 && S.size(1) == H && S.size(2) == D &&
                  S.size(3) == V,
              "S pool must be [slots, H, D, V]");
  TORCH_CHECK(slots.numel() == pos0.numel(), "ragged metadata");
}

Tensor gla_scan(Tensor proj, int64_t q_off, int64_t k_off, int64_t v_off,
                int64_t r_off, Tensor a2t, Tensor bias, double tau, Tensor S,
                Tensor cu, Tensor slots, Tensor pos0, int64_t H, int64_t D,
                int64_t V) {
  check_gla(proj, q_off, k_off, v_off, r_off, a2t, bias, tau, S, slots, pos0,
            H, D, V);
  GLA_I32(cu);
  const int B = (int)slots.numel();
  TORCH_CHECK(cu.numel() == B + 1, "ragged metadata");
  auto out = torch::empty({proj.size(0), H * V},
                          proj.options().dtype(torch::kFloat));
  if (proj.size(0) == 0 || B == 0) return out;
  const int rc = tl_gla_scan(
      proj.data_ptr(), (int)proj.size(1), (int)q_off, (int)k_off, (int)v_off,
      (int)r_off, a2t.data_ptr(), bias.data_ptr(), (int)a2t.size(0),
      (float)(1.0 / tau), (float)(1.0 / std::sqrt((double)D)), S.data_ptr(),
      cu.data_ptr(), slots.data_ptr(), pos0.data_ptr(), out.data_ptr(), B,
      (int)H, (int)D, (int)V, gla_is_f32(proj), gla_stream());
  TORCH_CHECK(rc == 0, "gla_scan: head sizes outside the kernel's range");
  return out;
}

bool gla_chunks_ok(int64_t D, int64_t R, int64_t C) {
  return tl_gla_chunks_ok((int)D, (int)R, (int)C) != 0;
}

// cu_c [NC + 1] token offsets of the chunks (<= C tokens each); base / cnt
// [B] first chunk and chunk count per sequence
Tensor gla_chunks(Tensor proj, int64_t q_off, int64_t k_off, int64_t v_off,
                  int64_t r_off, Tensor a2t, Tensor bias, double tau,
                  Tensor S, Tensor cu_c, Tensor base, Tensor cnt,
                  Tensor slots, Tensor pos0, int64_t H, int64_t D, int64_t V,
                  int64_t C) {
  check_gla(proj, q_off, k_off, v_off, r_off, a2t, bias, tau, S, slots, pos0,
            H, D, V);
  GLA_I32(cu_c);
  GLA_I32(base);
  GLA_I32(cnt);
  const int B = (int)slots.numel();
  const int64_t NC = cu_c.numel() - 1;
  TORCH_CHECK(NC >= 0 && base.numel() == B && cnt.numel() == B,
              "per-sequence chunk metadata");
  TORCH_CHECK(tl_gla_chunks_ok((int)D, (int)a2t.size(0), (int)C),
              "gla_chunks: shape outside the kernels' range");
  auto o = proj.options().dtype(torch::kFloat);
  auto out = torch::empty({proj.size(0), H * V}, o);
  if (proj.size(0) == 0 || B == 0 || NC == 0) return out;
  auto U = torch::empty({NC, H, D, V}, o);
  auto dec = torch::empty({NC, H, D}, o);
  const int rc = tl_gla_chunks(
      proj.data_ptr(), (int)proj.size(1), (int)q_off, (int)k_off, (int)v_off,
      (int)r_off, a2t.data_ptr(), bias.data_ptr(), (int)a2t.size(0),
      (float)(1.0 / tau), (float)(1.0 / std::sqrt((double)D)), S.data_ptr(),
      cu_c.data_ptr(), (int)NC, base.data_ptr(), cnt.data_ptr(),
      slots.data_ptr(), pos0.data_ptr(), B, U.data_ptr(), dec.data_ptr(),
      out.data_ptr(), (int)H, (int)D, (int)V, (int)C, gla_is_f32(proj),
      gla_stream());
  TORCH_CHECK(rc == 0, "gla_chunks: launch refused");
  return out;
}

// fp32 logits h w^T (given, or computed here for few rows); the `top`
// largest and the softmax over them: (weights [T, top], indices [T, top])
std::vector<Tensor> moe_route(Tensor h, Tensor w, c10::optional<Tensor> z,
                              int64_t top) {
  GLA_IN(h);
  GLA_F32(w);
  TORCH_CHECK(h.dim() == 2 && w.dim() == 2 && w.size(1) == h.size(1),
              "h [T, W], w [E, W]");
  const int64_t T = h.size(0), E = w.size(0);
  TORCH_CHECK(top >= 1 && top <= E && top <= tl_moe_max_top() &&
                  E <= tl_moe_max_experts(),
              "router sizes outside the kernel's range");
  if (z.has_value()) {
    GLA_F32(z.value());
    TORCH_CHECK(z->dim() == 2 && z->size(0) == T && z->size(1) == E,
                "logits must be [T, E]");
  }
  auto wt = torch::empty({T, top}, w.options());
  auto idx = torch::empty({T, top}, w.options().dtype(torch::kInt));
  tl_moe_route(h.data_ptr(), w.data_ptr(),
               z.has_value() ? z->data_ptr() : nullptr, wt.data_ptr(),
               idx.data_ptr(), T, (int)h.size(1), (int)E, (int)top,
               gla_is_f32(h), gla_stream());
  return {wt, idx};
}

// fp32 logits z[:, col:col + E]: scores = softmax over all E, the `top`
// largest of score + corr chosen, weighted by their scores
std::vector<Tensor> moe_route_scores(Tensor z, int64_t col, int64_t E,
                                     c10::optional<Tensor> corr,
                                     int64_t top) {
  GLA_F32(z);
  TORCH_CHECK(z.dim() == 2 && col >= 0 && E >= 1 && col + E <= z.size(1),
              "logit columns out of range");
  TORCH_CHECK(top >= 1 && top <= E && top <= tl_moe_max_top() &&
                  E <= tl_moe_max_experts(),
              "router sizes outside the kernel's range");
  if (corr.has_value()) {
    GLA_F32(corr.value());
    TORCH_CHECK(corr->numel() == E, "one correction per expert");
  }
  const int64_t T = z.size(0);
  auto wt = torch::empty({T, top}, z.options());
  auto idx = torch::empty({T, top}, z.options().dtype(torch::kInt));
  tl_moe_route_scores((const float*)z.data_ptr() + col, z.size(1),
                      corr.has_value() ? corr->data_ptr() : nullptr,
                      wt.data_ptr(), idx.data_ptr(), T, (int)E, (int)top,
                      gla_stream());
  return {wt, idx};
}

// idx [T, top] int32 in [0, E): (segments [E + 1], token of every sorted
// pair [P], sorted position of every pair [T, top])
std::vector<Tensor> moe_sort(Tensor idx, int64_t E) {
  GLA_I32(idx);
  TORCH_CHECK(idx.dim() == 2 && E >= 1 && E <= tl_moe_max_experts(),
              "idx must be [T, top]");
  const int64_t P = idx.numel();
  TORCH_CHECK(P < (1LL << 30), "too many pairs");
  auto seg = torch::empty({E + 1}, idx.options());
  auto tok = torch::empty({P}, idx.options());
  auto rank = torch::empty(idx.sizes(), idx.options());
  const int nb = tl_moe_sort_blocks((int)P);
  auto hist = torch::empty({nb, E}, idx.options());
  tl_moe_sort(idx.data_ptr(), (int)P, (int)E, (int)idx.size(1),
              seg.data_ptr(), tok.data_ptr(), rank.data_ptr(),
              hist.data_ptr(), gla_stream());
  return {seg, tok, rank};
}

// out[p] = x[tok ? tok[p] : p] w[e]^T for the pairs p of expert e
Tensor moe_gemm_stacked(Tensor x, c10::optional<Tensor> tok, Tensor seg,
                        Tensor w) {
  GLA_IN(x);
  GLA_IN(w);
  GLA_I32(seg);
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && w.size(2) == x.size(1) &&
                  w.scalar_type() == x.scalar_type() &&
                  seg.numel() == w.size(0) + 1,
              "x [*, K], w [E, N, K], seg [E + 1]");
  const int is_f32 = gla_is_f32(x);
  int64_t P = x.size(0);
  const void* ti = nullptr;
  if (tok.has_value()) {
    GLA_I32(tok.value());
    P = tok->numel();
    ti = tok->data_ptr();
  }
  const int64_t E = w.size(0), N = w.size(1), K = w.size(2);
  auto out = torch::empty({P, N}, x.options());
  if (P == 0) return out;
  const bool mfma = !is_f32 && K % 32 == 0 && N % 64 == 0;
  if (mfma && P <= 128)
    tl_moe_rows(x.data_ptr(), ti, seg.data_ptr(), w.data_ptr(),
                out.data_ptr(), (int)P, (int)E, (int)N, (int)K, gla_stream());
  else if (mfma && P >= 64 * E && P >= 1024)
    tl_moe_tiles(x.data_ptr(), ti, seg.data_ptr(), w.data_ptr(),
                 out.data_ptr(), (int)P, (int)E, (int)N, (int)K,
                 gla_stream());
  else if (mfma)
    tl_moe_gemm_stacked(x.data_ptr(), ti, seg.data_ptr(), w.data_ptr(),
                        out.data_ptr(), (int)E, (int)N, (int)K, gla_stream());
  else
    tl_grouped_any(x.data_ptr(), ti, seg.data_ptr(), w.data_ptr(),
                   out.data_ptr(), (int)P, (int)E, (int)N, (int)K, is_f32,
                   gla_stream());
  return out;
}

// sum_j wt[t][j] y[rank[t][j]] (+ sigmoid(sg[t][sg_col]) * shared[t]); with
// `ident` pairs at sorted positions >= n_real[0] stand for the token's row of
// it
Tensor moe_combine(Tensor y, Tensor rank, Tensor wt,
                   c10::optional<Tensor> shared, c10::optional<Tensor> sg,
                   int64_t sg_col, c10::optional<Tensor> ident,
                   c10::optional<Tensor> n_real) {
  GLA_IN(y);
  GLA_I32(rank);
  GLA_F32(wt);
  TORCH_CHECK(y.dim() == 2 && rank.dim() == 2 && wt.sizes() == rank.sizes() &&
                  y.size(0) == rank.numel(),
              "y [T * top, W], rank and weights [T, top]");
  const int64_t T = rank.size(0), W = y.size(1);
  int ldg = 0;
  if (shared.has_value()) {
    GLA_IN(shared.value());
    TORCH_CHECK(shared->dim() == 2 && shared->size(0) == T &&
                    shared->size(1) == W &&
                    shared->scalar_type() == y.scalar_type(),
                "the shared expert's output must be [T, W]");
    if (sg.has_value()) {
      GLA_IN(sg.value());
      TORCH_CHECK(sg->dim() == 2 && sg->size(0) == T && sg_col >= 0 &&
                      sg_col < sg->size(1) &&
                      sg->scalar_type() == y.scalar_type(),
                  "gate column out of range");
      ldg = (int)sg->size(1);
    }
  }
  if (ident.has_value()) {
    GLA_IN(ident.value());
    TORCH_CHECK(n_real.has_value() && ident->dim() == 2 &&
                    ident->size(0) == T && ident->size(1) == W &&
                    ident->scalar_type() == y.scalar_type(),
                "identity rows must be [T, W]");
    GLA_I32(n_real.value());
  }
  auto out = torch::empty({T, W}, y.options());
  tl_moe_combine(y.data_ptr(), rank.data_ptr(), wt.data_ptr(),
                 shared.has_value() ? shared->data_ptr() : nullptr,
                 shared.has_value() && sg.has_value() ? sg->data_ptr()
                                                      : nullptr,
                 ldg, (int)sg_col,
                 ident.has_value() ? ident->data_ptr() : nullptr,
                 ident.has_value() ? n_real->data_ptr() : nullptr,
                 out.data_ptr(), T, (int)W, (int)rank.size(1), gla_is_f32(y), gla_stream());
  return out;
}

// the routed experts of a step in one call: sort, gate|up product,
// activation, down product, combine (gate_up [E, 2 ff, W], down [E, W, ff]).
// Indices E .. E + identity - 1 are identity experts: their pairs sort behind
// the others, no product reads them, and the combine adds the token's h.
Tensor moe_experts(Tensor h, Tensor wt, Tensor idx, Tensor gate_up,
                   Tensor down, int64_t act, double lim, double alpha,
                   int64_t identity, c10::optional<Tensor> shared,
                   c10::optional<Tensor> sg, int64_t sg_col) {
  TORCH_CHECK(gate_up.dim() == 3 && down.dim() == 3 && h.dim() == 2 &&
                  gate_up.size(1) == 2 * down.size(2) &&
                  gate_up.size(0) == down.size(0) &&
                  down.size(1) == h.size(1) && idx.dim() == 2 &&
                  idx.size(0) == h.size(0) && act >= 0 && act <= 4 &&
                  identity >= 0,
              "h [T, W], idx [T, top], gate_up [E, 2 ff, W], down [E, W, ff]");
  const int64_t E = gate_up.size(0);
  auto s = moe_sort(idx, E + identity);
  Tensor seg = s[0].narrow(0, 0, E + 1);
  Tensor a = moe_gemm_stacked(h, s[1], seg, gate_up);
  const int64_t ff = down.size(2);
  auto b = torch::empty({a.size(0), ff}, a.options());
  tl_act_gate(a.data_ptr(), 2 * ff, ff % 8 == 0, b.data_ptr(), a.size(0),
              (int)ff, (int)act, (float)lim, (float)alpha, gla_is_f32(a),
              gla_stream());
  Tensor y = moe_gemm_stacked(b, c10::nullopt, seg, down);
  c10::optional<Tensor> ident, n_real;
  if (identity > 0) {
    ident = h;
    n_real = s[0].narrow(0, E, 1);
  }
  return moe_combine(y, s[2], wt, shared, sg, sg_col, ident, n_real);
}

}  // namespace

void register_gla_ops(pybind11::module& mod) {
  mod.def("gla_scan", &gla_scan,
          "gated linear attention over ragged sequences (slot state)");
  mod.def("gla_chunks_ok", &gla_chunks_ok,
          "whether the chunk kernels serve a shape");
  mod.def("gla_chunks", &gla_chunks,
          "gated linear attention, chunk form on fp32 MFMA");
  mod.def("moe_route", &moe_route,
          "top-k router with the softmax over the chosen logits");
  mod.def("moe_route_scores", &moe_route_scores,
          "top-k router on corrected softmax scores, logits given");
  mod.def("moe_sort", &moe_sort, "expert-sorted (token, choice) pairs");
  mod.def("moe_gemm_stacked", &moe_gemm_stacked,
          "grouped product with stacked experts, any size, bf16 or fp32");
  mod.def("moe_experts", &moe_experts,
          "sort, grouped products, activation and combine in one call");
  mod.def("moe_combine", &moe_combine,
          "weighted sum of a token's experts plus a gated shared expert");
}
