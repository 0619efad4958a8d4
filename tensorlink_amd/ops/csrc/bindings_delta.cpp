// Python bindings for the gated delta rule (scan and chunk form), the bigram
// embedding and the thin fp32 projections. Host-side glue and shape checks
// only; registered into the main module by register_delta_ops().

#include <torch/extension.h>

#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

extern "C" {
int tl_delta_chunk_tokens();
int tl_delta_chunks_ok(int D, int R);
int tl_delta_row_pad(int D);
int tl_delta_col_pad(int V);
int tl_delta_chunks(const void* x, int ldx, int q_off, int k_off, int v_off,
                    const void* proj, int ldr, int r_off, int R,
                    const void* b, int ldb, int b_off, const void* a2t,
                    const void* dt_bias, const void* A_log, float qscale,
                    void* S, const void* cu_c, int NC, const void* base,
                    const void* cnt, const void* slots, const void* pos0,
                    int B, void* W, void* Q, void* Kt, void* Bm, void* U,
                    void* dec, void* out, int H, int G, int D, int V,
                    int is_f32, hipStream_t stream);
int tl_delta_scan(const void* x, int ldx, int q_off, int k_off, int v_off,
                  const void* proj, int ldr, int r_off, int R, const void* b,
                  int ldb, int b_off, const void* a2t, const void* dt_bias,
                  const void* A_log, float qscale, void* S, const void* cu,
                  const void* slots, const void* pos0, void* out, int B,
                  int H, int G, int D, int V, int is_f32, hipStream_t stream);
void tl_bigram_embed(const void* tokens, const void* embed, const void* table,
                     void* prev, const void* tok_seq, const void* cu,
                     const void* slots, const void* pos0, void* X, int64_t T,
                     int W, int64_t vocab, int64_t n, int64_t mul_prev,
                     int64_t mul_cur, int is_f32, hipStream_t stream);
void tl_thin_linear(const void* h, const void* w, const void* bias, void* out,
                    int64_t T, int W, int N, int is_f32, hipStream_t stream);
}

namespace {

using torch::Tensor;

hipStream_t delta_stream() {
  return c10::hip::getCurrentHIPStream().stream();
}

#define DL_IN(t)                                     \
  TORCH_CHECK((t).is_cuda(), #t " must be on GPU");  \
  TORCH_CHECK((t).is_contiguous(), #t " must be contiguous")
#define DL_F32(t) \
  DL_IN(t);       \
  TORCH_CHECK((t).scalar_type() == torch::kFloat, #t " must be fp32")
#define DL_I32(t) \
  DL_IN(t);       \
  TORCH_CHECK((t).scalar_type() == torch::kInt, #t " must be int32")

int delta_is_f32(const Tensor& t) {
  TORCH_CHECK(t.scalar_type() == torch::kFloat ||
                  t.scalar_type() == torch::kBFloat16,
              "activations must be fp32 or bf16");
  return t.scalar_type() == torch::kFloat ? 1 : 0;
}

// x [T, *] fp32 with q [G*D] | k [G*D] | v [H*V]; proj [T, *] with the
// low-rank columns; b [T, *] fp32 raw step sizes
void check_delta(const Tensor& x, int64_t q_off, int64_t k_off, int64_t v_off,
                 const Tensor& proj, int64_t r_off, const Tensor& b,
                 int64_t b_off, const Tensor& a2t, const Tensor& dt_bias,
                 const Tensor& A_log, const Tensor& S, const Tensor& slots,
                 const Tensor& pos0, int64_t H, int64_t G, int64_t D,
                 int64_t V) {
  DL_F32(x);
  DL_IN(proj);
  DL_F32(b);
  DL_F32(a2t);
  DL_F32(dt_bias);
  DL_F32(A_log);
  DL_F32(S);
  DL_I32(slots);
  DL_I32(pos0);
  TORCH_CHECK(x.dim() == 2 && proj.dim() == 2 && b.dim() == 2 &&
                  a2t.dim() == 2 && proj.size(0) == x.size(0) &&
                  b.size(0) == x.size(0),
              "x, proj, b [T, *], a2t [R, H*D]");
  TORCH_CHECK(H >= 1 && G >= 1 && H % G == 0 && D >= 1 && V >= 1, "sizes");
  TORCH_CHECK(q_off >= 0 && k_off >= 0 && v_off >= 0 &&
                  q_off + G * D <= x.size(1) && k_off + G * D <= x.size(1) &&
                  v_off + H * V <= x.size(1) && r_off >= 0 &&
                  r_off + a2t.size(0) <= proj.size(1) && b_off >= 0 &&
                  b_off + H <= b.size(1),
              "columns out of range");
  TORCH_CHECK(a2t.size(0) >= 1 && a2t.size(1) == H * D &&
                  dt_bias.numel() == H * D && A_log.numel() == H,
              "decay weights must be [R, H*D], [H*D] and [H]");
  TORCH_CHECK(S.dim() == 4 && S.size(1) == H && S.size(2) == D &&
                  S.size(3) == V,
              "S pool must be [slots, H, D, V]");
  TORCH_CHECK(slots.numel() == pos0.numel(), "ragged metadata");
}

Tensor delta_scan(Tensor x, int64_t q_off, int64_t k_off, int64_t v_off,
                  Tensor proj, int64_t r_off, Tensor b, int64_t b_off,
                  Tensor a2t, Tensor dt_bias, Tensor A_log, Tensor S,
                  Tensor cu, Tensor slots, Tensor pos0, int64_t H, int64_t G,
                  int64_t D, int64_t V) {
  check_delta(x, q_off, k_off, v_off, proj, r_off, b, b_off, a2t, dt_bias,
              A_log, S, slots, pos0, H, G, D, V);
  DL_I32(cu);
  const int B = (int)slots.numel();
  TORCH_CHECK(cu.numel() == B + 1, "ragged metadata");
  auto out = torch::empty({x.size(0), H * V}, x.options());
  if (x.size(0) == 0 || B == 0) return out;
  const int rc = tl_delta_scan(
      x.data_ptr(), (int)x.size(1), (int)q_off, (int)k_off, (int)v_off,
      proj.data_ptr(), (int)proj.size(1), (int)r_off, (int)a2t.size(0),
      b.data_ptr(), (int)b.size(1), (int)b_off, a2t.data_ptr(),
      dt_bias.data_ptr(), A_log.data_ptr(),
      (float)(1.0 / std::sqrt((double)D)), S.data_ptr(), cu.data_ptr(),
      slots.data_ptr(), pos0.data_ptr(), out.data_ptr(), B, (int)H, (int)G,
      (int)D, (int)V, delta_is_f32(proj), delta_stream());
  TORCH_CHECK(rc == 0, "delta_scan: head sizes outside the kernel's range");
  return out;
}

int64_t delta_chunk_tokens() { return tl_delta_chunk_tokens(); }

bool delta_chunks_ok(int64_t D, int64_t R) {
  return tl_delta_chunks_ok((int)D, (int)R) != 0;
}

// cu_c [NC + 1] token offsets of the chunks; base / cnt
// [B] first chunk and chunk count per sequence
Tensor delta_chunks(Tensor x, int64_t q_off, int64_t k_off, int64_t v_off,
                    Tensor proj, int64_t r_off, Tensor b, int64_t b_off,
                    Tensor a2t, Tensor dt_bias, Tensor A_log, Tensor S,
                    Tensor cu_c, Tensor base, Tensor cnt, Tensor slots,
                    Tensor pos0, int64_t H, int64_t G, int64_t D,
                    int64_t V) {
  check_delta(x, q_off, k_off, v_off, proj, r_off, b, b_off, a2t, dt_bias,
              A_log, S, slots, pos0, H, G, D, V);
  DL_I32(cu_c);
  DL_I32(base);
  DL_I32(cnt);
  const int B = (int)slots.numel();
  const int64_t NC = cu_c.numel() - 1;
  TORCH_CHECK(NC >= 0 && base.numel() == B && cnt.numel() == B,
              "per-sequence chunk metadata");
  TORCH_CHECK(tl_delta_chunks_ok((int)D, (int)a2t.size(0)),
              "delta_chunks: shape outside the kernels' range");
  auto out = torch::empty({x.size(0), H * V}, x.options());
  if (x.size(0) == 0 || B == 0 || NC == 0) return out;
  const int64_t DP = tl_delta_row_pad((int)D), VP = tl_delta_col_pad((int)V);
  const int64_t n = NC * H, C = tl_delta_chunk_tokens();
  auto W = torch::empty({n, C, DP}, x.options());
  auto Q = torch::empty({n, C, DP}, x.options());
  auto Kt = torch::empty({n, DP, C}, x.options());
  auto Bm = torch::empty({n, C, C}, x.options());
  auto U = torch::empty({n, C, VP}, x.options());
  auto dec = torch::empty({n, DP}, x.options());
  const int rc = tl_delta_chunks(
      x.data_ptr(), (int)x.size(1), (int)q_off, (int)k_off, (int)v_off,
      proj.data_ptr(), (int)proj.size(1), (int)r_off, (int)a2t.size(0),
      b.data_ptr(), (int)b.size(1), (int)b_off, a2t.data_ptr(),
      dt_bias.data_ptr(), A_log.data_ptr(),
      (float)(1.0 / std::sqrt((double)D)), S.data_ptr(), cu_c.data_ptr(),
      (int)NC, base.data_ptr(), cnt.data_ptr(), slots.data_ptr(),
      pos0.data_ptr(), B, W.data_ptr(), Q.data_ptr(), Kt.data_ptr(),
      Bm.data_ptr(), U.data_ptr(), dec.data_ptr(), out.data_ptr(), (int)H,
      (int)G, (int)D, (int)V, delta_is_f32(proj), delta_stream());
  TORCH_CHECK(rc == 0, "delta_chunks: launch refused");
  return out;
}

// fp32 [T, W] = embed[token] + table[hashed bigram row]; prev [slots] int32
Tensor bigram_embed(Tensor tokens, Tensor embed, Tensor table, Tensor prev,
                    Tensor tok_seq, Tensor cu, Tensor slots, Tensor pos0,
                    int64_t mul_prev, int64_t mul_cur) {
  DL_IN(tokens);
  DL_IN(embed);
  DL_IN(table);
  DL_I32(prev);
  DL_I32(tok_seq);
  DL_I32(cu);
  DL_I32(slots);
  DL_I32(pos0);
  TORCH_CHECK(tokens.scalar_type() == torch::kLong && tokens.dim() == 1,
              "tokens must be int64 [T]");
  TORCH_CHECK(embed.dim() == 2 && table.dim() == 2 && table.size(0) >= 2 &&
                  table.size(1) == embed.size(1) &&
                  table.scalar_type() == embed.scalar_type(),
              "embed [V, W], table [n + 1, W] of one dtype");
  const int64_t T = tokens.numel(), W = embed.size(1);
  TORCH_CHECK(tok_seq.numel() == T && cu.numel() == slots.numel() + 1 &&
                  pos0.numel() == slots.numel(),
              "ragged metadata");
  auto X = torch::empty({T, W}, embed.options().dtype(torch::kFloat));
  tl_bigram_embed(tokens.data_ptr(), embed.data_ptr(), table.data_ptr(),
                  prev.data_ptr(), tok_seq.data_ptr(), cu.data_ptr(),
                  slots.data_ptr(), pos0.data_ptr(), X.data_ptr(), T, (int)W,
                  embed.size(0), table.size(0) - 1, mul_prev, mul_cur,
                  delta_is_f32(embed), delta_stream());
  return X;
}

// fp32 [T, N] = h w^T + bias
Tensor thin_linear(Tensor h, Tensor w, c10::optional<Tensor> bias) {
  DL_IN(h);
  DL_IN(w);
  TORCH_CHECK(h.dim() == 2 && w.dim() == 2 && w.size(1) == h.size(1) &&
                  w.scalar_type() == h.scalar_type(),
              "h [T, W], w [N, W] of one dtype");
  if (bias.has_value()) {
    DL_F32(bias.value());
    TORCH_CHECK(bias->numel() == w.size(0), "bias must be [N]");
  }
  auto out = torch::empty({h.size(0), w.size(0)},
                          h.options().dtype(torch::kFloat));
  tl_thin_linear(h.data_ptr(), w.data_ptr(),
                 bias.has_value() ? bias->data_ptr() : nullptr,
                 out.data_ptr(), h.size(0), (int)h.size(1), (int)w.size(0),
                 delta_is_f32(h), delta_stream());
  return out;
}

}  // namespace

void register_delta_ops(pybind11::module& mod) {
  mod.def("delta_scan", &delta_scan,
          "gated delta rule over ragged sequences (slot state)");
  mod.def("delta_chunk_tokens", &delta_chunk_tokens,
          "tokens per chunk of the chunk form");
  mod.def("delta_chunks_ok", &delta_chunks_ok,
          "whether the chunk kernels serve a shape");
  mod.def("delta_chunks", &delta_chunks,
          "gated delta rule, chunk form on fp32 MFMA");
  mod.def("bigram_embed", &bigram_embed,
          "token embedding plus a hashed bigram embedding");
  mod.def("thin_linear", &thin_linear,
          "fp32 results of a projection to few outputs, few rows");
}
