// torch custom-op bindings (namespace `dlia`) of the kernels for stacks with plain-weight norms on both sides of every sublayer,
// bigram embeddings, mapped passes of a repeated stretch and per-head query / key norms. As everywhere in this library, shapes,
// types and devices are checked on the host before anything is launched.
#include <torch/library.h>
#include <ATen/ATen.h>
#include <ATen/hip/impl/HIPGuardImplMasqueradingAsCUDA.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>
#include <c10/util/Optional.h>

#include "launch.h"

namespace {

using at::Tensor;
using OptTensor = const std::optional<Tensor>&;

inline hipStream_t cur_stream() { return c10::hip::getCurrentHIPStreamMasqueradingAsCUDA().stream(); }

#define DLIA_CHECK(cond, ...) TORCH_CHECK(cond, "dlia: ", __VA_ARGS__)
#define DLIA_ON_DEVICE_OF(t) \
  DLIA_CHECK((t).is_cuda(), #t " must be a GPU tensor"); \
  const c10::hip::HIPGuardMasqueradingAsCUDA dlia_device_guard_((t).device())

inline bool is_f32(const Tensor& t) { return t.scalar_type() == at::kFloat; }
inline void check_f32(const Tensor& t, const char* name) {
  DLIA_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous(), name, " must be contiguous float32 on the GPU");
}
inline void check_i32(const Tensor& t, const char* name) {
  DLIA_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous(), name, " must be contiguous int32 on the GPU");
}
inline void check_act(const Tensor& t, const char* name) {
  DLIA_CHECK(t.is_cuda() && (t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16), name, " must be float32 or bfloat16 on the GPU");
}
inline void check_mat(const Tensor& t, const char* name) {
  DLIA_CHECK(t.dim() == 2 && (t.size(1) == 1 || t.stride(1) == 1), name, " must be 2-D with unit inner stride");
}
inline void check_fmat(const Tensor& t, const char* name) {
  check_mat(t, name);
  DLIA_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat, name, " must be float32 on the GPU");
}
inline const float* opt_f32(OptTensor t, int64_t n, const char* name) {
  if (!t.has_value()) return nullptr;
  check_f32(*t, name);
  DLIA_CHECK(t->numel() >= n, name, " has too few elements");
  return t->data_ptr<float>();
}

// out [T, H] fp32 = table[id] * scale (+ bigram[hash(previous id, id)]); cat [T, 2 H]: the second half (and with cat_both the first)
// gets the same row in the table's type. pages [blocks, 32]: every token's id at its place in its sequence's blocks.
void embed_bigram(Tensor out, const std::optional<Tensor>& cat, bool cat_both, const Tensor& ids, const Tensor& table, double scale,
                  OptTensor bigram, int64_t mul_prev, int64_t mul_cur, const std::optional<Tensor>& pages, const Tensor& tok_pos,
                  const Tensor& tok_seq, const Tensor& block_table) {
  DLIA_ON_DEVICE_OF(out);
  check_f32(out, "out"); check_i32(ids, "ids"); check_act(table, "table");
  check_i32(tok_pos, "tok_pos"); check_i32(tok_seq, "tok_seq"); check_i32(block_table, "block_table");
  const int64_t T = out.size(0), H = out.size(1);
  DLIA_CHECK(out.dim() == 2 && table.dim() == 2 && table.is_contiguous() && table.size(1) == H && table.size(0) >= 1 && ids.numel() >= T &&
             tok_pos.numel() >= T && tok_seq.numel() >= T && block_table.dim() == 2, "embed_bigram: out [T, H], table [vocab, H], per-token metadata");
  void* cp = nullptr; long ldc = 0;
  if (cat.has_value()) {
    check_mat(*cat, "cat");
    DLIA_CHECK(cat->is_cuda() && cat->scalar_type() == table.scalar_type() && cat->size(0) >= T && cat->size(1) == 2 * H, "embed_bigram: cat [T, 2 H] of the table's type");
    cp = cat->data_ptr(); ldc = cat->stride(0);
  }
  const void* bp = nullptr; int* pp = nullptr; int64_t buckets = 1, blocks = 0;
  if (bigram.has_value()) {
    DLIA_CHECK(bigram->is_cuda() && bigram->dim() == 2 && bigram->is_contiguous() && bigram->scalar_type() == table.scalar_type() &&
               bigram->size(1) == H && bigram->size(0) >= 2 && mul_prev >= 0 && mul_cur >= 0 && mul_prev < (1ll << 31) && mul_cur < (1ll << 31),
               "embed_bigram: bigram [buckets + 1, H] of the table's type, multipliers below 2^31");
    DLIA_CHECK(pages.has_value(), "embed_bigram: the bigram table needs the pages of token ids");
    check_i32(*pages, "pages");
    DLIA_CHECK(pages->dim() == 2 && pages->size(1) == 32, "embed_bigram: pages [blocks, 32]");
    bp = bigram->data_ptr(); buckets = bigram->size(0) - 1; pp = pages->data_ptr<int>(); blocks = pages->size(0);
  }
  dlia_embed_bigram(out.data_ptr<float>(), cp, ldc, cat_both ? 1 : 0, ids.data_ptr<int>(), table.data_ptr(), is_f32(table), (float)scale, bp,
                    (int)buckets, (long)mul_prev, (long)mul_cur, pp, tok_pos.data_ptr<int>(), tok_seq.data_ptr<int>(), block_table.data_ptr<int>(),
                    (int)T, (int)block_table.size(1), (int)blocks, (int)block_table.size(0), (int)H, (int)table.size(0), cur_stream());
}

int64_t sandwich_join_max_width(bool vec) { return dlia_sandwich_join_max_width(vec ? 1 : 0); }

// y = ya (as it is, or the sum of its first dimension's partial results) + the token's rows of ey; x += rms(y) wb; out = rms(x) wn, or x itself without wn. Without wb only the second half.
void sandwich_join(const std::optional<Tensor>& out, Tensor x, OptTensor ya, OptTensor ey, OptTensor pair_row, int64_t top,
                   OptTensor wb, OptTensor wn, double eps) {
  DLIA_ON_DEVICE_OF(x);
  check_fmat(x, "x");
  const int64_t T = x.size(0), H = x.size(1);
  const float *ap = nullptr, *ep = nullptr; const int* pp = nullptr;
  long lda = 0, step = 0; int parts = 1;
  if (ya.has_value()) {
    DLIA_CHECK(ya->is_cuda() && ya->scalar_type() == at::kFloat && (ya->dim() == 2 || ya->dim() == 3) && (ya->size(-1) == 1 || ya->stride(-1) == 1) &&
               ya->size(-1) == H && ya->size(-2) >= T, "sandwich_join: ya float32 [T, H] or [parts, T, H]");
    ap = ya->data_ptr<float>(); lda = ya->stride(-2);
    if (ya->dim() == 3) { parts = (int)ya->size(0); step = ya->stride(0); }
  }
  if (ey.has_value()) {
    check_f32(*ey, "ey");
    DLIA_CHECK(ey->dim() == 2 && ey->size(1) == H && pair_row.has_value() && top >= 1, "sandwich_join: expert rows [rows, H] with their places");
    check_i32(*pair_row, "pair_row");
    DLIA_CHECK(pair_row->numel() >= T * top, "sandwich_join: pair_row [T, top]");
    ep = ey->data_ptr<float>(); pp = pair_row->data_ptr<int>();
  }
  DLIA_CHECK((ap || ep) == wb.has_value(), "sandwich_join: a sublayer's output comes with its norm's weight");
  void* op = nullptr; long ldo = 0; int of32 = 1;
  if (out.has_value()) {
    check_act(*out, "out"); check_mat(*out, "out");
    DLIA_CHECK(out->size(0) >= T && out->size(1) == H, "sandwich_join: out [T, H]");
    op = out->data_ptr(); ldo = out->stride(0); of32 = is_f32(*out);
  }
  DLIA_CHECK(op || wb.has_value(), "sandwich_join: nothing to do");
  const int rc = dlia_sandwich_join(op, of32, ldo, x.data_ptr<float>(), x.stride(0), ap, lda, parts, step, ep, pp, (int)top, opt_f32(wb, H, "wb"),
                                    opt_f32(wn, H, "wn"), (int)T, (int)H, (float)eps, cur_stream());
  DLIA_CHECK(rc == 0, "sandwich_join: rows of ", H, " are beyond what the kernel holds in registers");
}

// z [T, q | k (| v at col_v) ...]; q_out [T, H d]; layout 0: kc [blocks, G, 32, d], vc [blocks, G, 32, dv]; 1: vc [blocks, G, dv, 32];
// 2: kc [blocks, G, 2, 32 d] in fragment order, no vc.
void qk_prep(const Tensor& z, int64_t H, int64_t G, int64_t d, int64_t dv, int64_t col_v, OptTensor qw, OptTensor kw, bool unit, double eps,
             int64_t dims, bool interleaved, OptTensor cos_t, OptTensor sin_t, Tensor q_out, Tensor kc, const std::optional<Tensor>& vc,
             int64_t layout, const Tensor& tok_pos, const Tensor& tok_seq, const Tensor& block_table) {
  DLIA_ON_DEVICE_OF(kc);
  check_act(z, "z"); check_mat(z, "z"); check_act(q_out, "q_out"); check_mat(q_out, "q_out"); check_act(kc, "kc");
  check_i32(tok_pos, "tok_pos"); check_i32(tok_seq, "tok_seq"); check_i32(block_table, "block_table");
  const int64_t T = z.size(0);
  DLIA_CHECK(H >= 1 && G >= 1 && H % G == 0 && d >= 1 && dv >= 1 && (col_v >= 0 || dv == d), "qk_prep: head geometry");
  DLIA_CHECK(z.size(1) >= (H + G) * d && (col_v < 0 || (col_v >= (H + G) * d && z.size(1) >= col_v + G * dv)), "qk_prep: columns of z");
  DLIA_CHECK(q_out.size(0) >= T && q_out.size(1) == H * d && tok_pos.numel() >= T && tok_seq.numel() >= T && block_table.dim() == 2, "qk_prep: rows");
  DLIA_CHECK(dims >= 0 && dims % 2 == 0 && dims <= d && qw.has_value() == kw.has_value(), "qk_prep: rotated entries, norm weights");
  DLIA_CHECK(layout >= 0 && layout <= 2 && kc.is_contiguous() && kc.dim() == 4 && kc.size(1) == G, "qk_prep: caches [blocks, G, ., .]");
  void* vp = nullptr;
  if (layout == 2) {
    DLIA_CHECK(!vc.has_value() && kc.size(2) == 2 && kc.size(3) == 32 * d && d == dv && (d == 64 || d == 128) && kc.scalar_type() == at::kBFloat16,
               "qk_prep: fragment-ordered cache [blocks, G, 2, 32 d] in bfloat16, d = dv of 64 or 128");
  } else {
    DLIA_CHECK(vc.has_value(), "qk_prep: a value cache");
    check_act(*vc, "vc");
    DLIA_CHECK(kc.size(2) == 32 && kc.size(3) == d && vc->is_contiguous() && vc->dim() == 4 && vc->size(0) == kc.size(0) && vc->size(1) == G &&
               vc->size(layout == 1 ? 2 : 3) == dv && vc->size(layout == 1 ? 3 : 2) == 32 && vc->scalar_type() == kc.scalar_type(),
               "qk_prep: kc [blocks, G, 32, d], vc [blocks, G, 32, dv] (or [blocks, G, dv, 32]) of one type");
    vp = vc->data_ptr();
  }
  const float *cp = nullptr, *sp = nullptr; int table_pos = 0;
  if (dims > 0) {
    DLIA_CHECK(cos_t.has_value() && sin_t.has_value(), "qk_prep: rotation needs its tables");
    check_f32(*cos_t, "cos"); check_f32(*sin_t, "sin");
    DLIA_CHECK(cos_t->dim() == 2 && cos_t->size(1) == dims / 2 && sin_t->sizes() == cos_t->sizes(), "qk_prep: tables [positions, dims / 2]");
    cp = cos_t->data_ptr<float>(); sp = sin_t->data_ptr<float>(); table_pos = (int)cos_t->size(0);
  }
  const int rc = dlia_qk_prep(z.data_ptr(), is_f32(z), z.stride(0), (int)T, (int)H, (int)G, (int)d, (int)dv, (int)col_v, opt_f32(qw, d, "qw"),
                              opt_f32(kw, d, "kw"), unit ? 1 : 0, (float)eps, (int)dims, interleaved ? 1 : 0, cp, sp, table_pos, q_out.data_ptr(),
                              is_f32(q_out), q_out.stride(0), kc.data_ptr(), vp, is_f32(kc), (int)layout, tok_pos.data_ptr<int>(),
                              tok_seq.data_ptr<int>(), block_table.data_ptr<int>(), (int)block_table.size(1), (int)kc.size(0),
                              (int)block_table.size(0), cur_stream());
  DLIA_CHECK(rc == 0, "qk_prep: types or sizes not taken (heads up to 512 entries; an fp32 cache takes fp32 rows; fragment order wants aligned rows)");
}

// act [M, F] = relu(z)^2 from z [M, >= F], or relu(gate) * up from gate | up in z [M, >= 2 F]
void relu_act(Tensor act, const Tensor& z, bool glu) {
  DLIA_ON_DEVICE_OF(act);
  check_act(act, "act"); check_mat(act, "act"); check_act(z, "z"); check_mat(z, "z");
  DLIA_CHECK(z.size(0) >= act.size(0) && z.size(1) >= (glu ? 2 : 1) * act.size(1), "relu_act: act [M, F] from z [M, F] or [M, 2 F]");
  dlia_relu_act(act.data_ptr(), is_f32(act), act.stride(0), z.data_ptr(), is_f32(z), z.stride(0), (int)act.size(0), (int)act.size(1), glu ? 1 : 0,
                cur_stream());
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(dlia, m) {
  m.def("embed_bigram(Tensor(a!) out, Tensor(b!)? cat, bool cat_both, Tensor ids, Tensor table, float scale, Tensor? bigram, int mul_prev, int mul_cur, Tensor(c!)? pages, Tensor tok_pos, Tensor tok_seq, Tensor block_table) -> ()");
  m.def("sandwich_join_max_width(bool vec) -> int");
  m.def("sandwich_join(Tensor(a!)? out, Tensor(b!) x, Tensor? ya, Tensor? ey, Tensor? pair_row, int top, Tensor? wb, Tensor? wn, float eps) -> ()");
  m.def("qk_prep(Tensor z, int H, int G, int d, int dv, int col_v, Tensor? qw, Tensor? kw, bool unit, float eps, int dims, bool interleaved, Tensor? cos_t, Tensor? sin_t, Tensor(a!) q_out, Tensor(b!) kc, Tensor(c!)? vc, int layout, Tensor tok_pos, Tensor tok_seq, Tensor block_table) -> ()");
  m.def("relu_act(Tensor(a!) act, Tensor z, bool glu) -> ()");
}

TORCH_LIBRARY_IMPL(dlia, CUDA, m) {
  m.impl("embed_bigram", &embed_bigram);
  m.impl("sandwich_join", &sandwich_join);
  m.impl("qk_prep", &qk_prep);
  m.impl("relu_act", &relu_act);
}

TORCH_LIBRARY_IMPL(dlia, CompositeExplicitAutograd, m) {
  m.impl("sandwich_join_max_width", &sandwich_join_max_width);
}
