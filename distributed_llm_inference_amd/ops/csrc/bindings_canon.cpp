// torch custom-op bindings (namespace `dlia`) of the kernels for stacks with convolved sublayer inputs, a learned average over
// depth, linear attention with decays, PolyNorm and experts chosen by token id. As everywhere in this library, shapes, types
// and devices are checked on the host before anything is launched.
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

inline int64_t carry_rows(const Tensor& carry, int64_t K, int64_t H, const char* name) {
  check_f32(carry, name);
  DLIA_CHECK(carry.dim() == 3 && carry.size(1) == K - 1 && carry.size(2) == H, name, " must be [slots, taps - 1, H]");
  return carry.size(0);
}

// x <- x_in + ya + yb + ew * (the token's expert rows); hist[navg] <- x and x <- sum_j coef[j] hist[j] when hist is given; rs <- the row
// factors of the next norm (nw). out given (steps of single tokens): g = h + conv(h), with the slots' rings. close_carry given
// (other steps): the last h of every sequence of the sublayer that closes (norm weight close_w, factors in rs) go to its ring.
void stream_join(const std::optional<Tensor>& out, Tensor x, const Tensor& x_in, OptTensor ya, OptTensor yb, OptTensor ey,
                 OptTensor pair_row, int64_t top, double ew, const std::optional<Tensor>& hist, int64_t navg, OptTensor coef, OptTensor nw,
                 Tensor rs, OptTensor close_w, const std::optional<Tensor>& close_carry, OptTensor taps, const std::optional<Tensor>& carry,
                 const Tensor& tok_pos, const Tensor& tok_seq, double eps) {
  DLIA_ON_DEVICE_OF(x);
  check_f32(x, "x"); check_f32(x_in, "x_in"); check_f32(rs, "rs"); check_i32(tok_pos, "tok_pos"); check_i32(tok_seq, "tok_seq");
  DLIA_CHECK(x.dim() == 2, "stream_join: x [T, H]");
  const int64_t T = x.size(0), H = x.size(1);
  DLIA_CHECK(x_in.dim() == 2 && x_in.size(0) >= T && x_in.size(1) == H && rs.numel() >= T && tok_pos.numel() >= T && tok_seq.numel() >= T,
             "stream_join: x_in [T, H], rs, tok_pos, tok_seq [T]");
  auto rows = [&](OptTensor y, const char* name, long& ld) -> const float* {
    if (!y.has_value()) return nullptr;
    check_fmat(*y, name);
    DLIA_CHECK(y->size(0) >= T && y->size(1) == H, name, " must be [T, H]");
    ld = y->stride(0);
    return y->data_ptr<float>();
  };
  long ldya = 0, ldyb = 0;
  const float *yap = rows(ya, "ya", ldya), *ybp = rows(yb, "yb", ldyb), *eyp = nullptr;
  const int* prp = nullptr;
  if (ey.has_value()) {
    check_f32(*ey, "ey");
    DLIA_CHECK(ey->dim() == 2 && ey->size(1) == H && top >= 1 && pair_row.has_value(), "stream_join: ey [rows, H] with its pairs");
    check_i32(*pair_row, "pair_row");
    DLIA_CHECK(pair_row->numel() >= T * top, "stream_join: pair_row [T * top]");
    eyp = ey->data_ptr<float>(); prp = pair_row->data_ptr<int>();
  }
  float* hp = nullptr; long hs = 0;
  if (hist.has_value()) {
    DLIA_CHECK(hist->is_cuda() && hist->scalar_type() == at::kFloat && hist->dim() == 3 && hist->size(0) > navg && navg >= 1 && hist->size(1) >= T &&
               hist->size(2) == H && hist->stride(2) == 1 && hist->stride(1) == H && coef.has_value(), "stream_join: hist [> navg, T, H] with navg + 1 coefficients");
    DLIA_CHECK(hist->data_ptr<float>() != x.data_ptr<float>(), "stream_join: the stream is not a row of the history");
    hp = hist->data_ptr<float>(); hs = hist->stride(0);
  }
  int64_t K = 0, srows = 0;
  const float* tp = nullptr; float* cp = nullptr; float* ccp = nullptr;
  if (taps.has_value()) {
    check_f32(*taps, "taps");
    DLIA_CHECK(taps->dim() == 2 && taps->size(0) >= 1 && taps->size(1) == H, "stream_join: taps [taps, H]");
    K = taps->size(0); tp = taps->data_ptr<float>();
  }
  if (close_carry.has_value()) {
    DLIA_CHECK(close_carry->dim() == 3 && close_w.has_value() && (K == 0 || K == close_carry->size(1) + 1) && !out.has_value(),
               "stream_join: the closing ring comes with its norm weight, in steps whose convolution runs apart");
    K = close_carry->size(1) + 1;
    srows = carry_rows(*close_carry, K, H, "close_carry"); ccp = close_carry->data_ptr<float>();
  }
  if (carry.has_value()) {
    DLIA_CHECK(tp && out.has_value(), "stream_join: a ring comes with its taps, in steps of single tokens");
    srows = carry_rows(*carry, K, H, "carry"); cp = carry->data_ptr<float>();
  }
  void* op = nullptr; long ldo = 0; int of32 = 1;
  if (out.has_value()) {
    check_act(*out, "out"); check_mat(*out, "out");
    DLIA_CHECK(out->size(0) >= T && out->size(1) == H && nw.has_value() && (!tp || K == 1 || cp), "stream_join: out [T, H] with the next norm's weight and the ring");
    op = out->data_ptr(); ldo = out->stride(0); of32 = is_f32(*out);
  }
  const int rc = dlia_stream_join(op, of32, ldo, x.data_ptr<float>(), x_in.data_ptr<float>(), yap, ldya, ybp, ldyb, eyp, prp, (int)top, (float)ew, hp,
                                  hs, (int)navg, opt_f32(coef, navg + 1, "coef"), opt_f32(nw, H, "nw"), rs.data_ptr<float>(), opt_f32(close_w, H, "close_w"),
                                  ccp, tp, cp, (int)K, tok_pos.data_ptr<int>(), tok_seq.data_ptr<int>(), (int)T, (int)srows, (int)H, (float)eps, cur_stream());
  DLIA_CHECK(rc == 0, "stream_join: rows of ", H, " entries are wider than the kernel takes");
}

// g = h + conv(h), h = x rs (1 + nw); earlier h from the step's rows or from the slots' rings.
void canon_conv(Tensor out, const Tensor& x, const Tensor& rs, const Tensor& nw, OptTensor taps, OptTensor carry, const Tensor& tok_pos,
                const Tensor& tok_seq) {
  DLIA_ON_DEVICE_OF(x);
  check_f32(x, "x"); check_f32(rs, "rs"); check_f32(nw, "nw"); check_i32(tok_pos, "tok_pos"); check_i32(tok_seq, "tok_seq");
  check_act(out, "out"); check_mat(out, "out");
  DLIA_CHECK(x.dim() == 2, "canon_conv: x [T, H]");
  const int64_t T = x.size(0), H = x.size(1);
  DLIA_CHECK(out.size(0) >= T && out.size(1) == H && rs.numel() >= T && nw.numel() == H && tok_pos.numel() >= T && tok_seq.numel() >= T, "canon_conv: shapes");
  int64_t K = 0, srows = 0;
  const float *tp = nullptr, *cp = nullptr;
  if (taps.has_value()) {
    check_f32(*taps, "taps");
    DLIA_CHECK(taps->dim() == 2 && taps->size(0) >= 1 && taps->size(1) == H && (taps->size(0) == 1 || carry.has_value()), "canon_conv: taps [taps, H] with their ring");
    K = taps->size(0); tp = taps->data_ptr<float>();
    if (carry.has_value()) { srows = carry_rows(*carry, K, H, "carry"); cp = carry->data_ptr<float>(); }
  }
  dlia_canon_conv(out.data_ptr(), is_f32(out), out.stride(0), x.data_ptr<float>(), rs.data_ptr<float>(), nw.data_ptr<float>(), tp, cp, (int)K,
                  tok_pos.data_ptr<int>(), tok_seq.data_ptr<int>(), (int)T, (int)srows, (int)H, cur_stream());
}

void poly_norm(Tensor out, const Tensor& z, const Tensor& coef, double eps) {
  DLIA_ON_DEVICE_OF(out);
  check_act(out, "out"); check_mat(out, "out"); check_fmat(z, "z"); check_f32(coef, "coef");
  DLIA_CHECK(z.size(0) >= out.size(0) && z.size(1) >= out.size(1) && coef.numel() == 4, "poly_norm: out [T, F] from z [T, >= F], four numbers");
  dlia_poly_norm(out.data_ptr(), is_f32(out), out.stride(0), z.data_ptr<float>(), z.stride(0), coef.data_ptr<float>(), (int)out.size(0),
                 (int)out.size(1), (float)eps, cur_stream());
}

int64_t linear_attention_ws_floats(int64_t rows, int64_t B, int64_t H, int64_t d, int64_t dv, bool per_channel) {
  return dlia_linear_attention_ws_floats((int)rows, (int)B, (int)H, (int)d, (int)dv, per_channel ? 1 : 0);
}

// out [T, H dv] = rms(o) norm_w silu(g) per head; z [T, .]: q | k | v | g (| low-rank projection) at the given columns; state
// [slots, H, d, dv]. head_decay [2, H] (decay, its log2), or a2t [rank, H d] and a_b [H d].
void linear_attention(Tensor out, const Tensor& z, Tensor state, OptTensor head_decay, OptTensor a2t, OptTensor a_b, OptTensor norm_w,
                      const Tensor& q_start, const Tensor& ctx, const Tensor& slots, int64_t H, int64_t d, int64_t dv, int64_t col_q,
                      int64_t col_k, int64_t col_v, int64_t col_g, int64_t col_a, double qscale, double inv_tau, double eps, int64_t max_q,
                      const std::optional<Tensor>& ws) {
  DLIA_ON_DEVICE_OF(out);
  check_act(out, "out"); check_mat(out, "out"); check_fmat(z, "z"); check_f32(state, "state");
  check_i32(q_start, "q_start"); check_i32(ctx, "ctx"); check_i32(slots, "slots");
  const int64_t T = out.size(0), B = ctx.numel(), ZC = z.size(1);
  DLIA_CHECK(H >= 1 && d >= 1 && d <= 512 && dv >= 1 && dv <= 512 && out.size(1) == H * dv && z.size(0) >= T, "linear_attention: key / value sizes up to 512, out [T, H dv]");
  DLIA_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == d && state.size(3) == dv, "linear_attention: state [slots, H, d, dv]");
  DLIA_CHECK(q_start.numel() >= B + 1 && slots.numel() >= B && max_q >= 0 && max_q <= T && (max_q != 1 || T <= B), "linear_attention: metadata");
  auto span = [&](int64_t col, int64_t n) { return col >= 0 && col + n <= ZC; };
  DLIA_CHECK(span(col_q, H * d) && span(col_k, H * d) && span(col_v, H * dv) && span(col_g, H * dv), "linear_attention: columns");
  int64_t rank = 0;
  if (!head_decay.has_value()) {
    DLIA_CHECK(a2t.has_value() && a_b.has_value() && a2t->dim() == 2 && a2t->size(1) == H * d, "linear_attention: decays per head, or a2t [rank, H d] with its bias");
    rank = a2t->size(0);
    DLIA_CHECK(span(col_a, rank), "linear_attention: columns of the low-rank projection");
  }
  const int rc = dlia_linear_attention(out.data_ptr(), is_f32(out), out.stride(0), z.data_ptr<float>(), z.stride(0), state.data_ptr<float>(),
                                       opt_f32(head_decay, 2 * H, "head_decay"), opt_f32(a2t, rank * H * d, "a2t"), opt_f32(a_b, H * d, "a_b"), (int)rank,
                                       opt_f32(norm_w, dv, "norm_w"), q_start.data_ptr<int>(), ctx.data_ptr<int>(), slots.data_ptr<int>(), (int)B, (int)T,
                                       (int)max_q, (int)H, (int)d, (int)dv, (int)state.size(0), (int)col_q, (int)col_k, (int)col_v, (int)col_g, (int)col_a,
                                       (float)qscale, (float)inv_tau, (float)eps, const_cast<float*>(opt_f32(ws, 1, "ws")),
                                       ws.has_value() ? (long)ws->numel() : 0, cur_stream());
  DLIA_CHECK(rc != 2, "linear_attention: a step with portions needs the workspace (linear_attention_ws_floats)");
  DLIA_CHECK(rc == 0, "linear_attention: sizes");
}

int64_t stream_join_max_width(bool vec) { return dlia_stream_join_max_width(vec ? 1 : 0); }

// One plan per routed layer from the step's token ids. desc [layers, 8] on the host and on the device (the same numbers).
void moe_table_plan(Tensor tiles, Tensor row_tok, Tensor pair_row, const Tensor& tables, const Tensor& ids, const Tensor& desc,
                    const Tensor& desc_host, int64_t T, int64_t vocab, int64_t big_pairs) {
  DLIA_ON_DEVICE_OF(tiles);
  check_i32(tiles, "tiles"); check_i32(row_tok, "row_tok"); check_i32(pair_row, "pair_row"); check_i32(tables, "tables"); check_i32(ids, "ids"); check_i32(desc, "desc");
  DLIA_CHECK(desc_host.device().is_cpu() && desc_host.scalar_type() == at::kInt && desc_host.is_contiguous() && desc_host.dim() == 2 && desc_host.size(1) == 8 &&
             desc.sizes() == desc_host.sizes() && ids.numel() >= T && T >= 0 && vocab >= 1 && big_pairs >= 0, "moe_table_plan: descriptors [layers, 8], ids [T]");
  const int* dh = desc_host.data_ptr<int>();
  for (int64_t l = 0; l < desc_host.size(0); ++l, dh += 8) {
    const int64_t top = dh[1], E = dh[2], pairs = T * top, tr = dh[6] && pairs >= big_pairs ? 128 : 32, nt = (pairs + tr - 1) / tr + E;
    DLIA_CHECK(top >= 1 && E >= 1 && E <= 1024 && dh[0] >= 0 && dh[0] + vocab * top <= tables.numel() && dh[3] >= 0 && dh[3] + 1 + nt <= tiles.numel() &&
               dh[4] >= 0 && dh[4] + nt * tr <= row_tok.numel() && dh[5] >= 0 && dh[5] + pairs <= pair_row.numel(), "moe_table_plan: layer ", l, " does not fit its buffers");
  }
  dlia_moe_table_plan(tiles.data_ptr<int>(), row_tok.data_ptr<int>(), pair_row.data_ptr<int>(), tables.data_ptr<int>(), ids.data_ptr<int>(),
                      desc.data_ptr<int>(), (int)desc_host.size(0), (int)T, (int)vocab, (int)big_pairs, cur_stream());
}

void glu_act(Tensor act, const Tensor& z, double limit, bool gated) {
  DLIA_ON_DEVICE_OF(act);
  check_act(act, "act"); check_mat(act, "act"); check_fmat(z, "z");
  DLIA_CHECK(z.size(0) >= act.size(0) && z.size(1) >= 2 * act.size(1) + (gated ? 1 : 0), "glu_act: act [M, F] from gate | up (| one number) in z");
  dlia_glu_act(act.data_ptr(), is_f32(act), act.stride(0), z.data_ptr<float>(), z.stride(0), (int)act.size(0), (int)act.size(1), (float)limit,
               gated ? 1 : 0, cur_stream());
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(dlia, m) {
  m.def("stream_join(Tensor(a!)? out, Tensor(b!) x, Tensor x_in, Tensor? ya, Tensor? yb, Tensor? ey, Tensor? pair_row, int top, float ew, Tensor(c!)? hist, int navg, Tensor? coef, Tensor? nw, Tensor(d!) rs, Tensor? close_w, Tensor(e!)? close_carry, Tensor? taps, Tensor(f!)? carry, Tensor tok_pos, Tensor tok_seq, float eps) -> ()");
  m.def("stream_join_max_width(bool vec) -> int");
  m.def("canon_conv(Tensor(a!) out, Tensor x, Tensor rs, Tensor nw, Tensor? taps, Tensor? carry, Tensor tok_pos, Tensor tok_seq) -> ()");
  m.def("poly_norm(Tensor(a!) out, Tensor z, Tensor coef, float eps) -> ()");
  m.def("linear_attention_ws_floats(int rows, int B, int H, int d, int dv, bool per_channel) -> int");
  m.def("linear_attention(Tensor(a!) out, Tensor z, Tensor(b!) state, Tensor? head_decay, Tensor? a2t, Tensor? a_b, Tensor? norm_w, Tensor q_start, Tensor ctx, Tensor slots, int H, int d, int dv, int col_q, int col_k, int col_v, int col_g, int col_a, float qscale, float inv_tau, float eps, int max_q, Tensor(c!)? ws) -> ()");
  m.def("moe_table_plan(Tensor(a!) tiles, Tensor(b!) row_tok, Tensor(c!) pair_row, Tensor tables, Tensor ids, Tensor desc, Tensor desc_host, int T, int vocab, int big_pairs) -> ()");
  m.def("glu_act(Tensor(a!) act, Tensor z, float limit, bool gated) -> ()");
}

TORCH_LIBRARY_IMPL(dlia, CUDA, m) {
  m.impl("stream_join", &stream_join);
  m.impl("canon_conv", &canon_conv);
  m.impl("poly_norm", &poly_norm);
  m.impl("linear_attention", &linear_attention);
  m.impl("moe_table_plan", &moe_table_plan);
  m.impl("glu_act", &glu_act);
}

TORCH_LIBRARY_IMPL(dlia, CompositeExplicitAutograd, m) {
  m.impl("stream_join_max_width", &stream_join_max_width);
  m.impl("linear_attention_ws_floats", &linear_attention_ws_floats);
}
