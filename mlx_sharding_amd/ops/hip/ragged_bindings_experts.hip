// Python bindings of the routed experts.
#include "ragged_bindings.h"
#include "ragged_experts.h"

extern "C" {
void launch_expert_route(const RouteArgs*, bool, hipStream_t);
void launch_expert_plan(const PlanArgs*, hipStream_t);
void launch_expert_gemm(const ExpertGemmArgs*, int, bool, hipStream_t);
void launch_expert_combine(const CombineArgs*, bool, hipStream_t);
void launch_token_gate(const TokenGateArgs*, bool, hipStream_t);
}

namespace {

Tensor int_rows(const Tensor& like, std::vector<int64_t> sizes) {
  return torch::empty(sizes, like.options().dtype(torch::kInt32));
}

// h [N, K], w [total / 16, K / 32, 64, 8], correction [total] or none
// -> chosen [N, top], weights [N, top], ranks [N, top], histograms
std::tuple<Tensor, Tensor, Tensor, Tensor> expert_route(
    Tensor h, Tensor w, c10::optional<Tensor> correction, int64_t total,
    int64_t experts, int64_t top, bool sigmoid, bool normalize) {
  const bool f32 = is_f32(h, "h");
  check_like(w, h, "router");
  RouteArgs a = {};
  a.sigmoid = sigmoid;
  a.normalize = normalize;
  a.hstride = rows2(h, "h");
  a.n = h.size(0);
  a.K = (int)h.size(1);
  a.total = (int)total;
  TORCH_CHECK(a.K % EX_STEP == 0 && a.hstride % 8 == 0);
  TORCH_CHECK(w.dim() == 4 && w.is_contiguous() &&
              w.size(0) == (a.total + 15) / 16 && w.size(1) == a.K / 32 &&
              w.size(2) == 64 && w.size(3) == 8, "router not packed for h");
  aligned16(h, "h");
  aligned16(w, "router");
  a.experts = (int)experts;
  a.top = (int)top;
  TORCH_CHECK(a.total <= EX_MAXTOTAL && experts >= 1 && experts <= a.total &&
              top >= 1 && top <= a.total);
  if (correction) {
    check_like(*correction, h, "correction");
    TORCH_CHECK(correction->is_contiguous() && correction->numel() == total);
    a.correction = correction->data_ptr();
  }
  const long blocks = (a.n + EX_TOK - 1) / EX_TOK;
  auto idx = int_rows(h, {a.n, top}), rank = int_rows(h, {a.n, top});
  auto hist = int_rows(h, {blocks, experts});
  auto weight = torch::empty({a.n, top}, h.options().dtype(torch::kFloat32));
  a.h = h.data_ptr();
  a.w = w.data_ptr();
  a.idx = idx.data_ptr<int>();
  a.weight = weight.data_ptr<float>();
  a.rank = rank.data_ptr<int>();
  a.hist = hist.data_ptr<int>();
  if (a.n) launch_expert_route(&a, f32, stream());
  return {idx, weight, rank, hist};
}

// -> rows of the pairs [N, top], tokens of the rows [N * top], tiles [*, 3], and
// the rows' weights [N * top] if weight is given
std::tuple<Tensor, Tensor, Tensor, c10::optional<Tensor>> expert_plan(
    Tensor idx, Tensor rank, Tensor hist, c10::optional<Tensor> weight,
    int64_t experts, int64_t tile) {
  PlanArgs a = {};
  TORCH_CHECK(idx.dim() == 2 && hist.dim() == 2);
  a.n = idx.size(0);
  a.top = (int)idx.size(1);
  a.experts = (int)experts;
  a.tile = (int)tile;
  a.n_blocks = (int)hist.size(0);
  TORCH_CHECK(tile >= 1 && experts >= 1 && experts <= EX_MAXTOTAL &&
              hist.size(1) == experts &&
              a.n_blocks == (a.n + EX_TOK - 1) / EX_TOK);
  const long pairs = a.n * a.top;
  TORCH_CHECK(pairs < (1L << 31), "too many tokens in one step");
  // every expert may leave one tile unfilled, and none has more than all pairs
  a.n_tiles = (int)(pairs / tile + std::min<long>(experts, pairs));
  TORCH_CHECK(a.n_tiles <= 65535 * 16L);
  auto where = int_rows(idx, {a.n, a.top}), tokens = int_rows(idx, {pairs});
  auto tiles = int_rows(idx, {a.n_tiles, 3});
  a.idx = ints(idx, pairs, "idx");
  a.rank = ints(rank, pairs, "rank");
  a.hist = ints(hist, 0, "hist");
  a.where = where.data_ptr<int>();
  a.tokens = tokens.data_ptr<int>();
  a.tiles = tiles.data_ptr<int>();
  c10::optional<Tensor> scale;
  if (weight) {
    check_f32(*weight, "weight");
    TORCH_CHECK(weight->numel() == pairs);
    scale = torch::empty({pairs}, weight->options());
    a.weight = weight->data_ptr<float>();
    a.scale = scale->data_ptr<float>();
  }
  if (a.n) launch_expert_plan(&a, stream());
  return {where, tokens, tiles, scale};
}

// x rows (of `tokens`, or the pairs' own) times w [experts, O, K] and the rows'
// scale -> [pairs, O], half of it for gated units; rows padded to whole vectors
Tensor expert_gemm(Tensor x, c10::optional<Tensor> tokens, Tensor tiles,
                   Tensor w, c10::optional<Tensor> scale, int64_t tile,
                   int64_t pairs, int64_t act, double limit, double alpha) {
  const bool f32 = is_f32(x, "x");
  check_like(w, x, "w");
  ExpertGemmArgs a = {};
  a.xstride = rows2(x, "x");
  TORCH_CHECK(w.dim() == 3 && w.is_contiguous() && x.size(1) == w.size(2));
  a.O = (int)w.size(1);
  a.K = (int)w.size(2);
  TORCH_CHECK(a.K % EX_STEP == 0 && a.xstride % 8 == 0);
  TORCH_CHECK(tile == 16 || tile == 128, "tiles hold 16 or 128 pairs");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 3);
  a.n_tiles = (int)tiles.size(0);
  TORCH_CHECK(tile == 128 || a.n_tiles <= 65535);
  aligned16(x, "x");
  aligned16(w, "w");
  if (tokens) a.tokens = ints(*tokens, pairs, "tokens");
  else TORCH_CHECK(x.size(0) >= pairs);
  TORCH_CHECK(act == EX_NONE || act == EX_RELU2 || act == EX_CLAMPED_GLU);
  a.act = (int)act;
  a.limit = (float)limit;
  a.alpha = (float)alpha;
  int outs = a.O;
  if (act == EX_CLAMPED_GLU) {
    // gate and up projection are padded to whole 16-row tiles each
    TORCH_CHECK(a.O % 32 == 0, "gated units come in tiles of 16");
    outs /= 2;
  }
  if (scale) {
    check_f32(*scale, "scale");
    TORCH_CHECK(scale->numel() >= pairs);
    a.scale = scale->data_ptr<float>();
  }
  a.ostride = (outs + 7) / 8 * 8;
  auto out = torch::empty({pairs, a.ostride}, x.options());
  a.x = x.data_ptr();
  a.w = w.data_ptr();
  a.out = out.data_ptr();
  a.tiles = ints(tiles, 0, "tiles");
  if (a.n_tiles) launch_expert_gemm(&a, (int)tile, f32, stream());
  return out;
}

// x [N, W] += weighted rows of d (or of h where the pair has none)
c10::optional<Tensor> expert_combine(Tensor x, Tensor h, Tensor d, Tensor where,
                                     Tensor weight, bool copy) {
  check_f32(x, "x");
  const bool f32 = is_f32(h, "h");
  check_like(d, h, "d");
  CombineArgs a = {};
  a.n = x.size(0);
  a.W = (int)x.size(1);
  a.hstride = rows2(h, "h");
  a.dstride = rows2(d, "d");
  TORCH_CHECK(h.size(0) == a.n && h.size(1) >= a.W && d.size(1) >= a.W &&
              a.hstride % 8 == 0 && a.dstride % 8 == 0);
  TORCH_CHECK(where.dim() == 2 && where.size(0) == a.n &&
              weight.sizes() == where.sizes());
  check_f32(weight, "weight");
  a.top = (int)where.size(1);
  for (const Tensor* t : {&x, &h, &d}) aligned16(*t, "operand");
  c10::optional<Tensor> out;
  if (copy) {
    out = torch::empty(x.sizes(), h.options());
    a.copy = out->data_ptr();
  }
  a.x = x.data_ptr<float>();
  a.h = h.data_ptr();
  a.d = d.data_ptr();
  a.where = ints(where, a.n * a.top, "where");
  a.weight = weight.data_ptr<float>();
  if (a.n) launch_expert_combine(&a, f32, stream());
  return out;
}

// gelu_tanh(x w^T) * e for a few rows of the fp32 residual; w packed for e's
// columns
Tensor token_gate(Tensor x, Tensor w, Tensor e) {
  check_f32(x, "x");
  const bool f32 = is_f32(w, "w");
  check_like(e, w, "e");
  TokenGateArgs a = {};
  a.n = (int)x.size(0);
  a.K = (int)x.size(1);
  a.O = (int)e.size(1);
  TORCH_CHECK(a.K % EX_STEP == 0 && w.dim() == 4 && w.is_contiguous() &&
              w.size(0) == (a.O + 15) / 16 && w.size(1) == a.K / 32 &&
              w.size(2) == 64 && w.size(3) == 8, "w not packed for x");
  aligned16(x, "x");
  aligned16(w, "w");
  a.estride = rows2(e, "e");
  TORCH_CHECK(e.size(0) == a.n);
  auto out = torch::empty({a.n, a.O}, w.options());
  a.x = x.data_ptr<float>();
  a.w = w.data_ptr();
  a.e = e.data_ptr();
  a.out = out.data_ptr();
  if (a.n) launch_token_gate(&a, f32, stream());
  return out;
}

}  // namespace

void bind_experts(pybind11::module_& m) {
  m.def("expert_route", &expert_route);
  m.def("expert_plan", &expert_plan);
  m.def("expert_gemm", &expert_gemm);
  m.def("expert_combine", &expert_combine);
  m.def("token_gate", &token_gate);
}
