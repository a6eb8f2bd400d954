// Python bindings of the causal convolutions and the selective scan.
#include "ragged_bindings.h"
#include "ragged_recurrent.h"

extern "C" {
void launch_conv_short(const ConvArgs*, bool, hipStream_t);
void launch_conv_long(const ConvArgs*, bool, hipStream_t);
int norm_conv_width();
void launch_norm_conv_short(const NormConvArgs*, bool, hipStream_t);
bool scan_has(int, int);
void launch_scan(const ScanArgs*, int, int, bool, bool, hipStream_t);
}

namespace {

using Maybe = c10::optional<Tensor>;

// weights [taps, C] and history [slots, taps - 1, C] of a convolution
int check_conv(const Tensor& w, const Tensor& hist, const Tensor& like, long C) {
  check_like(w, like, "w");
  check_like(hist, like, "history");
  TORCH_CHECK(w.dim() == 2 && w.is_contiguous() && w.size(1) == C,
              "w must be [taps, channels]");
  const long taps = w.size(0);
  TORCH_CHECK(taps >= 1 && taps <= RC_MAXTAPS, "convolutions have 1 to ",
              RC_MAXTAPS, " taps");
  TORCH_CHECK(hist.dim() == 3 && hist.is_contiguous() &&
                  hist.size(1) == taps - 1 && hist.size(2) == C,
              "history must be [slots, taps - 1, channels]");
  return (int)taps;
}

ConvArgs conv_args(const Tensor& h, const Tensor& w, const Maybe& bias,
                   const Tensor& hist, const Tensor& out, const Tensor& cu,
                   const Tensor& pos0, const Tensor& slots, int64_t n_req,
                   bool add, bool silu) {
  const bool f32 = is_f32(h, "h");
  ConvArgs a = {};
  a.hstride = rows2(h, "h");
  a.C = (int)h.size(1);
  a.taps = check_conv(w, hist, h, a.C);
  check_like(out, h, "out");
  TORCH_CHECK(out.dim() == 2 && out.is_contiguous() && out.size(1) >= a.C);
  a.Cp = (int)out.size(1);
  const int v = f32 ? 4 : 8;
  auto whole = [&](const Tensor& t, long stride) {
    return ((uintptr_t)t.data_ptr()) % 16 == 0 && stride % v == 0;
  };
  a.vec = whole(h, a.hstride) && whole(w, a.C) && whole(hist, a.C) &&
          whole(out, a.Cp) && a.C % v == 0;
  if (bias) {
    check_like(*bias, h, "bias");
    TORCH_CHECK(bias->numel() == a.C && bias->is_contiguous());
    a.vec = a.vec && whole(*bias, a.C);
    a.bias = bias->data_ptr();
  }
  a.h = h.data_ptr();
  a.w = w.data_ptr();
  a.hist = hist.data_ptr();
  a.out = out.data_ptr();
  a.cu = ints(cu, n_req + 1, "cu");
  a.pos0 = ints(pos0, n_req, "pos0");
  a.slots = ints(slots, n_req, "slots");
  a.add = add;
  a.silu = silu;
  return a;
}

// The first n_req requests, n_tok tokens.
void conv_short(Tensor h, Tensor w, Maybe bias, Tensor hist, Tensor out,
                Tensor cu, Tensor pos0, Tensor slots, int64_t n_req,
                int64_t n_tok, bool add, bool silu) {
  auto a = conv_args(h, w, bias, hist, out, cu, pos0, slots, n_req, add, silu);
  TORCH_CHECK(n_tok <= h.size(0) && n_tok <= out.size(0));
  a.n_short = (int)n_req;
  if (n_req) launch_conv_short(&a, is_f32(h, "h"), stream());
}

// The n_long requests after the first n_short; row 0 of h is token h_base.
void conv_long(Tensor h, Tensor w, Maybe bias, Tensor hist, Tensor out,
               Tensor cu, Tensor pos0, Tensor slots, Tensor tok_entry,
               Tensor chunks, int64_t n_short, int64_t n_long, int64_t tok_base,
               int64_t h_base, bool add, bool silu) {
  auto a = conv_args(h, w, bias, hist, out, cu, pos0, slots, n_short + n_long,
                     add, silu);
  TORCH_CHECK(h_base >= 0 && h_base <= tok_base &&
                  out.size(0) == h.size(0) + h_base,
              "rows of h must reach to the batch's end");
  TORCH_CHECK(chunks.dim() == 2 && chunks.size(1) == 2);
  a.tok_entry = ints(tok_entry, out.size(0), "tok_entry");
  a.chunks = ints(chunks, 0, "chunks");
  a.n_chunks = (int)chunks.size(0);
  a.n_short = (int)n_short;
  a.n_long = (int)n_long;
  a.h_base = (int)h_base;
  if (n_long && a.n_chunks) launch_conv_long(&a, is_f32(h, "h"), stream());
}

// Whether norm_conv_short has rows of W columns and this y.
bool norm_conv_fits(int64_t W, Maybe y) {
  return W % 4 == 0 && W <= norm_conv_width() &&
         (!y || (rows2(*y, "y") % 4 == 0 && ((uintptr_t)y->data_ptr()) % 16 == 0));
}

void norm_conv_short(Tensor x, Maybe y, Maybe w_post, Tensor g, double eps,
                     Tensor w, Tensor hist, Tensor out, Tensor cu, Tensor pos0,
                     Tensor slots, int64_t n_req, int64_t n_tok) {
  check_f32(x, "x");
  const bool f32 = is_f32(out, "out");
  TORCH_CHECK(x.dim() == 2);
  const long W = x.size(1);
  TORCH_CHECK(norm_conv_fits(W, y), "rows do not fit the kernel");
  NormConvArgs a = {};
  a.taps = check_conv(w, hist, out, W);
  TORCH_CHECK(out.dim() == 2 && out.is_contiguous() && out.size(1) >= W &&
              out.size(1) % 4 == 0 && n_tok <= x.size(0) &&
              n_tok <= out.size(0));
  for (const Tensor* t : {&x, &w, &hist, &out}) aligned16(*t, "operand");
  if (y) {
    check_like(*y, out, "y");
    TORCH_CHECK(y->sizes() == x.sizes());
    a.y = y->data_ptr();
    a.ystride = rows2(*y, "y");
    if (w_post) {
      check_like(*w_post, out, "w_post");
      TORCH_CHECK(w_post->numel() == W && w_post->is_contiguous());
      aligned16(*w_post, "w_post");
      a.w_post = w_post->data_ptr();
    }
  }
  check_like(g, out, "g");
  TORCH_CHECK(g.numel() == 1, "the norm's weight must be one number");
  a.x = x.data_ptr<float>();
  a.g = g.data_ptr();
  a.w = w.data_ptr();
  a.hist = hist.data_ptr();
  a.out = out.data_ptr();
  a.cu = ints(cu, n_req + 1, "cu");
  a.pos0 = ints(pos0, n_req, "pos0");
  a.slots = ints(slots, n_req, "slots");
  a.W = (int)W;
  a.Wp = (int)out.size(1);
  a.n_short = (int)n_req;
  a.eps = (float)eps;
  if (n_req) launch_norm_conv_short(&a, f32, stream());
}

ScanArgs scan_args(const Tensor& x, const Tensor& z, const Tensor& dt,
                   const Tensor& bias, const Tensor& bc, const Tensor& A,
                   const Tensor& D, const Tensor& state, const Tensor& out,
                   const Tensor& pos0, const Tensor& slots, int64_t n_req,
                   int64_t part, int64_t parts, int64_t b0, int64_t c0) {
  is_f32(x, "x");
  ScanArgs a = {};
  TORCH_CHECK(scan_has((int)part, (int)parts), "no scan of ", part, " x ",
              parts, " states");
  const long N = x.size(0), C = x.size(1), Np = part * parts;
  a.xs = rows2(x, "x");
  a.zs = rows2(z, "z");
  a.ds = rows2(dt, "dt");
  a.bs = rows2(bc, "bc");
  for (const Tensor* t : {&z, &dt, &bc, &out}) check_like(*t, x, "scan operand");
  TORCH_CHECK(z.sizes() == x.sizes() && dt.sizes() == x.sizes() &&
              bc.size(0) == N);
  TORCH_CHECK(b0 >= 0 && c0 >= 0 && b0 + Np <= bc.size(1) &&
              c0 + Np <= bc.size(1) && b0 % 8 == 0 && c0 % 8 == 0 &&
              a.bs % 8 == 0);
  aligned16(bc, "bc");
  check_f32(bias, "bias");
  check_f32(D, "D");
  check_f32(A, "A");
  check_f32(state, "state");
  TORCH_CHECK(bias.numel() == C && D.numel() == C && A.numel() == Np * C);
  TORCH_CHECK(state.dim() == 4 && state.size(1) == 1 && state.size(2) == Np &&
              state.size(3) == C);
  TORCH_CHECK(out.is_contiguous() && out.sizes() == x.sizes());
  a.x = x.data_ptr();
  a.z = z.data_ptr();
  a.dt = dt.data_ptr();
  a.bc = bc.data_ptr();
  a.bias = bias.data_ptr<float>();
  a.A = A.data_ptr<float>();
  a.D = D.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.out = out.data_ptr();
  a.pos0 = ints(pos0, n_req, "pos0");
  a.slots = ints(slots, n_req, "slots");
  a.C = (int)C;
  a.Np = (int)Np;
  a.b0 = (int)b0;
  a.c0 = (int)c0;
  return a;
}

void scan_short(Tensor x, Tensor z, Tensor dt, Tensor bias, Tensor bc, Tensor A,
                Tensor D, Tensor state, Tensor out, Tensor cu, Tensor pos0,
                Tensor slots, int64_t n_req, int64_t n_tok, int64_t part,
                int64_t parts, int64_t b0, int64_t c0) {
  auto a = scan_args(x, z, dt, bias, bc, A, D, state, out, pos0, slots, n_req,
                     part, parts, b0, c0);
  TORCH_CHECK(n_tok <= x.size(0) && n_req <= 65535);
  a.cu = ints(cu, n_req + 1, "cu");
  a.n_short = (int)n_req;
  if (n_req)
    launch_scan(&a, (int)part, (int)parts, true, is_f32(x, "x"), stream());
}

// spans [*, 4]: (first token, tokens, request, whether its portion ends)
void scan_long(Tensor x, Tensor z, Tensor dt, Tensor bias, Tensor bc, Tensor A,
               Tensor D, Tensor state, Tensor out, Tensor pos0, Tensor slots,
               Tensor spans, Tensor span_cu, int64_t n_short, int64_t n_long,
               int64_t part, int64_t parts, int64_t b0, int64_t c0) {
  auto a = scan_args(x, z, dt, bias, bc, A, D, state, out, pos0, slots,
                     n_short + n_long, part, parts, b0, c0);
  TORCH_CHECK(spans.dim() == 2 && spans.size(1) == 4 &&
              spans.size(0) <= 65535 && n_long <= 65535 && a.Np <= 65535);
  a.spans = ints(spans, 0, "spans");
  a.span_cu = ints(span_cu, n_long + 1, "span_cu");
  a.n_short = (int)n_short;
  a.n_long = (int)n_long;
  a.n_spans = (int)spans.size(0);
  if (a.n_spans == 0) return;
  Tensor ends, inits, sums;
  if (a.n_spans > n_long) {
    auto o = A.options();
    ends = torch::empty({a.n_spans, a.Np, a.C}, o);
    inits = torch::empty({a.n_spans, a.Np, a.C}, o);
    sums = torch::empty({a.n_spans, a.C}, o);
    a.ends = ends.data_ptr<float>();
    a.inits = inits.data_ptr<float>();
    a.sums = sums.data_ptr<float>();
  }
  launch_scan(&a, (int)part, (int)parts, false, is_f32(x, "x"), stream());
}

}  // namespace

void bind_recurrent(pybind11::module_& m) {
  m.def("conv_short", &conv_short);
  m.def("conv_long", &conv_long);
  m.def("norm_conv_fits", &norm_conv_fits);
  m.def("norm_conv_short", &norm_conv_short);
  m.def("scan_short", &scan_short);
  m.def("scan_long", &scan_long);
}
