// Python bindings of the ragged-batch kernels (extension _hip_ragged).
// Every operand's device, type, shape and alignment is checked here, before
// anything is launched.

#include "ragged_bindings.h"
#include "ragged_grouped.h"
#include "ragged_prefill.h"

struct AddNormArgs {
  float* x;
  const void *y, *y_bias, *w_post, *w_next;
  void* h;
  const int* where;
  long rows, ystride;
  int W, Wh, top;
  float eps, off, mult;
  bool one_next;
};

extern "C" {
void launch_clamped_glu(const void*, const void*, const void*, const void*,
                        void*, long, int, long, long, float, float, bool, bool,
                        hipStream_t);
void launch_glu_strided(const void*, const void*, void*, long, int, long, long,
                        bool, hipStream_t);
void launch_glu_any(const void*, const void*, void*, long, int, long, long,
                    bool, bool, hipStream_t);
void launch_add_norm(const AddNormArgs*, bool, hipStream_t);
void launch_latent_append(const void*, long, const void*, float, void*, void*,
                          long, int, int, int, int, int, int, int,
                          const float*, const float*, const int*, const int*,
                          const int*, int, long, bool, hipStream_t);
void launch_latent_gather(const void*, void*, const int*, int, int, bool,
                          hipStream_t);
void launch_latent_attn_short(const void*, const void*, const void*, void*,
                              float*, float*, const int*, const int*,
                              const int*, int, int, int, long, int, int, int,
                              int, float, int, int, int, bool, hipStream_t);
void launch_latent_attn_long_bf16(const LatentLongArgs*, int, int,
                                  hipStream_t);
void launch_latent_attn_long_f32(const LatentLongArgs*, int, int, hipStream_t);
int delta_short_rows(int, int, int);
void launch_grouped_append(const GroupedRowArgs*, void*, float*, const int*,
                           const int*, const int*, int, int, long, bool,
                           hipStream_t);
void launch_grouped_turn(const GroupedRowArgs*, void*, float*, const int*,
                         const int*, int, int, long, bool, bool, hipStream_t);
void launch_grouped_fill(const GroupedRowArgs*, const float*, const int*, int,
                         bool, hipStream_t);
void launch_grouped_attn_short_bf16(const GroupedAttnArgs*, int, int,
                                    hipStream_t);
void launch_grouped_attn_short_f32(const GroupedAttnArgs*, int, int,
                                   hipStream_t);
void launch_grouped_attn_long_bf16(const GroupedAttnArgs*, int, int,
                                   hipStream_t);
void launch_grouped_attn_long_f32(const GroupedAttnArgs*, int, int,
                                  hipStream_t);
void launch_gelu(const void*, void*, long, int, long, long, bool, bool,
                 hipStream_t);
void launch_cap_logits(const void*, float*, long, float, float, bool,
                       hipStream_t);
}

struct DeltaDims {
  int KH, H, D, V, taps;
  int qc, kc, vc, gc, ac, bc;
  long ystride, zstride;
  bool channels, sigmoid;
};

struct DeltaLongArgs {
  const void *y, *z, *conv_w, *A_log, *dt_bias, *norm_w;
  float* state;
  void *conv_state, *out;
  float *qn, *kn, *lg, *bt, *tm, *am, *ge, *o, *qg, *kg, *kl;
  void* vn;
  const int *cu, *pos0, *slots, *tok_entry, *chunks, *chunk_cu;
  int n_short, n_long, tok_base, n_chunks, Dp, Vp;
  long n_tok;
  float eps;
};

extern "C" {
void launch_delta_short(const void*, const void*, const void*, const void*,
                        const void*, const void*, float*, void*, void*, const int*,
                        const int*, const int*, const DeltaDims*, int, int,
                        float, bool, hipStream_t);
void launch_delta_long(const DeltaLongArgs*, const DeltaDims*, bool,
                       hipStream_t);
}

namespace {

Tensor glu(Tensor gate, Tensor up, bool gelu) {
  const bool f32 = is_f32(gate, "gate");
  check_like(up, gate, "up");
  TORCH_CHECK(gate.sizes() == up.sizes() && gate.dim() >= 1);
  const long I = gate.size(-1);
  auto g = gate.reshape({-1, I}), u = up.reshape({-1, I});
  if (g.stride(1) != 1) g = g.contiguous();
  if (u.stride(1) != 1) u = u.contiguous();
  auto y = torch::empty(gate.sizes(), gate.options());
  const long rows = g.size(0);
  if (rows == 0) return y;
  const long gs = rows2(g, "gate"), us = rows2(u, "up");
  const bool vec = !f32 && I % 4 == 0 && gs % 4 == 0 && us % 4 == 0 &&
                   ((uintptr_t)g.data_ptr()) % 8 == 0 &&
                   ((uintptr_t)u.data_ptr()) % 8 == 0;
  if (vec)
    launch_glu_strided(g.data_ptr(), u.data_ptr(), y.data_ptr(), rows, (int)I,
                       gs, us, gelu, stream());
  else
    launch_glu_any(g.data_ptr(), u.data_ptr(), y.data_ptr(), rows, (int)I, gs,
                   us, gelu, f32, stream());
  return y;
}

// gate and up [rows, C], possibly slices of wider rows; biases [C] or none
Tensor clamped_glu(Tensor gate, Tensor up, double limit, double alpha,
                   c10::optional<Tensor> gate_bias,
                   c10::optional<Tensor> up_bias) {
  const bool f32 = is_f32(gate, "gate");
  check_like(up, gate, "up");
  const long gs = rows2(gate, "gate"), us = rows2(up, "up");
  TORCH_CHECK(gate.sizes() == up.sizes());
  const long rows = gate.size(0), C = gate.size(1);
  auto out = torch::empty({rows, C}, gate.options());
  if (rows == 0 || C == 0) return out;
  bool vec = C % 8 == 0 && whole8(gate, gs) && whole8(up, us);
  auto bias = [&](const c10::optional<Tensor>& b) {
    if (!b) return (const void*)nullptr;
    check_like(*b, gate, "bias");
    TORCH_CHECK(b->numel() == C && b->is_contiguous());
    vec = vec && whole8(*b, 8);
    return (const void*)b->data_ptr();
  };
  const void *gb = bias(gate_bias), *ub = bias(up_bias);
  launch_clamped_glu(gate.data_ptr(), up.data_ptr(), gb, ub, out.data_ptr(),
                     rows, (int)C, gs, us, (float)limit, (float)alpha, vec, f32,
                     stream());
  return out;
}

// x [N, W] fp32 (updated in place when y is given, normed first when w_post
// is; where [N, top]: sums of rows of y; y_bias [W] added to y); returns h, `wide` columns of the next
// norm's rows or of x itself, or an empty tensor for wide == 0.
Tensor add_norm(Tensor x, c10::optional<Tensor> y, c10::optional<Tensor> w_post,
                c10::optional<Tensor> w_next, bool f32, double eps,
                double off, double mult, c10::optional<Tensor> where,
                int64_t wide, c10::optional<Tensor> y_bias) {
  check_f32(x, "x");
  TORCH_CHECK(x.dim() == 2, "x must be [rows, width]");
  const auto type = x.options().dtype(f32 ? torch::kFloat32 : torch::kBFloat16);
  auto h = torch::empty({wide ? x.size(0) : 0, wide}, type);
  AddNormArgs a = {};
  a.rows = x.size(0);
  a.W = (int)x.size(1);
  a.Wh = (int)wide;
  a.ystride = a.W;
  TORCH_CHECK(wide == 0 || wide >= a.W);
  if (y) {
    check_like(*y, h, "y");
    a.ystride = rows2(*y, "y");
    if (where) {
      TORCH_CHECK(where->dim() == 2 && where->size(0) == a.rows &&
                  y->size(1) >= a.W && y->size(0) == where->numel(),
                  "rows of y do not fit x");
      a.where = ints(*where, where->numel(), "where");
      a.top = (int)where->size(1);
    } else {
      TORCH_CHECK(y->sizes() == x.sizes(), "y must match x");
    }
    a.y = y->data_ptr();
    if (y_bias) {
      check_like(*y_bias, h, "y_bias");
      TORCH_CHECK(y_bias->numel() == a.W && y_bias->is_contiguous());
      a.y_bias = y_bias->data_ptr();
    }
    if (w_post) {
      check_like(*w_post, h, "w_post");
      TORCH_CHECK(w_post->numel() == a.W && w_post->is_contiguous());
      a.w_post = w_post->data_ptr();
    }
  }
  if (w_next) {
    check_like(*w_next, h, "w_next");
    TORCH_CHECK((w_next->numel() == a.W || w_next->numel() == 1) &&
                w_next->is_contiguous());
    a.w_next = w_next->data_ptr();
    a.one_next = w_next->numel() == 1;
  }
  if (a.rows == 0) return h;
  a.x = x.data_ptr<float>();
  a.h = wide ? h.data_ptr() : nullptr;
  a.eps = (float)eps;
  a.off = (float)off;
  a.mult = (float)mult;
  launch_add_norm(&a, f32, stream());
  return h;
}

// q [N, >= H * dq], rotated in place at qoff of every head; dkv [N, rank+rot]
// (optional) normed, rotated and written to its page rows.
void latent_append(c10::optional<Tensor> dkv, c10::optional<Tensor> norm_w,
                   double eps, Tensor pool, Tensor q, int64_t H, int64_t dq,
                   int64_t qoff, int64_t rank, int64_t rankp, int64_t rot,
                   int64_t rotp, Tensor cos, Tensor sin, Tensor tok_pos,
                   Tensor tok_entry, Tensor pages) {
  const bool f32 = is_f32(q, "q");
  const long N = q.size(0);
  const long qs = rows2(q, "q");
  TORCH_CHECK(q.size(1) >= H * dq && qoff >= 0 && qoff + rot <= dq);
  check_like(pool, q, "pool");
  TORCH_CHECK(pool.is_contiguous() && pool.dim() == 2 &&
              pool.size(1) == rankp + rotp);
  check_f32(cos, "cos");
  check_f32(sin, "sin");
  TORCH_CHECK(rot % 2 == 0 && cos.size(1) == rot / 2 &&
              sin.sizes() == cos.sizes());
  TORCH_CHECK(rank <= rankp && rot <= rotp && rotp % 2 == 0);
  TORCH_CHECK(pages.dim() == 2);
  long ds = 0;
  if (dkv) {
    check_like(*dkv, q, "dkv");
    ds = rows2(*dkv, "dkv");
    TORCH_CHECK(dkv->size(0) == N && dkv->size(1) >= rank + rot && norm_w);
    check_like(*norm_w, q, "norm_w");
    TORCH_CHECK(norm_w->numel() == rank && norm_w->is_contiguous());
  }
  if (N == 0) return;
  launch_latent_append(
      dkv ? dkv->data_ptr() : nullptr, ds, dkv ? norm_w->data_ptr() : nullptr,
      (float)eps, pool.data_ptr(), q.data_ptr(), qs, (int)H, (int)dq,
      (int)qoff, (int)rank, (int)rankp, (int)rot, (int)rotp,
      cos.data_ptr<float>(), sin.data_ptr<float>(), ints(tok_pos, N, "tok_pos"),
      ints(tok_entry, N, "tok_entry"), ints(pages, 0, "pages"),
      (int)pages.size(1), N, f32, stream());
}

Tensor latent_gather(Tensor pool, Tensor blocks, int64_t rows) {
  const bool f32 = is_f32(pool, "pool");
  TORCH_CHECK(pool.is_contiguous() && pool.dim() == 2 &&
              pool.size(1) % 8 == 0 && pool.size(0) % RG_PAGE == 0);
  TORCH_CHECK(blocks.dim() == 2 && blocks.size(1) == 3 &&
              rows == blocks.size(0) * RG_PAGE);
  auto out = torch::empty({rows, pool.size(1)}, pool.options());
  if (rows)
    launch_latent_gather(pool.data_ptr(), out.data_ptr(),
                         ints(blocks, 0, "blocks"), (int)blocks.size(0),
                         (int)pool.size(1), f32, stream());
  return out;
}

// q_abs [H, Nt, rankp], q [N, >= H*dq] (rotated) -> [H, Nt, rankp]
Tensor latent_attn_short(Tensor q_abs, Tensor q, Tensor pool, Tensor cu,
                         Tensor pos0, Tensor pages, int64_t n_req,
                         int64_t max_len, int64_t max_keys, int64_t dq,
                         int64_t qoff, int64_t rotp, double scale) {
  const bool f32 = is_f32(q_abs, "q_abs");
  check_like(q, q_abs, "q");
  check_like(pool, q_abs, "pool");
  TORCH_CHECK(q_abs.dim() == 3 && q_abs.is_contiguous());
  const long H = q_abs.size(0), Nt = q_abs.size(1), rankp = q_abs.size(2);
  TORCH_CHECK(rankp % 64 == 0 && rankp <= 1024 && rotp % 32 == 0);
  const long nd = rankp / 64;
  TORCH_CHECK(nd == 1 || nd == 2 || nd == 4 || nd == 8 || nd == 16,
              "latent width must be padded to 64 * 2^k");
  TORCH_CHECK(pool.is_contiguous() && pool.size(1) == rankp + rotp);
  const long qs = rows2(q, "q");
  TORCH_CHECK(q.size(0) >= Nt && q.size(1) >= H * dq && qoff + rotp <= dq &&
              qs % 8 == 0 && dq % 8 == 0 && qoff % 8 == 0);
  aligned16(q, "q");
  aligned16(q_abs, "q_abs");
  TORCH_CHECK(pages.dim() == 2 && pages.size(0) >= n_req);
  auto out = torch::empty_like(q_abs);
  if (Nt == 0 || n_req == 0) return out;
  const long tiles = (max_len * H + 15) / 16;
  // enough blocks for the chip, at least two key tiles per slice
  long nsplit = std::max<long>(1, 1024 / std::max<long>(1, n_req * tiles));
  nsplit = std::min<long>(nsplit, std::max<long>(1, max_keys / 64));
  nsplit = std::min<long>(nsplit, 64);
  Tensor po, ml;
  if (nsplit > 1) {
    auto o = q_abs.options().dtype(torch::kFloat32);
    po = torch::empty({H, Nt, nsplit, rankp}, o);
    ml = torch::empty({H, Nt, nsplit, 2}, o);
  }
  launch_latent_attn_short(
      q_abs.data_ptr(), q.data_ptr(), pool.data_ptr(), out.data_ptr(),
      nsplit > 1 ? po.data_ptr<float>() : nullptr,
      nsplit > 1 ? ml.data_ptr<float>() : nullptr, ints(cu, n_req + 1, "cu"),
      ints(pos0, n_req, "pos0"), ints(pages, 0, "pages"), (int)pages.size(1),
      (int)H, (int)Nt, qs, (int)dq, (int)qoff, (int)rankp, (int)rotp,
      (float)scale, (int)n_req, (int)nsplit, (int)tiles, f32, stream());
  return out;
}

// q [N, >= H*dq] (rotated), kx [St, H*dimp], lat [St, rankp+rotp],
// vt [H*vdp, St] -> [N - tok_base, H*vdp]
Tensor latent_attn_long(Tensor q, Tensor kx, Tensor lat, Tensor vt,
                        Tensor tiles, Tensor cu, Tensor pos0, Tensor cuk,
                        int64_t n_short, int64_t tok_base, int64_t H,
                        int64_t dimp, int64_t rotp, double scale) {
  const bool f32 = is_f32(q, "q");
  check_like(kx, q, "kx");
  check_like(lat, q, "lat");
  check_like(vt, q, "vt");
  const long dq = dimp + rotp;
  const long St = lat.size(0);
  const long vdp = vt.size(0) / H;
  TORCH_CHECK(kx.is_contiguous() && kx.size(0) == St && kx.size(1) == H * dimp);
  TORCH_CHECK(lat.is_contiguous() && lat.dim() == 2 && lat.size(1) > rotp);
  TORCH_CHECK(vt.is_contiguous() && vt.size(1) == St && vt.size(0) == H * vdp);
  TORCH_CHECK(St % LP_KT == 0 && dimp % 32 == 0 && rotp % 32 == 0);
  const long qs = rows2(q, "q");
  TORCH_CHECK(q.size(1) >= H * dq && qs % 8 == 0);
  aligned16(q, "q");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2);
  const int step = f32 ? 4 : 2;
  const int nks = (int)((dq / 32 + step - 1) / step) * step;
  const int ndh = (int)(vdp / 16);
  const bool ok_k = nks <= 8;
  const bool ok_v = f32 ? (ndh == 4 || ndh == 16)
                        : (ndh == 2 || ndh == 4 || ndh == 8 || ndh == 16);
  TORCH_CHECK(ok_k && ok_v && vdp % 16 == 0, "unsupported head shape ", dq,
              "/", vdp);
  auto out = torch::empty({q.size(0) - tok_base, H * vdp}, q.options());
  LatentLongArgs a;
  a.q = q.data_ptr();
  a.kx = kx.data_ptr();
  a.lat = lat.data_ptr();
  a.vt = vt.data_ptr();
  a.out = out.data_ptr();
  a.tiles = ints(tiles, 0, "tiles");
  a.cu = ints(cu, n_short + 2, "cu");
  a.pos0 = ints(pos0, n_short + 1, "pos0");
  a.cuk = ints(cuk, 2, "cuk");
  a.n_short = (int)n_short;
  a.tok_base = (int)tok_base;
  a.n_tiles = (int)tiles.size(0);
  a.H = (int)H;
  a.dq = (int)dq;
  a.dimp = (int)dimp;
  a.rankp = (int)(lat.size(1) - rotp);
  a.W = (int)lat.size(1);
  a.St = St;
  a.qstride = qs;
  a.scale = (float)scale;
  if (a.n_tiles == 0) return out;
  if (f32)
    launch_latent_attn_long_f32(&a, nks, ndh, stream());
  else
    launch_latent_attn_long_bf16(&a, nks, ndh, stream());
  return out;
}

// y [N, *] has q, k, v and beta; gate and decay are columns of y as well (one
// decay per head), or of z (one per head and key channel)
DeltaDims delta_dims(const Tensor& y, const c10::optional<Tensor>& z,
                     const Tensor& conv_w, int64_t KH, int64_t H, int64_t D,
                     int64_t V, const std::vector<int64_t>& cols,
                     bool sigmoid) {
  DeltaDims d;
  TORCH_CHECK(KH > 0 && H % KH == 0 && cols.size() == 6);
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.is_contiguous() &&
              conv_w.size(0) == 2 * KH * D + H * V);
  d.KH = (int)KH;
  d.H = (int)H;
  d.D = (int)D;
  d.V = (int)V;
  d.taps = (int)conv_w.size(1);
  TORCH_CHECK(d.taps >= 1 && d.taps <= 8, "convolutions have 1 to 8 taps");
  TORCH_CHECK(D <= 512 && V <= 512 && delta_short_rows((int)D, (int)V, 512) > 0,
              "state of a head is too large: ", D, " x ", V);
  d.channels = z.has_value();
  d.sigmoid = sigmoid;
  const int64_t w[6] = {KH * D, KH * D, H * V, H * V, d.channels ? H * D : H, H};
  for (int i = 0; i < 6; ++i) {
    const Tensor& rows = d.channels && (i == 3 || i == 4) ? *z : y;
    TORCH_CHECK(cols[i] >= 0 && cols[i] + w[i] <= rows.size(1));
  }
  d.qc = (int)cols[0];
  d.kc = (int)cols[1];
  d.vc = (int)cols[2];
  d.gc = (int)cols[3];
  d.ac = (int)cols[4];
  d.bc = (int)cols[5];
  d.ystride = d.zstride = rows2(y, "y");
  if (z) {
    check_like(*z, y, "z");
    TORCH_CHECK(z->size(0) == y.size(0));
    d.zstride = rows2(*z, "z");
  }
  return d;
}

void check_delta(const Tensor& y, const Tensor& conv_w, const Tensor& A_log,
                 const Tensor& dt, const Tensor& norm_w, const Tensor& state,
                 const Tensor& conv_state, const Tensor& out,
                 const DeltaDims& d) {
  for (const auto* t : {&conv_w, &A_log, &dt, &norm_w, &conv_state, &out})
    check_like(*t, y, "delta operand");
  TORCH_CHECK(A_log.numel() == d.H &&
              dt.numel() == (d.channels ? (long)d.H * d.D : d.H) &&
              norm_w.numel() == d.V && A_log.is_contiguous() &&
              dt.is_contiguous() && norm_w.is_contiguous());
  check_f32(state, "state");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == d.H &&
              state.size(2) == d.D && state.size(3) == d.V);
  TORCH_CHECK(conv_state.is_contiguous() && conv_state.dim() == 3 &&
              conv_state.size(0) == state.size(0) &&
              conv_state.size(1) == conv_w.size(0) &&
              conv_state.size(2) == d.taps - 1);
  TORCH_CHECK(out.is_contiguous() && out.size(0) == y.size(0) &&
              out.size(1) == (long)d.H * d.V);
}

// Short portions of y's batch; rows of out that belong to them are written.
void delta_short(Tensor y, Tensor conv_w, Tensor A_log, Tensor dt,
                 Tensor norm_w, Tensor state, Tensor conv_state, Tensor out,
                 Tensor cu, Tensor pos0, Tensor slots, int64_t n_req,
                 int64_t max_len, int64_t KH, int64_t H, int64_t D, int64_t V,
                 std::vector<int64_t> cols, double eps, c10::optional<Tensor> z,
                 bool sigmoid) {
  const bool f32 = is_f32(y, "y");
  auto d = delta_dims(y, z, conv_w, KH, H, D, V, cols, sigmoid);
  check_delta(y, conv_w, A_log, dt, norm_w, state, conv_state, out, d);
  TORCH_CHECK(max_len >= 1 && max_len <= 16, "short portions have 1 to 16 "
              "tokens");
  if (n_req == 0) return;
  launch_delta_short(y.data_ptr(), z ? z->data_ptr() : y.data_ptr(),
                     conv_w.data_ptr(), A_log.data_ptr(),
                     dt.data_ptr(), norm_w.data_ptr(), state.data_ptr<float>(),
                     conv_state.data_ptr(), out.data_ptr(),
                     ints(cu, n_req + 1, "cu"), ints(pos0, n_req, "pos0"),
                     ints(slots, n_req, "slots"), &d, (int)n_req, (int)max_len,
                     (float)eps, f32, stream());
}

// Long portions: requests n_short.. of the batch, tokens tok_base..
void delta_long(Tensor y, Tensor conv_w, Tensor A_log, Tensor dt,
                Tensor norm_w, Tensor state, Tensor conv_state, Tensor out,
                Tensor cu, Tensor pos0, Tensor slots, Tensor tok_entry,
                Tensor chunks, Tensor chunk_cu, int64_t n_short,
                int64_t n_long, int64_t tok_base, int64_t KH, int64_t H,
                int64_t D, int64_t V, std::vector<int64_t> cols, double eps,
                c10::optional<Tensor> z, bool sigmoid) {
  const bool f32 = is_f32(y, "y");
  auto d = delta_dims(y, z, conv_w, KH, H, D, V, cols, sigmoid);
  check_delta(y, conv_w, A_log, dt, norm_w, state, conv_state, out, d);
  const long n = y.size(0) - tok_base;
  if (n <= 0 || n_long == 0) return;
  TORCH_CHECK(chunks.dim() == 2 && chunks.size(1) == 2);
  TORCH_CHECK(n * H < (1L << 31), "too many tokens in one step");
  for (const Tensor* t : {&y, &norm_w, z ? &*z : &y})
    TORCH_CHECK(((uintptr_t)t->data_ptr()) % 8 == 0, "unaligned operand");
  const long nc = chunks.size(0);
  // depths 16 * 2^k take the walk with a fixed depth
  long Dp = 16;
  while (Dp < D) Dp *= 2;
  if (Dp > 128) Dp = (D + 15) / 16 * 16;
  const long Vp = (V + 15) / 16 * 16;
  auto fo = y.options().dtype(torch::kFloat32);
  auto qn = torch::empty({n, KH, Dp}, fo), kn = torch::empty({n, KH, Dp}, fo);
  auto vn = torch::empty({n, H, Vp}, y.options());
  auto bt = torch::empty({n, H}, fo);
  auto tm = torch::empty({nc, H, 64, 64}, fo);
  auto am = torch::empty({nc, H, 64, 64}, fo);
  auto o = torch::empty({n, H, Vp}, fo);
  DeltaLongArgs a = {};
  Tensor lg, ge, qg, kg, kl;
  if (d.channels) {
    qg = torch::empty({n, H, Dp}, fo);
    kg = torch::empty({n, H, Dp}, fo);
    kl = torch::empty({n, H, Dp}, fo);
    ge = torch::empty({nc, H, Dp}, fo);
    a.qg = qg.data_ptr<float>();
    a.kg = kg.data_ptr<float>();
    a.kl = kl.data_ptr<float>();
  } else {
    lg = torch::empty({n, H}, fo);
    ge = torch::empty({nc, H, 2, 64}, fo);
    a.lg = lg.data_ptr<float>();
  }
  a.y = y.data_ptr();
  a.z = z ? z->data_ptr() : y.data_ptr();
  a.conv_w = conv_w.data_ptr();
  a.A_log = A_log.data_ptr();
  a.dt_bias = dt.data_ptr();
  a.norm_w = norm_w.data_ptr();
  a.state = state.data_ptr<float>();
  a.conv_state = conv_state.data_ptr();
  a.out = out.data_ptr();
  a.qn = qn.data_ptr<float>();
  a.kn = kn.data_ptr<float>();
  a.bt = bt.data_ptr<float>();
  a.tm = tm.data_ptr<float>();
  a.am = am.data_ptr<float>();
  a.ge = ge.data_ptr<float>();
  a.o = o.data_ptr<float>();
  a.vn = vn.data_ptr();
  a.cu = ints(cu, n_short + n_long + 1, "cu");
  a.pos0 = ints(pos0, n_short + n_long, "pos0");
  a.slots = ints(slots, n_short + n_long, "slots");
  a.tok_entry = ints(tok_entry, y.size(0), "tok_entry");
  a.chunks = ints(chunks, 0, "chunks");
  a.chunk_cu = ints(chunk_cu, n_long + 1, "chunk_cu");
  a.n_short = (int)n_short;
  a.n_long = (int)n_long;
  a.tok_base = (int)tok_base;
  a.n_chunks = (int)nc;
  a.Dp = (int)Dp;
  a.Vp = (int)Vp;
  a.n_tok = n;
  a.eps = (float)eps;
  launch_delta_long(&a, &d, f32, stream());
}

// ---------------------------------------------------------------------------
// Grouped attention
// ---------------------------------------------------------------------------

void check_pool(const Tensor& pool, const Tensor& like, long width) {
  check_like(pool, like, "pool");
  TORCH_CHECK(pool.is_contiguous() && pool.dim() == 2 &&
                  pool.size(1) == width && pool.size(0) % RG_PAGE == 0,
              "pool must be pages of ", width, " elements per token");
  aligned16(pool, "pool");
}

GroupedRowArgs grouped_rows(const Tensor& y, const c10::optional<Tensor>& wq,
                            const c10::optional<Tensor>& wk, double eps,
                            const c10::optional<Tensor>& vmix,
                            const c10::optional<Tensor>& first,
                            const Tensor& pool, int64_t H, int64_t G, int64_t D,
                            int64_t V, int64_t dimp, int64_t vdp,
                            bool own = true, bool by_head = false) {
  TORCH_CHECK(G > 0 && H > 0 && H % G == 0 && D > 0 && V > 0);
  TORCH_CHECK(dimp % 32 == 0 && D <= dimp && vdp % 16 == 0 && V <= vdp &&
              dimp <= 512 && vdp <= 512);
  GroupedRowArgs a = {};
  a.ystride = rows2(y, "y");
  TORCH_CHECK(y.size(1) >= (own ? (H + G) * D + G * V : H * D));
  check_pool(pool, y, G * (dimp + vdp));
  a.vec = D % 8 == 0 && V % 8 == 0 && whole8(y, a.ystride);
  auto weight = [&](const c10::optional<Tensor>& w, long n, const char* name) {
    if (!w) return (const void*)nullptr;
    check_like(*w, y, name);
    TORCH_CHECK(w->numel() == n && w->is_contiguous());
    a.vec = a.vec && whole8(*w, 8);
    return (const void*)w->data_ptr();
  };
  a.wq = weight(wq, by_head ? D : H * D, "wq");
  a.wk = weight(wk, by_head ? D : G * D, "wk");
  if (first) {
    TORCH_CHECK(vmix && vmix->numel() == 1);
    check_like(*vmix, y, "vmix");
    check_like(*first, y, "first");
    a.fstride = rows2(*first, "first");
    TORCH_CHECK(first->size(0) == y.size(0) && first->size(1) == G * V);
    a.vec = a.vec && whole8(*first, a.fstride);
    a.vmix = vmix->data_ptr();
    a.first = first->data_ptr();
  }
  a.y = y.data_ptr();
  a.pool = pool.data_ptr();
  a.H = (int)H;
  a.G = (int)G;
  a.D = (int)D;
  a.V = (int)V;
  a.dimp = (int)dimp;
  a.vdp = (int)vdp;
  a.eps = (float)eps;
  return a;
}

// y [N, q | k | v | ...] -> queries [N, H, dimp] and the keys' inverse rms [N]
std::tuple<Tensor, Tensor> grouped_append(
    Tensor y, c10::optional<Tensor> wq, c10::optional<Tensor> wk, double eps,
    c10::optional<Tensor> vmix, c10::optional<Tensor> first, Tensor pool,
    int64_t H, int64_t G, int64_t D, int64_t V, int64_t dimp, int64_t vdp,
    Tensor tok_pos, Tensor tok_entry, Tensor pages, int64_t direct) {
  const bool f32 = is_f32(y, "y");
  auto a = grouped_rows(y, wq, wk, eps, vmix, first, pool, H, G, D, V, dimp,
                        vdp);
  const long N = y.size(0);
  TORCH_CHECK(pages.dim() == 2 && direct >= 0 && direct <= N);
  auto q = torch::empty({N, H, dimp}, y.options());
  auto kinv = torch::empty({N}, y.options().dtype(torch::kFloat32));
  if (N)
    launch_grouped_append(&a, q.data_ptr(), kinv.data_ptr<float>(),
                          ints(tok_pos, N, "tok_pos"),
                          ints(tok_entry, N, "tok_entry"),
                          ints(pages, 0, "pages"), (int)pages.size(1),
                          (int)direct, N, f32, stream());
  return {q, kinv};
}

using Table = c10::optional<Tensor>;

// rotation tables [positions, pairs] for the first 2 * pairs of `size` columns
void turn_tables(const Table& cos, const Table& sin, long size, const float** c,
                 const float** s, int* pairs) {
  TORCH_CHECK(cos.has_value() == sin.has_value());
  if (!cos) return;
  check_f32(*cos, "cos");
  check_f32(*sin, "sin");
  TORCH_CHECK(cos->dim() == 2 && cos->sizes() == sin->sizes() &&
              2 * cos->size(1) <= size, "rotation tables do not fit");
  *c = cos->data_ptr<float>();
  *s = sin->data_ptr<float>();
  *pairs = (int)cos->size(1);
}

void grouped_turns(GroupedRowArgs& a, bool head_norm, const Table& qk_cos,
                   const Table& qk_sin, const Table& v_cos, const Table& v_sin,
                   const Tensor& tok_pos, long n) {
  a.head_norm = head_norm;
  turn_tables(qk_cos, qk_sin, a.D, &a.qk_cos, &a.qk_sin, &a.qk_pairs);
  turn_tables(v_cos, v_sin, a.V, &a.v_cos, &a.v_sin, &a.v_pairs);
  a.tok_pos = ints(tok_pos, n, "tok_pos");
  for (const auto* t : {&qk_cos, &qk_sin, &v_cos, &v_sin})
    if (*t) aligned16(**t, "rotation table");
}

// y [N, q | k | v | ...] -> queries [N, H, dimp] and inverse rms of keys [N, G];
// wq, wk [D] weights of the norms per head; not own: y [N, q | ...], the queries
// alone
std::tuple<Tensor, Tensor> grouped_turn(
    Tensor y, c10::optional<Tensor> wq, c10::optional<Tensor> wk, double eps,
    bool head_norm, Table qk_cos, Table qk_sin, Table v_cos, Table v_sin,
    Tensor pool, int64_t H, int64_t G, int64_t D, int64_t V, int64_t dimp,
    int64_t vdp, Tensor tok_pos, Tensor tok_entry, Tensor pages, int64_t direct,
    bool own) {
  const bool f32 = is_f32(y, "y");
  const c10::optional<Tensor> none;
  TORCH_CHECK(head_norm || !(wq || wk), "weights without norms per head");
  auto a = grouped_rows(y, wq, wk, eps, none, none, pool, H, G, D, V, dimp, vdp,
                        own, true);
  const long N = y.size(0);
  TORCH_CHECK(pages.dim() == 2 && direct >= 0 && direct <= N);
  grouped_turns(a, head_norm, qk_cos, qk_sin, v_cos, v_sin, tok_pos, N);
  auto q = torch::empty({N, H, dimp}, y.options());
  auto kinv = torch::empty({N, G}, y.options().dtype(torch::kFloat32));
  if (N)
    launch_grouped_turn(&a, q.data_ptr(), kinv.data_ptr<float>(),
                        ints(tok_entry, N, "tok_entry"),
                        ints(pages, 0, "pages"), (int)pages.size(1),
                        (int)direct, N, own, f32, stream());
  return {q, kinv};
}

// fills [*, 4]: (page, token of its first slot, first slot, end slot)
void grouped_fill(Tensor y, c10::optional<Tensor> wk, Tensor kinv,
                  c10::optional<Tensor> vmix, c10::optional<Tensor> first,
                  Tensor pool, int64_t H, int64_t G, int64_t D, int64_t V,
                  int64_t dimp, int64_t vdp, Tensor fills, bool head_norm,
                  Table qk_cos, Table qk_sin, Table v_cos, Table v_sin,
                  Tensor tok_pos) {
  const bool f32 = is_f32(y, "y");
  const bool turns = head_norm || qk_cos || v_cos;
  auto a = grouped_rows(y, c10::nullopt, wk, 0.0, vmix, first, pool, H, G, D, V,
                        dimp, vdp, true, turns);
  check_f32(kinv, "kinv");
  grouped_turns(a, head_norm, qk_cos, qk_sin, v_cos, v_sin, tok_pos, y.size(0));
  TORCH_CHECK(kinv.numel() == y.size(0) * (turns ? G : 1) && G <= 65535);
  TORCH_CHECK(!(turns && first) && !(turns && !head_norm && wk),
              "norms per head or rotations beside norms of whole rows or "
              "blended values");
  TORCH_CHECK(fills.dim() == 2 && fills.size(1) == 4);
  if (fills.size(0))
    launch_grouped_fill(&a, kinv.data_ptr<float>(), ints(fills, 0, "fills"),
                        (int)fills.size(0), f32, stream());
}

int head_bucket(long n) { return n <= 64 ? 64 : n <= 128 ? 128 : n <= 256 ? 256 : 512; }

GroupedAttnArgs grouped_attn(const Tensor& q, const c10::optional<Tensor>& sink,
                             const Tensor& pool, const Tensor& out,
                             const Tensor& pages, int64_t G, int64_t V,
                             int64_t vdp, double scale, int64_t window,
                             const Table& v_cos, const Table& v_sin,
                             const Table& tok_pos, const Table& gate) {
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous());
  const long H = q.size(1), dimp = q.size(2);
  TORCH_CHECK(G > 0 && H % G == 0 && V > 0 && V <= vdp);
  TORCH_CHECK(dimp % 32 == 0 && vdp % 16 == 0 && dimp <= 512 && vdp <= 512);
  check_pool(pool, q, G * (dimp + vdp));
  check_like(out, q, "out");
  aligned16(q, "q");
  GroupedAttnArgs a = {};
  a.ostride = rows2(out, "out");
  TORCH_CHECK(out.size(0) == q.size(0) && out.size(1) == H * V);
  a.vec = V % 4 == 0 && a.ostride % 4 == 0 &&
          ((uintptr_t)out.data_ptr()) % 16 == 0;
  if (sink) {
    check_like(*sink, q, "sink");
    TORCH_CHECK(sink->numel() == H && sink->is_contiguous());
    a.sink = sink->data_ptr();
  }
  TORCH_CHECK(pages.dim() == 2);
  a.q = q.data_ptr();
  a.pool = pool.data_ptr();
  a.out = out.data_ptr();
  a.pages = ints(pages, 0, "pages");
  a.P = (int)pages.size(1);
  a.H = (int)H;
  a.G = (int)G;
  a.dimp = (int)dimp;
  a.V = (int)V;
  a.vdp = (int)vdp;
  a.scale = (float)scale;
  TORCH_CHECK(window >= 0 && window < (1L << 30));
  a.window = (int)window;
  int pairs = 0;
  turn_tables(v_cos, v_sin, V, &a.v_cos, &a.v_sin, &pairs);
  TORCH_CHECK(!v_cos || 2 * pairs == V, "values are turned back whole");
  TORCH_CHECK(!v_cos || tok_pos, "turning back needs positions");
  if (tok_pos) a.tok_pos = ints(*tok_pos, q.size(0), "tok_pos");
  if (gate) {
    check_like(*gate, q, "gate");
    a.gstride = rows2(*gate, "gate");
    TORCH_CHECK(gate->size(0) == q.size(0) && gate->size(1) == H);
    a.gate = gate->data_ptr();
  }
  return a;
}

// The first n_req requests of the batch, n_tok tokens; q [N, H, dimp], out [N, H * V].
void grouped_attn_short(Tensor q, c10::optional<Tensor> sink, Tensor pool,
                        Tensor out, Tensor cu, Tensor pos0, Tensor pages,
                        int64_t n_req, int64_t n_tok, int64_t max_len,
                        int64_t max_keys, int64_t G, int64_t V, int64_t vdp,
                        double scale, int64_t window, Table v_cos, Table v_sin,
                        Table tok_pos, Table gate) {
  const bool f32 = is_f32(q, "q");
  auto a = grouped_attn(q, sink, pool, out, pages, G, V, vdp, scale, window,
                        v_cos, v_sin, tok_pos, gate);
  // a block starts at the step that holds its first window's first key
  if (window) max_keys = std::min(max_keys, window + max_len + GA_STEP);
  TORCH_CHECK(pages.size(0) >= n_req && n_tok <= q.size(0));
  if (n_req == 0 || n_tok == 0) return;
  a.cu = ints(cu, n_req + 1, "cu");
  a.pos0 = ints(pos0, n_req, "pos0");
  a.n_req = (int)n_req;
  const long tiles = (max_len * (a.H / a.G) + 15) / 16;
  TORCH_CHECK(tiles <= 65535, "portion too long");
  a.row_tiles = (int)tiles;
  // enough blocks for the chip, at least one step of keys per wave
  long nsplit = std::max<long>(1, 1024 / (n_req * G * tiles));
  nsplit = std::min<long>(nsplit, std::max<long>(1, max_keys / 128));
  nsplit = std::min<long>(nsplit, GA_MAXSPLIT);
  a.nsplit = (int)nsplit;
  a.n_rows = n_tok * a.H;
  Tensor po, ml;
  if (nsplit > 1) {
    auto o = q.options().dtype(torch::kFloat32);
    po = torch::empty({a.n_rows, nsplit, vdp}, o);
    ml = torch::empty({a.n_rows, nsplit, 2}, o);
    a.part_o = po.data_ptr<float>();
    a.part_ml = ml.data_ptr<float>();
  }
  const int kb = head_bucket(a.dimp), vb = head_bucket(vdp);
  const bool big = kb == 512 || vb == 512;
  (f32 ? launch_grouped_attn_short_f32 : launch_grouped_attn_short_bf16)(
      &a, big ? 512 : kb, big ? 512 : vb, stream());
}

// The portions that tiles [*, 2] names: (request, first query).
void grouped_attn_long(Tensor q, c10::optional<Tensor> sink, Tensor pool,
                       Tensor out, Tensor tiles, Tensor cu, Tensor pos0,
                       Tensor pages, int64_t G, int64_t V, int64_t vdp,
                       double scale, int64_t window, Table v_cos, Table v_sin,
                       Table tok_pos, Table gate) {
  const bool f32 = is_f32(q, "q");
  auto a = grouped_attn(q, sink, pool, out, pages, G, V, vdp, scale, window,
                        v_cos, v_sin, tok_pos, gate);
  TORCH_CHECK(a.dimp <= 256 && vdp <= 256, "head sizes above 256");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2 &&
              tiles.size(0) <= 65535);
  a.tiles = ints(tiles, 0, "tiles");
  a.cu = ints(cu, 2, "cu");
  a.pos0 = ints(pos0, 1, "pos0");
  a.n_tiles = (int)tiles.size(0);
  if (a.n_tiles == 0) return;
  (f32 ? launch_grouped_attn_long_f32 : launch_grouped_attn_long_bf16)(
      &a, head_bucket(a.dimp), head_bucket(vdp), stream());
}

// Rows of C columns, possibly slices of wider ones.
void gelu(Tensor x, Tensor out) {
  const bool f32 = is_f32(x, "x");
  check_like(out, x, "out");
  const long xs = rows2(x, "x"), os = rows2(out, "out");
  TORCH_CHECK(x.sizes() == out.sizes());
  const long rows = x.size(0), C = x.size(1);
  if (rows == 0 || C == 0) return;
  const bool vec = C % 8 == 0 && whole8(x, xs) && whole8(out, os);
  launch_gelu(x.data_ptr(), out.data_ptr(), rows, (int)C, xs, os, vec, f32,
              stream());
}

Tensor cap_logits(Tensor z, double scale, double limit) {
  const bool f32 = is_f32(z, "z");
  TORCH_CHECK(limit != 0.0);
  auto c = z.contiguous();
  aligned16(c, "z");
  auto o = torch::empty(z.sizes(), z.options().dtype(torch::kFloat32));
  if (c.numel())
    launch_cap_logits(c.data_ptr(), o.data_ptr<float>(), c.numel(),
                      (float)scale, (float)limit, f32, stream());
  return o;
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("glu", &glu);
  m.def("clamped_glu", &clamped_glu, py::arg("gate"), py::arg("up"),
        py::arg("limit"), py::arg("alpha"), py::arg("gate_bias") = py::none(),
        py::arg("up_bias") = py::none());
  m.def("add_norm", &add_norm, py::arg("x"), py::arg("y"), py::arg("w_post"),
        py::arg("w_next"), py::arg("f32"), py::arg("eps"), py::arg("offset"),
        py::arg("mult"), py::arg("where"), py::arg("wide"),
        py::arg("y_bias") = py::none());
  m.def("latent_append", &latent_append);
  m.def("latent_gather", &latent_gather);
  m.def("latent_attn_short", &latent_attn_short);
  m.def("latent_attn_long", &latent_attn_long);
  m.def("delta_short", &delta_short);
  m.def("delta_long", &delta_long);
  m.def("grouped_append", &grouped_append);
  m.def("grouped_turn", &grouped_turn);
  m.def("grouped_fill", &grouped_fill);
  m.def("grouped_attn_short", &grouped_attn_short, py::arg("q"),
        py::arg("sink"), py::arg("pool"), py::arg("out"), py::arg("cu"),
        py::arg("pos0"), py::arg("pages"), py::arg("n_req"), py::arg("n_tok"),
        py::arg("max_len"), py::arg("max_keys"), py::arg("kv_heads"),
        py::arg("vdim"), py::arg("vdp"), py::arg("scale"),
        py::arg("window") = 0, py::arg("v_cos") = py::none(),
        py::arg("v_sin") = py::none(), py::arg("tok_pos") = py::none(),
        py::arg("gate") = py::none());
  m.def("grouped_attn_long", &grouped_attn_long, py::arg("q"),
        py::arg("sink"), py::arg("pool"), py::arg("out"), py::arg("tiles"),
        py::arg("cu"), py::arg("pos0"), py::arg("pages"), py::arg("kv_heads"),
        py::arg("vdim"), py::arg("vdp"), py::arg("scale"),
        py::arg("window") = 0, py::arg("v_cos") = py::none(),
        py::arg("v_sin") = py::none(), py::arg("tok_pos") = py::none(),
        py::arg("gate") = py::none());
  m.def("gelu", &gelu);
  m.def("cap_logits", &cap_logits);
  bind_recurrent(m);
  bind_experts(m);
  m.attr("PAGE") = RG_PAGE;
}
