// Norms around a 32-bit residual stream, and the short-row work of paged
// latent attention (latent norm, rotation, append, gather).
#include "ragged_common.h"

#define RN_BLOCK 256

// ---------------------------------------------------------------------------
// One sublayer boundary in one kernel, one block per row:
//   y += y_bias                           (y_bias == null: y as it is)
//   x += mult * rms(y) * (w_post + off)   (y == null: x unchanged;
//                                          w_post == null: x += mult * y)
//   h  = rms(x) * (w_next + off)      (w_next == null: h = x; h == null: no h)
// x is the fp32 residual; y and h are T; w_next holds W weights or one for all
// (one_next).  Rows of h have Wh columns, those past W become zero.  NR > 0
// keeps the row in registers (NR groups of VEC elements per thread); NR == 0
// re-reads it.  SUM: row i of y is the sum of its rows where[i, 0 .. top - 1],
// -1 for none.
// ---------------------------------------------------------------------------

template <typename T, int VEC>
__device__ __forceinline__ void rn_load(const T* p, float (&o)[VEC]) {
  if constexpr (VEC == 4) {
    f32x4 v = load4(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = v[j];
  } else {
    o[0] = (float)p[0];
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void rn_store(T* p, const float (&o)[VEC]) {
  if constexpr (VEC == 4) {
    store4(p, f32x4{o[0], o[1], o[2], o[3]});
  } else {
    p[0] = (T)o[0];
  }
}

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

template <typename T, int VEC, int NR, bool SUM>
__global__ __launch_bounds__(RN_BLOCK) void add_norm_kernel(
    const AddNormArgs a) {
  __shared__ float scratch[RN_BLOCK / WAVE];
  const long row = blockIdx.x;
  const int W = a.W;
  float* xr = a.x + row * W;
  const T* y = (const T*)a.y;
  const T* w_post = (const T*)a.w_post;
  const T* w_next = (const T*)a.w_next;
  T* hr = a.h ? (T*)a.h + row * a.Wh : nullptr;
  const int step = RN_BLOCK * VEC;
  constexpr int NA = NR > 0 ? NR : 1;
  float xv[NA][VEC];

  auto load_y = [&](int c, float (&o)[VEC]) {
    if constexpr (SUM) {
      const int* from = a.where + row * a.top;
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = 0.0f;
#pragma unroll 4
      for (int k = 0; k < a.top; ++k) {
        if (from[k] < 0) continue;
        float part[VEC];
        rn_load<T, VEC>(y + from[k] * a.ystride + c, part);
#pragma unroll
        for (int j = 0; j < VEC; ++j) o[j] += part[j];
      }
    } else {
      rn_load<T, VEC>(y + row * a.ystride + c, o);
    }
    if (a.y_bias) {
      float b[VEC];
      rn_load<T, VEC>((const T*)a.y_bias + c, b);
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] += b[j];
    }
  };

  float inv_y = a.mult;
  float yv[NA][VEC];
  if (y && !w_post) {
    if constexpr (NR > 0) {
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int c = i * step + threadIdx.x * VEC;
        if (c < W) load_y(c, yv[i]);
      }
    }
  } else if (y) {
    float ss = 0.0f;
    if constexpr (NR > 0) {
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int c = i * step + threadIdx.x * VEC;
        if (c < W) {
          load_y(c, yv[i]);
#pragma unroll
          for (int j = 0; j < VEC; ++j) ss += yv[i][j] * yv[i][j];
        }
      }
    } else {
      for (int c = threadIdx.x * VEC; c < W; c += step) {
        load_y(c, yv[0]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss += yv[0][j] * yv[0][j];
      }
    }
    ss = block_sum<RN_BLOCK>(ss, scratch);
    inv_y = a.mult / sqrtf(ss / (float)W + a.eps);
  }

  float ss = 0.0f;
  auto update = [&](int c, float (&xa)[VEC], float (&ya)[VEC]) {
    rn_load<float, VEC>(xr + c, xa);
    if (y && !w_post) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) xa[j] += ya[j] * inv_y;
      rn_store<float, VEC>(xr + c, xa);
    } else if (y) {
      float wv[VEC];
      rn_load<T, VEC>(w_post + c, wv);
#pragma unroll
      for (int j = 0; j < VEC; ++j) xa[j] += ya[j] * inv_y * (wv[j] + a.off);
      rn_store<float, VEC>(xr + c, xa);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += xa[j] * xa[j];
  };
  if constexpr (NR > 0) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int c = i * step + threadIdx.x * VEC;
      if (c < W) update(c, xv[i], yv[i]);
    }
  } else {
    for (int c = threadIdx.x * VEC; c < W; c += step) {
      if (y) load_y(c, yv[0]);
      update(c, xv[0], yv[0]);
    }
  }
  if (!hr) return;
  for (int c = W + threadIdx.x; c < a.Wh; c += RN_BLOCK) hr[c] = (T)0.0f;
  float inv = 1.0f;
  if (w_next) {
    ss = block_sum<RN_BLOCK>(ss, scratch);
    inv = 1.0f / sqrtf(ss / (float)W + a.eps);
  }
  const float one = a.one_next ? (float)w_next[0] : 0.0f;
  auto emit = [&](int c, float (&xa)[VEC]) {
    if (!w_next) {
      rn_store<T, VEC>(hr + c, xa);
      return;
    }
    float wv[VEC], o[VEC];
    if (a.one_next) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) wv[j] = one;
    } else {
      rn_load<T, VEC>(w_next + c, wv);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = xa[j] * inv * (wv[j] + a.off);
    rn_store<T, VEC>(hr + c, o);
  };
  if constexpr (NR > 0) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int c = i * step + threadIdx.x * VEC;
      if (c < W) emit(c, xv[i]);
    }
  } else {
    for (int c = threadIdx.x * VEC; c < W; c += step) {
      rn_load<float, VEC>(xr + c, xv[0]);
      emit(c, xv[0]);
    }
  }
}

template <typename T>
static void add_norm_t(const AddNormArgs& a, hipStream_t stream) {
  const bool vec = a.W % 4 == 0 && a.Wh % 4 == 0 && a.ystride % 4 == 0 &&
                   ((uintptr_t)a.y) % 16 == 0;
  const int nr = (a.W + RN_BLOCK * 4 - 1) / (RN_BLOCK * 4);
  dim3 grid((unsigned)a.rows), block(RN_BLOCK);
#define RN_GO(V, N)                                                 \
  do {                                                              \
    if (a.where)                                                    \
      add_norm_kernel<T, V, N, true><<<grid, block, 0, stream>>>(a); \
    else                                                            \
      add_norm_kernel<T, V, N, false><<<grid, block, 0, stream>>>(a); \
  } while (0)
  if (!vec)
    RN_GO(1, 0);
  else if (nr <= 1)
    RN_GO(4, 1);
  else if (nr <= 2)
    RN_GO(4, 2);
  else if (nr <= 4)
    RN_GO(4, 4);
  else if (nr <= 8)
    RN_GO(4, 8);
  else
    RN_GO(4, 0);
#undef RN_GO
}

extern "C" void launch_add_norm(const AddNormArgs* a, bool f32,
                                hipStream_t stream) {
  if (f32)
    add_norm_t<float>(*a, stream);
  else
    add_norm_t<__bf16>(*a, stream);
}

// ---------------------------------------------------------------------------
// Latent row work, one block per token:
//   pool[row(token)] = [ rms(d[:rank]) * w | 0 | rotate(d[rank:]) | 0 ]
//   q[token, h, qoff : qoff + rot] rotated in place for every head
// Rows are rankp + rotp wide; rotation pairs neighbours; cos/sin [*, rot/2].
// dkv == null (the layer reads another layer's rows): only q is rotated.
// ---------------------------------------------------------------------------

template <typename T>
__global__ __launch_bounds__(RN_BLOCK) void latent_append_kernel(
    const T* __restrict__ dkv, long dstride, const T* __restrict__ norm_w,
    float eps, T* __restrict__ pool, T* __restrict__ q, long qstride, int H,
    int dq, int qoff, int rank, int rankp, int rot, int rotp,
    const float* __restrict__ cost, const float* __restrict__ sint,
    const int* __restrict__ tok_pos, const int* __restrict__ tok_entry,
    const int* __restrict__ pages, int P) {
  __shared__ float scratch[RN_BLOCK / WAVE];
  const long t = blockIdx.x;
  const int pos = tok_pos[t];
  const int half = rot / 2;
  const float* c = cost + (long)pos * half;
  const float* s = sint + (long)pos * half;

  T* qt = q + t * qstride + qoff;
  for (int i = threadIdx.x; i < H * half; i += RN_BLOCK) {
    const int h = i / half, p = i - h * half;
    T* a = qt + (long)h * dq + 2 * p;
    const float u = (float)a[0], v = (float)a[1];
    a[0] = (T)(u * c[p] - v * s[p]);
    a[1] = (T)(v * c[p] + u * s[p]);
  }
  if (!dkv) return;

  const T* d = dkv + t * dstride;
  const long page = pages[(long)tok_entry[t] * P + pos / RG_PAGE];
  T* row = pool + (page * RG_PAGE + pos % RG_PAGE) * (long)(rankp + rotp);
  float ss = 0.0f;
  for (int i = threadIdx.x; i < rank; i += RN_BLOCK) {
    const float v = (float)d[i];
    ss += v * v;
  }
  ss = block_sum<RN_BLOCK>(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)rank + eps);
  for (int i = threadIdx.x; i < rankp; i += RN_BLOCK)
    row[i] = i < rank ? (T)((float)d[i] * inv * (float)norm_w[i]) : (T)0.0f;
  for (int p = threadIdx.x; p < rotp / 2; p += RN_BLOCK) {
    float o0 = 0.0f, o1 = 0.0f;
    if (p < half) {
      const float u = (float)d[rank + 2 * p], v = (float)d[rank + 2 * p + 1];
      o0 = u * c[p] - v * s[p];
      o1 = v * c[p] + u * s[p];
    }
    row[rankp + 2 * p] = (T)o0;
    row[rankp + 2 * p + 1] = (T)o1;
  }
}

extern "C" void launch_latent_append(
    const void* dkv, long dstride, const void* norm_w, float eps, void* pool,
    void* q, long qstride, int H, int dq, int qoff, int rank, int rankp,
    int rot, int rotp, const float* cost, const float* sint,
    const int* tok_pos, const int* tok_entry, const int* pages, int P,
    long n_tok, bool f32, hipStream_t stream) {
  dim3 grid((unsigned)n_tok), block(RN_BLOCK);
#define LA_GO(T)                                                            \
  latent_append_kernel<T><<<grid, block, 0, stream>>>(                      \
      (const T*)dkv, dstride, (const T*)norm_w, eps, (T*)pool, (T*)q,       \
      qstride, H, dq, qoff, rank, rankp, rot, rotp, cost, sint, tok_pos,    \
      tok_entry, pages, P)
  if (f32)
    LA_GO(float);
  else
    LA_GO(__bf16);
#undef LA_GO
}

// ---------------------------------------------------------------------------
// Pages -> contiguous rows.  One block per page: blocks[i] = (page, first
// destination row, valid rows); rows past the valid ones become zero.
// ---------------------------------------------------------------------------

template <typename T>
__global__ __launch_bounds__(RN_BLOCK) void latent_gather_kernel(
    const T* __restrict__ pool, T* __restrict__ dst,
    const int* __restrict__ blocks, int W) {
  const int* b = blocks + (long)blockIdx.x * 3;
  const T* src = pool + (long)b[0] * RG_PAGE * W;
  T* out = dst + (long)b[1] * W;
  const int nvec = W / 8;
  const int valid = b[2] * nvec;
  for (int i = threadIdx.x; i < RG_PAGE * nvec; i += RN_BLOCK) {
    if (i < valid)
      copy8(out + (long)i * 8, src + (long)i * 8);
    else
      zero8(out + (long)i * 8);
  }
}

extern "C" void launch_latent_gather(const void* pool, void* dst,
                                     const int* blocks, int n_blocks, int W,
                                     bool f32, hipStream_t stream) {
  dim3 grid((unsigned)n_blocks), block(RN_BLOCK);
  if (f32)
    latent_gather_kernel<float><<<grid, block, 0, stream>>>(
        (const float*)pool, (float*)dst, blocks, W);
  else
    latent_gather_kernel<__bf16><<<grid, block, 0, stream>>>(
        (const __bf16*)pool, (__bf16*)dst, blocks, W);
}
