// Row work around grouped attention: norms of the projections, rotations,
// blended values, writing keys and values to their pages; exact gelu; clamped
// gated units; capped logits.
#include "ragged_grouped.h"

#define GR_BLOCK 256

typedef float f32x8 __attribute__((ext_vector_type(8)));

// eight elements as they lie in memory, and their values
template <typename T>
using Raw8 = T __attribute__((ext_vector_type(8)));
template <typename T>
__device__ __forceinline__ Raw8<T> raw8(const T* p) {
  return *reinterpret_cast<const Raw8<T>*>(p);
}
__device__ __forceinline__ f32x8 value8(bf16x8 v) {
  f32x8 o;
#pragma unroll
  for (int j = 0; j < 8; ++j) o[j] = (float)v[j];
  return o;
}
__device__ __forceinline__ f32x8 value8(f32x8 v) { return v; }
template <typename T>
__device__ __forceinline__ f32x8 load8(const T* p) {
  return value8(raw8(p));
}
__device__ __forceinline__ void store8(__bf16* p, f32x8 v) {
  bf16x8 o;
#pragma unroll
  for (int j = 0; j < 8; ++j) o[j] = (__bf16)v[j];
  *reinterpret_cast<bf16x8*>(p) = o;
}
__device__ __forceinline__ void store8(float* p, f32x8 v) {
  store4(p, __builtin_shufflevector(v, v, 0, 1, 2, 3));
  store4(p + 4, __builtin_shufflevector(v, v, 4, 5, 6, 7));
}

// Columns c .. c + 7 of one head (`size` wide, zeros behind it).
template <typename T, bool VEC>
__device__ __forceinline__ f32x8 head8(const T* row, int c, int size) {
  f32x8 o = {0, 0, 0, 0, 0, 0, 0, 0};
  if constexpr (VEC) {
    if (c < size) o = load8(row + c);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (c + j < size) o[j] = (float)row[c + j];
  }
  return o;
}

__device__ __forceinline__ float squares(f32x8 v) {
  float s = 0.0f;
#pragma unroll
  for (int j = 0; j < 8; ++j) s += v[j] * v[j];
  return s;
}

// Columns c .. c + 7 of one head with their pairs rotated, as far as pairs are.
__device__ __forceinline__ f32x8 turn8(f32x8 v, const float* cos_t,
                                       const float* sin_t, int pairs, int pos,
                                       int c) {
  if (!cos_t || c >= 2 * pairs) return v;
  const float* cp = cos_t + (long)pos * pairs + c / 2;
  const float* sp = sin_t + (long)pos * pairs + c / 2;
  f32x4 cs = {1, 1, 1, 1}, sn = {0, 0, 0, 0};
  if (pairs % 4 == 0) {
    cs = load4(cp);
    sn = load4(sp);
  } else {
#pragma unroll
    for (int p = 0; p < 4; ++p)
      if (c / 2 + p < pairs) {
        cs[p] = cp[p];
        sn[p] = sp[p];
      }
  }
  f32x8 o;
#pragma unroll
  for (int p = 0; p < 4; ++p) {
    o[2 * p] = v[2 * p] * cs[p] - v[2 * p + 1] * sn[p];
    o[2 * p + 1] = v[2 * p + 1] * cs[p] + v[2 * p] * sn[p];
  }
  return o;
}

// The i-th chunk of eight columns of a row of heads padded to 8 * nc columns.
template <typename T, bool VEC>
__device__ __forceinline__ f32x8 chunk8(const T* row, int i, int size, int nc) {
  const int h = i / nc;
  return head8<T, VEC>(row + h * size, (i - h * nc) * 8, size);
}

// Where that chunk lies; what is past the row or in the padding reads another
// chunk of it, so that many loads are in flight together.
template <typename T>
__device__ __forceinline__ const T* chunk_at(const T* row, int i, int n,
                                             int size, int nc) {
  i = min(i, n - 1);
  const int h = i / nc;
  return row + h * size + min((i - h * nc) * 8, size - 8);
}

// Where eight columns of a key in slot r of its page go, from the head's base.
__device__ __forceinline__ int key_place(int r, int c, int dimp) {
  return ((r / 16 * (dimp / 32) + c / 32) * 64 + c / 8 % 4 * 16 + r % 16) * 8;
}

// One block per token: queries out [N, H, dimp]; keys and values of the first
// `direct` tokens go to their pages, the others only leave their keys' inverse
// rms.  NQ, NK: chunks of the projections a thread keeps (whole vectors only);
// 0: read twice.
template <typename T, bool VEC, int NQ, int NK>
__global__ __launch_bounds__(GR_BLOCK) void grouped_append_kernel(
    const GroupedRowArgs a, T* __restrict__ q, float* __restrict__ kinv,
    const int* __restrict__ tok_pos, const int* __restrict__ tok_entry,
    const int* __restrict__ pages, int P, int direct) {
  constexpr int AQ = NQ > 0 ? NQ : 1, AK = NK > 0 ? NK : 1;
  __shared__ float sums[2][GR_BLOCK / WAVE];
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const T* yq = (const T*)a.y + t * a.ystride;
  const T* yk = yq + (long)a.H * a.D;
  const T* yv = yk + (long)a.G * a.D;
  const T* wq = (const T*)a.wq;
  const T* wk = (const T*)a.wk;
  const int nc = a.dimp / 8, nq = a.H * nc, nk = a.G * nc;

  Raw8<T> rq[AQ], rqw[AQ], rk[AK], rkw[AK];
#pragma unroll
  for (int k = 0; k < NQ; ++k) {
    const int i = k * GR_BLOCK + tid;
    rq[k] = raw8(chunk_at(yq, i, nq, a.D, nc));
    rqw[k] = raw8(chunk_at(wq ? wq : yq, i, nq, a.D, nc));
  }
#pragma unroll
  for (int k = 0; k < NK; ++k) {
    const int i = k * GR_BLOCK + tid;
    rk[k] = raw8(chunk_at(yk, i, nk, a.D, nc));
    rkw[k] = raw8(chunk_at(wk ? wk : yk, i, nk, a.D, nc));
  }
  const bool write = t < direct;
  int r = 0;
  long page = 0;
  if (write) {
    const int pos = tok_pos[t];
    r = pos % RG_PAGE;
    page = pages[(long)tok_entry[t] * P + pos / RG_PAGE];
  }
  float sq = 0.0f, sk = 0.0f;
  f32x8 qv[AQ], kv[AK];
  const f32x8 none = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
  for (int k = 0; k < NQ; ++k) {
    const int i = k * GR_BLOCK + tid;
    qv[k] = i < nq && i % nc * 8 < a.D ? value8(rq[k]) : none;
    sq += squares(qv[k]);
  }
#pragma unroll
  for (int k = 0; k < NK; ++k) {
    const int i = k * GR_BLOCK + tid;
    kv[k] = i < nk && i % nc * 8 < a.D ? value8(rk[k]) : none;
    sk += squares(kv[k]);
  }
  if constexpr (NQ == 0)
    for (int i = tid; i < nq; i += GR_BLOCK)
      sq += squares(chunk8<T, VEC>(yq, i, a.D, nc));
  if constexpr (NK == 0)
    for (int i = tid; i < nk; i += GR_BLOCK)
      sk += squares(chunk8<T, VEC>(yk, i, a.D, nc));
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if (tid % WAVE == 0) {
    sums[0][tid / WAVE] = sq;
    sums[1][tid / WAVE] = sk;
  }
  __syncthreads();
  sq = sk = 0.0f;
#pragma unroll
  for (int w = 0; w < GR_BLOCK / WAVE; ++w) {
    sq += sums[0][w];
    sk += sums[1][w];
  }
  const float qi = 1.0f / sqrtf(sq / (float)(a.H * a.D) + a.eps);
  const float ki = 1.0f / sqrtf(sk / (float)(a.G * a.D) + a.eps);
  if (tid == 0) kinv[t] = ki;

  T* qo = q + t * a.H * a.dimp;
#pragma unroll
  for (int k = 0; k < NQ; ++k) {
    const int i = k * GR_BLOCK + tid;
    if (i < nq)
      store8(qo + (long)i * 8, wq ? qv[k] * qi * value8(rqw[k]) : qv[k]);
  }
  if constexpr (NQ == 0) {
    for (int i = tid; i < nq; i += GR_BLOCK) {
      f32x8 v = chunk8<T, VEC>(yq, i, a.D, nc);
      if (wq) v = v * qi * chunk8<T, VEC>(wq, i, a.D, nc);
      store8(qo + (long)i * 8, v);
    }
  }
  if (!write) return;

  const long PW = (long)RG_PAGE * (a.dimp + a.vdp);
  T* base = (T*)a.pool + page * a.G * PW;
  auto key_at = [&](int i) {
    const int g = i / nc, c = (i - g * nc) * 8;
    return base + g * PW + key_place(r, c, a.dimp);
  };
#pragma unroll
  for (int k = 0; k < NK; ++k) {
    const int i = k * GR_BLOCK + tid;
    if (i < nk) store8(key_at(i), wk ? kv[k] * ki * value8(rkw[k]) : kv[k]);
  }
  if constexpr (NK == 0) {
    for (int i = tid; i < nk; i += GR_BLOCK) {
      f32x8 v = chunk8<T, VEC>(yk, i, a.D, nc);
      if (wk) v = v * ki * chunk8<T, VEC>(wk, i, a.D, nc);
      store8(key_at(i), v);
    }
  }
  const T* first = a.first ? (const T*)a.first + t * a.fstride : nullptr;
  const float lam = first ? (float)((const T*)a.vmix)[0] : 0.0f;
  for (int i = tid; i < a.G * a.vdp; i += GR_BLOCK) {
    const int g = i / a.vdp, d = i - g * a.vdp;
    float v = 0.0f;
    if (d < a.V) {
      v = (float)yv[g * a.V + d];
      if (first) v = (1.0f - lam) * v + lam * (float)first[g * a.V + d];
    }
    base[g * PW + RG_PAGE * a.dimp +
         ((d / 16 * 2 + r / 32) * 64 + r / 4 % 4 * 16 + d % 16) * 8 +
         r / 16 % 2 * 4 + r % 4] = (T)v;
  }
}

// The same with norms per head and rotations: `sub` lanes (a power of two) share
// one head of one token, each eight of its columns.  Items of a token are its
// query heads, keys and values, or the query heads alone; keys' inverse rms
// [N, G].
template <typename T, bool VEC>
__global__ __launch_bounds__(GR_BLOCK) void grouped_turn_kernel(
    const GroupedRowArgs a, T* __restrict__ q, float* __restrict__ kinv,
    const int* __restrict__ tok_entry, const int* __restrict__ pages, int P,
    int direct, int sub, long n_tok, int items) {
  const long at = ((long)blockIdx.x * GR_BLOCK + threadIdx.x) / sub;
  const int c = threadIdx.x % sub * 8;
  const long t = min(at / items, n_tok - 1);
  const bool live = at / items < n_tok;
  const int j = (int)(at - at / items * items);
  const int pos = a.tok_pos[t];
  const bool value = j >= a.H + a.G;
  const int size = value ? a.V : a.D;
  const T* src = (const T*)a.y + t * a.ystride +
                 (value ? (long)(a.H + a.G) * a.D + (long)(j - a.H - a.G) * a.V
                        : (long)j * a.D);
  f32x8 v = head8<T, VEC>(src, c, size);
  if (a.head_norm) {
    float ss = squares(v);
    for (int o = 1; o < sub; o <<= 1) ss += __shfl_xor(ss, o, WAVE);
    const float inv = 1.0f / sqrtf(ss / (float)a.D + a.eps);
    if (!value) {
      v = v * inv;
      const T* w = (const T*)(j < a.H ? a.wq : a.wk);
      if (w) v = v * head8<T, VEC>(w, c, a.D);
    }
    if (live && c == 0 && !value && j >= a.H) kinv[t * a.G + j - a.H] = inv;
  }
  if (value)
    v = turn8(v, a.v_cos, a.v_sin, a.v_pairs, pos, c);
  else
    v = turn8(v, a.qk_cos, a.qk_sin, a.qk_pairs, pos, c);
  if (!live) return;
  if (j < a.H) {
    if (c < a.dimp) store8(q + (t * a.H + j) * a.dimp + c, v);
    return;
  }
  if (t >= direct) return;
  const int r = pos % RG_PAGE;
  const long page = pages[(long)tok_entry[t] * P + pos / RG_PAGE];
  const int g = value ? j - a.H - a.G : j - a.H;
  T* base = (T*)a.pool + (page * a.G + g) * RG_PAGE * (a.dimp + a.vdp);
  if (!value) {
    if (c < a.dimp) store8(base + key_place(r, c, a.dimp), v);
    return;
  }
  base += RG_PAGE * a.dimp;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int d = c + i;
    if (d < a.vdp)
      base[((d / 16 * 2 + r / 32) * 64 + r / 4 % 4 * 16 + d % 16) * 8 +
           r / 16 % 2 * 4 + r % 4] = (T)v[i];
  }
}

// One block per (page, key/value head): the slots lo .. hi - 1 of a page from
// tokens t + slot; later slots become zero, earlier ones stay.
//   fills[i] = (page, t, lo, hi)
// TURN: norms per head (wk is one head's weights) and rotations in place of
// norms of rows and blended values.
template <typename T, bool VEC, bool TURN>
__global__ __launch_bounds__(GR_BLOCK) void grouped_fill_kernel(
    const GroupedRowArgs a, const float* __restrict__ kinv,
    const int* __restrict__ fills) {
  __shared__ T sv[RG_PAGE][64 + 4];
  const int* f = fills + (long)blockIdx.x * 4;
  const int g = blockIdx.y;
  const long t = f[1];
  const int lo = f[2], hi = f[3];
  const int tid = threadIdx.x;
  const T* y = (const T*)a.y;
  const T* wk = a.wk ? (const T*)a.wk + (TURN ? 0 : g * a.D) : nullptr;
  const long koff = (long)(a.H + g) * a.D;
  const long voff = (long)(a.H + a.G) * a.D + (long)g * a.V;
  T* base = (T*)a.pool +
            ((long)f[0] * a.G + g) * RG_PAGE * (a.dimp + a.vdp);

  const int nk = a.dimp / 32;
  for (int i = tid; i < 4 * nk * 64; i += GR_BLOCK) {
    const int tile = i / 64, lane = i % 64;
    const int s = tile / nk * 16 + lane % 16;
    const int c = tile % nk * 32 + lane / 16 * 8;
    if (s < lo) continue;
    f32x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
    if (s < hi) {
      v = head8<T, VEC>(y + (t + s) * a.ystride + koff, c, a.D);
      if constexpr (TURN) {
        if (a.head_norm) v = v * kinv[(t + s) * a.G + g];
        if (wk) v = v * head8<T, VEC>(wk, c, a.D);
        v = turn8(v, a.qk_cos, a.qk_sin, a.qk_pairs, a.tok_pos[t + s], c);
      } else {
        if (wk) v = v * kinv[t + s] * head8<T, VEC>(wk, c, a.D);
      }
    }
    store8(base + (long)i * 8, v);
  }

  base += RG_PAGE * a.dimp;
  const T* first = (const T*)a.first;
  const float lam = first ? (float)((const T*)a.vmix)[0] : 0.0f;
  for (int d0 = 0; d0 < a.vdp; d0 += 64) {
    if (d0) __syncthreads();
    for (int i = tid; i < RG_PAGE * 8; i += GR_BLOCK) {
      const int s = i / 8, c = d0 + i % 8 * 8;
      f32x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (s >= lo && s < hi) {
        v = head8<T, VEC>(y + (t + s) * a.ystride + voff, c, a.V);
        if constexpr (TURN)
          v = turn8(v, a.v_cos, a.v_sin, a.v_pairs, a.tok_pos[t + s], c);
        else if (first)
          v = (1.0f - lam) * v +
              lam * head8<T, VEC>(
                        first + (t + s) * a.fstride + (long)g * a.V, c, a.V);
      }
      T* o = &sv[s][i % 8 * 8];
      store4(o, f32x4{v[0], v[1], v[2], v[3]});
      store4(o + 4, f32x4{v[4], v[5], v[6], v[7]});
    }
    __syncthreads();
    const int tiles = min(4, (a.vdp - d0) / 16);
    for (int i = tid; i < tiles * 128; i += GR_BLOCK) {
      const int lane = i % 64;
      const int s = i / 64 % 2 * 32 + lane / 16 * 4;  // first key of the eight
      const int d = i / 128 * 16 + lane % 16;
      T* o = base + ((long)(d0 / 16) * 128 + i) * 8;
      f32x8 v;
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = (float)sv[s + (j < 4 ? j : 12 + j)][d];
      if (s >= lo) {
        store8(o, v);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (s + (j < 4 ? j : 12 + j) >= lo) o[j] = (T)v[j];
      }
    }
  }
}

extern "C" void launch_grouped_append(const GroupedRowArgs* a, void* q,
                                      float* kinv, const int* tok_pos,
                                      const int* tok_entry, const int* pages,
                                      int P, int direct, long n_tok, bool f32,
                                      hipStream_t stream) {
  dim3 grid((unsigned)n_tok), block(GR_BLOCK);
  const int nq = (a->H * (a->dimp / 8) + GR_BLOCK - 1) / GR_BLOCK;
  const int nk = (a->G * (a->dimp / 8) + GR_BLOCK - 1) / GR_BLOCK;
#define GR_GO(T, VEC, NQ, NK)                                        \
  grouped_append_kernel<T, VEC, NQ, NK><<<grid, block, 0, stream>>>( \
      *a, (T*)q, kinv, tok_pos, tok_entry, pages, P, direct)
#define GR_ROW(T)                                              \
  do {                                                         \
    if (!a->vec) GR_GO(T, false, 0, 0);                        \
    else if (nq > 4) GR_GO(T, true, 0, 0);                     \
    else if (nq <= 1) GR_GO(T, true, 1, 1);                    \
    else if (nq <= 2 && nk <= 1) GR_GO(T, true, 2, 1);         \
    else if (nk <= 1) GR_GO(T, true, 4, 1);                    \
    else GR_GO(T, true, 4, 4);                                 \
  } while (0)
  if (f32) GR_ROW(float);
  else GR_ROW(__bf16);
#undef GR_ROW
#undef GR_GO
}

extern "C" void launch_grouped_turn(const GroupedRowArgs* a, void* q,
                                    float* kinv, const int* tok_entry,
                                    const int* pages, int P, int direct,
                                    long n_tok, bool own, bool f32,
                                    hipStream_t stream) {
  int sub = 1;
  while (sub * 8 < a->dimp || sub * 8 < a->vdp) sub *= 2;
  const int items = a->H + (own ? 2 * a->G : 0);
  const long lanes = n_tok * items * sub;
  dim3 grid((unsigned)((lanes + GR_BLOCK - 1) / GR_BLOCK)), block(GR_BLOCK);
#define GR_GO(T, VEC)                                                        \
  grouped_turn_kernel<T, VEC><<<grid, block, 0, stream>>>(                   \
      *a, (T*)q, kinv, tok_entry, pages, P, direct, sub, n_tok, items)
  if (f32) {
    if (a->vec) GR_GO(float, true);
    else GR_GO(float, false);
  } else {
    if (a->vec) GR_GO(__bf16, true);
    else GR_GO(__bf16, false);
  }
#undef GR_GO
}

extern "C" void launch_grouped_fill(const GroupedRowArgs* a, const float* kinv,
                                    const int* fills, int n_fills, bool f32,
                                    hipStream_t stream) {
  dim3 grid((unsigned)n_fills, (unsigned)a->G), block(GR_BLOCK);
  const bool turn = a->head_norm || a->qk_cos || a->v_cos;
#define GR_TURN(T, VEC, TURN)                                           \
  grouped_fill_kernel<T, VEC, TURN><<<grid, block, 0, stream>>>(*a, kinv, \
                                                               fills)
#define GR_GO(T, VEC)               \
  do {                              \
    if (turn) GR_TURN(T, VEC, true); \
    else GR_TURN(T, VEC, false);    \
  } while (0)
  if (f32) {
    if (a->vec) GR_GO(float, true);
    else GR_GO(float, false);
  } else {
    if (a->vec) GR_GO(__bf16, true);
    else GR_GO(__bf16, false);
  }
#undef GR_GO
#undef GR_TURN
}

// ---------------------------------------------------------------------------
// Exact gelu, x * Phi(x), on strided rows.
// ---------------------------------------------------------------------------

template <typename T>
__device__ __forceinline__ float gelu_erf(float x);
template <>
__device__ __forceinline__ float gelu_erf<float>(float x) {
  return 0.5f * x * (1.0f + erff(x * 0.70710678118654752440f));
}
// For bf16 results: erfc by the rational approximation 7.1.26 of Abramowitz
// and Stegun, Handbook of Mathematical Functions (error below 1.5e-7).
template <>
__device__ __forceinline__ float gelu_erf<__bf16>(float x) {
  const float z = fabsf(x) * 0.70710678118654752440f;
  const float t = __builtin_amdgcn_rcpf(fmaf(0.3275911f, z, 1.0f));
  float p = fmaf(t, 1.061405429f, -1.453152027f);
  p = fmaf(t, p, 1.421413741f);
  p = fmaf(t, p, -0.284496736f);
  p = fmaf(t, p, 0.254829592f);
  const float tail = 0.5f * p * t *
                     __builtin_amdgcn_exp2f(-1.44269504088896340736f * z * z);
  return x * (x < 0.0f ? tail : 1.0f - tail);
}

template <typename T, bool VEC>
__global__ __launch_bounds__(GR_BLOCK) void gelu_kernel(
    const T* __restrict__ x, T* __restrict__ o, int C, long xs, long os) {
  const long row = blockIdx.y;
  const T* xr = x + row * xs;
  T* orow = o + row * os;
  if constexpr (VEC) {
    const int c = (blockIdx.x * GR_BLOCK + threadIdx.x) * 8;
    if (c >= C) return;
    f32x8 v = load8(xr + c);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = gelu_erf<T>(v[j]);
    store8(orow + c, v);
  } else {
    const int c = blockIdx.x * GR_BLOCK + threadIdx.x;
    if (c < C) orow[c] = (T)gelu_erf<T>((float)xr[c]);
  }
}

extern "C" void launch_gelu(const void* x, void* o, long rows, int C, long xs,
                            long os, bool vec, bool f32, hipStream_t stream) {
  const int per = GR_BLOCK * (vec ? 8 : 1);
  const long most = 65535;  // rows of one launch
#define GR_GO(T, VEC)                                                        \
  for (long r = 0; r < rows; r += most) {                                    \
    dim3 grid((unsigned)((C + per - 1) / per),                               \
              (unsigned)(rows - r < most ? rows - r : most));                \
    gelu_kernel<T, VEC><<<grid, dim3(GR_BLOCK), 0, stream>>>(                \
        (const T*)x + r * xs, (T*)o + r * os, C, xs, os);                    \
  }
  if (f32) {
    if (vec) { GR_GO(float, true) } else { GR_GO(float, false) }
  } else {
    if (vec) { GR_GO(__bf16, true) } else { GR_GO(__bf16, false) }
  }
#undef GR_GO
}

// ---------------------------------------------------------------------------
// Clamped gated unit on strided rows (and biases, if there are any):
// g sigmoid(alpha g) (u + 1), g at most limit, u within +-limit.
// ---------------------------------------------------------------------------

template <typename T, bool VEC>
__global__ __launch_bounds__(GR_BLOCK) void clamped_glu_kernel(
    const T* __restrict__ gate, const T* __restrict__ up,
    const T* __restrict__ gate_b, const T* __restrict__ up_b, T* __restrict__ o,
    long rows, int C, long gs, long us, float limit, float alpha) {
  constexpr int V = VEC ? 8 : 1;
  const int per = C / V;  // whole vectors, or elements
  const long total = rows * per, step = (long)gridDim.x * GR_BLOCK;
  for (long i = (long)blockIdx.x * GR_BLOCK + threadIdx.x; i < total; i += step) {
    const long r = i / per;
    const int c = (int)(i - r * per) * V;
    if constexpr (VEC) {
      f32x8 g = load8(gate + r * gs + c), u = load8(up + r * us + c);
      if (gate_b) g = g + load8(gate_b + c);
      if (up_b) u = u + load8(up_b + c);
#pragma unroll
      for (int j = 0; j < 8; ++j) g[j] = clamped_glu_of<T>(g[j], u[j], limit, alpha);
      store8(o + r * C + c, g);
    } else {
      const float g = (float)gate[r * gs + c] + (gate_b ? (float)gate_b[c] : 0.0f);
      const float u = (float)up[r * us + c] + (up_b ? (float)up_b[c] : 0.0f);
      o[r * C + c] = (T)clamped_glu_of<T>(g, u, limit, alpha);
    }
  }
}

extern "C" void launch_clamped_glu(const void* gate, const void* up,
                                   const void* gate_b, const void* up_b,
                                   void* o, long rows, int C, long gs, long us,
                                   float limit, float alpha, bool vec, bool f32,
                                   hipStream_t stream) {
  const long want = (rows * (vec ? C / 8 : C) + GR_BLOCK - 1) / GR_BLOCK;
  dim3 grid((unsigned)(want < 16384 ? want : 16384)), block(GR_BLOCK);
#define GR_GO(T, VEC)                                                     \
  clamped_glu_kernel<T, VEC><<<grid, block, 0, stream>>>(                 \
      (const T*)gate, (const T*)up, (const T*)gate_b, (const T*)up_b, (T*)o, \
      rows, C, gs, us, limit, alpha)
  if (f32) {
    if (vec) GR_GO(float, true);
    else GR_GO(float, false);
  } else {
    if (vec) GR_GO(__bf16, true);
    else GR_GO(__bf16, false);
  }
#undef GR_GO
}

// limit * tanh(z * scale / limit), four columns at a time.
template <typename T>
__device__ __forceinline__ float tanh_any(float x);
template <>
__device__ __forceinline__ float tanh_any<float>(float x) {
  return tanhf(x);
}
// logits that come in bf16: tanh by its definition, off by 1e-7 at most
template <>
__device__ __forceinline__ float tanh_any<__bf16>(float x) {
  const float e = __builtin_amdgcn_exp2f(2.88539008177792681472f * fabsf(x));
  return copysignf(1.0f - 2.0f * __builtin_amdgcn_rcpf(e + 1.0f), x);
}

template <typename T>
__global__ __launch_bounds__(GR_BLOCK) void cap_logits_kernel(
    const T* __restrict__ z, float* __restrict__ o, long n, float scale,
    float limit) {
  const float by = scale / limit;
  const long step = (long)gridDim.x * GR_BLOCK * 4;
  for (long i = ((long)blockIdx.x * GR_BLOCK + threadIdx.x) * 4; i < n;
       i += step) {
    if (i + 4 <= n) {
      f32x4 v = load4(z + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = limit * tanh_any<T>(v[j] * by);
      store4(o + i, v);
    } else {
      for (long j = i; j < n; ++j)
        o[j] = limit * tanh_any<T>((float)z[j] * by);
    }
  }
}

extern "C" void launch_cap_logits(const void* z, float* o, long n, float scale,
                                  float limit, bool f32, hipStream_t stream) {
  const long want = (n + GR_BLOCK * 4 - 1) / (GR_BLOCK * 4);
  dim3 grid((unsigned)(want < 16384 ? want : 16384)), block(GR_BLOCK);
  if (f32)
    cap_logits_kernel<float><<<grid, block, 0, stream>>>((const float*)z, o, n,
                                                         scale, limit);
  else
    cap_logits_kernel<__bf16><<<grid, block, 0, stream>>>((const __bf16*)z, o,
                                                          n, scale, limit);
}
