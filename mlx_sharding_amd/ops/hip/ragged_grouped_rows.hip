// Row work around grouped attention: norms of the projections, blended
// values, writing keys and values to their pages; exact gelu; capped logits.
#include "ragged_grouped.h"

#define GR_BLOCK 256

template <typename T>
__device__ __forceinline__ void load8(const T* p, float (&o)[8]) {
  const f32x4 a = load4(p), b = load4(p + 4);
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    o[j] = a[j];
    o[4 + j] = b[j];
  }
}

template <typename T>
__device__ __forceinline__ void store8(T* p, const float (&v)[8]);
template <>
__device__ __forceinline__ void store8(__bf16* p, const float (&v)[8]) {
  bf16x8 o;
#pragma unroll
  for (int j = 0; j < 8; ++j) o[j] = (__bf16)v[j];
  *reinterpret_cast<bf16x8*>(p) = o;
}
template <>
__device__ __forceinline__ void store8(float* p, const float (&v)[8]) {
  store4(p, f32x4{v[0], v[1], v[2], v[3]});
  store4(p + 4, f32x4{v[4], v[5], v[6], v[7]});
}

// Columns c .. c + 7 of one head (`size` wide, zeros behind it).
template <typename T, bool VEC>
__device__ __forceinline__ void head8(const T* row, int c, int size,
                                      float (&o)[8]) {
  if (VEC && c < size) {
    load8(row + c, o);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      o[j] = !VEC && c + j < size ? (float)row[c + j] : 0.0f;
  }
}

// normed columns: row and weight of one head, times the row's inverse rms
template <typename T, bool VEC>
__device__ __forceinline__ void normed8(const T* row, const T* w, int c,
                                        int size, float inv, float (&o)[8]) {
  head8<T, VEC>(row, c, size, o);
  if (w) {
    float wv[8];
    head8<T, VEC>(w, c, size, wv);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = o[j] * inv * wv[j];
  }
}

template <typename T, bool VEC>
__device__ __forceinline__ float square_sum(const T* p, int n) {
  float s = 0.0f;
  if constexpr (VEC) {
    for (int i = threadIdx.x * 8; i < n; i += GR_BLOCK * 8) {
      float v[8];
      load8(p + i, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) s += v[j] * v[j];
    }
  } else {
    for (int i = threadIdx.x; i < n; i += GR_BLOCK)
      s += (float)p[i] * (float)p[i];
  }
  return s;
}

// One block per token: q out [N, H, dimp]; the first `direct` tokens' keys and
// values go to their pages, the others only leave their keys' inverse rms.
template <typename T, bool VEC>
__global__ __launch_bounds__(GR_BLOCK) void grouped_append_kernel(
    const GroupedRowArgs a, T* __restrict__ q, float* __restrict__ kinv,
    const int* __restrict__ tok_pos, const int* __restrict__ tok_entry,
    const int* __restrict__ pages, int P, int direct) {
  __shared__ float scratch[2][GR_BLOCK / WAVE];
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const T* yq = (const T*)a.y + t * a.ystride;
  const T* yk = yq + (long)a.H * a.D;
  const T* yv = yk + (long)a.G * a.D;
  const T* wq = (const T*)a.wq;
  const T* wk = (const T*)a.wk;

  float sq = wq ? square_sum<T, VEC>(yq, a.H * a.D) : 0.0f;
  float sk = wk ? square_sum<T, VEC>(yk, a.G * a.D) : 0.0f;
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if (tid % WAVE == 0) {
    scratch[0][tid / WAVE] = sq;
    scratch[1][tid / WAVE] = sk;
  }
  __syncthreads();
  sq = sk = 0.0f;
#pragma unroll
  for (int w = 0; w < GR_BLOCK / WAVE; ++w) {
    sq += scratch[0][w];
    sk += scratch[1][w];
  }
  const float qi = 1.0f / sqrtf(sq / (float)(a.H * a.D) + a.eps);
  const float ki = 1.0f / sqrtf(sk / (float)(a.G * a.D) + a.eps);
  if (tid == 0) kinv[t] = ki;

  const int nc = a.dimp / 8;
  T* qo = q + t * a.H * a.dimp;
  for (int i = tid; i < a.H * nc; i += GR_BLOCK) {
    const int h = i / nc, c = (i - h * nc) * 8;
    float v[8];
    normed8<T, VEC>(yq + h * a.D, wq ? wq + h * a.D : nullptr, c, a.D, qi, v);
    store8(qo + (long)i * 8, v);
  }
  if (t >= direct) return;

  const int pos = tok_pos[t], r = pos % RG_PAGE;
  const long page = pages[(long)tok_entry[t] * P + pos / RG_PAGE];
  const long PW = (long)RG_PAGE * (a.dimp + a.vdp);
  T* base = (T*)a.pool + page * a.G * PW;
  for (int i = tid; i < a.G * nc; i += GR_BLOCK) {
    const int g = i / nc, c = (i - g * nc) * 8;
    float v[8];
    normed8<T, VEC>(yk + g * a.D, wk ? wk + g * a.D : nullptr, c, a.D, ki, v);
    store8(base + g * PW +
               ((r / 16 * (a.dimp / 32) + c / 32) * 64 + c / 8 % 4 * 16 +
                r % 16) * 8, v);
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

// One block per (page, key/value head): the slots lo .. hi - 1 of a page from
// tokens t + slot; later slots become zero, earlier ones stay.
//   fills[i] = (page, t, lo, hi)
template <typename T, bool VEC>
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
  const T* wk = a.wk ? (const T*)a.wk + g * a.D : nullptr;
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
    float v[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    if (s < hi)
      normed8<T, VEC>(y + (t + s) * a.ystride + koff, wk, c, a.D,
                      wk ? kinv[t + s] : 1.0f, v);
    store8(base + (long)i * 8, v);
  }

  base += RG_PAGE * a.dimp;
  const T* first = (const T*)a.first;
  const float lam = first ? (float)((const T*)a.vmix)[0] : 0.0f;
  for (int d0 = 0; d0 < a.vdp; d0 += 64) {
    if (d0) __syncthreads();
    for (int i = tid; i < RG_PAGE * 8; i += GR_BLOCK) {
      const int s = i / 8, c = d0 + i % 8 * 8;
      float v[8] = {0, 0, 0, 0, 0, 0, 0, 0};
      if (s >= lo && s < hi) {
        head8<T, VEC>(y + (t + s) * a.ystride + voff, c, a.V, v);
        if (first) {
          float u[8];
          head8<T, VEC>(first + (t + s) * a.fstride + (long)g * a.V, c, a.V, u);
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = (1.0f - lam) * v[j] + lam * u[j];
        }
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
      float v[8];
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
#define GR_GO(T, VEC)                                        \
  grouped_append_kernel<T, VEC><<<grid, block, 0, stream>>>( \
      *a, (T*)q, kinv, tok_pos, tok_entry, pages, P, direct)
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
#define GR_GO(T, VEC) \
  grouped_fill_kernel<T, VEC><<<grid, block, 0, stream>>>(*a, kinv, fills)
  if (f32) {
    if (a->vec) GR_GO(float, true);
    else GR_GO(float, false);
  } else {
    if (a->vec) GR_GO(__bf16, true);
    else GR_GO(__bf16, false);
  }
#undef GR_GO
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
    float v[8];
    load8(xr + c, v);
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

// limit * tanh(z * scale / limit)
template <typename T>
__global__ __launch_bounds__(GR_BLOCK) void cap_logits_kernel(
    const T* __restrict__ z, float* __restrict__ o, long n, float scale,
    float limit) {
  const long step = (long)gridDim.x * GR_BLOCK;
  for (long i = (long)blockIdx.x * GR_BLOCK + threadIdx.x; i < n; i += step)
    o[i] = limit * tanhf((float)z[i] * scale / limit);
}

extern "C" void launch_cap_logits(const void* z, float* o, long n, float scale,
                                  float limit, bool f32, hipStream_t stream) {
  const long want = (n + GR_BLOCK - 1) / GR_BLOCK;
  dim3 grid((unsigned)(want < 8192 ? want : 8192)), block(GR_BLOCK);
  if (f32)
    cap_logits_kernel<float><<<grid, block, 0, stream>>>((const float*)z, o, n,
                                                         scale, limit);
  else
    cap_logits_kernel<__bf16><<<grid, block, 0, stream>>>((const __bf16*)z, o,
                                                          n, scale, limit);
}
