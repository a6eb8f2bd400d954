// Causal convolutions over time with their histories in slots, alone and fused
// with the norm before them, and the selective scan.
//
// A request at position 0 starts from zeros whatever its slot holds.
#include "ragged_recurrent.h"

#define RC_BLOCK 256
#define RC_TT 8        // tokens per block of a long portion
#define RC_CHUNK 64    // tokens per entry of `chunks`
#define RC_SUB (RC_CHUNK / RC_TT)

// N elements as they lie in memory
template <typename T, int N>
struct Raw {
  typedef T Vec __attribute__((ext_vector_type(N)));
  Vec v;
  __device__ __forceinline__ void load(const T* p) {
    v = *reinterpret_cast<const Vec*>(p);
  }
  __device__ __forceinline__ void store(T* p) const {
    *reinterpret_cast<Vec*>(p) = v;
  }
  __device__ __forceinline__ void clear() {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = (T)0.0f;
  }
  __device__ __forceinline__ float at(int i) const { return (float)v[i]; }
  __device__ __forceinline__ void set(int i, float x) { v[i] = (T)x; }
};
template <typename T>
struct Raw<T, 1> {
  T v;
  __device__ __forceinline__ void load(const T* p) { v = *p; }
  __device__ __forceinline__ void store(T* p) const { *p = v; }
  __device__ __forceinline__ void clear() { v = (T)0.0f; }
  __device__ __forceinline__ float at(int) const { return (float)v; }
  __device__ __forceinline__ void set(int, float x) { v = (T)x; }
};

template <typename T>
__device__ __forceinline__ float silu_of(float z);
template <>
__device__ __forceinline__ float silu_of<float>(float z) {
  return silu_f(z);
}
template <>
__device__ __forceinline__ float silu_of<__bf16>(float z) {
  return z * __builtin_amdgcn_rcpf(
                 1.0f + __builtin_amdgcn_exp2f(-1.44269504088896340736f * z));
}

// What one token's convolution gives from the last HT + 1 rows, newest last;
// rows and weights past the real taps are zero.
template <typename T, int V, int HT>
__device__ __forceinline__ Raw<T, V> convolved(const Raw<T, V>* rows,
                                               const Raw<T, V> (&w)[HT + 1],
                                               const Raw<T, V>& bias,
                                               const ConvArgs& a) {
  Raw<T, V> o;
#pragma unroll
  for (int i = 0; i < V; ++i) {
    float s = bias.at(i);
#pragma unroll
    for (int j = 0; j <= HT; ++j) s += w[j].at(i) * rows[j].at(i);
    if (a.silu) s = silu_of<T>(s);
    if (a.add) s += rows[HT].at(i);
    o.set(i, s);
  }
  return o;
}

template <typename T, int V, int HT>
__device__ __forceinline__ void load_taps(const ConvArgs& a, int c,
                                          Raw<T, V> (&w)[HT + 1],
                                          Raw<T, V>& bias) {
  const int pad = HT + 1 - a.taps;  // the newest tap is w[HT]
#pragma unroll
  for (int j = 0; j <= HT; ++j) {
    w[j].clear();
    if (j >= pad) w[j].load((const T*)a.w + (long)(j - pad) * a.C + c);
  }
  bias.clear();
  if (a.bias) bias.load((const T*)a.bias + c);
}

// Portions of up to 16 tokens: a thread walks one request's tokens for V
// channels.  grid (requests, channel groups)
template <typename T, int V, int HT>
__global__ __launch_bounds__(RC_BLOCK) void conv_short_kernel(const ConvArgs a) {
  const int e = blockIdx.x;
  const int c = (blockIdx.y * RC_BLOCK + threadIdx.x) * V;
  if (c >= a.Cp) return;
  const int t0 = a.cu[e], n = a.cu[e + 1] - t0;
  T* out = (T*)a.out + (long)t0 * a.Cp + c;
  if (c >= a.C) {
    Raw<T, V> none;
    none.clear();
    for (int t = 0; t < n; ++t) none.store(out + (long)t * a.Cp);
    return;
  }
  const bool fresh = a.pos0[e] == 0;
  const int hist = a.taps - 1;
  T* hp = (T*)a.hist + (long)a.slots[e] * hist * a.C + c;
  Raw<T, V> w[HT + 1], bias, rows[HT + 1];
  load_taps<T, V, HT>(a, c, w, bias);
#pragma unroll
  for (int j = 0; j < HT; ++j) {
    rows[j].clear();
    if (j >= HT - hist && !fresh) rows[j].load(hp + (long)(j - HT + hist) * a.C);
  }
  const T* h = (const T*)a.h + (long)(t0 - a.h_base) * a.hstride + c;
  for (int t = 0; t < n; ++t) {
    rows[HT].load(h + (long)t * a.hstride);
    convolved<T, V, HT>(rows, w, bias, a).store(out + (long)t * a.Cp);
#pragma unroll
    for (int j = 0; j < HT; ++j) rows[j] = rows[j + 1];
  }
#pragma unroll
  for (int j = 0; j < HT; ++j)
    if (j >= HT - hist) rows[j].store(hp + (long)(j - HT + hist) * a.C);
}

// Long portions: RC_TT tokens by V channels a thread, all rows asked for first.
// grid (chunks * RC_SUB, channel groups)
template <typename T, int V, int HT>
__global__ __launch_bounds__(RC_BLOCK) void conv_long_kernel(const ConvArgs a) {
  const int chunk = blockIdx.x / RC_SUB, sub = blockIdx.x % RC_SUB;
  const int t0 = a.chunks[2 * chunk] + sub * RC_TT;
  const int len = min(RC_TT, a.chunks[2 * chunk + 1] - sub * RC_TT);
  const int c = (blockIdx.y * RC_BLOCK + threadIdx.x) * V;
  if (len <= 0 || c >= a.Cp) return;
  T* out = (T*)a.out + (long)t0 * a.Cp + c;
  if (c >= a.C) {
    Raw<T, V> none;
    none.clear();
    for (int t = 0; t < len; ++t) none.store(out + (long)t * a.Cp);
    return;
  }
  const int e = a.tok_entry[t0];
  const int rel = t0 - a.cu[e];  // place within the portion
  const bool fresh = a.pos0[e] == 0;
  const int hist = a.taps - 1;
  const T* hp = (const T*)a.hist + (long)a.slots[e] * hist * a.C + c;
  const T* h = (const T*)a.h + (long)(t0 - a.h_base) * a.hstride + c;
  Raw<T, V> w[HT + 1], bias, rows[HT + RC_TT];
#pragma unroll
  for (int j = 0; j < HT + RC_TT; ++j) {
    const int t = j - HT;
    if (t >= 0) {
      // tokens past the end repeat the last one and are not stored
      rows[j].load(h + (long)min(t, len - 1) * a.hstride);
    } else {
      rows[j].clear();
      if (t >= -hist) {
        if (rel + t >= 0)
          rows[j].load(h + (long)t * a.hstride);
        else if (!fresh)
          rows[j].load(hp + (long)(hist + rel + t) * a.C);
      }
    }
  }
  load_taps<T, V, HT>(a, c, w, bias);
#pragma unroll
  for (int t = 0; t < RC_TT; ++t)
    if (t < len)
      convolved<T, V, HT>(rows + t, w, bias, a).store(out + (long)t * a.Cp);
}

// The last inputs of long portions; runs after the convolution has read the
// ones before.  grid (long requests, channel groups)
template <typename T>
__global__ __launch_bounds__(RC_BLOCK) void conv_tail_kernel(const ConvArgs a) {
  const int e = a.n_short + blockIdx.x;
  const int c = blockIdx.y * RC_BLOCK + threadIdx.x;
  if (c >= a.C) return;
  const int t0 = a.cu[e], n = a.cu[e + 1] - t0;
  const bool fresh = a.pos0[e] == 0;
  const int hist = a.taps - 1;
  T* hp = (T*)a.hist + (long)a.slots[e] * hist * a.C + c;
  for (int j = 0; j < hist; ++j) {  // ascending: reads stay ahead of writes
    const int s = n - hist + j;
    T v = (T)0.0f;
    if (s >= 0)
      v = ((const T*)a.h)[(long)(t0 - a.h_base + s) * a.hstride + c];
    else if (!fresh)
      v = hp[(long)(hist + s) * a.C];
    hp[(long)j * a.C] = v;
  }
}

#define RC_TAPS(T, V, KERNEL, GRID)                                   \
  do {                                                                \
    if (a->taps <= 4)                                                 \
      KERNEL<T, V, 3><<<GRID, dim3(RC_BLOCK), 0, stream>>>(*a);       \
    else                                                              \
      KERNEL<T, V, RC_MAXTAPS - 1><<<GRID, dim3(RC_BLOCK), 0, stream>>>(*a); \
  } while (0)

static dim3 conv_grid(int x, int Cp, int v) {
  const int per = RC_BLOCK * v;
  return dim3((unsigned)x, (unsigned)((Cp + per - 1) / per));
}

extern "C" void launch_conv_short(const ConvArgs* a, bool f32,
                                  hipStream_t stream) {
#define RC_GO(T, V) \
  RC_TAPS(T, V, conv_short_kernel, conv_grid(a->n_short, a->Cp, V))
  if (f32) {
    if (a->vec) RC_GO(float, 4);
    else RC_GO(float, 1);
  } else {
    if (a->vec) RC_GO(__bf16, 8);
    else RC_GO(__bf16, 1);
  }
#undef RC_GO
}

extern "C" void launch_conv_long(const ConvArgs* a, bool f32,
                                 hipStream_t stream) {
#define RC_GO(T, V) \
  RC_TAPS(T, V, conv_long_kernel, conv_grid(a->n_chunks * RC_SUB, a->Cp, V))
  if (f32) {
    if (a->vec) RC_GO(float, 4);
    else RC_GO(float, 1);
  } else {
    if (a->vec) RC_GO(__bf16, 8);
    else RC_GO(__bf16, 1);
  }
#undef RC_GO
  if (a->taps < 2) return;
  const dim3 grid = conv_grid(a->n_long, a->C, 1);
  if (f32)
    conv_tail_kernel<float><<<grid, dim3(RC_BLOCK), 0, stream>>>(*a);
  else
    conv_tail_kernel<__bf16><<<grid, dim3(RC_BLOCK), 0, stream>>>(*a);
}

// ---------------------------------------------------------------------------
// A sublayer boundary of short portions in one kernel, one block per request:
//   x += y, or rms(y) * w_post;  h = rms(x) * g;  out = h + conv(h)
// A thread keeps NR groups of four columns and their history in registers.
// ---------------------------------------------------------------------------

template <typename T, int NT, int NR, int HT>
__global__ __launch_bounds__(NT) void norm_conv_short_kernel(
    const NormConvArgs a) {
  __shared__ float scratch[NT / WAVE];
  const int e = blockIdx.x;
  const int t0 = a.cu[e], n = a.cu[e + 1] - t0;
  const bool fresh = a.pos0[e] == 0;
  const int W = a.W, hist = a.taps - 1, pad = HT - hist;
  const T* w = (const T*)a.w;
  T* hp = (T*)a.hist + (long)a.slots[e] * hist * W;
  const float g = (float)((const T*)a.g)[0];
  Raw<T, 4> rows[NR][HT + 1];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int c = (i * NT + threadIdx.x) * 4;
#pragma unroll
    for (int j = 0; j < HT; ++j) {
      rows[i][j].clear();
      if (j >= pad && !fresh && c < W) rows[i][j].load(hp + (long)(j - pad) * W + c);
    }
  }
  for (int t = 0; t < n; ++t) {
    float* xr = a.x + (long)(t0 + t) * W;
    f32x4 xv[NR], yv[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int c = (i * NT + threadIdx.x) * 4;
      xv[i] = yv[i] = f32x4{0, 0, 0, 0};
      if (c < W) {
        xv[i] = load4(xr + c);
        if (a.y) yv[i] = load4((const T*)a.y + (long)(t0 + t) * a.ystride + c);
      }
    }
    if (a.y) {
      float inv = 1.0f;
      if (a.w_post) {
        float ss = 0.0f;
#pragma unroll
        for (int i = 0; i < NR; ++i)
#pragma unroll
          for (int k = 0; k < 4; ++k) ss += yv[i][k] * yv[i][k];
        inv = 1.0f / sqrtf(block_sum<NT>(ss, scratch) / (float)W + a.eps);
      }
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int c = (i * NT + threadIdx.x) * 4;
        if (c >= W) continue;
        f32x4 p = {1, 1, 1, 1};
        if (a.w_post) p = load4((const T*)a.w_post + c);
#pragma unroll
        for (int k = 0; k < 4; ++k) xv[i][k] += yv[i][k] * inv * p[k];
        store4(xr + c, xv[i]);
      }
    }
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < NR; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k) ss += xv[i][k] * xv[i][k];
    const float inv =
        1.0f / sqrtf(block_sum<NT>(ss, scratch) / (float)W + a.eps);
    T* out = (T*)a.out + (long)(t0 + t) * a.Wp;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int c = (i * NT + threadIdx.x) * 4;
      if (c >= W) continue;
      f32x4 o = {0, 0, 0, 0};
#pragma unroll
      for (int k = 0; k < 4; ++k) rows[i][HT].set(k, xv[i][k] * inv * g);
#pragma unroll
      for (int j = 0; j <= HT; ++j) {
        if (j < pad) continue;
        const f32x4 wv = load4(w + (long)(j - pad) * W + c);
#pragma unroll
        for (int k = 0; k < 4; ++k) o[k] += wv[k] * rows[i][j].at(k);
      }
#pragma unroll
      for (int k = 0; k < 4; ++k) o[k] += rows[i][HT].at(k);
      store4(out + c, o);
#pragma unroll
      for (int j = 0; j < HT; ++j) rows[i][j] = rows[i][j + 1];
    }
    for (int c = W + threadIdx.x; c < a.Wp; c += NT) out[c] = (T)0.0f;
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int c = (i * NT + threadIdx.x) * 4;
    if (c >= W) continue;
#pragma unroll
    for (int j = 0; j < HT; ++j)
      if (j >= pad) rows[i][j].store(hp + (long)(j - pad) * W + c);
  }
}

// widest row of the kernel
extern "C" int norm_conv_width() { return 1024 * 4 * 2; }

template <typename T>
static void norm_conv_t(const NormConvArgs* a, hipStream_t stream) {
#define NC_GO(NT, NR)                                                      \
  do {                                                                     \
    if (a->taps <= 4)                                                      \
      norm_conv_short_kernel<T, NT, NR, 3>                                 \
          <<<dim3((unsigned)a->n_short), dim3(NT), 0, stream>>>(*a);       \
    else                                                                   \
      norm_conv_short_kernel<T, NT, NR, RC_MAXTAPS - 1>                    \
          <<<dim3((unsigned)a->n_short), dim3(NT), 0, stream>>>(*a);       \
  } while (0)
  if (a->W <= 1024) NC_GO(256, 1);
  else if (a->W <= 2048) NC_GO(512, 1);
  else if (a->W <= 4096) NC_GO(1024, 1);
  else NC_GO(1024, 2);
#undef NC_GO
}

extern "C" void launch_norm_conv_short(const NormConvArgs* a, bool f32,
                                       hipStream_t stream) {
  if (f32) norm_conv_t<float>(a, stream);
  else norm_conv_t<__bf16>(a, stream);
}

// ---------------------------------------------------------------------------
// Selective scan.  Per channel c and state n, with d = softplus(dt + bias):
//   S <- exp(d A) S + d x B;  y = sum_n S C + D x;  out = y silu(z)
// A wave takes 64 / PARTS neighbouring channels; PARTS lanes share a channel,
// NS states each.  Where a lane has all states of its channel, B and C are the
// same for the whole wave and are read as scalars.
//
// Long portions are cut into spans.  Unless every portion is a single span, a
// first pass finds what each span adds to a zero state and the sum of its
// steps (the decay over a span is exp(A sum)), a second one carries the states
// from span to span, and the last one runs all spans from their first states.
// ---------------------------------------------------------------------------

// exponent of a decay: bf16 works in powers of two, float in powers of e
template <typename T>
__device__ __forceinline__ constexpr float decay_unit() {
  return sizeof(T) == 2 ? 1.44269504088896340736f : 1.0f;
}
template <typename T>
__device__ __forceinline__ float decay_exp(float x);
template <>
__device__ __forceinline__ float decay_exp<__bf16>(float x) {
  return __builtin_amdgcn_exp2f(x);
}
template <>
__device__ __forceinline__ float decay_exp<float>(float x) {
  return expf(x);
}

typedef const __attribute__((address_space(4))) unsigned* ScalarWords;

template <int NS>
__device__ __forceinline__ void load_uniform(const __bf16* p, float (&o)[NS]) {
  ScalarWords s = (ScalarWords)(uintptr_t)p;
#pragma unroll
  for (int i = 0; i < NS / 2; ++i) {
    const unsigned u = s[i];
    o[2 * i] = __uint_as_float(u << 16);
    o[2 * i + 1] = __uint_as_float(u & 0xffff0000u);
  }
}
template <int NS>
__device__ __forceinline__ void load_uniform(const float* p, float (&o)[NS]) {
  ScalarWords s = (ScalarWords)(uintptr_t)p;
#pragma unroll
  for (int i = 0; i < NS; ++i) o[i] = __uint_as_float(s[i]);
}

// NS coefficients of one token: of the whole wave, or of a lane's part
template <typename T, int NS, int PARTS>
__device__ __forceinline__ void load_coeffs(const T* p, int part,
                                            float (&o)[NS]) {
  if constexpr (PARTS == 1) {
    load_uniform<NS>(p, o);
  } else {
#pragma unroll
    for (int i = 0; i < NS; i += 8) {
      Raw<T, 8> r;
      r.load(p + part * NS + i);
#pragma unroll
      for (int j = 0; j < 8; ++j) o[i + j] = r.at(j);
    }
  }
}

template <int PARTS>
__device__ __forceinline__ float sum_parts(float y) {
#pragma unroll
  for (int o = WAVE / PARTS; o < WAVE; o <<= 1) y += __shfl_xor(y, o, WAVE);
  return y;
}

#define SS_BLOCK 256
#define SS_AHEAD 4  // tokens whose inputs are asked for together

template <typename T, int NS, int PARTS>
struct ScanLane {
  int c, part;
  bool live;
  float A[NS], S[NS], bias, D;

  __device__ __forceinline__ ScanLane(const ScanArgs& a) {
    const int lane = threadIdx.x & (WAVE - 1);
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    constexpr int CPW = WAVE / PARTS;
    c = (blockIdx.x * (SS_BLOCK / WAVE) + wid) * CPW + lane % CPW;
    part = lane / CPW;
    live = c < a.C;
    c = min(c, a.C - 1);  // lanes past the end repeat the last channel
#pragma unroll
    for (int i = 0; i < NS; ++i)
      A[i] = a.A[(long)(part * NS + i) * a.C + c] * decay_unit<T>();
    bias = a.bias[c];
    D = a.D[c];
  }
  // [states padded, C] from `p`
  __device__ __forceinline__ void load(const ScanArgs& a, const float* p,
                                       bool zero) {
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const float v = p[(long)(part * NS + i) * a.C + c];
      S[i] = zero ? 0.0f : v;
    }
  }
  __device__ __forceinline__ void save(const ScanArgs& a, float* p) const {
    if (!live) return;
#pragma unroll
    for (int i = 0; i < NS; ++i) p[(long)(part * NS + i) * a.C + c] = S[i];
  }
  // n tokens from t0 on; returns the sum of their steps
  template <bool OUT>
  __device__ __forceinline__ float walk(const ScanArgs& a, int t0, int n) {
    const T* xp = (const T*)a.x + (long)t0 * a.xs + c;
    const T* zp = (const T*)a.z + (long)t0 * a.zs + c;
    const T* dp = (const T*)a.dt + (long)t0 * a.ds + c;
    const T* bp = (const T*)a.bc + (long)t0 * a.bs;
    T* op = (T*)a.out + (long)t0 * a.C + c;
    float total = 0.0f;
    T xr[SS_AHEAD], zr[SS_AHEAD], dr[SS_AHEAD];
    auto ask = [&](int t) {
#pragma unroll
      for (int u = 0; u < SS_AHEAD; ++u) {
        const int s = min(t + u, n - 1);
        xr[u] = xp[(long)s * a.xs];
        dr[u] = dp[(long)s * a.ds];
        if constexpr (OUT) zr[u] = zp[(long)s * a.zs];
      }
    };
    ask(0);
    for (int t = 0; t < n; t += SS_AHEAD) {
      float x[SS_AHEAD], d[SS_AHEAD], z[SS_AHEAD];
#pragma unroll
      for (int u = 0; u < SS_AHEAD; ++u) {
        x[u] = (float)xr[u];
        d[u] = (float)dr[u] + bias;
        z[u] = OUT ? (float)zr[u] : 0.0f;
      }
      if (t + SS_AHEAD < n) ask(t + SS_AHEAD);
#pragma unroll
      for (int u = 0; u < SS_AHEAD; ++u) {
        if (t + u >= n) break;
        const float step = softplus_of<T>(d[u]);
        const float in = step * x[u];
        float B[NS], C[NS];
        load_coeffs<T, NS, PARTS>(bp + (long)(t + u) * a.bs + a.b0, part, B);
        if constexpr (OUT)
          load_coeffs<T, NS, PARTS>(bp + (long)(t + u) * a.bs + a.c0, part, C);
        float y = 0.0f;
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          S[i] = decay_exp<T>(step * A[i]) * S[i] + B[i] * in;
          if constexpr (OUT) y += S[i] * C[i];
        }
        total += step;
        if constexpr (OUT) {
          y = sum_parts<PARTS>(y) + D * x[u];
          if (live && part == 0)
            op[(long)(t + u) * a.C] = (T)(y * silu_of<T>(z[u]));
        }
      }
    }
    return total;
  }
};

// grid (channel groups, requests)
template <typename T, int NS, int PARTS>
__global__ __launch_bounds__(SS_BLOCK) void scan_short_kernel(
    const ScanArgs a) {
  const int e = blockIdx.y;
  const int t0 = a.cu[e], n = a.cu[e + 1] - t0;
  float* state = a.state + (long)a.slots[e] * a.Np * a.C;
  ScanLane<T, NS, PARTS> s(a);
  s.load(a, state, a.pos0[e] == 0);
  s.template walk<true>(a, t0, n);
  s.save(a, state);
}

// grid (channel groups, spans); first: what the span adds to a zero state
template <typename T, int NS, int PARTS, bool FIRST>
__global__ __launch_bounds__(SS_BLOCK) void scan_span_kernel(const ScanArgs a) {
  const int j = blockIdx.y;
  const int t0 = a.spans[4 * j], n = a.spans[4 * j + 1];
  const int e = a.spans[4 * j + 2];
  const bool ends = a.spans[4 * j + 3] != 0;
  if (FIRST && ends) return;
  ScanLane<T, NS, PARTS> s(a);
  const long at = (long)j * a.Np * a.C;
  if constexpr (FIRST) {
#pragma unroll
    for (int i = 0; i < NS; ++i) s.S[i] = 0.0f;
    const float total = s.template walk<false>(a, t0, n);
    s.save(a, a.ends + at);
    if (s.live && s.part == 0) a.sums[(long)j * a.C + s.c] = total;
  } else {
    float* state = a.state + (long)a.slots[e] * a.Np * a.C;
    // with inits, a portion's first span must not read the state, which its
    // last span may have written already
    if (a.inits) s.load(a, a.inits + at, false);
    else s.load(a, state, a.pos0[e] == 0);
    s.template walk<true>(a, t0, n);
    if (ends) s.save(a, state);
  }
}

// grid (channel groups, padded states, long requests)
template <typename T>
__global__ __launch_bounds__(SS_BLOCK) void scan_carry_kernel(
    const float* __restrict__ ends, const float* __restrict__ sums,
    const float* __restrict__ state, const float* __restrict__ A,
    float* __restrict__ inits, const int* __restrict__ span_cu,
    const int* __restrict__ pos0, const int* __restrict__ slots, int n_short,
    int C, int Np) {
  const int c = blockIdx.x * SS_BLOCK + threadIdx.x;
  if (c >= C) return;
  const long n = blockIdx.y;
  const int e = n_short + blockIdx.z;
  const float k = A[n * C + c] * decay_unit<T>();
  float S = 0.0f;
  if (pos0[e] != 0) S = state[((long)slots[e] * Np + n) * C + c];
  const int j1 = span_cu[blockIdx.z + 1];
  int j = span_cu[blockIdx.z];
  const long step = (long)Np * C;
  const float* ep = ends + j * step + n * C + c;
  const float* sp = sums + (long)j * C + c;
  float* ip = inits + j * step + n * C + c;
  constexpr int U = 8;
  for (; j < j1; j += U) {
    float ev[U], sv[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      // a portion's last span has no end of its own; nothing follows it
      const int k2 = max(0, min(u, j1 - 2 - j));
      ev[u] = j1 - 2 >= j ? ep[k2 * step] : 0.0f;
      sv[u] = j1 - 2 >= j ? sp[(long)k2 * C] : 0.0f;
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (j + u < j1) {
        ip[u * step] = S;
        S = decay_exp<T>(k * sv[u]) * S + ev[u];
      }
    }
    ep += U * step;
    sp += (long)U * C;
    ip += U * step;
  }
}

template <typename T, int NS, int PARTS>
static void scan_go(const ScanArgs* a, bool is_short, hipStream_t stream) {
  const int per = SS_BLOCK / PARTS;
  const unsigned groups = (unsigned)((a->C + per - 1) / per);
  if (is_short) {
    scan_short_kernel<T, NS, PARTS>
        <<<dim3(groups, (unsigned)a->n_short), dim3(SS_BLOCK), 0, stream>>>(*a);
    return;
  }
  const dim3 grid(groups, (unsigned)a->n_spans);
  if (a->inits) {
    scan_span_kernel<T, NS, PARTS, true>
        <<<grid, dim3(SS_BLOCK), 0, stream>>>(*a);
    scan_carry_kernel<T>
        <<<dim3((unsigned)((a->C + SS_BLOCK - 1) / SS_BLOCK), (unsigned)a->Np,
                (unsigned)a->n_long),
           dim3(SS_BLOCK), 0, stream>>>(a->ends, a->sums, a->state, a->A,
                                        a->inits, a->span_cu, a->pos0,
                                        a->slots, a->n_short, a->C, a->Np);
  }
  scan_span_kernel<T, NS, PARTS, false>
      <<<grid, dim3(SS_BLOCK), 0, stream>>>(*a);
}

template <typename T>
static bool scan_t(const ScanArgs* a, int part, int parts, bool is_short,
                   hipStream_t stream) {
#define SS_CASE(NS, P)                              \
  case NS * 100 + P:                                \
    scan_go<T, NS, P>(a, is_short, stream);         \
    return true
  switch (part * 100 + parts) {
    SS_CASE(8, 1); SS_CASE(16, 1); SS_CASE(32, 1); SS_CASE(32, 2);
    SS_CASE(32, 4); SS_CASE(32, 8); SS_CASE(32, 16);
    default: return false;
  }
#undef SS_CASE
}

extern "C" bool scan_has(int part, int parts) {
  return parts == 1 ? part == 8 || part == 16 || part == 32
                    : part == 32 && (parts == 2 || parts == 4 || parts == 8 ||
                                     parts == 16);
}

extern "C" void launch_scan(const ScanArgs* a, int part, int parts,
                            bool is_short, bool f32, hipStream_t stream) {
  if (f32) scan_t<float>(a, part, parts, is_short, stream);
  else scan_t<__bf16>(a, part, parts, is_short, stream);
}
