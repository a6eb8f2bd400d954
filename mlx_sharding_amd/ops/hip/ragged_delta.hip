// Gated delta rule over a ragged batch, state in slots.
//
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// with q, k, v behind a short causal convolution and silu, q and k unit
// vectors, and one decay g per head, or one per head and key channel (rows of
// S).  The state [D, V] and everything that enters the recurrence are fp32 in
// either element type.
//
//  * short portions (decoding): one kernel does convolution, norms, gates,
//    recurrence, output norm and gate; the state lives in registers.
//  * long portions: chunks of 64 tokens.  With G the running log decay of the
//    chunk, S0 the state before it, and
//        L[i,j] = beta_i exp(G_i - G_j) k_i.k_j   (j < i)
//        A[i,j] =        exp(G_i - G_j) q_i.k_j   (j <= i)
//    the writes are U = (I + L)^-1 diag(beta) (V - diag(exp G) K S0), the
//    outputs O = diag(exp G) Q S0 + A U, and the next state
//    exp(G_last) S0 + K^T diag(exp(G_last - G)) U.  One kernel makes
//    (I + L)^-1 diag(beta) and A of all chunks at once, a second walks the
//    chunks of a (request, head, 16 value columns).  All products run on the
//    fp32 matrix cores.
//  * decays per channel: exp(G) is a vector then, and L and A sum
//    k_i[d] k_j[d] exp(G_i[d] - G_j[d]) over channels.  Between the tokens of two
//    neighbouring blocks, with the second block's begin as reference, that is a
//    product of two factors, the decay from there to i and the one from j to
//    there; both are running products of decays of at most 1, so nothing
//    overflows and no difference of large logarithms is taken.  Every pair of a
//    chunk lies in two such blocks of 1, 2, 4, 8, 16 or more tokens.
//
// A request at position 0 starts from a zero state whatever its slot holds.
#include "ragged_common.h"

#define DR_CHUNK 64
#define DR_MAXTAPS 8
#define DR_SHORT 16  // most tokens of a short portion

struct DeltaDims {
  int KH, H, D, V, taps;
  int qc, kc, vc, gc, ac, bc;  // column offsets in a projection row; gate (gc)
  long ystride, zstride;       // and decay (ac) in rows z of their own
  bool channels;               // decays per head and key channel
  bool sigmoid;                // the output gate; else silu
};

__device__ __forceinline__ float log_decay(float a, float A_log, float dt) {
  return -expf(A_log) * softplus_f(a + dt);
}

// the factor of one step
template <typename T>
__device__ __forceinline__ float decay_of(float a, float rate, float dt);
template <>
__device__ __forceinline__ float decay_of<float>(float a, float rate, float dt) {
  return expf(-rate * softplus_of<float>(a + dt));
}
template <>
__device__ __forceinline__ float decay_of<__bf16>(float a, float rate, float dt) {
  return __builtin_amdgcn_exp2f(-1.44269504088896340736f * rate *
                                softplus_of<__bf16>(a + dt));
}

__device__ __forceinline__ float out_gate(float x, bool sigmoid) {
  const float s = sigmoid_f(x);
  return sigmoid ? s : x * s;
}

// ---------------------------------------------------------------------------
// Short portions.  Block = (request, q/k head); its r = H / KH value heads
// follow one another.  Threads: VT along V (power of two), DG groups along D,
// RPT state rows per thread.
// ---------------------------------------------------------------------------

// EXACT: the threads tile the state without a remainder.  CH: decays per channel.
template <typename T, int RPT, int NT, bool EXACT, bool CH>
__global__ __launch_bounds__(NT, RPT <= 32 ? 4 : 2) void delta_short_kernel(
    const T* __restrict__ y, const T* __restrict__ z,
    const T* __restrict__ conv_w,
    const T* __restrict__ A_log, const T* __restrict__ dt_bias,
    const T* __restrict__ norm_w, float* __restrict__ state,
    T* __restrict__ conv_state, T* __restrict__ out,
    const int* __restrict__ cu, const int* __restrict__ pos0,
    const int* __restrict__ slots, DeltaDims dm, int VT, float q_scale,
    float eps) {
  const int e = blockIdx.x;
  const int kh = blockIdx.y;
  const int t0 = cu[e];
  const int n = min(cu[e + 1] - t0, DR_SHORT);
  const bool fresh = pos0[e] == 0;
  const long slot = slots[e];
  const int D = dm.D, V = dm.V;
  const int DG = NT / VT;
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = tid / WAVE;
  const int C = 2 * dm.KH * D + dm.H * V;
  const int hist = dm.taps - 1;

  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* qk = reinterpret_cast<float*>(smem);  // [n][2][D]
  float* kq = qk + (long)n * 2 * D;            // [n]
  float* vb = kq + DR_SHORT;                   // [n][V]
  float* red = vb + (long)n * V;               // [2][DG][VT]
  float* scratch = red + 2 * NT;               // [NT / WAVE]
  float* gd = scratch + NT / WAVE;             // [n][D], decays per channel

  const int v = tid & (VT - 1);
  const int dg = tid / VT;
  const int d0 = dg * RPT;
  const int rep = dm.H / dm.KH;
  // this thread's part of a head's state; asked for as early as possible
  float S[RPT];
  auto load_state = [&](int h) {
    // uniform row base + one lane offset: no address per row and lane
    const float* sp = state + ((slot * dm.H + h) * (long)D) * V;
    const int vc = EXACT ? v : min(v, V - 1);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const float x = EXACT ? sp[d0 * V + v] : sp[min(d0 + i, D - 1) * V + vc];
      S[i] = fresh ? 0.0f : x;
      if (EXACT) sp += V;
    }
  };
  load_state(kh * rep);

  // convolution + silu of channel c (column col of y) for all n tokens
  auto convolve = [&](int c, int col, float* dst, int dstep) {
    float w[DR_MAXTAPS], x[DR_MAXTAPS];
    T* cs = conv_state + (slot * C + c) * hist;
    // taps sit at the end of w/x, so the index of the newest is fixed
    const int pad = DR_MAXTAPS - dm.taps;
#pragma unroll
    for (int j = 0; j < DR_MAXTAPS; ++j) {
      w[j] = j >= pad ? (float)conv_w[(long)c * dm.taps + j - pad] : 0.0f;
      x[j] = (j >= pad && j < DR_MAXTAPS - 1 && !fresh) ? (float)cs[j - pad]
                                                        : 0.0f;
    }
    for (int t = 0; t < n; ++t) {
      x[DR_MAXTAPS - 1] = (float)y[(long)(t0 + t) * dm.ystride + col];
      float a = 0.0f;
#pragma unroll
      for (int j = 0; j < DR_MAXTAPS; ++j) a += w[j] * x[j];
      dst[(long)t * dstep] = silu_f(a);
#pragma unroll
      for (int j = 0; j < DR_MAXTAPS - 1; ++j) x[j] = x[j + 1];
    }
    // x[j] now holds the input one step older than slot j + 1: the last
    // taps - 1 inputs are x[pad .. MAXTAPS - 2]
#pragma unroll
    for (int j = 0; j < DR_MAXTAPS - 1; ++j)
      if (j >= pad) cs[j - pad] = (T)x[j];
  };

  for (int i = tid; i < 2 * D; i += NT) {
    const int which = i / D, d = i - which * D;
    const int c = which * dm.KH * D + kh * D + d;
    convolve(c, (which ? dm.kc : dm.qc) + kh * D + d, qk + i, 2 * D);
  }
  __syncthreads();
  for (int r = wid; r < 2 * n; r += NT / WAVE) {
    float* row = qk + (long)r * D;
    float ss = 0.0f;
    for (int d = lane; d < D; d += WAVE) ss += row[d] * row[d];
    ss = wave_sum(ss);
    const float s = (r & 1 ? 1.0f : q_scale) / sqrtf(ss + 1e-6f);
    for (int d = lane; d < D; d += WAVE) row[d] *= s;
  }
  __syncthreads();
  for (int t = wid; t < n; t += NT / WAVE) {
    float a = 0.0f;
    for (int d = lane; d < D; d += WAVE)
      a += qk[(long)t * 2 * D + d] * qk[(long)t * 2 * D + D + d];
    a = wave_sum(a);
    if (lane == 0) kq[t] = a;
  }

  for (int hh = 0; hh < rep; ++hh) {
    const int h = kh * rep + hh;
    __syncthreads();
    for (int i = tid; i < V; i += NT)
      convolve(2 * dm.KH * D + h * V + i, dm.vc + h * V + i, vb + i, V);
    const float Al = (float)A_log[h], dt = CH ? 0.0f : (float)dt_bias[h];
    if constexpr (CH) {
      const float rate = expf(Al);
      for (int i = tid; i < n * D; i += NT) {
        const int t = i / D, d = i - t * D;
        gd[i] = decay_of<T>((float)z[(t0 + t) * dm.zstride + dm.ac + h * D + d],
                            rate, (float)dt_bias[h * D + d]);
      }
    }
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const T* yt = y + (long)(t0 + t) * dm.ystride;
      const T* zt = z + (long)(t0 + t) * dm.zstride;
      const float g =
          CH ? 1.0f : expf(log_decay((float)zt[dm.ac + h], Al, dt));
      const float beta = sigmoid_f((float)yt[dm.bc + h]);
      const float* qr = qk + (long)t * 2 * D;
      const float* kr = qr + D;
      float sk = 0.0f, sq = 0.0f;
#pragma unroll
      for (int i = 0; i < RPT; ++i)
        if (EXACT || d0 + i < D) {
          if (CH) S[i] *= gd[t * D + d0 + i];
          sk += S[i] * kr[d0 + i];
          sq += S[i] * qr[d0 + i];
        }
      red[dg * VT + v] = sk;
      red[NT + dg * VT + v] = sq;
      __syncthreads();
      sk = 0.0f;
      sq = 0.0f;
      for (int i = 0; i < DG; ++i) {
        sk += red[i * VT + v];
        sq += red[NT + i * VT + v];
      }
      const float vv = v < V ? vb[(long)t * V + v] : 0.0f;
      const float u = beta * (vv - g * sk);
      const float o = g * sq + kq[t] * u;
#pragma unroll
      for (int i = 0; i < RPT; ++i)
        if (EXACT || d0 + i < D) S[i] = g * S[i] + kr[d0 + i] * u;
      const bool mine = dg == 0 && v < V;
      const float ss = block_sum<NT>(mine ? o * o : 0.0f, scratch);
      if (mine) {
        const float gate = out_gate((float)zt[dm.gc + h * V + v], dm.sigmoid);
        out[(long)(t0 + t) * ((long)dm.H * V) + h * V + v] =
            (T)(o / sqrtf(ss / (float)V + eps) * (float)norm_w[v] * gate);
      }
    }
    float* sp = state + ((slot * dm.H + h) * (long)D) * V;
    if (EXACT || v < V) {
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        if (EXACT || d0 + i < D) sp[d0 * V + v] = S[i];
        sp += V;
      }
    }
    if (hh + 1 < rep) load_state(h + 1);
  }
}

static int pow2_at_least(int v) {
  int p = 16;
  while (p < v) p *= 2;
  return p;
}

// state rows per thread, or 0 if the head is too large for the kernel
extern "C" int delta_short_rows(int D, int V, int nt) {
  const int vt = pow2_at_least(V);
  if (vt > nt) return 0;
  const int need = (D + nt / vt - 1) / (nt / vt);
  for (int r : {4, 16, 32, 64, 128})
    if (need <= r) return r;
  return 0;
}

#define DR_NT 512

template <typename T, bool CH>
static void delta_short_t(const void* y, const void* z, const void* conv_w,
                          const void* A_log, const void* dt_bias,
                          const void* norm_w, float* state, void* conv_state,
                          void* out, const int* cu, const int* pos0,
                          const int* slots, const DeltaDims& dm, int n_req,
                          int max_len, float eps, hipStream_t stream) {
  const int vt = pow2_at_least(dm.V);
  const int rpt = delta_short_rows(dm.D, dm.V, DR_NT);
  const size_t smem = ((size_t)max_len * ((CH ? 3 : 2) * dm.D + dm.V) +
                       DR_SHORT + 2 * DR_NT + DR_NT / WAVE) * sizeof(float);
  const float q_scale = 1.0f / sqrtf((float)dm.D);
  dim3 grid((unsigned)n_req, (unsigned)dm.KH), block(DR_NT);
#define DS_ONE(R, X)                                                         \
  do {                                                                       \
    if (smem > 65536)                                                        \
      (void)hipFuncSetAttribute(                                             \
          reinterpret_cast<const void*>(                                     \
              &delta_short_kernel<T, R, DR_NT, X, CH>),                      \
          hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);            \
    delta_short_kernel<T, R, DR_NT, X, CH><<<grid, block, smem, stream>>>(   \
        (const T*)y, (const T*)z, (const T*)conv_w, (const T*)A_log,         \
        (const T*)dt_bias, (const T*)norm_w, state, (T*)conv_state, (T*)out, \
        cu, pos0, slots, dm, vt, q_scale, eps);                              \
  } while (0)
#define DS_GO(R)                                                             \
  do {                                                                       \
    if (dm.V == vt && dm.D == R * (DR_NT / vt))                              \
      DS_ONE(R, true);                                                       \
    else                                                                     \
      DS_ONE(R, false);                                                      \
  } while (0)
  switch (rpt) {
    case 4: DS_GO(4); break;
    case 16: DS_GO(16); break;
    case 32: DS_GO(32); break;
    case 64: DS_GO(64); break;
    case 128: DS_GO(128); break;
    default: break;
  }
#undef DS_GO
#undef DS_ONE
}

extern "C" void launch_delta_short(const void* y, const void* z,
                                   const void* conv_w, const void* A_log,
                                   const void* dt_bias, const void* norm_w,
                                   float* state, void* conv_state, void* out,
                                   const int* cu, const int* pos0,
                                   const int* slots, const DeltaDims* dm,
                                   int n_req, int max_len, float eps, bool f32,
                                   hipStream_t stream) {
#define DS_TYPE(T, CH)                                                        \
  delta_short_t<T, CH>(y, z, conv_w, A_log, dt_bias, norm_w, state,           \
                       conv_state, out, cu, pos0, slots, *dm, n_req, max_len, \
                       eps, stream)
  if (dm->channels) {
    if (f32) DS_TYPE(float, true);
    else DS_TYPE(__bf16, true);
  } else {
    if (f32) DS_TYPE(float, false);
    else DS_TYPE(__bf16, false);
  }
#undef DS_TYPE
}

// ---------------------------------------------------------------------------
// Long portions, step 1: convolution, silu, unit norms, gates.
// q, k -> fp32 [n, KH, Dp] (zero padded), v -> T [n, H, Vp], log decay and
// beta -> fp32 [n, H].  One wave per (16 tokens of a chunk, piece): a piece is
// a q or k head, 64 * CW value channels, or the gates.  A lane keeps its CW
// neighbouring channels' inputs of all 16 tokens and their history in
// registers.  NU: channel groups per lane and q/k head, D <= 64 * CW * NU.
// ---------------------------------------------------------------------------

// CW neighbouring elements at once (1 or 2)
template <typename T, int CW>
struct __attribute__((aligned(CW * sizeof(T)))) Lanes {
  T v[CW];
};

template <typename T, int CW>
__device__ __forceinline__ void load_lanes(const T* p, float (&o)[CW]) {
  const Lanes<T, CW> t = *reinterpret_cast<const Lanes<T, CW>*>(p);
#pragma unroll
  for (int k = 0; k < CW; ++k) o[k] = (float)t.v[k];
}

template <typename T, int CW>
__device__ __forceinline__ void store_lanes(T* p, const float (&o)[CW]) {
  Lanes<T, CW> t;
#pragma unroll
  for (int k = 0; k < CW; ++k) t.v[k] = (T)o[k];
  *reinterpret_cast<Lanes<T, CW>*>(p) = t;
}

#define DC_BLOCK 256
#define DC_TT 16
#define DC_SUB (DR_CHUNK / DC_TT)

template <typename T, int NU, int CW>
__global__ __launch_bounds__(DC_BLOCK) void delta_conv_kernel(
    const T* __restrict__ y, const T* __restrict__ conv_w,
    const T* __restrict__ A_log, const T* __restrict__ dt_bias,
    const T* __restrict__ conv_state, float* __restrict__ qo,
    float* __restrict__ ko, T* __restrict__ vo, float* __restrict__ lg,
    float* __restrict__ bt, const int* __restrict__ cu,
    const int* __restrict__ pos0, const int* __restrict__ slots,
    const int* __restrict__ tok_entry, const int* __restrict__ chunks,
    int tok_base, DeltaDims dm, int Dp, int Vp, float q_scale) {
  const int chunk = blockIdx.x / DC_SUB, sub = blockIdx.x % DC_SUB;
  const int t0 = chunks[2 * chunk] + sub * DC_TT;
  const int len = min(DC_TT, chunks[2 * chunk + 1] - sub * DC_TT);
  const int lane = threadIdx.x & (WAVE - 1);
  const int piece = __builtin_amdgcn_readfirstlane(
      blockIdx.y * (DC_BLOCK / WAVE) + threadIdx.x / WAVE);
  const int D = dm.D, V = dm.V;
  const int n_qk = 2 * dm.KH;
  const int n_v = (dm.H * Vp + WAVE * CW - 1) / (WAVE * CW);
  if (len <= 0 || piece > n_qk + n_v) return;
  const long i0 = t0 - tok_base;          // row among the long tokens
  const int e = tok_entry[t0];
  const int rel = t0 - cu[e];             // place within the portion
  const bool fresh = pos0[e] == 0;
  const int hist = dm.taps - 1;
  const int C = 2 * dm.KH * D + dm.H * V;
  const T* cs = conv_state + (long)slots[e] * C * hist;
  const T* yt = y + (long)t0 * dm.ystride;

  // channels c.. (columns col.. of y): convolved, silu'd values of 16 tokens
  auto convolve = [&](int c, int col, float (&o)[DC_TT][CW]) {
    float x[DC_TT + DR_MAXTAPS - 1][CW], w[DR_MAXTAPS][CW];
#pragma unroll
    for (int k = 0; k < DC_TT + DR_MAXTAPS - 1; ++k) {
      const int t = k - (DR_MAXTAPS - 1);
#pragma unroll
      for (int q = 0; q < CW; ++q) x[k][q] = 0.0f;
      if (t >= 0) {
        // tokens past the end repeat the last one and are not stored
        load_lanes<T, CW>(yt + (long)min(t, len - 1) * dm.ystride + col, x[k]);
      } else if (t >= -hist) {
        if (rel + t >= 0)
          load_lanes<T, CW>(yt + (long)t * dm.ystride + col, x[k]);
        else if (!fresh)
#pragma unroll
          for (int q = 0; q < CW; ++q)
            x[k][q] = (float)cs[(long)(c + q) * hist + hist + rel + t];
      }
    }
    const int pad = DR_MAXTAPS - dm.taps;
#pragma unroll
    for (int j = 0; j < DR_MAXTAPS; ++j)
#pragma unroll
      for (int q = 0; q < CW; ++q)
        w[j][q] = j >= pad ? (float)conv_w[(long)(c + q) * dm.taps + j - pad]
                           : 0.0f;
#pragma unroll
    for (int t = 0; t < DC_TT; ++t)
#pragma unroll
      for (int q = 0; q < CW; ++q) {
        float a = 0.0f;
#pragma unroll
        for (int j = 0; j < DR_MAXTAPS; ++j)
          if (j >= pad) a += w[j][q] * x[t + j][q];
        o[t][q] = silu_f(a);
      }
  };

  if (piece < n_qk) {
    const int which = piece / dm.KH, kh = piece - which * dm.KH;
    float o[NU][DC_TT][CW];
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const int d = (lane + u * WAVE) * CW;
      if (d < D) {
        convolve(which * dm.KH * D + kh * D + d,
                 (which ? dm.kc : dm.qc) + kh * D + d, o[u]);
      } else {
#pragma unroll
        for (int t = 0; t < DC_TT; ++t)
#pragma unroll
          for (int q = 0; q < CW; ++q) o[u][t][q] = 0.0f;
      }
    }
    float* dst = (which ? ko : qo) + (i0 * dm.KH + kh) * Dp;
#pragma unroll
    for (int t = 0; t < DC_TT; ++t) {
      float ss = 0.0f;
#pragma unroll
      for (int u = 0; u < NU; ++u)
#pragma unroll
        for (int q = 0; q < CW; ++q) ss += o[u][t][q] * o[u][t][q];
      ss = wave_sum(ss);
      const float s = (which ? 1.0f : q_scale) / sqrtf(ss + 1e-6f);
      if (t < len) {
#pragma unroll
        for (int u = 0; u < NU; ++u) {
          const int d = (lane + u * WAVE) * CW;
#pragma unroll
          for (int q = 0; q < CW; ++q) o[u][t][q] *= s;
          if (d < Dp)
            store_lanes<float, CW>(dst + (long)t * dm.KH * Dp + d, o[u][t]);
        }
      }
    }
  } else if (piece < n_qk + n_v) {
    const int j = ((piece - n_qk) * WAVE + lane) * CW;
    if (j >= dm.H * Vp) return;
    const int h = j / Vp, v = j - h * Vp;
    float o[DC_TT][CW];
    if (v < V) {
      convolve(2 * dm.KH * D + h * V + v, dm.vc + h * V + v, o);
    } else {
#pragma unroll
      for (int t = 0; t < DC_TT; ++t)
#pragma unroll
        for (int q = 0; q < CW; ++q) o[t][q] = 0.0f;
    }
#pragma unroll
    for (int t = 0; t < DC_TT; ++t)
      if (t < len)
        store_lanes<T, CW>(vo + (i0 + t) * ((long)dm.H * Vp) + j, o[t]);
  } else {
    for (int j = lane; j < len * dm.H; j += WAVE) {
      const int t = j / dm.H, h = j - t * dm.H;
      const T* yr = yt + (long)t * dm.ystride;
      if (!dm.channels)
        lg[(i0 + t) * dm.H + h] =
            log_decay((float)yr[dm.ac + h], (float)A_log[h], (float)dt_bias[h]);
      bt[(i0 + t) * dm.H + h] = sigmoid_f((float)yr[dm.bc + h]);
    }
  }
}

// The last taps - 1 inputs of every channel; runs after the convolution.
template <typename T>
__global__ __launch_bounds__(DC_BLOCK) void delta_conv_state_kernel(
    const T* __restrict__ y, T* __restrict__ conv_state,
    const int* __restrict__ cu, const int* __restrict__ pos0,
    const int* __restrict__ slots, int n_short, DeltaDims dm) {
  const int e = n_short + blockIdx.x;
  const int c = blockIdx.y * DC_BLOCK + threadIdx.x;
  const int D = dm.D, V = dm.V;
  const int nq = dm.KH * D;
  const int C = 2 * nq + dm.H * V;
  if (c >= C) return;
  const int col = c < nq ? dm.qc + c
                         : (c < 2 * nq ? dm.kc + c - nq : dm.vc + c - 2 * nq);
  const int hist = dm.taps - 1;
  const int t0 = cu[e], n = cu[e + 1] - t0;
  const bool fresh = pos0[e] == 0;
  T* cs = conv_state + ((long)slots[e] * C + c) * hist;
  for (int j = 0; j < hist; ++j) {  // ascending: reads stay ahead of writes
    const int s = n - hist + j;
    if (s >= 0)
      cs[j] = y[(long)(t0 + s) * dm.ystride + col];
    else
      cs[j] = fresh ? (T)0.0f : cs[hist + s];
  }
}

// ---------------------------------------------------------------------------
// Step 2, all chunks at once.  Block = (chunk, head), 4 waves; wave w makes
// rows 16w..16w+15 of the two Gram matrices, wave 0 then inverts I + L, one
// column per lane.
//   tm [chunks, H, 64, 64]  (I + L)^-1 diag(beta)
//   am [chunks, H, 64, 64]  A (lower tiles only)
//   ge [chunks, H, 2, 64]   exp(G), exp(G_last - G)
// ---------------------------------------------------------------------------

#define DR_LS 68

// (I + L)^-1 times `by`, one column per lane; ls: L, rows of DR_LS
__device__ __forceinline__ void invert_unit(const float* ls, float by, float* tm,
                                            int lane) {
  float x[DR_CHUNK];
#pragma unroll
  for (int i = 0; i < DR_CHUNK; ++i) {
    float a0 = i == lane ? 1.0f : 0.0f, a1 = 0.0f, a2 = 0.0f, a3 = 0.0f;
    const float* row = ls + i * DR_LS;
#pragma unroll
    for (int j = 0; j + 4 <= i; j += 4) {
      const f32x4 l4 = load4(row + j);
      a0 -= l4[0] * x[j];
      a1 -= l4[1] * x[j + 1];
      a2 -= l4[2] * x[j + 2];
      a3 -= l4[3] * x[j + 3];
    }
#pragma unroll
    for (int j = i & ~3; j < i; ++j) a0 -= row[j] * x[j];
    x[i] = (a0 + a1) + (a2 + a3);
    tm[i * 64 + lane] = x[i] * by;
  }
}

__global__ __launch_bounds__(256) void delta_chunk_kernel(
    const float* __restrict__ qn, const float* __restrict__ kn,
    const float* __restrict__ lg, const float* __restrict__ bt,
    float* __restrict__ tm, float* __restrict__ am, float* __restrict__ ge,
    const int* __restrict__ chunks, int tok_base, int KH, int H, int Dp) {
  const int c = blockIdx.x, h = blockIdx.y;
  const int kh = h / (H / KH);
  const int i0 = chunks[2 * c] - tok_base;
  const int len = chunks[2 * c + 1];
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = tid / WAVE;
  const int lr = lane & 15, g4 = lane >> 4;

  __shared__ double gs[DR_CHUNK];
  __shared__ float bs[DR_CHUNK];
  __shared__ __attribute__((aligned(16))) float ls[DR_CHUNK * DR_LS];

  const long ch = (long)c * H + h;
  if (wid == 0) {
    // running sum of log decays; differences of it must stay exact to fp32,
    // also behind strong decays, hence double
    const bool in = lane < len;
    double g = in ? (double)lg[(long)(i0 + lane) * H + h] : 0.0;
#pragma unroll
    for (int off = 1; off < WAVE; off <<= 1) {
      const double o = __shfl_up(g, off, WAVE);
      if (lane >= off) g += o;
    }
    const double last = __shfl(g, WAVE - 1, WAVE);
    gs[lane] = g;
    bs[lane] = in ? bt[(long)(i0 + lane) * H + h] : 0.0f;
    ge[ch * 128 + lane] = expf((float)g);
    ge[ch * 128 + 64 + lane] = expf((float)(last - g));
  }

  f32x4 kk[4], qk[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    kk[j] = f32x4{0, 0, 0, 0};
    qk[j] = f32x4{0, 0, 0, 0};
  }
  // rows past the end repeat the last one: their beta is 0
  const int ra = min(wid * 16 + lr, len - 1);
  const float* kbase = kn + ((long)i0 * KH + kh) * Dp + g4 * 4;
  const float* qbase = qn + ((long)i0 * KH + kh) * Dp + g4 * 4;
  const long rstride = (long)KH * Dp;
  for (int d = 0; d < Dp; d += 16) {
    const f32x4 ka = load4(kbase + ra * rstride + d);
    const f32x4 qa = load4(qbase + ra * rstride + d);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j > wid) continue;
      const int rb = min(j * 16 + lr, len - 1);
      const f32x4 kb = load4(kbase + rb * rstride + d);
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        kk[j] = mma4(ka[s], kb[s], kk[j]);
        qk[j] = mma4(qa[s], kb[s], qk[j]);
      }
    }
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    if (j > wid) continue;
    const int col = j * 16 + lr;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = wid * 16 + g4 * 4 + r;
      const float dec = col <= row ? expf((float)(gs[row] - gs[col])) : 0.0f;
      ls[row * DR_LS + col] = col < row ? bs[row] * dec * kk[j][r] : 0.0f;
      am[ch * 4096 + row * 64 + col] = dec * qk[j][r];
    }
  }
  __syncthreads();
  if (wid == 0) invert_unit(ls, bs[lane], tm + ch * 4096, lane);
}

// The same for decays per channel, and what the walk multiplies the state with:
//   qg, kg [tokens, H, Dp]  q and k with the decay from the chunk's begin
//   kl     [tokens, H, Dp]  k with the decay to the chunk's end
//   gl     [chunks, H, Dp]  the decay of the whole chunk
// Wave w has token rows 16w..16w+15, a lane one of them and four of each 16
// channels.  Per 16 channels, running products over blocks of 1, 2, 4, 8 and 16
// rows grow by one exchange between lanes each: `from` decays from the row's
// block's begin to the row, `to` from the row to its block's end.
#define DCH_STEPS 4                    // steps of 16 channels between barriers
#define DCH_LS (DCH_STEPS * 16 + 4)

// VEC: channels and rows of z are whole vectors of 4.
template <typename T, bool VEC>
__global__ __launch_bounds__(256, 2) void delta_chunk_channels_kernel(
    const float* __restrict__ qn, const float* __restrict__ kn,
    const T* __restrict__ z, const T* __restrict__ A_log,
    const T* __restrict__ dt_bias, const float* __restrict__ bt,
    float* __restrict__ tm, float* __restrict__ am, float* __restrict__ qg,
    float* __restrict__ kg, float* __restrict__ kl, float* __restrict__ gl,
    const int* __restrict__ chunks, int tok_base, DeltaDims dm, int Dp) {
  const int c = blockIdx.x, h = blockIdx.y;
  const int H = dm.H, KH = dm.KH, D = dm.D;
  const int kh = h / (H / KH);
  const int i0 = chunks[2 * c] - tok_base;
  const int len = chunks[2 * c + 1];
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, g4 = lane >> 4;

  __shared__ float bs[DR_CHUNK];
  __shared__ __attribute__((aligned(16))) float ms[4][DCH_STEPS * 16];
  // k with the decay to its wave's last row; later I + L
  __shared__ __attribute__((aligned(16))) float ls[DR_CHUNK * DR_LS];
  static_assert(DCH_LS <= DR_LS, "");

  const long ch = (long)c * H + h;
  if (wid == 0) bs[lane] = lane < len ? bt[(long)(i0 + lane) * H + h] : 0.0f;

  const int row = wid * 16 + lr;
  const bool in = row < len;
  // rows past the end repeat the last one with k = q = 0, decay 1 and beta 0
  const long tok = i0 + min(row, len - 1);
  const float* kp = kn + (tok * KH + kh) * Dp + g4 * 4;
  const float* qp = qn + (tok * KH + kh) * Dp + g4 * 4;
  const T* zp = z + (tok_base + tok) * dm.zstride + dm.ac + (long)h * D;
  const T* dp = dt_bias + (long)h * D;
  const long at = ((long)(i0 + row) * H + h) * Dp + g4 * 4;
  const float rate = expf((float)A_log[h]);
  const f32x4 zero = {0, 0, 0, 0}, one = {1, 1, 1, 1};

  f32x4 kk[4], qk[4], kko[3], qko[3];
#pragma unroll
  for (int i = 0; i < 4; ++i) kk[i] = qk[i] = zero;
#pragma unroll
  for (int i = 0; i < 3; ++i) kko[i] = qko[i] = zero;
  float diag = 0.0f;

  for (int d0 = 0; d0 < Dp; d0 += DCH_STEPS * 16) {
    f32x4 ka[DCH_STEPS], qa[DCH_STEPS], kb[DCH_STEPS];
    f32x4 za[DCH_STEPS], dt[DCH_STEPS];
    // everything a slice reads is asked for first
#pragma unroll
    for (int s = 0; s < DCH_STEPS; ++s) {
      const int ds = min(d0 + s * 16, Dp - 16), d = ds + g4 * 4;
      ka[s] = load4(kp + ds);
      qa[s] = load4(qp + ds);
      if constexpr (VEC) {
        const int dc = min(d, D - 4);
        za[s] = load4(zp + dc);
        dt[s] = load4(dp + dc);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int dc = min(d + j, D - 1);
          za[s][j] = (float)zp[dc];
          dt[s][j] = (float)dp[dc];
        }
      }
    }
#pragma unroll
    for (int s = 0; s < DCH_STEPS; ++s) {
      const int ds = d0 + s * 16;
      if (ds >= Dp) continue;
      const f32x4 k = in ? ka[s] : zero, q = in ? qa[s] : zero;
      f32x4 from, to = one;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float g = decay_of<T>(za[s][j], rate, dt[s][j]);
        from[j] = in && ds + g4 * 4 + j < D ? g : 1.0f;
        diag += q[j] * k[j];
      }
#pragma unroll
      for (int l = 0; l < 4; ++l) {
        const int half = 1 << l;
        const f32x4 kf = k * from, qf = q * from, kt = k * to;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          kk[l] = mma4(kf[j], kt[j], kk[l]);
          qk[l] = mma4(qf[j], kt[j], qk[l]);
        }
        // the other half's whole decay: of the first for rows of the second
        const bool second = lr & half;
        const int src = (lane & ~(2 * half - 1)) + (second ? half : 2 * half) - 1;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float other = __shfl(from[j], src, WAVE);
          if (second) from[j] *= other;
          else to[j] *= other;
        }
      }
      ka[s] = k * from;
      qa[s] = q * from;
      kb[s] = k * to;
      store4(ls + row * DCH_LS + s * 16 + g4 * 4, kb[s]);
      if (lr == 15) store4(&ms[wid][s * 16 + g4 * 4], from);
    }
    __syncthreads();
    // blocks before this wave's, the nearest first
#pragma unroll
    for (int b = 2; b >= 0; --b) {
      if (b >= wid) continue;
#pragma unroll
      for (int s = 0; s < DCH_STEPS; ++s) {
        if (d0 + s * 16 >= Dp) continue;
        const f32x4 k = load4(ls + (b * 16 + lr) * DCH_LS + s * 16 + g4 * 4);
        const f32x4 m = load4(&ms[b][s * 16 + g4 * 4]);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          kko[b] = mma4(ka[s][j], k[j], kko[b]);
          qko[b] = mma4(qa[s][j], k[j], qko[b]);
        }
        ka[s] = ka[s] * m;
        qa[s] = qa[s] * m;
      }
    }
    // and those behind it
#pragma unroll
    for (int b = 1; b < 4; ++b) {
      if (b <= wid) continue;
#pragma unroll
      for (int s = 0; s < DCH_STEPS; ++s)
        if (d0 + s * 16 < Dp)
          kb[s] = kb[s] * load4(&ms[b][s * 16 + g4 * 4]);
    }
    if (in) {
#pragma unroll
      for (int s = 0; s < DCH_STEPS; ++s) {
        const int ds = d0 + s * 16;
        if (ds >= Dp) continue;
        store4(kg + at + ds, ka[s]);
        store4(qg + at + ds, qa[s]);
        store4(kl + at + ds, kb[s]);
      }
    }
    if (tid < DCH_STEPS * 16 && d0 + tid < Dp)
      gl[ch * Dp + d0 + tid] =
          (ms[0][tid] * ms[1][tid]) * (ms[2][tid] * ms[3][tid]);
    __syncthreads();
  }
  diag += __shfl_xor(diag, 16, WAVE);
  diag += __shfl_xor(diag, 32, WAVE);  // of this lane's row: q.k

#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = wid * 16 + g4 * 4 + r;
    const float b = bs[i];
#pragma unroll
    for (int j = 0; j < 3; ++j) {
      if (j >= wid) continue;
      ls[i * DR_LS + j * 16 + lr] = b * kko[j][r];
      am[ch * 4096 + i * 64 + j * 16 + lr] = qko[j][r];
    }
    // the level that separates the row from the column
    const int local = g4 * 4 + r;
    float kv = 0.0f, qv = local == lr ? diag : 0.0f;
#pragma unroll
    for (int l = 0; l < 4; ++l)
      if (local > lr && (local ^ lr) >> l == 1) {
        kv = kk[l][r];
        qv = qk[l][r];
      }
    ls[i * DR_LS + row] = b * kv;
    am[ch * 4096 + i * 64 + row] = qv;
  }
  __syncthreads();
  if (wid == 0) invert_unit(ls, bs[lane], tm + ch * 4096, lane);
}

// ---------------------------------------------------------------------------
// Step 3: the walk.  Block = (value column tile, head, request), 4 waves;
// wave w owns token rows 16w..16w+15 of a chunk and state row tiles w, w+4,...
// A operands come straight from global memory as vectors (the contraction
// order inside 16 is permuted the same way on both sides).  CH: decays per
// channel; q, k and kt (k as the state takes it up) come with their decays, one
// row per value head (KH == H), and ge is the chunk's decay [chunks, H, Dp].
// ---------------------------------------------------------------------------

template <typename T, bool CH>
__global__ __launch_bounds__(256) void delta_walk_kernel(
    const float* __restrict__ qn, const float* __restrict__ kn,
    const float* __restrict__ kt, const T* __restrict__ vn, const float* __restrict__ tm,
    const float* __restrict__ am, const float* __restrict__ ge,
    float* __restrict__ state, float* __restrict__ o,
    const int* __restrict__ chunks, const int* __restrict__ chunk_cu,
    const int* __restrict__ pos0, const int* __restrict__ slots, int n_short,
    int tok_base, int KH, int H, int D, int Dp, int V, int Vp) {
  const int v0 = blockIdx.x * 16;
  const int h = blockIdx.y;
  const int e = blockIdx.z;
  const int kh = h / (H / KH);
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = tid / WAVE;
  const int lr = lane & 15, g4 = lane >> 4;

  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* ss = reinterpret_cast<float*>(smem);  // [Dp][17] state columns
  float* xs = ss + Dp * 17;                    // [64][17] V - exp(G) K S
  float* us = xs + 64 * 17;                    // [64][17] U
  float* uw = us + 64 * 17;                    // [64][17] exp(G_last - G) U

  const bool fresh = pos0[n_short + e] == 0;
  float* sg = state + ((long)slots[n_short + e] * H + h) * (long)D * V;
  for (int i = tid; i < Dp * 16; i += 256) {
    const int d = i >> 4, v = v0 + (i & 15);
    ss[d * 17 + (i & 15)] =
        (!fresh && d < D && v < V) ? sg[(long)d * V + v] : 0.0f;
  }
  __syncthreads();

  const long rstride = (long)KH * Dp;
  const f32x4 zero = {0, 0, 0, 0};
  const int row = wid * 16 + lr;            // A-operand row
  for (int c = chunk_cu[e]; c < chunk_cu[e + 1]; ++c) {
    const int i0 = chunks[2 * c] - tok_base;
    const int len = chunks[2 * c + 1];
    const long ch = (long)c * H + h;
    const float* kp = kn + ((long)i0 * KH + kh) * Dp;
    const float* qp = qn + ((long)i0 * KH + kh) * Dp;
    const float* tp = kt + ((long)i0 * KH + kh) * Dp;
    const float* gc = ge + ch * (CH ? Dp : 128);

    f32x4 ks = zero, qs = zero;
    {
      const float* ka = kp + row * rstride + g4 * 4;
      const float* qa = qp + row * rstride + g4 * 4;
      const bool in = row < len;
#pragma unroll 4
      for (int d = 0; d < Dp; d += 16) {
        const f32x4 a = in ? load4(ka + d) : zero;
        const f32x4 b = in ? load4(qa + d) : zero;
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          const float sv = ss[(d + g4 * 4 + s) * 17 + lr];
          ks = mma4(a[s], sv, ks);
          qs = mma4(b[s], sv, qs);
        }
      }
    }
    float gr[4], gl[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = wid * 16 + g4 * 4 + r;
      gr[r] = CH ? 1.0f : gc[i];
      gl[r] = CH ? 1.0f : gc[64 + i];
      const float v =
          i < len ? (float)vn[((long)(i0 + i) * H + h) * Vp + v0 + lr] : 0.0f;
      xs[i * 17 + lr] = v - gr[r] * ks[r];
    }
    __syncthreads();
    f32x4 u = zero;
    const float* ta = tm + ch * 4096 + row * 64 + g4 * 4;
    for (int j = 0; j <= wid; ++j) {
      const f32x4 a = load4(ta + j * 16);
#pragma unroll
      for (int s = 0; s < 4; ++s)
        u = mma4(a[s], xs[(j * 16 + g4 * 4 + s) * 17 + lr], u);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = wid * 16 + g4 * 4 + r;
      us[i * 17 + lr] = u[r];
      uw[i * 17 + lr] = u[r] * gl[r];
    }
    __syncthreads();
    f32x4 oc;
#pragma unroll
    for (int r = 0; r < 4; ++r) oc[r] = gr[r] * qs[r];
    const float* aa = am + ch * 4096 + row * 64 + g4 * 4;
    for (int j = 0; j <= wid; ++j) {
      const f32x4 a = load4(aa + j * 16);
#pragma unroll
      for (int s = 0; s < 4; ++s)
        oc = mma4(a[s], us[(j * 16 + g4 * 4 + s) * 17 + lr], oc);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = wid * 16 + g4 * 4 + r;
      if (i < len) o[((long)(i0 + i) * H + h) * Vp + v0 + lr] = oc[r];
    }
    for (int d0 = wid * 16; d0 < Dp; d0 += 64) {
      f32x4 sn;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        sn[r] = gc[CH ? d0 + g4 * 4 + r : 63] * ss[(d0 + g4 * 4 + r) * 17 + lr];
      const float* ka = tp + d0 + lr;
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          const int i = j * 16 + g4 * 4 + s;
          const float a = i < len ? ka[i * rstride] : 0.0f;
          sn = mma4(a, uw[i * 17 + lr], sn);
        }
#pragma unroll
      for (int r = 0; r < 4; ++r) ss[(d0 + g4 * 4 + r) * 17 + lr] = sn[r];
    }
    __syncthreads();
  }
  for (int i = tid; i < Dp * 16; i += 256) {
    const int d = i >> 4, v = v0 + (i & 15);
    if (d < D && v < V) sg[(long)d * V + v] = ss[d * 17 + (i & 15)];
  }
}

// The same walk with the state depth fixed at 16 * ND: every global operand
// of the next chunk is fetched into registers right after the current chunk
// used it, so its latency passes behind the products that remain.  Rows past
// the end of a chunk repeat its last one: their beta is 0, so they write
// nothing, and their outputs are not stored.
template <typename T, int ND, bool CH>
__global__ __launch_bounds__(256, 1) void delta_walk_fixed_kernel(
    const float* __restrict__ qn, const float* __restrict__ kn,
    const float* __restrict__ ktn, const T* __restrict__ vn, const float* __restrict__ tm,
    const float* __restrict__ am, const float* __restrict__ ge,
    float* __restrict__ state, float* __restrict__ o,
    const int* __restrict__ chunks, const int* __restrict__ chunk_cu,
    const int* __restrict__ pos0, const int* __restrict__ slots, int n_short,
    int tok_base, int KH, int H, int D, int V, int Vp) {
  constexpr int Dp = ND * 16;
  constexpr int NT = (ND + 3) / 4;  // state row tiles per wave
  const int v0 = blockIdx.x * 16;
  const int h = blockIdx.y;
  const int e = blockIdx.z;
  const int kh = h / (H / KH);
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, g4 = lane >> 4;

  __shared__ float ss[Dp * 17];  // state columns
  __shared__ float xs[64 * 17];  // V - exp(G) K S
  __shared__ float us[64 * 17];  // U
  __shared__ float uw[64 * 17];  // exp(G_last - G) U

  const bool fresh = pos0[n_short + e] == 0;
  float* sg = state + ((long)slots[n_short + e] * H + h) * (long)D * V;
  for (int i = tid; i < Dp * 16; i += 256) {
    const int d = i >> 4, v = v0 + (i & 15);
    ss[d * 17 + (i & 15)] =
        (!fresh && d < D && v < V) ? sg[(long)d * V + v] : 0.0f;
  }

  const long rstride = (long)KH * Dp;
  const f32x4 zero = {0, 0, 0, 0};
  const int row = wid * 16 + lr;            // A-operand row
  const int row_c = wid * 16 + g4 * 4;      // first C row

  f32x4 kf[ND], qf[ND], tf[4], af[4], kt[NT][4];
  float vf[4], gr[4], gl[4], g_all;
  f32x4 gd[NT];  // decays of this lane's state rows

  auto load_rows = [&](int i0, int len) {
    const long at = ((long)(i0 + min(row, len - 1)) * KH + kh) * Dp + g4 * 4;
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      kf[d] = load4(kn + at + d * 16);
      qf[d] = load4(qn + at + d * 16);
    }
  };
  auto load_misc = [&](int c, int i0, int len) {
    const float* gc = ge + ((long)c * H + h) * (CH ? Dp : 128);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = row_c + r;
      vf[r] = (float)vn[((long)(i0 + min(i, len - 1)) * H + h) * Vp + v0 + lr];
      gr[r] = CH ? 1.0f : gc[i];
      gl[r] = CH ? 1.0f : gc[64 + i];
    }
    if (!CH) g_all = gc[63];
  };
  auto load_decay = [&](int c) {
    if constexpr (CH) {
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const int d0 = wid * 16 + n * 64;
        if (d0 < Dp) gd[n] = load4(ge + ((long)c * H + h) * Dp + d0 + g4 * 4);
      }
    }
  };
  auto load_mat = [&](const float* m, int c, f32x4 (&f)[4]) {
    const float* p = m + ((long)c * H + h) * 4096 + row * 64 + g4 * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) f[j] = load4(p + j * 16);
  };
  auto load_kt = [&](int i0, int len) {
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int d0 = wid * 16 + n * 64;
      if (d0 >= Dp) continue;
      const float* ka = ktn + ((long)i0 * KH + kh) * Dp + d0 + lr;
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          const int i = min(j * 16 + g4 * 4 + s, len - 1);
          kt[n][j][s] = ka[i * rstride];
        }
    }
  };

  const int c_end = chunk_cu[e + 1];
  int c = chunk_cu[e];
  int i0 = chunks[2 * c] - tok_base, len = chunks[2 * c + 1];
  load_rows(i0, len);
  load_misc(c, i0, len);
  load_mat(tm, c, tf);
  load_mat(am, c, af);
  load_kt(i0, len);
  load_decay(c);
  __syncthreads();

  for (; c < c_end; ++c) {
    const int cn = min(c + 1, c_end - 1);  // the last one is fetched twice
    const int j0 = chunks[2 * cn] - tok_base;
    const int jl = chunks[2 * cn + 1];

    f32x4 ks = zero, qs = zero;
#pragma unroll
    for (int d = 0; d < ND; ++d)
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const float sv = ss[(d * 16 + g4 * 4 + s) * 17 + lr];
        ks = mma4(kf[d][s], sv, ks);
        qs = mma4(qf[d][s], sv, qs);
      }
    load_rows(j0, jl);
    f32x4 oc;
    float glk[4];
    const float g_now = g_all;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      xs[(row_c + r) * 17 + lr] = vf[r] - gr[r] * ks[r];
      oc[r] = gr[r] * qs[r];
      glk[r] = gl[r];
    }
    load_misc(cn, j0, jl);
    __syncthreads();

    f32x4 u = zero;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wid) {
#pragma unroll
        for (int s = 0; s < 4; ++s)
          u = mma4(tf[j][s], xs[(j * 16 + g4 * 4 + s) * 17 + lr], u);
      }
    load_mat(tm, cn, tf);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      us[(row_c + r) * 17 + lr] = u[r];
      uw[(row_c + r) * 17 + lr] = u[r] * glk[r];
    }
    __syncthreads();

#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wid) {
#pragma unroll
        for (int s = 0; s < 4; ++s)
          oc = mma4(af[j][s], us[(j * 16 + g4 * 4 + s) * 17 + lr], oc);
      }
    load_mat(am, cn, af);
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (row_c + r < len)
        o[((long)(i0 + row_c + r) * H + h) * Vp + v0 + lr] = oc[r];

#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int d0 = wid * 16 + n * 64;
      if (d0 >= Dp) continue;
      f32x4 sn;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        sn[r] = (CH ? gd[n][r] : g_now) * ss[(d0 + g4 * 4 + r) * 17 + lr];
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int s = 0; s < 4; ++s)
          sn = mma4(kt[n][j][s], uw[(j * 16 + g4 * 4 + s) * 17 + lr], sn);
#pragma unroll
      for (int r = 0; r < 4; ++r) ss[(d0 + g4 * 4 + r) * 17 + lr] = sn[r];
    }
    load_kt(j0, jl);
    load_decay(cn);
    __syncthreads();
    i0 = j0;
    len = jl;
  }
  for (int i = tid; i < Dp * 16; i += 256) {
    const int d = i >> 4, v = v0 + (i & 15);
    if (d < D && v < V) sg[(long)d * V + v] = ss[d * 17 + (i & 15)];
  }
}

// ---------------------------------------------------------------------------
// Step 4: output norm over V, weight, gate.  One wave per (token, head).
// ---------------------------------------------------------------------------

// NV groups of CW channels per lane, V <= 64 * CW * NV; DG_ROWS rows per wave
// in flight.
#define DG_ROWS 8

template <typename T, int NV, int CW>
__global__ __launch_bounds__(256) void delta_gate_kernel(
    const float* __restrict__ o, const T* __restrict__ z,
    const T* __restrict__ norm_w, T* __restrict__ out, long n, int tok_base,
    DeltaDims dm, int Vp, float eps) {
  const int lane = threadIdx.x & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const long w0 = ((long)blockIdx.x * 4 + wid) * DG_ROWS;
  const long rows = n * dm.H;
  float ov[DG_ROWS][NV][CW], gv[DG_ROWS][NV][CW];
#pragma unroll
  for (int k = 0; k < DG_ROWS; ++k) {
    const int wi = (int)min(w0 + k, rows - 1);
    const int i = wi / dm.H;
    const int h = wi - i * dm.H;
    const T* gr = z + (long)(tok_base + i) * dm.zstride + dm.gc + h * dm.V;
    const float* orow = o + (long)wi * Vp;
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int v = min((lane + u * WAVE) * CW, dm.V - CW);
      load_lanes<float, CW>(orow + v, ov[k][u]);
      load_lanes<T, CW>(gr + v, gv[k][u]);
    }
  }
  float wv[NV][CW];
#pragma unroll
  for (int u = 0; u < NV; ++u)
    load_lanes<T, CW>(norm_w + min((lane + u * WAVE) * CW, dm.V - CW), wv[u]);
#pragma unroll
  for (int k = 0; k < DG_ROWS; ++k) {
    const long wi = w0 + k;
    if (wi >= rows) return;
    float ss = 0.0f;
#pragma unroll
    for (int u = 0; u < NV; ++u)
      if ((lane + u * WAVE) * CW < dm.V) {
#pragma unroll
        for (int q = 0; q < CW; ++q) ss += ov[k][u][q] * ov[k][u][q];
      }
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)dm.V + eps);
    // row wi of [tokens * heads, V]
    T* dst = out + (tok_base * (long)dm.H + wi) * dm.V;
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int v = (lane + u * WAVE) * CW;
      float r[CW];
#pragma unroll
      for (int q = 0; q < CW; ++q)
        r[q] = ov[k][u][q] * inv * wv[u][q] * out_gate(gv[k][u][q], dm.sigmoid);
      if (v < dm.V) store_lanes<T, CW>(dst + v, r);
    }
  }
}

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

// KH: heads that q, k and kt have
template <typename T, bool CH>
static void delta_walk_t(const DeltaLongArgs& a, const DeltaDims& dm,
                         const float* q, const float* k, const float* kt, int KH,
                         dim3 grid, hipStream_t stream) {
  const dim3 block(256);
#define DW_GO(N)                                                              \
  delta_walk_fixed_kernel<T, N, CH><<<grid, block, 0, stream>>>(              \
      q, k, kt, (const T*)a.vn, a.tm, a.am, a.ge, a.state, a.o, a.chunks,     \
      a.chunk_cu, a.pos0, a.slots, a.n_short, a.tok_base, KH, dm.H, dm.D,     \
      dm.V, a.Vp)
  if (a.Dp == 16) DW_GO(1);
  else if (a.Dp == 32) DW_GO(2);
  else if (a.Dp == 64) DW_GO(4);
  else if (a.Dp == 128) DW_GO(8);
  else {
    const size_t smem = ((size_t)a.Dp + 3 * 64) * 17 * sizeof(float);
    delta_walk_kernel<T, CH><<<grid, block, smem, stream>>>(
        q, k, kt, (const T*)a.vn, a.tm, a.am, a.ge, a.state, a.o, a.chunks,
        a.chunk_cu, a.pos0, a.slots, a.n_short, a.tok_base, KH, dm.H, dm.D,
        a.Dp, dm.V, a.Vp);
  }
#undef DW_GO
}

template <typename T>
static void delta_long_t(const DeltaLongArgs& a, const DeltaDims& dm,
                         hipStream_t stream) {
  const int C = 2 * dm.KH * dm.D + dm.H * dm.V;
  const float q_scale = 1.0f / sqrtf((float)dm.D);
  dim3 block(DC_BLOCK);
  // pairs of channels per lane where the sizes allow it
  const bool pair = dm.D % 2 == 0 && dm.V % 2 == 0 && dm.ystride % 2 == 0;
  const int cw = pair ? 2 : 1;
  const int pieces =
      2 * dm.KH + (dm.H * a.Vp + WAVE * cw - 1) / (WAVE * cw) + 1;
  dim3 g1((unsigned)(a.n_chunks * DC_SUB),
          (unsigned)((pieces + DC_BLOCK / WAVE - 1) / (DC_BLOCK / WAVE)));
#define DC_GO(N, W)                                                          \
  delta_conv_kernel<T, N, W><<<g1, block, 0, stream>>>(                      \
      (const T*)a.y, (const T*)a.conv_w, (const T*)a.A_log,                  \
      (const T*)a.dt_bias, (const T*)a.conv_state, a.qn, a.kn, (T*)a.vn,     \
      a.lg, a.bt, a.cu, a.pos0, a.slots, a.tok_entry, a.chunks, a.tok_base,  \
      dm, a.Dp, a.Vp, q_scale)
  if (pair) {
    if (a.Dp <= 128) DC_GO(1, 2);
    else if (a.Dp <= 256) DC_GO(2, 2);
    else DC_GO(4, 2);
  } else {
    if (a.Dp <= 64) DC_GO(1, 1);
    else if (a.Dp <= 128) DC_GO(2, 1);
    else if (a.Dp <= 256) DC_GO(4, 1);
    else DC_GO(8, 1);
  }
#undef DC_GO
  dim3 g2((unsigned)a.n_long, (unsigned)((C + DC_BLOCK - 1) / DC_BLOCK));
  if (dm.taps > 1)
    delta_conv_state_kernel<T><<<g2, block, 0, stream>>>(
        (const T*)a.y, (T*)a.conv_state, a.cu, a.pos0, a.slots, a.n_short, dm);
  dim3 g3((unsigned)a.n_chunks, (unsigned)dm.H);
  dim3 g4((unsigned)(a.Vp / 16), (unsigned)dm.H, (unsigned)a.n_long);
  if (dm.channels) {
    const bool vec = dm.D % 4 == 0 && dm.ac % 4 == 0 && dm.zstride % 4 == 0 &&
                     ((uintptr_t)a.z | (uintptr_t)a.dt_bias) % 16 == 0;
#define DCH_GO(V)                                                              \
  delta_chunk_channels_kernel<T, V><<<g3, block, 0, stream>>>(                 \
      a.qn, a.kn, (const T*)a.z, (const T*)a.A_log, (const T*)a.dt_bias, a.bt, \
      a.tm, a.am, a.qg, a.kg, a.kl, a.ge, a.chunks, a.tok_base, dm, a.Dp)
    if (vec) DCH_GO(true);
    else DCH_GO(false);
#undef DCH_GO
    delta_walk_t<T, true>(a, dm, a.qg, a.kg, a.kl, dm.H, g4, stream);
  } else {
    delta_chunk_kernel<<<g3, block, 0, stream>>>(
        a.qn, a.kn, a.lg, a.bt, a.tm, a.am, a.ge, a.chunks, a.tok_base, dm.KH,
        dm.H, a.Dp);
    delta_walk_t<T, false>(a, dm, a.qn, a.kn, a.kn, dm.KH, g4, stream);
  }
  dim3 g5((unsigned)((a.n_tok * dm.H + 4 * DG_ROWS - 1) / (4 * DG_ROWS)));
#define DG_GO(N, W)                                                          \
  delta_gate_kernel<T, N, W><<<g5, block, 0, stream>>>(                      \
      a.o, (const T*)a.z, (const T*)a.norm_w, (T*)a.out, a.n_tok,            \
      a.tok_base, dm, a.Vp, a.eps)
  if (pair && dm.gc % 2 == 0 && dm.zstride % 2 == 0) {
    if (dm.V <= 128) DG_GO(1, 2);
    else if (dm.V <= 256) DG_GO(2, 2);
    else DG_GO(4, 2);
  } else {
    if (dm.V <= 64) DG_GO(1, 1);
    else if (dm.V <= 128) DG_GO(2, 1);
    else if (dm.V <= 256) DG_GO(4, 1);
    else DG_GO(8, 1);
  }
#undef DG_GO
}

extern "C" void launch_delta_long(const DeltaLongArgs* a, const DeltaDims* dm,
                                  bool f32, hipStream_t stream) {
  if (f32)
    delta_long_t<float>(*a, *dm, stream);
  else
    delta_long_t<__bf16>(*a, *dm, stream);
}
