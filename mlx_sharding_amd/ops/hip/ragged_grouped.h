// Grouped softmax attention over a ragged batch and a paged cache of keys and
// values.
//
// A page holds, for each key/value head, 64 keys and then 64 values in the
// order in which the matrix cores take them (fragments of 64 lanes x 8
// elements):
//   keys    tile (16 keys x 32 dims):   lane = (dim / 8 % 4, key % 16)
//   values  tile (16 dims x 32 keys):   lane = (key / 4 % 4, dim % 16), a
//           lane's elements are keys 0..3 and 16..19 past its first
// so a wave's operand is one coalesced load and a page goes to LDS by plain
// copies.  Scores are computed transposed (keys x queries): a lane holds one
// query, and its scores of two key tiles are the value product's operand
// without leaving the lane.
//
// The optional sink is one more term of the softmax's denominator, with
// neither key nor value; it enters once, when a row is finished.  With a window
// a token sees its last `window` tokens; pages before all of a block's windows
// are not visited.  Where values were rotated by their positions, a finished
// row is turned back by its own.  A gate multiplies a finished row of a head by
// the sigmoid of one number.
#pragma once

#include "ragged_common.h"

struct GroupedRowArgs {
  const void *y, *wq, *wk, *vmix, *first;  // all but y may be null
  void* pool;
  long ystride, fstride;
  int H, G, D, V, dimp, vdp;
  float eps;
  bool vec;  // heads, rows and bases are whole vectors of 8
  // rotations by position, [positions, pairs]: the first 2 * qk_pairs
  // dimensions of queries and keys, the first 2 * v_pairs of values
  const float *qk_cos, *qk_sin, *v_cos, *v_sin;
  int qk_pairs, v_pairs;
  const int* tok_pos;
  bool head_norm;  // queries and keys over their own root mean squares, times
                   // weights [D] if wq, wk are given
};

struct GroupedAttnArgs {
  const void *q, *sink, *pool;
  void* out;
  float *part_o, *part_ml;
  const int *cu, *pos0, *pages, *tiles;
  int P, H, G, dimp, V, vdp;
  int n_req, nsplit, row_tiles, n_tiles;
  long n_rows, ostride;
  float scale;
  bool vec;  // rows of out take vectors of 4
  int window;                 // 0: every earlier token is seen
  const float *v_cos, *v_sin; // [positions, V / 2] or null
  const int* tok_pos;
  const void* gate;           // [tokens, H] or null
  long gstride;
};

#define GA_BLOCK 256
#define GA_WAVES (GA_BLOCK / WAVE)
#define GA_STEP 32     // keys per step of a wave, decode
#define GA_QT 128      // queries per block, prompts
#define GA_MAXSPLIT WAVE
#define GA_NONE -1e30f

// Softmax arguments: bf16 works in powers of two, float in powers of e.
template <typename T>
__device__ __forceinline__ constexpr float sm_unit() {
  return sizeof(T) == 2 ? 1.44269504088896340736f : 1.0f;
}
template <typename T>
__device__ __forceinline__ float sm_exp(float x);
template <>
__device__ __forceinline__ float sm_exp<__bf16>(float x) {
  return __builtin_amdgcn_exp2f(x);
}
template <>
__device__ __forceinline__ float sm_exp<float>(float x) {
  return expf(x);
}

template <typename T>
__device__ __forceinline__ void frag_zero(Frag<T>& f);
template <>
__device__ __forceinline__ void frag_zero(Frag<__bf16>& f) {
#pragma unroll
  for (int j = 0; j < 8; ++j) f.v[j] = (__bf16)0.0f;
}
template <>
__device__ __forceinline__ void frag_zero(Frag<float>& f) {
  f.a = f32x4{0, 0, 0, 0};
  f.b = f32x4{0, 0, 0, 0};
}

// zero the elements of a value fragment from key `n` of its 32 on
__device__ __forceinline__ void frag_cut(Frag<__bf16>& f, int lg, int n) {
#pragma unroll
  for (int j = 0; j < 8; ++j)
    if (lg * 4 + (j < 4 ? j : 12 + j) >= n) f.v[j] = (__bf16)0.0f;
}
__device__ __forceinline__ void frag_cut(Frag<float>& f, int lg, int n) {
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    if (lg * 4 + j >= n) f.a[j] = 0.0f;
    if (lg * 4 + 16 + j >= n) f.b[j] = 0.0f;
  }
}

template <typename T>
__device__ __forceinline__ void store_cols(T* o, int col, int V, f32x4 v,
                                           bool vec) {
  if (vec) {
    if (col < V) store4(o + col, v);
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (col + j < V) o[col + j] = (T)v[j];
  }
}

// columns col .. col + 3 of a finished row at `pos`, turned back
__device__ __forceinline__ f32x4 turn_back(const GroupedAttnArgs& a, int pos,
                                           int col, f32x4 v) {
  if (!a.v_cos || col >= a.V) return v;
  const int half = a.V / 2, p = col / 2, q = min(p + 1, half - 1);
  const float* c = a.v_cos + (long)pos * half;
  const float* s = a.v_sin + (long)pos * half;
  return f32x4{v[0] * c[p] + v[1] * s[p], v[1] * c[p] - v[0] * s[p],
               v[2] * c[q] + v[3] * s[q], v[3] * c[q] - v[2] * s[q]};
}

// what a head's finished row of a token is multiplied by
template <typename T>
__device__ __forceinline__ float gate_of(const GroupedAttnArgs& a, long tok,
                                         int h) {
  return a.gate ? sigmoid_f((float)((const T*)a.gate)[tok * a.gstride + h])
                : 1.0f;
}

// the first token that one at `pos` sees
__device__ __forceinline__ int first_seen(const GroupedAttnArgs& a, int pos) {
  return a.window ? max(0, pos - a.window + 1) : 0;
}

// ---------------------------------------------------------------------------
// Short portions and decoding.  A query row is one (token, head) pair of one
// request and key/value head; a block serves 16 of them over one slice of the
// keys, its waves take every fourth step of 32 keys, straight from the pages
// into registers, and are merged through LDS.
//   grid (requests * key/value heads, slices, row tiles)
// NK, ND: 32-wide key and 16-wide value tiles of a head, rounded up; tiles
// past the real ones repeat the last and meet zero queries or are not stored.
// ---------------------------------------------------------------------------

template <typename T, int NK, int ND>
__global__ __launch_bounds__(GA_BLOCK) void grouped_attn_short_kernel(
    const GroupedAttnArgs a) {
  constexpr int CH = ND < 8 ? ND : 8;  // value tiles merged at a time
  constexpr int CW = CH * 16 + 4;
  constexpr bool AHEAD = sizeof(T) == 2 && 2 * NK + ND <= 24;
  __shared__ float so[GA_WAVES][16][CW];
  __shared__ float sm[GA_WAVES][16], sl[GA_WAVES][16], sw[16];

  const int e = blockIdx.x / a.G, g = blockIdx.x % a.G;
  const int R = a.H / a.G;
  const int r0 = blockIdx.z * 16;
  const int t0 = a.cu[e];
  const int rows = (a.cu[e + 1] - t0) * R;
  if (r0 >= rows) return;
  const int p0 = a.pos0[e];
  const int S = p0 + min(r0 + 15, rows - 1) / R + 1;  // keys these rows see
  const int s0 = first_seen(a, p0 + r0 / R) / GA_STEP * GA_STEP;
  const int steps = (S - s0 + GA_STEP - 1) / GA_STEP;
  const int per = (steps + a.nsplit - 1) / a.nsplit * GA_STEP;
  const int lo = s0 + blockIdx.y * per;
  const int hi = min(S, lo + per);

  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, lg = lane >> 4;
  const int nk = a.dimp / 32, nd = a.vdp / 16;
  const long PW = (long)RG_PAGE * (a.dimp + a.vdp);
  const T* pool = (const T*)a.pool;

  const int my_row = min(r0 + lr, rows - 1);
  const int my_tok = my_row / R;
  const int my_head = g * R + my_row - my_tok * R;
  const int limit = min(p0 + my_tok + 1, hi);
  const int from = first_seen(a, p0 + my_tok);
  const float scale = a.scale * sm_unit<T>();

  Frag<T> qf[NK];
  {
    const T* q = (const T*)a.q +
                 ((long)(t0 + my_tok) * a.H + my_head) * a.dimp + lg * 8;
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      qf[k].load(q + min(k, nk - 1) * 32);
      if (k >= nk) frag_zero(qf[k]);
    }
  }

  float m_run = GA_NONE, l_run = 0.0f;
  f32x4 acc[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) acc[d] = f32x4{0, 0, 0, 0};

  const int* table = a.pages + (long)e * a.P;
  int t = lo + wid * GA_STEP;
  long page = t < hi ? table[t / RG_PAGE] : 0;
  for (; t < hi; t += GA_WAVES * GA_STEP) {
    const T* base = pool + (page * a.G + g) * PW + lane * 8;
    const T* kp = base + (t % RG_PAGE) * a.dimp;
    const T* vp = base + RG_PAGE * a.dimp + t % RG_PAGE * 16;
    const int t_next = t + GA_WAVES * GA_STEP;
    if (t_next < hi) page = table[t_next / RG_PAGE];
    Frag<T> kf[2][NK], vf[AHEAD ? ND : 1];
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int k = 0; k < NK; ++k)
        kf[s][k].load(kp + (s * nk + min(k, nk - 1)) * 512);
    if constexpr (AHEAD) {
#pragma unroll
      for (int d = 0; d < ND; ++d) vf[d].load(vp + min(d, nd - 1) * 1024);
      __builtin_amdgcn_sched_barrier(0);
    }
    f32x4 sc[2];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      sc[s] = f32x4{0, 0, 0, 0};
#pragma unroll
      for (int k = 0; k < NK; ++k) sc[s] = mma(kf[s][k], qf[k], sc[s]);
    }
    float p[8], mx = GA_NONE;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int key = t + lg * 4 + (j < 4 ? j : 12 + j);
      p[j] = key < limit && key >= from ? sc[j / 4][j % 4] * scale : GA_NONE;
      mx = fmaxf(mx, p[j]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
    const float m_new = fmaxf(m_run, mx);
    const float alpha = sm_exp<T>(m_run - m_new);
    m_run = m_new;
    float sum = 0.0f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      p[j] = p[j] == GA_NONE ? 0.0f : sm_exp<T>(p[j] - m_new);
      sum += p[j];
    }
    sum += __shfl_xor(sum, 16, WAVE);
    sum += __shfl_xor(sum, 32, WAVE);
    l_run = l_run * alpha + sum;
    Frag<T> ph, pl;
    split_weights(p, ph, pl);
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      Frag<T> v;
      if constexpr (AHEAD) v = vf[d];
      else v.load(vp + min(d, nd - 1) * 1024);
      // what lies behind the last key may be anything
      if (t + GA_STEP > S) frag_cut(v, lg, S - t);
      f32x4 c4 = acc[d];
#pragma unroll
      for (int j = 0; j < 4; ++j) c4[j] *= alpha;
      acc[d] = mma_weights(v, ph, pl, c4);
    }
  }

  if (lg == 0) {
    sm[wid][lr] = m_run;
    sl[wid][lr] = l_run;
  }
  __syncthreads();
  float sink = 0.0f, M = GA_NONE;
  const bool last = a.nsplit == 1;
#pragma unroll
  for (int w = 0; w < GA_WAVES; ++w) M = fmaxf(M, sm[w][lr]);
  if (last && a.sink) {
    sink = (float)((const T*)a.sink)[my_head] * sm_unit<T>();
    M = fmaxf(M, sink);
  }
  float L = last && a.sink ? sm_exp<T>(sink - M) : 0.0f;
#pragma unroll
  for (int w = 0; w < GA_WAVES; ++w) L += sl[w][lr] * sm_exp<T>(sm[w][lr] - M);
  const float mine = sm_exp<T>(m_run - M);
  if (tid < 16) {
    if (last) {
      sw[lr] = gate_of<T>(a, t0 + my_tok, my_head) / L;
    } else {
      sw[lr] = 1.0f;
      if (r0 + lr < rows) {
        const long orow = (long)(t0 + my_tok) * a.H + my_head;
        float* ml = a.part_ml + (orow * a.nsplit + blockIdx.y) * 2;
        ml[0] = M;
        ml[1] = L;
      }
    }
  }
#pragma unroll
  for (int c = 0; c < ND / CH; ++c) {
    if (c) __syncthreads();
#pragma unroll
    for (int d = 0; d < CH; ++d) {
      f32x4 c4 = acc[c * CH + d];
#pragma unroll
      for (int j = 0; j < 4; ++j) c4[j] *= mine;
      *reinterpret_cast<f32x4*>(&so[wid][lr][d * 16 + lg * 4]) = c4;
    }
    __syncthreads();
    for (int i = tid; i < 16 * CH * 4; i += GA_BLOCK) {
      const int r = i / (CH * 4), w = (i % (CH * 4)) * 4;
      const int col = c * CH * 16 + w;
      if (r0 + r >= rows || col >= a.vdp) continue;
      f32x4 v = {0, 0, 0, 0};
#pragma unroll
      for (int k = 0; k < GA_WAVES; ++k) {
        const f32x4 u = *reinterpret_cast<const f32x4*>(&so[k][r][w]);
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] += u[j];
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] *= sw[r];
      const int tok = (r0 + r) / R, h = g * R + (r0 + r) % R;
      if (last)
        store_cols((T*)a.out + (long)(t0 + tok) * a.ostride + (long)h * a.V,
                   col, a.V, turn_back(a, p0 + tok, col, v), a.vec);
      else
        store4(a.part_o +
                   (((long)(t0 + tok) * a.H + h) * a.nsplit + blockIdx.y) *
                       a.vdp + col, v);
    }
  }
}

// One block per (token, head): merges the slices of the keys and the sink.
template <typename T>
__global__ __launch_bounds__(128) void grouped_attn_merge_kernel(
    const GroupedAttnArgs a) {
  const long row = blockIdx.x;
  const int h = (int)(row % a.H), n = a.nsplit;
  const float* ml = a.part_ml + row * n * 2;
  __shared__ float w[GA_MAXSPLIT];  // weight of each slice
  if (threadIdx.x < WAVE) {
    const int s = threadIdx.x;
    const float ms = s < n ? ml[2 * s] : GA_NONE;
    float M = wave_max(ms), sink = 0.0f;
    if (a.sink) {
      sink = (float)((const T*)a.sink)[h] * sm_unit<T>();
      M = fmaxf(M, sink);
    }
    const float e = s < n ? sm_exp<T>(ms - M) : 0.0f;
    float L = wave_sum(s < n ? ml[2 * s + 1] * e : 0.0f);
    if (a.sink) L += sm_exp<T>(sink - M);
    w[s] = e / L * gate_of<T>(a, row / a.H, h);
  }
  __syncthreads();
  T* out = (T*)a.out + row / a.H * a.ostride + (long)h * a.V;
  for (int d = threadIdx.x * 4; d < a.vdp; d += 512) {
    const float* p = a.part_o + row * n * a.vdp + d;
    f32x4 o = {0, 0, 0, 0};
#pragma unroll 8
    for (int s = 0; s < n; ++s) {
      const f32x4 v = load4(p + (long)s * a.vdp);
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] += v[j] * w[s];
    }
    if (a.v_cos) o = turn_back(a, a.tok_pos[row / a.H], d, o);
    store_cols(out, d, a.V, o, a.vec);
  }
}

template <typename T, int NK, int ND>
static void grouped_attn_short_go(const GroupedAttnArgs& a,
                                  hipStream_t stream) {
  dim3 grid((unsigned)(a.n_req * a.G), (unsigned)a.nsplit,
            (unsigned)a.row_tiles);
  grouped_attn_short_kernel<T, NK, ND>
      <<<grid, dim3(GA_BLOCK), 0, stream>>>(a);
  if (a.nsplit > 1)
    grouped_attn_merge_kernel<T>
        <<<dim3((unsigned)a.n_rows), dim3(128), 0, stream>>>(a);
}

// ---------------------------------------------------------------------------
// Prompts.  A block serves 128 queries of one head, 32 a wave; pages go to
// LDS as they are, the next one while this one is worked on.
//   grid (heads, query tiles): neighbouring blocks are other key/value heads,
//   and blocks go round the XCDs, so heads that share keys share an L2.
//   tiles[i] = (request, first query within the portion)
// ---------------------------------------------------------------------------

// 16 bytes a lane from memory to LDS, lane after lane from `dst` on
__device__ __forceinline__ void to_lds(const void* src, void* dst) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) void*)src,
      (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

template <typename T, int NK, int ND>
__global__ __launch_bounds__(GA_BLOCK, sizeof(T) == 2 && NK + ND / 2 <= 8 ? 2 : 1)
void grouped_attn_long_kernel(
    const GroupedAttnArgs a) {
  constexpr int BUFS = sizeof(T) == 2 ? 2 : 1;
  const int R = a.H / a.G;
  const int g = blockIdx.x % a.G, h = g * R + blockIdx.x / a.G;
  const int e = a.tiles[2 * blockIdx.y];
  const int q0 = a.tiles[2 * blockIdx.y + 1];
  const int t0 = a.cu[e];
  const int n = a.cu[e + 1] - t0;
  const int p0 = a.pos0[e];
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, lg = lane >> 4;
  const int nk = a.dimp / 32, nd = a.vdp / 16;
  const int PW = RG_PAGE * (a.dimp + a.vdp);  // of one key/value head
  const int parts = PW * (int)sizeof(T) / 1024;
  const float scale = a.scale * sm_unit<T>();

  extern __shared__ __attribute__((aligned(16))) char smem[];

  const int* table = a.pages + (long)e * a.P;
  auto stage = [&](int p, long page) {
    const char* src = (const char*)((const T*)a.pool + (page * a.G + g) * PW);
    char* dst = smem + (size_t)(p % BUFS) * PW * sizeof(T);
    for (int i = wid; i < parts; i += GA_WAVES)
      to_lds(src + i * 1024 + lane * 16, dst + i * 1024);
  };

  const int hi = p0 + min(q0 + GA_QT, n);
  const int n_pages = (hi + RG_PAGE - 1) / RG_PAGE;
  const int first = first_seen(a, p0 + q0) / RG_PAGE;
  if constexpr (BUFS == 2) stage(first, table[first]);
  int next = table[min(first + 1, n_pages - 1)];

  const int w0 = q0 + wid * 32;  // this wave's first query
  Frag<T> qf[2][NK];
  int qpos[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = min(w0 + i * 16 + lr, n - 1);
    qpos[i] = p0 + r;
    const T* src =
        (const T*)a.q + ((long)(t0 + r) * a.H + h) * a.dimp + lg * 8;
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      qf[i][k].load(src + min(k, nk - 1) * 32);
      if (k >= nk) frag_zero(qf[i][k]);
    }
  }
  const int wave_lo = p0 + min(w0, n - 1);                // positions
  const int wave_hi = w0 < n ? p0 + min(w0 + 31, n - 1) + 1 : 0;
  const int wave_from = first_seen(a, wave_lo);
  int qfrom[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) qfrom[i] = first_seen(a, qpos[i]);

  float m_run[2] = {GA_NONE, GA_NONE}, l_run[2] = {0.0f, 0.0f};
  f32x4 acc[2][ND];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[i][d] = f32x4{0, 0, 0, 0};

  for (int p = first; p < n_pages; ++p) {
    if constexpr (BUFS == 1) {
      __syncthreads();
      stage(p, table[p]);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if constexpr (BUFS == 2)
      if (p + 1 < n_pages) {
        stage(p + 1, next);
        next = table[min(p + 2, n_pages - 1)];
      }
    const int t = p * RG_PAGE;
    if (t >= wave_hi || t + RG_PAGE <= wave_from) continue;
    const T* ks = (const T*)smem + (p % BUFS) * PW + lane * 8;
    const T* vs = ks + RG_PAGE * a.dimp;

    f32x4 sc[2][4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      sc[0][s] = f32x4{0, 0, 0, 0};
      sc[1][s] = f32x4{0, 0, 0, 0};
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        Frag<T> f;
        f.load(ks + (s * nk + min(k, nk - 1)) * 512);
        sc[0][s] = mma(f, qf[0][k], sc[0][s]);
        sc[1][s] = mma(f, qf[1][k], sc[1][s]);
      }
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j) sc[i][s][j] *= scale;
    if (t + RG_PAGE - 1 > wave_lo) {
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (t + s * 16 + lg * 4 + j > qpos[i]) sc[i][s][j] = GA_NONE;
    }
    // the last query's window begins last
    if (t < first_seen(a, wave_hi - 1)) {
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (t + s * 16 + lg * 4 + j < qfrom[i]) sc[i][s][j] = GA_NONE;
    }
    float alpha[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      float mx = GA_NONE;
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j) mx = fmaxf(mx, sc[i][s][j]);
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      const float m_new = fmaxf(m_run[i], mx);
      alpha[i] = sm_exp<T>(m_run[i] - m_new);
      m_run[i] = m_new;
      // a window may begin behind its block's first page: no score yet
      const float m_ref = m_new == GA_NONE ? 0.0f : m_new;
      float sum = 0.0f;
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float w = sm_exp<T>(sc[i][s][j] - m_ref);
          sc[i][s][j] = w;
          sum += w;
        }
      sum += __shfl_xor(sum, 16, WAVE);
      sum += __shfl_xor(sum, 32, WAVE);
      l_run[i] = l_run[i] * alpha[i] + sum;
    }
    if (!__all(alpha[0] == 1.0f && alpha[1] == 1.0f)) {
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int d = 0; d < ND; ++d)
#pragma unroll
          for (int j = 0; j < 4; ++j) acc[i][d][j] *= alpha[i];
    }
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
      Frag<T> ph[2], pl[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        float w[8];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          w[j] = sc[i][2 * hh][j];
          w[4 + j] = sc[i][2 * hh + 1][j];
        }
        split_weights(w, ph[i], pl[i]);
      }
#pragma unroll
      for (int d = 0; d < ND; ++d) {
        Frag<T> f;
        f.load(vs + (min(d, nd - 1) * 2 + hh) * 512);
        acc[0][d] = mma_weights(f, ph[0], pl[0], acc[0][d]);
        acc[1][d] = mma_weights(f, ph[1], pl[1], acc[1][d]);
      }
    }
  }

  float sink = 0.0f;
  if (a.sink) sink = (float)((const T*)a.sink)[h] * sm_unit<T>();
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = w0 + i * 16 + lr;
    if (r >= n) continue;
    float f = 1.0f / l_run[i];
    if (a.sink) {
      const float M = fmaxf(m_run[i], sink);
      f = sm_exp<T>(m_run[i] - M);
      f /= l_run[i] * f + sm_exp<T>(sink - M);
    }
    f *= gate_of<T>(a, t0 + r, h);
    T* o = (T*)a.out + (long)(t0 + r) * a.ostride + (long)h * a.V;
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      f32x4 c4 = acc[i][d];
#pragma unroll
      for (int j = 0; j < 4; ++j) c4[j] *= f;
      c4 = turn_back(a, p0 + r, d * 16 + lg * 4, c4);
      store_cols(o, d * 16 + lg * 4, a.V, c4, a.vec);
    }
  }
}

template <typename T, int NK, int ND>
static void grouped_attn_long_go(const GroupedAttnArgs& a, hipStream_t stream) {
  const size_t smem = (size_t)(sizeof(T) == 2 ? 2 : 1) * RG_PAGE *
                      (a.dimp + a.vdp) * sizeof(T);
  if (smem > 65536)
    (void)hipFuncSetAttribute(
        reinterpret_cast<const void*>(&grouped_attn_long_kernel<T, NK, ND>),
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  grouped_attn_long_kernel<T, NK, ND>
      <<<dim3((unsigned)a.H, (unsigned)a.n_tiles), dim3(GA_BLOCK), smem,
         stream>>>(a);
}
