// Routed experts: router, placement of (token, expert) pairs, grouped matrix
// products, weighted gather.
//
// Pairs are sorted by expert and cut into tiles of one expert.  The placement is
// made from per-block histograms without atomics on memory, so nothing has to
// be cleared beforehand and the kernels may be captured in a graph.
#include "ragged_experts.h"

#define EX_BLOCK 256
#define EX_WAVES (EX_BLOCK / WAVE)

// ---------------------------------------------------------------------------
// Router.  A block has 16 tokens and 16 waves: 128 experts at a time, half of
// the waves for each 64 of them, eight parts of the contraction, which meet in
// LDS.  Then a wave per token makes scores and picks.
// ---------------------------------------------------------------------------

#define RT_BLOCK 1024
#define RT_WAVES (RT_BLOCK / WAVE)
#define RT_PARTS 8
#define RT_LS (128 + 4)

template <typename T>
__global__ __launch_bounds__(RT_BLOCK) void expert_route_kernel(
    const RouteArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int totalp = (a.total + 63) / 64 * 64;
  float* part = reinterpret_cast<float*>(smem);        // [parts][16][RT_LS]
  float* choices = part;                               // later: [waves][totalp]
  const int shared_n = max(RT_PARTS * EX_TOK * RT_LS, RT_WAVES * totalp);
  float* logits = part + shared_n;                     // [16][totalp]
  int* counts = reinterpret_cast<int*>(logits + EX_TOK * totalp);  // [experts]
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, lg = lane >> 4;
  const long t0 = (long)blockIdx.x * EX_TOK;
  const int n = (int)min((long)EX_TOK, a.n - t0);

  for (int e = tid; e < a.experts; e += RT_BLOCK) counts[e] = 0;
  const T* hrow =
      (const T*)a.h + (t0 + min(lr, n - 1)) * a.hstride + lg * 8;
  const int steps = a.K / 32;
  const int per = (steps + RT_PARTS - 1) / RT_PARTS;
  const int half = wid / RT_PARTS, which = wid % RT_PARTS;
  const int s0 = which * per, s1 = min(steps, s0 + per);
  for (int e0 = 0; e0 < a.total; e0 += 128) {
    const int first = e0 + half * 64;
    const int tiles = max(0, min(4, (a.total - first + 15) / 16));
    f32x4 acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4{0, 0, 0, 0};
    // operands of 16 experts by 32 columns lie together, lane after lane
    const T* w = (const T*)a.w + (long)first / 16 * steps * 512 + lane * 8;
    const long next = (long)steps * 512;
#pragma unroll 8
    for (int s = s0; s < s1; ++s) {
      Frag<T> b, f[4];
      b.load(hrow + s * 32);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (i < tiles) f[i].load(w + i * next + s * 512);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (i < tiles) acc[i] = mma(f[i], b, acc[i]);
    }
    __syncthreads();  // the sums of the last round are read
#pragma unroll
    for (int i = 0; i < 4; ++i)
      store4(part + (which * EX_TOK + lr) * RT_LS + half * 64 + i * 16 + lg * 4,
             acc[i]);
    __syncthreads();
    for (int i = tid; i < EX_TOK * 128; i += RT_BLOCK) {
      const int t = i / 128, e = i % 128;
      if (e0 + e >= totalp) continue;
      float z = 0.0f;
#pragma unroll
      for (int w = 0; w < RT_PARTS; ++w)
        z += part[(w * EX_TOK + t) * RT_LS + e];
      logits[t * totalp + e0 + e] = z;
    }
  }
  __syncthreads();

  for (int t = wid; t < n; t += RT_WAVES) {
    const float* z = logits + t * totalp;
    float* choice = choices + wid * totalp;
    float mx = -INFINITY, inv = 1.0f;
    if (!a.sigmoid) {
      for (int e = lane; e < a.total; e += WAVE) mx = fmaxf(mx, z[e]);
      mx = wave_max(mx);
      float sum = 0.0f;
      for (int e = lane; e < a.total; e += WAVE) sum += expf(z[e] - mx);
      inv = 1.0f / wave_sum(sum);
    }
    auto score = [&](int e) {
      return a.sigmoid ? sigmoid_f(z[e]) : expf(z[e] - mx) * inv;
    };
    // a lane writes and reads only its own choices; logits order uncorrected
    // scores, also where those round to the same
    for (int e = lane; e < a.total; e += WAVE)
      choice[e] = a.correction ? score(e) + (float)((const T*)a.correction)[e]
                               : z[e];
    float picked = 0.0f, mine = 0.0f;
    int my_e = 0;
    for (int k = 0; k < a.top; ++k) {
      float best = -INFINITY;
      int at = a.total;
      for (int e = lane; e < a.total; e += WAVE)
        if (choice[e] > best) {
          best = choice[e];
          at = e;
        }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float v = __shfl_xor(best, o, WAVE);
        const int w = __shfl_xor(at, o, WAVE);
        if (v > best || (v == best && w < at)) {
          best = v;
          at = w;
        }
      }
      at = min(at, a.total - 1);
      if (at % WAVE == lane) choice[at] = -INFINITY;
      const float s = score(at);  // without the correction
      picked += s;
      if (lane == k % WAVE) {
        mine = s;
        my_e = at;
      }
      // a full round of lanes, or the last ones: store what they hold
      if (k % WAVE == WAVE - 1 || k == a.top - 1) {
        const int base = k / WAVE * WAVE;
        if (base + lane <= k) {
          const long p = (t0 + t) * a.top + base + lane;
          a.idx[p] = my_e;
          a.weight[p] = mine;
          a.rank[p] = my_e < a.experts ? atomicAdd(&counts[my_e], 1) : 0;
        }
      }
    }
    if (!a.normalize) continue;
    const float by = 1.0f / (picked + 1e-20f);
    for (int k = lane; k < a.top; k += WAVE)
      a.weight[(t0 + t) * a.top + k] *= by;
  }
  __syncthreads();
  for (int e = tid; e < a.experts; e += RT_BLOCK)
    a.hist[(long)blockIdx.x * a.experts + e] = counts[e];
}

extern "C" void launch_expert_route(const RouteArgs* a, bool f32,
                                    hipStream_t stream) {
  const int totalp = (a->total + 63) / 64 * 64;
  const int parts = RT_PARTS * EX_TOK * RT_LS, picks = RT_WAVES * totalp;
  const size_t smem = (size_t)((parts > picks ? parts : picks) +
                               EX_TOK * totalp + a->experts) * 4;
  const dim3 grid((unsigned)((a->n + EX_TOK - 1) / EX_TOK));
#define EX_GO(T)                                                            \
  do {                                                                      \
    (void)hipFuncSetAttribute(                                              \
        reinterpret_cast<const void*>(&expert_route_kernel<T>),             \
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);             \
    expert_route_kernel<T><<<grid, dim3(RT_BLOCK), smem, stream>>>(*a);     \
  } while (0)
  if (f32) EX_GO(float);
  else EX_GO(__bf16);
#undef EX_GO
}

// ---------------------------------------------------------------------------
// Placement.  Every block sums the histograms of all router blocks and of those
// before its own EX_GROUPS ones, and places its own pairs; the first block also
// writes the tiles.  EP: experts side by side, PB / EP rows at a time.
// ---------------------------------------------------------------------------

#define PB 1024

__global__ __launch_bounds__(PB) void expert_plan_kernel(const PlanArgs a,
                                                         int EP) {
  __shared__ int all[PB], before[PB];         // partial sums, then by expert
  __shared__ int start[EX_MAXTOTAL + 1], first[EX_MAXTOTAL + 1];
  __shared__ int wsum[2][PB / WAVE];
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1), wid = tid / WAVE;
  const int b0 = blockIdx.x * EX_GROUPS;
  const int e = tid % EP, r0 = tid / EP, rows = PB / EP;
  int sum = 0, prev = 0;
  if (e < a.experts) {
    const int* h = a.hist + e;
#pragma unroll 8
    for (int r = r0; r < a.n_blocks; r += rows) {
      const int v = h[(long)r * a.experts];
      sum += v;
      prev += r < b0 ? v : 0;
    }
  }
  all[tid] = sum;
  before[tid] = prev;
  __syncthreads();
  for (int o = rows / 2; o > 0; o >>= 1) {
    if (r0 < o) {
      all[tid] += all[tid + o * EP];
      before[tid] += before[tid + o * EP];
    }
    __syncthreads();
  }
  // exclusive sums over experts of pairs and of tiles
  const int pairs = tid < a.experts ? all[tid] : 0;
  const int cuts = (pairs + a.tile - 1) / a.tile;
  int sp = pairs, st = cuts;
#pragma unroll
  for (int o = 1; o < WAVE; o <<= 1) {
    const int u = __shfl_up(sp, o, WAVE), v = __shfl_up(st, o, WAVE);
    if (lane >= o) {
      sp += u;
      st += v;
    }
  }
  if (lane == WAVE - 1) {
    wsum[0][wid] = sp;
    wsum[1][wid] = st;
  }
  __syncthreads();
  for (int w = 0; w < wid; ++w) {
    sp += wsum[0][w];
    st += wsum[1][w];
  }
  if (tid < a.experts) {
    start[tid] = sp - pairs;
    first[tid] = st - cuts;
  }
  if (tid == PB - 1) first[EX_MAXTOTAL] = st;
  __syncthreads();

  if (blockIdx.x == 0) {
    if (tid < a.experts) {
      for (int i = 0; i < cuts; ++i) {
        int* t = a.tiles + (long)(first[tid] + i) * 3;
        t[0] = tid;
        t[1] = start[tid] + i * a.tile;
        t[2] = min(a.tile, pairs - i * a.tile);
      }
    }
    for (int i = first[EX_MAXTOTAL] + tid; i < a.n_tiles; i += PB) {
      int* t = a.tiles + (long)i * 3;
      t[0] = t[1] = t[2] = 0;
    }
  }
  const long lo = (long)b0 * EX_TOK * a.top;
  const long hi = min(a.n, (long)(b0 + EX_GROUPS) * EX_TOK) * a.top;
  for (long p = lo + tid; p < hi; p += PB) {
    const int x = a.idx[p];
    if (x >= a.experts) {
      a.where[p] = -1;
      continue;
    }
    const int b = (int)(p / (EX_TOK * a.top));
    int at = start[x] + before[x] + a.rank[p];
    for (int r = b0; r < b; ++r) at += a.hist[(long)r * a.experts + x];
    a.where[p] = at;
    a.tokens[at] = (int)(p / a.top);
    if (a.weight) a.scale[at] = a.weight[p];
  }
}

extern "C" void launch_expert_plan(const PlanArgs* a, hipStream_t stream) {
  int EP = 1;
  while (EP < a->experts) EP *= 2;
  const int blocks = (a->n_blocks + EX_GROUPS - 1) / EX_GROUPS;
  expert_plan_kernel<<<dim3((unsigned)blocks), dim3(PB), 0, stream>>>(*a, EP);
}

// ---------------------------------------------------------------------------
// Few tokens per expert.  A block makes 32 outputs of up to 16 pairs; its waves
// split the contraction, operands go from memory to registers, partial sums
// meet in LDS.  The same body serves the gate of token rows, whose input is the
// fp32 residual.
// ---------------------------------------------------------------------------

#define SK_OUT 32

// 8 elements of a row of X as operand of type T
template <typename T>
__device__ __forceinline__ void load_as(Frag<T>& f, const T* p) {
  f.load(p);
}
__device__ __forceinline__ void load_as(Frag<__bf16>& f, const float* p) {
  const f32x4 u = load4(p), v = load4(p + 4);
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    f.v[j] = (__bf16)u[j];
    f.v[j + 4] = (__bf16)v[j];
  }
}

// red[wave][token][output] <- partial sums; w0, w1: this lane's weights of two
// tiles, WS elements from step to step; xr: its row of X
template <typename T, typename X, int WS>
__device__ __forceinline__ void skinny_sums(const T* w0, const T* w1,
                                            const X* xr, int K, int wid, int lr,
                                            int lg,
                                            float (*red)[16][SK_OUT + 4]) {
  constexpr int U = sizeof(T) == 2 ? 8 : 4;
  const int steps = K / 32;
  const int per = (steps + EX_WAVES - 1) / EX_WAVES;
  int s = wid * per;
  const int s1 = min(steps, s + per);
  f32x4 c0 = {0, 0, 0, 0}, c1 = {0, 0, 0, 0};
  for (; s + U <= s1; s += U) {
    Frag<T> a0[U], a1[U], b[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      a0[u].load(w0 + (s + u) * WS);
      a1[u].load(w1 + (s + u) * WS);
      load_as(b[u], xr + (s + u) * 32);
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      c0 = mma(a0[u], b[u], c0);
      c1 = mma(a1[u], b[u], c1);
    }
  }
  for (; s < s1; ++s) {
    Frag<T> a0, a1, b;
    a0.load(w0 + s * WS);
    a1.load(w1 + s * WS);
    load_as(b, xr + s * 32);
    c0 = mma(a0, b, c0);
    c1 = mma(a1, b, c1);
  }
  store4(&red[wid][lr][lg * 4], c0);
  store4(&red[wid][lr][16 + lg * 4], c1);
  __syncthreads();
}

// grid (output blocks, tiles).  GLU: 16 gated units, the first weight tile is
// their gate's, the second their up projection's.
template <typename T, bool GLU>
__global__ __launch_bounds__(EX_BLOCK) void expert_skinny_kernel(
    const ExpertGemmArgs a) {
  __shared__ __attribute__((aligned(16))) float red[EX_WAVES][16][SK_OUT + 4];
  const int* tile = a.tiles + (long)blockIdx.y * 3;
  const int e = tile[0], p0 = tile[1], n = tile[2];
  if (n == 0) return;
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, lg = lane >> 4;
  constexpr int OUT = GLU ? SK_OUT / 2 : SK_OUT;
  const int outs = GLU ? a.O / 2 : a.O;
  const int o0 = blockIdx.x * OUT;
  const T* w = (const T*)a.w + (long)e * a.O * a.K + lg * 8;
  const long p = p0 + min(lr, n - 1);
  const long row = a.tokens ? a.tokens[p] : p;
  const int r0 = min(o0 + lr, outs - 1);
  const int r1 = GLU ? outs + r0 : min(o0 + 16 + lr, outs - 1);
  skinny_sums<T, T, 32>(w + (long)r0 * a.K, w + (long)r1 * a.K,
                        (const T*)a.x + row * a.xstride + lg * 8, a.K, wid, lr,
                        lg, red);
  for (int i = tid; i < n * OUT; i += EX_BLOCK) {
    const int t = i / OUT, o = i % OUT;
    if (o0 + o >= outs) continue;
    float v = 0.0f, u = 0.0f;
#pragma unroll
    for (int k = 0; k < EX_WAVES; ++k) {
      v += red[k][t][o];
      if (GLU) u += red[k][t][16 + o];
    }
    const float scale = a.scale ? a.scale[p0 + t] : 1.0f;
    v *= scale;
    if constexpr (GLU) {
      v = clamped_glu_of<T>(v, u * scale, a.limit, a.alpha);
    } else if (a.act == EX_RELU2) {
      v = fmaxf(v, 0.0f);
      v *= v;
    }
    ((T*)a.out)[(p0 + t) * a.ostride + o0 + o] = (T)v;
  }
}

// gelu, tanh form
__device__ __forceinline__ float gelu_tanh_f(float z) {
  return 0.5f * z *
         (1.0f + tanhf(0.79788456080286535588f * (z + 0.044715f * z * z * z)));
}

// grid (output blocks, token tiles): gelu_tanh(W x) * e
template <typename T>
__global__ __launch_bounds__(EX_BLOCK) void token_gate_kernel(
    const TokenGateArgs a) {
  __shared__ __attribute__((aligned(16))) float red[EX_WAVES][16][SK_OUT + 4];
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, lg = lane >> 4;
  const int o0 = blockIdx.x * SK_OUT, t0 = blockIdx.y * 16;
  const int n = min(16, a.n - t0);
  // operands of 16 outputs by 32 columns lie together, lane after lane
  const int tiles = (a.O + 15) / 16;
  const T* w = (const T*)a.w + lane * 8;
  skinny_sums<T, float, 512>(
      w + (long)(o0 / 16) * a.K * 16,
      w + (long)min(o0 / 16 + 1, tiles - 1) * a.K * 16,
      a.x + (long)(t0 + min(lr, n - 1)) * a.K + lg * 8, a.K, wid, lr, lg, red);
  for (int i = tid; i < n * SK_OUT; i += EX_BLOCK) {
    const int t = i / SK_OUT, o = o0 + i % SK_OUT;
    if (o >= a.O) continue;
    float v = 0.0f;
#pragma unroll
    for (int k = 0; k < EX_WAVES; ++k) v += red[k][t][i % SK_OUT];
    const float e = (float)((const T*)a.e)[(t0 + t) * a.estride + o];
    ((T*)a.out)[(long)(t0 + t) * a.O + o] = (T)(gelu_tanh_f(v) * e);
  }
}

extern "C" void launch_token_gate(const TokenGateArgs* a, bool f32,
                                  hipStream_t stream) {
  const dim3 grid((unsigned)((a->O + SK_OUT - 1) / SK_OUT),
                  (unsigned)((a->n + 15) / 16));
  if (f32)
    token_gate_kernel<float><<<grid, dim3(EX_BLOCK), 0, stream>>>(*a);
  else
    token_gate_kernel<__bf16><<<grid, dim3(EX_BLOCK), 0, stream>>>(*a);
}

// ---------------------------------------------------------------------------
// Many tokens per expert.  A block takes 128 weight rows to up to 128 pairs, a
// wave 64 x 64 of them; of a gated unit, 16 rows of the gate and 16 of the up
// projection by turns, so that a lane has both halves of its outputs.  Rows of 128 bytes go to LDS without passing registers, the
// next step while this one is worked on; 16-byte pieces are swapped within a
// row (by the source address) so that reads of a column meet different banks.
// ---------------------------------------------------------------------------

#define WT_OUT 128
#define WT_TOK 128
#define WT_BYTES 128  // of a row per step

__device__ __forceinline__ void to_lds16(const void* src, void* dst) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) void*)src,
      (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

// contraction group kk of this step for row r
__device__ __forceinline__ void read_row(Frag<__bf16>& f, const char* base,
                                         int r, int kk, int lg) {
  const int q = kk * 4 + lg;
  f.load((const __bf16*)(base + r * WT_BYTES + ((q ^ (r & 7)) * 16)));
}
__device__ __forceinline__ void read_row(Frag<float>& f, const char* base,
                                         int r, int, int lg) {
  const int q = lg * 2;
  f.load44((const float*)(base + r * WT_BYTES + ((q ^ (r & 7)) * 16)),
           (const float*)(base + r * WT_BYTES + (((q + 1) ^ (r & 7)) * 16)));
}

// grid: one row of blocks per XCD, so that neighbouring tiles share an L2
template <typename T, bool GLU>
__global__ __launch_bounds__(EX_BLOCK, 2) void expert_wide_kernel(
    const ExpertGemmArgs a) {
  constexpr int STEP = WT_BYTES / (int)sizeof(T);   // elements per step
  constexpr int GROUPS = STEP / 32;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int obs = (a.O + WT_OUT - 1) / WT_OUT;
  const int work = obs * a.n_tiles;
  const int per = (work + 7) / 8;
  const int item = blockIdx.x % 8 * per + blockIdx.x / 8;
  if (item >= work || (int)blockIdx.x / 8 >= per) return;
  const int* tile = a.tiles + (long)(item / obs) * 3;
  const int e = tile[0], p0 = tile[1], n = tile[2];
  if (n == 0) return;
  const int o0 = item % obs * WT_OUT;
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lr = lane & 15, lg = lane >> 4;

  // a wave brings 32 rows of each operand, 8 at a time
  const int piece = ((lane & 7) ^ (lane >> 3)) * (16 / (int)sizeof(T));
  const T *ws[4], *xs[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = wid * 32 + i * 8 + (lane >> 3);
    int o = min(o0 + r, a.O - 1);
    if (GLU)
      o = r / 16 % 2 * (a.O / 2) + min(o0 / 2 + r / 32 * 16 + r % 16, a.O / 2 - 1);
    ws[i] = (const T*)a.w + ((long)e * a.O + o) * a.K + piece;
    const long p = p0 + min(r, n - 1);
    const long row = a.tokens ? a.tokens[p] : p;
    xs[i] = (const T*)a.x + row * a.xstride + piece;
  }
  auto stage = [&](int s, int buf) {
    char* base = smem + buf * (2 * WT_OUT * WT_BYTES) + wid * 32 * WT_BYTES;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      to_lds16(ws[i] + (long)s * STEP, base + i * 8 * WT_BYTES);
      to_lds16(xs[i] + (long)s * STEP,
               base + WT_OUT * WT_BYTES + i * 8 * WT_BYTES);
    }
  };
  const int wo = wid % 2 * 64, wt = wid / 2 * 64;  // this wave's corner
  f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0, 0, 0, 0};

  const int steps = a.K / STEP;
  stage(0, 0);
  for (int s = 0; s < steps; ++s) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (s + 1 < steps) stage(s + 1, (s + 1) & 1);
    const char* wb = smem + (s & 1) * (2 * WT_OUT * WT_BYTES);
    const char* xb = wb + WT_OUT * WT_BYTES;
#pragma unroll
    for (int kk = 0; kk < GROUPS; ++kk) {
      Frag<T> fw[4], fx[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        read_row(fw[i], wb, wo + i * 16 + lr, kk, lg);
        read_row(fx[i], xb, wt + i * 16 + lr, kk, lg);
      }
      // the block that multiplies goes before the one that loads
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mma(fw[i], fx[j], acc[i][j]);
      __builtin_amdgcn_s_setprio(0);
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = wt + j * 16 + lr;
    if (t >= n) continue;
    T* out = (T*)a.out + (long)(p0 + t) * a.ostride;
    const float scale = a.scale ? a.scale[p0 + t] : 1.0f;
    const int outs = GLU ? a.O / 2 : a.O;
#pragma unroll
    for (int i = 0; i < 4; i += GLU ? 2 : 1) {
      const int o = GLU ? (o0 + wo) / 2 + i * 8 + lg * 4
                        : o0 + wo + i * 16 + lg * 4;
      f32x4 v = acc[i][j];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        v[k] *= scale;
        if constexpr (GLU) {
          v[k] = clamped_glu_of<T>(v[k], acc[i + 1][j][k] * scale, a.limit, a.alpha);
        } else if (a.act == EX_RELU2) {
          v[k] = fmaxf(v[k], 0.0f);
          v[k] *= v[k];
        }
      }
      if (o + 4 <= outs) {
        store4(out + o, v);  // rows of out begin at whole vectors
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (o + k < outs) out[o + k] = (T)v[k];
      }
    }
  }
}

extern "C" void launch_expert_gemm(const ExpertGemmArgs* a, int tile, bool f32,
                                   hipStream_t stream) {
  const bool glu = a->act == EX_CLAMPED_GLU;
  const dim3 block(EX_BLOCK);
  if (tile == 16) {
    const dim3 grid((unsigned)((a->O + SK_OUT - 1) / SK_OUT),
                    (unsigned)a->n_tiles);
#define EX_GO(T)                                                     \
  do {                                                               \
    if (glu)                                                         \
      expert_skinny_kernel<T, true><<<grid, block, 0, stream>>>(*a); \
    else                                                             \
      expert_skinny_kernel<T, false><<<grid, block, 0, stream>>>(*a); \
  } while (0)
    if (f32) EX_GO(float);
    else EX_GO(__bf16);
#undef EX_GO
    return;
  }
  const size_t smem = 2 * 2 * WT_OUT * WT_BYTES;
  const long work = (long)((a->O + WT_OUT - 1) / WT_OUT) * a->n_tiles;
  const dim3 grid((unsigned)((work + 7) / 8 * 8));
#define EX_GO(T)                                                      \
  do {                                                                \
    if (glu)                                                          \
      expert_wide_kernel<T, true><<<grid, block, smem, stream>>>(*a); \
    else                                                              \
      expert_wide_kernel<T, false><<<grid, block, smem, stream>>>(*a); \
  } while (0)
  if (f32) EX_GO(float);
  else EX_GO(__bf16);
#undef EX_GO
}

// ---------------------------------------------------------------------------
// x[t] += sum_k weight * (d[where] or, for an identity expert, h[t])
// ---------------------------------------------------------------------------

template <typename T, int V>
__global__ __launch_bounds__(EX_BLOCK) void expert_combine_kernel(
    const CombineArgs a) {
  const long t = blockIdx.x;
  const int* where = a.where + t * a.top;
  const float* weight = a.weight + t * a.top;
  const T* h = (const T*)a.h + t * a.hstride;
  float* x = a.x + t * a.W;
  const int c = (blockIdx.y * EX_BLOCK + threadIdx.x) * V;
  if (c < a.W) {
    float s[V];
#pragma unroll
    for (int i = 0; i < V; ++i) s[i] = 0.0f;
#pragma unroll 4
    for (int k = 0; k < a.top; ++k) {
      const int p = where[k];
      const float w = weight[k];
      const T* src = p < 0 ? h : (const T*)a.d + (long)p * a.dstride;
      if constexpr (V == 4) {
        const f32x4 v = load4(src + c);
#pragma unroll
        for (int i = 0; i < 4; ++i) s[i] += w * v[i];
      } else {
        s[0] += w * (float)src[c];
      }
    }
    if constexpr (V == 4) {
      f32x4 v = load4(x + c);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] += s[i];
      store4(x + c, v);
      if (a.copy) store4((T*)a.copy + t * a.W + c, v);
    } else {
      const float v = x[c] + s[0];
      x[c] = v;
      if (a.copy) ((T*)a.copy)[t * a.W + c] = (T)v;
    }
  }
}

extern "C" void launch_expert_combine(const CombineArgs* a, bool f32,
                                      hipStream_t stream) {
  const bool vec = a->W % 4 == 0;
  const int per = EX_BLOCK * (vec ? 4 : 1);
  const dim3 grid((unsigned)a->n, (unsigned)((a->W + per - 1) / per));
  const dim3 block(EX_BLOCK);
#define EX_GO(T)                                                  \
  do {                                                            \
    if (vec) \
      expert_combine_kernel<T, 4><<<grid, block, 0, stream>>>(*a); \
    else \
      expert_combine_kernel<T, 1><<<grid, block, 0, stream>>>(*a);     \
  } while (0)
  if (f32) EX_GO(float);
  else EX_GO(__bf16);
#undef EX_GO
}
