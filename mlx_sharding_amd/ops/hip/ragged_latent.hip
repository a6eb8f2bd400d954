// Latent attention over a ragged batch and a paged cache of latent rows.
//
// Two kernels, one per way of reading the cache:
//  * absorbed (short portions, decoding): W_uk is folded into the query and
//    W_uv into the output, so all heads attend the cached rows themselves —
//    rank + rot values per key instead of heads * (dim + rot + vdim).
//  * expanded (long portions): keys and values of the whole prefix are made
//    from the gathered rows by library GEMMs, then ordinary causal attention.
// Scores and weights stay fp32; bf16 weights enter the value product as a
// high and a low part.
#include "ragged_common.h"

#define LA_BLOCK 256
#define LA_KT 32  // keys per tile, absorbed
#define LA_MAXSPLIT WAVE

// ---------------------------------------------------------------------------
// Absorbed.  A query row is one (token, head) pair of one request; a block
// serves 16 rows of one request over one slice of its keys.  The key tile is
// staged once in LDS, row-major, and read as rows (scores) and as columns
// (values).  Scores are computed transposed (keys x rows), so a lane holds
// one query row and the softmax needs two shuffles.
//   grid (short requests, splits, row tiles)
// ND: 16-wide latent column tiles per wave; rankp == 64 * ND.
// ---------------------------------------------------------------------------

template <typename T, int ND>
__global__ __launch_bounds__(LA_BLOCK) void latent_attn_short_kernel(
    const T* __restrict__ q_abs,  // [H, Nt, rankp]
    const T* __restrict__ q,      // row qstride, head dq, rotated part at qoff
    const T* __restrict__ pool,   // rows of rankp + rotp
    T* __restrict__ out,          // [H, Nt, rankp]             (1 split)
    float* __restrict__ part_o,   // [H, Nt, splits, rankp]
    float* __restrict__ part_ml,  // [H, Nt, splits, 2]
    const int* __restrict__ cu, const int* __restrict__ pos0,
    const int* __restrict__ pages, int P, int H, int Nt, long qstride, int dq,
    int qoff, int rotp, float scale) {
  constexpr int rankp = 64 * ND;
  const int e = blockIdx.x;
  const int split = blockIdx.y;
  const int nsplit = gridDim.y;
  const int r0 = blockIdx.z * 16;
  const int t0 = cu[e];
  const int rows = (cu[e + 1] - t0) * H;
  if (r0 >= rows) return;
  const int p0 = pos0[e];
  const int last_tok = min(r0 + 15, rows - 1) / H;
  const int S = p0 + last_tok + 1;       // keys any row of this tile sees
  const int tiles = (S + LA_KT - 1) / LA_KT;
  const int per = (tiles + nsplit - 1) / nsplit * LA_KT;
  const int lo = split * per;
  const int hi = min(S, lo + per);

  const int W = rankp + rotp;
  const int WS = W + 8;
  const int nvec = W / 8;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  T* qs = reinterpret_cast<T*>(smem);    // [16][WS]
  T* ks = qs + 16 * WS;                  // [LA_KT][WS]
  float* sp = reinterpret_cast<float*>(ks + LA_KT * WS);  // [2][LA_KT][17]

  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = tid / WAVE;
  const int lr = lane & 15, lg = lane >> 4;

  for (int i = tid; i < 16 * nvec; i += LA_BLOCK) {
    const int r = i / nvec, c = (i - r * nvec) * 8;
    const int row = min(r0 + r, rows - 1);
    const int tok = row / H, h = row - tok * H;
    const T* src = c < rankp
                       ? q_abs + ((long)h * Nt + t0 + tok) * rankp + c
                       : q + (long)(t0 + tok) * qstride + (long)h * dq + qoff +
                             (c - rankp);
    copy8(qs + r * WS + c, src);
  }

  const int my_row = min(r0 + lr, rows - 1);
  const int my_tok = my_row / H;
  const int my_head = my_row - my_tok * H;
  const int limit = min(p0 + my_tok + 1, hi);

  float m_run = -1e30f, l_run = 0.0f;
  f32x4 acc[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) acc[d] = f32x4{0, 0, 0, 0};

  const int sub = wid & 1, part = wid >> 1;
  const int nk = W / 32;
  const int k_lo = part ? (nk + 1) / 2 : 0;
  const int k_hi = part ? nk : (nk + 1) / 2;

  for (int t = lo; t < hi; t += LA_KT) {
    __syncthreads();
    {
      const long page = pages[(long)e * P + t / RG_PAGE];
      const T* src = pool + (page * RG_PAGE + t % RG_PAGE) * (long)W;
      const int valid = min(LA_KT, S - t);
      for (int i = tid; i < LA_KT * nvec; i += LA_BLOCK) {
        const int r = i / nvec, c = (i - r * nvec) * 8;
        if (r < valid)
          copy8(ks + r * WS + c, src + (long)r * W + c);
        else
          zero8(ks + r * WS + c);
      }
    }
    __syncthreads();
    {
      f32x4 c4 = {0, 0, 0, 0};
      const T* ka = ks + (sub * 16 + lr) * WS + lg * 8;
      const T* qb = qs + lr * WS + lg * 8;
      for (int k = k_lo; k < k_hi; ++k) {
        Frag<T> a, b;
        a.load(ka + k * 32);
        b.load(qb + k * 32);
        c4 = mma(a, b, c4);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        sp[(part * LA_KT + sub * 16 + lg * 4 + j) * 17 + lr] = c4[j];
    }
    __syncthreads();
    float p[8];
    float mx = -1e30f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int k = lg * 8 + j;
      const float s =
          (sp[k * 17 + lr] + sp[(LA_KT + k) * 17 + lr]) * scale;
      p[j] = (t + k < limit) ? s : -1e30f;
      mx = fmaxf(mx, p[j]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
    const float m_new = fmaxf(m_run, mx);
    const float alpha = softmax_exp<T>(m_run - m_new);
    m_run = m_new;
    float sum = 0.0f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      p[j] = (p[j] <= -1e29f) ? 0.0f : softmax_exp<T>(p[j] - m_new);
      sum += p[j];
    }
    sum += __shfl_xor(sum, 16, WAVE);
    sum += __shfl_xor(sum, 32, WAVE);
    l_run = l_run * alpha + sum;
    Frag<T> ph, pl;
    split_weights(p, ph, pl);
    const T* va = ks + (lg * 8) * WS + wid * ND * 16 + lr;
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      Frag<T> a;
      a.load_strided(va + d * 16, WS);
      f32x4 c4 = acc[d];
#pragma unroll
      for (int j = 0; j < 4; ++j) c4[j] *= alpha;
      acc[d] = mma_weights(a, ph, pl, c4);
    }
  }

  if (r0 + lr >= rows) return;
  const long orow = (long)my_head * Nt + t0 + my_tok;
  const int dcol = wid * ND * 16 + lg * 4;
  if (nsplit == 1) {
    const float rinv = 1.0f / l_run;
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      f32x4 c4 = acc[d];
#pragma unroll
      for (int j = 0; j < 4; ++j) c4[j] *= rinv;
      store4(out + orow * rankp + dcol + d * 16, c4);
    }
    return;
  }
  float* po = part_o + (orow * nsplit + split) * rankp + dcol;
#pragma unroll
  for (int d = 0; d < ND; ++d) store4(po + d * 16, acc[d]);
  if (wid == 0 && lg == 0) {
    part_ml[(orow * nsplit + split) * 2] = m_run;
    part_ml[(orow * nsplit + split) * 2 + 1] = l_run;
  }
}

// One block per (head, token): merges the slices of the keys.
template <typename T>
__global__ __launch_bounds__(128) void latent_attn_merge_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml,
    T* __restrict__ out, int nsplit, int rankp) {
  const long row = blockIdx.x;
  const float* ml = part_ml + row * nsplit * 2;
  __shared__ float w[LA_MAXSPLIT];  // weight of each slice
  if (threadIdx.x < WAVE) {
    const int s = threadIdx.x;
    const float ms = s < nsplit ? ml[2 * s] : -1e30f;
    const float m = wave_max(ms);
    const float e = s < nsplit ? softmax_exp<T>(ms - m) : 0.0f;
    const float l = wave_sum(s < nsplit ? ml[2 * s + 1] * e : 0.0f);
    w[s] = e / l;
  }
  __syncthreads();
  for (int d = threadIdx.x * 4; d < rankp; d += 512) {
    const float* p = part_o + row * nsplit * rankp + d;
    f32x4 o = {0, 0, 0, 0};
#pragma unroll 8
    for (int s = 0; s < nsplit; ++s) {
      const f32x4 v = load4(p + (long)s * rankp);
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] += v[j] * w[s];
    }
    store4(out + row * rankp + d, o);
  }
}

template <typename T>
static void latent_attn_short_t(const void* q_abs, const void* q,
                                const void* pool, void* out, float* part_o,
                                float* part_ml, const int* cu, const int* pos0,
                                const int* pages, int P, int H, int Nt,
                                long qstride, int dq, int qoff, int rankp,
                                int rotp, float scale, int n_req, int nsplit,
                                int row_tiles, hipStream_t stream) {
  const int WS = rankp + rotp + 8;
  const size_t smem =
      (size_t)(16 + LA_KT) * WS * sizeof(T) + 2 * LA_KT * 17 * sizeof(float);
  dim3 grid((unsigned)n_req, (unsigned)nsplit, (unsigned)row_tiles);
  dim3 block(LA_BLOCK);
#define LS_GO(N)                                                           \
  do {                                                                     \
    if (smem > 65536)                                                      \
      (void)hipFuncSetAttribute(                                           \
          reinterpret_cast<const void*>(&latent_attn_short_kernel<T, N>),  \
          hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);          \
    latent_attn_short_kernel<T, N><<<grid, block, smem, stream>>>(         \
        (const T*)q_abs, (const T*)q, (const T*)pool, (T*)out, part_o,     \
        part_ml, cu, pos0, pages, P, H, Nt, qstride, dq, qoff, rotp, scale); \
  } while (0)
  switch (rankp / 64) {
    case 1: LS_GO(1); break;
    case 2: LS_GO(2); break;
    case 4: LS_GO(4); break;
    case 8: LS_GO(8); break;
    default: LS_GO(16); break;
  }
#undef LS_GO
  if (nsplit > 1) {
    dim3 mgrid((unsigned)(H * Nt)), mblock(128);
    latent_attn_merge_kernel<T><<<mgrid, mblock, 0, stream>>>(
        part_o, part_ml, (T*)out, nsplit, rankp);
  }
}

extern "C" void launch_latent_attn_short(
    const void* q_abs, const void* q, const void* pool, void* out,
    float* part_o, float* part_ml, const int* cu, const int* pos0,
    const int* pages, int P, int H, int Nt, long qstride, int dq, int qoff,
    int rankp, int rotp, float scale, int n_req, int nsplit, int row_tiles,
    bool f32, hipStream_t stream) {
  if (f32)
    latent_attn_short_t<float>(q_abs, q, pool, out, part_o, part_ml, cu, pos0,
                               pages, P, H, Nt, qstride, dq, qoff, rankp, rotp,
                               scale, n_req, nsplit, row_tiles, stream);
  else
    latent_attn_short_t<__bf16>(q_abs, q, pool, out, part_o, part_ml, cu, pos0,
                                pages, P, H, Nt, qstride, dq, qoff, rankp,
                                rotp, scale, n_req, nsplit, row_tiles, stream);
}
