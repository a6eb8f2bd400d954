// Expanded latent attention for long portions (flash style, causal, ragged).
//
// Block: 4 waves x 32 query rows of one head; key tiles of 64.  Scores are
// computed transposed (keys x queries): a lane holds one query per group and
// its scores are, without any shuffle, the B operand of the value product
// O^T = V^T P^T, because the contraction order over keys is free.  V arrives
// already transposed ([heads * vdim, keys], straight from the GEMM that
// expands the latent), so both operands are vector loads.
//
//   grid (heads, query tiles): neighbouring blocks are different heads, and
//   blocks go round the XCDs, so a head's keys stay in one XCD's L2.
//   tiles[i] = (request, first query row within the portion)
#pragma once

#include "ragged_common.h"

#define LP_BLOCK 256
#define LP_QT 128
#define LP_KT 64

template <typename T, int NKS, int NDH>
__global__ __launch_bounds__(LP_BLOCK) void latent_attn_long_kernel(
    const T* __restrict__ q,    // row qstride, head dq: [dimp | rotp]
    const T* __restrict__ kx,   // [St, H * dimp]
    const T* __restrict__ lat,  // [St, rankp + rotp]
    const T* __restrict__ vt,   // [H * vdp, St]
    T* __restrict__ out,        // [long tokens, H * vdp]
    const int* __restrict__ tiles, const int* __restrict__ cu,
    const int* __restrict__ pos0, const int* __restrict__ cuk, int n_short,
    int tok_base, long St, int H, long qstride, int dq, int dimp, int rankp,
    int W, float scale) {
  constexpr int KS = NKS * 32 + 8;
  constexpr int VS = LP_KT + 8;
  constexpr int vdp = NDH * 16;
  const int h = blockIdx.x;
  const int e = tiles[2 * blockIdx.y];
  const int q0 = tiles[2 * blockIdx.y + 1];
  const int t0 = cu[e];
  const int n = cu[e + 1] - t0;
  const int p0 = pos0[e];
  const long kb = cuk[e - n_short];
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wid = tid / WAVE;
  const int lr = lane & 15, lg = lane >> 4;

  extern __shared__ __attribute__((aligned(16))) char smem[];
  T* ks = reinterpret_cast<T*>(smem);  // [LP_KT][KS]
  T* vs = ks + LP_KT * KS;             // [vdp][VS]

  Frag<T> qf[2][NKS];
  int qpos[2];
#pragma unroll
  for (int g = 0; g < 2; ++g) {
    const int r = min(q0 + wid * 32 + g * 16 + lr, n - 1);
    qpos[g] = p0 + r;
    const T* src = q + (long)(t0 + r) * qstride + (long)h * dq + lg * 8;
#pragma unroll
    for (int k = 0; k < NKS; ++k) {
      if (k * 32 < dq) qf[g][k].load(src + k * 32);
      else qf[g][k].load(src);  // meets zero key columns
    }
  }
  const int wave_hi = p0 + min(q0 + wid * 32 + 31, n - 1) + 1;
  const int hi = p0 + min(q0 + LP_QT, n);

  float m_run[2] = {-1e30f, -1e30f}, l_run[2] = {0.0f, 0.0f};
  f32x4 acc[2][NDH];
#pragma unroll
  for (int g = 0; g < 2; ++g)
#pragma unroll
    for (int d = 0; d < NDH; ++d) acc[g][d] = f32x4{0, 0, 0, 0};

  for (int t = 0; t < hi; t += LP_KT) {
    __syncthreads();
    for (int i = tid; i < LP_KT * NKS * 4; i += LP_BLOCK) {
      const int r = i / (NKS * 4), c = (i % (NKS * 4)) * 8;
      const long row = kb + t + r;
      if (c < dimp)
        copy8(ks + r * KS + c, kx + row * ((long)H * dimp) + (long)h * dimp + c);
      else if (c < dq)
        copy8(ks + r * KS + c, lat + row * W + rankp + (c - dimp));
      else
        zero8(ks + r * KS + c);
    }
    for (int i = tid; i < vdp * (LP_KT / 8); i += LP_BLOCK) {
      const int d = i / (LP_KT / 8), c = (i % (LP_KT / 8)) * 8;
      copy8(vs + d * VS + c, vt + ((long)h * vdp + d) * St + kb + t + c);
    }
    __syncthreads();
    if (t >= wave_hi) continue;

    f32x4 sc[2][4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      sc[0][s] = f32x4{0, 0, 0, 0};
      sc[1][s] = f32x4{0, 0, 0, 0};
      const T* ka = ks + (s * 16 + lr) * KS + lg * 8;
#pragma unroll
      for (int k = 0; k < NKS; ++k) {
        Frag<T> a;
        a.load(ka + k * 32);
        sc[0][s] = mma(a, qf[0][k], sc[0][s]);
        sc[1][s] = mma(a, qf[1][k], sc[1][s]);
      }
    }
    float alpha[2];
#pragma unroll
    for (int g = 0; g < 2; ++g) {
      float mx = -1e30f;
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int key = t + s * 16 + lg * 4 + j;
          const float v = key <= qpos[g] ? sc[g][s][j] * scale : -1e30f;
          sc[g][s][j] = v;
          mx = fmaxf(mx, v);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      const float m_new = fmaxf(m_run[g], mx);
      alpha[g] = softmax_exp<T>(m_run[g] - m_new);
      m_run[g] = m_new;
      float sum = 0.0f;
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float v = sc[g][s][j];
          const float p = v <= -1e29f ? 0.0f : softmax_exp<T>(v - m_new);
          sc[g][s][j] = p;
          sum += p;
        }
      sum += __shfl_xor(sum, 16, WAVE);
      sum += __shfl_xor(sum, 32, WAVE);
      l_run[g] = l_run[g] * alpha[g] + sum;
#pragma unroll
      for (int d = 0; d < NDH; ++d)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[g][d][j] *= alpha[g];
    }
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
      Frag<T> ph[2], pl[2];
#pragma unroll
      for (int g = 0; g < 2; ++g) {
        float p[8];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          p[j] = sc[g][2 * hh][j];
          p[4 + j] = sc[g][2 * hh + 1][j];
        }
        split_weights(p, ph[g], pl[g]);
      }
#pragma unroll
      for (int d = 0; d < NDH; ++d) {
        Frag<T> a;
        const T* va = vs + (d * 16 + lr) * VS + hh * 32 + lg * 4;
        a.load44(va, va + 16);
        acc[0][d] = mma_weights(a, ph[0], pl[0], acc[0][d]);
        acc[1][d] = mma_weights(a, ph[1], pl[1], acc[1][d]);
      }
    }
  }

#pragma unroll
  for (int g = 0; g < 2; ++g) {
    const int r = q0 + wid * 32 + g * 16 + lr;
    if (r >= n) continue;
    const float rinv = 1.0f / l_run[g];
    T* o = out + (long)(t0 - tok_base + r) * ((long)H * vdp) + (long)h * vdp +
           lg * 4;
#pragma unroll
    for (int d = 0; d < NDH; ++d) {
      f32x4 c4 = acc[g][d];
#pragma unroll
      for (int j = 0; j < 4; ++j) c4[j] *= rinv;
      store4(o + d * 16, c4);
    }
  }
}

struct LatentLongArgs {
  const void *q, *kx, *lat, *vt;
  void* out;
  const int *tiles, *cu, *pos0, *cuk;
  int n_short, tok_base, n_tiles, H, dq, dimp, rankp, W;
  long St, qstride;
  float scale;
};

template <typename T, int NKS, int NDH>
static void latent_attn_long_go(const LatentLongArgs& a, hipStream_t stream) {
  const size_t smem = ((size_t)LP_KT * (NKS * 32 + 8) +
                       (size_t)NDH * 16 * (LP_KT + 8)) * sizeof(T);
  if (smem > 65536)
    (void)hipFuncSetAttribute(
        reinterpret_cast<const void*>(&latent_attn_long_kernel<T, NKS, NDH>),
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  dim3 grid((unsigned)a.H, (unsigned)a.n_tiles), block(LP_BLOCK);
  latent_attn_long_kernel<T, NKS, NDH><<<grid, block, smem, stream>>>(
      (const T*)a.q, (const T*)a.kx, (const T*)a.lat, (const T*)a.vt,
      (T*)a.out, a.tiles, a.cu, a.pos0, a.cuk, a.n_short, a.tok_base, a.St,
      a.H, a.qstride, a.dq, a.dimp, a.rankp, a.W, a.scale);
}
