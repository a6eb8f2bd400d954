// Shared pieces of the ragged-batch kernels (paged latent attention, gated
// delta rule, fp32-residual norms).
//
// Every kernel is a template over the element type T of activations and
// weights: __bf16 (serving) or float (true 32-bit arithmetic throughout).
// Matrix products go through one abstraction, a 16x16 tile with a contraction
// step of 32:
//   A (16x32): lane holds row l&15,  8 elements of contraction group l>>4
//   B (32x16): lane holds col l&15,  8 elements of contraction group l>>4
//   C (16x16): lane holds col l&15,  rows (l>>4)*4 + 0..3
// bf16: one mfma_f32_16x16x32_bf16.  float: eight mfma_f32_16x16x4_f32, step s
// contracting element s of every group — the same operands, true fp32.
// The order of contraction indices inside the step is free as long as A and B
// agree, which the attention kernels use to feed scores back without a
// shuffle.
#pragma once

#include "hip_common.h"

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

#define RG_PAGE 64  // tokens per cache page

template <typename T>
struct Frag;

template <>
struct Frag<__bf16> {
  bf16x8 v;
  __device__ __forceinline__ void load(const __bf16* p) {
    v = *reinterpret_cast<const bf16x8*>(p);
  }
  // elements 0..3 from p0, 4..7 from p1
  __device__ __forceinline__ void load44(const __bf16* p0, const __bf16* p1) {
    bf16x4 a = *reinterpret_cast<const bf16x4*>(p0);
    bf16x4 b = *reinterpret_cast<const bf16x4*>(p1);
    v = __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
  }
  __device__ __forceinline__ void load_strided(const __bf16* p, int stride) {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = p[j * stride];
  }
};

template <>
struct Frag<float> {
  f32x4 a, b;
  __device__ __forceinline__ void load(const float* p) {
    a = *reinterpret_cast<const f32x4*>(p);
    b = *reinterpret_cast<const f32x4*>(p + 4);
  }
  __device__ __forceinline__ void load44(const float* p0, const float* p1) {
    a = *reinterpret_cast<const f32x4*>(p0);
    b = *reinterpret_cast<const f32x4*>(p1);
  }
  __device__ __forceinline__ void load_strided(const float* p, int stride) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      a[j] = p[j * stride];
      b[j] = p[(j + 4) * stride];
    }
  }
};

__device__ __forceinline__ f32x4 mma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

__device__ __forceinline__ f32x4 mma(const Frag<__bf16>& a,
                                     const Frag<__bf16>& b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}

__device__ __forceinline__ f32x4 mma(const Frag<float>& a,
                                     const Frag<float>& b, f32x4 c) {
#pragma unroll
  for (int s = 0; s < 4; ++s) c = mma4(a.a[s], b.a[s], c);
#pragma unroll
  for (int s = 0; s < 4; ++s) c = mma4(a.b[s], b.b[s], c);
  return c;
}

// Softmax weights (fp32) times A: in bf16 the weights enter as a high and a low
// part, so that they keep about 16 bits instead of 8.
__device__ __forceinline__ f32x4 mma_weights(const Frag<__bf16>& a,
                                             const Frag<__bf16>& hi,
                                             const Frag<__bf16>& lo, f32x4 c) {
  c = mma(a, hi, c);
  return mma(a, lo, c);
}

__device__ __forceinline__ f32x4 mma_weights(const Frag<float>& a,
                                             const Frag<float>& hi,
                                             const Frag<float>&, f32x4 c) {
  return mma(a, hi, c);
}

__device__ __forceinline__ void split_weights(const float (&p)[8],
                                              Frag<__bf16>& hi,
                                              Frag<__bf16>& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const __bf16 h = (__bf16)p[j];
    hi.v[j] = h;
    lo.v[j] = (__bf16)(p[j] - (float)h);
  }
}

__device__ __forceinline__ void split_weights(const float (&p)[8],
                                              Frag<float>& hi, Frag<float>&) {
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    hi.a[j] = p[j];
    hi.b[j] = p[j + 4];
  }
}

// exp of a non-positive softmax argument
template <typename T>
__device__ __forceinline__ float softmax_exp(float x);
template <>
__device__ __forceinline__ float softmax_exp<__bf16>(float x) {
  return __expf(x);
}
template <>
__device__ __forceinline__ float softmax_exp<float>(float x) {
  return expf(x);
}

// four consecutive elements
__device__ __forceinline__ void store4(__bf16* p, f32x4 v) {
  bf16x4 o;
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = (__bf16)v[j];
  *reinterpret_cast<bf16x4*>(p) = o;
}
__device__ __forceinline__ void store4(float* p, f32x4 v) {
  *reinterpret_cast<f32x4*>(p) = v;
}
__device__ __forceinline__ f32x4 load4(const __bf16* p) {
  bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
  return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}
__device__ __forceinline__ f32x4 load4(const float* p) {
  return *reinterpret_cast<const f32x4*>(p);
}

// 8 elements, one (bf16) or two (float) 16-byte moves
__device__ __forceinline__ void copy8(__bf16* d, const __bf16* s) {
  *reinterpret_cast<bf16x8*>(d) = *reinterpret_cast<const bf16x8*>(s);
}
__device__ __forceinline__ void copy8(float* d, const float* s) {
  reinterpret_cast<f32x4*>(d)[0] = reinterpret_cast<const f32x4*>(s)[0];
  reinterpret_cast<f32x4*>(d)[1] = reinterpret_cast<const f32x4*>(s)[1];
}
__device__ __forceinline__ void zero8(__bf16* d) {
  *reinterpret_cast<f32x4*>(d) = f32x4{0, 0, 0, 0};
}
__device__ __forceinline__ void zero8(float* d) {
  reinterpret_cast<f32x4*>(d)[0] = f32x4{0, 0, 0, 0};
  reinterpret_cast<f32x4*>(d)[1] = f32x4{0, 0, 0, 0};
}

__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float sigmoid_f(float x) {
  return 1.0f / (1.0f + expf(-x));
}
__device__ __forceinline__ float softplus_f(float x) {
  return fmaxf(x, 0.0f) + log1pf(expf(-fabsf(x)));
}

// sigmoid for bf16 results from the hardware's power of two, off by about 1e-7
template <typename T>
__device__ __forceinline__ float sigmoid_of(float x);
template <>
__device__ __forceinline__ float sigmoid_of<float>(float x) {
  return sigmoid_f(x);
}
template <>
__device__ __forceinline__ float sigmoid_of<__bf16>(float x) {
  return __builtin_amdgcn_rcpf(
      1.0f + __builtin_amdgcn_exp2f(-1.44269504088896340736f * x));
}

// ln(1 + e^x).  For bf16 operands: the logarithm of 1 + u from the instruction
// where u is not small, else its series; both to about 1e-6 of the result.
template <typename T>
__device__ __forceinline__ float softplus_of(float x);
template <>
__device__ __forceinline__ float softplus_of<float>(float x) {
  return softplus_f(x);
}
template <>
__device__ __forceinline__ float softplus_of<__bf16>(float d) {
  const float u = __builtin_amdgcn_exp2f(-1.44269504088896340736f * fabsf(d));
  const float large = 0.69314718055994530942f * __builtin_amdgcn_logf(1.0f + u);
  // u - u^2/2 + ... + u^5/5, off by u^6/6
  float small = fmaf(u, 0.2f, -0.25f);
  small = fmaf(u, small, 0.33333333333333333333f);
  small = fmaf(u, small, -0.5f);
  small = fmaf(u, small * u, u);
  return fmaxf(d, 0.0f) + (u < 0.04f ? small : large);
}

// g sigmoid(alpha g) (u + 1), g at most `limit`, u within +-limit
template <typename T>
__device__ __forceinline__ float clamped_glu_of(float g, float u, float limit,
                                                float alpha) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_of<T>(alpha * g) * (u + 1.0f);
}
