// Activation element types of the kernels that run in bf16 or wholly in 32-bit, and the scalar
// functions the fp32-residual designs add to dmath.h.
#pragma once

#include "dmath.h"

// value of an activation element, and an fp32 value as one (rounded for bf16)
__device__ __forceinline__ float act_f(bf16_t v) { return dm_bf2f(v); }
__device__ __forceinline__ float act_f(float v) { return v; }
template <typename A>
__device__ __forceinline__ A act_of(float v);
template <>
__device__ __forceinline__ bf16_t act_of<bf16_t>(float v) { return dm_f2bf(v); }
template <>
__device__ __forceinline__ float act_of<float>(float v) { return v; }

// N (4 or 8) consecutive elements, aligned to their size
template <int N>
__device__ __forceinline__ void act_load(const bf16_t* p, float (&v)[N]) {
  if constexpr (N == 8) {
    const uint4 w = *reinterpret_cast<const uint4*>(p);
    v[0] = dm_bf2f_lo(w.x); v[1] = dm_bf2f_hi(w.x); v[2] = dm_bf2f_lo(w.y); v[3] = dm_bf2f_hi(w.y);
    v[4] = dm_bf2f_lo(w.z); v[5] = dm_bf2f_hi(w.z); v[6] = dm_bf2f_lo(w.w); v[7] = dm_bf2f_hi(w.w);
  } else {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    v[0] = dm_bf2f_lo(w.x); v[1] = dm_bf2f_hi(w.x); v[2] = dm_bf2f_lo(w.y); v[3] = dm_bf2f_hi(w.y);
  }
}
template <int N>
__device__ __forceinline__ void act_load(const float* p, float (&v)[N]) {
#pragma unroll
  for (int c = 0; c < N / 4; ++c) {
    const float4 w = reinterpret_cast<const float4*>(p)[c];
    v[4 * c] = w.x; v[4 * c + 1] = w.y; v[4 * c + 2] = w.z; v[4 * c + 3] = w.w;
  }
}
__device__ __forceinline__ void act_store4(bf16_t* p, const float (&v)[4]) {
  *reinterpret_cast<uint2*>(p) = make_uint2(dm_f2bf2(v[0], v[1]), dm_f2bf2(v[2], v[3]));
}
__device__ __forceinline__ void act_store4(float* p, const float (&v)[4]) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}

// tanh: the odd power series up to x^9 below 1/4 (its remainder there is below 1e-8 of the value),
// 1 - 2 / (e^2x + 1) above
__device__ __forceinline__ float dm_tanh(float x) {
  const float a = __builtin_fabsf(x);
  const float x2 = x * x;
  float s = 62.0f / 2835.0f;
  s = dm_fma(s, x2, -17.0f / 315.0f);
  s = dm_fma(s, x2, 2.0f / 15.0f);
  s = dm_fma(s, x2, -1.0f / 3.0f);
  s = dm_fma(s * x2, x, x);
  const float t = 1.0f - 2.0f / (dm_exp(2.0f * a) + 1.0f);
  return a < 0.25f ? s : (x < 0.0f ? -t : t);
}

// gelu by its tanh approximation
__device__ __forceinline__ float dm_gelu_tanh(float z) {
  const float u = 0.7978845608028654f * dm_fma(0.044715f * z * z, z, z);
  return 0.5f * z * (1.0f + dm_tanh(u));
}

// log(sigmoid(x))
__device__ __forceinline__ float dm_log_sigmoid(float x) {
  return __builtin_fminf(x, 0.0f) - dm_log1p(dm_exp(-__builtin_fabsf(x)));
}

// 2^x as the hardware gives it: for the matrix-core kernels, which agree with the exact ones to
// rounding
__device__ __forceinline__ float dm_exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

// sum and maximum over lanes l, l ^ 16, l ^ 32, l ^ 48
__device__ __forceinline__ float dm_sum_groups16(float v) {
  float a, b;
  dm_row_swap<32>(v, a, b);
  v = a + b;
  dm_row_swap<16>(v, a, b);
  return a + b;
}
__device__ __forceinline__ float dm_max_groups16(float v) {
  float a, b;
  dm_row_swap<32>(v, a, b);
  v = b > a ? b : a;
  dm_row_swap<16>(v, a, b);
  return b > a ? b : a;
}
