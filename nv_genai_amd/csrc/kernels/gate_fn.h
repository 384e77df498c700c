// Helpers of the recurrences: scalar loads of either activation type, gate functions, the fp32 MFMA.
#pragma once
#include "common.h"

namespace nga {

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<uint16_t>(const uint16_t* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }

// fp32 activations take the library functions, bf16 ones the hardware exp2 / log2 / reciprocal
template <typename T> struct GateFn;
template <> struct GateFn<float> {
  static __device__ __forceinline__ float exp(float x) { return expf(x); }
  static __device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
  static __device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
};
template <> struct GateFn<uint16_t> {
  static __device__ __forceinline__ float exp(float x) { return __builtin_amdgcn_exp2f(1.4426950408889634f * x); }
  static __device__ __forceinline__ float sigmoid(float z) {
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
  }
  static __device__ __forceinline__ float softplus(float z) {
    const float e = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z));
    // ln(1 + e) for e in (0, 1]; below 2^-12 the series (1 + e would drop e's low bits)
    const float l = e < 2.44140625e-4f ? e - 0.5f * e * e : 0.6931471805599453f * __builtin_amdgcn_logf(1.0f + e);
    return fmaxf(z, 0.f) + l;
  }
};

__device__ __forceinline__ f32x4 mfma32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

}  // namespace

}  // namespace nga
