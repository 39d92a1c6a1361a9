// Element access shared by the kernels that come in a bf16 and an fp32
// build: storage type S is uint16_t (bf16 bits) or float, math is fp32.
#pragma once
#include "common.h"

namespace helix {

template <typename S>
__device__ __forceinline__ float ld1(const S* p);
template <>
__device__ __forceinline__ float ld1<uint16_t>(const uint16_t* p) {
  return bf16_to_f32(*p);
}
template <>
__device__ __forceinline__ float ld1<float>(const float* p) { return *p; }

template <typename S>
__device__ __forceinline__ void st1(S* p, float v);
template <>
__device__ __forceinline__ void st1<uint16_t>(uint16_t* p, float v) {
  *p = f32_to_bf16(v);
}
template <>
__device__ __forceinline__ void st1<float>(float* p, float v) { *p = v; }

// N consecutive elements (N = 4 or 8); p is aligned to N elements.
template <int N>
__device__ __forceinline__ void ldv(const uint16_t* p, float* out) {
  typedef __attribute__((ext_vector_type(N))) uint16_t V;
  const V v = *reinterpret_cast<const V*>(p);
#pragma unroll
  for (int i = 0; i < N; ++i) out[i] = bf16_to_f32(v[i]);
}
template <int N>
__device__ __forceinline__ void ldv(const float* p, float* out) {
#pragma unroll
  for (int j = 0; j < N; j += 4) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p + j);
#pragma unroll
    for (int i = 0; i < 4; ++i) out[j + i] = v[i];
  }
}
template <int N>
__device__ __forceinline__ void stv(uint16_t* p, const float* in) {
  typedef __attribute__((ext_vector_type(N))) uint16_t V;
  V v;
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = f32_to_bf16(in[i]);
  *reinterpret_cast<V*>(p) = v;
}
template <int N>
__device__ __forceinline__ void stv(float* p, const float* in) {
#pragma unroll
  for (int j = 0; j < N; j += 4) {
    f32x4 v;
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = in[j + i];
    *reinterpret_cast<f32x4*>(p + j) = v;
  }
}

// Two floats -> two bf16 (round to nearest even), a in the low half; one
// v_cvt_pk_bf16_f32 on gfx950.
__device__ __forceinline__ uint32_t pack_bf16(float a, float b) {
  typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
  const bf16x2 v = __builtin_convertvector(f32x2{a, b}, bf16x2);
  return __builtin_bit_cast(uint32_t, v);
}

// exp / tanh per storage type: the fp32 build takes the library functions,
// the bf16 build the native exponential (absolute error of the capped
// score below 1e-5 for caps up to a few hundred).
template <typename S>
__device__ __forceinline__ float exp_s(float x) { return __expf(x); }
template <>
__device__ __forceinline__ float exp_s<float>(float x) { return expf(x); }

template <typename S>
__device__ __forceinline__ float tanh_s(float x) {
  return 1.f - 2.f * __builtin_amdgcn_rcpf(1.f + __expf(2.f * x));
}
template <>
__device__ __forceinline__ float tanh_s<float>(float x) { return tanhf(x); }

// Attention score from a raw dot product: scale, optional soft cap
// (cap > 0), then the per-head distance bias.
template <typename S>
__device__ __forceinline__ float cap_and_bias(float dot, float scale,
                                              float cap, float inv_cap,
                                              float slope, int dist) {
  float s = dot * scale;
  if (cap > 0.f) s = cap * tanh_s<S>(s * inv_cap);
  return s - slope * (float)dist;
}

}  // namespace helix
