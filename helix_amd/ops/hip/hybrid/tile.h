// Small pieces shared by the kernels of hybrid models.
#pragma once
#include "../elem.h"

namespace helix {

__device__ __forceinline__ u16x8 ld_u16x8(const uint16_t* p) {
  return *reinterpret_cast<const u16x8*>(p);
}

// D[16 x 16] += A[16 x 32] B[32 x 16]. Lane (hi = lane / 16, lo = lane % 16)
// holds A[lo][8 hi + i], B[8 hi + i][lo] and D[4 hi + r][lo].
__device__ __forceinline__ floatx4 mfma16(u16x8 a, u16x8 b, floatx4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(
      __builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0,
      0);
}

// Where row r of a tile is stored in LDS when its products should leave 8
// neighbouring rows to a lane: rows 8 a + 4 s + b of a group of 32 go to
// 16 s + 4 a + b, so an A operand of half s is 16 rows in a row (no bank
// conflicts) and lane hi ends up with rows 8 hi + 4 s + r of its result.
__device__ __forceinline__ int paired_row(int r) {
  return (r & ~31) | (r & 4) << 2 | (r & 24) >> 1 | (r & 3);
}

__device__ __forceinline__ u16x8 pack8(const float* v) {
  u32x4 u;
#pragma unroll
  for (int i = 0; i < 4; ++i) u[i] = pack_bf16(v[2 * i], v[2 * i + 1]);
  return __builtin_bit_cast(u16x8, u);
}

// v = hi + lo with two bf16 terms (about 17 significant bits).
__device__ __forceinline__ void split8(const float* v, u16x8& hi, u16x8& lo) {
  hi = pack8(v);
  float rest[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) rest[i] = v[i] - bf16_to_f32(hi[i]);
  lo = pack8(rest);
}

__device__ __forceinline__ void st_bf16x4(uint16_t* p, const float* v) {
  *reinterpret_cast<u32x2*>(p) =
      u32x2{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])};
}

template <typename S>
__device__ __forceinline__ float sigmoid_s(float x) {
  return 1.f / (1.f + exp_s<S>(-x));
}
template <typename S>
__device__ __forceinline__ float silu_s(float x) {
  return x / (1.f + exp_s<S>(-x));
}

// log(1 + e^x)
__device__ __forceinline__ float softplus(float x) {
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}

// Sum over a workgroup of up to 16 waves; red: 16 floats. Callers that use
// red again put a barrier between.
__device__ __forceinline__ float group_sum(float v, float* red) {
  v = wave_reduce_sum(v);
  const int wid = threadIdx.x / WAVE, nw = blockDim.x / WAVE;
  if ((threadIdx.x & (WAVE - 1)) == 0) red[wid] = v;
  __syncthreads();
  float s = 0.f;
  for (int i = 0; i < nw; ++i) s += red[i];
  return s;
}

}  // namespace helix
