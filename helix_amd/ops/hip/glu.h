// act(gate) * up over fused projections, for every gated feed-forward.
#pragma once
#include "hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

namespace helix {

struct Silu {
  template <typename S>
  static __device__ __forceinline__ float run(float x) { return silu_s<S>(x); }
};

// x * (1 + tanh(u)) / 2 = x * sigmoid(2 u), u = sqrt(2/pi)(x + 0.044715 x^3)
struct GeluTanh {
  template <typename S>
  static __device__ __forceinline__ float run(float x) {
    const float u = 0.7978845608028654f * (x + 0.044715f * x * x * x);
    return x / (1.f + exp_s<S>(-2.f * u));
  }
};

template <typename S, class Act, int N>
__global__ void glu_kernel(S* __restrict__ out, const S* __restrict__ z,
                           int64_t z_stride, int up_at, int F,
                           int64_t total) {
  const int64_t i = ((int64_t)blockIdx.x * blockDim.x + threadIdx.x);
  if (i >= total) return;
  const int nv = F / N;
  const int64_t t = i / nv;
  const int d = (int)(i - t * nv) * N;
  const S* zr = z + t * z_stride;
  if constexpr (N == 1) {
    st1(out + t * F + d,
        Act::template run<S>(ld1(zr + d)) * ld1(zr + up_at + d));
  } else {
    float g[N], u[N];
    ldv<N>(zr + d, g);
    ldv<N>(zr + up_at + d, u);
#pragma unroll
    for (int j = 0; j < N; ++j) g[j] = Act::template run<S>(g[j]) * u[j];
    stv<N>(out + t * F + d, g);
  }
}

template <typename S, class Act>
void launch_glu_as(torch::Tensor out, torch::Tensor z, int up_at) {
  const int64_t T = out.size(0);
  const int F = out.size(1);
  auto stream = at::hip::getCurrentHIPStream();
  const bool vec = F % 8 == 0 && up_at % 8 == 0 && z.stride(0) % 8 == 0;
  const int64_t total = T * F / (vec ? 8 : 1);
  const dim3 grid((total + 255) / 256);
  if (vec)
    hipLaunchKernelGGL((glu_kernel<S, Act, 8>), grid, dim3(256), 0, stream,
                       (S*)out.data_ptr(), (const S*)z.data_ptr(),
                       z.stride(0), up_at, F, total);
  else
    hipLaunchKernelGGL((glu_kernel<S, Act, 1>), grid, dim3(256), 0, stream,
                       (S*)out.data_ptr(), (const S*)z.data_ptr(),
                       z.stride(0), up_at, F, total);
}

// out [T, F] <- Act(z[:, :F]) * z[:, up_at : up_at + F]
template <class Act>
void launch_glu(torch::Tensor out, torch::Tensor z, int64_t up_at) {
  TORCH_CHECK(out.dim() == 2 && out.is_contiguous() && z.stride(1) == 1);
  TORCH_CHECK(z.scalar_type() == out.scalar_type() &&
              z.size(0) == out.size(0));
  TORCH_CHECK(out.size(1) <= up_at && up_at + out.size(1) <= z.size(1));
  if (out.numel() == 0) return;
  if (z.scalar_type() == torch::kBFloat16)
    launch_glu_as<uint16_t, Act>(out, z, up_at);
  else if (z.scalar_type() == torch::kFloat32)
    launch_glu_as<float, Act>(out, z, up_at);
  else
    TORCH_CHECK(false, "gated activation: bf16 or fp32");
}

}  // namespace helix
