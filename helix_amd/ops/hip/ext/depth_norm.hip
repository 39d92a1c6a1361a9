// fp32 residual stream with depth averaging, fused with the RMS norm that
// feeds the next layer.
//
//   X_new  = x + y                        (layer result)
//   x'     = sum_{j<n} c[j] X_j + c[n] X_new
//   h      = x' / sqrt(mean(x'^2) + eps) * w
//
// One workgroup per token. Everything is read once: the averaged row stays
// in registers between the sum and the norm. The history is [depth, T, W]
// fp32, so each X_j row is one contiguous streak.
#include "../elem.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int VEC = 4;

__device__ __forceinline__ float row_sum(float v, float* red) {
  v = wave_reduce_sum(v);
  const int wid = threadIdx.x / WAVE, nw = blockDim.x / WAVE;
  if ((threadIdx.x & (WAVE - 1)) == 0) red[wid] = v;
  __syncthreads();
  float s = 0.f;
  for (int i = 0; i < nw; ++i) s += red[i];
  return s;
}

// NV = 4-float vectors per thread; 4 * NV * blockDim.x >= W, W % 4 == 0.
template <typename S, int NV>
__global__ void depth_norm_kernel(
    S* __restrict__ h, float* x_out, const float* x, const S* __restrict__ y,
    int64_t y_stride, float* __restrict__ hist, int64_t hist_stride,
    int n_prev, int store_new, const float* __restrict__ coef,
    const float* __restrict__ w, float eps, int W) {
  __shared__ float red[16];
  const int64_t row = (int64_t)blockIdx.x * W;
  const S* yrow = y + (int64_t)blockIdx.x * y_stride;
  float a[NV][VEC];
  float ss = 0.f;
  const float c_new = coef[n_prev];
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * blockDim.x + threadIdx.x) * VEC;
    if (d < W) {
      float b[VEC];
      ldv<VEC>(x + row + d, a[v]);
      ldv<VEC>(yrow + d, b);
#pragma unroll
      for (int i = 0; i < VEC; ++i) a[v][i] += b[i];
      if (store_new) stv<VEC>(hist + n_prev * hist_stride + row + d, a[v]);
#pragma unroll
      for (int i = 0; i < VEC; ++i) a[v][i] *= c_new;
    }
  }
#pragma unroll 4
  for (int j = 0; j < n_prev; ++j) {
    const float c = coef[j];
    const float* hj = hist + j * hist_stride + row;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int d = (v * blockDim.x + threadIdx.x) * VEC;
      if (d < W) {
        float b[VEC];
        ldv<VEC>(hj + d, b);
#pragma unroll
        for (int i = 0; i < VEC; ++i) a[v][i] += c * b[i];
      }
    }
  }
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * blockDim.x + threadIdx.x) * VEC;
    if (d < W) {
      if (x_out != nullptr) stv<VEC>(x_out + row + d, a[v]);
#pragma unroll
      for (int i = 0; i < VEC; ++i) ss += a[v][i] * a[v][i];
    }
  }
  const float inv = 1.f / sqrtf(row_sum(ss, red) / W + eps);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * blockDim.x + threadIdx.x) * VEC;
    if (d < W) {
      float ww[VEC];
      ldv<VEC>(w + d, ww);
#pragma unroll
      for (int i = 0; i < VEC; ++i) a[v][i] = a[v][i] * inv * ww[i];
      stv<VEC>(h + row + d, a[v]);
    }
  }
}

// Any W: scalar accesses, the averaged row is kept in x_row (dynamic LDS).
template <typename S>
__global__ void depth_norm_any_kernel(
    S* __restrict__ h, float* x_out, const float* x, const S* __restrict__ y,
    int64_t y_stride, float* __restrict__ hist, int64_t hist_stride,
    int n_prev, int store_new, const float* __restrict__ coef,
    const float* __restrict__ w, float eps, int W) {
  extern __shared__ float x_row[];
  __shared__ float red[16];
  const int64_t row = (int64_t)blockIdx.x * W;
  float ss = 0.f;
  for (int d = threadIdx.x; d < W; d += blockDim.x) {
    const float fresh = x[row + d] + ld1(y + blockIdx.x * y_stride + d);
    if (store_new) hist[n_prev * hist_stride + row + d] = fresh;
    float a = coef[n_prev] * fresh;
    for (int j = 0; j < n_prev; ++j)
      a += coef[j] * hist[j * hist_stride + row + d];
    if (x_out != nullptr) x_out[row + d] = a;
    x_row[d] = a;
    ss += a * a;
  }
  const float inv = 1.f / sqrtf(row_sum(ss, red) / W + eps);
  for (int d = threadIdx.x; d < W; d += blockDim.x)
    st1(h + row + d, x_row[d] * inv * w[d]);
}

// hist[0][t] = embed[ids[t]] in fp32 and its norm.
template <typename S>
__global__ void embed_norm_kernel(S* __restrict__ h, float* __restrict__ x,
                                  const int64_t* __restrict__ ids,
                                  const S* __restrict__ embed,
                                  const float* __restrict__ w, float eps,
                                  int W, int vocab) {
  __shared__ float red[16];
  const int64_t row = (int64_t)blockIdx.x * W;
  int64_t id = ids[blockIdx.x];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const S* e = embed + id * W;
  float ss = 0.f;
  for (int d = threadIdx.x; d < W; d += blockDim.x) {
    const float a = ld1(e + d);
    x[row + d] = a;
    ss += a * a;
  }
  const float inv = 1.f / sqrtf(row_sum(ss, red) / W + eps);
  for (int d = threadIdx.x; d < W; d += blockDim.x)
    st1(h + row + d, ld1(e + d) * inv * w[d]);
}

template <typename S>
void launch_depth(torch::Tensor h, c10::optional<torch::Tensor> x_out,
                  torch::Tensor x, torch::Tensor y, torch::Tensor hist,
                  int n_prev, bool store_new, torch::Tensor coef,
                  torch::Tensor w, float eps) {
  const int T = x.size(0), W = x.size(1);
  auto stream = at::hip::getCurrentHIPStream();
  S* hp = (S*)h.data_ptr();
  float* xo = x_out.has_value() ? x_out->data_ptr<float>() : nullptr;
  const float* xp = x.data_ptr<float>();
  const S* yp = (const S*)y.data_ptr();
  float* hist_p = hist.data_ptr<float>();
  const int64_t hs = hist.stride(0);
  const float* cp = coef.data_ptr<float>();
  const float* wp = w.data_ptr<float>();
#define HELIX_DEPTH(NV, THREADS)                                             \
  hipLaunchKernelGGL((depth_norm_kernel<S, NV>), dim3(T), dim3(THREADS), 0,  \
                     stream, hp, xo, xp, yp, y.stride(0), hist_p, hs,        \
                     n_prev, (int)store_new, cp, wp, eps, W)
  const bool vec_ok = W % VEC == 0 && y.stride(0) % VEC == 0;
  // few rows: spread each over more waves (latency), many: keep the
  // workgroup small so several share a CU
  const int want = T <= 512 ? 1024 : 256;
  if (vec_ok && W <= want * VEC) {
    const int threads = cdiv(cdiv(W, VEC), WAVE) * WAVE;
    HELIX_DEPTH(1, std::min(threads, want));
  } else if (vec_ok && W <= want * VEC * 2) {
    HELIX_DEPTH(2, want);
  } else if (vec_ok && W <= want * VEC * 4) {
    HELIX_DEPTH(4, want);
  } else if (vec_ok && W <= want * VEC * 8) {
    HELIX_DEPTH(8, want);
  } else {
    TORCH_CHECK(W <= 15000, "width ", W, " needs W % 4 == 0");
    hipLaunchKernelGGL((depth_norm_any_kernel<S>), dim3(T), dim3(256),
                       W * sizeof(float), stream, hp, xo, xp, yp,
                       y.stride(0), hist_p, hs, n_prev, (int)store_new, cp,
                       wp, eps, W);
  }
#undef HELIX_DEPTH
}

}  // namespace

// hist: [depth, T, W] fp32 holding X_0 .. X_{n_prev-1}; X_{n_prev} is
// appended when store_new. x and x_out may be the same tensor.
void depth_norm(torch::Tensor h, c10::optional<torch::Tensor> x_out,
                torch::Tensor x, torch::Tensor y, torch::Tensor hist,
                int64_t n_prev, bool store_new, torch::Tensor coef,
                torch::Tensor w, double eps) {
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(x.is_contiguous() && h.is_contiguous() && hist.is_contiguous());
  TORCH_CHECK(x.scalar_type() == torch::kFloat32 &&
              hist.scalar_type() == torch::kFloat32 &&
              coef.scalar_type() == torch::kFloat32 &&
              w.scalar_type() == torch::kFloat32);
  TORCH_CHECK(h.scalar_type() == y.scalar_type());
  TORCH_CHECK(h.numel() == T * W && w.numel() == W);
  TORCH_CHECK(y.size(0) == T && y.size(1) == W && y.stride(1) == 1);
  TORCH_CHECK(hist.size(1) == T && hist.size(2) == W);
  TORCH_CHECK(n_prev + (store_new ? 1 : 0) <= hist.size(0));
  TORCH_CHECK(coef.numel() == n_prev + 1, "depth coefficients");
  if (x_out.has_value())
    TORCH_CHECK(x_out->is_contiguous() && x_out->numel() == T * W &&
                x_out->scalar_type() == torch::kFloat32);
  if (T == 0) return;
  if (h.scalar_type() == torch::kBFloat16)
    launch_depth<uint16_t>(h, x_out, x, y, hist, n_prev, store_new, coef, w,
                           (float)eps);
  else if (h.scalar_type() == torch::kFloat32)
    launch_depth<float>(h, x_out, x, y, hist, n_prev, store_new, coef, w,
                        (float)eps);
  else
    TORCH_CHECK(false, "depth_norm: bf16 or fp32");
}

void embed_norm(torch::Tensor h, torch::Tensor x, torch::Tensor ids,
                torch::Tensor embed, torch::Tensor w, double eps) {
  const int64_t T = ids.size(0), W = embed.size(1);
  TORCH_CHECK(h.is_contiguous() && x.is_contiguous() &&
              embed.is_contiguous() && ids.is_contiguous());
  TORCH_CHECK(h.numel() == T * W && x.numel() == T * W && w.numel() == W);
  TORCH_CHECK(ids.scalar_type() == torch::kInt64);
  TORCH_CHECK(x.scalar_type() == torch::kFloat32 &&
              w.scalar_type() == torch::kFloat32);
  TORCH_CHECK(h.scalar_type() == embed.scalar_type());
  if (T == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
#define HELIX_EMBED(S)                                                       \
  hipLaunchKernelGGL((embed_norm_kernel<S>), dim3(T), dim3(256), 0, stream,  \
                     (S*)h.data_ptr(), x.data_ptr<float>(),                  \
                     ids.data_ptr<int64_t>(), (const S*)embed.data_ptr(),    \
                     w.data_ptr<float>(), (float)eps, (int)W,                \
                     (int)embed.size(0))
  if (h.scalar_type() == torch::kBFloat16) HELIX_EMBED(uint16_t);
  else if (h.scalar_type() == torch::kFloat32) HELIX_EMBED(float);
  else TORCH_CHECK(false, "embed_norm: bf16 or fp32");
#undef HELIX_EMBED
}
