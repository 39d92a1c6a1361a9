// The fp32 residual stream of looped layers and the norms around it.
//
//   v = x + mult * (ls * y);  tap <- v;  v += embed[id];  v += step
//   x_out <- v;  h = v / sqrt(mean(v^2) + eps) * w
//
// One workgroup per token; the row stays in registers between sum and norm.
#include "../glu.h"

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

struct Stream {
  const float* x;              // null: the row starts from zero
  const float* ls;
  const int64_t* ids;          // null: no embedding is added
  const float* step;           // null: no step vector
  const float* w;
  float* x_out;
  float* tap;
  int64_t y_stride;
  float mult, eps;
  int W, vocab;
};

// N consecutive elements at d of row t.
template <typename S, int N>
__device__ __forceinline__ void stream_row(float (&a)[N], const Stream& s,
                                           const S* y, const S* embed,
                                           int64_t t, int64_t id, int d) {
  const int64_t at = t * s.W + d;
#pragma unroll
  for (int i = 0; i < N; ++i) a[i] = 0.f;
  float b[N];
  if (s.x != nullptr) {
    float c[N];
    if constexpr (N == 1) {
      a[0] = s.x[at];
      b[0] = ld1(y + t * s.y_stride + d);
      c[0] = s.ls[d];
    } else {
      ldv<N>(s.x + at, a);
      ldv<N>(y + t * s.y_stride + d, b);
      ldv<N>(s.ls + d, c);
    }
#pragma unroll
    for (int i = 0; i < N; ++i) a[i] += s.mult * (c[i] * b[i]);
  }
  if (s.tap != nullptr) {
    if constexpr (N == 1) s.tap[at] = a[0]; else stv<N>(s.tap + at, a);
  }
  if (s.ids != nullptr) {
    if constexpr (N == 1) b[0] = ld1(embed + id * s.W + d);
    else ldv<N>(embed + id * s.W + d, b);
#pragma unroll
    for (int i = 0; i < N; ++i) a[i] += b[i];
  }
  if (s.step != nullptr) {
    if constexpr (N == 1) b[0] = s.step[d]; else ldv<N>(s.step + d, b);
#pragma unroll
    for (int i = 0; i < N; ++i) a[i] += b[i];
  }
  if (s.x_out != nullptr) {
    if constexpr (N == 1) s.x_out[at] = a[0]; else stv<N>(s.x_out + at, a);
  }
}

__device__ __forceinline__ int64_t token_id(const Stream& s, int64_t t) {
  if (s.ids == nullptr) return 0;
  const int64_t id = s.ids[t];
  return id < 0 ? 0 : (id >= s.vocab ? s.vocab - 1 : id);
}

// NV vectors of 4 per thread; 4 * NV * blockDim.x >= W, W % 4 == 0.
template <typename S, int NV>
__global__ void residual_norm_kernel(S* __restrict__ h, const S* y,
                                     const S* embed, Stream s) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x, id = token_id(s, t);
  float a[NV][4];
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * blockDim.x + threadIdx.x) * 4;
    if (d < s.W) {
      stream_row<S, 4>(a[v], s, y, embed, t, id, d);
#pragma unroll
      for (int i = 0; i < 4; ++i) ss += a[v][i] * a[v][i];
    }
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / s.W + s.eps);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * blockDim.x + threadIdx.x) * 4;
    if (d < s.W) {
      float w[4];
      ldv<4>(s.w + d, w);
#pragma unroll
      for (int i = 0; i < 4; ++i) a[v][i] *= inv * w[i];
      stv<4>(h + t * s.W + d, a[v]);
    }
  }
}

// Any width: the row waits in LDS.
template <typename S>
__global__ void residual_norm_any_kernel(S* __restrict__ h, const S* y,
                                         const S* embed, Stream s) {
  extern __shared__ float row[];
  __shared__ float red[16];
  const int64_t t = blockIdx.x, id = token_id(s, t);
  float ss = 0.f;
  for (int d = threadIdx.x; d < s.W; d += blockDim.x) {
    float a[1];
    stream_row<S, 1>(a, s, y, embed, t, id, d);
    row[d] = a[0];
    ss += a[0] * a[0];
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / s.W + s.eps);
  for (int d = threadIdx.x; d < s.W; d += blockDim.x)
    st1(h + t * s.W + d, row[d] * inv * s.w[d]);
}

template <typename S>
void launch_residual(torch::Tensor h, OptT y, OptT embed, Stream s, int T) {
  auto stream = at::hip::getCurrentHIPStream();
  S* hp = (S*)h.data_ptr();
  const S* yp = y.has_value() ? (const S*)y->data_ptr() : nullptr;
  const S* ep = embed.has_value() ? (const S*)embed->data_ptr() : nullptr;
  // few rows: spread each over more waves; many: several rows to a CU
  const int want = T <= 512 ? 1024 : 256, vecs = cdiv(s.W, 4);
  const bool vec = s.W % 4 == 0 && s.y_stride % 4 == 0;
#define HELIX_RES(NV, THREADS)                                               \
  hipLaunchKernelGGL((residual_norm_kernel<S, NV>), dim3(T), dim3(THREADS),  \
                     0, stream, hp, yp, ep, s)
  if (vec && vecs <= want)
    HELIX_RES(1, std::min(want, cdiv(vecs, WAVE) * WAVE));
  else if (vec && vecs <= 2 * want) HELIX_RES(2, want);
  else if (vec && vecs <= 4 * want) HELIX_RES(4, want);
  else if (vec && vecs <= 8 * want) HELIX_RES(8, want);
  else {
    TORCH_CHECK(s.W <= 15000, "width ", s.W, " needs W % 4 == 0");
    hipLaunchKernelGGL((residual_norm_any_kernel<S>), dim3(T), dim3(256),
                       s.W * sizeof(float), stream, hp, yp, ep, s);
  }
#undef HELIX_RES
}

// ------------------------------------------------------------- grouped norm

// One workgroup per (row, group); NV vectors of 8 per thread.
template <typename S, int NV>
__global__ void group_norm_kernel(S* __restrict__ out,
                                  const S* __restrict__ y,
                                  const float* __restrict__ w, float eps,
                                  int groups, int size) {
  __shared__ float red[16];
  const int64_t at = (int64_t)blockIdx.x * size;
  const float* wg = w + (int64_t)(blockIdx.x % groups) * size;
  float a[NV][8];
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * blockDim.x + threadIdx.x) * 8;
    if (d < size) {
      ldv<8>(y + at + d, a[v]);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += a[v][i] * a[v][i];
    }
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / size + eps);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * blockDim.x + threadIdx.x) * 8;
    if (d < size) {
      float ww[8];
      ldv<8>(wg + d, ww);
#pragma unroll
      for (int i = 0; i < 8; ++i) a[v][i] *= inv * ww[i];
      stv<8>(out + at + d, a[v]);
    }
  }
}

template <typename S>
__global__ void group_norm_any_kernel(S* __restrict__ out,
                                      const S* __restrict__ y,
                                      const float* __restrict__ w, float eps,
                                      int groups, int size) {
  __shared__ float red[16];
  const int64_t at = (int64_t)blockIdx.x * size;
  const float* wg = w + (int64_t)(blockIdx.x % groups) * size;
  float ss = 0.f;
  for (int d = threadIdx.x; d < size; d += blockDim.x) {
    const float v = ld1(y + at + d);
    ss += v * v;
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / size + eps);
  for (int d = threadIdx.x; d < size; d += blockDim.x)
    st1(out + at + d, ld1(y + at + d) * inv * wg[d]);
}

template <typename S>
void launch_group_norm(torch::Tensor out, torch::Tensor y, int groups,
                       torch::Tensor w, float eps) {
  const int size = y.size(1) / groups;
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(y.size(0) * groups);
#define HELIX_GN(K, THREADS)                                                 \
  hipLaunchKernelGGL((K), grid, dim3(THREADS), 0, stream,                    \
                     (S*)out.data_ptr(), (const S*)y.data_ptr(),             \
                     w.data_ptr<float>(), eps, groups, size)
  if (size % 8 == 0 && size <= 2048)
    HELIX_GN((group_norm_kernel<S, 1>), cdiv(cdiv(size, 8), WAVE) * WAVE);
  else if (size % 8 == 0 && size <= 16384)
    HELIX_GN((group_norm_kernel<S, 4>), 512);
  else
    HELIX_GN((group_norm_any_kernel<S>), 256);
#undef HELIX_GN
}

void check_f32(const OptT& t, int64_t n, const char* what) {
  if (!t.has_value()) return;
  TORCH_CHECK(t->is_cuda() && t->scalar_type() == torch::kFloat32 &&
                  t->is_contiguous() && t->numel() == n,
              what);
}

bool supported(const torch::Tensor& t) {
  return t.scalar_type() == torch::kBFloat16 ||
         t.scalar_type() == torch::kFloat32;
}

}  // namespace

void residual_norm(torch::Tensor h, OptT x, OptT y, OptT ls, double mult,
                   OptT ids, OptT embed, OptT step, torch::Tensor w,
                   double eps, OptT x_out, OptT tap) {
  TORCH_CHECK(h.dim() == 2 && h.is_contiguous() && supported(h));
  const int64_t T = h.size(0), W = h.size(1);
  TORCH_CHECK(x.has_value() || ids.has_value(), "nothing to norm");
  check_f32(x, T * W, "x");
  check_f32(x_out, T * W, "x_out");
  check_f32(tap, T * W, "tap");
  check_f32(step, W, "step");
  check_f32(w, W, "w");
  Stream s{};
  s.y_stride = 4;
  if (x.has_value()) {
    TORCH_CHECK(y.has_value() && ls.has_value());
    check_f32(ls, W, "ls");
    TORCH_CHECK(y->scalar_type() == h.scalar_type() && y->size(0) == T &&
                y->size(1) == W && y->stride(1) == 1);
    s.x = x->data_ptr<float>();
    s.ls = ls->data_ptr<float>();
    s.y_stride = y->stride(0);
  } else {
    y = c10::nullopt;
  }
  if (ids.has_value()) {
    TORCH_CHECK(embed.has_value() && embed->is_contiguous() &&
                embed->scalar_type() == h.scalar_type() &&
                embed->size(1) == W && embed->size(0) > 0);
    TORCH_CHECK(ids->scalar_type() == torch::kInt64 && ids->numel() == T &&
                ids->is_contiguous());
    s.ids = ids->data_ptr<int64_t>();
    s.vocab = embed->size(0);
  }
  if (step.has_value()) s.step = step->data_ptr<float>();
  if (x_out.has_value()) s.x_out = x_out->data_ptr<float>();
  if (tap.has_value()) s.tap = tap->data_ptr<float>();
  s.w = w.data_ptr<float>();
  s.mult = (float)mult;
  s.eps = (float)eps;
  s.W = W;
  if (T == 0) return;
  if (h.scalar_type() == torch::kBFloat16)
    launch_residual<uint16_t>(h, y, embed, s, T);
  else
    launch_residual<float>(h, y, embed, s, T);
}

void silu_mul(torch::Tensor out, torch::Tensor z, int64_t up_at) {
  launch_glu<Silu>(out, z, up_at);
}

void group_rms_norm(torch::Tensor out, torch::Tensor y, int64_t groups,
                    torch::Tensor w, double eps) {
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && out.is_contiguous() &&
              supported(y));
  TORCH_CHECK(out.scalar_type() == y.scalar_type() &&
              out.numel() == y.numel());
  TORCH_CHECK(groups > 0 && y.size(1) % groups == 0);
  check_f32(w, y.size(1), "w");
  if (y.numel() == 0) return;
  if (y.scalar_type() == torch::kBFloat16)
    launch_group_norm<uint16_t>(out, y, groups, w, (float)eps);
  else
    launch_group_norm<float>(out, y, groups, w, (float)eps);
}
