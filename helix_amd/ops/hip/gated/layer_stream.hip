// The fp32 residual stream of layers that norm before and after a sublayer
// (layer norm), and of loops that mix the embedding in by a projection.
//
// A row v comes from one of
//   ADD    x + norm(y)                      a sublayer's result
//   EMBED  scale * embed[id]
//   ENTER  a (+ b) + e_scale * e + step     a pass of the loop begins
// goes to x_out (and tap), and leaves as its layer norm in the storage type
// or as two bf16 terms v = hi + lo, the operands of the loop's projection.
//
// One workgroup per token; the row stays in registers through both norms,
// whose variance is taken from the deviations.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

enum Source { ADD, EMBED, ENTER };

struct Stream {
  const float* x;
  const float *wy, *by;        // ADD: norm of y
  const int64_t* ids;          // EMBED
  const float *a, *b, *e, *step;  // ENTER; b and step may be null
  const float *w, *bias;       // norm of the result; null: no norm
  float *x_out, *tap;
  void *hi, *lo;               // two terms; null: none
  int64_t y_stride;
  float scale, eps;
  int W, vocab;
};

template <int N>
__device__ __forceinline__ void ldf(const float* p, float* v) {
  if constexpr (N == 1) v[0] = *p; else ldv<N>(p, v);
}
template <int N>
__device__ __forceinline__ void lds_(const uint16_t* p, float* v) {
  if constexpr (N == 1) v[0] = ld1(p); else ldv<N>(p, v);
}
template <int N>
__device__ __forceinline__ void lds_(const float* p, float* v) {
  ldf<N>(p, v);
}
template <int N, typename S>
__device__ __forceinline__ void sts(S* p, const float* v) {
  if constexpr (N == 1) st1(p, v[0]); else stv<N>(p, v);
}

// v <- (v - mean) / sqrt(variance + eps) * w + bias over the workgroup's row
template <int NV, int N>
__device__ __forceinline__ void norm_row(float (&v)[NV][N], const float* w,
                                         const float* bias, int W, float eps,
                                         float* red) {
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if ((i * blockDim.x + threadIdx.x) * N < W)
#pragma unroll
      for (int j = 0; j < N; ++j) s += v[i][j];
  const float mean = group_sum(s, red) / W;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if ((i * blockDim.x + threadIdx.x) * N < W)
#pragma unroll
      for (int j = 0; j < N; ++j) {
        v[i][j] -= mean;
        ss += v[i][j] * v[i][j];
      }
  const float inv = 1.f / sqrtf(group_sum(ss, red + 16) / W + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int d = (i * blockDim.x + threadIdx.x) * N;
    if (d < W) {
      float g[N], c[N];
      ldf<N>(w + d, g);
      ldf<N>(bias + d, c);
#pragma unroll
      for (int j = 0; j < N; ++j) v[i][j] = v[i][j] * inv * g[j] + c[j];
    }
  }
}

// NV vectors of N values per thread; N * NV * blockDim.x >= W, W % N == 0.
template <typename S, int SRC, int NV, int N>
__global__ void layer_stream_kernel(S* __restrict__ h, const S* y,
                                    const S* embed, Stream s) {
  __shared__ float red[64];
  const int64_t t = blockIdx.x, row = t * s.W;
  float v[NV][N];
  if constexpr (SRC == ADD) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = (i * blockDim.x + threadIdx.x) * N;
      if (d < s.W) lds_<N>(y + t * s.y_stride + d, v[i]);
    }
    norm_row<NV, N>(v, s.wy, s.by, s.W, s.eps, red);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = (i * blockDim.x + threadIdx.x) * N;
      if (d < s.W) {
        float x[N];
        ldf<N>(s.x + row + d, x);
#pragma unroll
        for (int j = 0; j < N; ++j) v[i][j] += x[j];
      }
    }
  } else if constexpr (SRC == EMBED) {
    const int64_t raw = s.ids[t];
    const int64_t id = raw < 0 ? 0 : (raw >= s.vocab ? s.vocab - 1 : raw);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = (i * blockDim.x + threadIdx.x) * N;
      if (d < s.W) {
        lds_<N>(embed + id * s.W + d, v[i]);
#pragma unroll
        for (int j = 0; j < N; ++j) v[i][j] *= s.scale;
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = (i * blockDim.x + threadIdx.x) * N;
      if (d < s.W) {
        float u[N];
        ldf<N>(s.a + row + d, v[i]);
        if (s.b != nullptr) {
          ldf<N>(s.b + row + d, u);
#pragma unroll
          for (int j = 0; j < N; ++j) v[i][j] += u[j];
        }
        ldf<N>(s.e + row + d, u);
#pragma unroll
        for (int j = 0; j < N; ++j) v[i][j] += s.scale * u[j];
        if (s.step != nullptr) {
          ldf<N>(s.step + d, u);
#pragma unroll
          for (int j = 0; j < N; ++j) v[i][j] += u[j];
        }
      }
    }
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int d = (i * blockDim.x + threadIdx.x) * N;
    if (d < s.W) {
      if (s.x_out != nullptr) sts<N>(s.x_out + row + d, v[i]);
      if (s.tap != nullptr) sts<N>(s.tap + row + d, v[i]);
      if constexpr (sizeof(S) == 2) {
        if (s.hi != nullptr) {
          float rest[N];
#pragma unroll
          for (int j = 0; j < N; ++j) {
            const uint16_t top = f32_to_bf16(v[i][j]);
            rest[j] = v[i][j] - bf16_to_f32(top);
          }
          sts<N>((S*)s.hi + row + d, v[i]);
          sts<N>((S*)s.lo + row + d, rest);
        }
      }
    }
  }
  if (s.w == nullptr) return;
  norm_row<NV, N>(v, s.w, s.bias, s.W, s.eps, red + 32);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int d = (i * blockDim.x + threadIdx.x) * N;
    if (d < s.W) sts<N>(h + row + d, v[i]);
  }
}

template <typename S, int SRC>
void launch(OptT h, OptT y, OptT embed, Stream s, int T) {
  auto stream = at::hip::getCurrentHIPStream();
  S* hp = h.has_value() ? (S*)h->data_ptr() : nullptr;
  const S* yp = y.has_value() ? (const S*)y->data_ptr() : nullptr;
  const S* ep = embed.has_value() ? (const S*)embed->data_ptr() : nullptr;
  const int N = s.W % 4 == 0 && s.y_stride % 4 == 0 ? 4 : 1;
  const int vecs = s.W / N;
  // few rows: spread each over more waves; many: several rows to a CU
  const int want = T <= 512 || vecs > 2048 ? 512 : 256;
  TORCH_CHECK(vecs <= 8 * 512 * (N == 1 ? 4 : 1), "width ", s.W,
              " is too large");
  int nv = 1;
  while (nv * want < vecs) nv *= 2;
  const int threads = std::min(want, cdiv(vecs, WAVE) * WAVE);
#define HELIX_LS(NV, N)                                                      \
  hipLaunchKernelGGL((layer_stream_kernel<S, SRC, NV, N>), dim3(T),          \
                     dim3(threads), 0, stream, hp, yp, ep, s)
  if (N == 4) {
    if (nv == 1) HELIX_LS(1, 4);
    else if (nv == 2) HELIX_LS(2, 4);
    else if (nv == 4) HELIX_LS(4, 4);
    else HELIX_LS(8, 4);
  } else {
    if (nv <= 4) HELIX_LS(4, 1);
    else HELIX_LS(32, 1);
  }
#undef HELIX_LS
}

template <int SRC>
void launch(bool bf16, OptT h, OptT y, OptT embed, Stream s, int T) {
  if (T == 0) return;
  if (bf16) launch<uint16_t, SRC>(h, y, embed, s, T);
  else launch<float, SRC>(h, y, embed, s, T);
}

const float* f32(const OptT& t, int64_t n, const char* what) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->scalar_type() == torch::kFloat32 &&
                  t->is_contiguous() && t->numel() == n,
              what);
  return t->data_ptr<float>();
}

// The pieces every source shares; true for bf16 storage.
bool outputs(Stream& s, int64_t T, int64_t W, torch::ScalarType type, OptT h,
             OptT w, OptT b, OptT x_out, OptT tap, OptT terms, double eps) {
  TORCH_CHECK(type == torch::kBFloat16 || type == torch::kFloat32);
  TORCH_CHECK(h.has_value() == w.has_value() &&
              w.has_value() == b.has_value());
  if (h.has_value())
    TORCH_CHECK(h->is_contiguous() && h->size(0) == T && h->size(1) == W &&
                h->scalar_type() == type);
  s.w = f32(w, W, "norm weight");
  s.bias = f32(b, W, "norm bias");
  s.x_out = (float*)f32(x_out, T * W, "x_out");
  s.tap = (float*)f32(tap, T * W, "tap");
  if (terms.has_value()) {
    TORCH_CHECK(terms->is_contiguous() && terms->numel() == 2 * T * W &&
                terms->scalar_type() == torch::kBFloat16 &&
                type == torch::kBFloat16);
    s.hi = terms->data_ptr();
    s.lo = (uint16_t*)s.hi + T * W;
  }
  s.W = W;
  s.eps = (float)eps;
  s.y_stride = 4;
  return type == torch::kBFloat16;
}

}  // namespace

void stream_add(OptT h, torch::Tensor x, torch::Tensor y, torch::Tensor wy,
                torch::Tensor by, OptT w, OptT b, double eps, OptT x_out,
                OptT tap, OptT terms) {
  TORCH_CHECK(x.dim() == 2 && y.dim() == 2);
  const int64_t T = x.size(0), W = x.size(1);
  Stream s{};
  const bool bf16 = outputs(s, T, W, y.scalar_type(), h, w, b, x_out, tap,
                            terms, eps);
  TORCH_CHECK(y.size(0) == T && y.size(1) == W && y.stride(1) == 1);
  s.x = f32(x, T * W, "x");
  s.wy = f32(wy, W, "weight of y's norm");
  s.by = f32(by, W, "bias of y's norm");
  s.y_stride = y.stride(0);
  launch<ADD>(bf16, h, y, c10::nullopt, s, T);
}

void stream_embed(OptT h, torch::Tensor ids, torch::Tensor embed,
                  double scale, OptT w, OptT b, double eps, OptT x_out,
                  OptT terms) {
  const int64_t T = ids.numel(), W = embed.size(1);
  Stream s{};
  const bool bf16 = outputs(s, T, W, embed.scalar_type(), h, w, b, x_out,
                            c10::nullopt, terms, eps);
  TORCH_CHECK(ids.scalar_type() == torch::kInt64 && ids.is_contiguous() &&
              embed.is_contiguous() && embed.size(0) > 0);
  s.ids = ids.data_ptr<int64_t>();
  s.vocab = embed.size(0);
  s.scale = (float)scale;
  launch<EMBED>(bf16, h, c10::nullopt, embed, s, T);
}

void stream_enter(torch::Tensor h, torch::Tensor a, OptT a2, torch::Tensor e,
                  double e_scale, OptT step, torch::Tensor w, torch::Tensor b,
                  double eps, OptT x_out) {
  const int64_t T = h.size(0), W = h.size(1);
  Stream s{};
  const bool bf16 = outputs(s, T, W, h.scalar_type(), h, w, b, x_out,
                            c10::nullopt, c10::nullopt, eps);
  s.a = f32(a, T * W, "a");
  s.b = f32(a2, T * W, "a2");
  s.e = f32(e, T * W, "e");
  s.step = f32(step, W, "step");
  s.scale = (float)e_scale;
  launch<ENTER>(bf16, h, c10::nullopt, c10::nullopt, s, T);
}
