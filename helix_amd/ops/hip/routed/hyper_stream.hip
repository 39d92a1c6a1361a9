// Several fp32 residual streams side by side (hyper-connections), with an
// elementwise norm (tanh(alpha u) w + b).
//
//   x_t <- sum_s mix[s, t] x_s + out[t] y         a sublayer's result y
//   h   <- norm(sum_s into[s] x_s)                what the next one reads
//
// One launch does both: nothing of it crosses columns, so a thread owns some
// columns of one token and the old streams are read once. y is a row, or
// made here from a mixture's routed rows: the weighted sum of up to K expert
// results, with identity experts returning the sublayer's own input.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr int NT = 256;
constexpr int MAX_STREAMS = 8;

enum Source { EMBED, ROW, ROUTED };

struct Hyper {
  float* x;                    // [T, NS, W]
  const float *mix, *out;      // [NS, NS] from, to; [NS]
  const float* into;           // [NS]
  const float *alpha, *w, *b;  // norm: scalar, [W], [W]
  float* tap;                  // [T, W] or null: sum of the new streams
  // EMBED
  const int64_t *ids, *pos;
  int64_t vocab, places;
  // ROUTED
  const int* slot;             // [T, K] row of `rows`, negative: identity
  const float* weight;         // [T, K]
  int64_t y_stride, total;
  int W, K;
};

template <typename S, int N>
__device__ __forceinline__ void get(const S* p, float* v) {
  if constexpr (N == 1) v[0] = ld1(p); else ldv<N>(p, v);
}
template <typename S, int N>
__device__ __forceinline__ void put(S* p, const float* v) {
  if constexpr (N == 1) st1(p, v[0]); else stv<N>(p, v);
}

// tanh; the bf16 build by the native exponential
template <typename S>
__device__ __forceinline__ float tanh_of(float x) { return tanh_s<S>(x); }

// y: EMBED the token table, ROW the results, ROUTED the experts' rows;
// other: EMBED the position table, ROUTED the sublayer's input.
template <typename S, int SRC, int NS, int N>
__global__ __launch_bounds__(NT) void hyper_stream_kernel(
    S* __restrict__ h, const S* __restrict__ y, const S* __restrict__ other,
    Hyper m) {
  const int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x;
  if (i >= m.total) return;
  const int cols = m.W / N;
  const int64_t t = i / cols;
  const int d = (int)(i - t * cols) * N;
  float* xr = m.x + t * NS * m.W + d;

  float v[NS][N], r[N];
  if constexpr (SRC == EMBED) {
    const int64_t id = min(max(m.ids[t], (int64_t)0), m.vocab - 1);
    const int64_t p = min(max(m.pos[t], (int64_t)0), m.places - 1);
    float e[N];
    get<S, N>(y + id * m.W + d, e);
    get<S, N>(other + p * m.W + d, r);
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int j = 0; j < N; ++j) v[s][j] = e[j] + r[j];
  } else {
    float x[NS][N];
#pragma unroll
    for (int s = 0; s < NS; ++s) get<float, N>(xr + s * m.W, x[s]);
    if constexpr (SRC == ROW) {
      get<S, N>(y + t * m.y_stride + d, r);
    } else {
      float self = 0.f;
#pragma unroll
      for (int j = 0; j < N; ++j) r[j] = 0.f;
#pragma unroll 4
      for (int k = 0; k < m.K; ++k) {
        const int at = m.slot[t * m.K + k];
        const float g = m.weight[t * m.K + k];
        float e[N];
        // row 0 may never have been written: selected, not multiplied by 0
        get<S, N>(y + (int64_t)max(at, 0) * m.W + d, e);
        self += at < 0 ? g : 0.f;
#pragma unroll
        for (int j = 0; j < N; ++j) r[j] += at < 0 ? 0.f : g * e[j];
      }
      if (self != 0.f) {
        float e[N];
        get<S, N>(other + t * m.W + d, e);
#pragma unroll
        for (int j = 0; j < N; ++j) r[j] += self * e[j];
      }
    }
#pragma unroll
    for (int q = 0; q < NS; ++q) {
      const float o = m.out[q];
#pragma unroll
      for (int j = 0; j < N; ++j) v[q][j] = o * r[j];
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        const float c = m.mix[s * NS + q];
#pragma unroll
        for (int j = 0; j < N; ++j) v[q][j] += c * x[s][j];
      }
    }
  }
  float u[N], sum[N];
#pragma unroll
  for (int j = 0; j < N; ++j) u[j] = sum[j] = 0.f;
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    const float c = m.into[s];
    put<float, N>(xr + s * m.W, v[s]);
#pragma unroll
    for (int j = 0; j < N; ++j) {
      u[j] += c * v[s][j];
      sum[j] += v[s][j];
    }
  }
  if (m.tap != nullptr) put<float, N>(m.tap + t * m.W + d, sum);
  const float alpha = m.alpha[0];
  float w[N], b[N];
  get<float, N>(m.w + d, w);
  get<float, N>(m.b + d, b);
#pragma unroll
  for (int j = 0; j < N; ++j) u[j] = tanh_of<S>(alpha * u[j]) * w[j] + b[j];
  put<S, N>(h + t * m.W + d, u);
}

// rows <- cap * tanh(rows / cap), fp32 in place
__global__ __launch_bounds__(NT) void softcap_kernel(float* __restrict__ x,
                                                     float cap,
                                                     int64_t n) {
  const int64_t i = ((int64_t)blockIdx.x * NT + threadIdx.x) * 4;
  if (i + 4 <= n) {
    float v[4];
    ldv<4>(x + i, v);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = cap * tanhf(v[j] / cap);
    stv<4>(x + i, v);
  } else {
    for (int64_t j = i; j < n; ++j) x[j] = cap * tanhf(x[j] / cap);
  }
}

const float* f32(const torch::Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kFloat32 &&
                  t.is_contiguous() && t.numel() == n,
              what);
  return t.data_ptr<float>();
}

template <typename S, int SRC, int NS>
void launch_as(Hyper m, torch::Tensor h, torch::Tensor y, OptT other) {
  auto stream = at::hip::getCurrentHIPStream();
  const S* op = other.has_value() ? (const S*)other->data_ptr() : nullptr;
  const bool vec = m.W % 4 == 0 && m.y_stride % 4 == 0 &&
                   (uintptr_t)y.data_ptr() % 16 == 0;
  m.total = h.size(0) * (m.W / (vec ? 4 : 1));
  const dim3 grid((m.total + NT - 1) / NT);
#define HELIX_HS(N)                                                          \
  hipLaunchKernelGGL((hyper_stream_kernel<S, SRC, NS, N>), grid, dim3(NT),   \
                     0, stream, (S*)h.data_ptr(), (const S*)y.data_ptr(),    \
                     op, m)
  if (vec) HELIX_HS(4);
  else HELIX_HS(1);
#undef HELIX_HS
}

template <int SRC>
void launch(Hyper m, int64_t streams, torch::Tensor h, torch::Tensor y,
            OptT other) {
  TORCH_CHECK(y.scalar_type() == h.scalar_type());
  if (h.size(0) == 0) return;
#define HELIX_NS(NS)                                                         \
  case NS:                                                                   \
    if (h.scalar_type() == torch::kBFloat16)                                 \
      launch_as<uint16_t, SRC, NS>(m, h, y, other);                          \
    else                                                                     \
      launch_as<float, SRC, NS>(m, h, y, other);                             \
    break;
  switch (streams) {
    HELIX_NS(1) HELIX_NS(2) HELIX_NS(3) HELIX_NS(4)
    HELIX_NS(5) HELIX_NS(6) HELIX_NS(7) HELIX_NS(8)
  }
#undef HELIX_NS
}

Hyper common(const torch::Tensor& h, const torch::Tensor& x,
             const torch::Tensor& into, const torch::Tensor& alpha,
             const torch::Tensor& w, const torch::Tensor& b, OptT tap) {
  Hyper m{};
  TORCH_CHECK(x.dim() == 3 && h.dim() == 2 && h.is_contiguous());
  const int64_t T = h.size(0), W = h.size(1), NS = x.size(1);
  TORCH_CHECK(NS >= 1 && NS <= MAX_STREAMS, NS, " streams, at most ",
              MAX_STREAMS);
  TORCH_CHECK(x.size(0) == T && x.size(2) == W);
  TORCH_CHECK(h.scalar_type() == torch::kBFloat16 ||
              h.scalar_type() == torch::kFloat32);
  m.x = (float*)f32(x, T * NS * W, "streams");
  m.into = f32(into, NS, "input coefficients");
  m.alpha = f32(alpha, 1, "alpha");
  m.w = f32(w, W, "norm weight");
  m.b = f32(b, W, "norm bias");
  if (tap.has_value()) m.tap = (float*)f32(*tap, T * W, "tap");
  m.W = W;
  m.y_stride = W;
  return m;
}

}  // namespace

void hyper_embed(torch::Tensor h, torch::Tensor x, torch::Tensor ids,
                 torch::Tensor pos, torch::Tensor embed, torch::Tensor places,
                 torch::Tensor into, torch::Tensor alpha, torch::Tensor w,
                 torch::Tensor b) {
  Hyper m = common(h, x, into, alpha, w, b, c10::nullopt);
  for (const auto& t : {ids, pos})
    TORCH_CHECK(t.scalar_type() == torch::kInt64 && t.is_contiguous() &&
                t.numel() == h.size(0));
  for (const auto& t : {embed, places})
    TORCH_CHECK(t.dim() == 2 && t.is_contiguous() && t.size(0) > 0 &&
                t.size(1) == m.W && t.scalar_type() == h.scalar_type());
  m.ids = ids.data_ptr<int64_t>();
  m.pos = pos.data_ptr<int64_t>();
  m.vocab = embed.size(0);
  m.places = places.size(0);
  launch<EMBED>(m, x.size(1), h, embed, places);
}

void hyper_step(torch::Tensor h, torch::Tensor x, torch::Tensor y,
                torch::Tensor mix, torch::Tensor out, torch::Tensor into,
                torch::Tensor alpha, torch::Tensor w, torch::Tensor b,
                OptT tap) {
  Hyper m = common(h, x, into, alpha, w, b, tap);
  const int64_t NS = x.size(1);
  m.mix = f32(mix, NS * NS, "mix");
  m.out = f32(out, NS, "output coefficients");
  TORCH_CHECK(y.dim() == 2 && y.size(0) == h.size(0) && y.size(1) == m.W &&
              y.stride(1) == 1);
  m.y_stride = y.stride(0);
  launch<ROW>(m, NS, h, y, c10::nullopt);
}

// rows [P, W]; slot and weight [T, K]; self [T, W]: the sublayer's input.
void hyper_step_routed(torch::Tensor h, torch::Tensor x, torch::Tensor rows,
                       torch::Tensor slot, torch::Tensor weight,
                       torch::Tensor self, torch::Tensor mix,
                       torch::Tensor out, torch::Tensor into,
                       torch::Tensor alpha, torch::Tensor w, torch::Tensor b,
                       OptT tap) {
  Hyper m = common(h, x, into, alpha, w, b, tap);
  const int64_t NS = x.size(1), T = h.size(0);
  m.mix = f32(mix, NS * NS, "mix");
  m.out = f32(out, NS, "output coefficients");
  TORCH_CHECK(slot.dim() == 2 && slot.size(0) == T &&
              slot.scalar_type() == torch::kInt32 && slot.is_contiguous());
  m.K = slot.size(1);
  m.slot = slot.data_ptr<int>();
  m.weight = f32(weight, T * m.K, "weights");
  TORCH_CHECK(rows.dim() == 2 && rows.is_contiguous() &&
              rows.size(0) >= T * m.K && rows.size(1) == m.W);
  TORCH_CHECK(self.is_contiguous() && self.numel() == T * m.W &&
              self.scalar_type() == h.scalar_type());
  launch<ROUTED>(m, NS, h, rows, self);
}

void softcap(torch::Tensor x, double cap) {
  f32(x, x.numel(), "softcap: fp32");
  TORCH_CHECK(cap > 0 && (uintptr_t)x.data_ptr() % 16 == 0);
  const int64_t n = x.numel();
  if (n == 0) return;
  hipLaunchKernelGGL(softcap_kernel, dim3((n + 4 * NT - 1) / (4 * NT)),
                     dim3(NT), 0, at::hip::getCurrentHIPStream(),
                     x.data_ptr<float>(), (float)cap, n);
}
