// What happens to fused query / key / value projections before attention:
// whole-projection RMS norms, rotation ("halves": dimension i turns with
// i + n), the write to the paged cache.
//
// The cosines and sines of a step are made once for all layers that turn
// alike. Keys go to pages [G][block][dim_pad], values to pages
// [G][vdim][block]: 8 tokens of one value dimension are 16 bytes in a row.
// Values may be the unrotated keys, and may be rotated over their full size.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr int NT = 256;

// cs[t][i] = (cos, sin) of pos[t] * freqs[i]; whole turns come off in double.
__global__ void rotary_table_kernel(float2* __restrict__ cs,
                                    const int64_t* __restrict__ pos,
                                    const double* __restrict__ freqs, int n,
                                    int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x;
  if (i >= total) return;
  double turns = (double)pos[i / n] * freqs[i % n] * 0.15915494309189535;
  turns -= rint(turns);
  float s, c;
  sincospif(2.f * (float)turns, &s, &c);
  cs[i] = make_float2(c, s);
}

struct Epilogue {
  const float2 *cs, *vcs;      // [T][nk], [T][nv] or null
  const float *qw, *kw;        // whole-row norm weights or null
  const int64_t* slots;
  int64_t z_stride, T;
  int q_at, k_at, v_at, H, G, D, Dp, E, nk, nv, bs, per;
  int q_rows, kv_rows;         // tokens whose queries / keys are wanted
  float eps;
};

template <typename S, int N>
__device__ __forceinline__ void get(const S* p, float* v) {
  if constexpr (N == 1) {
    v[0] = ld1(p);
  } else if constexpr (N == 2) {
    v[0] = ld1(p);
    v[1] = ld1(p + 1);
  } else {
    ldv<N>(p, v);
  }
}
template <typename S, int N>
__device__ __forceinline__ void put(S* p, const float* v) {
  if constexpr (N == 1) st1(p, v[0]); else stv<N>(p, v);
}

template <typename S, int N>
__device__ __forceinline__ float row_inv(const S* z, int n, float eps,
                                         float* red) {
  float ss = 0.f;
  for (int i = threadIdx.x * N; i < n; i += NT * N) {
    float v[N];
    get<S, N>(z + i, v);
#pragma unroll
    for (int j = 0; j < N; ++j) ss += v[j] * v[j];
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / n + eps);
  __syncthreads();
  return inv;
}

// Unit u of head h of one row z [heads][D]: N pairs of the turned part, or N
// dimensions of the rest. store(dim, values) takes the results.
template <typename S, int N, class Store>
__device__ __forceinline__ void turn_unit(const S* z, int h, int u, int D,
                                          const float2* cs, int n, float inv,
                                          const float* w, Store store) {
  const int pu = n / N;
  const int d = u < pu ? u * N : 2 * n + (u - pu) * N;
  const int at = h * D + d;
  float a[N], b[N];
  get<S, N>(z + at, a);
  if (w != nullptr) {
    float g[N];
    get<float, N>(w + at, g);
#pragma unroll
    for (int j = 0; j < N; ++j) a[j] *= inv * g[j];
  }
  if (u < pu) {
    get<S, N>(z + at + n, b);
    if (w != nullptr) {
      float g[N];
      get<float, N>(w + at + n, g);
#pragma unroll
      for (int j = 0; j < N; ++j) b[j] *= inv * g[j];
    }
    float r[2 * N];
    get<float, 2 * N>((const float*)(cs + d), r);
#pragma unroll
    for (int j = 0; j < N; ++j) {
      const float p = a[j] * r[2 * j] - b[j] * r[2 * j + 1];
      b[j] = b[j] * r[2 * j] + a[j] * r[2 * j + 1];
      a[j] = p;
    }
    store(d + n, b);
  }
  store(d, a);
}

// Units of a head: the turned pairs, then the rest.
__device__ __forceinline__ int units_of(int D, int n, int N) {
  return n / N + (D - 2 * n) / N;
}

constexpr int PER = 16;                       // tokens of a workgroup at most

// The first q_rows workgroups have a token's queries each, the others keys and
// values of `per` neighbouring tokens. Values go out token by token of one
// dimension, so that a page's 16-byte runs are written at once.
template <typename S, int N>
__global__ __launch_bounds__(NT) void attn_epilogue_kernel(
    S* __restrict__ q, S* __restrict__ kc, S* __restrict__ vc,
    const S* __restrict__ z, Epilogue m) {
  __shared__ float red[16], invs[PER];
  __shared__ int64_t slots[PER];
  const int pad = m.Dp - m.D;
  if ((int)blockIdx.x < m.q_rows) {
    const int64_t t = blockIdx.x;
    const S* zq = z + t * m.z_stride + m.q_at;
    float inv = 1.f;
    if (m.qw != nullptr) inv = row_inv<S, N>(zq, m.H * m.D, m.eps, red);
    S* qt = q + t * m.H * m.Dp;
    const int units = units_of(m.D, m.nk, N);
    for (int i = threadIdx.x; i < m.H * units; i += NT) {
      const int h = i / units;
      turn_unit<S, N>(zq, h, i - h * units, m.D, m.cs + t * m.nk, m.nk, inv,
                      m.qw, [&](int d, const float* v) {
                        put<S, N>(qt + h * m.Dp + d, v);
                      });
    }
    for (int i = threadIdx.x; i < m.H * pad; i += NT)
      st1(qt + i / pad * m.Dp + m.D + i % pad, 0.f);
    return;
  }
  const int64_t t0 = (int64_t)(blockIdx.x - m.q_rows) * m.per;
  const int nt = (int)min((int64_t)m.per, m.T - t0);
  if ((int)threadIdx.x < nt) slots[threadIdx.x] = m.slots[t0 + threadIdx.x];
  if (m.kw != nullptr) {
    const int lane = threadIdx.x & (WAVE - 1), n = m.G * m.D;
    for (int t = threadIdx.x / WAVE; t < nt; t += NT / WAVE) {
      const S* zk = z + (t0 + t) * m.z_stride + m.k_at;
      float ss = 0.f;
      for (int i = lane * N; i < n; i += WAVE * N) {
        float v[N];
        get<S, N>(zk + i, v);
#pragma unroll
        for (int j = 0; j < N; ++j) ss += v[j] * v[j];
      }
      ss = wave_reduce_sum(ss);
      if (lane == 0) invs[t] = 1.f / sqrtf(ss / n + m.eps);
    }
  }
  __syncthreads();
  {
    const int units = units_of(m.D, m.nk, N), all = m.G * units;
    for (int i = threadIdx.x; i < nt * all; i += NT) {
      const int t = i / all, g = (i - t * all) / units;
      const int64_t slot = slots[t];
      if (slot < 0) continue;
      S* kt = kc + ((slot / m.bs * m.G + g) * m.bs + slot % m.bs) * m.Dp;
      turn_unit<S, N>(z + (t0 + t) * m.z_stride + m.k_at, g,
                      i - t * all - g * units, m.D, m.cs + (t0 + t) * m.nk,
                      m.nk, m.kw != nullptr ? invs[t] : 1.f, m.kw,
                      [&](int d, const float* v) { put<S, N>(kt + d, v); });
    }
    for (int i = threadIdx.x; i < nt * m.G * pad; i += NT) {
      const int t = i / (m.G * pad), g = i / pad % m.G;
      const int64_t slot = slots[t];
      if (slot >= 0)
        st1(kc + ((slot / m.bs * m.G + g) * m.bs + slot % m.bs) * m.Dp +
                m.D + i % pad, 0.f);
    }
  }
  const int units = units_of(m.E, m.nv, N);
  for (int i = threadIdx.x; i < nt * m.G * units; i += NT) {
    const int t = i % nt, u = i / nt, g = u / units;
    const int64_t slot = slots[t];
    if (slot < 0) continue;
    S* vt = vc + (slot / m.bs * m.G + g) * m.E * m.bs + slot % m.bs;
    turn_unit<S, N>(z + (t0 + t) * m.z_stride + m.v_at, g, u - g * units,
                    m.E, m.vcs + (t0 + t) * m.nv, m.nv, 1.f, nullptr,
                    [&](int d, const float* v) {
#pragma unroll
                      for (int j = 0; j < N; ++j)
                        st1(vt + (int64_t)(d + j) * m.bs, v[j]);
                    });
  }
}

// fp32: factor of a query's scores by its position,
// 1 + coef * ln(floor((p + 1) / every) + 1).
__global__ void query_temperature_kernel(float* __restrict__ out,
                                         const int64_t* __restrict__ pos,
                                         float coef, double every, int T) {
  const int t = blockIdx.x * NT + threadIdx.x;
  if (t >= T) return;
  const double n = floor((double)(pos[t] + 1) / every) + 1.0;
  out[t] = 1.f + coef * logf((float)n);
}

template <typename S>
void launch(OptT q, torch::Tensor kc, torch::Tensor vc,
            torch::Tensor z, Epilogue m) {
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(m.q_rows + (m.kv_rows + m.per - 1) / m.per);
  S* qp = q.has_value() ? (S*)q->data_ptr() : nullptr;
  const bool vec = m.nk % 8 == 0 && m.nv % 8 == 0 && m.D % 8 == 0 &&
                   m.E % 8 == 0 && m.q_at % 8 == 0 && m.k_at % 8 == 0 &&
                   m.v_at % 8 == 0 && m.z_stride % 8 == 0 &&
                   (uintptr_t)z.data_ptr() % 16 == 0;
#define HELIX_EP(N)                                                          \
  hipLaunchKernelGGL((attn_epilogue_kernel<S, N>), grid, dim3(NT), 0,        \
                     stream, qp, (S*)kc.data_ptr(),                          \
                     (S*)vc.data_ptr(), (const S*)z.data_ptr(), m)
  if (vec) HELIX_EP(8);
  else HELIX_EP(1);
#undef HELIX_EP
}

const float2* table(const OptT& t, int64_t T, int& n) {
  n = 0;
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->scalar_type() == torch::kFloat32 && t->is_contiguous() &&
              t->dim() == 3 && t->size(0) == T && t->size(2) == 2);
  n = t->size(1);
  return (const float2*)t->data_ptr<float>();
}

const float* weight(const OptT& t, int64_t n) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->scalar_type() == torch::kFloat32 && t->is_contiguous() &&
              t->numel() == n);
  return t->data_ptr<float>();
}

}  // namespace

void rotary_table(torch::Tensor cs, torch::Tensor pos, torch::Tensor freqs) {
  const int64_t T = pos.numel(), n = freqs.numel();
  TORCH_CHECK(cs.scalar_type() == torch::kFloat32 && cs.is_contiguous() &&
              cs.numel() == T * n * 2);
  TORCH_CHECK(pos.scalar_type() == torch::kInt64 && pos.is_contiguous());
  TORCH_CHECK(freqs.scalar_type() == torch::kFloat64 &&
              freqs.is_contiguous());
  const int64_t total = T * n;
  if (total == 0) return;
  hipLaunchKernelGGL(rotary_table_kernel, dim3((total + NT - 1) / NT),
                     dim3(NT), 0, at::hip::getCurrentHIPStream(),
                     (float2*)cs.data_ptr<float>(), pos.data_ptr<int64_t>(),
                     freqs.data_ptr<double>(), (int)n, total);
}

void query_temperature(torch::Tensor out, torch::Tensor pos, double coef,
                       double every) {
  const int T = pos.numel();
  TORCH_CHECK(out.scalar_type() == torch::kFloat32 && out.is_contiguous() &&
              out.numel() == T && every > 0);
  TORCH_CHECK(pos.scalar_type() == torch::kInt64 && pos.is_contiguous());
  if (T == 0) return;
  hipLaunchKernelGGL(query_temperature_kernel, dim3((T + NT - 1) / NT),
                     dim3(NT), 0, at::hip::getCurrentHIPStream(),
                     out.data_ptr<float>(), pos.data_ptr<int64_t>(),
                     (float)coef, every, T);
}

void attn_epilogue(OptT q, torch::Tensor kc, torch::Tensor vc,
                   torch::Tensor z, int64_t q_at, int64_t k_at, int64_t v_at,
                   int64_t heads, int64_t dim, torch::Tensor slots, OptT cs,
                   OptT vcs, OptT qw, OptT kw, double eps, bool write_kv) {
  Epilogue m{};
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4);
  m.T = z.size(0);
  m.H = heads;
  m.Dp = kc.size(3);
  m.q_rows = q.has_value() ? m.T : 0;
  m.kv_rows = write_kv ? m.T : 0;
  m.G = kc.size(1);
  m.bs = kc.size(2);
  m.E = vc.size(2);
  m.D = dim;
  TORCH_CHECK(m.Dp % 8 == 0 && dim > 0 && dim <= m.Dp);
  TORCH_CHECK(vc.size(0) == kc.size(0) && vc.size(1) == m.G &&
              vc.size(3) == m.bs);
  if (q.has_value())
    TORCH_CHECK(q->dim() == 3 && q->size(0) == m.T && q->size(1) == m.H &&
                q->size(2) == m.Dp && q->is_contiguous() &&
                q->scalar_type() == z.scalar_type());
  for (const auto& t : {kc, vc})
    TORCH_CHECK(t.is_contiguous() && t.scalar_type() == z.scalar_type());
  TORCH_CHECK(z.stride(1) == 1);
  if (q.has_value()) TORCH_CHECK(q_at + m.H * dim <= z.size(1));
  if (write_kv)
    TORCH_CHECK(k_at >= 0 && k_at + m.G * dim <= z.size(1) && v_at >= 0 &&
                v_at + m.G * m.E <= z.size(1));
  TORCH_CHECK(slots.scalar_type() == torch::kInt64 && slots.numel() == m.T &&
              slots.is_contiguous());
  m.cs = table(cs, m.T, m.nk);
  m.vcs = table(vcs, m.T, m.nv);
  TORCH_CHECK(2 * m.nk <= m.D && 2 * m.nv <= m.E);
  m.qw = weight(qw, (int64_t)m.H * dim);
  m.kw = weight(kw, (int64_t)m.G * dim);
  m.slots = slots.data_ptr<int64_t>();
  m.z_stride = z.stride(0);
  m.q_at = q_at;
  m.k_at = k_at;
  m.v_at = v_at;
  m.eps = (float)eps;
  if (m.q_rows + m.kv_rows == 0) return;
  m.per = m.T > 1024 ? PER : 1;
  if (z.scalar_type() == torch::kBFloat16) launch<uint16_t>(q, kc, vc, z, m);
  else if (z.scalar_type() == torch::kFloat32) launch<float>(q, kc, vc, z, m);
  else TORCH_CHECK(false, "attention epilogue: bf16 or fp32");
}
