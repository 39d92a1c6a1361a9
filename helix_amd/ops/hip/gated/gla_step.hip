// Gated linear attention, a token at a time.
//
//   alpha = sigmoid(a2 a1 + b)^(1/tau)              per key channel
//   S <- diag(alpha) S + k v^T;  o = S^T q
//   y = out_scale * rms_norm(o) * w * silu(g)       per head
//
// or (FIXED) with a constant decay per head, q, k and v through silu, and o
// itself as the result:
//
//   S <- decay S + silu(k) silu(v)^T;  y = S^T silu(q)
//
// A workgroup owns one head's [D, E] matrix (TX threads with 4 values each
// across, TY down), reads it once and writes it once: the state is the
// traffic. Everything else of the mixer happens in the same launch. Spans of
// tokens (32-bit engines) keep the state in registers.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

struct Step {
  const void* a2;              // [H * D, rank_pad], storage type
  const float *a2_b, *norm;    // [H * D], [E]
  const float* decay;          // FIXED: [H]
  float* state;                // [slots, H, D, Ep]
  const int* slots;
  const int64_t* pos;          // per row
  const int* cu;               // spans: [B + 1] rows; null: a token each
  int64_t z_stride, y_stride;
  int q_at, k_at, v_at, g_at, a_at, H, D, E, Ep, rank, rank_pad;
  float inv_tau, q_scale, out_scale, eps;
};

// silu as it is stored
template <typename S>
__device__ __forceinline__ float stored_silu(const S* p) {
  S v;
  st1(&v, silu_s<S>(ld1(p)));
  return ld1(&v);
}

// NI: state rows per thread (D <= TY NI).
template <typename S, int TX, int TY, int NI, bool FIXED>
__global__ __launch_bounds__(TX* TY) void gla_step_kernel(
    S* __restrict__ y, const S* __restrict__ z, Step m) {
  constexpr int NT = TX * TY, NW = NT / WAVE;
  __shared__ float qs[TY * NI], ks[TY * NI], as[TY * NI], vs[TX * 4];
  __shared__ float part[NW][TX * 4], red[32];
  extern __shared__ float a1[];               // [rank_pad]
  const int b = blockIdx.x, h = blockIdx.y;
  const int tid = threadIdx.x, tx = tid % TX, ty = tid / TX;
  const int row0 = m.cu ? m.cu[b] : b, row1 = m.cu ? m.cu[b + 1] : b + 1;
  if (row0 >= row1) return;
  const int slot = m.slots[b], e = tx * 4;
  float* st = m.state + ((int64_t)max(slot, 0) * m.H + h) * m.D * m.Ep + e;

  float s[NI][4];
  const bool carried = slot >= 0 && m.pos[row0] > 0 && e < m.Ep;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int n = i * TY + ty;
    if (carried && n < m.D) {
      ldv<4>(st + (int64_t)n * m.Ep, s[i]);
    } else {
#pragma unroll
      for (int v = 0; v < 4; ++v) s[i][v] = 0.f;
    }
  }

  for (int row = row0; row < row1; ++row) {
    const S* zr = z + row * m.z_stride;
    if constexpr (!FIXED) {
      for (int r = tid; r < m.rank_pad; r += NT)
        a1[r] = r < m.rank ? ld1(zr + m.a_at + r) : 0.f;
    }
    __syncthreads();
    for (int d = tid; d < TY * NI; d += NT) {
      float a = 1.f, q = 0.f, k = 0.f;
      if (d < m.D) {
        const int c = h * m.D + d;
        if constexpr (FIXED) {
          as[d] = m.decay[h];
          qs[d] = stored_silu(zr + m.q_at + c);
          ks[d] = stored_silu(zr + m.k_at + c);
          continue;
        }
        float x = m.a2_b[c];
        const S* w = (const S*)m.a2 + (int64_t)c * m.rank_pad;
        for (int r = 0; r < m.rank_pad; r += 8) {
          float u[8];
          ldv<8>(w + r, u);
#pragma unroll
          for (int i = 0; i < 8; ++i) x += a1[r + i] * u[i];
        }
        a = expf(-softplus(-x) * m.inv_tau);
        q = ld1(zr + m.q_at + c) * m.q_scale;
        k = ld1(zr + m.k_at + c);
      }
      as[d] = a;
      qs[d] = q;
      ks[d] = k;
    }
    for (int i = tid; i < TX * 4; i += NT)
      vs[i] = i >= m.E ? 0.f
              : FIXED  ? stored_silu(zr + m.v_at + h * m.E + i)
                       : ld1(zr + m.v_at + h * m.E + i);
    __syncthreads();
    float acc[4] = {0.f, 0.f, 0.f, 0.f}, v[4];
    ldv<4>(vs + e, v);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int n = i * TY + ty;
      const float a = as[n], k = ks[n], q = qs[n];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[i][j] = a * s[i][j] + k * v[j];
        acc[j] += q * s[i][j];
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
#pragma unroll
      for (int off = TX; off < WAVE; off *= 2)
        acc[j] += __shfl_xor(acc[j], off, WAVE);
    }
    if ((tid & (WAVE - 1)) < TX) stv<4>(part[tid / WAVE] + e, acc);
    __syncthreads();
    float o = 0.f;
    if (tid < m.E) {
#pragma unroll
      for (int w = 0; w < NW; ++w) o += part[w][tid];
    }
    if constexpr (FIXED) {
      if (tid < m.E) st1(y + row * m.y_stride + h * m.E + tid, o);
      if (row + 1 < row1) __syncthreads();
      continue;
    }
    const float inv = 1.f / sqrtf(group_sum(o * o, red) / m.E + m.eps);
    if (tid < m.E) {
      const int c = h * m.E + tid;
      st1(y + row * m.y_stride + c,
          m.out_scale * o * inv * m.norm[tid] *
              silu_s<S>(ld1(zr + m.g_at + c)));
    }
    if (row + 1 < row1) __syncthreads();
  }
  if (slot >= 0 && e < m.Ep) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int n = i * TY + ty;
      if (n < m.D) stv<4>(st + (int64_t)n * m.Ep, s[i]);
    }
  }
}

const float* f32(const torch::Tensor& t, int64_t n) {
  TORCH_CHECK(t.scalar_type() == torch::kFloat32 && t.is_contiguous() &&
              t.numel() == n);
  return t.data_ptr<float>();
}

template <typename S, bool FIXED>
void launch(torch::Tensor y, torch::Tensor z, Step m, int B) {
  const dim3 grid(B, m.H);
#define HELIX_GLA(TX, TY, NI)                                                \
  hipLaunchKernelGGL((gla_step_kernel<S, TX, TY, NI, FIXED>), grid,          \
                     dim3(TX * TY), m.rank_pad * 4,                          \
                     at::hip::getCurrentHIPStream(),                         \
                     (S*)y.data_ptr(),                                       \
                     (const S*)z.data_ptr(), m)
#define HELIX_GLA_D(TX, TY)                                                  \
  if (m.D <= TY * 2) HELIX_GLA(TX, TY, 2);                                   \
  else if (m.D <= TY * 4) HELIX_GLA(TX, TY, 4);                              \
  else if (m.D <= TY * 8) HELIX_GLA(TX, TY, 8);                              \
  else HELIX_GLA(TX, TY, 16)
  if (m.E <= 32) { HELIX_GLA_D(8, 32); }
  else if (m.E <= 64) { HELIX_GLA_D(16, 16); }
  else if (m.E <= 128) { HELIX_GLA_D(32, 16); }
  else { HELIX_GLA_D(64, 16); }
#undef HELIX_GLA_D
#undef HELIX_GLA
}

// What both forms share; the number of sequences.
int arguments(Step& m, const torch::Tensor& y, const torch::Tensor& z,
              int64_t q_at, int64_t k_at, int64_t v_at, int64_t vdim,
              const torch::Tensor& state, const torch::Tensor& slots,
              const torch::Tensor& pos, const OptT& cu) {
  TORCH_CHECK(state.dim() == 4);
  const int64_t T = z.size(0);
  m.H = state.size(1);
  m.D = state.size(2);
  m.Ep = state.size(3);
  m.E = vdim;
  TORCH_CHECK(m.D <= 256 && m.E <= 256, "heads of at most 256 x 256, got ",
              m.D, " x ", m.E);
  TORCH_CHECK(m.Ep % 4 == 0 && m.Ep >= m.E && m.E > 0 && m.D > 0);
  TORCH_CHECK(z.dim() == 2 && z.stride(1) == 1 && y.stride(1) == 1 &&
              y.size(0) == T && y.size(1) == m.H * m.E &&
              y.scalar_type() == z.scalar_type());
  const int64_t width = z.size(1);
  TORCH_CHECK(q_at + m.H * m.D <= width && k_at + m.H * m.D <= width &&
              v_at + m.H * m.E <= width);
  m.state = (float*)f32(state, state.numel());
  const int B = cu.has_value() ? cu->numel() - 1 : T;
  TORCH_CHECK(slots.scalar_type() == torch::kInt32 && slots.numel() == B &&
              slots.is_contiguous());
  TORCH_CHECK(pos.scalar_type() == torch::kInt64 && pos.numel() == T &&
              pos.is_contiguous());
  if (cu.has_value()) {
    TORCH_CHECK(cu->scalar_type() == torch::kInt32 && cu->is_contiguous());
    m.cu = cu->data_ptr<int>();
  }
  m.slots = slots.data_ptr<int>();
  m.pos = pos.data_ptr<int64_t>();
  m.z_stride = z.stride(0);
  m.y_stride = y.stride(0);
  m.q_at = q_at;
  m.k_at = k_at;
  m.v_at = v_at;
  return T == 0 ? 0 : B;
}

}  // namespace

// z and y rows: one token of sequence r each, or (with cu) the concatenated
// tokens of cu.numel() - 1 sequences.
void gla_step(torch::Tensor y, torch::Tensor z, int64_t q_at, int64_t k_at,
              int64_t v_at, int64_t g_at, int64_t a_at, int64_t vdim, int64_t rank,
              torch::Tensor a2, torch::Tensor a2_b, torch::Tensor norm,
              double tau, double q_scale, double out_scale, double eps,
              torch::Tensor state, torch::Tensor slots, torch::Tensor pos,
              OptT cu) {
  Step m{};
  const int B = arguments(m, y, z, q_at, k_at, v_at, vdim, state, slots, pos,
                          cu);
  m.rank = rank;
  m.rank_pad = a2.size(1);
  TORCH_CHECK(a2.dim() == 2 && a2.is_contiguous() &&
              a2.size(0) == (int64_t)m.H * m.D && m.rank_pad % 8 == 0 &&
              rank >= 1 && rank <= m.rank_pad && m.rank_pad <= 4096 &&
              a2.scalar_type() == z.scalar_type());
  TORCH_CHECK(g_at + m.H * m.E <= z.size(1) && a_at + m.rank <= z.size(1));
  m.a2 = a2.data_ptr();
  m.a2_b = f32(a2_b, (int64_t)m.H * m.D);
  m.norm = f32(norm, m.E);
  m.g_at = g_at;
  m.a_at = a_at;
  m.inv_tau = (float)(1.0 / tau);
  m.q_scale = (float)q_scale;
  m.out_scale = (float)out_scale;
  m.eps = (float)eps;
  if (B == 0) return;
  if (z.scalar_type() == torch::kBFloat16) launch<uint16_t, false>(y, z, m, B);
  else if (z.scalar_type() == torch::kFloat32) launch<float, false>(y, z, m, B);
  else TORCH_CHECK(false, "gla: bf16 or fp32");
}

// The form with a constant decay per head; y is o.
void decay_step(torch::Tensor y, torch::Tensor z, int64_t q_at, int64_t k_at,
                int64_t v_at, int64_t vdim, torch::Tensor decay,
                torch::Tensor state, torch::Tensor slots, torch::Tensor pos,
                OptT cu) {
  Step m{};
  const int B = arguments(m, y, z, q_at, k_at, v_at, vdim, state, slots, pos,
                          cu);
  m.decay = f32(decay, m.H);
  if (B == 0) return;
  if (z.scalar_type() == torch::kBFloat16) launch<uint16_t, true>(y, z, m, B);
  else if (z.scalar_type() == torch::kFloat32) launch<float, true>(y, z, m, B);
  else TORCH_CHECK(false, "decay_step: bf16 or fp32");
}
