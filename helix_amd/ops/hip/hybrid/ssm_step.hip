// Mamba-2 mixer, a token at a time.
//
//   xBC = silu(conv(inputs));  dt = softplus(raw + bias)
//   S <- exp(-exp(A_log) dt) S + dt B x^T;  y = (S^T C + D x) silu(z)
//
// A workgroup owns one head's [state, vdim] matrix (16 threads across the
// values, 16 down the state), reads it once and writes it once: the state is
// the traffic. Single tokens do their convolution here; spans of tokens
// (32-bit engines) take it from conv_span and keep the state in registers.
//
// Ring entry pos % taps holds the raw inputs of position pos, so the entry
// that a step writes is one that no workgroup of the step reads.
#include "tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr int NT = 256;
constexpr int TX = 16, TY = NT / TX;

struct Step {
  const float *conv, *conv_b, *dt_bias, *A_log, *D;
  float* state;                // [slots, H, N, P]
  const int* slots;
  const int64_t* pos;          // per row
  const int* cu;               // spans: [B + 1] rows; null: a token each
  int64_t z_stride, y_stride;
  int z_at, xbc_at, dt_at, H, P, N, G, taps, C;
};

// NI: state rows per thread (N <= 16 NI), VEC: values per thread.
template <typename S, int VEC, int NI>
__global__ __launch_bounds__(NT) void ssm_step_kernel(
    S* __restrict__ y, const S* __restrict__ z, const S* __restrict__ xbc,
    S* ring, Step m) {
  extern __shared__ float sh[];               // x [TX * VEC], B [N], C [N]
  __shared__ float part[NT / WAVE][TX * VEC];
  float *xs = sh, *Bs = sh + TX * VEC, *Cs = Bs + m.N;
  const int b = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * TX * VEC;
  const int tid = threadIdx.x, tx = tid % TX, ty = tid / TX;
  const int row0 = m.cu ? m.cu[b] : b, row1 = m.cu ? m.cu[b + 1] : b + 1;
  const int slot = m.slots[b];
  const int hpg = m.H / m.G, g = h / hpg, inner = m.H * m.P;
  const int p = p0 + tx * VEC, np = min(TX * VEC, m.P - p0);
  const bool mine = p < m.P;
  float* st = m.state + ((int64_t)slot * m.H + h) * m.N * m.P + p;

  float s[NI][VEC];
  const bool carried = slot >= 0 && m.pos[row0] > 0 && mine;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int n = i * TY + ty;
    if (carried && n < m.N) {
      if constexpr (VEC == 4) ldv<4>(st + (int64_t)n * m.P, s[i]);
      else s[i][0] = st[(int64_t)n * m.P];
    } else {
#pragma unroll
      for (int v = 0; v < VEC; ++v) s[i][v] = 0.f;
    }
  }
  const float decay = -expf(m.A_log[h]), bias = m.dt_bias[h], Dh = m.D[h];

  for (int row = row0; row < row1; ++row) {
    // inputs of this token: the head's values, its group's B and C
    for (int i = tid; i < np + 2 * m.N; i += NT) {
      const int c = i < np ? h * m.P + p0 + i
                           : (i < np + m.N
                                  ? inner + g * m.N + i - np
                                  : inner + (m.G + g) * m.N + i - np - m.N);
      float v;
      if (xbc != nullptr) {
        v = ld1(xbc + (int64_t)row * m.C + c);
      } else {
        const int64_t pos = m.pos[row];
        const S* own = z + row * m.z_stride + m.xbc_at + c;
        S* rs = ring + (int64_t)max(slot, 0) * m.taps * m.C + c;
        const float* w = m.conv + (int64_t)c * m.taps;
        float a = m.conv_b[c];
        for (int k = m.taps - 1; k > 0; --k)
          if (slot >= 0 && pos >= k)
            a += w[m.taps - 1 - k] * ld1(rs + (pos - k) % m.taps * m.C);
        a += w[m.taps - 1] * ld1(own);
        // values belong to their head, B and C to the group's first one
        if (slot >= 0 && (i < np || (h % hpg == 0 && p0 == 0)))
          rs[pos % m.taps * m.C] = *own;
        S q;
        st1(&q, silu_s<S>(a));                // as the span path stores it
        v = ld1(&q);
      }
      if (i < np) xs[i] = v; else Bs[i - np] = v;
    }
    const float dt =
        softplus(ld1(z + row * m.z_stride + m.dt_at + h) + bias);
    const float keep = expf(decay * dt);
    __syncthreads();
    float acc[VEC], x[VEC];
#pragma unroll
    for (int v = 0; v < VEC; ++v) {
      acc[v] = 0.f;
      x[v] = mine ? xs[tx * VEC + v] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int n = i * TY + ty;
      if (n < m.N) {
        const float bn = dt * Bs[n], cn = Cs[n];
#pragma unroll
        for (int v = 0; v < VEC; ++v) {
          s[i][v] = keep * s[i][v] + bn * x[v];
          acc[v] += cn * s[i][v];
        }
      }
    }
#pragma unroll
    for (int v = 0; v < VEC; ++v) {
      acc[v] += __shfl_xor(acc[v], 16, WAVE);
      acc[v] += __shfl_xor(acc[v], 32, WAVE);
      if ((tid & (WAVE - 1)) < TX) part[tid / WAVE][tx * VEC + v] = acc[v];
    }
    __syncthreads();
    if (tid < np) {
      float o = Dh * xs[tid];
#pragma unroll
      for (int w = 0; w < NT / WAVE; ++w) o += part[w][tid];
      const int c = h * m.P + p0 + tid;
      o *= silu_s<S>(ld1(z + row * m.z_stride + m.z_at + c));
      st1(y + row * m.y_stride + c, o);
    }
    if (row + 1 < row1) __syncthreads();
  }
  if (slot >= 0 && mine) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int n = i * TY + ty;
      if (n < m.N) {
        if constexpr (VEC == 4) stv<4>(st + (int64_t)n * m.P, s[i]);
        else st[(int64_t)n * m.P] = s[i][0];
      }
    }
  }
}

// silu(conv) of prompt portions, a thread per channel and block of tokens;
// the first block of a sequence reads the ring and, being the only one that
// does, refills it.
constexpr int SPAN = 64;

template <typename S>
__global__ __launch_bounds__(NT) void conv_span_kernel(
    S* __restrict__ out, const S* __restrict__ z, int64_t z_stride,
    int xbc_at, const float* __restrict__ conv,
    const float* __restrict__ conv_b, S* ring, const int* __restrict__ slots,
    const int64_t* __restrict__ pos, const int* __restrict__ cu, int taps,
    int C) {
  const int b = blockIdx.y, c = blockIdx.x * NT + threadIdx.x;
  const int row0 = cu[b], len = cu[b + 1] - row0;
  const int t0 = blockIdx.z * SPAN;
  if (c >= C || t0 >= len) return;
  const int slot = slots[b];
  const int64_t p0 = pos[row0];
  S* rs = ring + (int64_t)max(slot, 0) * taps * C + c;
  const S* zc = z + (int64_t)row0 * z_stride + xbc_at + c;
  const float* w = conv + (int64_t)c * taps;
  for (int t = t0; t < min(len, t0 + SPAN); ++t) {
    float a = conv_b[c];
    for (int k = taps - 1; k >= 0; --k) {
      if (k <= t)
        a += w[taps - 1 - k] * ld1(zc + (int64_t)(t - k) * z_stride);
      else if (slot >= 0 && p0 + t >= k)
        a += w[taps - 1 - k] * ld1(rs + (p0 + t - k) % taps * C);
    }
    st1(out + (int64_t)(row0 + t) * C + c, silu_s<S>(a));
  }
  // tokens past the first block are at least SPAN >= taps - 1 in
  if (t0 == 0 && slot >= 0)
    for (int t = max(0, len - taps); t < len; ++t)
      rs[(p0 + t) % taps * C] = zc[(int64_t)t * z_stride];
}

template <typename S, int VEC>
void launch_step(torch::Tensor y, torch::Tensor z, OptT xbc,
                 torch::Tensor ring, Step m, int B) {
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(B, m.H, cdiv(m.P, TX * VEC));
  const int lds = (TX * VEC + 2 * m.N) * sizeof(float);
#define HELIX_STEP(NI)                                                       \
  hipLaunchKernelGGL((ssm_step_kernel<S, VEC, NI>), grid, dim3(NT), lds,     \
                     stream, (S*)y.data_ptr(), (const S*)z.data_ptr(),       \
                     xbc.has_value() ? (const S*)xbc->data_ptr() : nullptr,  \
                     (S*)ring.data_ptr(), m)
  const int ni = cdiv(m.N, TY);
  if (ni <= 2) HELIX_STEP(2);
  else if (ni <= 4) HELIX_STEP(4);
  else if (ni <= 8) HELIX_STEP(8);
  else if (ni <= 16) HELIX_STEP(16);
  else HELIX_STEP(32);
#undef HELIX_STEP
}

void check_f32(const torch::Tensor& t, int64_t n) {
  TORCH_CHECK(t.scalar_type() == torch::kFloat32 && t.is_contiguous() &&
              t.numel() == n);
}

}  // namespace

// z and y rows: one token of sequence r each, or (with xbc and cu) the
// concatenated tokens of cu.numel() - 1 sequences.
void ssm_step(torch::Tensor y, torch::Tensor z, OptT xbc, int64_t z_at,
              int64_t xbc_at, int64_t dt_at, torch::Tensor conv,
              torch::Tensor conv_b, torch::Tensor dt_bias,
              torch::Tensor A_log, torch::Tensor D, torch::Tensor ring,
              torch::Tensor state, torch::Tensor slots, torch::Tensor pos,
              OptT cu) {
  TORCH_CHECK(state.dim() == 4 && ring.dim() == 3);
  Step m{};
  m.H = state.size(1);
  m.N = state.size(2);
  m.P = state.size(3);
  m.taps = ring.size(1);
  m.C = ring.size(2);
  const int64_t T = z.size(0), inner = (int64_t)m.H * m.P;
  TORCH_CHECK(m.N > 0 && (m.C - inner) % (2 * m.N) == 0 && m.C > inner);
  m.G = (m.C - inner) / (2 * m.N);
  TORCH_CHECK(m.H % m.G == 0);
  TORCH_CHECK(m.N <= 512, "state size ", m.N, " > 512");
  TORCH_CHECK(z.stride(1) == 1 && y.stride(1) == 1 && y.size(0) == T &&
              y.size(1) == inner);
  TORCH_CHECK(z_at + inner <= z.size(1) && xbc_at + m.C <= z.size(1) &&
              dt_at + m.H <= z.size(1));
  check_f32(conv, (int64_t)m.C * m.taps);
  check_f32(conv_b, m.C);
  check_f32(dt_bias, m.H);
  check_f32(A_log, m.H);
  check_f32(D, m.H);
  check_f32(state, state.numel());
  TORCH_CHECK(ring.is_contiguous() && ring.size(0) == state.size(0));
  TORCH_CHECK(z.scalar_type() == y.scalar_type() &&
              z.scalar_type() == ring.scalar_type());
  TORCH_CHECK(xbc.has_value() == cu.has_value());
  const int B = cu.has_value() ? cu->numel() - 1 : T;
  TORCH_CHECK(slots.scalar_type() == torch::kInt32 && slots.numel() == B &&
              slots.is_contiguous());
  TORCH_CHECK(pos.scalar_type() == torch::kInt64 && pos.numel() == T &&
              pos.is_contiguous());
  if (xbc.has_value()) {
    TORCH_CHECK(xbc->is_contiguous() && xbc->scalar_type() == z.scalar_type()
                && xbc->size(0) == T && xbc->size(1) == m.C);
    TORCH_CHECK(cu->scalar_type() == torch::kInt32 && cu->is_contiguous());
    m.cu = cu->data_ptr<int>();
  }
  m.conv = conv.data_ptr<float>();
  m.conv_b = conv_b.data_ptr<float>();
  m.dt_bias = dt_bias.data_ptr<float>();
  m.A_log = A_log.data_ptr<float>();
  m.D = D.data_ptr<float>();
  m.state = state.data_ptr<float>();
  m.slots = slots.data_ptr<int>();
  m.pos = pos.data_ptr<int64_t>();
  m.z_stride = z.stride(0);
  m.y_stride = y.stride(0);
  m.z_at = z_at;
  m.xbc_at = xbc_at;
  m.dt_at = dt_at;
  if (B == 0 || T == 0) return;
  const bool vec = m.P % 4 == 0;
  if (z.scalar_type() == torch::kBFloat16) {
    if (vec) launch_step<uint16_t, 4>(y, z, xbc, ring, m, B);
    else launch_step<uint16_t, 1>(y, z, xbc, ring, m, B);
  } else {
    TORCH_CHECK(z.scalar_type() == torch::kFloat32, "ssm: bf16 or fp32");
    if (vec) launch_step<float, 4>(y, z, xbc, ring, m, B);
    else launch_step<float, 1>(y, z, xbc, ring, m, B);
  }
}

void conv_span(torch::Tensor out, torch::Tensor z, int64_t xbc_at,
               torch::Tensor conv, torch::Tensor conv_b, torch::Tensor ring,
               torch::Tensor slots, torch::Tensor pos, torch::Tensor cu,
               int64_t max_len) {
  const int taps = ring.size(1), C = ring.size(2), B = cu.numel() - 1;
  TORCH_CHECK(out.is_contiguous() && ring.is_contiguous() &&
              out.size(0) == z.size(0) && out.size(1) == C &&
              z.stride(1) == 1 && xbc_at + C <= z.size(1));
  TORCH_CHECK(out.scalar_type() == z.scalar_type() &&
              ring.scalar_type() == z.scalar_type());
  TORCH_CHECK(taps - 1 <= SPAN, "at most ", SPAN + 1, " taps");
  check_f32(conv, (int64_t)C * taps);
  check_f32(conv_b, C);
  TORCH_CHECK(slots.scalar_type() == torch::kInt32 && slots.numel() == B &&
              slots.is_contiguous() && cu.scalar_type() == torch::kInt32 &&
              cu.is_contiguous());
  TORCH_CHECK(pos.scalar_type() == torch::kInt64 && pos.is_contiguous() &&
              pos.numel() == z.size(0));
  if (B == 0 || z.size(0) == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(cdiv(C, NT), B, cdiv((int)max_len, SPAN));
#define HELIX_CONV(S)                                                        \
  hipLaunchKernelGGL((conv_span_kernel<S>), grid, dim3(NT), 0, stream,       \
                     (S*)out.data_ptr(), (const S*)z.data_ptr(),             \
                     z.stride(0), (int)xbc_at, conv.data_ptr<float>(),       \
                     conv_b.data_ptr<float>(), (S*)ring.data_ptr(),          \
                     slots.data_ptr<int>(), pos.data_ptr<int64_t>(),         \
                     cu.data_ptr<int>(), taps, C)
  if (z.scalar_type() == torch::kBFloat16) HELIX_CONV(uint16_t);
  else if (z.scalar_type() == torch::kFloat32) HELIX_CONV(float);
  else TORCH_CHECK(false, "conv_span: bf16 or fp32");
#undef HELIX_CONV
}
