// Linear attention with a constant decay per head over prompt portions: the
// operands of the chunk recurrence (gla_chunks), and the norm behind it.
//
// With a the head's decay and n the tokens of a chunk of up to 64:
//
//   qe_i = silu(q_i) a^(i+1)      ke_j = silu(k_j) a^(n-1-j)
//   A_ij = a^(i-j) silu(q_i) . silu(k_j)  for j <= i,     ec = a^n
//
// silu(q), silu(k), silu(v) are bf16, as single tokens store them; whatever
// has a decay in it leaves as two bf16 terms (17 bits).
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int NT = 256;
constexpr int L = 64;                         // tokens of a chunk
constexpr int SL = 32;                        // channels worked on at a time
constexpr int PB = SL + 8;                    // pitch, bf16 rows
constexpr int PS = SL + 1;                    // pitch, columns read

struct Operands {
  const float* log_decay;      // [H] base 2
  const int *row, *count;      // per chunk
  int64_t z_stride;
  int q_at, k_at, v_at, H, D, Dp, E, Pp, vec;
};

__device__ __forceinline__ float power(float log_decay, int n) {
  return __builtin_amdgcn_exp2f(log_decay * (float)n);
}

// silu of columns c0 .. c0 + 31 of the chunk's rows, 8 per thread; zero past
// column n or row count.
__device__ __forceinline__ u16x8 silu_slice(const uint16_t* z, int64_t stride,
                                            int c0, int n, int count,
                                            bool vec) {
  const int t = threadIdx.x / 4, d = c0 + threadIdx.x % 4 * 8;
  u16x8 raw = {0, 0, 0, 0, 0, 0, 0, 0};
  if (t < count) {
    const uint16_t* p = z + t * stride + d;
    if (vec) {
      if (d < n) raw = ld_u16x8(p);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (d + i < n) raw[i] = p[i];
    }
  }
  float v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = silu_s<uint16_t>(bf16_to_f32(raw[i]));
  return pack8(v);
}

// grid (chunks, heads)
__global__ __launch_bounds__(NT) void decay_operands_kernel(
    uint16_t* __restrict__ qe, uint16_t* __restrict__ ke,
    uint16_t* __restrict__ am, uint16_t* __restrict__ vt,
    float* __restrict__ ec, const uint16_t* __restrict__ z, Operands m) {
  __shared__ __attribute__((aligned(16))) uint16_t qb[L * PB], kb[L * PB];
  __shared__ float cols[L * PS];              // keys, later values
  const int n = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int count = m.count[n];
  const uint16_t* zr = z + (int64_t)m.row[n] * m.z_stride;
  const int64_t nh = (int64_t)n * m.H + h;
  uint16_t* qo = qe + nh * 2 * L * m.Dp;
  uint16_t* ko = ke + nh * 2 * L * m.Dp;
  const float la = m.log_decay[h];
  // the score blocks (I, J <= I) of this wave; heads start elsewhere, so
  // that the long rows do not all meet on one SIMD
  const int I = (wid + h) & 3;
  floatx4 acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = floatx4{0, 0, 0, 0};
  const uint16_t *zq = zr + m.q_at + h * m.D, *zk = zr + m.k_at + h * m.D;
  const uint16_t* zv = zr + m.v_at + h * m.E;
  const int t = tid / 4, s = tid % 4 * 8;     // as rows are loaded
  const int kd = tid / 8, kt = tid % 8 * 8;   // as columns are stored
  const float fq = power(la, t + 1);
  float fk[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) fk[i] = power(la, max(count - 1 - kt - i, 0));

  u16x8 q = silu_slice(zq, m.z_stride, 0, m.D, count, m.vec);
  u16x8 k = silu_slice(zk, m.z_stride, 0, m.D, count, m.vec);
  for (int d0 = 0; d0 < m.Dp; d0 += SL) {
    __syncthreads();                          // the last slice is done
    *reinterpret_cast<u16x8*>(qb + t * PB + s) = q;
    *reinterpret_cast<u16x8*>(kb + t * PB + s) = k;
    float v[8];
    u16x8 a, b;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      cols[t * PS + s + i] = bf16_to_f32(k[i]);
      v[i] = bf16_to_f32(q[i]) * fq;
    }
    split8(v, a, b);
    *reinterpret_cast<u16x8*>(qo + t * m.Dp + d0 + s) = a;
    *reinterpret_cast<u16x8*>(qo + (L + t) * m.Dp + d0 + s) = b;
    __syncthreads();
    if (d0 + SL < m.Dp) {
      q = silu_slice(zq, m.z_stride, d0 + SL, m.D, count, m.vec);
      k = silu_slice(zk, m.z_stride, d0 + SL, m.D, count, m.vec);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = cols[(kt + i) * PS + kd] * fk[i];
    split8(v, a, b);
    *reinterpret_cast<u16x8*>(ko + (d0 + kd) * L + kt) = a;
    *reinterpret_cast<u16x8*>(ko + (m.Dp + d0 + kd) * L + kt) = b;
    // scores: rows j of a block's result, columns i
    const u16x8 qf = ld_u16x8(qb + (I * 16 + lo) * PB + hi * 8);
#pragma unroll
    for (int J = 0; J < 4; ++J)
      if (J <= I)
        acc[J] = mfma16(ld_u16x8(kb + (J * 16 + lo) * PB + hi * 8), qf,
                        acc[J]);
  }
  if (tid < m.Dp) ec[nh * m.Dp + tid] = power(la, count);

  uint16_t* ao = am + nh * 2 * L * L + (I * 16 + lo) * L + hi * 4;
#pragma unroll
  for (int J = 0; J < 4; ++J) {
    float x[4], rest[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int back = (I - J) * 16 + lo - hi * 4 - r;
      x[r] = back >= 0 ? acc[J][r] * power(la, back) : 0.f;
      rest[r] = x[r] - bf16_to_f32(f32_to_bf16(x[r]));
    }
    st_bf16x4(ao + J * 16, x);
    st_bf16x4(ao + L * L + J * 16, rest);
  }
  // values, transposed
  u16x8 w = silu_slice(zv, m.z_stride, 0, m.E, count, m.vec);
  for (int e0 = 0; e0 < m.Pp; e0 += SL) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 8; ++i) cols[t * PS + s + i] = bf16_to_f32(w[i]);
    if (e0 + SL < m.Pp)
      w = silu_slice(zv, m.z_stride, e0 + SL, m.E, count, m.vec);
    __syncthreads();
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = cols[(kt + i) * PS + kd];
    if (e0 + kd < m.Pp)
      *reinterpret_cast<u16x8*>(vt + (nh * m.Pp + e0 + kd) * L + kt) =
          pack8(v);
  }
}

// y <- rms_norm(o) * w * sigmoid(g) over whole rows; a workgroup per row.
template <typename S, int N>
__global__ __launch_bounds__(NT) void row_norm_gate_kernel(
    S* __restrict__ y, const S* __restrict__ o, const S* __restrict__ g,
    const float* __restrict__ w, int64_t y_stride, int64_t o_stride,
    int64_t g_stride, int n, float eps) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const S *po = o + t * o_stride, *pg = g + t * g_stride;
  S* py = y + t * y_stride;
  float ss = 0.f;
  for (int i = threadIdx.x * N; i < n; i += NT * N) {
    float v[N];
    if constexpr (N == 1) v[0] = ld1(po + i); else ldv<N>(po + i, v);
#pragma unroll
    for (int j = 0; j < N; ++j) ss += v[j] * v[j];
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / n + eps);
  for (int i = threadIdx.x * N; i < n; i += NT * N) {
    if constexpr (N == 1) {
      st1(py + i, ld1(po + i) * inv * w[i] * sigmoid_s<S>(ld1(pg + i)));
    } else {
      float v[N], c[N], x[N];
      ldv<N>(po + i, v);
      ldv<N>(w + i, c);
      ldv<N>(pg + i, x);
#pragma unroll
      for (int j = 0; j < N; ++j) v[j] *= inv * c[j] * sigmoid_s<S>(x[j]);
      stv<N>(py + i, v);
    }
  }
}

void check(const torch::Tensor& t, torch::ScalarType type, int64_t n) {
  TORCH_CHECK(t.scalar_type() == type && t.is_contiguous() && t.numel() == n,
              "decay chunks: operand of ", t.numel(), " values, want ", n);
}

template <typename S>
void launch_norm(torch::Tensor y, torch::Tensor o, torch::Tensor g,
                 torch::Tensor w, double eps, bool vec) {
  auto stream = at::hip::getCurrentHIPStream();
#define HELIX_RN(N)                                                          \
  hipLaunchKernelGGL((row_norm_gate_kernel<S, N>), dim3(o.size(0)),          \
                     dim3(NT), 0, stream, (S*)y.data_ptr(),                  \
                     (const S*)o.data_ptr(), (const S*)g.data_ptr(),         \
                     w.data_ptr<float>(), y.stride(0), o.stride(0),          \
                     g.stride(0), (int)o.size(1), (float)eps)
  if (vec) HELIX_RN(8);
  else HELIX_RN(1);
#undef HELIX_RN
}

}  // namespace

void decay_operands(torch::Tensor qe, torch::Tensor ke, torch::Tensor am,
                    torch::Tensor vt, torch::Tensor ec, torch::Tensor z,
                    int64_t q_at, int64_t k_at, int64_t v_at, int64_t dim,
                    int64_t vdim, torch::Tensor log_decay, torch::Tensor row,
                    torch::Tensor count) {
  TORCH_CHECK(qe.dim() == 5 && vt.dim() == 4);
  const int64_t n = qe.size(0);
  Operands m{};
  m.H = qe.size(1);
  m.D = dim;
  m.Dp = qe.size(4);
  m.E = vdim;
  m.Pp = vt.size(2);
  TORCH_CHECK(m.D > 0 && m.D <= m.Dp && m.Dp % 32 == 0 && m.Dp <= 256 &&
              m.E > 0 && m.E <= m.Pp && m.Pp % 16 == 0);
  const int64_t nh = n * m.H;
  check(qe, torch::kBFloat16, nh * 2 * L * m.Dp);
  check(ke, torch::kBFloat16, nh * 2 * L * m.Dp);
  check(am, torch::kBFloat16, nh * 2 * L * L);
  check(vt, torch::kBFloat16, nh * m.Pp * L);
  check(ec, torch::kFloat32, nh * m.Dp);
  check(log_decay, torch::kFloat32, m.H);
  check(row, torch::kInt32, n);
  check(count, torch::kInt32, n);
  TORCH_CHECK(z.scalar_type() == torch::kBFloat16 && z.stride(1) == 1);
  const int64_t width = z.size(1);
  TORCH_CHECK(q_at + m.H * m.D <= width && k_at + m.H * m.D <= width &&
              v_at + m.H * m.E <= width);
  m.log_decay = log_decay.data_ptr<float>();
  m.row = row.data_ptr<int>();
  m.count = count.data_ptr<int>();
  m.z_stride = z.stride(0);
  m.q_at = q_at;
  m.k_at = k_at;
  m.v_at = v_at;
  m.vec = m.D % 8 == 0 && m.E % 8 == 0 && q_at % 8 == 0 && k_at % 8 == 0 &&
          v_at % 8 == 0 && m.z_stride % 8 == 0 &&
          (uintptr_t)z.data_ptr() % 16 == 0;
  if (n == 0) return;
  hipLaunchKernelGGL(decay_operands_kernel, dim3(n, m.H), dim3(NT), 0,
                     at::hip::getCurrentHIPStream(), (uint16_t*)qe.data_ptr(),
                     (uint16_t*)ke.data_ptr(), (uint16_t*)am.data_ptr(),
                     (uint16_t*)vt.data_ptr(), ec.data_ptr<float>(),
                     (const uint16_t*)z.data_ptr(), m);
}

void row_norm_gate(torch::Tensor y, torch::Tensor o, torch::Tensor g,
                   torch::Tensor w, double eps) {
  TORCH_CHECK(o.dim() == 2);
  const int64_t T = o.size(0), n = o.size(1);
  check(w, torch::kFloat32, n);
  bool vec = n % 8 == 0;
  for (const auto& t : {y, o, g}) {
    TORCH_CHECK(t.scalar_type() == o.scalar_type() && t.size(0) == T &&
                t.size(1) == n && t.stride(1) == 1);
    vec = vec && t.stride(0) % 8 == 0 && (uintptr_t)t.data_ptr() % 16 == 0;
  }
  if (T == 0 || n == 0) return;
  if (o.scalar_type() == torch::kBFloat16)
    launch_norm<uint16_t>(y, o, g, w, eps, vec);
  else if (o.scalar_type() == torch::kFloat32)
    launch_norm<float>(y, o, g, w, eps, vec);
  else
    TORCH_CHECK(false, "row_norm_gate: bf16 or fp32");
}
