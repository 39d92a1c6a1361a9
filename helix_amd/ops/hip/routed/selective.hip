// Selective scan (Mamba-1): a linear recurrence per channel c and state n
//
//   dt = softplus(raw + bias)
//   S[n] <- exp(dt A[n]) S[n] + dt x B[n];   y = sum_n S[n] C[n] + D x
//
// whose decays differ per channel, state and token, so there is no product
// form: a lane has a channel and keeps its states in registers. The result
// leaves as y silu(z). The causal convolution ahead of it is a launch of its
// own, since projections of its result come in between.
//
// State is [slots, N, C]: neighbouring lanes have neighbouring channels, B
// and C of a token are the same for all of them and come by scalar loads. A
// is kept as [N, C] times log2(e).
//
// Prompts: one wave per 64 channels and sequence where that fills the chip.
// Where it does not, sequences are cut into chunks: every chunk's scan from
// zero, then the chunks' entry states one after the other, then the scan
// from those.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float exp2_(float x) {
  return __builtin_amdgcn_exp2f(x);
}

// log(1 + e^x) to a few units in the last place: small exponentials by the
// series of log(1 + e).
template <typename S>
__device__ __forceinline__ float softplus_of(float x) {
  const float e = exp2_(-fabsf(x) * LOG2E);
  const float small =
      e * (1.f - e * (0.5f - e * (0.33333333f - e * (0.25f - e * 0.2f))));
  const float big = __builtin_amdgcn_logf(1.f + e) * 0.6931471805599453f;
  return fmaxf(x, 0.f) + (e < 0.03125f ? small : big);
}
template <>
__device__ __forceinline__ float softplus_of<float>(float x) {
  return softplus(x);
}

template <int N>
__device__ __forceinline__ void ldf(const float* p, float* v) {
  if constexpr (N == 1) v[0] = *p; else ldv<N>(p, v);
}
template <typename S, int N>
__device__ __forceinline__ void get(const S* p, float* v) {
  if constexpr (N == 1) v[0] = ld1(p); else ldv<N>(p, v);
}
template <typename S, int N>
__device__ __forceinline__ void put(S* p, const float* v) {
  if constexpr (N == 1) st1(p, v[0]); else stv<N>(p, v);
}

// ---------------------------------------------------------------- convolution

// Ring entry pos % taps holds the raw inputs of position pos. A thread has N
// channels of a block of tokens; the first block of a sequence reads the
// ring and, being the only one that does, refills it.
constexpr int CT = 256, SPAN = 32;

template <typename S, int N, int TAPS>
__global__ __launch_bounds__(CT) void conv_silu_kernel(
    S* __restrict__ out, const S* __restrict__ z, int64_t z_stride, int x_at,
    const float* __restrict__ conv, const float* __restrict__ bias, S* ring,
    const int* __restrict__ slots, const int64_t* __restrict__ pos,
    const int* __restrict__ cu, int taps_, int C) {
  const int taps = TAPS ? TAPS : taps_;
  const int b = blockIdx.y, c = (blockIdx.x * CT + threadIdx.x) * N;
  const int row0 = cu ? cu[b] : b, len = cu ? cu[b + 1] - row0 : 1;
  const int t0 = blockIdx.z * SPAN;
  if (c >= C || t0 >= len) return;
  const int slot = slots[b];
  const int64_t p0 = pos[row0];
  S* rs = ring + (int64_t)max(slot, 0) * taps * C + c;
  const S* zc = z + (int64_t)row0 * z_stride + x_at + c;
  // taps are stored [taps][C]
  const float* w = conv + c;
  float bv[N];
  ldf<N>(bias + c, bv);
  // raw inputs of token t (before the portion: what the ring holds)
  auto input = [&](int t, float* v) {
#pragma unroll
    for (int j = 0; j < N; ++j) v[j] = 0.f;
    if (t >= 0)
      get<S, N>(zc + (int64_t)t * z_stride, v);
    else if (slot >= 0 && p0 + t >= 0)
      get<S, N>(rs + (p0 + t) % taps * C, v);
  };
  if constexpr (TAPS > 0) {
    float wv[TAPS][N], win[TAPS][N];
#pragma unroll
    for (int k = 0; k < TAPS; ++k) ldf<N>(w + (int64_t)k * C, wv[k]);
#pragma unroll
    for (int k = 0; k < TAPS - 1; ++k) input(t0 - TAPS + 1 + k, win[k]);
    const int t1 = min(len, t0 + SPAN);
    for (int t = t0; t < t1; ++t) {
      get<S, N>(zc + (int64_t)t * z_stride, win[TAPS - 1]);
      float a[N];
#pragma unroll
      for (int j = 0; j < N; ++j) a[j] = bv[j];
#pragma unroll
      for (int k = 0; k < TAPS; ++k)
#pragma unroll
        for (int j = 0; j < N; ++j) a[j] += wv[k][j] * win[k][j];
#pragma unroll
      for (int k = 0; k < TAPS - 1; ++k)
#pragma unroll
        for (int j = 0; j < N; ++j) win[k][j] = win[k + 1][j];
#pragma unroll
      for (int j = 0; j < N; ++j) a[j] = silu_s<S>(a[j]);
      put<S, N>(out + (int64_t)(row0 + t) * C + c, a);
    }
  } else {
    for (int t = t0; t < min(len, t0 + SPAN); ++t) {
      float a[N];
#pragma unroll
      for (int j = 0; j < N; ++j) a[j] = bv[j];
      for (int k = 0; k < taps; ++k) {
        float v[N], g[N];
        input(t - taps + 1 + k, v);
        ldf<N>(w + (int64_t)k * C, g);
#pragma unroll
        for (int j = 0; j < N; ++j) a[j] += g[j] * v[j];
      }
#pragma unroll
      for (int j = 0; j < N; ++j) a[j] = silu_s<S>(a[j]);
      put<S, N>(out + (int64_t)(row0 + t) * C + c, a);
    }
  }
  // tokens past the first block are at least SPAN >= taps - 1 in
  if (t0 == 0 && slot >= 0)
    for (int t = max(0, len - taps); t < len; ++t) {
      float v[N];
      get<S, N>(zc + (int64_t)t * z_stride, v);
      put<S, N>(rs + (p0 + t) % taps * C, v);
    }
}

// ----------------------------------------------------------------------- scan

struct Scan {
  const float *dt, *bias;      // [T, C] raw step sizes, [C]
  const float *bc, *A, *D;     // [T, ..] rows with B and C; [N, C]; [C]
  float* state;                // [slots, N, C]
  const int* slots;
  const int64_t* pos;
  const int* cu;               // [B + 1]
  // chunks
  const int *row, *count;      // per chunk
  const int* first;            // [B + 1] chunks of a sequence
  float *entry, *sums;         // [chunks, N, C], [chunks, C]
  int64_t z_stride, y_stride, bc_stride;
  int z_at, b_at, c_at, C, N;
};

// Single tokens: a thread has V channels and walks over their states.
template <typename S, int V>
__global__ __launch_bounds__(CT) void scan_step_kernel(
    S* __restrict__ y, const S* __restrict__ x, const S* __restrict__ z,
    Scan m) {
  const int b = blockIdx.y, c = (blockIdx.x * CT + threadIdx.x) * V;
  if (c >= m.C) return;
  const int slot = m.slots[b];
  float* st = m.state + (int64_t)max(slot, 0) * m.N * m.C + c;
  const bool carried = slot >= 0 && m.pos[b] > 0;
  const float *B = m.bc + b * m.bc_stride + m.b_at,
              *Cc = m.bc + b * m.bc_stride + m.c_at;
  float xv[V], dt[V], u[V], acc[V], g[V];
  get<S, V>(x + (int64_t)b * m.C + c, xv);
  ldf<V>(m.dt + (int64_t)b * m.C + c, dt);
  ldf<V>(m.bias + c, u);
  ldf<V>(m.D + c, acc);
#pragma unroll
  for (int j = 0; j < V; ++j) {
    dt[j] = softplus_of<S>(dt[j] + u[j]);
    u[j] = dt[j] * xv[j];
    acc[j] *= xv[j];
  }
#pragma unroll 4
  for (int n = 0; n < m.N; ++n) {
    float s[V], a[V];
#pragma unroll
    for (int j = 0; j < V; ++j) s[j] = 0.f;
    if (carried) ldf<V>(st + (int64_t)n * m.C, s);
    ldf<V>(m.A + (int64_t)n * m.C + c, a);
    const float bn = B[n], cn = Cc[n];
#pragma unroll
    for (int j = 0; j < V; ++j) {
      s[j] = exp2_(dt[j] * a[j]) * s[j] + u[j] * bn;
      acc[j] += s[j] * cn;
    }
    if (slot >= 0) put<float, V>(st + (int64_t)n * m.C, s);
  }
  get<S, V>(z + b * m.z_stride + m.z_at + c, g);
#pragma unroll
  for (int j = 0; j < V; ++j) acc[j] *= silu_s<S>(g[j]);
  put<S, V>(y + b * m.y_stride + c, acc);
}

constexpr int ST = 64;                        // channels of a workgroup
constexpr int TT = 4;                         // tokens loaded at a time
typedef const __attribute__((address_space(4))) float* uniform_f32;

enum Pass { WHOLE, LOCAL, FINAL };

// NS: states in registers (N <= NS; B and C are zero from N to NS). WHOLE: sequences from their slots'
// state and back. LOCAL: chunks from zero, only the state they end with.
// FINAL: chunks from their entry state, only results.
template <typename S, int NS, int PASS>
__global__ __launch_bounds__(ST) void scan_kernel(
    S* __restrict__ y, const S* __restrict__ x, const S* __restrict__ z,
    Scan m) {
  const int u = blockIdx.y, lane = threadIdx.x;
  const int c0 = blockIdx.x * ST, c = min(c0 + lane, m.C - 1);
  const bool mine = c0 + lane < m.C;
  int row0, len, slot = -1;
  bool carried = false;
  if constexpr (PASS == WHOLE) {
    row0 = m.cu[u];
    len = m.cu[u + 1] - row0;
    if (len <= 0) return;
    slot = m.slots[u];
    carried = slot >= 0 && m.pos[row0] > 0;
  } else {
    row0 = m.row[u];
    len = m.count[u];
  }
  float* st = PASS == WHOLE
                  ? m.state + (int64_t)max(slot, 0) * m.N * m.C + c
                  : m.entry + (int64_t)u * m.N * m.C + c;
  float s[NS], a[NS], total = 0.f;
#pragma unroll
  for (int n = 0; n < NS; ++n) {
    const int64_t at = (int64_t)min(n, m.N - 1) * m.C;
    a[n] = m.A[at + c];
    s[n] = n < m.N && (PASS == FINAL || carried) ? st[at] : 0.f;
  }
  const float bias = m.bias[c], D = m.D[c];
  const S* xp = x + (int64_t)row0 * m.C + c;
  const float* dp = m.dt + (int64_t)row0 * m.C + c;
  const S* zp = z + row0 * m.z_stride + m.z_at + c;
  S* yp = PASS == LOCAL ? nullptr : y + row0 * m.y_stride + c;

  float dr[TT];
  S xr[TT], zr[TT];
  auto load = [&](int t) {
#pragma unroll
    for (int i = 0; i < TT; ++i) {
      const int64_t r = min(t + i, len - 1);
      xr[i] = xp[r * m.C];
      dr[i] = dp[r * m.C];
      if constexpr (PASS != LOCAL) zr[i] = zp[r * m.z_stride];
    }
  };
  // uniform: scalar registers
  constexpr bool AHEAD = NS <= 16;
  float b[NS], c_[NS], nb[NS], nc[NS];
  auto fetch = [&](int t, float* bn, float* cn) {
    const uniform_f32 r = (uniform_f32)(uintptr_t)(
        m.bc + (int64_t)(row0 + min(t, len - 1)) * m.bc_stride);
#pragma unroll
    for (int n = 0; n < NS; ++n) {
      bn[n] = r[m.b_at + n];
      if constexpr (PASS != LOCAL) cn[n] = r[m.c_at + n];
    }
  };
  load(0);
  if constexpr (AHEAD) fetch(0, b, c_);
  for (int t = 0; t < len; t += TT) {
    float xv[TT], dv[TT], zv[TT];
#pragma unroll
    for (int i = 0; i < TT; ++i) {
      // past the end: a step of size zero changes nothing
      dv[i] = t + i < len ? softplus_of<S>(dr[i] + bias) : 0.f;
      xv[i] = ld1(&xr[i]);
      if constexpr (PASS != LOCAL) zv[i] = ld1(&zr[i]);
    }
    if (t + TT < len) load(t + TT);
#pragma unroll
    for (int i = 0; i < TT; ++i) {
      if constexpr (AHEAD) {
        // a token's B and C are on their way while the one before it is
        // worked on; nothing moves across the fences
        fetch(t + i + 1, nb, nc);
        __builtin_amdgcn_sched_barrier(0);
      } else {
        fetch(t + i, b, c_);
      }
      const float w = dv[i] * xv[i];
      if constexpr (PASS == LOCAL) total += dv[i];
      float acc[4] = {D * xv[i], 0.f, 0.f, 0.f};
#pragma unroll
      for (int n = 0; n < NS; ++n) {
        s[n] = exp2_(dv[i] * a[n]) * s[n] + w * b[n];
        if constexpr (PASS != LOCAL) acc[n & 3] += s[n] * c_[n];
      }
      if constexpr (PASS != LOCAL) {
        const float o = (acc[0] + acc[1]) + (acc[2] + acc[3]);
        if (mine && t + i < len)
          st1(yp + (int64_t)(t + i) * m.y_stride, o * silu_s<S>(zv[i]));
      }
      if constexpr (AHEAD) {
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int n = 0; n < NS; ++n) {
          b[n] = nb[n];
          c_[n] = nc[n];
        }
      }
    }
  }
  if constexpr (PASS != FINAL) {
    if (mine && (PASS == LOCAL || slot >= 0))
#pragma unroll
      for (int n = 0; n < NS; ++n)
        if (n < m.N) st[(int64_t)n * m.C] = s[n];
  }
  if constexpr (PASS == LOCAL)
    if (mine) m.sums[(int64_t)u * m.C + c] = total;
}

// The chunks' ends become their entry states; the last end goes to the slot.
__global__ __launch_bounds__(CT) void scan_carry_kernel(Scan m) {
  const int c = blockIdx.x * CT + threadIdx.x, n = blockIdx.y, b = blockIdx.z;
  if (c >= m.C) return;
  const int slot = m.slots[b], n0 = m.first[b], n1 = m.first[b + 1];
  if (n0 >= n1) return;
  float* st = m.state + ((int64_t)max(slot, 0) * m.N + n) * m.C + c;
  const bool carried = slot >= 0 && m.pos[m.cu[b]] > 0;
  const float a = m.A[(int64_t)n * m.C + c];
  float s = carried ? *st : 0.f;
  for (int k = n0; k < n1; ++k) {
    float* e = m.entry + ((int64_t)k * m.N + n) * m.C + c;
    const float end = *e;
    *e = s;
    s = exp2_(a * m.sums[(int64_t)k * m.C + c]) * s + end;
  }
  if (slot >= 0) *st = s;
}

const float* f32(const torch::Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kFloat32 &&
                  t.is_contiguous() && t.numel() == n,
              what);
  return t.data_ptr<float>();
}

void check_rows(const torch::Tensor& slots, const torch::Tensor& pos,
                int64_t B, int64_t T) {
  TORCH_CHECK(slots.scalar_type() == torch::kInt32 && slots.numel() == B &&
              slots.is_contiguous());
  TORCH_CHECK(pos.scalar_type() == torch::kInt64 && pos.numel() == T &&
              pos.is_contiguous());
}

const int* i32(const torch::Tensor& t, int64_t n) {
  TORCH_CHECK(t.scalar_type() == torch::kInt32 && t.is_contiguous() &&
              t.numel() == n);
  return t.data_ptr<int>();
}

Scan arguments(const torch::Tensor& y, const torch::Tensor& x,
               const torch::Tensor& z, int64_t z_at, const torch::Tensor& dt,
               const torch::Tensor& bias, const torch::Tensor& bc,
               int64_t b_at, int64_t c_at, const torch::Tensor& A,
               const torch::Tensor& D, const torch::Tensor& state) {
  Scan m{};
  TORCH_CHECK(state.dim() == 3 && x.dim() == 2 && z.dim() == 2 &&
              y.dim() == 2 && bc.dim() == 2);
  m.N = state.size(1);
  m.C = state.size(2);
  const int64_t T = x.size(0);
  TORCH_CHECK(x.is_contiguous() && x.size(1) == m.C);
  TORCH_CHECK(z.size(0) == T && z.stride(1) == 1 && z_at >= 0 &&
              z_at + m.C <= z.size(1) && y.size(0) == T &&
              y.size(1) == m.C && y.stride(1) == 1);
  TORCH_CHECK(x.scalar_type() == z.scalar_type() &&
              x.scalar_type() == y.scalar_type());
  TORCH_CHECK(bc.size(0) == T && bc.stride(1) == 1 &&
              bc.scalar_type() == torch::kFloat32 && b_at >= 0 &&
              b_at + m.N <= bc.size(1) && c_at >= 0 &&
              c_at + m.N <= bc.size(1));
  m.dt = f32(dt, T * m.C, "step sizes");
  m.bias = f32(bias, m.C, "bias of the step sizes");
  m.A = f32(A, (int64_t)m.N * m.C, "A");
  m.D = f32(D, m.C, "D");
  m.state = (float*)f32(state, state.numel(), "state");
  m.bc = bc.data_ptr<float>();
  m.bc_stride = bc.stride(0);
  m.z_stride = z.stride(0);
  m.y_stride = y.stride(0);
  m.z_at = z_at;
  m.b_at = b_at;
  m.c_at = c_at;
  return m;
}

// Columns that B and C take in a row.
int columns_of(int N) {
  int n = 8;
  while (n < N) n *= 2;
  return n;
}

template <int PASS>
void launch_scan(torch::Tensor y, torch::Tensor x, torch::Tensor z, Scan m,
                 int units) {
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(cdiv(m.C, ST), units);
#define HELIX_SCAN_S(S, NS)                                                  \
  hipLaunchKernelGGL((scan_kernel<S, NS, PASS>), grid, dim3(ST), 0, stream,  \
                     (S*)y.data_ptr(), (const S*)x.data_ptr(),               \
                     (const S*)z.data_ptr(), m)
#define HELIX_SCAN(NS)                                                       \
  do {                                                                       \
    if (x.scalar_type() == torch::kBFloat16) HELIX_SCAN_S(uint16_t, NS);     \
    else HELIX_SCAN_S(float, NS);                                            \
  } while (0)
  if (m.N <= 8) HELIX_SCAN(8);
  else if (m.N <= 16) HELIX_SCAN(16);
  else if (m.N <= 32) HELIX_SCAN(32);
  else if (m.N <= 64) HELIX_SCAN(64);
  else HELIX_SCAN(128);
#undef HELIX_SCAN
#undef HELIX_SCAN_S
}

}  // namespace

// Most states per channel, and the columns that N take in B's and C's rows
// (zero from N on).
int64_t scan_max_state() { return 128; }
int64_t scan_columns(int64_t N) { return columns_of(N); }

// out [T, C] <- silu of the causal convolution of z's columns x_at ..; conv
// [taps, C]. z rows: one token of sequence r each, or (with cu) the
// concatenated tokens of cu.numel() - 1 sequences.
void conv_silu(torch::Tensor out, torch::Tensor z, int64_t x_at,
               torch::Tensor conv, torch::Tensor bias, torch::Tensor ring,
               torch::Tensor slots, torch::Tensor pos, OptT cu,
               int64_t max_len) {
  TORCH_CHECK(ring.dim() == 3 && ring.is_contiguous() && z.dim() == 2);
  const int taps = ring.size(1), C = ring.size(2);
  const int64_t T = z.size(0);
  const int B = cu.has_value() ? cu->numel() - 1 : T;
  TORCH_CHECK(out.is_contiguous() && out.size(0) == T && out.size(1) == C &&
              z.stride(1) == 1 && x_at >= 0 && x_at + C <= z.size(1));
  TORCH_CHECK(out.scalar_type() == z.scalar_type() &&
              ring.scalar_type() == z.scalar_type());
  TORCH_CHECK(taps >= 1 && taps - 1 <= SPAN, "at most ", SPAN + 1, " taps");
  f32(conv, (int64_t)C * taps, "taps");
  f32(bias, C, "bias");
  check_rows(slots, pos, B, T);
  const int* cup = cu.has_value() ? i32(*cu, B + 1) : nullptr;
  if (B == 0 || T == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const bool vec = C % 4 == 0 && x_at % 4 == 0 && z.stride(0) % 4 == 0 &&
                   (uintptr_t)z.data_ptr() % 16 == 0;
  const dim3 grid(cdiv(C, CT * (vec ? 4 : 1)), B,
                  cu.has_value() ? cdiv((int)max_len, SPAN) : 1);
#define HELIX_CONV(S, N, TAPS)                                               \
  hipLaunchKernelGGL((conv_silu_kernel<S, N, TAPS>), grid, dim3(CT), 0,      \
                     stream, (S*)out.data_ptr(), (const S*)z.data_ptr(),     \
                     z.stride(0), (int)x_at, conv.data_ptr<float>(),         \
                     bias.data_ptr<float>(), (S*)ring.data_ptr(),            \
                     slots.data_ptr<int>(), pos.data_ptr<int64_t>(), cup,    \
                     taps, C)
#define HELIX_CONV_T(S, N)                                                   \
  do {                                                                       \
    if (taps == 4) HELIX_CONV(S, N, 4);                                      \
    else HELIX_CONV(S, N, 0);                                                \
  } while (0)
  if (z.scalar_type() == torch::kBFloat16) {
    if (vec) HELIX_CONV_T(uint16_t, 4);
    else HELIX_CONV_T(uint16_t, 1);
  } else {
    TORCH_CHECK(z.scalar_type() == torch::kFloat32, "conv_silu: bf16 or fp32");
    if (vec) HELIX_CONV_T(float, 4);
    else HELIX_CONV_T(float, 1);
  }
#undef HELIX_CONV_T
#undef HELIX_CONV
}

void scan_step(torch::Tensor y, torch::Tensor x, torch::Tensor z,
               int64_t z_at, torch::Tensor dt, torch::Tensor bias,
               torch::Tensor bc, int64_t b_at, int64_t c_at, torch::Tensor A,
               torch::Tensor D, torch::Tensor state, torch::Tensor slots,
               torch::Tensor pos) {
  Scan m = arguments(y, x, z, z_at, dt, bias, bc, b_at, c_at, A, D, state);
  const int B = x.size(0);
  check_rows(slots, pos, B, B);
  m.slots = slots.data_ptr<int>();
  m.pos = pos.data_ptr<int64_t>();
  if (B == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  bool vec = m.C % 4 == 0 && z_at % 4 == 0 && m.z_stride % 4 == 0 &&
             m.y_stride % 4 == 0;
  for (const auto& t : {y, x, z, dt, state})
    vec = vec && (uintptr_t)t.data_ptr() % 16 == 0;
  // few rows: a channel to a thread, more waves
  if ((int64_t)B * m.C < 256 * 1024) vec = false;
  const dim3 grid(cdiv(m.C, CT * (vec ? 4 : 1)), B);
#define HELIX_STEP(S, V)                                                     \
  hipLaunchKernelGGL((scan_step_kernel<S, V>), grid, dim3(CT), 0, stream,    \
                     (S*)y.data_ptr(), (const S*)x.data_ptr(),               \
                     (const S*)z.data_ptr(), m)
  if (x.scalar_type() == torch::kBFloat16) {
    if (vec) HELIX_STEP(uint16_t, 4);
    else HELIX_STEP(uint16_t, 1);
  } else {
    TORCH_CHECK(x.scalar_type() == torch::kFloat32, "scan: bf16 or fp32");
    if (vec) HELIX_STEP(float, 4);
    else HELIX_STEP(float, 1);
  }
#undef HELIX_STEP
}

// Prompt portions; with row .. sums in chunks (entry [chunks, N, C], sums
// [chunks, C] are scratch).
void scan_prompt(torch::Tensor y, torch::Tensor x, torch::Tensor z,
                 int64_t z_at, torch::Tensor dt, torch::Tensor bias,
                 torch::Tensor bc, int64_t b_at, int64_t c_at,
                 torch::Tensor A, torch::Tensor D, torch::Tensor state,
                 torch::Tensor slots, torch::Tensor pos, torch::Tensor cu,
                 OptT row, OptT count, OptT first, OptT entry, OptT sums) {
  Scan m = arguments(y, x, z, z_at, dt, bias, bc, b_at, c_at, A, D, state);
  const int B = slots.numel();
  check_rows(slots, pos, B, x.size(0));
  TORCH_CHECK(m.N <= scan_max_state(), "state size ", m.N);
  const int64_t cols = columns_of(m.N);
  TORCH_CHECK(b_at + cols <= bc.size(1) && c_at + cols <= bc.size(1) &&
                  std::abs(b_at - c_at) >= cols,
              "B and C take ", cols, " columns each");
  TORCH_CHECK(x.scalar_type() == torch::kBFloat16 ||
              x.scalar_type() == torch::kFloat32);
  m.slots = slots.data_ptr<int>();
  m.pos = pos.data_ptr<int64_t>();
  m.cu = i32(cu, B + 1);
  if (B == 0 || x.size(0) == 0) return;
  if (!row.has_value()) {
    launch_scan<WHOLE>(y, x, z, m, B);
    return;
  }
  TORCH_CHECK(count.has_value() && first.has_value() && entry.has_value() &&
              sums.has_value());
  const int n = row->numel();
  m.row = i32(*row, n);
  m.count = i32(*count, n);
  m.first = i32(*first, B + 1);
  m.entry = (float*)f32(*entry, (int64_t)n * m.N * m.C, "entry states");
  m.sums = (float*)f32(*sums, (int64_t)n * m.C, "sums of step sizes");
  if (n == 0) return;
  launch_scan<LOCAL>(y, x, z, m, n);
  hipLaunchKernelGGL(scan_carry_kernel, dim3(cdiv(m.C, CT), m.N, B), dim3(CT),
                     0, at::hip::getCurrentHIPStream(), m);
  launch_scan<FINAL>(y, x, z, m, n);
}
