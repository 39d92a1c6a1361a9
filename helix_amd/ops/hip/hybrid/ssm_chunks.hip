// Mamba-2 mixer over prompt portions, 64 tokens at a time on MFMA.
//
// With a_t = -exp(A_log) dt_t summed from the chunk's start to A_t, and S the
// state that enters the chunk:
//
//   y_i = e^(A_i) S^T C_i + sum_{j<=i} e^(A_i - A_j) dt_j (C_i . B_j) x_j
//   S  <- e^(A_63) S + sum_j e^(A_63 - A_j) dt_j B_j x_j^T
//
// conv_chunks makes the chunk's operands: convolution, silu, x and B also
// transposed, step sizes and their sums. ssm_chunks carries a head's state
// from chunk to chunk in fp32 registers. B, C and x enter the products as
// the bf16 they are; whatever has a decay or the state in it (S, the score
// matrix, the weighted x) enters as two bf16 terms, 17 significant bits.
//
// Layouts per chunk: xt [H, Pp, 64], b and c [64, G, Np], bt [G, Np, 64],
// da [H, 2, 64] (A_t and dt_t). Tokens past a portion's end and state
// columns past N are zero.
#include "tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr int NT = 256;
constexpr int L = 64;                         // tokens of a chunk
constexpr int LP = L + 8;

struct Conv {
  const float *conv, *conv_b, *dt_bias, *A_log;
  const int* slots;
  const int64_t* pos;
  const int* cu;
  const int* seq;              // per chunk
  const int* row;
  const int* count;
  int64_t z_stride;
  int xbc_at, dt_at, H, P, Pp, N, Np, G, taps, C;
};

// grid (chunks, channel blocks of 64 + blocks of 4 heads for da)
__global__ __launch_bounds__(NT) void conv_chunks_kernel(
    uint16_t* __restrict__ xt, uint16_t* __restrict__ b,
    uint16_t* __restrict__ bt, uint16_t* __restrict__ c,
    float* __restrict__ da, const uint16_t* __restrict__ z, uint16_t* ring,
    Conv m) {
  extern __shared__ __attribute__((aligned(16))) float sh[];
  const int n = blockIdx.x, tid = threadIdx.x;
  const int row = m.row[n], count = m.count[n], sq = m.seq[n];
  const int pb = cdiv(m.P, 64), nb = cdiv(m.Np, 64);
  int y = blockIdx.y;

  if (y >= m.H * pb + 2 * m.G * nb) {         // a wave per head
    const int h = (y - m.H * pb - 2 * m.G * nb) * 4 + tid / WAVE;
    const int t = tid & (WAVE - 1);
    if (h >= m.H) return;
    float dt = 0.f;
    if (t < count)
      dt = softplus(
          bf16_to_f32(z[(row + t) * m.z_stride + m.dt_at + h]) +
          m.dt_bias[h]);
    float a = -expf(m.A_log[h]) * dt;
#pragma unroll
    for (int off = 1; off < WAVE; off *= 2) {
      const float up = __shfl_up(a, off, WAVE);
      if (t >= off) a += up;
    }
    float* o = da + ((int64_t)n * m.H + h) * 2 * L;
    o[t] = a;
    o[L + t] = dt;
    return;
  }

  // which 64 channels, and where they go
  int kind = 0, unit, part, c0, nc;
  if (y < m.H * pb) {
    unit = y / pb;
    part = y % pb * 64;
    c0 = unit * m.P + part;
    nc = min(64, m.P - part);
  } else {
    y -= m.H * pb;
    kind = 1 + y / (m.G * nb);
    unit = y % (m.G * nb) / nb;
    part = y % nb * 64;
    c0 = m.H * m.P + ((kind - 1) * m.G + unit) * m.N + part;
    nc = min(64, m.N - part);                 // may be none: padding
  }
  const int before = m.taps - 1, rows = L + before;
  constexpr int IP = 65;
  float* in = sh;                             // [rows][IP]
  uint16_t* ol = (uint16_t*)(sh + ((rows * IP + 3) & ~3));   // [L][LP]
  const int seq0 = m.cu[sq], slot = m.slots[sq];
  const int64_t p0 = m.pos[row];
  uint16_t* rs = ring + (int64_t)max(slot, 0) * m.taps * m.C + c0;
  for (int i = tid; i < rows * 64; i += NT) {
    const int r = i / 64, ch = i % 64, t = r - before;
    float v = 0.f;
    if (ch < nc && t < count) {
      if (row + t >= seq0)
        v = bf16_to_f32(z[(row + t) * m.z_stride + m.xbc_at + c0 + ch]);
      else if (slot >= 0 && p0 + t >= 0)
        v = bf16_to_f32(rs[(p0 + t) % m.taps * m.C + ch]);
    }
    in[r * IP + ch] = v;
  }
  __syncthreads();
  // The first chunk is the only reader of the ring; it also refills it with
  // the portion's last inputs.
  if (row == seq0 && slot >= 0) {
    const int len = m.cu[sq + 1] - seq0, k = min(m.taps, len);
    for (int i = tid; i < k * 64; i += NT) {
      const int t = len - k + i / 64, ch = i % 64;
      if (ch < nc)
        rs[(p0 + t) % m.taps * m.C + ch] =
            z[(int64_t)(seq0 + t) * m.z_stride + m.xbc_at + c0 + ch];
    }
  }
  const int ch = tid >> 2, t0 = (tid & 3) * 16;
  float acc[16];
  const bool live = ch < nc;
  const float bias = live ? m.conv_b[c0 + ch] : 0.f;
#pragma unroll
  for (int i = 0; i < 16; ++i) acc[i] = bias;
  for (int k = 0; k < m.taps; ++k) {
    const float w = live ? m.conv[(int64_t)(c0 + ch) * m.taps + k] : 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] += w * in[(t0 + i + k) * IP + ch];
  }
#pragma unroll
  for (int i = 0; i < 16; ++i)
    acc[i] = live && t0 + i < count ? silu_s<uint16_t>(acc[i]) : 0.f;

  const u16x8 lo = pack8(acc), hi = pack8(acc + 8);
  uint16_t* t_out = nullptr;
  if (kind == 0 && part + ch < m.Pp)
    t_out = xt + (((int64_t)n * m.H + unit) * m.Pp + part + ch) * L;
  else if (kind == 1 && part + ch < m.Np)
    t_out = bt + (((int64_t)n * m.G + unit) * m.Np + part + ch) * L;
  if (t_out != nullptr) {
    *reinterpret_cast<u16x8*>(t_out + t0) = lo;
    *reinterpret_cast<u16x8*>(t_out + t0 + 8) = hi;
  }
  if (kind == 0) return;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    ol[(t0 + i) * LP + ch] = lo[i];
    ol[(t0 + 8 + i) * LP + ch] = hi[i];
  }
  __syncthreads();
  uint16_t* o = kind == 1 ? b : c;
  for (int i = tid; i < L * 8; i += NT) {
    const int t = i / 8, d = i % 8 * 8;
    if (part + d < m.Np)
      *reinterpret_cast<u16x8*>(
          o + (((int64_t)n * L + t) * m.G + unit) * m.Np + part + d) =
          *reinterpret_cast<u16x8*>(ol + t * LP + d);
  }
}

struct Chunks {
  const float* da;
  const float* D;
  float* state;                // [slots, H, N, P]
  const int* slots;
  const int64_t* pos;
  const int* cu;
  const int* first;            // [B + 1] chunks of a sequence
  int64_t z_stride, y_stride;
  int z_at, H, P, Pp, N, Np, G, vec;
};

// NK: 32-wide steps of the state size. Wave w: tokens 16 w .. of the output,
// values 16 w .. of the state.
template <int NK>
__global__ __launch_bounds__(NT, NK > 4 ? 1 : 2) void ssm_chunks_kernel(
    uint16_t* __restrict__ y, const uint16_t* __restrict__ z,
    const uint16_t* __restrict__ xt, const uint16_t* __restrict__ b,
    const uint16_t* __restrict__ bt, const uint16_t* __restrict__ c,
    Chunks m) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  const int NP = m.Np + 8;
  uint16_t* bl = lds;                         // [64 tokens][NP]
  uint16_t* btl = bl + L * NP;                // [Np][LP]
  uint16_t* xl = btl + m.Np * LP;             // [64 values][LP]
  uint16_t* sh = xl + 64 * LP;                // [64 values][NP]
  uint16_t* sl = sh + 64 * NP;
  float* al = (float*)(sl + 64 * NP);         // [64] sums, [64] steps
  float* dl = al + L;

  const int seq = blockIdx.y, h = blockIdx.x, p0 = blockIdx.z * 64;
  const int g = h / (m.H / m.G);
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int np = min(64, m.P - p0), rowsp = min(64, m.Pp - p0);
  const int row0 = m.cu[seq], row1 = m.cu[seq + 1];
  const int slot = m.slots[seq];
  const int n0 = m.first[seq], n1 = m.first[seq + 1];
  const int ks = m.Np / 32, ns = m.Np / 16, per = m.Np / 8;
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};

  // this wave's 16 columns of the state: lane has column lo, rows 4 hi + r
  const int pcol = p0 + wid * 16 + lo;
  floatx4 S[NK * 2];
  float* st = m.state + ((int64_t)max(slot, 0) * m.H + h) * m.N * m.P + pcol;
  const bool carried = slot >= 0 && m.pos[row0] > 0 && pcol < m.P;
#pragma unroll
  for (int t = 0; t < NK * 2; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = t * 16 + hi * 4 + r;
      S[t][r] = carried && n < m.N ? st[(int64_t)n * m.P] : 0.f;
    }

  u16x8 breg[NK], btreg[NK], xreg[2], creg[NK];
  float areg = 0.f;
  auto load = [&](int n) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = i * NT + tid;
      breg[i] = btreg[i] = zero;
      if (e < L * per)
        breg[i] = ld_u16x8(
            b + (((int64_t)n * L + e / per) * m.G + g) * m.Np + e % per * 8);
      if (e < m.Np * 8)
        btreg[i] =
            ld_u16x8(bt + ((int64_t)n * m.G + g) * m.Np * L + e * 8);
      creg[i] = i < ks ? ld_u16x8(c + (((int64_t)n * L + wid * 16 + lo) *
                                           m.G + g) * m.Np +
                                  i * 32 + hi * 8)
                       : zero;
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = i * NT + tid;
      xreg[i] = e < rowsp * 8
                    ? ld_u16x8(xt + (((int64_t)n * m.H + h) * m.Pp + p0) * L +
                               e * 8)
                    : zero;
    }
    if (tid < 2 * L) areg = m.da[((int64_t)n * m.H + h) * 2 * L + tid];
  };

  load(n0);
  for (int n = n0; n < n1; ++n) {
    __syncthreads();                          // the last chunk is done
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = i * NT + tid;
      if (e < L * per)
        *reinterpret_cast<u16x8*>(bl + e / per * NP + e % per * 8) = breg[i];
      if (e < m.Np * 8)
        *reinterpret_cast<u16x8*>(btl + e / 8 * LP + e % 8 * 8) = btreg[i];
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = i * NT + tid;
      *reinterpret_cast<u16x8*>(xl + e / 8 * LP + e % 8 * 8) = xreg[i];
    }
    if (tid < 2 * L) al[tid] = areg;
#pragma unroll
    for (int t = 0; t < NK * 2; ++t)
      if (t < ns) {
        const float hi4[4] = {S[t][0], S[t][1], S[t][2], S[t][3]};
        uint16_t* at = sh + (wid * 16 + lo) * NP + t * 16 + hi * 4;
        st_bf16x4(at, hi4);
        float lo4[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) lo4[r] = hi4[r] - bf16_to_f32(at[r]);
        st_bf16x4(sl + (wid * 16 + lo) * NP + t * 16 + hi * 4, lo4);
      }
    u16x8 cf[NK];
#pragma unroll
    for (int k = 0; k < NK; ++k) cf[k] = creg[k];
    __syncthreads();
    if (n + 1 < n1) load(n + 1);

    // --- scores, transposed: lane has token i, 8 neighbouring j a group
    const int i = wid * 16 + lo;
    const float ai = al[i];
    u16x8 mh[2], mlow[2];
#pragma unroll
    for (int jp = 0; jp < 2; ++jp) {
      mh[jp] = mlow[jp] = zero;
      if (jp > (wid >> 1)) continue;
      float v[8];
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        floatx4 d = floatx4{0, 0, 0, 0};
        const uint16_t* br = bl + (jp * 32 + paired_row(lo, s)) * NP + hi * 8;
#pragma unroll
        for (int k = 0; k < NK; ++k)
          if (k < ks) d = mfma16(ld_u16x8(br + k * 32), cf[k], d);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = jp * 32 + hi * 8 + s * 4 + r;
          v[s * 4 + r] = j <= i ? d[r] * __expf(ai - al[j]) * dl[j] : 0.f;
        }
      }
      split8(v, mh[jp], mlow[jp]);
    }
    // --- outputs, transposed: lane has token i, values 4 hi + r
    const float ei = __expf(ai);
    const int64_t row = row0 + (int64_t)(n - n0) * L + i;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      if (t * 16 >= np) continue;
      floatx4 o = floatx4{0, 0, 0, 0};
      const uint16_t* s1 = sh + (t * 16 + lo) * NP + hi * 8;
      const uint16_t* s2 = sl + (t * 16 + lo) * NP + hi * 8;
#pragma unroll
      for (int k = 0; k < NK; ++k)
        if (k < ks) {
          o = mfma16(ld_u16x8(s1 + k * 32), cf[k], o);
          o = mfma16(ld_u16x8(s2 + k * 32), cf[k], o);
        }
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] *= ei;
#pragma unroll
      for (int jp = 0; jp < 2; ++jp) {
        if (jp > (wid >> 1)) continue;
        const u16x8 a = ld_u16x8(xl + (t * 16 + lo) * LP + jp * 32 + hi * 8);
        o = mfma16(a, mh[jp], o);
        o = mfma16(a, mlow[jp], o);
      }
      if (row < row1) {
        const int p = t * 16 + hi * 4;
        const int64_t zc = row * m.z_stride + m.z_at + h * m.P + p0 + p;
        uint16_t* dst = y + row * m.y_stride + h * m.P + p0 + p;
        if (m.vec) {
          if (p < np) {
            const u16x4 zz = *reinterpret_cast<const u16x4*>(z + zc);
            float v[4];
#pragma unroll
            for (int r = 0; r < 4; ++r)
              v[r] = (o[r] + m.D[h] * bf16_to_f32(xl[(p + r) * LP + i])) *
                     silu_s<uint16_t>(bf16_to_f32(zz[r]));
            st_bf16x4(dst, v);
          }
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (p + r < np)
              dst[r] = f32_to_bf16(
                  (o[r] + m.D[h] * bf16_to_f32(xl[(p + r) * LP + i])) *
                  silu_s<uint16_t>(bf16_to_f32(z[zc + r])));
        }
      }
    }
    // --- state
    if (wid * 16 < np) {
      const float end = al[L - 1], ee = __expf(end);
#pragma unroll
      for (int t = 0; t < NK * 2; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[t][r] *= ee;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const u16x8 x =
            ld_u16x8(xl + (wid * 16 + lo) * LP + kk * 32 + hi * 8);
        float v[8];
#pragma unroll
        for (int q = 0; q < 8; ++q) {
          const int j = kk * 32 + hi * 8 + q;
          v[q] = bf16_to_f32(x[q]) * (__expf(end - al[j]) * dl[j]);
        }
        u16x8 xh, xlow;
        split8(v, xh, xlow);
#pragma unroll
        for (int t = 0; t < NK * 2; ++t)
          if (t < ns) {
            const u16x8 a =
                ld_u16x8(btl + (t * 16 + lo) * LP + kk * 32 + hi * 8);
            S[t] = mfma16(a, xh, S[t]);
            S[t] = mfma16(a, xlow, S[t]);
          }
      }
    }
  }
  if (slot >= 0 && pcol < m.P) {
#pragma unroll
    for (int t = 0; t < NK * 2; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = t * 16 + hi * 4 + r;
        if (n < m.N) st[(int64_t)n * m.P] = S[t][r];
      }
  }
}

void check(const torch::Tensor& t, torch::ScalarType type, int64_t n) {
  TORCH_CHECK(t.scalar_type() == type && t.is_contiguous() && t.numel() == n,
              "ssm chunks: operand of ", t.numel(), " values, want ", n);
}

int chunk_lds(int Np) {
  return (3 * L * (Np + 8) + Np * LP + 64 * LP) * 2 + 2 * L * 4;
}

}  // namespace

bool ssm_chunks_fit(torch::Tensor z, int64_t vdim, int64_t state,
                    int64_t taps) {
  return z.scalar_type() == torch::kBFloat16 && state <= 256 && taps <= 65 &&
         vdim > 0;
}

void conv_chunks(torch::Tensor xt, torch::Tensor b, torch::Tensor bt,
                 torch::Tensor c, torch::Tensor da, torch::Tensor z,
                 int64_t xbc_at, int64_t dt_at, int64_t vdim, int64_t state,
                 torch::Tensor conv, torch::Tensor conv_b,
                 torch::Tensor dt_bias, torch::Tensor A_log,
                 torch::Tensor ring, torch::Tensor slots, torch::Tensor pos,
                 torch::Tensor cu, torch::Tensor seq, torch::Tensor row,
                 torch::Tensor count) {
  const auto BF = torch::kBFloat16, F32 = torch::kFloat32;
  const auto I32 = torch::kInt32;
  Conv m{};
  const int64_t n = seq.numel(), T = z.size(0);
  m.H = xt.size(1);
  m.P = vdim;
  m.Pp = xt.size(2);
  m.N = state;
  m.G = b.size(2);
  m.Np = b.size(3);
  m.taps = ring.size(1);
  m.C = ring.size(2);
  TORCH_CHECK(ssm_chunks_fit(z, vdim, state, m.taps));
  TORCH_CHECK(m.Pp >= m.P && m.Pp % 16 == 0 && m.Np >= m.N &&
              m.Np % 32 == 0 && m.C == m.H * m.P + 2 * m.G * m.N);
  check(xt, BF, n * m.H * m.Pp * L);
  check(b, BF, n * L * m.G * m.Np);
  check(c, BF, b.numel());
  check(bt, BF, b.numel());
  check(da, F32, n * m.H * 2 * L);
  check(conv, F32, (int64_t)m.C * m.taps);
  check(conv_b, F32, m.C);
  check(dt_bias, F32, m.H);
  check(A_log, F32, m.H);
  check(ring, BF, ring.numel());
  check(cu, I32, slots.numel() + 1);
  check(slots, I32, slots.numel());
  check(row, I32, n);
  check(count, I32, n);
  check(seq, I32, n);
  check(pos, torch::kInt64, T);
  TORCH_CHECK(z.stride(1) == 1 && xbc_at + m.C <= z.size(1) &&
              dt_at + m.H <= z.size(1));
  m.conv = conv.data_ptr<float>();
  m.conv_b = conv_b.data_ptr<float>();
  m.dt_bias = dt_bias.data_ptr<float>();
  m.A_log = A_log.data_ptr<float>();
  m.slots = slots.data_ptr<int>();
  m.pos = pos.data_ptr<int64_t>();
  m.cu = cu.data_ptr<int>();
  m.seq = seq.data_ptr<int>();
  m.row = row.data_ptr<int>();
  m.count = count.data_ptr<int>();
  m.z_stride = z.stride(0);
  m.xbc_at = xbc_at;
  m.dt_at = dt_at;
  if (n == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const int rows = L + m.taps - 1;
  const int lds = ((rows * 65 + 3) & ~3) * 4 + L * LP * 2;
  const dim3 grid(n, m.H * cdiv(m.P, 64) + 2 * m.G * cdiv(m.Np, 64) +
                         cdiv(m.H, 4));
  hipLaunchKernelGGL(conv_chunks_kernel, grid, dim3(NT), lds, stream,
                     (uint16_t*)xt.data_ptr(), (uint16_t*)b.data_ptr(),
                     (uint16_t*)bt.data_ptr(), (uint16_t*)c.data_ptr(),
                     da.data_ptr<float>(), (const uint16_t*)z.data_ptr(),
                     (uint16_t*)ring.data_ptr(), m);
}

void ssm_chunks(torch::Tensor y, torch::Tensor z, int64_t z_at, int64_t vdim,
                int64_t state_size, torch::Tensor xt, torch::Tensor b,
                torch::Tensor bt, torch::Tensor c, torch::Tensor da,
                torch::Tensor D, torch::Tensor state, torch::Tensor slots,
                torch::Tensor pos, torch::Tensor cu, torch::Tensor first) {
  const auto BF = torch::kBFloat16, F32 = torch::kFloat32;
  const auto I32 = torch::kInt32;
  Chunks m{};
  const int64_t n = xt.size(0);
  const int B = slots.numel();
  m.H = xt.size(1);
  m.P = vdim;
  m.Pp = xt.size(2);
  m.N = state_size;
  m.G = b.size(2);
  m.Np = b.size(3);
  TORCH_CHECK(ssm_chunks_fit(z, vdim, state_size, 1) && m.H % m.G == 0);
  TORCH_CHECK(m.Pp >= m.P && m.Pp % 16 == 0 && m.Np >= m.N &&
              m.Np % 32 == 0 && m.Np <= 256);
  check(xt, BF, n * m.H * m.Pp * L);
  check(b, BF, n * L * m.G * m.Np);
  check(c, BF, b.numel());
  check(bt, BF, b.numel());
  check(da, F32, n * m.H * 2 * L);
  check(D, F32, m.H);
  check(state, F32, state.size(0) * m.H * m.N * m.P);
  check(slots, I32, B);
  check(cu, I32, B + 1);
  check(first, I32, B + 1);
  check(pos, torch::kInt64, z.size(0));
  TORCH_CHECK(z.stride(1) == 1 && y.stride(1) == 1 &&
              z.size(0) == y.size(0) && y.size(1) == m.H * m.P &&
              y.scalar_type() == BF && z_at + m.H * m.P <= z.size(1));
  m.da = da.data_ptr<float>();
  m.D = D.data_ptr<float>();
  m.state = state.data_ptr<float>();
  m.slots = slots.data_ptr<int>();
  m.pos = pos.data_ptr<int64_t>();
  m.cu = cu.data_ptr<int>();
  m.first = first.data_ptr<int>();
  m.z_stride = z.stride(0);
  m.y_stride = y.stride(0);
  m.z_at = z_at;
  m.vec = m.P % 4 == 0 && z_at % 4 == 0 && m.z_stride % 4 == 0 &&
          m.y_stride % 4 == 0 && (uintptr_t)z.data_ptr() % 8 == 0 &&
          (uintptr_t)y.data_ptr() % 8 == 0;
  if (B == 0 || n == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(m.H, B, cdiv(m.P, 64));
  const int lds = chunk_lds(m.Np);
#define HELIX_SSM(NK)                                                        \
  do {                                                                       \
    static const hipError_t big = hipFuncSetAttribute(                       \
        (const void*)ssm_chunks_kernel<NK>,                                  \
        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);             \
    TORCH_CHECK(big == hipSuccess, "LDS size refused");                      \
    hipLaunchKernelGGL((ssm_chunks_kernel<NK>), grid, dim3(NT), lds, stream, \
                       (uint16_t*)y.data_ptr(),                              \
                       (const uint16_t*)z.data_ptr(),                        \
                       (const uint16_t*)xt.data_ptr(),                       \
                       (const uint16_t*)b.data_ptr(),                        \
                       (const uint16_t*)bt.data_ptr(),                       \
                       (const uint16_t*)c.data_ptr(), m);                    \
  } while (0)
  if (m.Np <= 32) HELIX_SSM(1);
  else if (m.Np <= 64) HELIX_SSM(2);
  else if (m.Np <= 128) HELIX_SSM(4);
  else HELIX_SSM(8);
#undef HELIX_SSM
}
