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
// da [H, 3, 64] (A_t, dt_t and e^(A_63 - A_t) dt_t). Tokens past a portion's end and state
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
  int xbc_at, dt_at, H, P, Pp, N, Np, G, taps, C, vec;
};

// grid (chunks, channel blocks of 64 + blocks of 4 heads for da)
__global__ __launch_bounds__(NT) void conv_chunks_kernel(
    uint16_t* __restrict__ xt, uint16_t* __restrict__ b,
    uint16_t* __restrict__ bt, uint16_t* __restrict__ c,
    float* __restrict__ da, const uint16_t* __restrict__ z, uint16_t* ring,
    Conv m) {
  extern __shared__ __attribute__((aligned(16))) uint16_t sh[];
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
    float* o = da + ((int64_t)n * m.H + h) * 3 * L;
    o[t] = a;
    o[L + t] = dt;
    o[2 * L + t] = __expf(__shfl(a, WAVE - 1, WAVE) - a) * dt;
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
  // Inputs in LDS, a row per token: the chunk's own and those before it.
  const int before = m.taps - 1, rows = L + before;
  uint16_t* in = sh;                          // [rows][LP]
  uint16_t* tl = in + rows * LP;              // [64 channels][LP] result
  uint16_t* rl = tl + 64 * LP;                // [64 tokens][LP] result
  const int seq0 = m.cu[sq], slot = m.slots[sq];
  const int64_t p0 = m.pos[row];
  const uint16_t* zc = z + m.xbc_at + c0;
  uint16_t* rs = ring + (int64_t)max(slot, 0) * m.taps * m.C + c0;
  if (m.vec) {
    for (int i = tid; i < rows * 8; i += NT) {
      const int r = i / 8, ch = i % 8 * 8, t = r - before;
      u16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (ch < nc && t < count) {
        if (row + t >= seq0)
          v = ld_u16x8(zc + (row + t) * m.z_stride + ch);
        else if (slot >= 0 && p0 + t >= 0)
          v = ld_u16x8(rs + (p0 + t) % m.taps * m.C + ch);
      }
      *reinterpret_cast<u16x8*>(in + r * LP + ch) = v;
    }
  } else {
    for (int i = tid; i < rows * 64; i += NT) {
      const int r = i / 64, ch = i % 64, t = r - before;
      uint16_t v = 0;
      if (ch < nc && t < count) {
        if (row + t >= seq0) v = zc[(row + t) * m.z_stride + ch];
        else if (slot >= 0 && p0 + t >= 0)
          v = rs[(p0 + t) % m.taps * m.C + ch];
      }
      in[r * LP + ch] = v;
    }
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
            zc[(int64_t)(seq0 + t) * m.z_stride + ch];
    }
  }
  // A thread has two neighbouring channels of 8 tokens.
  const int ch = tid % 32 * 2, t0 = tid / 32 * 8;
  const int ca = c0 + min(ch, max(nc, 1) - 1);
  const int cb = c0 + min(ch + 1, max(nc, 1) - 1);
  float u[8], v[8];
  if (nc > 0) {
    const float b0 = m.conv_b[ca], b1 = m.conv_b[cb];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      u[i] = b0;
      v[i] = b1;
    }
    const uint16_t* src = in + t0 * LP + ch;
    auto tap = [&](int k, const uint32_t* x) {
      const float w0 = m.conv[(int64_t)ca * m.taps + k];
      const float w1 = m.conv[(int64_t)cb * m.taps + k];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        u[i] += w0 * bf16_to_f32((uint16_t)x[i]);
        v[i] += w1 * bf16_to_f32((uint16_t)(x[i] >> 16));
      }
    };
    if (m.taps == 4) {
      uint32_t x[11];
#pragma unroll
      for (int i = 0; i < 11; ++i)
        x[i] = *reinterpret_cast<const uint32_t*>(src + i * LP);
#pragma unroll
      for (int k = 0; k < 4; ++k) tap(k, x + k);
    } else {
      for (int k = 0; k < m.taps; ++k) {
        uint32_t x[8];
#pragma unroll
        for (int i = 0; i < 8; ++i)
          x[i] = *reinterpret_cast<const uint32_t*>(src + (i + k) * LP);
        tap(k, x);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    u[i] = ch < nc && t0 + i < count ? silu_s<uint16_t>(u[i]) : 0.f;
    v[i] = ch + 1 < nc && t0 + i < count ? silu_s<uint16_t>(v[i]) : 0.f;
  }
  if (kind != 2) {
    *reinterpret_cast<u16x8*>(tl + ch * LP + t0) = pack8(u);
    *reinterpret_cast<u16x8*>(tl + (ch + 1) * LP + t0) = pack8(v);
  }
  if (kind != 0) {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      *reinterpret_cast<uint32_t*>(rl + (t0 + i) * LP + ch) =
          pack_bf16(u[i], v[i]);
  }
  __syncthreads();
  if (kind != 2) {
    const int width = kind == 0 ? m.Pp : m.Np;
    uint16_t* o = kind == 0
                      ? xt + (((int64_t)n * m.H + unit) * m.Pp + part) * L
                      : bt + (((int64_t)n * m.G + unit) * m.Np + part) * L;
    for (int i = tid; i < 64 * 8; i += NT)
      if (part + i / 8 < width)
        *reinterpret_cast<u16x8*>(o + i * 8) =
            ld_u16x8(tl + i / 8 * LP + i % 8 * 8);
  }
  if (kind != 0) {
    uint16_t* o = kind == 1 ? b : c;
    for (int i = tid; i < L * 8; i += NT) {
      const int t = i / 8, d = i % 8 * 8;
      if (part + d < m.Np)
        *reinterpret_cast<u16x8*>(
            o + (((int64_t)n * L + t) * m.G + unit) * m.Np + part + d) =
            ld_u16x8(rl + t * LP + d);
    }
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

// NK: 32-wide steps of the state size; PW: 16-value tiles of a workgroup.
// Wave w has tokens 16 w .. of the output, and of the state the value tile
// w % PW in its share of the rows.
template <int NK, int PW>
__global__ __launch_bounds__(NT, NK > 4 ? 1 : 2) void ssm_chunks_kernel(
    uint16_t* __restrict__ y, const uint16_t* __restrict__ z,
    const uint16_t* __restrict__ xt, const uint16_t* __restrict__ b,
    const uint16_t* __restrict__ bt, const uint16_t* __restrict__ c,
    Chunks m) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  constexpr int PB = PW * 16, ST = NK * PW / 2, XL = PW / 2;
  const int NP = m.Np + 8;
  uint16_t* bl = lds;                         // [64 tokens][NP]
  uint16_t* btl = bl + L * NP;                // [Np][LP]
  uint16_t* xl = btl + m.Np * LP;             // [PB values][LP]
  uint16_t* sh = xl + PB * LP;                // [PB values][NP]
  uint16_t* sl = sh + PB * NP;
  float* al = (float*)(sl + PB * NP);         // sums, steps, weights: [64]
  float *dl = al + L, *wl = dl + L;

  // neighbouring heads share B and C: an XCD gets a contiguous range
  const int h = m.H % 8 ? blockIdx.x
                        : (blockIdx.x & 7) * (m.H / 8) + (blockIdx.x >> 3);
  const int seq = blockIdx.y, p0 = blockIdx.z * PB;
  const int g = h / (m.H / m.G);
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int np = min(PB, m.P - p0), rowsp = min(PB, m.Pp - p0);
  const int row0 = m.cu[seq], row1 = m.cu[seq + 1];
  const int slot = m.slots[seq];
  const int n0 = m.first[seq], n1 = m.first[seq + 1];
  const int ks = m.Np / 32, per = m.Np / 8;
  // this wave's 16 columns of the state: lane has column lo, rows 4 hi + r
  // of the nts row tiles from nt0 on
  const int pt = wid % PW, pcol = p0 + pt * 16 + lo;
  const int nts = m.Np * PW / 64, nt0 = wid / PW * nts;
  floatx4 S[ST];
  float* st = m.state + ((int64_t)max(slot, 0) * m.H + h) * m.N * m.P + pcol;
  const bool carried = slot >= 0 && m.pos[row0] > 0 && pcol < m.P;
#pragma unroll
  for (int t = 0; t < ST; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = (nt0 + t) * 16 + hi * 4 + r;
      S[t][r] = carried && t < nts && n < m.N ? st[(int64_t)n * m.P] : 0.f;
    }

  u16x8 breg[NK], btreg[NK], xreg[XL], creg[NK];
  float areg = 0.f;
  // No branches, so that all loads are under way at once: indices past the
  // end are clamped and their values not stored.
  auto load = [&](int n) {
    const int64_t at = (int64_t)n * L * m.G * m.Np;
    const uint16_t* bn = b + at + g * m.Np;
    const uint16_t* btn = bt + at + (int64_t)g * m.Np * L;
    const uint16_t* cn =
        c + at + ((int64_t)(wid * 16 + lo) * m.G + g) * m.Np + hi * 8;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = min(i * NT + tid, L * per - 1);
      breg[i] = ld_u16x8(bn + (int64_t)(e / per) * m.G * m.Np + e % per * 8);
      btreg[i] = ld_u16x8(btn + e * 8);
      creg[i] = ld_u16x8(cn + min(i, ks - 1) * 32);
    }
    const uint16_t* xn = xt + (((int64_t)n * m.H + h) * m.Pp + p0) * L;
#pragma unroll
    for (int i = 0; i < XL; ++i)
      xreg[i] = ld_u16x8(xn + min(i * NT + tid, rowsp * 8 - 1) * 8);
    areg = m.da[((int64_t)n * m.H + h) * 3 * L + min(tid, 3 * L - 1)];
  };

  const float Dh = m.D[h];
  load(n0);
  for (int n = n0; n < n1; ++n) {
    __syncthreads();                          // the last chunk is done
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = i * NT + tid;
      if (e < L * per)
        *reinterpret_cast<u16x8*>(bl + paired_row(e / per) * NP +
                                  e % per * 8) = breg[i];
      if (e < m.Np * 8)
        *reinterpret_cast<u16x8*>(btl + e / 8 * LP + e % 8 * 8) = btreg[i];
    }
#pragma unroll
    for (int i = 0; i < XL; ++i) {
      const int e = i * NT + tid;
      *reinterpret_cast<u16x8*>(xl + e / 8 * LP + e % 8 * 8) = xreg[i];
    }
    if (tid < 3 * L) al[tid] = areg;
#pragma unroll
    for (int t = 0; t < ST; ++t)
      if (t < nts) {
        const uint32_t u0 = pack_bf16(S[t][0], S[t][1]);
        const uint32_t u1 = pack_bf16(S[t][2], S[t][3]);
        const int at = (pt * 16 + lo) * NP + (nt0 + t) * 16 + hi * 4;
        *reinterpret_cast<u32x2*>(sh + at) = u32x2{u0, u1};
        const float rest[4] = {
            S[t][0] - bf16_to_f32((uint16_t)u0),
            S[t][1] - bf16_to_f32((uint16_t)(u0 >> 16)),
            S[t][2] - bf16_to_f32((uint16_t)u1),
            S[t][3] - bf16_to_f32((uint16_t)(u1 >> 16))};
        st_bf16x4(sl + at, rest);
      }
    u16x8 cf[NK];
#pragma unroll
    for (int k = 0; k < NK; ++k) cf[k] = creg[k];
    __syncthreads();
    // this chunk's gates and the next one's operands are on their way while
    // the products run
    const int i = wid * 16 + lo;
    const int64_t row = row0 + (int64_t)(n - n0) * L + i;
    const uint16_t* zr =
        z + min(row, (int64_t)row1 - 1) * m.z_stride + m.z_at + h * m.P + p0;
    u16x4 zreg[PW];
    if (m.vec) {
#pragma unroll
      for (int t = 0; t < PW; ++t)
        zreg[t] = *reinterpret_cast<const u16x4*>(
            zr + min(t * 16 + hi * 4, np - 4));
    }
    if (n + 1 < n1) load(n + 1);

    // --- scores, transposed: lane has token i, 8 neighbouring j a group
    const float ai = al[i];
    u16x8 mh[2], mlow[2];
#pragma unroll
    for (int jp = 0; jp < 2; ++jp) {
      if (jp > (wid >> 1)) continue;
      float v[8];
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        floatx4 d = floatx4{0, 0, 0, 0};
        const uint16_t* br = bl + (jp * 32 + s * 16 + lo) * NP + hi * 8;
#pragma unroll
        for (int k = 0; k < NK; ++k)
          if (k < ks) d = mfma16(ld_u16x8(br + k * 32), cf[k], d);
        const int j = jp * 32 + hi * 8 + s * 4;
        const f32x4 aj = *reinterpret_cast<const f32x4*>(al + j);
        const f32x4 dj = *reinterpret_cast<const f32x4*>(dl + j);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          v[s * 4 + r] = j + r <= i ? d[r] * __expf(ai - aj[r]) * dj[r] : 0.f;
      }
      split8(v, mh[jp], mlow[jp]);
    }
    // --- outputs, transposed: lane has token i, values 4 hi + r
    const float ei = __expf(ai);
#pragma unroll
    for (int t = 0; t < PW; ++t) {
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
        uint16_t* dst = y + row * m.y_stride + h * m.P + p0 + p;
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r)
          v[r] = o[r] + Dh * bf16_to_f32(xl[(p + r) * LP + i]);
        if (m.vec) {
          if (p < np) {
#pragma unroll
            for (int r = 0; r < 4; ++r)
              v[r] *= silu_s<uint16_t>(bf16_to_f32(zreg[t][r]));
            st_bf16x4(dst, v);
          }
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (p + r < np)
              dst[r] = f32_to_bf16(
                  v[r] * silu_s<uint16_t>(bf16_to_f32(zr[p + r])));
        }
      }
    }
    // --- state
    if (pt * 16 < np) {
      const float ee = __expf(al[L - 1]);
#pragma unroll
      for (int t = 0; t < ST; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[t][r] *= ee;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const u16x8 x =
            ld_u16x8(xl + (pt * 16 + lo) * LP + kk * 32 + hi * 8);
        float v[8], w[8];
        ldv<8>(wl + kk * 32 + hi * 8, w);
#pragma unroll
        for (int q = 0; q < 8; ++q) v[q] = bf16_to_f32(x[q]) * w[q];
        u16x8 xh, xlow;
        split8(v, xh, xlow);
#pragma unroll
        for (int t = 0; t < ST; ++t)
          if (t < nts) {
            const u16x8 a = ld_u16x8(btl + ((nt0 + t) * 16 + lo) * LP +
                                     kk * 32 + hi * 8);
            S[t] = mfma16(a, xh, S[t]);
            S[t] = mfma16(a, xlow, S[t]);
          }
      }
    }
  }
  if (slot >= 0 && pcol < m.P) {
#pragma unroll
    for (int t = 0; t < ST; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = (nt0 + t) * 16 + hi * 4 + r;
        if (t < nts && n < m.N) st[(int64_t)n * m.P] = S[t][r];
      }
  }
}

void check(const torch::Tensor& t, torch::ScalarType type, int64_t n) {
  TORCH_CHECK(t.scalar_type() == type && t.is_contiguous() && t.numel() == n,
              "ssm chunks: operand of ", t.numel(), " values, want ", n);
}

int chunk_lds(int Np, int PB) {
  return ((L + 2 * PB) * (Np + 8) + (Np + PB) * LP) * 2 + 3 * L * 4;
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
  check(da, F32, n * m.H * 3 * L);
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
  // 16-byte loads: every block of channels starts on 8 and is whole
  m.vec = m.P % 8 == 0 && m.N % 8 == 0 && m.C % 8 == 0 && xbc_at % 8 == 0 &&
          m.z_stride % 8 == 0 && (uintptr_t)z.data_ptr() % 16 == 0;
  const int lds = (L + m.taps - 1 + 64 + L) * LP * 2;
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
  check(da, F32, n * m.H * 3 * L);
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
  // few heads and sequences: half the values to a workgroup
  const int PW = (int64_t)m.H * B * cdiv(m.P, 64) < 256 ? 2 : 4;
  const dim3 grid(m.H, B, cdiv(m.P, PW * 16));
  const int lds = chunk_lds(m.Np, PW * 16);
#define HELIX_SSM_P(NK, PW)                                                  \
  do {                                                                       \
    static const hipError_t big = hipFuncSetAttribute(                       \
        (const void*)ssm_chunks_kernel<NK, PW>,                              \
        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);             \
    TORCH_CHECK(big == hipSuccess, "LDS size refused");                      \
    hipLaunchKernelGGL((ssm_chunks_kernel<NK, PW>), grid, dim3(NT), lds,     \
                       stream, (uint16_t*)y.data_ptr(),                      \
                       (const uint16_t*)z.data_ptr(),                        \
                       (const uint16_t*)xt.data_ptr(),                       \
                       (const uint16_t*)b.data_ptr(),                        \
                       (const uint16_t*)bt.data_ptr(),                       \
                       (const uint16_t*)c.data_ptr(), m);                    \
  } while (0)
#define HELIX_SSM(NK)                                                        \
  if (PW == 4) HELIX_SSM_P(NK, 4); else HELIX_SSM_P(NK, 2)
  if (m.Np <= 32) { HELIX_SSM(1); }
  else if (m.Np <= 64) { HELIX_SSM(2); }
  else if (m.Np <= 128) { HELIX_SSM(4); }
  else { HELIX_SSM(8); }
#undef HELIX_SSM
#undef HELIX_SSM_P
}
