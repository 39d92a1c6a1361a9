// Gated linear attention over prompt portions, 64 tokens at a time on MFMA.
//
// With c_t the running sum of a chunk's log decays (per key channel) and S
// the state that enters it:
//
//   o_i = S^T (q_i e^(c_i)) + sum_{j<=i} A_ij v_j
//   A_ij = sum_d q_i[d] k_j[d] e^(c_i[d] - c_j[d])
//   S  <- diag(e^(c_63)) S + sum_j (k_j e^(c_63 - c_j)) v_j^T
//
// gla_operands makes a chunk's operands. No power there overflows,
// however fast a channel decays: A's blocks of 16 x 16 take the start of the
// later block as reference. On the diagonal keys then have positive ones;
// where a channel decays by more than 2^-100 in 16 tokens, that block is
// summed pair by pair in fp32. gla_chunks carries a head's state from
// chunk to chunk in fp32 registers. v enters the products as the bf16 it is,
// whatever has a decay or the state in it as two bf16 terms (17 bits).
//
// Operands per chunk and head: qe [2, 64, Dp], ke [2, Dp, 64], am
// [2, 64, 64] (two terms each), vt [Pp, 64], ec [Dp] (fp32, e^(c_63)).
// Tokens past a portion's end and channels past D are zero.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int NT = 256;
constexpr int L = 64;                         // tokens of a chunk
constexpr int LP = L + 8;
constexpr int SL = 32;                        // channels worked on at a time
constexpr int PV = 36;                        // pitch, rows read as vectors
constexpr int PS = 33;                        // pitch, columns read
constexpr float LOG2E_ = 1.4426950408889634f;

struct Operands {
  const uint16_t* a2;          // [H * D, rank_pad]
  const float* a2_b;           // [H * D]
  const int *row, *count;      // per chunk
  int64_t z_stride;
  int q_at, k_at, v_at, a_at, H, D, Dp, E, Pp, rank, rank_pad, vec;
  float unit, q_scale;         // unit: 1 / tau
};

// Columns c0 .. c0 + 31 of the chunk's rows, 8 per thread; nothing past
// column n or row count.
__device__ __forceinline__ u16x8 load_slice(const uint16_t* z, int64_t stride,
                                            int c0, int n, int count,
                                            bool vec) {
  const int t = threadIdx.x / 4, d = c0 + threadIdx.x % 4 * 8;
  u16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
  if (t >= count) return v;
  const uint16_t* p = z + t * stride + d;
  if (vec) {
    if (d < n) v = ld_u16x8(p);
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (d + i < n) v[i] = p[i];
  }
  return v;
}

__device__ __forceinline__ float exp2_(float x) {
  return __builtin_amdgcn_exp2f(x);
}

// log2(1 + 2^x)
__device__ __forceinline__ float softplus2(float x) {
  return fmaxf(x, 0.f) +
         __builtin_amdgcn_logf(1.f + exp2_(-fabsf(x)));
}

// Most a channel may decay within 16 tokens (as a power of two) for the
// diagonal blocks to be products.
constexpr float STEEP = -100.f;

// grid (chunks, heads). Decays are kept as base-2 logarithms.
__global__ __launch_bounds__(NT) void gla_operands_kernel(
    uint16_t* __restrict__ qe, uint16_t* __restrict__ ke,
    uint16_t* __restrict__ am, uint16_t* __restrict__ vt,
    float* __restrict__ ec, const uint16_t* __restrict__ z, Operands m) {
  __shared__ __attribute__((aligned(16))) float qs[L * PV];
  __shared__ float ks[L * PS];                // keys (later values)
  __shared__ float cs[L * PS];                // log decays, summed
  __shared__ float ends[4][SL];               // of every 16 tokens
  const int n = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int count = m.count[n];
  const uint16_t* zr = z + (int64_t)m.row[n] * m.z_stride;
  const int64_t nh = (int64_t)n * m.H + h;
  uint16_t* qo = qe + nh * 2 * L * m.Dp;
  uint16_t* ko = ke + nh * 2 * L * m.Dp;
  // the score blocks (I, J <= I) of this wave; heads start elsewhere, so
  // that the long rows do not all meet on one SIMD
  const int I = (wid + h) & 3;
  floatx4 acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = floatx4{0, 0, 0, 0};

  // inputs of the decays: wave w has tokens 16 w ..
  auto rank_terms = [&](int r) {
    u16x8 a = {0, 0, 0, 0, 0, 0, 0, 0};
    const int t = wid * 16 + lo;
    if (t < count && r < m.rank) {
      const uint16_t* ap = zr + t * m.z_stride + m.a_at + r;
      if (m.vec && r + 8 <= m.rank) {
        a = ld_u16x8(ap);
      } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
          if (r + i < m.rank) a[i] = ap[i];
      }
    }
    return a;
  };
  const u16x8 a0 = rank_terms(hi * 8);
  const uint16_t *zq = zr + m.q_at + h * m.D, *zk = zr + m.k_at + h * m.D;
  // a slice's queries, keys and decay weights are under way one slice ahead
  u16x8 qreg, kreg, b0[2];
  auto load = [&](int d0) {
    qreg = load_slice(zq, m.z_stride, d0, m.D, count, m.vec);
    kreg = load_slice(zk, m.z_stride, d0, m.D, count, m.vec);
#pragma unroll
    for (int u = 0; u < 2; ++u)
      b0[u] = ld_u16x8(m.a2 + (int64_t)(h * m.D + min(d0 + u * 16 + lo,
                                                      m.D - 1)) *
                                  m.rank_pad + hi * 8);
  };

  load(0);
  for (int d0 = 0; d0 < m.Dp; d0 += SL) {
    float v[8], w[8];
    const int t = tid / 4, s = tid % 4 * 8;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[i] = bf16_to_f32(qreg[i]);
      w[i] = bf16_to_f32(kreg[i]);
    }
    // a lane has 4 tokens of two channels
    floatx4 x[2];
#pragma unroll
    for (int u = 0; u < 2; ++u)
      x[u] = mfma16(a0, b0[u], floatx4{0, 0, 0, 0});
    for (int r = 32 + hi * 8; r < m.rank_pad; r += 32) {
      const u16x8 a = rank_terms(r);
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const int c = min(d0 + u * 16 + lo, m.D - 1);
        x[u] = mfma16(
            a, ld_u16x8(m.a2 + (int64_t)(h * m.D + c) * m.rank_pad + r),
            x[u]);
      }
    }
    if (d0 + SL < m.Dp) load(d0 + SL);
    float part[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int c = d0 + u * 16 + lo;
      const float bias = c < m.D ? m.a2_b[h * m.D + c] : 0.f;
      float sum = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const bool in = c < m.D && wid * 16 + hi * 4 + r < count;
        // log2(sigmoid(y)^(1/tau)) = -softplus2(-y log2(e)) / tau
        const float g = -softplus2(-(x[u][r] + bias) * LOG2E_) * m.unit;
        sum += in ? g : 0.f;
        x[u][r] = sum;
      }
      float up = __shfl_up(sum, 16, WAVE);
      if (hi >= 1) sum += up;
      up = __shfl_up(sum, 32, WAVE);
      if (hi >= 2) sum += up;
      part[u] = sum - x[u][3];                // of the lanes before
    }
    __syncthreads();                          // the last slice is done
#pragma unroll
    for (int u = 0; u < 2; ++u)
      if (hi == 3) ends[wid][u * 16 + lo] = part[u] + x[u][3];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[i] *= m.q_scale;
      ks[t * PS + s + i] = w[i];
    }
    stv<8>(qs + t * PV + s, v);
    __syncthreads();
    bool steep = false;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float base = part[u];
#pragma unroll
      for (int i = 0; i < 3; ++i)
        if (i < wid) base += ends[i][u * 16 + lo];
#pragma unroll
      for (int r = 0; r < 4; ++r)
        cs[(wid * 16 + hi * 4 + r) * PS + u * 16 + lo] = base + x[u][r];
      steep |= ends[I][u * 16 + lo] < STEEP;
    }
    steep = __any(steep);
    __syncthreads();
    // queries and keys with their decays
    u16x8 a, b;
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= exp2_(cs[t * PS + s + i]);
    split8(v, a, b);
    *reinterpret_cast<u16x8*>(qo + t * m.Dp + d0 + s) = a;
    *reinterpret_cast<u16x8*>(qo + (L + t) * m.Dp + d0 + s) = b;
    const int kd = tid / 8, kt = tid % 8 * 8;
    const float end = cs[(L - 1) * PS + kd];
#pragma unroll
    for (int i = 0; i < 8; ++i)
      w[i] = ks[(kt + i) * PS + kd] * exp2_(end - cs[(kt + i) * PS + kd]);
    split8(w, a, b);
    *reinterpret_cast<u16x8*>(ko + (d0 + kd) * L + kt) = a;
    *reinterpret_cast<u16x8*>(ko + (m.Dp + d0 + kd) * L + kt) = b;
    if (tid < SL) ec[nh * m.Dp + d0 + tid] = exp2_(cs[(L - 1) * PS + tid]);

    // scores: rows j of a block's result, columns i
    const int i = I * 16 + lo;
    float ref[8], q[8];
#pragma unroll
    for (int c = 0; c < 8; ++c) {
      const int d = hi * 8 + c;
      ref[c] = I > 0 ? cs[(I * 16 - 1) * PS + d] : 0.f;
      q[c] = qs[i * PV + d] * exp2_(cs[i * PS + d] - ref[c]);
    }
    u16x8 qh, ql;
    split8(q, qh, ql);
#pragma unroll
    for (int J = 0; J < 4; ++J) {
      if (J > I || (J == I && steep)) continue;
      const int j = J * 16 + lo;
      float k[8];
#pragma unroll
      for (int c = 0; c < 8; ++c)
        k[c] = ks[j * PS + hi * 8 + c] *
               exp2_(ref[c] - cs[j * PS + hi * 8 + c]);
      u16x8 kh, kl;
      split8(k, kh, kl);
      acc[J] = mfma16(kh, qh, acc[J]);
      acc[J] = mfma16(kh, ql, acc[J]);
      acc[J] = mfma16(kl, qh, acc[J]);
    }
    if (steep)
#pragma unroll
      for (int J = 0; J < 4; ++J)
        if (J == I)
          for (int d = 0; d < SL; ++d) {
            const float qd = qs[i * PV + d], cd = cs[i * PS + d];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int j = J * 16 + hi * 4 + r;
              if (j <= i)
                acc[J][r] += qd * ks[j * PS + d] * exp2_(cd - cs[j * PS + d]);
            }
          }
  }

  const uint16_t* zv = zr + m.v_at + h * m.E;
  u16x8 vreg = load_slice(zv, m.z_stride, 0, m.E, count, m.vec);
  uint16_t* ao = am + nh * 2 * L * L + (I * 16 + lo) * L + hi * 4;
#pragma unroll
  for (int J = 0; J < 4; ++J) {
    float x[4], rest[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      x[r] = J < I || (J == I && hi * 4 + r <= lo) ? acc[J][r] : 0.f;
      rest[r] = x[r] - bf16_to_f32(f32_to_bf16(x[r]));
    }
    st_bf16x4(ao + J * 16, x);
    st_bf16x4(ao + L * L + J * 16, rest);
  }
  // values, transposed
  for (int e0 = 0; e0 < m.Pp; e0 += SL) {
    float v[8];
    const u16x8 raw = vreg;
    if (e0 + SL < m.Pp) vreg = load_slice(zv, m.z_stride, e0 + SL, m.E, count,
                                          m.vec);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 8; ++i)
      ks[tid / 4 * PS + tid % 4 * 8 + i] = bf16_to_f32(raw[i]);
    __syncthreads();
    const int e = e0 + tid / 8, t = tid % 8 * 8;
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = ks[(t + i) * PS + tid / 8];
    if (e < m.Pp)
      *reinterpret_cast<u16x8*>(vt + (nh * m.Pp + e) * L + t) = pack8(v);
  }
}

struct Chunks {
  const float* ec;
  float* state;                // [slots, H, D, Ep]
  const int* slots;
  const int64_t* pos;
  const int* cu;
  const int* first;            // [B + 1] chunks of a sequence
  int64_t o_stride;
  int H, D, Dp, E, Ep, Pp, vec;
};

// A chunk's operands on their way to one thread.
template <int NK, int XL>
struct Stage {
  u16x8 k[NK * 2], q[2][NK], a[2][2], x[XL];
  float e;
};

// NK: 32-wide steps of the key channels; PW: 16-value tiles of a workgroup.
// Wave w has tokens 16 w .. of the output, and of the state the value tile
// w % PW in its share of the rows. FULL: every tile is a whole one, so
// nothing branches and the products of different tiles overlap (a chunk
// waits for the one before, so the chunk's own latency is the time).
template <int NK, int PW, bool FULL>
__global__ __launch_bounds__(NT, NK > 4 ? 1 : 2) void gla_chunks_kernel(
    uint16_t* __restrict__ o, const uint16_t* __restrict__ qe,
    const uint16_t* __restrict__ ke, const uint16_t* __restrict__ am,
    const uint16_t* __restrict__ vt, Chunks m) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  constexpr int PB = PW * 16, ST = NK * PW / 2, XL = PW / 2;
  constexpr int KR = NK * 2;                  // 16-byte loads of ke's terms
  const int NP = m.Dp + 8;
  uint16_t* kl = lds;                         // [2 Dp][LP] keys' terms
  uint16_t* xl = kl + 2 * m.Dp * LP;          // [PB values][LP]
  uint16_t* sh = xl + PB * LP;                // [PB values][NP] state
  uint16_t* sl = sh + PB * NP;
  float* el = (float*)(sl + PB * NP);         // [Dp]

  // neighbouring heads of a chunk are neighbours in memory
  const int h = m.H % 8 ? blockIdx.x
                        : (blockIdx.x & 7) * (m.H / 8) + (blockIdx.x >> 3);
  const int seq = blockIdx.y, p0 = blockIdx.z * PB;
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int np = min(PB, m.E - p0), rowsp = min(PB, m.Pp - p0);
  const int row0 = m.cu[seq], row1 = m.cu[seq + 1];
  const int slot = m.slots[seq];
  const int n0 = m.first[seq], n1 = m.first[seq + 1];
  if (n0 >= n1) return;
  const int ks = m.Dp / 32;
  // this wave's 16 columns of the state: lane has column lo, rows 4 hi + r
  // of the nts row tiles from nt0 on
  const int pt = wid % PW, pcol = p0 + pt * 16 + lo;
  const int nts = m.Dp * PW / 64, nt0 = wid / PW * nts;
  floatx4 S[ST];
  float* st = m.state + ((int64_t)max(slot, 0) * m.H + h) * m.D * m.Ep + pcol;
  const bool carried = slot >= 0 && m.pos[row0] > 0 && pcol < m.E;
#pragma unroll
  for (int t = 0; t < ST; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = (nt0 + t) * 16 + hi * 4 + r;
      S[t][r] = carried && t < nts && n < m.D ? st[(int64_t)n * m.Ep] : 0.f;
    }

  Stage<NK, XL> in;
  // No branches, so that all loads are under way at once: indices past the
  // end are clamped and their values not stored or not used.
  auto load = [&](int n) {
    const int64_t nh = (int64_t)n * m.H + h;
    const uint16_t* kn = ke + nh * 2 * L * m.Dp;
#pragma unroll
    for (int i = 0; i < KR; ++i)
      in.k[i] = ld_u16x8(kn + min(i * NT + tid, m.Dp * 16 - 1) * 8);
    const uint16_t* qn = qe + (nh * 2 * L + wid * 16 + lo) * m.Dp + hi * 8;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int k = 0; k < NK; ++k)
        in.q[s][k] = ld_u16x8(qn + (int64_t)s * L * m.Dp + min(k, ks - 1) * 32);
      const uint16_t* an =
          am + ((nh * 2 + s) * L + wid * 16 + lo) * L + hi * 8;
      in.a[s][0] = ld_u16x8(an);
      in.a[s][1] = ld_u16x8(an + 32);
    }
    const uint16_t* xn = vt + (nh * m.Pp + p0) * L;
#pragma unroll
    for (int i = 0; i < XL; ++i)
      in.x[i] = ld_u16x8(xn + min(i * NT + tid, rowsp * 8 - 1) * 8);
    in.e = m.ec[nh * m.Dp + min(tid, m.Dp - 1)];
  };

  load(n0);
  for (int n = n0; n < n1; ++n) {
    __syncthreads();                          // the last chunk is done
#pragma unroll
    for (int i = 0; i < KR; ++i) {
      const int e = i * NT + tid;
      if (FULL || e < m.Dp * 16)
        *reinterpret_cast<u16x8*>(kl + e / 8 * LP + e % 8 * 8) = in.k[i];
    }
#pragma unroll
    for (int i = 0; i < XL; ++i) {
      const int e = i * NT + tid;
      *reinterpret_cast<u16x8*>(xl + e / 8 * LP + e % 8 * 8) = in.x[i];
    }
    if (tid < m.Dp) el[tid] = in.e;
#pragma unroll
    for (int t = 0; t < ST; ++t)
      if (FULL || t < nts) {
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
    u16x8 qf[2][NK], af[2][2];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int k = 0; k < NK; ++k) qf[s][k] = in.q[s][k];
      af[s][0] = in.a[s][0];
      af[s][1] = in.a[s][1];
    }
    __syncthreads();
    if (n + 1 < n1) load(n + 1);

    // --- outputs, transposed: lane has token i, values 4 hi + r
    const int i = wid * 16 + lo;
    const int64_t row = row0 + (int64_t)(n - n0) * L + i;
#pragma unroll
    for (int t = 0; t < PW; ++t) {
      if (!FULL && t * 16 >= np) continue;
      floatx4 d = floatx4{0, 0, 0, 0};
      const uint16_t* s1 = sh + (t * 16 + lo) * NP + hi * 8;
      const uint16_t* s2 = sl + (t * 16 + lo) * NP + hi * 8;
#pragma unroll
      for (int k = 0; k < NK; ++k)
        if (FULL || k < ks) {
          const u16x8 a = ld_u16x8(s1 + k * 32);
          d = mfma16(a, qf[0][k], d);
          d = mfma16(a, qf[1][k], d);
          d = mfma16(ld_u16x8(s2 + k * 32), qf[0][k], d);
        }
#pragma unroll
      for (int jp = 0; jp < 2; ++jp) {
        if (!FULL && jp > (wid >> 1)) continue;  // zero there
        const u16x8 a = ld_u16x8(xl + (t * 16 + lo) * LP + jp * 32 + hi * 8);
        d = mfma16(a, af[0][jp], d);
        d = mfma16(a, af[1][jp], d);
      }
      if (row < row1) {
        const int p = t * 16 + hi * 4;
        uint16_t* dst = o + row * m.o_stride + h * m.E + p0 + p;
        if (m.vec) {
          const float v[4] = {d[0], d[1], d[2], d[3]};
          if (p < np) st_bf16x4(dst, v);
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (p + r < np) dst[r] = f32_to_bf16(d[r]);
        }
      }
    }
    // --- state
    if (FULL || pt * 16 < np) {
#pragma unroll
      for (int t = 0; t < ST; ++t)
        if (FULL || t < nts) {
          const f32x4 ee = *reinterpret_cast<const f32x4*>(
              el + (nt0 + t) * 16 + hi * 4);
#pragma unroll
          for (int r = 0; r < 4; ++r) S[t][r] *= ee[r];
        }
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const u16x8 x =
            ld_u16x8(xl + (pt * 16 + lo) * LP + kk * 32 + hi * 8);
#pragma unroll
        for (int t = 0; t < ST; ++t)
          if (FULL || t < nts) {
            const uint16_t* a =
                kl + ((nt0 + t) * 16 + lo) * LP + kk * 32 + hi * 8;
            S[t] = mfma16(ld_u16x8(a), x, S[t]);
            S[t] = mfma16(ld_u16x8(a + m.Dp * LP), x, S[t]);
          }
      }
    }
  }
  if (slot >= 0 && pcol < m.E) {
#pragma unroll
    for (int t = 0; t < ST; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = (nt0 + t) * 16 + hi * 4 + r;
        if (t < nts && n < m.D) st[(int64_t)n * m.Ep] = S[t][r];
      }
  }
}

// y <- scale * rms_norm(o per head) * w * silu(g); LN lanes have a head,
// each K vectors of N values.
template <int N, int K>
__global__ __launch_bounds__(NT) void head_norm_gate_kernel(
    uint16_t* __restrict__ y, const uint16_t* __restrict__ o,
    const uint16_t* __restrict__ g, const float* __restrict__ w,
    int64_t y_stride, int64_t g_stride, int H, int E, int LN, float scale,
    float eps, int64_t units) {
  const int64_t u = ((int64_t)blockIdx.x * NT + threadIdx.x) / LN;
  const int lane = threadIdx.x % LN;
  const bool live = u < units;
  const int64_t t = u / H;
  const int h = (int)(u - t * H);
  float v[K][N], ss = 0.f;
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int e = (k * LN + lane) * N;
    if (live && e < E) {
      const uint16_t* p = o + u * E + e;
      if constexpr (N == 1) v[k][0] = bf16_to_f32(*p); else ldv<N>(p, v[k]);
#pragma unroll
      for (int i = 0; i < N; ++i) ss += v[k][i] * v[k][i];
    }
  }
  for (int off = 1; off < LN; off *= 2) ss += __shfl_xor(ss, off, WAVE);
  const float inv = scale / sqrtf(ss / E + eps);
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int e = (k * LN + lane) * N;
    if (live && e < E) {
      const uint16_t* gp = g + t * g_stride + h * E + e;
      uint16_t* yp = y + t * y_stride + h * E + e;
      if constexpr (N == 1) {
        *yp = f32_to_bf16(v[k][0] * inv * w[e] *
                          silu_s<uint16_t>(bf16_to_f32(*gp)));
      } else {
        float x[N], c[N];
        ldv<N>(gp, x);
        ldv<N>(w + e, c);
#pragma unroll
        for (int i = 0; i < N; ++i)
          x[i] = v[k][i] * inv * c[i] * silu_s<uint16_t>(x[i]);
        stv<N>(yp, x);
      }
    }
  }
}

void check(const torch::Tensor& t, torch::ScalarType type, int64_t n) {
  TORCH_CHECK(t.scalar_type() == type && t.is_contiguous() && t.numel() == n,
              "gla chunks: operand of ", t.numel(), " values, want ", n);
}

// The operands' sizes; channels in Dp, values in Pp.
void check_operands(const torch::Tensor& qe, const torch::Tensor& ke,
                    const torch::Tensor& am, const torch::Tensor& vt,
                    const torch::Tensor& ec, int64_t D, int64_t E) {
  TORCH_CHECK(qe.dim() == 5 && vt.dim() == 4);
  const int64_t nh = qe.size(0) * qe.size(1), Dp = qe.size(4);
  const int64_t Pp = vt.size(2);
  TORCH_CHECK(D > 0 && D <= Dp && Dp % 32 == 0 && Dp <= 256 && E > 0 &&
              E <= Pp && Pp % 16 == 0);
  check(qe, torch::kBFloat16, nh * 2 * L * Dp);
  check(ke, torch::kBFloat16, nh * 2 * L * Dp);
  check(am, torch::kBFloat16, nh * 2 * L * L);
  check(vt, torch::kBFloat16, nh * Pp * L);
  check(ec, torch::kFloat32, nh * Dp);
}

}  // namespace

bool gla_chunks_fit(torch::Tensor z, int64_t dim) {
  return z.scalar_type() == torch::kBFloat16 && dim <= 256;
}

void gla_operands(torch::Tensor qe, torch::Tensor ke, torch::Tensor am,
                  torch::Tensor vt, torch::Tensor ec, torch::Tensor z,
                  int64_t q_at, int64_t k_at, int64_t v_at, int64_t a_at,
                  int64_t dim, int64_t vdim, int64_t rank, torch::Tensor a2,
                  torch::Tensor a2_b, double tau, double q_scale,
                  torch::Tensor row, torch::Tensor count) {
  check_operands(qe, ke, am, vt, ec, dim, vdim);
  const int64_t n = qe.size(0);
  Operands m{};
  m.H = qe.size(1);
  m.D = dim;
  m.Dp = qe.size(4);
  m.E = vdim;
  m.Pp = vt.size(2);
  m.rank = rank;
  m.rank_pad = a2.size(1);
  check(a2, torch::kBFloat16, (int64_t)m.rank_pad * m.H * m.D);
  TORCH_CHECK(rank >= 1 && rank <= m.rank_pad && m.rank_pad % 32 == 0);
  check(a2_b, torch::kFloat32, (int64_t)m.H * m.D);
  check(row, torch::kInt32, n);
  check(count, torch::kInt32, n);
  TORCH_CHECK(gla_chunks_fit(z, dim) && z.stride(1) == 1);
  const int64_t width = z.size(1);
  TORCH_CHECK(q_at + m.H * m.D <= width && k_at + m.H * m.D <= width &&
              v_at + m.H * m.E <= width && a_at + m.rank <= width);
  m.a2 = (const uint16_t*)a2.data_ptr();
  m.a2_b = a2_b.data_ptr<float>();
  m.row = row.data_ptr<int>();
  m.count = count.data_ptr<int>();
  m.z_stride = z.stride(0);
  m.q_at = q_at;
  m.k_at = k_at;
  m.v_at = v_at;
  m.a_at = a_at;
  m.unit = (float)(1.0 / tau);
  m.q_scale = (float)q_scale;
  m.vec = m.D % 8 == 0 && m.E % 8 == 0 && q_at % 8 == 0 && k_at % 8 == 0 &&
          v_at % 8 == 0 && a_at % 8 == 0 && m.z_stride % 8 == 0 &&
          (uintptr_t)z.data_ptr() % 16 == 0;
  if (n == 0) return;
  hipLaunchKernelGGL(gla_operands_kernel, dim3(n, m.H), dim3(NT), 0,
                     at::hip::getCurrentHIPStream(), (uint16_t*)qe.data_ptr(),
                     (uint16_t*)ke.data_ptr(), (uint16_t*)am.data_ptr(),
                     (uint16_t*)vt.data_ptr(), ec.data_ptr<float>(),
                     (const uint16_t*)z.data_ptr(), m);
}

void gla_chunks(torch::Tensor o, torch::Tensor qe, torch::Tensor ke,
                torch::Tensor am, torch::Tensor vt, torch::Tensor ec,
                int64_t vdim, torch::Tensor state, torch::Tensor slots,
                torch::Tensor pos, torch::Tensor cu, torch::Tensor first) {
  TORCH_CHECK(state.dim() == 4);
  Chunks m{};
  m.H = state.size(1);
  m.D = state.size(2);
  m.Ep = state.size(3);
  m.E = vdim;
  check_operands(qe, ke, am, vt, ec, m.D, m.E);
  m.Dp = qe.size(4);
  m.Pp = vt.size(2);
  const int64_t n = qe.size(0);
  const int B = slots.numel();
  TORCH_CHECK(qe.size(1) == m.H && m.Ep >= m.E);
  check(state, torch::kFloat32, state.numel());
  check(slots, torch::kInt32, B);
  check(cu, torch::kInt32, B + 1);
  check(first, torch::kInt32, B + 1);
  check(pos, torch::kInt64, o.size(0));
  TORCH_CHECK(o.dim() == 2 && o.stride(1) == 1 && o.size(1) == m.H * m.E &&
              o.scalar_type() == torch::kBFloat16);
  m.ec = ec.data_ptr<float>();
  m.state = state.data_ptr<float>();
  m.slots = slots.data_ptr<int>();
  m.pos = pos.data_ptr<int64_t>();
  m.cu = cu.data_ptr<int>();
  m.first = first.data_ptr<int>();
  m.o_stride = o.stride(0);
  m.vec = m.E % 4 == 0 && m.o_stride % 4 == 0 &&
          (uintptr_t)o.data_ptr() % 8 == 0;
  if (B == 0 || n == 0) return;
  // few heads and sequences: half the values to a workgroup
  const int PW = (int64_t)m.H * B * cdiv(m.E, 64) < 256 ? 2 : 4;
  const int PB = PW * 16;
  const dim3 grid(m.H, B, cdiv(m.E, PB));
  const int lds =
      (2 * m.Dp * LP + PB * LP + 2 * PB * (m.Dp + 8)) * 2 + m.Dp * 4;
  const bool full = m.E % PB == 0 && (m.Dp & (m.Dp - 1)) == 0;
#define HELIX_GC_F(NK, PW, FULL)                                             \
  do {                                                                       \
    static const hipError_t big = hipFuncSetAttribute(                       \
        (const void*)gla_chunks_kernel<NK, PW, FULL>,                        \
        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);             \
    TORCH_CHECK(big == hipSuccess, "LDS size refused");                      \
    hipLaunchKernelGGL((gla_chunks_kernel<NK, PW, FULL>), grid, dim3(NT),    \
                       lds,                                                  \
                       at::hip::getCurrentHIPStream(),                       \
                       (uint16_t*)o.data_ptr(),                              \
                       (const uint16_t*)qe.data_ptr(),                       \
                       (const uint16_t*)ke.data_ptr(),                       \
                       (const uint16_t*)am.data_ptr(),                       \
                       (const uint16_t*)vt.data_ptr(), m);                   \
  } while (0)
#define HELIX_GC_P(NK, PW)                                                   \
  if (full) HELIX_GC_F(NK, PW, true); else HELIX_GC_F(NK, PW, false)
#define HELIX_GC(NK)                                                         \
  if (PW == 4) { HELIX_GC_P(NK, 4); } else { HELIX_GC_P(NK, 2); }
  if (m.Dp <= 32) { HELIX_GC(1); }
  else if (m.Dp <= 64) { HELIX_GC(2); }
  else if (m.Dp <= 128) { HELIX_GC(4); }
  else { HELIX_GC(8); }
#undef HELIX_GC
#undef HELIX_GC_P
#undef HELIX_GC_F
}

void head_norm_gate(torch::Tensor y, torch::Tensor o, torch::Tensor g,
                    torch::Tensor w, double scale, double eps) {
  const int64_t T = o.size(0), E = w.numel();
  TORCH_CHECK(o.dim() == 2 && o.is_contiguous() && E > 0 && E <= 256 &&
              o.size(1) % E == 0);
  const int H = o.size(1) / E;
  for (const auto& t : {y, o, g})
    TORCH_CHECK(t.scalar_type() == torch::kBFloat16 && t.size(0) == T &&
                t.size(1) == o.size(1) && t.stride(1) == 1);
  check(w, torch::kFloat32, E);
  if (T == 0) return;
  const bool vec = E % 8 == 0 && y.stride(0) % 8 == 0 &&
                   g.stride(0) % 8 == 0 &&
                   (uintptr_t)y.data_ptr() % 16 == 0 &&
                   (uintptr_t)g.data_ptr() % 16 == 0;
  int LN = 1;
  while (LN < 64 && LN * (vec ? 8 : 1) < E) LN *= 2;
  const int64_t units = T * H;
  const dim3 grid((units * LN + NT - 1) / NT);
#define HELIX_HN(N, K)                                                       \
  hipLaunchKernelGGL((head_norm_gate_kernel<N, K>), grid, dim3(NT), 0,       \
                     at::hip::getCurrentHIPStream(),                         \
                     (uint16_t*)y.data_ptr(), (const uint16_t*)o.data_ptr(), \
                     (const uint16_t*)g.data_ptr(), w.data_ptr<float>(),     \
                     y.stride(0), g.stride(0), H, (int)E, LN, (float)scale,  \
                     (float)eps, units)
  if (vec) HELIX_HN(8, 1);
  else HELIX_HN(1, 4);
#undef HELIX_HN
}
