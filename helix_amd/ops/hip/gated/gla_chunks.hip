// Gated linear attention over prompt portions, 64 tokens at a time on MFMA.
//
// With c_t the running sum of a chunk's log decays (per key channel) and S
// the state that enters it:
//
//   o_i = S^T (q_i e^(c_i)) + sum_{j<=i} A_ij v_j
//   A_ij = sum_d q_i[d] k_j[d] e^(c_i[d] - c_j[d])
//   S  <- diag(e^(c_63)) S + sum_j (k_j e^(c_63 - c_j)) v_j^T
//
// gla_operands makes a chunk's operands. No exponent there is ever positive,
// however fast a channel decays: A's blocks of 16 x 16 off the diagonal take
// the start of the later block as reference, those on it multiply keys by
// one decay after another in fp32. gla_chunks carries a head's state from
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
constexpr int PA = 68;

struct Operands {
  const float *a2, *a2_b;      // [rank, H * D], [H * D]
  const int *row, *count;      // per chunk
  int64_t z_stride;
  int q_at, k_at, v_at, a_at, H, D, Dp, E, Pp, rank, vec;
  float inv_tau, q_scale;
};

// Columns c0 .. c0 + 31 of the chunk's rows, 8 per thread; nothing past
// column n or row count.
__device__ __forceinline__ void load_slice(float* v, const uint16_t* z,
                                           int64_t stride, int c0, int n,
                                           int count, bool vec) {
  const int t = threadIdx.x / 4, d = c0 + threadIdx.x % 4 * 8;
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = 0.f;
  if (t >= count) return;
  const uint16_t* p = z + t * stride + d;
  if (vec) {
    if (d < n) ldv<8>(p, v);
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (d + i < n) v[i] = bf16_to_f32(p[i]);
  }
}

// grid (chunks, heads)
__global__ __launch_bounds__(NT) void gla_operands_kernel(
    uint16_t* __restrict__ qe, uint16_t* __restrict__ ke,
    uint16_t* __restrict__ am, uint16_t* __restrict__ vt,
    float* __restrict__ ec, const uint16_t* __restrict__ z, Operands m) {
  extern __shared__ __attribute__((aligned(16))) float sh[];
  float* qs = sh;                             // [64][PV] queries
  float* al = qs + L * PV;                    // [64][PV] decays
  float* ks = al + L * PV;                    // [64][PS] keys (later values)
  float* cs = ks + L * PS;                    // [64][PS] log decays, summed
  float* pre = cs + L * PS;                   // [8][SL]
  float* a1 = pre + 8 * SL;                   // [64][rank]
  float* as = sh;                             // [64][PA] in the end
  const int n = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int count = m.count[n];
  const uint16_t* zr = z + (int64_t)m.row[n] * m.z_stride;
  const int64_t nh = (int64_t)n * m.H + h;
  uint16_t* qo = qe + nh * 2 * L * m.Dp;
  uint16_t* ko = ke + nh * 2 * L * m.Dp;

  for (int i = tid; i < L * m.rank; i += NT) {
    const int t = i / m.rank, r = i % m.rank;
    a1[i] = t < count ? bf16_to_f32(zr[t * m.z_stride + m.a_at + r]) : 0.f;
  }

  floatx4 off[2];                             // blocks wid, wid + 4 of six
  off[0] = off[1] = floatx4{0, 0, 0, 0};
  float dg[16];                               // diagonal block wid, column j
#pragma unroll
  for (int i = 0; i < 16; ++i) dg[i] = 0.f;
  const int j = lane >> 2, dq = (lane & 3) * 8;

  for (int d0 = 0; d0 < m.Dp; d0 += SL) {
    float v[8], w[8];
    const int t = tid / 4, s = tid % 4 * 8;
    load_slice(v, zr + m.q_at + h * m.D, m.z_stride, d0, m.D, count, m.vec);
    load_slice(w, zr + m.k_at + h * m.D, m.z_stride, d0, m.D, count, m.vec);
    __syncthreads();                          // the last slice is done
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[i] *= m.q_scale;
      ks[t * PS + s + i] = w[i];
    }
    stv<8>(qs + t * PV + s, v);
    {
      // decays: a thread has 8 tokens of a channel
      const int d = tid % SL, tg = tid / SL, c = d0 + d;
      float x[8], sum = 0.f;
      const float bias = c < m.D ? m.a2_b[h * m.D + c] : 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) x[i] = bias;
      if (c < m.D)
        for (int r = 0; r < m.rank; ++r) {
          const float wr = m.a2[(int64_t)r * m.H * m.D + h * m.D + c];
#pragma unroll
          for (int i = 0; i < 8; ++i)
            x[i] += a1[(tg * 8 + i) * m.rank + r] * wr;
        }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int tt = tg * 8 + i;
        const float g = tt < count && c < m.D
                            ? -softplus(-x[i]) * m.inv_tau : 0.f;
        sum += g;
        al[tt * PV + d] = expf(g);
        x[i] = sum;
      }
      pre[tg * SL + d] = sum;
      __syncthreads();
      float base = 0.f;
      for (int i = 0; i < tg; ++i) base += pre[i * SL + d];
#pragma unroll
      for (int i = 0; i < 8; ++i) cs[(tg * 8 + i) * PS + d] = base + x[i];
    }
    __syncthreads();
    // queries and keys with their decays
    u16x8 a, b;
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= expf(cs[t * PS + s + i]);
    split8(v, a, b);
    *reinterpret_cast<u16x8*>(qo + t * m.Dp + d0 + s) = a;
    *reinterpret_cast<u16x8*>(qo + (L + t) * m.Dp + d0 + s) = b;
    const int kd = tid / 8, kt = tid % 8 * 8;
    const float end = cs[(L - 1) * PS + kd];
#pragma unroll
    for (int i = 0; i < 8; ++i)
      w[i] = ks[(kt + i) * PS + kd] * expf(end - cs[(kt + i) * PS + kd]);
    split8(w, a, b);
    *reinterpret_cast<u16x8*>(ko + (d0 + kd) * L + kt) = a;
    *reinterpret_cast<u16x8*>(ko + (m.Dp + d0 + kd) * L + kt) = b;
    if (tid < SL) ec[nh * m.Dp + d0 + tid] = expf(cs[(L - 1) * PS + tid]);

    // diagonal block: key j meets queries i >= j, decaying on the way
    float kk[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) kk[i] = ks[(wid * 16 + j) * PS + dq + i];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float q[8], g[8], sum = 0.f;
      ldv<8>(qs + (wid * 16 + i) * PV + dq, q);
      ldv<8>(al + (wid * 16 + i) * PV + dq, g);
#pragma unroll
      for (int c = 0; c < 8; ++c) {
        kk[c] *= i > j ? g[c] : 1.f;
        sum += q[c] * kk[c];
      }
      dg[i] += i >= j ? sum : 0.f;
    }
    // blocks (I, J), I > J: rows j of the result, columns i
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int blk = wid + u * 4;
      if (blk >= 6) continue;
      const int I = blk < 1 ? 1 : (blk < 3 ? 2 : 3);
      const int J = blk - I * (I - 1) / 2;
      float q[8], k[8];
#pragma unroll
      for (int c = 0; c < 8; ++c) {
        const int d = hi * 8 + c;
        const float ref = cs[(I * 16 - 1) * PS + d];
        q[c] = qs[(I * 16 + lo) * PV + d] *
               expf(cs[(I * 16 + lo) * PS + d] - ref);
        k[c] = ks[(J * 16 + lo) * PS + d] *
               expf(ref - cs[(J * 16 + lo) * PS + d]);
      }
      u16x8 qh, ql, kh, kl;
      split8(q, qh, ql);
      split8(k, kh, kl);
      off[u] = mfma16(kh, qh, off[u]);
      off[u] = mfma16(kh, ql, off[u]);
      off[u] = mfma16(kl, qh, off[u]);
    }
  }

  // the score matrix, through LDS
  __syncthreads();
  for (int i = tid; i < L * PA; i += NT) as[i] = 0.f;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    float x = dg[i];
    x += __shfl_xor(x, 1, WAVE);
    x += __shfl_xor(x, 2, WAVE);
    if ((lane & 3) == 0) as[(wid * 16 + i) * PA + wid * 16 + j] = x;
  }
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int blk = wid + u * 4;
    if (blk >= 6) continue;
    const int I = blk < 1 ? 1 : (blk < 3 ? 2 : 3);
    const int J = blk - I * (I - 1) / 2;
    *reinterpret_cast<floatx4*>(as + (I * 16 + lo) * PA + J * 16 + hi * 4) =
        off[u];
  }
  __syncthreads();
  uint16_t* ao = am + nh * 2 * L * L;
  {
    const int i = tid / 4, c0 = tid % 4 * 16;
#pragma unroll
    for (int c = 0; c < 16; c += 8) {
      float v[8];
      ldv<8>(as + i * PA + c0 + c, v);
      u16x8 a, b;
      split8(v, a, b);
      *reinterpret_cast<u16x8*>(ao + i * L + c0 + c) = a;
      *reinterpret_cast<u16x8*>(ao + (L + i) * L + c0 + c) = b;
    }
  }
  // values, transposed
  for (int e0 = 0; e0 < m.Pp; e0 += SL) {
    float v[8];
    load_slice(v, zr + m.v_at + h * m.E, m.z_stride, e0, m.E, count, m.vec);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 8; ++i) ks[tid / 4 * PS + tid % 4 * 8 + i] = v[i];
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

// NK: 32-wide steps of the key channels; PW: 16-value tiles of a workgroup.
// Wave w has tokens 16 w .. of the output, and of the state the value tile
// w % PW in its share of the rows.
template <int NK, int PW>
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

  u16x8 kreg[KR], qreg[2][NK], areg[2][2], xreg[XL];
  float ereg = 0.f;
  // No branches, so that all loads are under way at once: indices past the
  // end are clamped and their values not stored or not used.
  auto load = [&](int n) {
    const int64_t nh = (int64_t)n * m.H + h;
    const uint16_t* kn = ke + nh * 2 * L * m.Dp;
#pragma unroll
    for (int i = 0; i < KR; ++i)
      kreg[i] = ld_u16x8(kn + min(i * NT + tid, m.Dp * 16 - 1) * 8);
    const uint16_t* qn = qe + (nh * 2 * L + wid * 16 + lo) * m.Dp + hi * 8;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int k = 0; k < NK; ++k)
        qreg[s][k] = ld_u16x8(qn + (int64_t)s * L * m.Dp + min(k, ks - 1) * 32);
      const uint16_t* an =
          am + ((nh * 2 + s) * L + wid * 16 + lo) * L + hi * 8;
      areg[s][0] = ld_u16x8(an);
      areg[s][1] = ld_u16x8(an + 32);
    }
    const uint16_t* xn = vt + (nh * m.Pp + p0) * L;
#pragma unroll
    for (int i = 0; i < XL; ++i)
      xreg[i] = ld_u16x8(xn + min(i * NT + tid, rowsp * 8 - 1) * 8);
    ereg = m.ec[nh * m.Dp + min(tid, m.Dp - 1)];
  };

  load(n0);
  for (int n = n0; n < n1; ++n) {
    __syncthreads();                          // the last chunk is done
#pragma unroll
    for (int i = 0; i < KR; ++i) {
      const int e = i * NT + tid;
      if (e < m.Dp * 16)
        *reinterpret_cast<u16x8*>(kl + e / 8 * LP + e % 8 * 8) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < XL; ++i) {
      const int e = i * NT + tid;
      *reinterpret_cast<u16x8*>(xl + e / 8 * LP + e % 8 * 8) = xreg[i];
    }
    if (tid < m.Dp) el[tid] = ereg;
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
    u16x8 qf[2][NK], af[2][2];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int k = 0; k < NK; ++k) qf[s][k] = qreg[s][k];
      af[s][0] = areg[s][0];
      af[s][1] = areg[s][1];
    }
    __syncthreads();
    if (n + 1 < n1) load(n + 1);

    // --- outputs, transposed: lane has token i, values 4 hi + r
    const int i = wid * 16 + lo;
    const int64_t row = row0 + (int64_t)(n - n0) * L + i;
#pragma unroll
    for (int t = 0; t < PW; ++t) {
      if (t * 16 >= np) continue;
      floatx4 d = floatx4{0, 0, 0, 0};
      const uint16_t* s1 = sh + (t * 16 + lo) * NP + hi * 8;
      const uint16_t* s2 = sl + (t * 16 + lo) * NP + hi * 8;
#pragma unroll
      for (int k = 0; k < NK; ++k)
        if (k < ks) {
          const u16x8 a = ld_u16x8(s1 + k * 32);
          d = mfma16(a, qf[0][k], d);
          d = mfma16(a, qf[1][k], d);
          d = mfma16(ld_u16x8(s2 + k * 32), qf[0][k], d);
        }
#pragma unroll
      for (int jp = 0; jp < 2; ++jp) {
        if (jp > (wid >> 1)) continue;
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
    if (pt * 16 < np) {
#pragma unroll
      for (int t = 0; t < ST; ++t)
        if (t < nts) {
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
          if (t < nts) {
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
                  int64_t dim, int64_t vdim, torch::Tensor a2,
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
  m.rank = a2.size(0);
  check(a2, torch::kFloat32, (int64_t)m.rank * m.H * m.D);
  check(a2_b, torch::kFloat32, (int64_t)m.H * m.D);
  check(row, torch::kInt32, n);
  check(count, torch::kInt32, n);
  TORCH_CHECK(gla_chunks_fit(z, dim) && z.stride(1) == 1);
  const int64_t width = z.size(1);
  TORCH_CHECK(q_at + m.H * m.D <= width && k_at + m.H * m.D <= width &&
              v_at + m.H * m.E <= width && a_at + m.rank <= width);
  m.a2 = a2.data_ptr<float>();
  m.a2_b = a2_b.data_ptr<float>();
  m.row = row.data_ptr<int>();
  m.count = count.data_ptr<int>();
  m.z_stride = z.stride(0);
  m.q_at = q_at;
  m.k_at = k_at;
  m.v_at = v_at;
  m.a_at = a_at;
  m.inv_tau = (float)(1.0 / tau);
  m.q_scale = (float)q_scale;
  m.vec = m.D % 8 == 0 && m.E % 8 == 0 && q_at % 8 == 0 && k_at % 8 == 0 &&
          v_at % 8 == 0 && m.z_stride % 8 == 0 &&
          (uintptr_t)z.data_ptr() % 16 == 0;
  if (n == 0) return;
  const int lds = (2 * L * PV + 2 * L * PS + 8 * SL + L * m.rank) * 4;
  TORCH_CHECK(m.rank >= 1 && lds <= 160 * 1024, "rank ", m.rank);
  static const hipError_t big = hipFuncSetAttribute(
      (const void*)gla_operands_kernel,
      hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  TORCH_CHECK(big == hipSuccess, "LDS size refused");
  hipLaunchKernelGGL(gla_operands_kernel, dim3(n, m.H), dim3(NT), lds,
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
#define HELIX_GC_P(NK, PW)                                                   \
  do {                                                                       \
    static const hipError_t big = hipFuncSetAttribute(                       \
        (const void*)gla_chunks_kernel<NK, PW>,                              \
        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);             \
    TORCH_CHECK(big == hipSuccess, "LDS size refused");                      \
    hipLaunchKernelGGL((gla_chunks_kernel<NK, PW>), grid, dim3(NT), lds,     \
                       at::hip::getCurrentHIPStream(),                       \
                       (uint16_t*)o.data_ptr(),                              \
                       (const uint16_t*)qe.data_ptr(),                       \
                       (const uint16_t*)ke.data_ptr(),                       \
                       (const uint16_t*)am.data_ptr(),                       \
                       (const uint16_t*)vt.data_ptr(), m);                   \
  } while (0)
#define HELIX_GC(NK)                                                         \
  if (PW == 4) HELIX_GC_P(NK, 4); else HELIX_GC_P(NK, 2)
  if (m.Dp <= 32) { HELIX_GC(1); }
  else if (m.Dp <= 64) { HELIX_GC(2); }
  else if (m.Dp <= 128) { HELIX_GC(4); }
  else { HELIX_GC(8); }
#undef HELIX_GC
#undef HELIX_GC_P
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
