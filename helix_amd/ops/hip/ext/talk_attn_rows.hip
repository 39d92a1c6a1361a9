// Paged attention with talking heads, one query row at a time (decode).
//
// Talking heads mix the SOFTMAXED weights of all heads before they meet the
// values, so a head's output needs every head's denominator. Flash-decoding
// partials cannot be mixed after the fact without carrying H x G value sums,
// so the row is done in two streams over the window instead:
//
//   scores  s[h, j] = cap(q_h . k_j * scale) - slope_h * (i - j), fp32 to
//           scratch, with per-partition (max, sum). Reads K once.
//   values  p = exp(s - M) / L for all heads, w_h = sum_g talk[h, g] p_g in
//           fp32, out_h += w_h v. Reads V once; partitions simply add.
//   reduce  adds the partitions, applies the output gate, writes the row
//           (done by the value kernel itself when there is one partition).
//
// Scratch traffic is H*4 bytes per key against 2*G*(D+E) bytes of K/V.
// Grid: (rows, kv heads x head chunks, partitions); the partition count is
// sized by the host so small batches still fill the 256 CUs. Compiled for
// bf16 and fp32 storage; all math is fp32.
//
// bf16 runs both streams on MFMA, which is idle otherwise and keeps the VALU
// out of the way of the loads:
//
//   scores  4 tiles of 16 keys accumulate into ONE 16x16 result: tile u's
//           A operand holds the 4 queries in rows 4u..4u+3 and zeros
//           elsewhere, so lane (hi, lo) ends up with the 4 heads of key
//           16 hi + lo: a lane per key, no lane idle.
//   values  the mixed weights are the A operand, split into two bf16 terms
//           (17 significant bits), V pages are B operands as they lie.
//
// Cache layout: K [nblk, G, bs, Dp]; V [nblk, G, E, bs] (8 tokens of one
// value dim are one 16-byte load).
#include "../elem.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int NT = 128;
constexpr int NWV = NT / WAVE;
constexpr int CHUNK = 128;
constexpr int QUANT = 128;     // partition granularity in tokens
constexpr float NEG = -1e30f;

struct RowGeom {
  const int* bt;               // [.., bt_stride]
  int bt_stride;
  const int* row_seq;          // [R] block-table row; null: row index
  const int* row_len;          // [R] keys the row may see (own included)
  int window, H, G, bs, span, part, max_parts, hchunks;
};

// Per-thread (max, sum) of HC heads -> one pair per partition.
template <typename S, int HC>
__device__ __forceinline__ void store_stats(const float (&mx)[HC],
                                            const float (&sm)[HC],
                                            float (&red)[2][HC][NWV], int nh,
                                            float* ml, int64_t head0,
                                            int max_parts, int part) {
  const int wid = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
#pragma unroll
  for (int i = 0; i < HC; ++i) {
    const float wm = wave_reduce_max(mx[i]);
    const float ws = wave_reduce_sum(sm[i] * exp_s<S>(mx[i] - wm));
    if (lane == 0) {
      red[0][i][wid] = wm;
      red[1][i][wid] = ws;
    }
  }
  __syncthreads();
  if ((int)threadIdx.x < nh) {
    const int i = threadIdx.x;
    float M = NEG, L = 0.f;
    for (int w = 0; w < NWV; ++w) M = fmaxf(M, red[0][i][w]);
    for (int w = 0; w < NWV; ++w)
      L += red[1][i][w] * exp_s<S>(red[0][i][w] - M);
    float* o = ml + ((head0 + i) * max_parts + part) * 2;
    o[0] = M;
    o[1] = L;
  }
}

// Score pass, a thread per key.
template <typename S, int HC>
__global__ __launch_bounds__(NT) void row_scores_kernel(
    float* __restrict__ scores, float* __restrict__ ml,
    const S* __restrict__ q, const S* __restrict__ kc,
    const float* __restrict__ slopes, float scale, float cap, int Dp,
    RowGeom m) {
  extern __shared__ float q_lds[];            // [HC][Dp]
  __shared__ float red[2][HC][NWV];
  const int row = blockIdx.x, part = blockIdx.z;
  const int g = blockIdx.y / m.hchunks, hc = blockIdx.y % m.hchunks;
  const int HG = m.H / m.G;
  const int h0 = g * HG + hc * HC;
  const int nh = min(HC, HG - hc * HC);
  const int len = m.row_len[row];
  const int lo = m.window > 0 ? max(0, len - m.window) : 0;
  const int p0 = lo + part * m.part;
  const int p1 = min(len, p0 + m.part);
  if (p0 >= len) return;                      // nobody reads this partition
  for (int i = threadIdx.x; i < nh * Dp; i += NT)
    q_lds[i] = ld1(q + ((int64_t)row * m.H + h0) * Dp + i);
  for (int i = nh * Dp + threadIdx.x; i < HC * Dp; i += NT) q_lds[i] = 0.f;
  __syncthreads();

  const int* bt =
      m.bt + (int64_t)(m.row_seq ? m.row_seq[row] : row) * m.bt_stride;
  const float inv_cap = cap > 0.f ? 1.f / cap : 0.f;
  float slope[HC], mx[HC], sm[HC];
#pragma unroll
  for (int i = 0; i < HC; ++i) {
    slope[i] = (slopes != nullptr && i < nh) ? slopes[h0 + i] : 0.f;
    mx[i] = NEG;
    sm[i] = 0.f;
  }
  for (int tok = p0 + threadIdx.x; tok < p1; tok += CHUNK) {
    const S* krow =
        kc + (((int64_t)bt[tok / m.bs] * m.G + g) * m.bs + tok % m.bs) * Dp;
    float acc[HC];
#pragma unroll
    for (int i = 0; i < HC; ++i) acc[i] = 0.f;
    for (int j = 0; j < Dp; j += 8) {
      float k[8];
      ldv<8>(krow + j, k);
#pragma unroll
      for (int i = 0; i < HC; ++i)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[i] += q_lds[i * Dp + j + e] * k[e];
    }
#pragma unroll
    for (int i = 0; i < HC; ++i) {
      if (i < nh) {
        const float s = cap_and_bias<S>(acc[i], scale, cap, inv_cap,
                                        slope[i], len - 1 - tok);
        scores[((int64_t)row * m.H + h0 + i) * m.span + tok - lo] = s;
        const float mn = fmaxf(mx[i], s);
        sm[i] = sm[i] * exp_s<S>(mx[i] - mn) + exp_s<S>(s - mn);
        mx[i] = mn;
      }
    }
  }
  store_stats<S, HC>(mx, sm, red, nh, ml, (int64_t)row * m.H + h0,
                     m.max_parts, part);
}

// Score pass on MFMA. DT k-steps of 32 (Dp <= 32*DT); HC a multiple of 4.
template <int DT, int HC>
__global__ __launch_bounds__(NT) void row_scores_mfma_kernel(
    float* __restrict__ scores, float* __restrict__ ml,
    const uint16_t* __restrict__ q, const uint16_t* __restrict__ kc,
    const float* __restrict__ slopes, float scale, float cap, int Dp,
    RowGeom m) {
  __shared__ float red[2][HC][NWV];
  const int row = blockIdx.x, part = blockIdx.z;
  const int g = blockIdx.y / m.hchunks, hc = blockIdx.y % m.hchunks;
  const int HG = m.H / m.G;
  const int h0 = g * HG + hc * HC;
  const int nh = min(HC, HG - hc * HC);
  const int len = m.row_len[row];
  const int lo_key = m.window > 0 ? max(0, len - m.window) : 0;
  const int p0 = lo_key + part * m.part;
  const int p1 = min(len, p0 + m.part);
  if (p0 >= len) return;
  const int wid = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;

  // lane lo feeds head lo & 3 of every group of 4
  u16x8 qf[HC / 4][DT];
#pragma unroll
  for (int j = 0; j < HC / 4; ++j)
#pragma unroll
    for (int kt = 0; kt < DT; ++kt) {
      const int h = j * 4 + (lo & 3), d = kt * 32 + hi * 8;
      qf[j][kt] = h < nh && d < Dp
                      ? *reinterpret_cast<const u16x8*>(
                            q + ((int64_t)row * m.H + h0 + h) * Dp + d)
                      : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  const int* bt =
      m.bt + (int64_t)(m.row_seq ? m.row_seq[row] : row) * m.bt_stride;
  const float inv_cap = cap > 0.f ? 1.f / cap : 0.f;
  float slope[HC], mx[HC], sm[HC];
#pragma unroll
  for (int i = 0; i < HC; ++i) {
    slope[i] = (slopes != nullptr && i < nh) ? slopes[h0 + i] : 0.f;
    mx[i] = NEG;
    sm[i] = 0.f;
  }
  for (int base = p0 + wid * WAVE; base < p1; base += NWV * WAVE) {
    u16x8 kf[4][DT];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int tok = min(base + u * 16 + lo, p1 - 1);
      const uint16_t* kr =
          kc + (((int64_t)bt[tok / m.bs] * m.G + g) * m.bs + tok % m.bs) * Dp +
          hi * 8;
#pragma unroll
      for (int kt = 0; kt < DT; ++kt)
        kf[u][kt] = kt * 32 + hi * 8 < Dp
                        ? *reinterpret_cast<const u16x8*>(kr + kt * 32)
                        : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
    const int tok = base + lane;
#pragma unroll
    for (int j = 0; j < HC / 4; ++j) {
      floatx4 c = floatx4{0, 0, 0, 0};
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int kt = 0; kt < DT; ++kt) {
          u16x8 a = (lo >> 2) == u ? qf[j][kt]
                                   : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
          c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              *reinterpret_cast<bf16x8*>(&a),
              *reinterpret_cast<bf16x8*>(&kf[u][kt]), c, 0, 0, 0);
        }
      if (tok < p1) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = j * 4 + r;
          if (i < nh) {
            const float s = cap_and_bias<uint16_t>(
                c[r], scale, cap, inv_cap, slope[i], len - 1 - tok);
            scores[((int64_t)row * m.H + h0 + i) * m.span + tok - lo_key] = s;
            const float mn = fmaxf(mx[i], s);
            sm[i] = sm[i] * __expf(mx[i] - mn) + __expf(s - mn);
            mx[i] = mn;
          }
        }
      }
    }
  }
  store_stats<uint16_t, HC>(mx, sm, red, nh, ml, (int64_t)row * m.H + h0,
                            m.max_parts, part);
}

// Denominators of all heads and this workgroup's rows of the mixing matrix.
template <typename S, int HC>
__device__ __forceinline__ void load_mixing(float* M_lds, float* I_lds,
                                            float* T_lds, const float* ml,
                                            const float* talk, int row,
                                            int h0, int nh, int np,
                                            const RowGeom& m) {
  for (int h = threadIdx.x; h < m.H; h += NT) {
    const float* s = ml + ((int64_t)row * m.H + h) * m.max_parts * 2;
    float M = NEG, L = 0.f;
    for (int p = 0; p < np; ++p) M = fmaxf(M, s[2 * p]);
    for (int p = 0; p < np; ++p) L += s[2 * p + 1] * exp_s<S>(s[2 * p] - M);
    M_lds[h] = M;
    I_lds[h] = 1.f / L;
  }
  for (int i = threadIdx.x; i < m.H * HC; i += NT) {
    const int h = i / HC, c = i % HC;
    float t = 0.f;
    if (c < nh)
      t = talk != nullptr ? talk[(int64_t)(h0 + c) * m.H + h]
                          : (h == h0 + c ? 1.f : 0.f);
    T_lds[i] = t;
  }
  __syncthreads();
}

// w[i] += sum over all heads of talk * softmax weight, for one key whose
// scores start at s.
template <typename S, int HC>
__device__ __forceinline__ void mixed_weights(float (&w)[HC], const float* s,
                                              const float* M_lds,
                                              const float* I_lds,
                                              const float* T_lds,
                                              const RowGeom& m) {
#pragma unroll 8
  for (int h = 0; h < m.H; ++h) {
    const float p = exp_s<S>(s[(int64_t)h * m.span] - M_lds[h]) * I_lds[h];
#pragma unroll
    for (int i = 0; i < HC; ++i) w[i] += T_lds[h * HC + i] * p;
  }
}

// Value pass. w_lds holds the mixed weights of this workgroup's heads for
// one chunk; positions outside [p0, p1) weigh 0, so V is read in aligned
// groups of 8 tokens. Threads own value dims (one dim each, strided).
template <typename S, int HC>
__global__ __launch_bounds__(NT) void row_values_kernel(
    S* __restrict__ out, int64_t out_stride, float* __restrict__ tmp,
    const float* __restrict__ scores, const float* __restrict__ ml,
    const S* __restrict__ vc, const float* __restrict__ talk,
    const S* __restrict__ gate, int64_t gate_stride, int E, int nparts,
    RowGeom m) {
  extern __shared__ __attribute__((aligned(16))) float sh[];
  float* w_lds = sh;                          // [HC][CHUNK + 8]
  float* M_lds = w_lds + HC * (CHUNK + 8);    // [H]
  float* I_lds = M_lds + m.H;                 // [H] 1 / denominator
  float* T_lds = I_lds + m.H;                 // [H][HC] mixing columns
  const int row = blockIdx.x, part = blockIdx.z;
  const int g = blockIdx.y / m.hchunks, hc = blockIdx.y % m.hchunks;
  const int HG = m.H / m.G;
  const int h0 = g * HG + hc * HC;
  const int nh = min(HC, HG - hc * HC);
  const int len = m.row_len[row];
  const int lo = m.window > 0 ? max(0, len - m.window) : 0;
  const int p0 = lo + part * m.part;
  const int p1 = min(len, p0 + m.part);
  if (p0 >= len) return;
  load_mixing<S, HC>(M_lds, I_lds, T_lds, ml, talk, row, h0, nh,
                     cdiv(len - lo, m.part), m);
  const int* bt =
      m.bt + (int64_t)(m.row_seq ? m.row_seq[row] : row) * m.bt_stride;
  constexpr int ND = 4;                       // dims per thread: E <= 512
  float acc[ND][HC];
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int i = 0; i < HC; ++i) acc[d][i] = 0.f;

  // chunks start on 8-token boundaries
  for (int base = p0 & ~7; base < p1; base += CHUNK) {
    {
      const int tok = base + threadIdx.x;
      float w[HC];
#pragma unroll
      for (int i = 0; i < HC; ++i) w[i] = 0.f;
      if (tok >= p0 && tok < p1)
        mixed_weights<S, HC>(
            w, scores + (int64_t)row * m.H * m.span + tok - lo, M_lds, I_lds,
            T_lds, m);
#pragma unroll
      for (int i = 0; i < HC; ++i) w_lds[i * (CHUNK + 8) + threadIdx.x] = w[i];
    }
    __syncthreads();
    const int n8 = (min(CHUNK, p1 - base) + 7) / 8;
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      const int dim = d * NT + threadIdx.x;
      if (dim < E) {
#pragma unroll 4
        for (int j = 0; j < n8; ++j) {
          const int t8 = base + j * 8;
          float v[8];
          ldv<8>(vc + (((int64_t)bt[t8 / m.bs] * m.G + g) * E + dim) * m.bs +
                     t8 % m.bs, v);
          const int live = p1 - t8;           // stale tail: not even 0 * x
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const float ve = e < live ? v[e] : 0.f;
#pragma unroll
            for (int i = 0; i < HC; ++i)
              acc[d][i] += w_lds[i * (CHUNK + 8) + j * 8 + e] * ve;
          }
        }
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int d = 0; d < ND; ++d) {
    const int dim = d * NT + threadIdx.x;
    if (dim >= E) continue;
#pragma unroll
    for (int i = 0; i < HC; ++i) {
      if (i >= nh) continue;
      const int h = h0 + i;
      if (nparts == 1) {
        float o = acc[d][i];
        if (gate != nullptr)
          o /= 1.f + exp_s<S>(-ld1(gate + row * gate_stride + h));
        st1(out + row * out_stride + (int64_t)h * E + dim, o);
      } else {
        tmp[(((int64_t)row * m.H + h) * m.max_parts + part) * E + dim] =
            acc[d][i];
      }
    }
  }
}

// Value pass on MFMA (bf16). Waves own value tiles of 16 dims, ET of them at
// most (E <= 32 * ET for the 2 waves).
template <int ET, int HC>
__global__ __launch_bounds__(NT) void row_values_mfma_kernel(
    uint16_t* __restrict__ out, int64_t out_stride, float* __restrict__ tmp,
    const float* __restrict__ scores, const float* __restrict__ ml,
    const uint16_t* __restrict__ vc, const float* __restrict__ talk,
    const uint16_t* __restrict__ gate, int64_t gate_stride, int E, int nparts,
    RowGeom m) {
  extern __shared__ __attribute__((aligned(16))) float sh[];
  constexpr int WPITCH = CHUNK + 8;
  float* M_lds = sh;                          // [H]
  float* I_lds = M_lds + m.H;                 // [H] 1 / denominator
  float* T_lds = I_lds + m.H;                 // [H][HC] mixing columns
  __shared__ __attribute__((aligned(16))) uint16_t w_hi[HC * WPITCH];
  __shared__ __attribute__((aligned(16))) uint16_t w_lo[HC * WPITCH];
  const int row = blockIdx.x, part = blockIdx.z;
  const int g = blockIdx.y / m.hchunks, hc = blockIdx.y % m.hchunks;
  const int HG = m.H / m.G;
  const int h0 = g * HG + hc * HC;
  const int nh = min(HC, HG - hc * HC);
  const int len = m.row_len[row];
  const int lo_key = m.window > 0 ? max(0, len - m.window) : 0;
  const int p0 = lo_key + part * m.part;
  const int p1 = min(len, p0 + m.part);
  if (p0 >= len) return;
  load_mixing<uint16_t, HC>(M_lds, I_lds, T_lds, ml, talk, row, h0, nh,
                            cdiv(len - lo_key, m.part), m);
  const int* bt =
      m.bt + (int64_t)(m.row_seq ? m.row_seq[row] : row) * m.bt_stride;
  const int wid = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  floatx4 acc[ET];
#pragma unroll
  for (int c = 0; c < ET; ++c) acc[c] = floatx4{0, 0, 0, 0};

  for (int base = p0 & ~7; base < p1; base += CHUNK) {
    const int n32 = (min(CHUNK, p1 - base) + 31) / 32;
    {
      const int tok = base + threadIdx.x;
      float w[HC];
#pragma unroll
      for (int i = 0; i < HC; ++i) w[i] = 0.f;
      if (tok >= p0 && tok < p1)
        mixed_weights<uint16_t, HC>(
            w, scores + (int64_t)row * m.H * m.span + tok - lo_key, M_lds,
            I_lds, T_lds, m);
#pragma unroll
      for (int i = 0; i < HC; ++i) {
        const uint32_t h = pack_bf16(w[i], 0.f);
        w_hi[i * WPITCH + threadIdx.x] = (uint16_t)h;
        w_lo[i * WPITCH + threadIdx.x] = (uint16_t)pack_bf16(
            w[i] - __builtin_bit_cast(float, h << 16), 0.f);
      }
    }
    __syncthreads();
#pragma unroll 2
    for (int j = 0; j < n32; ++j) {
      const int t8 = base + j * 32 + hi * 8;
      const int tv = min(t8, (p1 - 1) & ~7);
      const uint16_t* vp =
          vc + (((int64_t)bt[tv / m.bs] * m.G + g) * E + lo) * m.bs +
          tv % m.bs;
      u16x8 vf[ET];
#pragma unroll
      for (int c = 0; c < ET; ++c) {
        const int dim0 = (c * NWV + wid) * 16;
        vf[c] = dim0 + lo < E ? *reinterpret_cast<const u16x8*>(
                                    vp + (int64_t)dim0 * m.bs)
                              : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
      }
      u16x8 ah = u16x8{0, 0, 0, 0, 0, 0, 0, 0}, al = ah;
      if (lo < HC) {
        ah = *reinterpret_cast<const u16x8*>(w_hi + lo * WPITCH + j * 32 +
                                             hi * 8);
        al = *reinterpret_cast<const u16x8*>(w_lo + lo * WPITCH + j * 32 +
                                             hi * 8);
      }
      const bool tail = base + j * 32 + 32 > p1;
#pragma unroll
      for (int c = 0; c < ET; ++c) {
        if (tail) {                           // stale slots: not even 0 * x
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if (t8 + e >= p1) vf[c][e] = 0;
        }
        const bf16x8 b = *reinterpret_cast<bf16x8*>(&vf[c]);
        acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            *reinterpret_cast<bf16x8*>(&al), b, acc[c], 0, 0, 0);
        acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            *reinterpret_cast<bf16x8*>(&ah), b, acc[c], 0, 0, 0);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int c = 0; c < ET; ++c) {
    const int dim = (c * NWV + wid) * 16 + lo;
    if (dim >= E) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = hi * 4 + r;
      if (i >= nh) continue;
      const int h = h0 + i;
      if (nparts == 1) {
        float o = acc[c][r];
        if (gate != nullptr)
          o /= 1.f + __expf(-bf16_to_f32(gate[row * gate_stride + h]));
        out[row * out_stride + (int64_t)h * E + dim] = f32_to_bf16(o);
      } else {
        tmp[(((int64_t)row * m.H + h) * m.max_parts + part) * E + dim] =
            acc[c][r];
      }
    }
  }
}

template <typename S>
__global__ __launch_bounds__(NT) void row_reduce_kernel(
    S* __restrict__ out, int64_t out_stride, const float* __restrict__ tmp,
    const S* __restrict__ gate, int64_t gate_stride, int E, RowGeom m) {
  const int row = blockIdx.x, h = blockIdx.y;
  const int len = m.row_len[row];
  const int lo = m.window > 0 ? max(0, len - m.window) : 0;
  const int np = cdiv(len - lo, m.part);
  const float* t = tmp + ((int64_t)row * m.H + h) * m.max_parts * E;
  float f = 1.f;
  if (gate != nullptr)
    f = 1.f / (1.f + exp_s<S>(-ld1(gate + row * gate_stride + h)));
  for (int d = threadIdx.x; d < E; d += NT) {
    float o = 0.f;
    for (int p = 0; p < np; ++p) o += t[(int64_t)p * E + d];
    st1(out + row * out_stride + (int64_t)h * E + d, o * f);
  }
}

template <typename S>
struct RowCall {
  S* out;
  int64_t out_stride;
  const S *q, *kc, *vc, *gate;
  int64_t gate_stride;
  const float *slopes, *talk;
  float *scores, *ml, *tmp;
  float scale, cap;
  int R, D, E, nparts;
  RowGeom m;
  hipStream_t stream;
};

template <typename S, int HC>
void launch_rows(RowCall<S>& c) {
  c.m.hchunks = cdiv(c.m.H / c.m.G, HC);
  const dim3 grid(c.R, c.m.G * c.m.hchunks, c.nparts);
  const size_t q_bytes = (size_t)HC * c.D * sizeof(float);
  hipLaunchKernelGGL((row_scores_kernel<S, HC>), grid, dim3(NT), q_bytes,
                     c.stream, c.scores, c.ml, c.q, c.kc, c.slopes, c.scale,
                     c.cap, c.D, c.m);
  const size_t v_bytes =
      (HC * (CHUNK + 8) + (2 + HC) * c.m.H) * sizeof(float);
  hipLaunchKernelGGL((row_values_kernel<S, HC>), grid, dim3(NT), v_bytes,
                     c.stream, c.out, c.out_stride, c.tmp, c.scores, c.ml,
                     c.vc, c.talk, c.gate, c.gate_stride, c.E, c.nparts, c.m);
  if (c.nparts > 1)
    hipLaunchKernelGGL((row_reduce_kernel<S>), dim3(c.R, c.m.H), dim3(NT), 0,
                       c.stream, c.out, c.out_stride, c.tmp, c.gate,
                       c.gate_stride, c.E, c.m);
}

template <int HC>
void launch_rows_mfma(RowCall<uint16_t>& c) {
  c.m.hchunks = cdiv(c.m.H / c.m.G, HC);
  const dim3 grid(c.R, c.m.G * c.m.hchunks, c.nparts);
#define HELIX_SCORES(DT)                                                     \
  hipLaunchKernelGGL((row_scores_mfma_kernel<DT, HC>), grid, dim3(NT), 0,    \
                     c.stream, c.scores, c.ml, c.q, c.kc, c.slopes, c.scale, \
                     c.cap, c.D, c.m)
  if (c.D <= 64) HELIX_SCORES(2);
  else HELIX_SCORES(4);
#undef HELIX_SCORES
  const size_t bytes = (2 + HC) * c.m.H * sizeof(float);
#define HELIX_VALUES(ET)                                                     \
  hipLaunchKernelGGL((row_values_mfma_kernel<ET, HC>), grid, dim3(NT),       \
                     bytes, c.stream, c.out, c.out_stride, c.tmp, c.scores,  \
                     c.ml, c.vc, c.talk, c.gate, c.gate_stride, c.E,         \
                     c.nparts, c.m)
  if (c.E <= 64) HELIX_VALUES(2);
  else if (c.E <= 128) HELIX_VALUES(4);
  else HELIX_VALUES(8);
#undef HELIX_VALUES
  if (c.nparts > 1)
    hipLaunchKernelGGL((row_reduce_kernel<uint16_t>), dim3(c.R, c.m.H),
                       dim3(NT), 0, c.stream, c.out, c.out_stride, c.tmp,
                       c.gate, c.gate_stride, c.E, c.m);
}

template <typename S>
void dispatch_rows(RowCall<S>& c) {
  const int HG = c.m.H / c.m.G;
  if constexpr (sizeof(S) == 2) {
    if (c.D <= 128 && c.E <= 256) {
      if (HG <= 4) launch_rows_mfma<4>(c);
      else launch_rows_mfma<8>(c);
      return;
    }
  }
  if (HG == 1) launch_rows<S, 1>(c);
  else if (HG == 2) launch_rows<S, 2>(c);
  else if (HG <= 4) launch_rows<S, 4>(c);
  else launch_rows<S, 8>(c);
}

}  // namespace

// out [R, H*E] (row stride free), q [R, H, Dp], caches as above,
// scores [>=R, H, span], ml [>=R, H, max_parts, 2],
// tmp [>=R, H, max_parts, E] (max_parts bounds the split); max_keys: bound on
// any row's visible keys (window applied).
void talk_attn_rows(torch::Tensor out, torch::Tensor q, torch::Tensor kc,
                    torch::Tensor vc, torch::Tensor block_tables,
                    c10::optional<torch::Tensor> row_seq,
                    torch::Tensor row_len, int64_t max_keys, double scale,
                    double cap, int64_t window,
                    c10::optional<torch::Tensor> slopes,
                    c10::optional<torch::Tensor> talk,
                    c10::optional<torch::Tensor> gate, torch::Tensor scores,
                    torch::Tensor ml, torch::Tensor tmp) {
  const int64_t R = q.size(0), H = q.size(1), Dp = q.size(2);
  if (R == 0) return;
  const int64_t G = kc.size(1), bs = kc.size(2), E = vc.size(2);
  TORCH_CHECK(q.is_contiguous() && kc.is_contiguous() && vc.is_contiguous());
  TORCH_CHECK(kc.size(3) == Dp && Dp % 8 == 0, "key rows padded to 8");
  TORCH_CHECK(vc.size(1) == G && vc.size(3) == bs && bs % 8 == 0 &&
              vc.size(0) == kc.size(0), "V cache is [nblk, G, E, bs]");
  TORCH_CHECK(H % G == 0 && E <= 512 && H <= 1024);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == R && out.size(1) == H * E &&
              out.stride(1) == 1);
  TORCH_CHECK(q.scalar_type() == kc.scalar_type() &&
              q.scalar_type() == vc.scalar_type() &&
              q.scalar_type() == out.scalar_type());
  TORCH_CHECK(block_tables.scalar_type() == torch::kInt32 &&
              block_tables.dim() == 2 && block_tables.stride(1) == 1);
  TORCH_CHECK(row_len.scalar_type() == torch::kInt32 &&
              row_len.numel() == R && row_len.is_contiguous());
  if (row_seq.has_value()) {
    TORCH_CHECK(row_seq->scalar_type() == torch::kInt32 &&
                row_seq->numel() == R && row_seq->is_contiguous());
  } else {
    TORCH_CHECK(block_tables.size(0) >= R);
  }
  if (slopes.has_value())
    TORCH_CHECK(slopes->scalar_type() == torch::kFloat32 &&
                slopes->numel() == H && slopes->is_contiguous());
  if (talk.has_value())
    TORCH_CHECK(talk->scalar_type() == torch::kFloat32 &&
                talk->numel() == H * H && talk->is_contiguous());
  if (gate.has_value())
    TORCH_CHECK(gate->scalar_type() == q.scalar_type() &&
                gate->size(0) == R && gate->size(1) == H &&
                gate->stride(1) == 1);
  TORCH_CHECK(scores.is_contiguous() && ml.is_contiguous() &&
              tmp.is_contiguous() &&
              scores.scalar_type() == torch::kFloat32 &&
              ml.scalar_type() == torch::kFloat32 &&
              tmp.scalar_type() == torch::kFloat32);
  const int64_t span = scores.size(2), max_parts = ml.size(2);
  TORCH_CHECK(scores.size(0) >= R && scores.size(1) == H &&
              ml.size(0) >= R && ml.size(1) == H && tmp.size(0) >= R &&
              tmp.size(1) == H && tmp.size(2) == max_parts &&
              tmp.size(3) == E);
  TORCH_CHECK(max_keys >= 1 && max_keys <= span, "score scratch too small");

  // partitions: enough workgroups for the chip, in whole QUANTs
  const int HG = H / G;
  const int hc = HG <= 4 ? 4 : 8;
  const int wg = R * G * cdiv(HG, hc);
  int nparts = std::max(1, 1024 / std::max(1, wg));
  nparts = std::min<int>({nparts, cdiv(max_keys, QUANT), (int)max_parts});
  const int part = cdiv(cdiv((int)max_keys, nparts), QUANT) * QUANT;
  nparts = cdiv(max_keys, part);

  auto fill = [&](auto& c) {
    using SP = decltype(c.out);
    c.out = (SP)out.data_ptr();
    c.out_stride = out.stride(0);
    c.q = (SP)q.data_ptr();
    c.kc = (SP)kc.data_ptr();
    c.vc = (SP)vc.data_ptr();
    c.gate = gate.has_value() ? (SP)gate->data_ptr() : nullptr;
    c.gate_stride = gate.has_value() ? gate->stride(0) : 0;
    c.slopes = slopes.has_value() ? slopes->data_ptr<float>() : nullptr;
    c.talk = talk.has_value() ? talk->data_ptr<float>() : nullptr;
    c.scores = scores.data_ptr<float>();
    c.ml = ml.data_ptr<float>();
    c.tmp = tmp.data_ptr<float>();
    c.scale = (float)scale;
    c.cap = (float)cap;
    c.R = R;
    c.D = Dp;
    c.E = E;
    c.nparts = nparts;
    c.m = RowGeom{block_tables.data_ptr<int>(), (int)block_tables.stride(0),
                  row_seq.has_value() ? row_seq->data_ptr<int>() : nullptr,
                  row_len.data_ptr<int>(), (int)window, (int)H, (int)G,
                  (int)bs, (int)span, part, (int)max_parts, 1};
    c.stream = at::hip::getCurrentHIPStream();
    dispatch_rows(c);
  };
  if (q.scalar_type() == torch::kBFloat16) {
    RowCall<uint16_t> c;
    fill(c);
  } else if (q.scalar_type() == torch::kFloat32) {
    RowCall<float> c;
    fill(c);
  } else {
    TORCH_CHECK(false, "talk_attn_rows: bf16 or fp32");
  }
}
