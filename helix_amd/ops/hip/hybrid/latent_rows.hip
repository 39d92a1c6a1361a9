// Latent attention, a query row at a time (decode and short prompts).
//
// With the key up-projection moved to the query, a row attends to the cached
// latents themselves, and all heads share one key and one value row:
//
//   absorb  q'_h = q_h W_uk                      [rank], beside the rotated
//   rows    o'_h = softmax(scale q'_h . row) c   over the cached rows
//   out     o_h  = gate_h W_uv o'_h
//
// The row kernel reads every cached row once for up to 32 heads. A tile of
// rows waits in LDS; it is the A operand of the scores as it lies and, read
// with the transposing LDS load, that of the values. A workgroup's 4 waves
// split rows x heads for the scores and the latent's dimensions for the
// values. Partitions of long rows are merged by a kernel of their own.
//
// Cache row: [latent, padded to 8 | shared rotated key part, padded to 8].
#include "tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr float NEG = -1e30f;
constexpr int NT = 256;

// ----------------------------------------------------------------- epilogue

struct Epilogue {
  const double* freqs;         // [pairs]; null: no rotation
  const int64_t* pos;
  const float* norm_w;
  const int64_t* slots;
  int64_t z_stride;
  int pairs, q_at, heads, dim_pad, head_cols, kv_at, rank, rank_pad, rot_dim,
      row;
  float amp, eps;
};

// The pair (u, v) at columns j, j + 1 of a head turns by its angle.
__device__ __forceinline__ void turn(float& u, float& v, const float* trig) {
  const float a = u * trig[0] - v * trig[1];
  v = v * trig[0] + u * trig[1];
  u = a;
}

// Rotates q in place, writes the cache row. One workgroup per token; the
// angles of the pairs are the same for all heads. N: elements of a thread's
// accesses; rank, dims and columns are multiples of it.
template <typename S, int N>
__global__ __launch_bounds__(NT) void latent_epilogue_kernel(
    S* __restrict__ z, S* __restrict__ cache, Epilogue e) {
  extern __shared__ __attribute__((aligned(16))) float trig[];  // [pairs][2]
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x;
  S* zr = z + t * e.z_stride;
  const S* kv = zr + e.kv_at;
  // the first query vector and the latent are under way during the angles
  const int per = 2 * e.pairs / N, nq = e.heads * per;
  auto q_at = [&](int i) {
    const int h = i / per;
    return zr + e.q_at + h * e.head_cols + e.dim_pad + (i - h * per) * N;
  };
  float q0[N], c0[N];
  if (tid < nq) ldv<N>(q_at(tid), q0);
  if (tid * N < e.rank) ldv<N>(kv + tid * N, c0);
  for (int i = tid; i < e.pairs; i += NT) {
    // whole turns off in double, the rest is a 32-bit angle
    const double turns =
        (double)e.pos[t] * e.freqs[i] * 0.15915494309189533577;
    const float a = (float)((turns - floor(turns)) * 6.28318530717958647693);
    float s, c;
    sincosf(a, &s, &c);
    trig[2 * i] = e.amp * c;
    trig[2 * i + 1] = e.amp * s;
  }
  float ss = 0.f;
  if (tid * N < e.rank) {
#pragma unroll
    for (int i = 0; i < N; ++i) ss += c0[i] * c0[i];
  }
  for (int d = (tid + NT) * N; d < e.rank; d += NT * N) {
    float v[N];
    ldv<N>(kv + d, v);
#pragma unroll
    for (int i = 0; i < N; ++i) ss += v[i] * v[i];
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / e.rank + e.eps);

  for (int i = tid; i < nq; i += NT) {
    S* q = q_at(i);
    if (i != tid) ldv<N>(q, q0);
    const float* tr = trig + i % per * N;
#pragma unroll
    for (int j = 0; j < N; j += 2) turn(q0[j], q0[j + 1], tr + j);
    stv<N>(q, q0);
  }
  const int64_t slot = e.slots[t];
  if (slot < 0) return;
  S* out = cache + slot * e.row;
  for (int d = tid * N; d < e.row; d += NT * N) {
    float v[N];
    if (d < e.rank) {
      float w[N];
      ldv<N>(kv + d, v);
      ldv<N>(e.norm_w + d, w);
#pragma unroll
      for (int i = 0; i < N; ++i) v[i] *= inv * w[i];
    } else if (d >= e.rank_pad && d < e.rank_pad + e.rot_dim) {
      ldv<N>(kv + d, v);
      const int j0 = d - e.rank_pad;
      if (j0 < 2 * e.pairs) {
#pragma unroll
        for (int j = 0; j < N; j += 2)
          turn(v[j], v[j + 1], trig + j0 + j);
      }
    } else {
#pragma unroll
      for (int i = 0; i < N; ++i) v[i] = 0.f;
    }
    stv<N>(out + d, v);
  }
}

// Any sizes.
template <typename S>
__global__ __launch_bounds__(NT) void latent_epilogue_any_kernel(
    S* __restrict__ z, S* __restrict__ cache, Epilogue e) {
  extern __shared__ float trig[];
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  S* zr = z + t * e.z_stride;
  for (int i = threadIdx.x; i < e.pairs; i += NT) {
    const double turns =
        (double)e.pos[t] * e.freqs[i] * 0.15915494309189533577;
    const float a = (float)((turns - floor(turns)) * 6.28318530717958647693);
    float s, c;
    sincosf(a, &s, &c);
    trig[2 * i] = e.amp * c;
    trig[2 * i + 1] = e.amp * s;
  }
  const S* kv = zr + e.kv_at;
  float ss = 0.f;
  for (int d = threadIdx.x; d < e.rank; d += NT) {
    const float v = ld1(kv + d);
    ss += v * v;
  }
  const float inv = 1.f / sqrtf(group_sum(ss, red) / e.rank + e.eps);
  const int64_t slot = e.slots[t];
  if (slot >= 0) {
    S* out = cache + slot * e.row;
    for (int d = threadIdx.x; d < e.row; d += NT) {
      float v = 0.f;
      if (d < e.rank) {
        v = ld1(kv + d) * inv * e.norm_w[d];
      } else if (d >= e.rank_pad && d < e.rank_pad + e.rot_dim) {
        const int j = d - e.rank_pad;
        v = ld1(kv + d);
        if (j < 2 * e.pairs) {
          float u = ld1(kv + e.rank_pad + (j & ~1));
          float w = ld1(kv + e.rank_pad + (j | 1));
          turn(u, w, trig + (j & ~1));
          v = (j & 1) ? w : u;
        }
      }
      st1(out + d, v);
    }
  }
  for (int i = threadIdx.x; i < e.heads * e.pairs; i += NT) {
    const int h = i / e.pairs, p = i - h * e.pairs;
    S* q = zr + e.q_at + h * e.head_cols + e.dim_pad + 2 * p;
    float u = ld1(q), v = ld1(q + 1);
    turn(u, v, trig + 2 * p);
    st1(q, u);
    st1(q + 1, v);
  }
}

// ------------------------------------------------------------------- absorb

// q' [R, H, rank_pad + rot_pad] on MFMA: D[rank, row] = ukt_h z^T. A wave
// has 16 rows and 8 tiles of the rank.
__global__ __launch_bounds__(NT) void absorb_mfma_kernel(
    uint16_t* __restrict__ q, const uint16_t* __restrict__ z,
    int64_t z_stride, int head_cols, int dim_pad,
    const uint16_t* __restrict__ ukt, int rank_pad, int row, int R, int H) {
  const int wid = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int h = blockIdx.y, r0 = blockIdx.x * 64 + wid * 16;
  if (r0 >= R) return;
  const int r = r0 + lo;
  const uint16_t* zh = z + (int64_t)min(r, R - 1) * z_stride + h * head_cols;
  uint16_t* qh = q + ((int64_t)min(r, R - 1) * H + h) * row;
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  floatx4 acc[8];
#pragma unroll
  for (int t = 0; t < 8; ++t) acc[t] = floatx4{0, 0, 0, 0};
  const int k0 = blockIdx.z * 128;
  for (int d0 = hi * 8; d0 < ((dim_pad + 31) & ~31); d0 += 32) {
    // clamped columns meet a zero, clamped rows are not stored
    const int d = min(d0, dim_pad - 8);
    const u16x8 raw = ld_u16x8(zh + d), b = d == d0 ? raw : zero;
    u16x8 a[8];
#pragma unroll
    for (int t = 0; t < 8; ++t)
      a[t] = ld_u16x8(ukt + ((int64_t)h * rank_pad +
                             min(k0 + t * 16 + lo, rank_pad - 1)) * dim_pad +
                      d);
#pragma unroll
    for (int t = 0; t < 8; ++t) acc[t] = mfma16(a[t], b, acc[t]);
  }
  if (r < R) {
#pragma unroll
    for (int t = 0; t < 8; ++t) {
      const int k = k0 + t * 16 + hi * 4;
      if (k < rank_pad) {
        const float v[4] = {acc[t][0], acc[t][1], acc[t][2], acc[t][3]};
        st_bf16x4(qh + k, v);
      }
    }
    if (blockIdx.z == 0)
      for (int d = hi * 8; d < row - rank_pad; d += 32)
        *reinterpret_cast<u16x8*>(qh + rank_pad + d) =
            ld_u16x8(zh + dim_pad + d);
  }
}

template <typename S>
__global__ __launch_bounds__(NT) void absorb_plain_kernel(
    S* __restrict__ q, const S* __restrict__ z, int64_t z_stride,
    int head_cols, int dim_pad, const S* __restrict__ uk, int rank_pad,
    int row, int H) {
  const int h = blockIdx.y;
  const S* zh = z + blockIdx.x * z_stride + h * head_cols;
  S* qh = q + ((int64_t)blockIdx.x * H + h) * row;
  for (int k = threadIdx.x; k < rank_pad; k += NT) {
    float a = 0.f;
    for (int d = 0; d < dim_pad; ++d)
      a += ld1(zh + d) * ld1(uk + ((int64_t)h * dim_pad + d) * rank_pad + k);
    st1(qh + k, a);
  }
  for (int d = threadIdx.x; d < row - rank_pad; d += NT)
    qh[rank_pad + d] = zh[dim_pad + d];
}

// --------------------------------------------------------------------- rows

struct Rows {
  const int* bt;
  const int* row_seq;          // table row of a query row; null: its index
  const int* row_len;
  int bt_stride, window, bs, row, rank_pad, H, parts;
  float scale;
};

// Which cached positions [p0, p1) a partition of a row covers (whole tiles,
// possibly none).
__device__ __forceinline__ void part_range(const Rows& m, int r, int part,
                                           int tile, int& p0, int& p1) {
  const int len = m.row_len[r];
  const int lo = m.window > 0 ? max(0, len - m.window) : 0;
  const int per = (len - lo + m.parts - 1) / m.parts;
  const int span = (per + tile - 1) / tile * tile;
  p0 = lo + part * span;
  p1 = min(len, p0 + span);
}

// Four keys of one value dimension from LDS. The 16 lanes of a quarter wave
// name 4 rows x 16 columns, 4 columns each (lane j: row j / 4, columns
// 4 (j % 4) ..), and get a column each.
__device__ __forceinline__ u16x4 ld_tr4(const uint16_t* p) {
  typedef __attribute__((ext_vector_type(4))) int16_t i16x4;
  auto v = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) i16x4*)p);
  return __builtin_bit_cast(u16x4, v);
}

// NK: 32-wide steps of the cache row; DT: 16-wide tiles of the latent per
// wave; HT: 16-head tiles. A tile of cached rows is 64 / HT of them.
template <int NK, int DT, int HT>
__global__ __launch_bounds__(NT, 2) void latent_rows_kernel(
    uint16_t* __restrict__ o, float* __restrict__ part_o,
    float* __restrict__ ml, const uint16_t* __restrict__ q,
    const uint16_t* __restrict__ cache, Rows m) {
  constexpr int KEYS = 64 / HT, KW = 4 / HT;
  constexpr int PITCH = NK * 32 + 8, PP = KEYS + 8;
  constexpr int NL = NK / HT;                 // 16-byte loads per thread
  static_assert(NK % HT == 0 && DT * 64 <= NK * 32, "tile");
  __shared__ uint16_t kv[KEYS * PITCH];
  __shared__ uint16_t pw[HT * 16 * PP];
  __shared__ float stat[4][16];
  __shared__ int slots[2][KEYS];              // cache rows of two tiles

  const int r = blockIdx.x, part = blockIdx.y, h0 = blockIdx.z * HT * 16;
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int wk = wid % KW, wh = wid / KW;
  const int64_t ml_at = ((int64_t)r * m.parts + part) * m.H;
  int p0, p1;
  part_range(m, r, part, KEYS, p0, p1);
  if (p0 >= p1) {
    if (ml != nullptr && tid < HT * 16 && h0 + tid < m.H) {
      ml[(ml_at + h0 + tid) * 2] = NEG;
      ml[(ml_at + h0 + tid) * 2 + 1] = 0.f;
    }
    return;
  }
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  const int hq = h0 + wh * 16 + lo;
  u16x8 qf[NK];
#pragma unroll
  for (int k = 0; k < NK; ++k) {
    const int d = k * 32 + hi * 8;
    qf[k] = hq < m.H && d < m.row
                ? ld_u16x8(q + ((int64_t)r * m.H + hq) * m.row + d)
                : zero;
  }
  const int* bt = m.bt + (int64_t)(m.row_seq ? m.row_seq[r] : r) * m.bt_stride;
  u16x8 reg[NL];
  auto load = [&](int buf) {
#pragma unroll
    for (int c = 0; c < NL; ++c) {
      // no branch, so that all loads are under way at once; columns past
      // the row meet zeros of the query
      const int e = c * NT + tid, key = e / (NK * 4);
      const int d = min(e % (NK * 4) * 8, m.row - 8);
      reg[c] = ld_u16x8(cache + (int64_t)slots[buf][key] * m.row + d);
    }
  };
  // page lookups run two tiles ahead of the rows, so no load waits for one
  auto slot_of = [&](int base) {
    const int tok = min(base + tid, p1 - 1);
    return bt[tok / m.bs] * m.bs + tok % m.bs;
  };
  floatx4 acc[HT][DT];
  float m_run[HT], l = 0.f;
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    m_run[t] = NEG;
#pragma unroll
    for (int d = 0; d < DT; ++d) acc[t][d] = floatx4{0, 0, 0, 0};
  }

  if (tid < KEYS) {
    slots[0][tid] = slot_of(p0);
    slots[1][tid] = slot_of(p0 + KEYS);
  }
  __syncthreads();
  load(0);
  int buf = 0;
  for (int base = p0; base < p1; base += KEYS, buf ^= 1) {
    __syncthreads();                          // the last tile is read
#pragma unroll
    for (int c = 0; c < NL; ++c) {
      const int e = c * NT + tid;
      *reinterpret_cast<u16x8*>(kv + e / (NK * 4) * PITCH +
                                e % (NK * 4) * 8) = reg[c];
    }
    __syncthreads();
    int ahead = 0;
    if (base + KEYS < p1) load(buf ^ 1);
    if (tid < KEYS) ahead = slot_of(base + 2 * KEYS);

    // scores of 16 rows x 16 heads: lane has rows 4 hi + i, head lo
    floatx4 s = floatx4{0, 0, 0, 0};
#pragma unroll
    for (int k = 0; k < NK; ++k)
      s = mfma16(ld_u16x8(kv + (wk * 16 + lo) * PITCH + k * 32 + hi * 8),
                 qf[k], s);
    float mx = NEG;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      s[i] = base + wk * 16 + hi * 4 + i < p1 ? s[i] * m.scale : NEG;
      mx = fmaxf(mx, s[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
    if (hi == 0) stat[wid][lo] = mx;
    __syncthreads();
    float corr[HT];
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      float mt = m_run[t];
#pragma unroll
      for (int k = 0; k < KW; ++k) mt = fmaxf(mt, stat[t * KW + k][lo]);
      corr[t] = __expf(m_run[t] - mt);
      m_run[t] = mt;
    }
    const float mine = HT == 1 ? m_run[0] : (wh ? m_run[HT - 1] : m_run[0]);
    l *= HT == 1 ? corr[0] : (wh ? corr[HT - 1] : corr[0]);
    float p[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      // a tile always has a row inside, so `mine` is a real score
      p[i] = __expf(s[i] - mine);
      l += p[i];
    }
    st_bf16x4(pw + (wh * 16 + lo) * PP + wk * 16 + hi * 4, p);
    __syncthreads();

    // values: D[dim, head] += c^T p
#pragma unroll
    for (int t = 0; t < HT; ++t)
#pragma unroll
      for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[t][d][i] *= corr[t];
#pragma unroll
    for (int kk = 0; kk < KEYS / 32; ++kk) {
      u16x8 pf[HT];
#pragma unroll
      for (int t = 0; t < HT; ++t)
        pf[t] = ld_u16x8(pw + (t * 16 + lo) * PP + kk * 32 + hi * 8);
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        const int at = (wid * DT + d) * 16;
        if (at < m.rank_pad) {
          const uint16_t* b = kv + (kk * 32 + hi * 8 + (lo >> 2)) * PITCH +
                              at + (lo & 3) * 4;
          const u16x4 a0 = ld_tr4(b), a1 = ld_tr4(b + 4 * PITCH);
          const u16x8 a = {a0[0], a0[1], a0[2], a0[3],
                           a1[0], a1[1], a1[2], a1[3]};
#pragma unroll
          for (int t = 0; t < HT; ++t) acc[t][d] = mfma16(a, pf[t], acc[t][d]);
        }
      }
    }
    if (tid < KEYS) slots[buf][tid] = ahead;  // this tile's are used
  }

  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  __syncthreads();
  if (hi == 0) stat[wid][lo] = l;
  __syncthreads();
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    float sum = 0.f;
#pragma unroll
    for (int k = 0; k < KW; ++k) sum += stat[t * KW + k][lo];
    const int h = h0 + t * 16 + lo;
    if (h >= m.H) continue;
    const float inv = m.parts == 1 ? 1.f / sum : 1.f;
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      const int at = (wid * DT + d) * 16 + hi * 4;
      if (at < m.rank_pad) {
        const float v[4] = {acc[t][d][0] * inv, acc[t][d][1] * inv,
                            acc[t][d][2] * inv, acc[t][d][3] * inv};
        if (m.parts == 1)
          st_bf16x4(o + ((int64_t)r * m.H + h) * m.rank_pad + at, v);
        else
          *reinterpret_cast<f32x4*>(part_o + (ml_at + h) * m.rank_pad + at) =
              f32x4{v[0], v[1], v[2], v[3]};
      }
    }
    if (ml != nullptr && wid == 0 && hi == 0) {
      ml[(ml_at + h) * 2] = m_run[t];
      ml[(ml_at + h) * 2 + 1] = sum;
    }
  }
}

// Any size, fp32 or bf16: a workgroup per (row, head), tiles of 256 cached
// rows, a thread per row for the scores and per dimensions for the values.
constexpr int PLAIN_DIMS = 8;                 // rank_pad <= 8 * NT

template <typename S>
__global__ __launch_bounds__(NT) void latent_rows_plain_kernel(
    S* __restrict__ o, const S* __restrict__ q, const S* __restrict__ cache,
    Rows m) {
  extern __shared__ float ql[];               // [row]
  __shared__ float pl[NT];
  __shared__ int64_t at[NT];
  __shared__ float red[16];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wid = tid / WAVE;
  int p0, p1;
  part_range(m, r, 0, 1, p0, p1);
  const int* bt = m.bt + (int64_t)(m.row_seq ? m.row_seq[r] : r) * m.bt_stride;
  const S* qr = q + ((int64_t)r * m.H + h) * m.row;
  for (int d = tid; d < m.row; d += NT) ql[d] = ld1(qr + d);
  float acc[PLAIN_DIMS], m_run = NEG, l = 0.f;
#pragma unroll
  for (int i = 0; i < PLAIN_DIMS; ++i) acc[i] = 0.f;
  for (int base = p0; base < p1; base += NT) {
    __syncthreads();
    const int tok = base + tid;
    float s = NEG;
    if (tok < p1) {
      at[tid] = ((int64_t)bt[tok / m.bs] * m.bs + tok % m.bs) * m.row;
      const S* row = cache + at[tid];
      float a = 0.f;
      for (int d = 0; d < m.row; d += 8) {
        float v[8];
        ldv<8>(row + d, v);
#pragma unroll
        for (int i = 0; i < 8; ++i) a += ql[d + i] * v[i];
      }
      s = a * m.scale;
    }
    const float wm = wave_reduce_max(s);
    if ((tid & (WAVE - 1)) == 0) red[wid] = wm;
    __syncthreads();
    float mn = m_run;
    for (int w = 0; w < NT / WAVE; ++w) mn = fmaxf(mn, red[w]);
    const float corr = exp_s<S>(m_run - mn);
    m_run = mn;
    const float p = tok < p1 ? exp_s<S>(s - mn) : 0.f;
    pl[tid] = p;
    l = l * corr + p;
    __syncthreads();
    const int n = min(NT, p1 - base);
#pragma unroll
    for (int i = 0; i < PLAIN_DIMS; ++i) {
      const int d = i * NT + tid;
      if (d < m.rank_pad) {
        float a = acc[i] * corr;
        for (int j = 0; j < n; ++j) a += pl[j] * ld1(cache + at[j] + d);
        acc[i] = a;
      }
    }
  }
  __syncthreads();
  const float inv = 1.f / group_sum(l, red);
#pragma unroll
  for (int i = 0; i < PLAIN_DIMS; ++i) {
    const int d = i * NT + tid;
    if (d < m.rank_pad)
      st1(o + ((int64_t)r * m.H + h) * m.rank_pad + d, acc[i] * inv);
  }
}

// -------------------------------------------------------------------- merge

// o'[r, h] from its partitions, a workgroup per (row, head): the waves take
// every fourth partition, 8 of them under way at once.
__global__ __launch_bounds__(NT) void latent_merge_kernel(
    uint16_t* __restrict__ o, const float* __restrict__ part_o,
    const float* __restrict__ ml, int H, int K, int parts) {
  __shared__ float sum[NT / WAVE][512];
  const int r = blockIdx.x, h = blockIdx.y;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const int lane = threadIdx.x & (WAVE - 1);
  const float* st = ml + ((int64_t)r * parts * H + h) * 2;
  float M = NEG, l = 0.f;
  for (int p = lane; p < parts; p += WAVE)
    M = fmaxf(M, st[(int64_t)p * H * 2]);
  M = wave_reduce_max(M);
  for (int p = lane; p < parts; p += WAVE)
    l += st[(int64_t)p * H * 2 + 1] * __expf(st[(int64_t)p * H * 2] - M);
  const float inv = 1.f / wave_reduce_sum(l);
  for (int d0 = 0; d0 < K; d0 += 512) {
    const int d = min(d0 + lane * 8, K - 8);
    const float* po = part_o + ((int64_t)r * parts * H + h) * K + d;
    float a[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    for (int p = wid; p < parts; p += 8 * (NT / WAVE)) {
      float b[8][8], w[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int64_t q = p + i * (NT / WAVE);
        w[i] = 0.f;
        if (q < parts) {                      // the same for all lanes
          const float* s = st + q * H * 2;
          w[i] = s[1] > 0.f ? __expf(s[0] - M) * inv : 0.f;
          ldv<8>(po + q * H * K, b[i]);
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (w[i] > 0.f) {                     // not an empty partition
#pragma unroll
          for (int j = 0; j < 8; ++j) a[j] += w[i] * b[i][j];
        }
    }
    stv<8>(&sum[wid][lane * 8], a);
    __syncthreads();
    if (wid == 0 && d0 + lane * 8 < K) {
#pragma unroll
      for (int w = 1; w < NT / WAVE; ++w)
#pragma unroll
        for (int j = 0; j < 8; ++j) a[j] += sum[w][lane * 8 + j];
      *reinterpret_cast<u16x8*>(o + ((int64_t)r * H + h) * K + d) = pack8(a);
    }
    __syncthreads();
  }
}

// ---------------------------------------------------------------------- out

// out[r, h E + e] = gate * sum_k uv[h E + e, k] o'[r, h, k]. A workgroup has
// RT tiles of 16 rows of one head; o' waits in LDS, the waves split the
// value dimensions.
template <int RT>
__global__ __launch_bounds__(NT) void latent_out_kernel(
    uint16_t* __restrict__ out, int64_t out_stride,
    const uint16_t* __restrict__ o, const uint16_t* __restrict__ uv,
    const uint16_t* __restrict__ gate, int64_t gate_stride, int R, int H,
    int E, int K, int vec) {
  extern __shared__ __attribute__((aligned(16))) uint16_t ol[];
  const int pitch = ((K + 31) & ~31) + 8, per = (pitch - 8) / 8;
  const int h = blockIdx.y, r0 = blockIdx.x * RT * 16;
  const int wid = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  for (int i = threadIdx.x; i < RT * 16 * per; i += NT) {
    const int t = i / per, d = i % per * 8;
    const u16x8 v = ld_u16x8(o + ((int64_t)min(r0 + t, R - 1) * H + h) * K +
                             min(d, K - 8));
    *reinterpret_cast<u16x8*>(ol + t * pitch + d) = d < K ? v : zero;
  }
  __syncthreads();
  for (int e0 = (blockIdx.z * 4 + wid) * 16; e0 < E;
       e0 += gridDim.z * 4 * 16) {
    floatx4 acc[RT];
#pragma unroll
    for (int t = 0; t < RT; ++t) acc[t] = floatx4{0, 0, 0, 0};
    const uint16_t* ur = uv + ((int64_t)h * E + min(e0 + lo, E - 1)) * K;
#pragma unroll 4
    for (int k = 0; k < pitch - 8; k += 32) {
      const u16x8 a = ld_u16x8(ur + min(k + hi * 8, K - 8));
#pragma unroll
      for (int t = 0; t < RT; ++t)
        acc[t] = mfma16(a, ld_u16x8(ol + (t * 16 + lo) * pitch + k + hi * 8),
                        acc[t]);
    }
#pragma unroll
    for (int t = 0; t < RT; ++t) {
      const int r = r0 + t * 16 + lo, e = e0 + hi * 4;
      if (r >= R || e >= E) continue;
      const float g = gate == nullptr ? 1.f
                                      : sigmoid_s<uint16_t>(bf16_to_f32(
                                            gate[r * gate_stride + h]));
      uint16_t* dst = out + r * out_stride + h * E + e;
      const float v[4] = {acc[t][0] * g, acc[t][1] * g, acc[t][2] * g,
                          acc[t][3] * g};
      if (vec) {
        st_bf16x4(dst, v);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (e + i < E) dst[i] = f32_to_bf16(v[i]);
      }
    }
  }
}

template <typename S>
__global__ __launch_bounds__(NT) void latent_out_plain_kernel(
    S* __restrict__ out, int64_t out_stride, const S* __restrict__ o,
    const S* __restrict__ uv, const S* __restrict__ gate,
    int64_t gate_stride, int H, int E, int K) {
  const int r = blockIdx.x, h = blockIdx.y;
  const S* oh = o + ((int64_t)r * H + h) * K;
  const float g =
      gate == nullptr ? 1.f : sigmoid_s<S>(ld1(gate + r * gate_stride + h));
  for (int e = threadIdx.x; e < E; e += NT) {
    const S* ur = uv + ((int64_t)h * E + e) * K;
    float a = 0.f;
    for (int k = 0; k < K; k += 8) {
      float u[8], v[8];
      ldv<8>(ur + k, u);
      ldv<8>(oh + k, v);
#pragma unroll
      for (int i = 0; i < 8; ++i) a += u[i] * v[i];
    }
    st1(out + r * out_stride + h * E + e, a * g);
  }
}

// ------------------------------------------------------------------ helpers

bool is_bf16(const torch::Tensor& t) {
  return t.scalar_type() == torch::kBFloat16;
}

void check_type(const torch::Tensor& t) {
  TORCH_CHECK(is_bf16(t) || t.scalar_type() == torch::kFloat32,
              "latent attention: bf16 or fp32");
}

Rows make_rows(torch::Tensor q, torch::Tensor cache, torch::Tensor bt,
               OptT row_seq, torch::Tensor row_len, int64_t rank_pad,
               double scale, int64_t window, int parts) {
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && cache.dim() == 4 &&
              cache.is_contiguous() && cache.size(1) == 1);
  TORCH_CHECK(q.size(2) == cache.size(3) && q.size(2) % 8 == 0 &&
              rank_pad % 8 == 0 && rank_pad <= q.size(2));
  TORCH_CHECK(q.scalar_type() == cache.scalar_type());
  TORCH_CHECK(bt.scalar_type() == torch::kInt32 && bt.dim() == 2 &&
              bt.stride(1) == 1);
  TORCH_CHECK(row_len.scalar_type() == torch::kInt32 &&
              row_len.numel() == q.size(0) && row_len.is_contiguous());
  if (row_seq.has_value()) {
    TORCH_CHECK(row_seq->scalar_type() == torch::kInt32 &&
                row_seq->numel() == q.size(0) && row_seq->is_contiguous());
  } else {
    TORCH_CHECK(bt.size(0) >= q.size(0));
  }
  Rows m{};
  m.bt = bt.data_ptr<int>();
  m.row_seq = row_seq.has_value() ? row_seq->data_ptr<int>() : nullptr;
  m.row_len = row_len.data_ptr<int>();
  m.bt_stride = bt.stride(0);
  m.window = window;
  m.bs = cache.size(2);
  m.row = q.size(2);
  m.rank_pad = rank_pad;
  m.H = q.size(1);
  m.parts = parts;
  m.scale = (float)scale;
  return m;
}

}  // namespace

void latent_epilogue(torch::Tensor z, int64_t q_at, int64_t heads,
                     int64_t dim_pad, int64_t head_cols, int64_t kv_at,
                     int64_t rank, int64_t rank_pad, int64_t rot_dim,
                     OptT freqs, double amp, torch::Tensor pos,
                     torch::Tensor norm_w, double eps, torch::Tensor cache,
                     torch::Tensor slots) {
  const int64_t T = z.size(0), row = cache.size(3);
  check_type(z);
  TORCH_CHECK(z.dim() == 2 && z.stride(1) == 1 && cache.dim() == 4 &&
              cache.is_contiguous() && cache.size(1) == 1 &&
              cache.scalar_type() == z.scalar_type());
  TORCH_CHECK(rank <= rank_pad && rank_pad + rot_dim <= row &&
              kv_at + row <= z.size(1) &&
              q_at + heads * head_cols <= z.size(1));
  TORCH_CHECK(pos.scalar_type() == torch::kInt64 && pos.numel() == T &&
              slots.scalar_type() == torch::kInt64 && slots.numel() == T &&
              pos.is_contiguous() && slots.is_contiguous());
  TORCH_CHECK(norm_w.scalar_type() == torch::kFloat32 &&
              norm_w.numel() == rank && norm_w.is_contiguous());
  Epilogue e{};
  if (freqs.has_value() && rot_dim > 0) {
    TORCH_CHECK(freqs->scalar_type() == torch::kFloat64 &&
                freqs->is_cuda() && freqs->is_contiguous());
    e.freqs = freqs->data_ptr<double>();
    e.pairs = freqs->numel();
  }
  TORCH_CHECK(2 * e.pairs <= rot_dim && dim_pad + 2 * e.pairs <= head_cols &&
              e.pairs <= 4096);
  e.pos = pos.data_ptr<int64_t>();
  e.norm_w = norm_w.data_ptr<float>();
  e.slots = slots.data_ptr<int64_t>();
  e.z_stride = z.stride(0);
  e.q_at = q_at;
  e.heads = heads;
  e.dim_pad = dim_pad;
  e.head_cols = head_cols;
  e.kv_at = kv_at;
  e.rank = rank;
  e.rank_pad = rank_pad;
  e.rot_dim = rot_dim;
  e.row = row;
  e.amp = (float)amp;
  e.eps = (float)eps;
  if (T == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const int lds = std::max(1, e.pairs) * 2 * sizeof(float);
  const bool vec = rank % 8 == 0 && rot_dim % 8 == 0 && e.pairs % 4 == 0 &&
                   rank_pad % 8 == 0 && row % 8 == 0 && dim_pad % 8 == 0 &&
                   head_cols % 8 == 0 && q_at % 8 == 0 && kv_at % 8 == 0 &&
                   e.z_stride % 8 == 0 && (uintptr_t)z.data_ptr() % 32 == 0;
#define HELIX_EPI(K, S)                                                      \
  hipLaunchKernelGGL((K), dim3(T), dim3(NT), lds, stream, (S*)z.data_ptr(),  \
                     (S*)cache.data_ptr(), e)
  if (is_bf16(z)) {
    if (vec && e.pairs > 0)
      HELIX_EPI((latent_epilogue_kernel<uint16_t, 8>), uint16_t);
    else
      HELIX_EPI((latent_epilogue_any_kernel<uint16_t>), uint16_t);
  } else {
    HELIX_EPI((latent_epilogue_any_kernel<float>), float);
  }
#undef HELIX_EPI
}

void latent_absorb(torch::Tensor q, torch::Tensor z, int64_t q_at,
                   int64_t head_cols, int64_t dim_pad, torch::Tensor uk,
                   torch::Tensor ukt, int64_t rank_pad) {
  check_type(z);
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && z.stride(1) == 1);
  const int R = q.size(0), H = q.size(1), row = q.size(2);
  TORCH_CHECK(z.size(0) == R && q_at + H * head_cols <= z.size(1));
  TORCH_CHECK(row == rank_pad + head_cols - dim_pad && dim_pad % 8 == 0 &&
              head_cols % 8 == 0 && rank_pad % 8 == 0 && q_at % 8 == 0);
  TORCH_CHECK(uk.is_contiguous() && ukt.is_contiguous() &&
              uk.numel() == (int64_t)H * dim_pad * rank_pad &&
              ukt.numel() == uk.numel());
  TORCH_CHECK(uk.scalar_type() == z.scalar_type() &&
              ukt.scalar_type() == z.scalar_type() &&
              q.scalar_type() == z.scalar_type());
  if (R == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  if (is_bf16(z)) {
    TORCH_CHECK(z.stride(0) % 8 == 0);
    hipLaunchKernelGGL(absorb_mfma_kernel,
                       dim3(cdiv(R, 64), H, cdiv(rank_pad, 128)), dim3(NT),
                       0, stream, (uint16_t*)q.data_ptr(),
                       (const uint16_t*)z.data_ptr() + q_at, z.stride(0),
                       (int)head_cols, (int)dim_pad,
                       (const uint16_t*)ukt.data_ptr(), (int)rank_pad, row,
                       R, H);
  } else {
    hipLaunchKernelGGL((absorb_plain_kernel<float>), dim3(R, H), dim3(NT), 0,
                       stream, (float*)q.data_ptr(),
                       (const float*)z.data_ptr() + q_at, z.stride(0),
                       (int)head_cols, (int)dim_pad,
                       (const float*)uk.data_ptr(), (int)rank_pad, row, H);
  }
}

// Whether the MFMA row kernel takes these sizes: q [R, H, row].
bool latent_rows_fits(torch::Tensor q, int64_t rank_pad) {
  return is_bf16(q) && q.size(2) <= 576 && rank_pad <= 512;
}

void latent_rows(OptT o, OptT part, OptT ml, torch::Tensor q,
                 torch::Tensor cache, torch::Tensor block_tables,
                 OptT row_seq, torch::Tensor row_len, int64_t rank_pad,
                 double scale, int64_t window) {
  TORCH_CHECK(latent_rows_fits(q, rank_pad));
  const int R = q.size(0), H = q.size(1);
  int parts = 1;
  if (o.has_value()) {
    TORCH_CHECK(!part.has_value() && !ml.has_value() && o->is_contiguous() &&
                is_bf16(*o) && o->numel() == (int64_t)R * H * rank_pad);
  } else {
    TORCH_CHECK(part.has_value() && ml.has_value() && part->dim() == 4);
    parts = part->size(1);
    TORCH_CHECK(part->is_contiguous() && ml->is_contiguous() &&
                part->scalar_type() == torch::kFloat32 &&
                ml->scalar_type() == torch::kFloat32 &&
                part->numel() == (int64_t)R * parts * H * rank_pad &&
                ml->numel() == (int64_t)R * parts * H * 2);
    TORCH_CHECK(parts > 1 && parts <= 65535);
  }
  Rows m = make_rows(q, cache, block_tables, row_seq, row_len, rank_pad,
                     scale, window, parts);
  if (R == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  uint16_t* op = o.has_value() ? (uint16_t*)o->data_ptr() : nullptr;
  float* pp = part.has_value() ? part->data_ptr<float>() : nullptr;
  float* mp = ml.has_value() ? ml->data_ptr<float>() : nullptr;
#define HELIX_ROWS(NK, DT, HT)                                               \
  hipLaunchKernelGGL((latent_rows_kernel<NK, DT, HT>),                       \
                     dim3(R, parts, cdiv(H, HT * 16)), dim3(NT), 0, stream,  \
                     op, pp, mp, (const uint16_t*)q.data_ptr(),              \
                     (const uint16_t*)cache.data_ptr(), m)
#define HELIX_ROWS_H(NK, DT)                                                 \
  if (H > 16) HELIX_ROWS(NK, DT, 2); else HELIX_ROWS(NK, DT, 1)
  if (m.row <= 128) { HELIX_ROWS_H(4, 2); }
  else if (m.row <= 320 && rank_pad <= 256) { HELIX_ROWS_H(10, 4); }
  else { HELIX_ROWS_H(18, 8); }
#undef HELIX_ROWS_H
#undef HELIX_ROWS
}

void latent_rows_plain(torch::Tensor o, torch::Tensor q, torch::Tensor cache,
                       torch::Tensor block_tables, OptT row_seq,
                       torch::Tensor row_len, double scale, int64_t window) {
  check_type(q);
  const int R = q.size(0), H = q.size(1), rank_pad = o.size(2);
  TORCH_CHECK(o.is_contiguous() && o.size(0) == R && o.size(1) == H &&
              o.scalar_type() == q.scalar_type());
  TORCH_CHECK(rank_pad <= PLAIN_DIMS * NT && q.size(2) <= 8192,
              "latent size ", rank_pad);
  Rows m = make_rows(q, cache, block_tables, row_seq, row_len, rank_pad,
                     scale, window, 1);
  if (R == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const int lds = m.row * sizeof(float);
  if (is_bf16(q))
    hipLaunchKernelGGL((latent_rows_plain_kernel<uint16_t>), dim3(R, H),
                       dim3(NT), lds, stream, (uint16_t*)o.data_ptr(),
                       (const uint16_t*)q.data_ptr(),
                       (const uint16_t*)cache.data_ptr(), m);
  else
    hipLaunchKernelGGL((latent_rows_plain_kernel<float>), dim3(R, H),
                       dim3(NT), lds, stream, (float*)o.data_ptr(),
                       (const float*)q.data_ptr(),
                       (const float*)cache.data_ptr(), m);
}

void latent_merge(torch::Tensor o, torch::Tensor part, torch::Tensor ml) {
  TORCH_CHECK(part.dim() == 4 && part.is_contiguous() &&
              part.scalar_type() == torch::kFloat32);
  const int R = part.size(0), parts = part.size(1), H = part.size(2);
  const int K = part.size(3);
  TORCH_CHECK(o.is_contiguous() && is_bf16(o) &&
              o.numel() == (int64_t)R * H * K && K % 8 == 0);
  TORCH_CHECK(ml.is_contiguous() && ml.scalar_type() == torch::kFloat32 &&
              ml.numel() == (int64_t)R * parts * H * 2);
  if (R == 0) return;
  hipLaunchKernelGGL(latent_merge_kernel, dim3(R, H), dim3(NT), 0,
                     at::hip::getCurrentHIPStream(), (uint16_t*)o.data_ptr(),
                     part.data_ptr<float>(), ml.data_ptr<float>(), H, K,
                     parts);
}

void latent_out(torch::Tensor out, torch::Tensor o, torch::Tensor uv,
                OptT gate) {
  check_type(out);
  TORCH_CHECK(o.dim() == 3 && o.is_contiguous() &&
              o.scalar_type() == out.scalar_type());
  const int R = o.size(0), H = o.size(1), K = o.size(2);
  TORCH_CHECK(uv.dim() == 2 && uv.is_contiguous() && uv.size(1) == K &&
              uv.size(0) % H == 0 && K % 8 == 0);
  const int E = uv.size(0) / H;
  TORCH_CHECK(out.size(0) == R && out.size(1) == H * E && out.stride(1) == 1);
  TORCH_CHECK(uv.scalar_type() == out.scalar_type());
  int64_t gs = 0;
  if (gate.has_value()) {
    TORCH_CHECK(gate->size(0) == R && gate->size(1) == H &&
                gate->stride(1) == 1 &&
                gate->scalar_type() == out.scalar_type());
    gs = gate->stride(0);
  }
  if (R == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  if (!is_bf16(out)) {
    hipLaunchKernelGGL((latent_out_plain_kernel<float>), dim3(R, H), dim3(NT),
                       0, stream, (float*)out.data_ptr(), out.stride(0),
                       (const float*)o.data_ptr(),
                       (const float*)uv.data_ptr(),
                       gate.has_value() ? (const float*)gate->data_ptr()
                                        : nullptr,
                       gs, H, E, K);
    return;
  }
  const int pitch = ((K + 31) & ~31) + 8;
  const int vec = E % 4 == 0 && out.stride(0) % 4 == 0 &&
                  (uintptr_t)out.data_ptr() % 8 == 0;
  const int zs = std::min(cdiv(E, 64), R <= 64 ? 8 : 1);
#define HELIX_OUT(RT)                                                        \
  hipLaunchKernelGGL((latent_out_kernel<RT>), dim3(cdiv(R, RT * 16), H, zs), \
                     dim3(NT), RT * 16 * pitch * 2, stream,                  \
                     (uint16_t*)out.data_ptr(), out.stride(0),               \
                     (const uint16_t*)o.data_ptr(),                          \
                     (const uint16_t*)uv.data_ptr(),                         \
                     gate.has_value() ? (const uint16_t*)gate->data_ptr()    \
                                      : nullptr,                             \
                     gs, R, H, E, K, vec)
  if (R > 16 && K <= 512) {
    HELIX_OUT(2);
  } else {
    TORCH_CHECK(K <= 1536, "latent size ", K);
    HELIX_OUT(1);
  }
#undef HELIX_OUT
}
