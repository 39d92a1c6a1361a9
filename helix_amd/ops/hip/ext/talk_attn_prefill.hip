// Prefill attention with talking heads on MFMA (bf16), straight from the
// paged cache.
//
// Mixing softmaxed weights across heads needs every head's denominator
// before any weight meets a value, so there are two kernels:
//
//   stats   log2-sum-exp of every (row, head). One wave owns 16 query rows
//           and HPW consecutive heads and streams the window's K once; no
//           LDS, no barrier. The 4 waves of a workgroup take neighbouring
//           row tiles of the same heads, so their K reads meet in L1.
//   values  one workgroup owns 16 query rows and ALL heads, a wave HPW of
//           them. Per 32 keys: each wave recomputes its heads' scores and
//           writes p = exp2(s - lse) to LDS; the mixing w = talk . p over
//           heads is an MFMA with the heads as the inner dimension (each
//           wave mixes its share of the 512 (row, key) pairs); w goes
//           through LDS to the waves that own the heads, which multiply
//           with V.
//
// The mixing keeps fp32 weights: p is split into two bf16 terms (17
// significant bits) and products accumulate in fp32; talk is split the same
// way unless it is exactly representable, as bf16 checkpoints are.
//
// V pages are stored [E][bs] (8 tokens of a dim contiguous), so V fragments
// are plain 16-byte loads and nothing is transposed in LDS.
//
// MFMA f32_16x16x32_bf16 lane layout (lo = l&15, hi = l>>4):
//   A: lane l holds A[row = lo][k = hi*8 + i]
//   B: lane l holds B[k = hi*8 + i][col = lo]
//   C: lane l holds C[row = hi*4 + r][col = lo]
#include "../elem.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int QT = 16;         // query rows per wave tile
constexpr int KT = 32;         // keys per tile
constexpr int WP = KT + 8;     // w row pitch (bf16), 16-byte multiple
constexpr float NEG = -1e30f;
constexpr float LOG2E = 1.44269504088896340736f;

struct PrefillArgs {
  uint16_t* out;               // [T, H*E], row stride out_stride
  int64_t out_stride;
  float* lse;                  // [T, H] log2-sum-exp
  const uint16_t* q;           // [T, H, Dp]
  const uint16_t* kc;          // [nblk, G, bs, Dp]
  const uint16_t* vc;          // [nblk, G, E, bs]
  const int* bt;               // [B, bt_stride]
  int bt_stride;
  const int* cu_q;             // [B+1] rows of q per sequence
  const int* seq_len;          // [B] keys per sequence, these rows included
  const float* slopes;         // [H] or null
  const float* talk;           // [H, H]
  const uint16_t* gate;        // [T, H] logits, row stride gate_stride
  int64_t gate_stride;
  float scale, cap;
  int window, H, G, Dp, E, bs;
};

// Scores in the base-2 domain: log2e * (cap * tanh(d * scale / cap)
// - slope * dist), or log2e * (d * scale - slope * dist) without a cap.
struct Score2 {
  float k, c1;
  bool capped;
  __device__ Score2(float scale, float cap) {
    capped = cap > 0.f;
    k = capped ? 2.f * LOG2E * scale / cap : LOG2E * scale;
    c1 = cap * LOG2E;
  }
  __device__ __forceinline__ float operator()(float d, float slope2,
                                              float dist) const {
    float s = d * k;
    if (capped)
      s = c1 - 2.f * c1 *
                   __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s));
    return s - slope2 * dist;
  }
};

// One wave's 16 query rows and HPW heads. FAST: pages of 16 tokens, key size
// exactly 32*DT, and all heads of a wave share their key/value head, so
// addresses are one base plus immediates.
template <int HPW, int DT, bool FAST>
struct WaveTile {
  const PrefillArgs& a;
  const int* bt;
  int q_start, qlen, len, ctx, qbase, lo, hi, hbase;
  bf16x8 qf[HPW][DT];
  float slope2[HPW];
  int kvh[HPW];

  __device__ __forceinline__ int bs() const { return FAST ? 16 : a.bs; }
  __device__ __forceinline__ int Dp() const { return FAST ? 32 * DT : a.Dp; }
  // does head i need other K / V rows than head i - 1?
  __device__ __forceinline__ bool fresh(int i) const {
    return i == 0 || (!FAST && kvh[i] != kvh[i - 1]);
  }
  int t_first, t_end, full_lo, full_hi;

  __device__ __forceinline__ WaveTile(const PrefillArgs& args, int seq,
                                      int qtile, int head0, int lane)
      : a(args) {
    bt = a.bt + (int64_t)seq * a.bt_stride;
    q_start = a.cu_q[seq];
    qlen = a.cu_q[seq + 1] - q_start;
    len = a.seq_len[seq];
    ctx = len - qlen;
    qbase = qtile * QT;
    lo = lane & 15;
    hi = lane >> 4;
    hbase = head0;
    const int kv_hi = min(len, ctx + qbase + QT);
    const int kv_lo = a.window > 0 ? max(0, ctx + qbase - a.window + 1) : 0;
    t_first = kv_lo / KT;
    t_end = (kv_hi + KT - 1) / KT;
    // tiles inside [full_lo, full_hi) are visible to all 16 rows
    full_hi = ctx + qbase + 1;
    full_lo = a.window > 0 ? max(0, ctx + qbase + QT - a.window) : 0;
  }
  __device__ __forceinline__ void load_q() {
    const int HG = a.H / a.G;
#pragma unroll
    for (int i = 0; i < HPW; ++i) {
      const int h = min(hbase + i, a.H - 1);  // idle heads repeat the last
      kvh[i] = h / HG;
      slope2[i] = a.slopes != nullptr ? a.slopes[h] * LOG2E : 0.f;
      const int r = qbase + lo;
#pragma unroll
      for (int kt = 0; kt < DT; ++kt) {
        const int d = kt * 32 + hi * 8;
        u16x8 raw = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
        if (r < qlen && d < Dp())
          raw = *reinterpret_cast<const u16x8*>(
              a.q + ((int64_t)(q_start + r) * a.H + h) * Dp() + d);
        qf[i][kt] = *reinterpret_cast<bf16x8*>(&raw);
      }
    }
  }
  // element offset of the key row this lane feeds (head 0 of the page)
  __device__ __forceinline__ int64_t key_row(int tok) const {
    const int t = min(tok, len - 1);
    return ((int64_t)bt[t / bs()] * a.G * bs() + t % bs()) * Dp();
  }
  __device__ __forceinline__ void load_k(u16x8 (&kf)[DT], int64_t row,
                                         int g) const {
    const uint16_t* p = a.kc + row + (int64_t)g * bs() * Dp() + hi * 8;
#pragma unroll
    for (int kt = 0; kt < DT; ++kt)
      kf[kt] = kt * 32 + hi * 8 < Dp()
                   ? *reinterpret_cast<const u16x8*>(p + kt * 32)
                   : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
  }
  __device__ __forceinline__ floatx4 dot(int i, u16x8 (&kf)[DT]) const {
    floatx4 s = floatx4{0, 0, 0, 0};
#pragma unroll
    for (int kt = 0; kt < DT; ++kt)
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          qf[i][kt], *reinterpret_cast<bf16x8*>(&kf[kt]), s, 0, 0, 0);
    return s;
  }
  // distance of C row r to key tp
  __device__ __forceinline__ int dist(int r, int tp) const {
    return ctx + qbase + hi * 4 + r - tp;
  }
  __device__ __forceinline__ bool masked(int d) const {
    return d < 0 || (a.window > 0 && d >= a.window);
  }
};

template <int HPW, int DT, bool FAST>
__global__ __launch_bounds__(256) void talk_stats_kernel(PrefillArgs a) {
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  // later tiles see more keys under a causal mask: start them first
  const int qtile = ((int)gridDim.x - 1 - (int)blockIdx.x) * 4 + wid;
  WaveTile<HPW, DT, FAST> w(a, blockIdx.y, qtile, blockIdx.z * HPW,
                      threadIdx.x & (WAVE - 1));
  if (w.qbase >= w.qlen) return;
  w.load_q();
  const Score2 score(a.scale, a.cap);
  float mx[HPW][4], sm[HPW][4];
#pragma unroll
  for (int i = 0; i < HPW; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      mx[i][r] = NEG;
      sm[i][r] = 0.f;
    }
  int64_t row0 = w.key_row(w.t_first * KT + w.lo);
  int64_t row1 = w.key_row(w.t_first * KT + 16 + w.lo);
  for (int t = w.t_first; t < w.t_end; ++t) {
    const int kb = t * KT;
    const bool full = kb >= w.full_lo && kb + KT <= w.full_hi;
    u16x8 k0[DT], k1[DT];
    w.load_k(k0, row0, w.kvh[0]);
    w.load_k(k1, row1, w.kvh[0]);
    const int64_t cur0 = row0, cur1 = row1;
    const int idist0 = w.dist(0, kb + w.lo);
    const float dist0 = (float)idist0;
    row0 = w.key_row(kb + KT + w.lo);         // next tile's page lookup
    row1 = w.key_row(kb + KT + 16 + w.lo);
#pragma unroll
    for (int i = 0; i < HPW; ++i) {
      if (i > 0 && w.fresh(i)) {
        w.load_k(k0, cur0, w.kvh[i]);
        w.load_k(k1, cur1, w.kvh[i]);
      }
      const floatx4 d0 = w.dot(i, k0), d1 = w.dot(i, k1);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float s0 = score(d0[r], w.slope2[i], dist0 + (float)r);
        float s1 = score(d1[r], w.slope2[i], dist0 + (float)(r - 16));
        if (!full) {
          if (w.masked(idist0 + r)) s0 = NEG;
          if (w.masked(idist0 + r - 16)) s1 = NEG;
        }
        const float mn = fmaxf(mx[i][r], fmaxf(s0, s1));
        sm[i][r] = sm[i][r] * __builtin_amdgcn_exp2f(mx[i][r] - mn) +
                   __builtin_amdgcn_exp2f(s0 - mn) +
                   __builtin_amdgcn_exp2f(s1 - mn);
        mx[i][r] = mn;
      }
    }
  }
  // combine the 16 lanes of a row
#pragma unroll
  for (int i = 0; i < HPW; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float M = mx[i][r];
#pragma unroll
      for (int off = 8; off > 0; off >>= 1)
        M = fmaxf(M, __shfl_xor(M, off, WAVE));
      float L = sm[i][r] * __builtin_amdgcn_exp2f(mx[i][r] - M);
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) L += __shfl_xor(L, off, WAVE);
      const int qrow = w.qbase + w.hi * 4 + r;
      if (w.lo == 0 && qrow < w.qlen && w.hbase + i < a.H)
        a.lse[(int64_t)(w.q_start + qrow) * a.H + w.hbase + i] =
            M + __builtin_amdgcn_logf(L);
    }
}

// HPW heads per wave, DT k-steps of 32 (Dp <= 32*DT), ET value tiles of 16
// (E <= 16*ET; FAST: equal). H <= 32. Register plan at 4 heads of 128: 128
// for the value sums, 64 for Q; everything else that lives across a tile
// (lse, the mixing matrix) waits in LDS.
template <int HPW, int DT, int ET, bool FAST>
__global__ __launch_bounds__(512) void talk_values_kernel(PrefillArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  const int lane = threadIdx.x & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const int nwaves = blockDim.x / WAVE;
  const int qtile = (int)gridDim.x - 1 - (int)blockIdx.x;
  WaveTile<HPW, DT, FAST> w(a, blockIdx.y, qtile, wid * HPW, lane);
  if (w.qbase >= w.qlen) return;              // whole workgroup
  w.load_q();
  const int lo = w.lo, hi = w.hi, H = a.H, hbase = w.hbase;
  const Score2 score(a.scale, a.cap);
  const int E = FAST ? 16 * ET : a.E;
  const int PP = ((H + 7) & ~7) + 8;          // p pitch: heads of one pair
  uint16_t* p_hi = lds;                       // [QT*KT][PP]
  uint16_t* p_lo = p_hi + QT * KT * PP;
  uint16_t* w_lds = p_lo + QT * KT * PP;      // [H][QT][WP]
  uint16_t* t_lds = w_lds + H * QT * WP;      // [2 terms][2][64 lanes][8]
  float* lse_lds = reinterpret_cast<float*>(t_lds + 4 * WAVE * 8);  // [H][QT]

  // mixing matrix as A operand: rows = new heads, inner = old heads
  bool t_exact = true;
  for (int m = 0; m < 2; ++m) {
    u16x8 fh, fl;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int row = m * 16 + lo, g = hi * 8 + e;
      const float t = row < H && g < H ? a.talk[row * H + g] : 0.f;
      fh[e] = f32_to_bf16(t);
      const float rest = t - bf16_to_f32(fh[e]);
      fl[e] = f32_to_bf16(rest);
      t_exact = t_exact && rest == 0.f;
    }
    if (wid == 0) {
      *reinterpret_cast<u16x8*>(t_lds + (m * WAVE + lane) * 8) = fh;
      *reinterpret_cast<u16x8*>(t_lds + ((2 + m) * WAVE + lane) * 8) = fl;
    }
  }
  t_exact = __all(t_exact);
  for (int i = threadIdx.x; i < H * QT; i += blockDim.x) {
    const int qrow = min(w.qbase + i % QT, w.qlen - 1);
    lse_lds[i] = a.lse[(int64_t)(w.q_start + qrow) * H + i / QT];
  }
  // head slots past H that the mixing reads: zero once
  for (int i = threadIdx.x; i < QT * KT; i += blockDim.x)
    for (int g = H; g < ((H + 7) & ~7); ++g) {
      p_hi[i * PP + g] = 0;
      p_lo[i * PP + g] = 0;
    }
  __syncthreads();
  floatx4 acc[HPW][ET];
#pragma unroll
  for (int i = 0; i < HPW; ++i)
#pragma unroll
    for (int c = 0; c < ET; ++c) acc[i][c] = floatx4{0, 0, 0, 0};

  for (int t = w.t_first; t < w.t_end; ++t) {
    const int kb = t * KT;
    const bool full = kb >= w.full_lo && kb + KT <= w.full_hi;
#pragma unroll 1
    for (int sub = 0; sub < 2; ++sub) {
      const int64_t row = w.key_row(kb + sub * 16 + lo);
      const int idist0 = w.dist(0, kb + sub * 16 + lo);
      const float dist0 = (float)idist0;
      u16x8 kf[DT];
      constexpr int HP = HPW < 2 ? 1 : 2;     // heads stored together
#pragma unroll
      for (int i0 = 0; i0 < HPW; i0 += HP) {
        float p[HP][4];
#pragma unroll
        for (int j = 0; j < HP; ++j) {
          const int i = i0 + j;
          if (w.fresh(i)) w.load_k(kf, row, w.kvh[i]);
          const floatx4 d = w.dot(i, kf);
          const f32x4 lse = *reinterpret_cast<const f32x4*>(
              lse_lds + min(hbase + i, H - 1) * QT + hi * 4);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            p[j][r] = __builtin_amdgcn_exp2f(
                score(d[r], w.slope2[i], dist0 + (float)r) - lse[r]);
            if (!full && w.masked(idist0 + r)) p[j][r] = 0.f;
          }
        }
        // (row, key) pair -> its heads, two bf16 terms
        const int h = hbase + i0;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int pos = ((hi * 4 + r) * KT + sub * 16 + lo) * PP + h;
          const float p0 = p[0][r], p1 = HP == 2 ? p[HP - 1][r] : 0.f;
          const uint32_t ph = pack_bf16(p0, p1);
          const uint32_t pl =
              pack_bf16(p0 - __builtin_bit_cast(float, ph << 16),
                        p1 - __builtin_bit_cast(float, ph & 0xffff0000u));
          if (HP == 2 && (FAST || h + 1 < H)) {
            *reinterpret_cast<uint32_t*>(p_hi + pos) = ph;
            *reinterpret_cast<uint32_t*>(p_lo + pos) = pl;
          } else if (FAST || h < H) {
            p_hi[pos] = (uint16_t)ph;
            p_lo[pos] = (uint16_t)pl;
          }
        }
      }
    }
    __syncthreads();

    // mix: 16 pairs (one row, 16 keys) per step
#pragma unroll 1
    for (int grp = wid; grp < QT * KT / 16; grp += nwaves) {
      u16x8 bh = u16x8{0, 0, 0, 0, 0, 0, 0, 0}, bl = bh;
      if (hi * 8 < H) {
        const int at = (grp * 16 + lo) * PP + hi * 8;
        bh = *reinterpret_cast<const u16x8*>(p_hi + at);
        bl = *reinterpret_cast<const u16x8*>(p_lo + at);
      }
      const bf16x8 ph = *reinterpret_cast<bf16x8*>(&bh);
      const bf16x8 pl = *reinterpret_cast<bf16x8*>(&bl);
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        if (m * 16 >= H) continue;
        const bf16x8 th = *reinterpret_cast<const bf16x8*>(
            t_lds + (m * WAVE + lane) * 8);
        floatx4 c = floatx4{0, 0, 0, 0};
        c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(th, pl, c, 0, 0, 0);
        if (!t_exact)
          c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              *reinterpret_cast<const bf16x8*>(
                  t_lds + ((2 + m) * WAVE + lane) * 8), ph, c, 0, 0, 0);
        c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(th, ph, c, 0, 0, 0);
        const uint32_t c01 = pack_bf16(c[0], c[1]);
        const uint32_t c23 = pack_bf16(c[2], c[3]);
        uint16_t* wp = w_lds + ((m * 16 + hi * 4) * QT + grp / 2) * WP +
                       (grp & 1) * 16 + lo;
        const int left = H - (m * 16 + hi * 4);
        if (left > 0) wp[0] = (uint16_t)c01;
        if (left > 1) wp[QT * WP] = (uint16_t)(c01 >> 16);
        if (left > 2) wp[2 * QT * WP] = (uint16_t)c23;
        if (left > 3) wp[3 * QT * WP] = (uint16_t)(c23 >> 16);
      }
    }
    __syncthreads();

    // values: this lane's 8 tokens; groups of 8 never straddle a page
    const int t8 = kb + hi * 8;
    const int tv = min(t8, w.len - 1);
    const uint16_t* vp =
        a.vc + ((int64_t)w.bt[tv / w.bs()] * a.G * E + lo) * w.bs() +
        (tv & ~7) % w.bs();
    const bool tail = kb + KT > w.len;
    bf16x8 wf[HPW];
#pragma unroll
    for (int i = 0; i < HPW; ++i)
      wf[i] = *reinterpret_cast<const bf16x8*>(
          w_lds + (min(hbase + i, H - 1) * QT + lo) * WP + hi * 8);
    const uint16_t* vp0 = vp + w.kvh[0] * E * w.bs();
#pragma unroll
    for (int c = 0; c < ET; ++c) {
      u16x8 vf = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
      for (int i = 0; i < HPW; ++i) {
        if (w.fresh(i) && (FAST || c * 16 + lo < E)) {
          vf = *reinterpret_cast<const u16x8*>(
              (i == 0 ? vp0 : vp + w.kvh[i] * E * w.bs()) +
              c * 16 * w.bs());
          if (tail) {                         // stale slots: not even 0 * x
#pragma unroll
            for (int e = 0; e < 8; ++e)
              if (t8 + e >= w.len) vf[e] = 0;
          }
        }
        acc[i][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            wf[i], *reinterpret_cast<bf16x8*>(&vf), acc[i][c], 0, 0, 0);
      }
    }
  }

  // ---- epilogue: gate and store ------------------------------------------
#pragma unroll
  for (int i = 0; i < HPW; ++i) {
    const int h = hbase + i;
    if (h >= H) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int qrow = w.qbase + hi * 4 + r;
      if (qrow >= w.qlen) continue;
      const int64_t row = w.q_start + qrow;
      float f = 1.f;
      if (a.gate != nullptr)
        f = 1.f / (1.f + __expf(-bf16_to_f32(a.gate[row * a.gate_stride + h])));
#pragma unroll
      for (int c = 0; c < ET; ++c) {
        const int dim = c * 16 + lo;
        if (FAST || dim < E)
          a.out[row * a.out_stride + (int64_t)h * E + dim] =
              f32_to_bf16(acc[i][c][r] * f);
      }
    }
  }
}

template <int HPW, int DT, int ET, bool FAST>
void launch(const PrefillArgs& a, int max_q, int B, hipStream_t stream) {
  const int groups = cdiv(a.H, HPW);
  hipLaunchKernelGGL((talk_stats_kernel<HPW, DT, FAST>),
                     dim3(cdiv(max_q, 4 * QT), B, groups), dim3(256), 0,
                     stream, a);
  const int PP = ((a.H + 7) & ~7) + 8;
  const int lds = (2 * QT * KT * PP + a.H * QT * WP + 4 * WAVE * 8) *
                      (int)sizeof(uint16_t) +
                  a.H * QT * (int)sizeof(float);
  auto* fn = talk_values_kernel<HPW, DT, ET, FAST>;
  static int granted = 64 << 10;              // default dynamic LDS limit
  if (lds > granted) {
    TORCH_CHECK(hipFuncSetAttribute(
                    (const void*)fn,
                    hipFuncAttributeMaxDynamicSharedMemorySize, lds) ==
                    hipSuccess, "dynamic LDS");
    granted = lds;
  }
  hipLaunchKernelGGL(fn, dim3(cdiv(max_q, QT), B), dim3(groups * WAVE), lds,
                     stream, a);
}

template <int HPW>
void by_size(const PrefillArgs& a, int max_q, int B, hipStream_t stream) {
  const bool even = a.bs == 16 && a.H % HPW == 0 && (a.H / a.G) % HPW == 0;
#define HELIX_ET(DT)                                                         \
  if (a.E <= 32) launch<HPW, DT, 2, false>(a, max_q, B, stream);             \
  else if (a.E <= 64) launch<HPW, DT, 4, false>(a, max_q, B, stream);        \
  else launch<HPW, DT, 8, false>(a, max_q, B, stream)
  if (even && a.Dp == 128 && a.E == 128)
    launch<HPW, 4, 8, true>(a, max_q, B, stream);
  else if (even && a.Dp == 64 && a.E == 64)
    launch<HPW, 2, 4, true>(a, max_q, B, stream);
  else if (a.Dp <= 64) { HELIX_ET(2); }
  else { HELIX_ET(4); }
#undef HELIX_ET
}

}  // namespace

// Largest shapes the MFMA kernel takes; callers use talk_attn_rows beyond.
bool talk_prefill_fits(int64_t H, int64_t Dp, int64_t E) {
  return H <= 32 && Dp <= 128 && E <= 128;
}

void talk_attn_prefill(torch::Tensor out, torch::Tensor q, torch::Tensor kc,
                       torch::Tensor vc, torch::Tensor block_tables,
                       torch::Tensor cu_seqlens, torch::Tensor seq_lens,
                       int64_t max_q, double scale, double cap,
                       int64_t window, c10::optional<torch::Tensor> slopes,
                       torch::Tensor talk,
                       c10::optional<torch::Tensor> gate,
                       torch::Tensor lse) {
  const int64_t T = q.size(0), H = q.size(1), Dp = q.size(2);
  const int64_t B = cu_seqlens.numel() - 1;
  if (T == 0 || B <= 0) return;
  const int64_t G = kc.size(1), bs = kc.size(2), E = vc.size(2);
  TORCH_CHECK(talk_prefill_fits(H, Dp, E) && H % G == 0);
  TORCH_CHECK(q.scalar_type() == torch::kBFloat16 &&
              kc.scalar_type() == torch::kBFloat16 &&
              vc.scalar_type() == torch::kBFloat16 &&
              out.scalar_type() == torch::kBFloat16);
  TORCH_CHECK(q.is_contiguous() && kc.is_contiguous() && vc.is_contiguous());
  TORCH_CHECK(kc.size(3) == Dp && Dp % 8 == 0 && bs % 8 == 0);
  TORCH_CHECK(vc.size(0) == kc.size(0) && vc.size(1) == G &&
              vc.size(3) == bs, "V cache is [nblk, G, E, bs]");
  TORCH_CHECK(out.dim() == 2 && out.size(0) == T && out.size(1) == H * E &&
              out.stride(1) == 1);
  TORCH_CHECK(block_tables.scalar_type() == torch::kInt32 &&
              block_tables.size(0) >= B && block_tables.stride(1) == 1);
  TORCH_CHECK(cu_seqlens.scalar_type() == torch::kInt32 &&
              cu_seqlens.is_contiguous());
  TORCH_CHECK(seq_lens.scalar_type() == torch::kInt32 &&
              seq_lens.numel() == B && seq_lens.is_contiguous());
  if (slopes.has_value())
    TORCH_CHECK(slopes->scalar_type() == torch::kFloat32 &&
                slopes->numel() == H && slopes->is_contiguous());
  TORCH_CHECK(talk.scalar_type() == torch::kFloat32 &&
              talk.numel() == H * H && talk.is_contiguous());
  TORCH_CHECK(lse.scalar_type() == torch::kFloat32 &&
              lse.numel() == T * H && lse.is_contiguous());
  if (gate.has_value())
    TORCH_CHECK(gate->scalar_type() == torch::kBFloat16 &&
                gate->size(0) == T && gate->size(1) == H &&
                gate->stride(1) == 1);
  PrefillArgs a;
  a.out = (uint16_t*)out.data_ptr();
  a.out_stride = out.stride(0);
  a.q = (const uint16_t*)q.data_ptr();
  a.kc = (const uint16_t*)kc.data_ptr();
  a.vc = (const uint16_t*)vc.data_ptr();
  a.bt = block_tables.data_ptr<int>();
  a.bt_stride = block_tables.stride(0);
  a.cu_q = cu_seqlens.data_ptr<int>();
  a.seq_len = seq_lens.data_ptr<int>();
  a.slopes = slopes.has_value() ? slopes->data_ptr<float>() : nullptr;
  a.talk = talk.data_ptr<float>();
  a.lse = lse.data_ptr<float>();
  a.gate = gate.has_value() ? (const uint16_t*)gate->data_ptr() : nullptr;
  a.gate_stride = gate.has_value() ? gate->stride(0) : 0;
  a.scale = (float)scale;
  a.cap = (float)cap;
  a.window = (int)window;
  a.H = H;
  a.G = G;
  a.Dp = Dp;
  a.E = E;
  a.bs = bs;
  auto stream = at::hip::getCurrentHIPStream();
  // heads of a wave should share their K and V rows; 8 waves at most
  const int HG = H / G;
  if (HG % 4 == 0 || H > 16) by_size<4>(a, max_q, B, stream);
  else if (HG % 2 == 0 || H > 8) by_size<2>(a, max_q, B, stream);
  else by_size<1>(a, max_q, B, stream);
}
