// Prefill attention with talking heads on MFMA (bf16), straight from the
// paged cache.
//
// One workgroup owns 16 query rows and ALL heads: mixing softmaxed weights
// across heads needs them side by side. Waves own HPW consecutive heads.
//
//   sweep 1  every wave streams the window's K once and keeps per-lane
//            running (max, sum) of its heads' scores. Waves are independent:
//            no LDS, no barrier; K rows go from L2 straight into B operands.
//   sweep 2  per 32 keys: waves recompute their heads' scores, write
//            p = exp(s - M) / L in fp32 to LDS; after a barrier each wave
//            forms w_h = sum_g talk[h, g] p_g for its heads in fp32 (the
//            mixing matrix sits in scalar registers), already in A-operand
//            layout, and multiplies with V.
//
// V pages are stored [E][bs] (8 tokens of a dim contiguous), so V fragments
// are plain 16-byte loads as well and nothing is transposed in LDS.
//
// MFMA f32_16x16x32_bf16 lane layout:
//   A: lane l holds A[row = l&15][k = (l>>4)*8 + i]
//   B: lane l holds B[k = (l>>4)*8 + i][col = l&15]
//   C: lane l holds C[row = (l>>4)*4 + r][col = l&15]
#include "elem.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int QT = 16;         // query rows per workgroup
constexpr int KT = 32;         // keys per sweep-2 tile
constexpr int PP = KT + 4;     // p row pitch (floats)
constexpr float NEG = -1e30f;

struct PrefillArgs {
  uint16_t* out;               // [T, H*E], row stride out_stride
  int64_t out_stride;
  const uint16_t* q;           // [T, H, Dp]
  const uint16_t* kc;          // [nblk, G, bs, Dp]
  const uint16_t* vc;          // [nblk, G, E, bs]
  const int* bt;               // [B, bt_stride]
  int bt_stride;
  const int* cu_q;             // [B+1] rows of q per sequence
  const int* seq_len;          // [B] keys per sequence, these rows included
  const float* slopes;         // [H] or null
  const float* talk;           // [H, H] or null
  const uint16_t* gate;        // [T, H] logits, row stride gate_stride
  int64_t gate_stride;
  float scale, cap;
  int window, H, G, Dp, E, bs;
};

// HPW heads per wave, DT k-steps of 32 (Dp <= 32*DT), ET value tiles of 16
// (E <= 16*ET).
template <int HPW, int DT, int ET>
__global__ __launch_bounds__(512) void talk_prefill_kernel(PrefillArgs a) {
  extern __shared__ float p_lds[];            // [H][QT][PP]
  const int seq = blockIdx.y;
  const int q_start = a.cu_q[seq];
  const int qlen = a.cu_q[seq + 1] - q_start;
  const int len = a.seq_len[seq];
  const int ctx = len - qlen;
  // later tiles see more keys under a causal mask: start them first
  const int qbase = ((int)gridDim.x - 1 - (int)blockIdx.x) * QT;
  if (qbase >= qlen) return;

  const int lane = threadIdx.x & (WAVE - 1);
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const int lo = lane & 15, hi = lane >> 4;
  const int H = a.H, G = a.G, HG = H / G;
  const int hbase = wid * HPW;
  const int* bt = a.bt + (int64_t)seq * a.bt_stride;
  const float inv_cap = a.cap > 0.f ? 1.f / a.cap : 0.f;

  bf16x8 qf[HPW][DT];
  float slope[HPW];
  int kvh[HPW];
#pragma unroll
  for (int i = 0; i < HPW; ++i) {
    const int h = min(hbase + i, H - 1);      // idle heads repeat the last
    kvh[i] = h / HG;
    slope[i] = a.slopes != nullptr ? a.slopes[h] : 0.f;
    const int r = qbase + lo;
#pragma unroll
    for (int kt = 0; kt < DT; ++kt) {
      const int d = kt * 32 + hi * 8;
      u16x8 raw = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (r < qlen && d < a.Dp)
        raw = *reinterpret_cast<const u16x8*>(
            a.q + ((int64_t)(q_start + r) * H + h) * a.Dp + d);
      qf[i][kt] = *reinterpret_cast<bf16x8*>(&raw);
    }
  }

  const int kv_hi = min(len, ctx + qbase + QT);
  const int kv_lo = a.window > 0 ? max(0, ctx + qbase - a.window + 1) : 0;
  const int t_first = kv_lo / KT, t_end = (kv_hi + KT - 1) / KT;
  const int qpos0 = ctx + qbase + hi * 4;     // position of C row r = 0
  // every (row, key) of a tile in [full_lo, full_hi) is visible
  const int full_hi = ctx + qbase + 1;
  const int full_lo =
      a.window > 0 ? max(0, ctx + qbase + QT - a.window) : 0;

  // element offset of the key row this lane feeds (head 0 of the page)
  auto key_row = [&](int tok) -> int64_t {
    const int t = min(tok, len - 1);
    return ((int64_t)bt[t / a.bs] * G * a.bs + t % a.bs) * a.Dp;
  };
  auto load_k = [&](u16x8 (&kf)[DT], int64_t row, int g) {
    const uint16_t* p = a.kc + row + (int64_t)g * a.bs * a.Dp;
#pragma unroll
    for (int kt = 0; kt < DT; ++kt) {
      const int d = kt * 32 + hi * 8;
      kf[kt] = d < a.Dp ? *reinterpret_cast<const u16x8*>(p + d)
                        : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  };
  auto dot = [&](const bf16x8 (&qq)[DT], u16x8 (&kf)[DT]) -> floatx4 {
    floatx4 s = floatx4{0, 0, 0, 0};
#pragma unroll
    for (int kt = 0; kt < DT; ++kt)
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          qq[kt], *reinterpret_cast<bf16x8*>(&kf[kt]), s, 0, 0, 0);
    return s;
  };
  auto score = [&](float d, int i, int r, int tp, bool full) -> float {
    const int dist = qpos0 + r - tp;
    float s = cap_and_bias<uint16_t>(d, a.scale, a.cap, inv_cap, slope[i],
                                     dist);
    if (!full && (dist < 0 || (a.window > 0 && dist >= a.window))) s = NEG;
    return s;
  };

  // ---- sweep 1: softmax statistics --------------------------------------
  float mx[HPW][4], sm[HPW][4];
#pragma unroll
  for (int i = 0; i < HPW; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      mx[i][r] = NEG;
      sm[i][r] = 0.f;
    }
  for (int t = t_first; t < t_end; ++t) {
    const int kb = t * KT;
    const bool full = kb >= full_lo && kb + KT <= full_hi;
    const int64_t row0 = key_row(kb + lo), row1 = key_row(kb + 16 + lo);
    u16x8 k0[DT], k1[DT];
#pragma unroll
    for (int i = 0; i < HPW; ++i) {
      if (i == 0 || kvh[i] != kvh[i - 1]) {
        load_k(k0, row0, kvh[i]);
        load_k(k1, row1, kvh[i]);
      }
      const floatx4 d0 = dot(qf[i], k0), d1 = dot(qf[i], k1);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float s0 = score(d0[r], i, r, kb + lo, full);
        const float s1 = score(d1[r], i, r, kb + 16 + lo, full);
        const float mn = fmaxf(mx[i][r], fmaxf(s0, s1));
        sm[i][r] = sm[i][r] * __expf(mx[i][r] - mn) + __expf(s0 - mn) +
                   __expf(s1 - mn);
        mx[i][r] = mn;
      }
    }
  }
  // combine the 16 lanes of a row; mx becomes M + log(L)
#pragma unroll
  for (int i = 0; i < HPW; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float M = mx[i][r];
#pragma unroll
      for (int off = 8; off > 0; off >>= 1)
        M = fmaxf(M, __shfl_xor(M, off, WAVE));
      float L = sm[i][r] * __expf(mx[i][r] - M);
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) L += __shfl_xor(L, off, WAVE);
      mx[i][r] = M;
      sm[i][r] = 1.f / L;
    }

  // ---- sweep 2: weights, mixing, values ----------------------------------
  floatx4 acc[HPW][ET];
#pragma unroll
  for (int i = 0; i < HPW; ++i)
#pragma unroll
    for (int c = 0; c < ET; ++c) acc[i][c] = floatx4{0, 0, 0, 0};

  for (int t = t_first; t < t_end; ++t) {
    const int kb = t * KT;
    const bool full = kb >= full_lo && kb + KT <= full_hi;
    {
      const int64_t row0 = key_row(kb + lo), row1 = key_row(kb + 16 + lo);
      u16x8 k0[DT], k1[DT];
#pragma unroll
      for (int i = 0; i < HPW; ++i) {
        if (i == 0 || kvh[i] != kvh[i - 1]) {
          load_k(k0, row0, kvh[i]);
          load_k(k1, row1, kvh[i]);
        }
        const floatx4 d0 = dot(qf[i], k0), d1 = dot(qf[i], k1);
        if (hbase + i < H) {
          float* pr = p_lds + ((hbase + i) * QT + hi * 4) * PP + lo;
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float s0 = score(d0[r], i, r, kb + lo, full);
            const float s1 = score(d1[r], i, r, kb + 16 + lo, full);
            pr[r * PP] = __expf(s0 - mx[i][r]) * sm[i][r];
            pr[r * PP + 16] = __expf(s1 - mx[i][r]) * sm[i][r];
          }
        }
      }
    }
    __syncthreads();

    float w[HPW][8];
    if (a.talk != nullptr) {
#pragma unroll
      for (int i = 0; i < HPW; ++i)
#pragma unroll
        for (int e = 0; e < 8; ++e) w[i][e] = 0.f;
      for (int g = 0; g < H; ++g) {
        const float* pr = p_lds + (g * QT + lo) * PP + hi * 8;
        float p[8];
        ldv<8>(pr, p);
#pragma unroll
        for (int i = 0; i < HPW; ++i) {
          const float tk = a.talk[min(hbase + i, H - 1) * H + g];
#pragma unroll
          for (int e = 0; e < 8; ++e) w[i][e] += tk * p[e];
        }
      }
    } else {
#pragma unroll
      for (int i = 0; i < HPW; ++i)
        ldv<8>(p_lds + (min(hbase + i, H - 1) * QT + lo) * PP + hi * 8, w[i]);
    }
    bf16x8 wf[HPW];
#pragma unroll
    for (int i = 0; i < HPW; ++i) {
      u16x8 raw;
#pragma unroll
      for (int e = 0; e < 8; ++e) raw[e] = f32_to_bf16(w[i][e]);
      wf[i] = *reinterpret_cast<bf16x8*>(&raw);
    }

    // V: this lane's 8 tokens; groups of 8 never straddle a page
    const int t8 = kb + hi * 8;
    const int tv = min(t8, len - 1);
    const int64_t vrow =
        (int64_t)bt[tv / a.bs] * G * a.E * a.bs + (tv & ~7) % a.bs;
    const bool tail = kb + KT > len;
#pragma unroll
    for (int c = 0; c < ET; ++c) {
      const int dim = c * 16 + lo;
      u16x8 vf = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
      for (int i = 0; i < HPW; ++i) {
        if (i == 0 || kvh[i] != kvh[i - 1]) {
          if (dim < a.E) {
            vf = *reinterpret_cast<const u16x8*>(
                a.vc + vrow + ((int64_t)kvh[i] * a.E + dim) * a.bs);
            if (tail) {                       // stale slots: not even 0 * x
#pragma unroll
              for (int e = 0; e < 8; ++e)
                if (t8 + e >= len) vf[e] = 0;
            }
          }
        }
        acc[i][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            wf[i], *reinterpret_cast<bf16x8*>(&vf), acc[i][c], 0, 0, 0);
      }
    }
    __syncthreads();
  }

  // ---- epilogue: gate and store ------------------------------------------
#pragma unroll
  for (int i = 0; i < HPW; ++i) {
    const int h = hbase + i;
    if (h >= H) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int qrow = qbase + hi * 4 + r;
      if (qrow >= qlen) continue;
      const int64_t row = q_start + qrow;
      float f = 1.f;
      if (a.gate != nullptr)
        f = 1.f / (1.f + __expf(-bf16_to_f32(a.gate[row * a.gate_stride + h])));
#pragma unroll
      for (int c = 0; c < ET; ++c) {
        const int dim = c * 16 + lo;
        if (dim < a.E)
          a.out[row * a.out_stride + (int64_t)h * a.E + dim] =
              f32_to_bf16(acc[i][c][r] * f);
      }
    }
  }
}

template <int HPW, int DT, int ET>
void launch(const PrefillArgs& a, int n_qtiles, int B, hipStream_t stream) {
  const int waves = cdiv(a.H, HPW);
  const int lds = a.H * QT * PP * (int)sizeof(float);
  auto* fn = talk_prefill_kernel<HPW, DT, ET>;
  static int granted = 64 << 10;              // default dynamic LDS limit
  if (lds > granted) {
    TORCH_CHECK(hipFuncSetAttribute(
                    (const void*)fn,
                    hipFuncAttributeMaxDynamicSharedMemorySize, lds) ==
                    hipSuccess, "dynamic LDS");
    granted = lds;
  }
  hipLaunchKernelGGL(fn, dim3(n_qtiles, B), dim3(waves * WAVE), lds, stream,
                     a);
}

template <int HPW>
void by_size(const PrefillArgs& a, int n_qtiles, int B, hipStream_t stream) {
#define HELIX_ET(DT)                                                         \
  if (a.E <= 32) launch<HPW, DT, 2>(a, n_qtiles, B, stream);                 \
  else if (a.E <= 64) launch<HPW, DT, 4>(a, n_qtiles, B, stream);            \
  else launch<HPW, DT, 8>(a, n_qtiles, B, stream)
  if (a.Dp <= 64) { HELIX_ET(2); }
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
                       c10::optional<torch::Tensor> talk,
                       c10::optional<torch::Tensor> gate) {
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
  if (talk.has_value())
    TORCH_CHECK(talk->scalar_type() == torch::kFloat32 &&
                talk->numel() == H * H && talk->is_contiguous());
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
  a.talk = talk.has_value() ? talk->data_ptr<float>() : nullptr;
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
  const int n_qtiles = cdiv((int)max_q, QT);
  if (H <= 8) by_size<1>(a, n_qtiles, B, stream);
  else if (H <= 16) by_size<2>(a, n_qtiles, B, stream);
  else by_size<4>(a, n_qtiles, B, stream);
}
