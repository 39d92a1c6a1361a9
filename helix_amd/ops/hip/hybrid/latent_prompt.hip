// Latent attention for prompts: keys and values of the visible context are
// spelled out per head by two GEMMs, this kernel is the attention itself.
//
//   k  [rows, H, dim_pad]   unrotated keys       kr [rows, rot_pad] shared
//   vt [H, E, rows]         values, transposed
//
// A workgroup has 128 queries of one head, each of its 4 waves 32 of them.
// Scores are computed transposed (key x query), so a lane has one query: the
// row statistics are per lane, and 8 neighbouring keys of a lane's scores
// are the B operand of the value product as they are. Tiles of 64 keys wait
// in LDS while the next one is on its way in registers.
#include "tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr int NT = 256;
constexpr int QT = 128;                       // queries of a workgroup
constexpr int KT = 64;                        // keys of a tile
constexpr float NEG = -1e30f;

struct Prompt {
  const int* cu;               // [B + 1] query rows
  const int* start;            // [B] first context row
  const int* length;           // [B] context rows, newest last
  int64_t z_stride, kr_stride, out_stride, gate_stride, rows;
  int head_cols, H, E, dim_pad, rot_pad, window, q_tiles, seqs, vec;
  float scale;                 // times log2(e)
};

template <int NK, int NV>
__global__ __launch_bounds__(NT, NK + NV > 16 ? 1 : 2)
void latent_prompt_kernel(uint16_t* __restrict__ out,
                          const uint16_t* __restrict__ q,
                          const uint16_t* __restrict__ k,
                          const uint16_t* __restrict__ kr,
                          const uint16_t* __restrict__ vt,
                          const uint16_t* __restrict__ gate, Prompt m) {
  constexpr int KP = NK * 32 + 8, VP = KT + 8;
  __shared__ uint16_t kl[KT * KP];
  __shared__ uint16_t vl[NV * 16 * VP];
  // all tiles of a (sequence, head) on one XCD: they share keys and values
  const int xcd = blockIdx.x & 7, at = blockIdx.x >> 3;
  const int sh = xcd + 8 * (at / m.q_tiles);
  if (sh >= m.seqs * m.H) return;
  const int b = sh / m.H, h = sh % m.H;
  // the latest tiles see the most keys: they go first
  const int q0 = (m.q_tiles - 1 - at % m.q_tiles) * QT;
  const int row0 = m.cu[b], qlen = m.cu[b + 1] - row0;
  if (q0 >= qlen) return;
  const int klen = m.length[b], ctx = klen - qlen;
  const int64_t k0 = m.start[b];

  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  u16x8 qf[2][NK];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int qi = min(q0 + wid * 32 + u * 16 + lo, qlen - 1);
    const uint16_t* qr = q + (row0 + qi) * m.z_stride + h * m.head_cols;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const int d = s * 32 + hi * 8;
      qf[u][s] = d < m.head_cols ? ld_u16x8(qr + d) : zero;
    }
  }

  // Loads without branches, so that all are under way at once: addresses
  // past the end are clamped. What they bring meets a zero query column, a
  // zero weight or a value dimension that is not stored.
  u16x8 kreg[NK], vreg[NV / 2];
  const uint16_t* kh = k + h * m.dim_pad;
  const uint16_t* vh = vt + (int64_t)h * m.E * m.rows;
  auto load = [&](int t) {
#pragma unroll
    for (int c = 0; c < NK; ++c) {
      const int e = c * NT + tid, key = e / (NK * 4);
      const int d = min(e % (NK * 4) * 8, m.head_cols - 8);
      const int64_t r = k0 + min(t + key, klen - 1);
      const uint16_t* src = d < m.dim_pad
                                ? kh + r * m.H * m.dim_pad + d
                                : kr + r * m.kr_stride + d - m.dim_pad;
      kreg[c] = ld_u16x8(src);
    }
#pragma unroll
    for (int c = 0; c < NV / 2; ++c) {
      const int e = c * NT + tid, dim = min(e / 8, m.E - 1);
      const int64_t r = min(k0 + t + e % 8 * 8, m.rows - 8);
      vreg[c] = ld_u16x8(vh + dim * m.rows + r);
    }
  };

  floatx4 acc[NV][2];
  float m_run[2] = {NEG, NEG}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int d = 0; d < NV; ++d) acc[d][0] = acc[d][1] = floatx4{0, 0, 0, 0};
  const int last = min(klen, ctx + q0 + QT);
  const int first =
      m.window > 0 ? max(0, ctx + q0 - m.window + 1) / KT * KT : 0;
  // of this wave
  const int qa = ctx + q0 + wid * 32, qz = qa + 31;

  load(first);
  for (int t = first; t < last; t += KT) {
    __syncthreads();
#pragma unroll
    for (int c = 0; c < NK; ++c) {
      const int e = c * NT + tid;
      *reinterpret_cast<u16x8*>(kl + paired_row(e / (NK * 4)) * KP +
                                e % (NK * 4) * 8) = kreg[c];
    }
#pragma unroll
    for (int c = 0; c < NV / 2; ++c) {
      const int e = c * NT + tid;
      *reinterpret_cast<u16x8*>(vl + e / 8 * VP + e % 8 * 8) = vreg[c];
    }
    __syncthreads();
    if (t + KT < last) load(t + KT);
    if (t > qz || (m.window > 0 && t + KT - 1 <= qa - m.window)) continue;

    floatx4 s[2][2][2];                       // [32 keys][half][query tile]
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        s[g][j][0] = s[g][j][1] = floatx4{0, 0, 0, 0};
        const uint16_t* row = kl + (g * 32 + j * 16 + lo) * KP + hi * 8;
#pragma unroll
        for (int c = 0; c < NK; ++c) {
          const u16x8 a = ld_u16x8(row + c * 32);
          s[g][j][0] = mfma16(a, qf[0][c], s[g][j][0]);
          s[g][j][1] = mfma16(a, qf[1][c], s[g][j][1]);
        }
      }
    const bool edge = t + KT - 1 > qa || t + KT > klen ||
                      (m.window > 0 && t <= qz - m.window);
    u16x8 pf[2][2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float p[2][8], mx = m_run[u];
      const int qi = qa + u * 16 + lo;
#pragma unroll
      for (int g = 0; g < 2; ++g)
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float v = s[g][i >> 2][u][i & 3] * m.scale;
          if (edge) {
            const int key = t + g * 32 + hi * 8 + i;
            if (key > qi || key >= klen ||
                (m.window > 0 && qi - key >= m.window))
              v = NEG;
          }
          p[g][i] = v;
          mx = fmaxf(mx, v);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      if (!__all(mx == m_run[u])) {
        const float corr = __builtin_amdgcn_exp2f(m_run[u] - mx);
        l[u] *= corr;
        m_run[u] = mx;
#pragma unroll
        for (int d = 0; d < NV; ++d)
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[d][u][i] *= corr;
      }
      // a query that has seen no key yet keeps weights of exactly zero
      const float base = mx <= NEG ? 0.f : mx;
#pragma unroll
      for (int g = 0; g < 2; ++g) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          p[g][i] = __builtin_amdgcn_exp2f(p[g][i] - base);
          l[u] += p[g][i];
        }
        pf[g][u] = pack8(p[g]);
      }
    }
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int d = 0; d < NV; ++d) {
        const u16x8 a = ld_u16x8(vl + (d * 16 + lo) * VP + g * 32 + hi * 8);
        acc[d][0] = mfma16(a, pf[g][0], acc[d][0]);
        acc[d][1] = mfma16(a, pf[g][1], acc[d][1]);
      }
  }

#pragma unroll
  for (int u = 0; u < 2; ++u) {
    l[u] += __shfl_xor(l[u], 16, WAVE);
    l[u] += __shfl_xor(l[u], 32, WAVE);
    const int qi = q0 + wid * 32 + u * 16 + lo;
    if (qi >= qlen) continue;
    const int64_t r = row0 + qi;
    float f = 1.f / l[u];
    if (gate != nullptr)
      f *= sigmoid_s<uint16_t>(bf16_to_f32(gate[r * m.gate_stride + h]));
#pragma unroll
    for (int d = 0; d < NV; ++d) {
      const int e = d * 16 + hi * 4;
      uint16_t* dst = out + r * m.out_stride + h * m.E + e;
      const float v[4] = {acc[d][u][0] * f, acc[d][u][1] * f,
                          acc[d][u][2] * f, acc[d][u][3] * f};
      if (m.vec) {
        if (e < m.E) st_bf16x4(dst, v);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (e + i < m.E) dst[i] = f32_to_bf16(v[i]);
      }
    }
  }
}

}  // namespace

bool latent_prompt_fits(torch::Tensor z, int64_t dim_pad, int64_t rot_pad,
                        int64_t vdim) {
  return z.scalar_type() == torch::kBFloat16 && dim_pad + rot_pad <= 256 &&
         vdim <= 256;
}

void latent_prompt(torch::Tensor out, torch::Tensor z, int64_t q_at,
                   int64_t head_cols, int64_t heads, torch::Tensor k,
                   torch::Tensor kr, torch::Tensor vt, torch::Tensor cu,
                   torch::Tensor start, torch::Tensor length, int64_t max_q,
                   double scale, int64_t window, OptT gate) {
  const int B = start.numel(), H = heads;
  TORCH_CHECK(k.dim() == 2 && k.is_contiguous() && k.size(1) % H == 0);
  const int64_t rows = k.size(0), dim_pad = k.size(1) / H;
  const int64_t rot_pad = kr.size(1), E = vt.size(0) / H;
  TORCH_CHECK(latent_prompt_fits(z, dim_pad, rot_pad, E));
  TORCH_CHECK(dim_pad + rot_pad == head_cols && dim_pad % 8 == 0 &&
              rot_pad % 8 == 0 && q_at % 8 == 0);
  TORCH_CHECK(z.stride(1) == 1 && z.stride(0) % 8 == 0 &&
              q_at + H * head_cols <= z.size(1));
  TORCH_CHECK(kr.size(0) == rows && kr.stride(1) == 1 &&
              kr.stride(0) % 8 == 0);
  TORCH_CHECK(vt.is_contiguous() && vt.size(1) == rows && rows % 8 == 0 &&
              vt.size(0) == H * E);
  for (const auto& t : {k, kr, vt, out})
    TORCH_CHECK(t.scalar_type() == torch::kBFloat16);
  for (const auto& t : {cu, start, length})
    TORCH_CHECK(t.scalar_type() == torch::kInt32 && t.is_contiguous());
  TORCH_CHECK(cu.numel() == B + 1 && length.numel() == B);
  TORCH_CHECK(out.size(0) == z.size(0) && out.size(1) == H * E &&
              out.stride(1) == 1);
  Prompt m{};
  if (gate.has_value()) {
    TORCH_CHECK(gate->size(0) == out.size(0) && gate->size(1) == H &&
                gate->stride(1) == 1 &&
                gate->scalar_type() == torch::kBFloat16);
    m.gate_stride = gate->stride(0);
  }
  if (B == 0 || out.size(0) == 0) return;
  m.cu = cu.data_ptr<int>();
  m.start = start.data_ptr<int>();
  m.length = length.data_ptr<int>();
  m.z_stride = z.stride(0);
  m.kr_stride = kr.stride(0);
  m.out_stride = out.stride(0);
  m.rows = rows;
  m.head_cols = head_cols;
  m.H = H;
  m.E = E;
  m.dim_pad = dim_pad;
  m.rot_pad = rot_pad;
  m.window = window;
  m.q_tiles = cdiv((int)max_q, QT);
  m.seqs = B;
  m.vec = E % 4 == 0 && out.stride(0) % 4 == 0 &&
          (uintptr_t)out.data_ptr() % 8 == 0;
  m.scale = (float)(scale * 1.4426950408889634);
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(8 * cdiv(B * H, 8) * m.q_tiles);
#define HELIX_LP(NK, NV)                                                     \
  hipLaunchKernelGGL((latent_prompt_kernel<NK, NV>), grid, dim3(NT), 0,      \
                     stream, (uint16_t*)out.data_ptr(),                      \
                     (const uint16_t*)z.data_ptr() + q_at,                   \
                     (const uint16_t*)k.data_ptr(),                          \
                     (const uint16_t*)kr.data_ptr(),                         \
                     (const uint16_t*)vt.data_ptr(),                         \
                     gate.has_value() ? (const uint16_t*)gate->data_ptr()    \
                                      : nullptr,                             \
                     m)
#define HELIX_LP_V(NK)                                                       \
  if (E <= 64) HELIX_LP(NK, 4);                                              \
  else if (E <= 128) HELIX_LP(NK, 8);                                        \
  else HELIX_LP(NK, 16)
  if (head_cols <= 64) { HELIX_LP_V(2); }
  else if (head_cols <= 128) { HELIX_LP_V(4); }
  else if (head_cols <= 192) { HELIX_LP_V(6); }
  else { HELIX_LP_V(8); }
#undef HELIX_LP_V
#undef HELIX_LP
}
