// Paged attention of prompt portions (bf16), causal.
//
// A workgroup has 128 queries of one head, each of its 4 waves 32 of them.
// Scores are computed transposed (key x query), so a lane has one query: row
// statistics are per lane, and 8 neighbouring keys of a lane's weights are
// an operand of the value product as they are. Tiles of 64 keys come
// straight from the pages (page numbers looked up a tile ahead) and wait in
// LDS while the next one is on its way in registers.
#include "attn.h"

using namespace helix;

namespace {

constexpr int NT = 256;
constexpr int QT = 128;                       // queries of a workgroup
constexpr int KT = 64;                        // keys of a tile

struct Prompt {
  Attn a;
  const int* cu;               // [B + 1] query rows
  const int* seq_lens;         // [B] keys, the newest tokens last
  int q_tiles, seqs, vec;
};

template <int NK, int NV, bool SIG>
__global__ __launch_bounds__(NT, NK + NV > 16 ? 1 : 2)
void attn_prompt_kernel(uint16_t* __restrict__ out,
                        const uint16_t* __restrict__ q,
                        const uint16_t* __restrict__ kc,
                        const uint16_t* __restrict__ vc, Prompt m) {
  constexpr int KP = NK * 32 + 8, VP = KT + 8;
  __shared__ uint16_t kl[KT * KP];
  __shared__ uint16_t vl[NV * 16 * VP];
  const Attn& A = m.a;
  // all tiles of a (sequence, head) on one XCD: they share keys and values,
  // and so do the heads of a group, which are neighbours there
  const int xcd = blockIdx.x & 7, at = blockIdx.x >> 3;
  const int total = m.seqs * A.H, chunk = cdiv(total, 8);
  const int sh = xcd * chunk + at / m.q_tiles;
  if (at / m.q_tiles >= chunk || sh >= total) return;
  const int b = sh / A.H, h = sh % A.H, g = h / (A.H / A.G);
  // the latest tiles see the most keys: they go first
  const int q0 = (m.q_tiles - 1 - at % m.q_tiles) * QT;
  const int row0 = m.cu[b], qlen = m.cu[b + 1] - row0;
  if (q0 >= qlen) return;
  const int klen = m.seq_lens[b], ctx = klen - qlen;
  const int* bt = A.bt + (int64_t)b * A.max_blocks;

  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  u16x8 qf[2][NK];
  float mul[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int qi = min(q0 + wid * 32 + u * 16 + lo, qlen - 1);
    const uint16_t* qr = q + (row0 + qi) * A.q_stride + h * A.Dp;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const int d = s * 32 + hi * 8;
      qf[u][s] = d < A.Dp ? ld_u16x8(qr + d) : zero;
    }
    mul[u] = head_mul(A, h) * row_mul(A, row0 + qi);
  }
  const float add = head_add(A, h);
  const int half = (A.E + 1) / 2;

  // Loads without branches, so that all are under way at once: what lies
  // past the end is clamped and meets a zero query column, a zero weight or
  // a value dimension that is not stored.
  u16x8 kreg[NK], vreg[NV / 2];
  int kpage[NK], vpage;
  auto pages = [&](int t) {
#pragma unroll
    for (int c = 0; c < NK; ++c)
      kpage[c] = bt[min(t + (c * NT + tid) / (NK * 4), klen - 1) / A.bs];
    vpage = bt[min(t + tid % 8 * 8, klen - 1) / A.bs];
  };
  auto load = [&](int t) {
#pragma unroll
    for (int c = 0; c < NK; ++c) {
      const int e = c * NT + tid;
      const int key = min(t + e / (NK * 4), klen - 1);
      kreg[c] = ld_u16x8(
          kc + (((int64_t)kpage[c] * A.G + g) * A.bs + key % A.bs) * A.Dp +
          min(e % (NK * 4) * 8, A.Dp - 8));
    }
    const uint16_t* vb = vc + ((int64_t)vpage * A.G + g) * A.E * A.bs +
                         (t + tid % 8 * 8) % A.bs;
#pragma unroll
    for (int c = 0; c < NV / 2; ++c) {
      const int r = c * 32 + tid / 8;         // row of the value tiles
      const int e = min((r >> 4 & 1) * half + (r >> 5) * 16 + (r & 15),
                        A.E - 1);
      vreg[c] = ld_u16x8(vb + (int64_t)e * A.bs);
    }
  };

  floatx4 acc[NV][2];
  float m_run[2] = {NEG, NEG}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int d = 0; d < NV; ++d) acc[d][0] = acc[d][1] = floatx4{0, 0, 0, 0};
  const int last = min(klen, ctx + q0 + QT);
  const int qa = ctx + q0 + wid * 32, qz = qa + 31;  // of this wave

  pages(0);
  load(0);
  pages(min(KT, last - 1));
  for (int t = 0; t < last; t += KT) {
    __syncthreads();
#pragma unroll
    for (int c = 0; c < NK; ++c) {
      const int e = c * NT + tid;
      *reinterpret_cast<u16x8*>(kl + paired_row(e / (NK * 4)) * KP +
                                e % (NK * 4) * 8) = kreg[c];
    }
#pragma unroll
    for (int c = 0; c < NV / 2; ++c)
      *reinterpret_cast<u16x8*>(vl + (c * 32 + tid / 8) * VP + tid % 8 * 8) =
          vreg[c];
    __syncthreads();
    if (t + KT < last) {
      load(t + KT);
      pages(t + 2 * KT);
    }
    if (t > qz) continue;

    floatx4 s[2][2][2];                       // [32 keys][half][query tile]
#pragma unroll
    for (int w = 0; w < 2; ++w)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        s[w][j][0] = s[w][j][1] = floatx4{0, 0, 0, 0};
        const uint16_t* row = kl + (w * 32 + j * 16 + lo) * KP + hi * 8;
#pragma unroll
        for (int c = 0; c < NK; ++c) {
          const u16x8 a = ld_u16x8(row + c * 32);
          s[w][j][0] = mfma16(a, qf[0][c], s[w][j][0]);
          s[w][j][1] = mfma16(a, qf[1][c], s[w][j][1]);
        }
      }
    const bool edge = t + KT - 1 > qa || t + KT > klen;
    u16x8 pf[2][2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float p[2][8], mx = m_run[u];
      const int qi = qa + u * 16 + lo;
#pragma unroll
      for (int w = 0; w < 2; ++w)
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float v = s[w][i >> 2][u][i & 3] * mul[u] + add;
          if (edge) {
            const int key = t + w * 32 + hi * 8 + i;
            if (key > qi || key >= klen) v = NEG;
          }
          p[w][i] = v;
          if constexpr (!SIG) mx = fmaxf(mx, v);
        }
      if constexpr (SIG) {
#pragma unroll
        for (int w = 0; w < 2; ++w) {
#pragma unroll
          for (int i = 0; i < 8; ++i) p[w][i] = sigmoid2(p[w][i]);
          pf[w][u] = pack8(p[w]);
        }
      } else {
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
        for (int w = 0; w < 2; ++w) {
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            p[w][i] = __builtin_amdgcn_exp2f(p[w][i] - base);
            l[u] += p[w][i];
          }
          pf[w][u] = pack8(p[w]);
        }
      }
    }
#pragma unroll
    for (int w = 0; w < 2; ++w)
#pragma unroll
      for (int d = 0; d < NV; ++d) {
        const u16x8 a = ld_u16x8(vl + (d * 16 + lo) * VP + w * 32 + hi * 8);
        acc[d][0] = mfma16(a, pf[w][0], acc[d][0]);
        acc[d][1] = mfma16(a, pf[w][1], acc[d][1]);
      }
  }

#pragma unroll
  for (int u = 0; u < 2; ++u) {
    float f = A.out_scale;
    if constexpr (!SIG) {
      l[u] += __shfl_xor(l[u], 16, WAVE);
      l[u] += __shfl_xor(l[u], 32, WAVE);
      f /= l[u];
    }
    const int qi = q0 + wid * 32 + u * 16 + lo;
    if (qi >= qlen) continue;
    const int64_t r = row0 + qi;
    uint16_t* dst = out + r * A.out_stride + h * A.E;
#pragma unroll
    for (int d = 0; d < NV; d += 2) {
      const int pair = d * 8 + hi * 4;
      if (pair >= half) continue;
      float x[4], y[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        x[i] = acc[d][u][i] * f;
        y[i] = acc[d + 1][u][i] * f;
        if (pair + i < half) turn_back(A, r, pair + i, x[i], y[i]);
      }
      if (A.gate != nullptr) {
        const int at = h * A.E + pair;
        const uint16_t* gp = (const uint16_t*)A.gate + r * A.gate_stride + at;
        if (m.vec) {
          float gx[4], gy[4];
          ldv<4>(gp, gx);
          ldv<4>(gp + half, gy);
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            x[i] *= sigmoid_s<uint16_t>(gx[i]);
            y[i] *= sigmoid_s<uint16_t>(gy[i]);
          }
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            if (pair + i >= half) continue;
            x[i] *= gate_of<uint16_t>(A, r, at + i);
            if (half + pair + i < A.E)
              y[i] *= gate_of<uint16_t>(A, r, at + half + i);
          }
        }
      }
      if (m.vec) {
        st_bf16x4(dst + pair, x);
        st_bf16x4(dst + half + pair, y);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          if (pair + i >= half) continue;
          dst[pair + i] = f32_to_bf16(x[i]);
          if (half + pair + i < A.E) dst[half + pair + i] = f32_to_bf16(y[i]);
        }
      }
    }
  }
}

}  // namespace

bool attn_fits(torch::Tensor q, int64_t vdim);

void attn_prompt(torch::Tensor out, torch::Tensor q, torch::Tensor kc,
                 torch::Tensor vc, torch::Tensor bt, torch::Tensor cu,
                 torch::Tensor seq_lens, int64_t max_q, double scale,
                 double out_scale, bool sigmoid, OptT temp, OptT bias,
                 OptT vcs, OptT row_scale, OptT gate) {
  TORCH_CHECK(q.dim() == 3 && q.scalar_type() == kc.scalar_type());
  const int64_t T = q.size(0), H = q.size(1);
  const int B = seq_lens.numel();
  Prompt m{};
  m.a = attn_args(kc, vc, bt, T, H, scale, out_scale, temp, bias, vcs,
                  row_scale, gate);
  query_rows(m.a, q);
  TORCH_CHECK(attn_fits(q, m.a.E));
  for (const auto& t : {cu, seq_lens})
    TORCH_CHECK(t.scalar_type() == torch::kInt32 && t.is_contiguous());
  TORCH_CHECK(cu.numel() == B + 1 && bt.size(0) >= B);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == T &&
              out.size(1) == H * m.a.E && out.stride(1) == 1 &&
              out.scalar_type() == torch::kBFloat16);
  if (B == 0 || T == 0) return;
  m.a.out_stride = out.stride(0);
  m.cu = cu.data_ptr<int>();
  m.seq_lens = seq_lens.data_ptr<int>();
  m.q_tiles = cdiv((int)max_q, QT);
  m.seqs = B;
  m.vec = m.a.E % 8 == 0 && out.stride(0) % 4 == 0 &&
          (uintptr_t)out.data_ptr() % 8 == 0 && m.a.gate_stride % 4 == 0 &&
          (uintptr_t)m.a.gate % 8 == 0;
  const dim3 grid(8 * cdiv(B * H, 8) * m.q_tiles);
#define HELIX_AP(NK, NV)                                                     \
  do {                                                                       \
    if (sigmoid)                                                             \
      hipLaunchKernelGGL((attn_prompt_kernel<NK, NV, true>), grid, dim3(NT), \
                         0, at::hip::getCurrentHIPStream(),                  \
                         (uint16_t*)out.data_ptr(),                          \
                         (const uint16_t*)q.data_ptr(),                      \
                         (const uint16_t*)kc.data_ptr(),                     \
                         (const uint16_t*)vc.data_ptr(), m);                 \
    else                                                                     \
      hipLaunchKernelGGL((attn_prompt_kernel<NK, NV, false>), grid,          \
                         dim3(NT), 0, at::hip::getCurrentHIPStream(),        \
                         (uint16_t*)out.data_ptr(),                          \
                         (const uint16_t*)q.data_ptr(),                      \
                         (const uint16_t*)kc.data_ptr(),                     \
                         (const uint16_t*)vc.data_ptr(), m);                 \
  } while (0)
  const int half = (m.a.E + 1) / 2, D = m.a.Dp;
  if (D <= 32 && half <= 16) HELIX_AP(1, 2);
  else if (D <= 64 && half <= 32) HELIX_AP(2, 4);
  else if (D <= 128 && half <= 64) HELIX_AP(4, 8);
  else HELIX_AP(8, 16);
#undef HELIX_AP
}
