// What the attention kernels of this folder share.
//
// Cache pages: keys [G][block][Dp], values [G][E][block]. Weights are a
// softmax, or each a sigmoid of its own score (no normalisation), from
// scores q.k * scale (* temp[head]) (+ bias[head]). Where values were cached
// turned by their position, a row's result is turned back by its own
// (vcs[row]: cosine and sine of every pair). A row may have a factor of its
// own on all its scores (row_scale), and its results a gate per value:
// sigmoid(gate[row][h E + e]).
//
// Value dimensions come in pairs (m, m + half), half = ceil(E / 2): tile 2 t
// of the value product has dimensions 16 t .. of the first half, tile 2 t + 1
// those of the second, so a lane holds both of a pair and turns them itself.
#pragma once
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

namespace helix {

constexpr float LOG2E = 1.4426950408889634f;
constexpr float NEG = -1e30f;

struct Attn {
  const int* bt;               // [seqs, max_blocks]
  const float *temp, *bias;    // [H] or null
  const float2* vcs;           // [rows, E / 2] or null
  const float* row_scale;      // [rows] or null
  const void* gate;            // [rows, H E] in the storage type, or null
  int64_t out_stride, q_stride, gate_stride;
  int max_blocks, bs, H, G, Dp, E;
  float scale, out_scale;
};

// score * log2(e) = dot * mul + add
__device__ __forceinline__ float head_mul(const Attn& m, int h) {
  return m.scale * LOG2E * (m.temp != nullptr ? m.temp[h] : 1.f);
}
__device__ __forceinline__ float head_add(const Attn& m, int h) {
  return m.bias != nullptr ? m.bias[h] * LOG2E : 0.f;
}

__device__ __forceinline__ float row_mul(const Attn& m, int64_t r) {
  return m.row_scale != nullptr ? m.row_scale[r] : 1.f;
}
// The gate's logits lie in the storage type, n-th value of row r.
template <typename S>
__device__ __forceinline__ float gate_of(const Attn& m, int64_t r, int n) {
  if (m.gate == nullptr) return 1.f;
  return sigmoid_s<S>(ld1((const S*)m.gate + r * m.gate_stride + n));
}

// 1 / (1 + 2^-x)
__device__ __forceinline__ float sigmoid2(float x) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-x));
}

// Turns the pair (a, b) of row r back.
__device__ __forceinline__ void turn_back(const Attn& m, int64_t r, int pair,
                                          float& a, float& b) {
  if (m.vcs == nullptr) return;
  const float2 c = m.vcs[r * (m.E / 2) + pair];
  const float u = a * c.x + b * c.y;
  b = b * c.x - a * c.y;
  a = u;
}

using OptT = c10::optional<torch::Tensor>;

// Per-row operands of the output: the values' own turn and the gate.
inline void row_operands(Attn& m, int64_t rows, torch::ScalarType type,
                         OptT vcs, OptT gate) {
  if (vcs.has_value()) {
    TORCH_CHECK(m.E % 2 == 0 && vcs->scalar_type() == torch::kFloat32 &&
                vcs->is_contiguous() && vcs->numel() == rows * m.E);
    m.vcs = (const float2*)vcs->data_ptr<float>();
  }
  if (gate.has_value()) {
    TORCH_CHECK(gate->dim() == 2 && gate->size(0) == rows &&
                gate->size(1) == m.H * m.E && gate->stride(1) == 1 &&
                gate->scalar_type() == type);
    m.gate = gate->data_ptr();
    m.gate_stride = gate->stride(0);
  }
}

// Queries [rows, H, Dp], the rows anywhere (16-byte aligned).
inline void query_rows(Attn& m, const torch::Tensor& q) {
  TORCH_CHECK(q.dim() == 3 && q.size(2) == m.Dp && q.stride(2) == 1 &&
              q.stride(1) == m.Dp && q.stride(0) % 8 == 0 &&
              (uintptr_t)q.data_ptr() % 16 == 0);
  m.q_stride = q.stride(0);
}

inline Attn attn_args(torch::Tensor kc, torch::Tensor vc, torch::Tensor bt,
                      int64_t rows, int64_t heads, double scale,
                      double out_scale, OptT temp, OptT bias, OptT vcs,
                      OptT row_scale, OptT gate) {
  Attn m{};
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.is_contiguous() &&
              vc.is_contiguous() && kc.scalar_type() == vc.scalar_type());
  m.H = heads;
  m.G = kc.size(1);
  m.bs = kc.size(2);
  m.Dp = kc.size(3);
  m.E = vc.size(2);
  TORCH_CHECK(m.G > 0 && m.H % m.G == 0 && m.bs % 8 == 0 && m.Dp % 8 == 0);
  TORCH_CHECK(vc.size(0) == kc.size(0) && vc.size(1) == m.G &&
              vc.size(3) == m.bs);
  TORCH_CHECK(bt.scalar_type() == torch::kInt32 && bt.dim() == 2 &&
              bt.stride(1) == 1);
  m.bt = bt.data_ptr<int>();
  m.max_blocks = bt.stride(0);
  for (const auto& t : {temp, bias})
    if (t.has_value())
      TORCH_CHECK(t->scalar_type() == torch::kFloat32 &&
                  t->is_contiguous() && t->numel() == heads);
  if (temp.has_value()) m.temp = temp->data_ptr<float>();
  if (bias.has_value()) m.bias = bias->data_ptr<float>();
  row_operands(m, rows, kc.scalar_type(), vcs, gate);
  if (row_scale.has_value()) {
    TORCH_CHECK(row_scale->scalar_type() == torch::kFloat32 &&
                row_scale->is_contiguous() && row_scale->numel() == rows);
    m.row_scale = row_scale->data_ptr<float>();
  }
  m.scale = (float)scale;
  m.out_scale = (float)out_scale;
  return m;
}

}  // namespace helix
