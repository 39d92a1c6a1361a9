// Epilogues of the fused input projection.
//
//  - unit_qkv_cache: per-head unit-RMS q and k (no weight), value mixing
//    with the values an earlier layer had for the same token, and the
//    paged-cache write. q/k: one workgroup per token. v: one workgroup per
//    16 tokens, transposed through LDS so that 16 lanes write the 16
//    neighbouring slots of one value dim.
//  - poly_norm: a N(z) + b N(z^2) + c N(z^3) + e over a token's feed-forward
//    vector, N = division by the root mean square.
//  - layer_epilogue: both in one launch, since both consume the same
//    projection output and neither fills the chip alone when few tokens
//    decode. grid.y selects the role.
//
// Cache layout: K [nblk, G, bs, Dp] with rows padded to Dp (zeros), so a
// row is a run of 16-byte loads; V TRANSPOSED inside a block,
// [nblk, G, E, bs], so 8 consecutive tokens of one value dim are one
// 16-byte load. That is the B operand of the weights-times-values MFMA, and
// it lets the attention kernels read V straight into registers.
#include "../elem.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int NT = 256;
constexpr int NW = NT / WAVE;

template <typename S>
struct QkvArgs {
  const S* z;              // [T, ...] projection output
  int64_t z_stride;
  int q_off, k_off, v_off;
  S* q_out;                // [T, H, Dp]
  S* k_cache;
  S* v_cache;
  const int64_t* slots;    // [T], < 0: no cache write
  S* v_first;              // [T, G*E]: written when first, else read
  const float* lam;        // null: no value mixing
  int first;
  float eps;
  int H, G, D, Dp, E, bs;
  int64_t T;
  int lph;                 // lanes per head of the vector path, 0: scalar
  int v_split;             // workgroups that share one token group's columns
};

template <typename S>
__device__ __forceinline__ void unit_head(const S* src, S* dst, int D,
                                          int Dp, float eps, int lane) {
  float ss = 0.f;
  for (int d = lane; d < D; d += WAVE) {
    const float v = ld1(src + d);
    ss += v * v;
  }
  ss = wave_reduce_sum(ss);
  const float inv = 1.f / sqrtf(ss / D + eps);
  for (int d = lane; d < Dp; d += WAVE) {
    st1(dst + d, d < D ? ld1(src + d) * inv : 0.f);
  }
}

// q and k heads of one token. vec: heads are runs of aligned 8-element
// vectors; lph lanes (a power of two) hold one head, 64 / lph heads a wave.
template <typename S>
__device__ __forceinline__ void qk_role(const QkvArgs<S>& p) {
  const int64_t t = blockIdx.x;
  if (t >= p.T) return;
  const int wid = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const S* src = p.z + t * p.z_stride;
  const int64_t slot = p.slots[t];
  const int64_t blk = slot >= 0 ? slot / p.bs : 0;
  const int off = slot >= 0 ? (int)(slot % p.bs) : 0;
  if (p.lph > 0) {
    const int per = WAVE / p.lph, sub = lane / p.lph;
    const int d = (lane % p.lph) * 8;
    for (int h0 = wid * per; h0 < p.H + p.G; h0 += NW * per) {
      const int h = h0 + sub;
      const bool live = h < p.H + p.G && d < p.D;
      float v[8];
      float ss = 0.f;
      if (live) {
        ldv<8>(src + (h < p.H ? p.q_off + h * p.D
                              : p.k_off + (h - p.H) * p.D) + d, v);
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += v[i] * v[i];
      }
      for (int o = p.lph / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, WAVE);
      if (!live) continue;
      const float inv = 1.f / sqrtf(ss / p.D + p.eps);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] *= inv;
      if (h < p.H)
        stv<8>(p.q_out + (t * p.H + h) * p.Dp + d, v);
      else if (slot >= 0)
        stv<8>(p.k_cache +
                   ((blk * p.G + h - p.H) * p.bs + off) * p.Dp + d, v);
    }
    return;
  }
  for (int h = wid; h < p.H + p.G; h += NW) {
    if (h < p.H) {
      unit_head<S>(src + p.q_off + h * p.D,
                   p.q_out + (t * p.H + h) * p.Dp, p.D, p.Dp, p.eps, lane);
    } else if (slot >= 0) {
      const int g = h - p.H;
      unit_head<S>(src + p.k_off + g * p.D,
                   p.k_cache + ((blk * p.G + g) * p.bs + off) * p.Dp, p.D,
                   p.Dp, p.eps, lane);
    }
  }
}

// Values of VTOK tokens, VCOL columns at a time. (g, e) = (i / E, i % E)
// makes a column of [blk, G, E, bs] one index i.
constexpr int VTOK = 16, VCOL = 128, VPITCH = VCOL + 1;

template <typename S>
__device__ __forceinline__ void v_role(const QkvArgs<S>& p, float* tile) {
  const int n = p.G * p.E;
  const int64_t t0 = (int64_t)(blockIdx.x / p.v_split) * VTOK;
  if (t0 >= p.T) return;
  const int nt = (int)min((int64_t)VTOK, p.T - t0);
  const float lam = (p.lam != nullptr && !p.first) ? *p.lam : 0.f;
  const int my = threadIdx.x % VTOK;          // token this lane writes
  const int64_t slot = my < nt ? p.slots[t0 + my] : -1;
  const int64_t dst = slot >= 0 ? slot / p.bs * n * p.bs + slot % p.bs : 0;
  for (int c0 = (blockIdx.x % p.v_split) * VCOL; c0 < n;
       c0 += p.v_split * VCOL) {
    const int nc = min(VCOL, n - c0);
    for (int i = threadIdx.x; i < nt * VCOL; i += NT) {
      const int tk = i / VCOL, c = i % VCOL;
      if (c >= nc) continue;
      float v = ld1(p.z + (t0 + tk) * p.z_stride + p.v_off + c0 + c);
      if (p.lam != nullptr) {
        S* carry = p.v_first + (t0 + tk) * n + c0 + c;
        if (p.first) st1(carry, v);
        else v = (1.f - lam) * v + lam * ld1(carry);
      }
      tile[tk * VPITCH + c] = v;
    }
    __syncthreads();
    if (slot >= 0)
      for (int c = threadIdx.x / VTOK; c < nc; c += NT / VTOK)
        st1(p.v_cache + dst + (int64_t)(c0 + c) * p.bs,
            tile[my * VPITCH + c]);
    __syncthreads();
  }
}

template <typename S>
struct PolyArgs {
  const S* z;
  int64_t z_stride;
  S* out;
  int64_t out_stride;
  const float* coef;       // a, b, c, e
  float eps;
  int F;
};

// VN: elements per access (8 when every row start is aligned, else 1).
template <typename S, int VN>
__device__ __forceinline__ void poly_role(const PolyArgs<S>& p, float* red) {
  const S* z = p.z + (int64_t)blockIdx.x * p.z_stride;
  S* o = p.out + (int64_t)blockIdx.x * p.out_stride;
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  for (int d = threadIdx.x * VN; d < p.F; d += NT * VN) {
    float e[VN];
    if constexpr (VN > 1) ldv<VN>(z + d, e);
    else e[0] = ld1(z + d);
#pragma unroll
    for (int i = 0; i < VN; ++i) {
      const float q = e[i] * e[i];
      s2 += q;
      s4 += q * q;
      s6 += q * q * q;
    }
  }
  s2 = wave_reduce_sum(s2);
  s4 = wave_reduce_sum(s4);
  s6 = wave_reduce_sum(s6);
  if ((threadIdx.x & (WAVE - 1)) == 0) {
    const int w = threadIdx.x / WAVE;
    red[w] = s2;
    red[NW + w] = s4;
    red[2 * NW + w] = s6;
  }
  __syncthreads();
  s2 = s4 = s6 = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) {
    s2 += red[w];
    s4 += red[NW + w];
    s6 += red[2 * NW + w];
  }
  const float n = (float)p.F;
  const float a = p.coef[0] / sqrtf(s2 / n + p.eps);
  const float b = p.coef[1] / sqrtf(s4 / n + p.eps);
  const float c = p.coef[2] / sqrtf(s6 / n + p.eps);
  const float e0 = p.coef[3];
  for (int d = threadIdx.x * VN; d < p.F; d += NT * VN) {
    float e[VN];
    if constexpr (VN > 1) ldv<VN>(z + d, e);
    else e[0] = ld1(z + d);
#pragma unroll
    for (int i = 0; i < VN; ++i)
      e[i] = ((c * e[i] + b) * e[i] + a) * e[i] + e0;
    if constexpr (VN > 1) stv<VN>(o + d, e);
    else st1(o + d, e[0]);
  }
}

template <typename S>
__global__ __launch_bounds__(NT) void unit_qkv_kernel(QkvArgs<S> p) {
  __shared__ float tile[VTOK * VPITCH];
  if (blockIdx.y == 0) qk_role<S>(p);
  else v_role<S>(p, tile);
}

template <typename S, int VN>
__global__ __launch_bounds__(NT) void poly_norm_kernel(PolyArgs<S> p) {
  __shared__ float red[3 * NW];
  poly_role<S, VN>(p, red);
}

template <typename S, int VN>
__global__ __launch_bounds__(NT) void layer_epilogue_kernel(QkvArgs<S> a,
                                                            PolyArgs<S> b) {
  __shared__ float sh[VTOK * VPITCH];
  if (blockIdx.y == 0) {
    if (blockIdx.x < a.T) poly_role<S, VN>(b, sh);
  } else if (blockIdx.y == 1) {
    qk_role<S>(a);
  } else {
    v_role<S>(a, sh);
  }
}

template <typename S>
QkvArgs<S> qkv_args(torch::Tensor z, int64_t q_off, int64_t k_off,
                    int64_t v_off, torch::Tensor q_out, torch::Tensor k_cache,
                    torch::Tensor v_cache, torch::Tensor slots,
                    c10::optional<torch::Tensor> v_first,
                    c10::optional<torch::Tensor> lam, bool first, int64_t D,
                    double eps) {
  QkvArgs<S> a;
  const int64_t T = z.size(0);
  a.H = q_out.size(1);
  a.Dp = q_out.size(2);
  a.G = k_cache.size(1);
  a.bs = k_cache.size(2);
  a.E = v_cache.size(2);
  a.D = D;
  TORCH_CHECK(z.dim() == 2 && z.stride(1) == 1);
  TORCH_CHECK(q_out.is_contiguous() && k_cache.is_contiguous() &&
              v_cache.is_contiguous() && slots.is_contiguous());
  TORCH_CHECK(q_out.size(0) == T && slots.numel() == T &&
              slots.scalar_type() == torch::kInt64);
  TORCH_CHECK(k_cache.size(3) == a.Dp && D <= a.Dp && v_cache.size(1) == a.G &&
              v_cache.size(3) == a.bs && v_cache.size(0) == k_cache.size(0));
  TORCH_CHECK(q_out.scalar_type() == z.scalar_type() &&
              k_cache.scalar_type() == z.scalar_type() &&
              v_cache.scalar_type() == z.scalar_type());
  TORCH_CHECK(q_off >= 0 && q_off + a.H * D <= z.size(1) && k_off >= 0 &&
              k_off + a.G * D <= z.size(1) && v_off >= 0 &&
              v_off + a.G * a.E <= z.size(1));
  a.lam = nullptr;
  a.v_first = nullptr;
  if (lam.has_value()) {
    TORCH_CHECK(lam->scalar_type() == torch::kFloat32 && lam->numel() == 1);
    TORCH_CHECK(v_first.has_value() && v_first->is_contiguous() &&
                v_first->scalar_type() == z.scalar_type() &&
                v_first->numel() == T * a.G * a.E,
                "value mixing needs equally shaped values in both layers");
    a.lam = lam->data_ptr<float>();
    a.v_first = (S*)v_first->data_ptr();
  }
  a.first = first;
  a.z = (const S*)z.data_ptr();
  a.z_stride = z.stride(0);
  a.q_off = q_off;
  a.k_off = k_off;
  a.v_off = v_off;
  a.q_out = (S*)q_out.data_ptr();
  a.k_cache = (S*)k_cache.data_ptr();
  a.v_cache = (S*)v_cache.data_ptr();
  a.slots = slots.data_ptr<int64_t>();
  a.eps = (float)eps;
  a.T = T;
  const uint64_t m = 8 * sizeof(S) - 1;
  const bool vec = D % 8 == 0 && D <= 8 * WAVE && q_off % 8 == 0 &&
                   k_off % 8 == 0 && a.z_stride % 8 == 0 &&
                   ((uint64_t)a.z & m) == 0;
  a.lph = 0;
  if (vec)
    for (a.lph = 1; a.lph * 8 < D;) a.lph *= 2;
  a.v_split = std::min(16, cdiv(a.G * a.E, VCOL));
  return a;
}

// workgroups along x: one per token, or per (token group, column share)
template <typename S>
int grid_x(const QkvArgs<S>& a) {
  return std::max((int)a.T, cdiv((int)a.T, VTOK) * a.v_split);
}

template <typename S>
PolyArgs<S> poly_args(torch::Tensor z, torch::Tensor out, torch::Tensor coef,
                      double eps) {
  TORCH_CHECK(z.dim() == 2 && out.dim() == 2 && z.sizes() == out.sizes() &&
              z.stride(1) == 1 && out.stride(1) == 1 &&
              z.scalar_type() == out.scalar_type());
  TORCH_CHECK(coef.numel() == 4 && coef.is_contiguous() &&
              coef.scalar_type() == torch::kFloat32);
  PolyArgs<S> b;
  b.z = (const S*)z.data_ptr();
  b.z_stride = z.stride(0);
  b.out = (S*)out.data_ptr();
  b.out_stride = out.stride(0);
  b.coef = coef.data_ptr<float>();
  b.eps = (float)eps;
  b.F = z.size(1);
  return b;
}

template <typename S>
bool poly_aligned(const PolyArgs<S>& b) {
  const uint64_t m = 8 * sizeof(S) - 1;
  return b.F % 8 == 0 && b.z_stride % 8 == 0 && b.out_stride % 8 == 0 &&
         ((uint64_t)b.z & m) == 0 && ((uint64_t)b.out & m) == 0;
}

}  // namespace

#define HELIX_BY_TYPE(t, what, ...)                                          \
  if ((t).scalar_type() == torch::kBFloat16) {                               \
    using S = uint16_t;                                                      \
    __VA_ARGS__                                                              \
  } else if ((t).scalar_type() == torch::kFloat32) {                         \
    using S = float;                                                         \
    __VA_ARGS__                                                              \
  } else {                                                                   \
    TORCH_CHECK(false, what ": bf16 or fp32");                               \
  }

void unit_qkv_cache(torch::Tensor z, int64_t q_off, int64_t k_off,
                    int64_t v_off, torch::Tensor q_out, torch::Tensor k_cache,
                    torch::Tensor v_cache, torch::Tensor slots,
                    c10::optional<torch::Tensor> v_first,
                    c10::optional<torch::Tensor> lam, bool first,
                    int64_t head_dim, double eps) {
  if (z.size(0) == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  HELIX_BY_TYPE(z, "unit_qkv_cache", {
    auto a = qkv_args<S>(z, q_off, k_off, v_off, q_out, k_cache, v_cache,
                         slots, v_first, lam, first, head_dim, eps);
    hipLaunchKernelGGL((unit_qkv_kernel<S>), dim3(grid_x(a), 2), dim3(NT), 0,
                       stream, a);
  })
}

void poly_norm(torch::Tensor out, torch::Tensor z, torch::Tensor coef,
               double eps) {
  if (z.size(0) == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  HELIX_BY_TYPE(z, "poly_norm", {
    auto b = poly_args<S>(z, out, coef, eps);
    if (poly_aligned(b))
      hipLaunchKernelGGL((poly_norm_kernel<S, 8>), dim3(z.size(0)), dim3(NT),
                         0, stream, b);
    else
      hipLaunchKernelGGL((poly_norm_kernel<S, 1>), dim3(z.size(0)), dim3(NT),
                         0, stream, b);
  })
}

void layer_epilogue(torch::Tensor z, int64_t q_off, int64_t k_off,
                    int64_t v_off, torch::Tensor q_out, torch::Tensor k_cache,
                    torch::Tensor v_cache, torch::Tensor slots,
                    c10::optional<torch::Tensor> v_first,
                    c10::optional<torch::Tensor> lam, bool first,
                    int64_t head_dim, double eps, torch::Tensor ff_out,
                    torch::Tensor ff_z, torch::Tensor coef) {
  if (z.size(0) == 0) return;
  TORCH_CHECK(ff_z.size(0) == z.size(0) &&
              ff_z.scalar_type() == z.scalar_type());
  auto stream = at::hip::getCurrentHIPStream();
  HELIX_BY_TYPE(z, "layer_epilogue", {
    auto a = qkv_args<S>(z, q_off, k_off, v_off, q_out, k_cache, v_cache,
                         slots, v_first, lam, first, head_dim, eps);
    auto b = poly_args<S>(ff_z, ff_out, coef, eps);
    if (poly_aligned(b))
      hipLaunchKernelGGL((layer_epilogue_kernel<S, 8>), dim3(grid_x(a), 3),
                         dim3(NT), 0, stream, a, b);
    else
      hipLaunchKernelGGL((layer_epilogue_kernel<S, 1>), dim3(grid_x(a), 3),
                         dim3(NT), 0, stream, a, b);
  })
}
