// Matrix products of a mixture's experts, all of them in one launch:
//
//   out[r] = act(w[e] a[row(r)])   for the rows r of every expert e
//
// over the tiles that place() made of the experts' common list. a's row is
// that of the list itself, or (gather) of the token a list entry belongs to.
// act: none, or the square of relu.
//
// bf16 comes in two shapes. A row or two per expert: a wave streams weights
// straight into MFMA operands, the waves of a workgroup share the inner
// dimension and meet in LDS at the end. More: tiles through LDS, filled by
// direct loads; 16-byte pieces of a row are stored crosswise (piece ^ row % 8),
// so that operands leave LDS without bank conflicts. fp32 and odd sizes run a plain kernel.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;
using OptT = c10::optional<torch::Tensor>;

namespace {

constexpr int NT = 256, NW = NT / WAVE;

struct Mix {
  const int4* tiles;           // expert (-1: none), first row, rows
  const int* order;            // gather: [P] (token, choice) of a row
  int64_t a_stride;
  int N, K, choices, relu2, n_tiles, m_tiles;
};

__device__ __forceinline__ int64_t source_row(const Mix& m, int r) {
  return m.order != nullptr ? m.order[r] / m.choices : r;
}

__device__ __forceinline__ float finish(const Mix& m, float v) {
  if (!m.relu2) return v;
  const float u = fmaxf(v, 0.f);
  return u * u;
}

// Workgroups of neighbouring tiles on one XCD.
__device__ __forceinline__ int xcd_chunk(int orig, int nwg) {
  const int q = nwg / 8, r = nwg % 8;
  const int xcd = orig % 8, pos = orig / 8;
  return (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + pos;
}

// --- streams: 16 MI rows x 16 NI columns of a workgroup; a wave has every
// fourth stretch of 32 U of the inner dimension.
template <int MI, int NI, int U>
__global__ __launch_bounds__(NT) void expert_rows_kernel(
    uint16_t* __restrict__ out, const uint16_t* __restrict__ a,
    const uint16_t* __restrict__ w, Mix m) {
  constexpr int BM = MI * 16, BN = NI * 16, PITCH = BN + 4;
  __shared__ __attribute__((aligned(16))) float part[NW][BM * PITCH];
  const int n_tile = blockIdx.x % m.n_tiles;
  const int4 tile = m.tiles[blockIdx.x / m.n_tiles];
  if (tile.x < 0) return;
  const int n0 = n_tile * BN;
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const uint16_t* ap[MI];
  const uint16_t* wp[NI];
#pragma unroll
  for (int i = 0; i < MI; ++i)
    ap[i] = a + source_row(m, tile.y + min(i * 16 + lo, tile.z - 1)) *
                    m.a_stride;
#pragma unroll
  for (int j = 0; j < NI; ++j)
    wp[j] = w + ((int64_t)tile.x * m.N + min(n0 + j * 16 + lo, m.N - 1)) * m.K;

  floatx4 acc[NI][MI];
#pragma unroll
  for (int j = 0; j < NI; ++j)
#pragma unroll
    for (int i = 0; i < MI; ++i) acc[j][i] = floatx4{0, 0, 0, 0};
  // past the end the weights meet zeros
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  u16x8 ar[U][MI], wr[U][NI];
  auto load = [&](int k0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * 32 + hi * 8, kc = min(k, m.K - 8);
#pragma unroll
      for (int j = 0; j < NI; ++j) wr[u][j] = ld_u16x8(wp[j] + kc);
#pragma unroll
      for (int i = 0; i < MI; ++i) {
        ar[u][i] = ld_u16x8(ap[i] + kc);
        if (k >= m.K) ar[u][i] = zero;
      }
    }
  };
  constexpr int STEP = NW * U * 32;
  int k0 = wid * U * 32;
  if (k0 < m.K) load(k0);
  for (; k0 < m.K; k0 += STEP) {
    u16x8 af[U][MI], wf[U][NI];
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
      for (int j = 0; j < NI; ++j) wf[u][j] = wr[u][j];
#pragma unroll
      for (int i = 0; i < MI; ++i) af[u][i] = ar[u][i];
    }
    if (k0 + STEP < m.K) load(k0 + STEP);
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int j = 0; j < NI; ++j)
#pragma unroll
        for (int i = 0; i < MI; ++i)
          acc[j][i] = mfma16(wf[u][j], af[u][i], acc[j][i]);
  }
  // lane: columns 4 hi + r of row lo
#pragma unroll
  for (int j = 0; j < NI; ++j)
#pragma unroll
    for (int i = 0; i < MI; ++i)
      *reinterpret_cast<floatx4*>(part[wid] + (i * 16 + lo) * PITCH + j * 16 +
                                  hi * 4) = acc[j][i];
  __syncthreads();
  for (int e = tid; e < BM * BN / 4; e += NT) {
    const int r = e / (BN / 4), c = e % (BN / 4) * 4;
    if (r >= tile.z) continue;
    f32x4 s = *reinterpret_cast<const f32x4*>(part[0] + r * PITCH + c);
#pragma unroll
    for (int q = 1; q < NW; ++q) {
      const f32x4 p =
          *reinterpret_cast<const f32x4*>(part[q] + r * PITCH + c);
#pragma unroll
      for (int i = 0; i < 4; ++i) s[i] += p[i];
    }
    uint16_t* o = out + (int64_t)(tile.y + r) * m.N + n0 + c;
    if (m.N % 4 == 0) {
      const float v[4] = {finish(m, s[0]), finish(m, s[1]), finish(m, s[2]),
                          finish(m, s[3])};
      if (n0 + c < m.N) st_bf16x4(o, v);
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + c + i < m.N) o[i] = f32_to_bf16(finish(m, s[i]));
    }
  }
}

// --- tiles: BM x BN of a workgroup, WM x WN waves, inner dimension in
// steps of 64 (K % 64 == 0). The next step's tiles are on their way to one
// half of LDS while the other is worked on.
constexpr int BK = 64;
// instruction classes of the scheduling hints
constexpr int MFMA = 0x008, DS_READ = 0x100;

template <int BM, int BN, int WM, int WN>
__global__ __launch_bounds__(WM* WN* WAVE) void expert_tiles_kernel(
    uint16_t* __restrict__ out, const uint16_t* __restrict__ a,
    const uint16_t* __restrict__ w, Mix m) {
  constexpr int TH = WM * WN * WAVE;
  constexpr int MI = BM / WM / 16, NI = BN / WN / 16;
  constexpr int AT = BM * BK / (TH * 8), WT = BN * BK / (TH * 8);
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  const int lin = xcd_chunk(blockIdx.x, gridDim.x);
  const int4 tile = m.tiles[lin / m.n_tiles];
  if (tile.x < 0) return;
  const int n0 = lin % m.n_tiles * BN;
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int wr = wid / WN, wc = wid % WN;

  // this thread's 16-byte pieces of either tile
  const uint16_t *ap[AT], *wp[WT];
  const int row0 = tid / 8;
#pragma unroll
  for (int i = 0; i < AT; ++i) {
    const int row = i * (TH / 8) + row0;
    ap[i] = a + source_row(m, tile.y + min(row, tile.z - 1)) * m.a_stride +
            ((tid & 7) ^ (row & 7)) * 8;
  }
#pragma unroll
  for (int i = 0; i < WT; ++i) {
    const int row = i * (TH / 8) + row0;
    wp[i] = w + ((int64_t)tile.x * m.N + min(n0 + row, m.N - 1)) * m.K +
            ((tid & 7) ^ (row & 7)) * 8;
  }
  auto load = [&](int k0, uint16_t* dst) {
#pragma unroll
    for (int i = 0; i < AT; ++i)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(ap[i] + k0),
          (__attribute__((address_space(3))) uint32_t*)(dst +
                                                        (i * TH + tid) * 8),
          16, 0, 0);
#pragma unroll
    for (int i = 0; i < WT; ++i)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(wp[i] + k0),
          (__attribute__((address_space(3))) uint32_t*)(
              dst + BM * BK + (i * TH + tid) * 8),
          16, 0, 0);
  };
  floatx4 acc[NI][MI];
#pragma unroll
  for (int j = 0; j < NI; ++j)
#pragma unroll
    for (int i = 0; i < MI; ++i) acc[j][i] = floatx4{0, 0, 0, 0};

  constexpr int HALF = (BM + BN) * BK;
  load(0, lds);
  for (int k0 = 0, cur = 0; k0 < m.K; k0 += BK, cur ^= 1) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (k0 + BK < m.K) load(k0 + BK, lds + (cur ^ 1) * HALF);
    const uint16_t* al = lds + cur * HALF + (wr * MI * 16 + lo) * BK;
    const uint16_t* wl = lds + cur * HALF + (BM + wc * NI * 16 + lo) * BK;
#pragma unroll
    for (int kk = 0; kk < BK / 32; ++kk) {
      const int piece = ((kk * 4 + hi) ^ (lo & 7)) * 8;
      u16x8 af[MI], wf[NI];
#pragma unroll
      for (int i = 0; i < MI; ++i) af[i] = ld_u16x8(al + i * 16 * BK + piece);
#pragma unroll
      for (int j = 0; j < NI; ++j) wf[j] = ld_u16x8(wl + j * 16 * BK + piece);
#pragma unroll
      for (int j = 0; j < NI; ++j)
#pragma unroll
        for (int i = 0; i < MI; ++i)
          acc[j][i] = mfma16(wf[j], af[i], acc[j][i]);
    }
    if constexpr (MI * NI == 32) {
      // the second half's operands leave LDS between the first products
      __builtin_amdgcn_sched_group_barrier(DS_READ, MI + NI, 0);
#pragma unroll
      for (int i = 0; i < MI + NI; ++i) {
        __builtin_amdgcn_sched_group_barrier(MFMA, 2, 0);
        __builtin_amdgcn_sched_group_barrier(DS_READ, 1, 0);
      }
      __builtin_amdgcn_sched_group_barrier(MFMA, 64 - 2 * (MI + NI), 0);
    }
  }
  // lane: columns 4 hi + r of row lo
#pragma unroll
  for (int i = 0; i < MI; ++i) {
    const int r = (wr * MI + i) * 16 + lo;
    if (r >= tile.z) continue;
    uint16_t* o = out + (int64_t)(tile.y + r) * m.N;
#pragma unroll
    for (int j = 0; j < NI; ++j) {
      const int c = n0 + (wc * NI + j) * 16 + hi * 4;
      if (m.N % 4 == 0) {
        const float v[4] = {finish(m, acc[j][i][0]), finish(m, acc[j][i][1]),
                            finish(m, acc[j][i][2]), finish(m, acc[j][i][3])};
        if (c < m.N) st_bf16x4(o + c, v);
      } else {
#pragma unroll
        for (int q = 0; q < 4; ++q)
          if (c + q < m.N) o[c + q] = f32_to_bf16(finish(m, acc[j][i][q]));
      }
    }
  }
}

template <int BM, int BN, int WM, int WN>
void launch_tiles(torch::Tensor out, torch::Tensor a, torch::Tensor w,
                  Mix m) {
  static const hipError_t big = hipFuncSetAttribute(
      (const void*)expert_tiles_kernel<BM, BN, WM, WN>,
      hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  TORCH_CHECK(big == hipSuccess, "LDS size refused");
  m.n_tiles = cdiv(m.N, BN);
  hipLaunchKernelGGL((expert_tiles_kernel<BM, BN, WM, WN>),
                     dim3(m.n_tiles * m.m_tiles), dim3(WM * WN * WAVE),
                     2 * (BM + BN) * BK * 2,
                     at::hip::getCurrentHIPStream(),
                     (uint16_t*)out.data_ptr(),
                     (const uint16_t*)a.data_ptr(),
                     (const uint16_t*)w.data_ptr(), m);
}

// --- any size and type: 32 x 32, fp32 inside.
constexpr int PT = 32;

template <typename S>
__global__ __launch_bounds__(NT) void expert_plain_kernel(
    S* __restrict__ out, const S* __restrict__ a, const S* __restrict__ w,
    Mix m) {
  __shared__ float al[PT][PT + 1], wl[PT][PT + 1];
  const int n0 = blockIdx.x % m.n_tiles * PT;
  const int4 tile = m.tiles[blockIdx.x / m.n_tiles];
  if (tile.x < 0) return;
  const int tid = threadIdx.x, x = tid % PT, y = tid / PT;  // y: 8 rows
  const S* we = w + (int64_t)tile.x * m.N * m.K;
  int64_t rows[4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
    rows[i] = source_row(m, tile.y + min(y + i * 8, tile.z - 1));
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < m.K; k0 += PT) {
    const int k = k0 + x;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = y + i * 8, c = min(n0 + r, m.N - 1);
      al[r][x] = k < m.K ? ld1(a + rows[i] * m.a_stride + k) : 0.f;
      wl[r][x] = k < m.K ? ld1(we + (int64_t)c * m.K + k) : 0.f;
    }
    __syncthreads();
    for (int q = 0; q < PT; ++q) {
      const float v = wl[x][q];
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] += al[y + i * 8][q] * v;
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = y + i * 8;
    if (r < tile.z && n0 + x < m.N)
      st1(out + (int64_t)(tile.y + r) * m.N + n0 + x, finish(m, acc[i]));
  }
}

}  // namespace

// Shapes the bf16 kernels take (16-byte pieces of rows).
bool experts_fit(torch::Tensor a, torch::Tensor w) {
  return a.scalar_type() == torch::kBFloat16 && w.size(2) % 8 == 0 &&
         a.stride(0) % 8 == 0 && (uintptr_t)a.data_ptr() % 16 == 0;
}

// tiles [n, 4] of at most `height` rows. kind: "stream" (height 32 or 64),
// "tile" (32, 64, 128 or 256; w.size(2) % 64 == 0), "plain" (32).
void expert_product(torch::Tensor out, torch::Tensor a, torch::Tensor w,
                    torch::Tensor tiles, OptT order, int64_t choices,
                    int64_t height, const std::string& kind, bool relu2) {
  TORCH_CHECK(out.dim() == 2 && a.dim() == 2 && w.dim() == 3);
  Mix m{};
  m.N = w.size(1);
  m.K = w.size(2);
  const int64_t P = out.size(0);
  TORCH_CHECK(out.is_contiguous() && out.size(1) == m.N && w.is_contiguous());
  TORCH_CHECK(a.stride(1) == 1 && a.size(1) == m.K &&
              a.scalar_type() == w.scalar_type() &&
              a.scalar_type() == out.scalar_type());
  TORCH_CHECK(tiles.scalar_type() == torch::kInt32 && tiles.is_contiguous() &&
              tiles.dim() == 2 && tiles.size(1) == 4);
  TORCH_CHECK(choices >= 1);
  if (order.has_value()) {
    TORCH_CHECK(order->scalar_type() == torch::kInt32 &&
                order->is_contiguous() && order->numel() == P &&
                a.size(0) * choices == P);
    m.order = order->data_ptr<int>();
  } else {
    TORCH_CHECK(a.size(0) == P);
  }
  m.tiles = (const int4*)tiles.data_ptr<int>();
  m.a_stride = a.stride(0);
  m.choices = choices;
  m.relu2 = relu2;
  m.m_tiles = tiles.size(0);
  if (P == 0 || m.m_tiles == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
#define HELIX_MIX(KERNEL, S, COLS)                                           \
  do {                                                                       \
    m.n_tiles = cdiv(m.N, COLS);                                             \
    hipLaunchKernelGGL(KERNEL, dim3(m.n_tiles * m.m_tiles), dim3(NT), 0,     \
                       stream, (S*)out.data_ptr(), (const S*)a.data_ptr(),   \
                       (const S*)w.data_ptr(), m);                           \
  } while (0)
  if (kind == "plain") {
    TORCH_CHECK(height == PT);
    if (a.scalar_type() == torch::kBFloat16)
      HELIX_MIX((expert_plain_kernel<uint16_t>), uint16_t, PT);
    else if (a.scalar_type() == torch::kFloat32)
      HELIX_MIX((expert_plain_kernel<float>), float, PT);
    else
      TORCH_CHECK(false, "experts: bf16 or fp32");
    return;
  }
  TORCH_CHECK(experts_fit(a, w) && (uintptr_t)w.data_ptr() % 16 == 0 &&
              (uintptr_t)out.data_ptr() % 8 == 0);
  if (kind == "tile") {
    TORCH_CHECK(m.K % BK == 0, "inner size ", m.K);
    if (height == 256) launch_tiles<256, 256, 2, 4>(out, a, w, m);
    else if (height == 128) launch_tiles<128, 128, 2, 2>(out, a, w, m);
    else if (height == 64) launch_tiles<64, 128, 1, 4>(out, a, w, m);
    else if (height == 32) launch_tiles<32, 128, 1, 4>(out, a, w, m);
    else TORCH_CHECK(false, "tiles of ", height, " rows");
    return;
  }
  TORCH_CHECK(kind == "stream", kind);
  if (height == 64) {
    HELIX_MIX((expert_rows_kernel<4, 2, 2>), uint16_t, 32);
  } else {
    TORCH_CHECK(height == 32, "streams of ", height, " rows");
    HELIX_MIX((expert_rows_kernel<2, 2, 2>), uint16_t, 32);
  }
#undef HELIX_MIX
}
