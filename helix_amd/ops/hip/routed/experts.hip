// Matrix products of a mixture's experts, all of them in one launch:
//
//   out[r] = act(w[e] a[row(r)])   for the rows r of every expert e
//
// over the tiles that place() made of the experts' common list. a's row is
// that of the list itself, or (gather) of the token a list entry belongs to.
// act: none, or the square of relu.
//
// bf16 comes in two shapes. Few rows per expert (decoding): the weights are
// the traffic, so a wave streams them straight into MFMA operands, the waves
// of a workgroup share the inner dimension and meet in LDS at the end. Many
// rows: tiles of 128 x 128 through LDS, filled by direct loads; 16-byte
// pieces of a row are stored crosswise (piece ^ row % 8), so that operands
// leave LDS without bank conflicts. fp32 and odd sizes run a plain kernel.
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

// --- few rows: 16 MI rows x 16 NI columns of a workgroup; a wave has every
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

// --- many rows: 128 x 128, inner dimension in steps of 64 (K % 64 == 0).
constexpr int BT = 128, BK = 64;

__global__ __launch_bounds__(NT) void expert_tiles_kernel(
    uint16_t* __restrict__ out, const uint16_t* __restrict__ a,
    const uint16_t* __restrict__ w, Mix m) {
  __shared__ __attribute__((aligned(16))) uint16_t al[BT * BK];
  __shared__ __attribute__((aligned(16))) uint16_t wl[BT * BK];
  const int lin = xcd_chunk(blockIdx.x, gridDim.x);
  const int4 tile = m.tiles[lin / m.n_tiles];
  if (tile.x < 0) return;
  const int n0 = lin % m.n_tiles * BT;
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int wr = wid >> 1, wc = wid & 1;      // 64 rows x 64 columns each

  // this thread's four 16-byte pieces of either tile
  constexpr int ITS = BT * BK / (NT * 8);
  const uint16_t *ap[ITS], *wp[ITS];
#pragma unroll
  for (int it = 0; it < ITS; ++it) {
    const int row = it * (NT / 8) + tid / 8;
    const int col = ((tid & 7) ^ (row & 7)) * 8;
    ap[it] = a + source_row(m, tile.y + min(row, tile.z - 1)) * m.a_stride +
             col;
    wp[it] = w + ((int64_t)tile.x * m.N + min(n0 + row, m.N - 1)) * m.K + col;
  }
  floatx4 acc[4][4];
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[j][i] = floatx4{0, 0, 0, 0};

  for (int k0 = 0; k0 < m.K; k0 += BK) {
    __syncthreads();
#pragma unroll
    for (int it = 0; it < ITS; ++it) {
      const int e = (it * NT + tid) * 8;
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(ap[it] + k0),
          (__attribute__((address_space(3))) uint32_t*)(al + e), 16, 0, 0);
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(wp[it] + k0),
          (__attribute__((address_space(3))) uint32_t*)(wl + e), 16, 0, 0);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < BK / 32; ++kk) {
      const int piece = ((kk * 4 + hi) ^ (lo & 7)) * 8;
      u16x8 af[4], wf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        af[i] = ld_u16x8(al + (wr * 64 + i * 16 + lo) * BK + piece);
        wf[i] = ld_u16x8(wl + (wc * 64 + i * 16 + lo) * BK + piece);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[j][i] = mfma16(wf[j], af[i], acc[j][i]);
    }
  }
  // lane: columns 4 hi + r of row lo
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = wr * 64 + i * 16 + lo;
    if (r >= tile.z) continue;
    uint16_t* o = out + (int64_t)(tile.y + r) * m.N;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = n0 + wc * 64 + j * 16 + hi * 4;
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

int64_t expert_tile_rows() { return BT; }

// tiles [n, 4] of at most `height` rows: 16, 32 or 64 (few rows), 128 (many
// rows; w.size(2) % 64 == 0), or 32 with plain.
void expert_product(torch::Tensor out, torch::Tensor a, torch::Tensor w,
                    torch::Tensor tiles, OptT order, int64_t choices,
                    int64_t height, bool relu2, bool plain) {
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
  if (plain) {
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
  if (height == BT) {
    TORCH_CHECK(m.K % BK == 0);
    HELIX_MIX(expert_tiles_kernel, uint16_t, BT);
  } else if (height == 64) {
    HELIX_MIX((expert_rows_kernel<4, 2, 2>), uint16_t, 32);
  } else if (height == 32) {
    HELIX_MIX((expert_rows_kernel<2, 2, 2>), uint16_t, 32);
  } else {
    TORCH_CHECK(height == 16, "tiles of ", height, " rows");
    HELIX_MIX((expert_rows_kernel<1, 2, 4>), uint16_t, 32);
  }
#undef HELIX_MIX
}
