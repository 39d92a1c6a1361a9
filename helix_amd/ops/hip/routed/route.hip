// Choice of experts, and the experts' token lists.
//
// route: softmax over all router outputs (fp32). Choice scores have a
// correction on top; only experts of the best groups can be chosen; the
// weights are the uncorrected scores of the chosen, normalised. A wave has a
// token at a time. Each workgroup also counts its tokens per expert and
// numbers them.
//
// place: a (token, choice) pair's row in the experts' common list, from the
// counts of all workgroups; no global atomics, nothing to clear. The list is
// cut into tiles of equal height, each of one expert.
#include "../hybrid/tile.h"
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

using namespace helix;

namespace {

constexpr int NT = 256, NW = NT / WAVE;
constexpr int MAX_OUTPUTS = 1024;             // router outputs
constexpr int PER = MAX_OUTPUTS / NT;
constexpr int MANY = 1024;                    // threads, many tokens

struct Route {
  int* ids;                    // [T, K]
  float* weights;              // [T, K]
  int* rank;                   // [T, K] within the workgroup and expert
  int* hist;                   // [workgroups, E]
  const float *z, *correction; // [T, n], [n]
  int64_t z_stride;
  int T, n, E, K, groups, size, keep, per;
};

// NJ: router outputs per lane
template <int NJ>
__global__ __launch_bounds__(MANY) void route_kernel(Route m) {
  extern __shared__ float sh[];
  const int wid = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int nw = blockDim.x / WAVE;
  float* choice = sh + wid * m.n;
  float* score = sh + (nw + wid) * m.n;
  float* best = sh + 2 * nw * m.n + wid * m.groups;
  int* count = (int*)(sh + 2 * nw * m.n + nw * m.groups);
  for (int e = threadIdx.x; e < m.E; e += blockDim.x) count[e] = 0;
  const int first = blockIdx.x * m.per;
  for (int i = 0; i < m.per; i += nw) {
    const int t = first + i + wid;
    const bool live = i + wid < m.per && t < m.T;
    const float* z = m.z + (int64_t)min(t, m.T - 1) * m.z_stride;
    float s[NJ], c[NJ], top = -INFINITY, sum = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int e = j * WAVE + lane;
      s[j] = e < m.n ? z[e] : -INFINITY;
      top = fmaxf(top, s[j]);
    }
    top = wave_reduce_max(top);
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      s[j] = expf(s[j] - top);
      sum += s[j];
    }
    sum = wave_reduce_sum(sum);
    __syncthreads();                          // the last token is done
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int e = j * WAVE + lane;
      s[j] /= sum;
      c[j] = e < m.n ? s[j] + m.correction[e] : -INFINITY;
      if (e < m.n) {
        choice[e] = c[j];
        score[e] = s[j];
      }
    }
    __syncthreads();
    if (m.keep < m.groups) {
      for (int g = lane; g < m.groups; g += WAVE) {
        float b = -INFINITY;
        for (int k = 0; k < m.size; ++k) b = fmaxf(b, choice[g * m.size + k]);
        best[g] = b;
      }
      __syncthreads();
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const int e = j * WAVE + lane;
        if (e >= m.n) continue;
        const int g = e / m.size;
        const float own = best[g];
        int ahead = 0;
        for (int k = 0; k < m.groups; ++k)
          ahead += best[k] > own || (best[k] == own && k < g);
        if (ahead >= m.keep) c[j] = -INFINITY;
      }
    }
    int mine = 0;
    float weight = 0.f, total = 0.f;
    for (int k = 0; k < m.K; ++k) {
      float v = c[0];
#pragma unroll
      for (int j = 1; j < NJ; ++j) v = fmaxf(v, c[j]);
      v = wave_reduce_max(v);
      int at = m.n - 1;                       // whatever the scores are
#pragma unroll
      for (int j = NJ - 1; j >= 0; --j) {     // the lowest index that has it
        const unsigned long long who = __ballot(c[j] == v);
        if (who != 0) at = min(j * WAVE + __builtin_ctzll(who), m.n - 1);
      }
#pragma unroll
      for (int j = 0; j < NJ; ++j)
        if (j * WAVE + lane == at) c[j] = -INFINITY;
      const float w = score[at];
      total += w;
      if (lane == k) {
        mine = at;
        weight = w;
      }
    }
    if (live && lane < m.K) {
      const int64_t p = (int64_t)t * m.K + lane;
      m.ids[p] = mine;
      m.weights[p] = weight / (total + 1e-20f);
      m.rank[p] = mine < m.E ? atomicAdd(count + mine, 1) : 0;
    }
  }
  __syncthreads();
  for (int e = threadIdx.x; e < m.E; e += blockDim.x)
    m.hist[(int64_t)blockIdx.x * m.E + e] = count[e];
}

struct Place {
  int* order;                  // [P] pair of a row of the list
  int* slot;                   // [P] row of a pair, -1: identity expert
  int4* tiles;                 // expert (-1: none), first row, rows
  const int *ids, *rank, *hist;
  int T, E, K, per, blocks, height, max_tiles;
};

__global__ __launch_bounds__(NT) void place_kernel(Place m) {
  __shared__ int at[MAX_OUTPUTS];             // this workgroup's first rows
  __shared__ int rows_of[MAX_OUTPUTS];
  __shared__ int sums[2][NW];
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  for (int e = tid; e < MAX_OUTPUTS; e += NT) at[e] = rows_of[e] = 0;
  __syncthreads();
  const int mine = blockIdx.x * m.E;
#pragma unroll 8
  for (int i = tid; i < m.blocks * m.E; i += NT) {
    const int c = m.hist[i], e = i % m.E;
    if (c != 0) {
      atomicAdd(rows_of + e, c);
      if (i < mine) atomicAdd(at + e, c);
    }
  }
  __syncthreads();
  // thread t has experts t PER ..
  int total[PER], rows = 0, tiles = 0;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    total[i] = rows_of[tid * PER + i];
    rows += total[i];
    tiles += (total[i] + m.height - 1) / m.height;
  }
  int r = rows, q = tiles;                    // running sums over threads
#pragma unroll
  for (int off = 1; off < WAVE; off <<= 1) {
    const int a = __shfl_up(r, off, WAVE), b = __shfl_up(q, off, WAVE);
    if (lane >= off) {
      r += a;
      q += b;
    }
  }
  if (lane == WAVE - 1) {
    sums[0][wid] = r;
    sums[1][wid] = q;
  }
  __syncthreads();
  r -= rows;
  q -= tiles;
  int all_tiles = 0;
#pragma unroll
  for (int w = 0; w < NW; ++w) {
    r += w < wid ? sums[0][w] : 0;
    q += w < wid ? sums[1][w] : 0;
    all_tiles += sums[1][w];
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int e = tid * PER + i;
    if (blockIdx.x == 0)
      for (int k = 0; k < total[i]; k += m.height, ++q)
        if (q < m.max_tiles)
          m.tiles[q] = make_int4(e, r + k, min(m.height, total[i] - k), 0);
    at[e] += r;
    r += total[i];
  }
  if (blockIdx.x == 0)
    for (int k = all_tiles + tid; k < m.max_tiles; k += NT)
      m.tiles[k] = make_int4(-1, 0, 0, 0);
  __syncthreads();
  const int p0 = blockIdx.x * m.per * m.K;
  const int p1 = min(m.T, (int)(blockIdx.x + 1) * m.per) * m.K;
  for (int p = p0 + tid; p < p1; p += NT) {
    const int e = m.ids[p];
    if (e < m.E) {
      const int s = at[e] + m.rank[p];
      m.order[s] = p;
      m.slot[p] = s;
    } else {
      m.slot[p] = -1;
    }
  }
}

void check(const torch::Tensor& t, torch::ScalarType type, int64_t n,
           const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == type && t.is_contiguous() &&
                  t.numel() == n,
              what);
}

}  // namespace

int64_t route_max_outputs() { return MAX_OUTPUTS; }

// per: tokens of a workgroup (the same for both launches).
void route(torch::Tensor ids, torch::Tensor weights, torch::Tensor rank,
           torch::Tensor hist, torch::Tensor z, torch::Tensor correction,
           int64_t experts, int64_t groups, int64_t keep, int64_t per) {
  TORCH_CHECK(ids.dim() == 2 && z.dim() == 2 && z.stride(1) == 1 &&
              z.scalar_type() == torch::kFloat32);
  Route m{};
  m.T = ids.size(0);
  m.K = ids.size(1);
  m.n = z.size(1);
  m.E = experts;
  m.groups = groups;
  m.keep = keep;
  m.per = per;
  TORCH_CHECK(z.size(0) == m.T && m.n >= 1 && m.n <= MAX_OUTPUTS &&
              m.E >= 0 && m.E <= m.n && groups >= 1 && m.n % groups == 0 &&
              keep >= 1 && keep <= groups && per >= 1);
  m.size = m.n / groups;
  TORCH_CHECK(m.K >= 1 && m.K <= WAVE && m.K <= keep * m.size,
              "top ", m.K, " of ", keep * m.size, " experts");
  const int64_t P = (int64_t)m.T * m.K, blocks = (m.T + per - 1) / per;
  check(ids, torch::kInt32, P, "ids");
  check(weights, torch::kFloat32, P, "weights");
  check(rank, torch::kInt32, P, "rank");
  check(hist, torch::kInt32, blocks * m.E, "hist");
  check(correction, torch::kFloat32, m.n, "correction");
  m.ids = ids.data_ptr<int>();
  m.weights = weights.data_ptr<float>();
  m.rank = rank.data_ptr<int>();
  m.hist = hist.data_ptr<int>();
  m.z = z.data_ptr<float>();
  m.z_stride = z.stride(0);
  m.correction = correction.data_ptr<float>();
  if (m.T == 0) return;
  const int threads = per >= 16 && m.n <= 256 ? MANY : NT;
  const int nw = threads / WAVE;
  const int lds = (2 * nw * m.n + nw * m.groups + m.E) * 4;
  const int nj = cdiv(m.n, WAVE);
#define HELIX_ROUTE(NJ)                                                      \
  hipLaunchKernelGGL(route_kernel<NJ>, dim3(blocks), dim3(threads), lds,     \
                     at::hip::getCurrentHIPStream(), m)
  if (nj <= 1) HELIX_ROUTE(1);
  else if (nj <= 2) HELIX_ROUTE(2);
  else if (nj <= 4) HELIX_ROUTE(4);
  else if (nj <= 8) HELIX_ROUTE(8);
  else HELIX_ROUTE(16);
#undef HELIX_ROUTE
}

void place(torch::Tensor order, torch::Tensor slot, torch::Tensor tiles,
           torch::Tensor ids, torch::Tensor rank, torch::Tensor hist,
           int64_t per, int64_t height) {
  TORCH_CHECK(ids.dim() == 2 && hist.dim() == 2 && tiles.dim() == 2 &&
              tiles.size(1) == 4 && per >= 1 && height >= 1);
  Place m{};
  m.T = ids.size(0);
  m.K = ids.size(1);
  m.blocks = hist.size(0);
  m.E = hist.size(1);
  m.per = per;
  m.height = height;
  m.max_tiles = tiles.size(0);
  const int64_t P = (int64_t)m.T * m.K;
  TORCH_CHECK(m.E <= MAX_OUTPUTS && m.blocks == (m.T + per - 1) / per &&
              P < (1 << 30));
  // every expert with rows has at most one tile that is not full
  TORCH_CHECK(m.max_tiles >= std::min<int64_t>(P, P / height + m.E));
  check(order, torch::kInt32, P, "order");
  check(slot, torch::kInt32, P, "slot");
  check(ids, torch::kInt32, P, "ids");
  check(rank, torch::kInt32, P, "rank");
  check(hist, torch::kInt32, (int64_t)m.blocks * m.E, "hist");
  check(tiles, torch::kInt32, (int64_t)m.max_tiles * 4, "tiles");
  m.order = order.data_ptr<int>();
  m.slot = slot.data_ptr<int>();
  m.tiles = (int4*)tiles.data_ptr<int>();
  m.ids = ids.data_ptr<int>();
  m.rank = rank.data_ptr<int>();
  m.hist = hist.data_ptr<int>();
  if (P == 0) return;
  hipLaunchKernelGGL(place_kernel, dim3(m.blocks), dim3(NT), 0,
                     at::hip::getCurrentHIPStream(), m);
}
