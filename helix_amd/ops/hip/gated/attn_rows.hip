// Paged attention of single query rows.
//
// bf16: a wave works alone on tiles of 32 keys. A lane loads key rows and
// value columns straight from the pages as MFMA operands: keys are permuted
// (paired_row) so that a lane ends up with the weights of 8 neighbouring
// keys of one query head, which are the other operand of the value product
// as they lie. Nothing passes through LDS until the four waves of a
// workgroup put their results together. The query heads of a key/value head
// share a tile. Loads of the next tile are under way while one is worked on.
//
// Long rows are cut into partitions, merged by a launch of their own. fp32
// and oversized heads run the plain kernel.
#include "attn.h"

using namespace helix;

namespace {

constexpr int NT = 256, NW = NT / WAVE;
constexpr int KT = 32;                        // keys of a tile

struct Rows {
  Attn a;
  const int* row_seq;          // null: row r is sequence r
  const int* row_len;
  float* part;                 // [R, parts, H, E] or null
  float2* ml;                  // [R, parts, H]
  int per, parts;              // query heads per key/value head
};

// Both values of a pair of head h, gated.
template <typename S>
__device__ __forceinline__ void store_pair(const Attn& A, S* out, int64_t row,
                                           int h, int pair, int half, float a,
                                           float b) {
  const int at = h * A.E + pair;
  S* o = out + row * A.out_stride + at;
  st1(o, a * gate_of<S>(A, row, at));
  if (half + pair < A.E) st1(o + half, b * gate_of<S>(A, row, at + half));
}

template <int NK, int NV, bool SIG>
__global__ __launch_bounds__(NT, NV > 8 ? 1 : 2) void attn_rows_kernel(
    uint16_t* __restrict__ out, const uint16_t* __restrict__ q,
    const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc,
    Rows m) {
  constexpr int PITCH = NV * 16 + 4;
  extern __shared__ __attribute__((aligned(16))) float sh[];
  const Attn& A = m.a;
  const int row = blockIdx.x, part = blockIdx.z;
  const int groups = cdiv(m.per, 16);
  const int g = blockIdx.y / groups, h0 = g * m.per + blockIdx.y % groups * 16;
  const int nh = min(16, (g + 1) * m.per - h0);
  const int seq = m.row_seq != nullptr ? m.row_seq[row] : row;
  const int len = m.row_len[row];
  const int tid = threadIdx.x, wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int lo = lane & 15, hi = lane >> 4;
  const int* bt = A.bt + (int64_t)seq * A.max_blocks;

  // this partition's tiles
  const int tiles = cdiv(len, KT), tp = cdiv(tiles, m.parts);
  const int t0 = part * tp, t1 = min(tiles, t0 + tp);

  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  u16x8 qf[NK];
  const uint16_t* qr = q + row * A.q_stride + (h0 + min(lo, nh - 1)) * A.Dp;
#pragma unroll
  for (int c = 0; c < NK; ++c) {
    const int d = c * 32 + hi * 8;
    qf[c] = lo < nh && d < A.Dp ? ld_u16x8(qr + d) : zero;
  }
  const float mul = head_mul(A, h0 + min(lo, nh - 1)) * row_mul(A, row);
  const float add = head_add(A, h0 + min(lo, nh - 1));

  // A lane's keys are in the group of 8 numbered lo / 4 (keys as operand)
  // and hi (values). Groups past the end read the last page; what they bring
  // is masked.
  const int half = (A.E + 1) / 2, last_page = (len - 1) / A.bs;
  int kp = 0, vp = 0;
  auto pages = [&](int t) {
    kp = bt[min((t * KT + (lo >> 2) * 8) / A.bs, last_page)];
    vp = bt[min((t * KT + hi * 8) / A.bs, last_page)];
  };
  u16x8 kr[2][NK], vr[NV];
  auto load = [&](int t) {
    const int ks = (t * KT + (lo >> 2) * 8) % A.bs + (lo & 3);
    const uint16_t* kb =
        kc + (((int64_t)kp * A.G + g) * A.bs + ks) * A.Dp;
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int c = 0; c < NK; ++c)
        kr[s][c] = ld_u16x8(kb + s * 4 * A.Dp +
                            min(c * 32 + hi * 8, A.Dp - 8));
    const uint16_t* vb = vc + ((int64_t)vp * A.G + g) * A.E * A.bs +
                         (t * KT + hi * 8) % A.bs;
#pragma unroll
    for (int d = 0; d < NV; ++d) {
      const int e = min((d & 1) * half + (d >> 1) * 16 + lo, A.E - 1);
      vr[d] = ld_u16x8(vb + (int64_t)e * A.bs);
    }
  };

  floatx4 acc[NV];
#pragma unroll
  for (int d = 0; d < NV; ++d) acc[d] = floatx4{0, 0, 0, 0};
  float m_run = NEG, l = 0.f;
  int t = t0 + wid;
  if (t < t1) {
    pages(t);
    load(t);
    pages(min(t + NW, t1 - 1));
  }
  for (; t < t1; t += NW) {
    u16x8 k[2][NK], v[NV];
#pragma unroll
    for (int c = 0; c < NK; ++c) {
      k[0][c] = kr[0][c];
      k[1][c] = kr[1][c];
    }
#pragma unroll
    for (int d = 0; d < NV; ++d) v[d] = vr[d];
    if (t + NW < t1) {
      load(t + NW);
      pages(min(t + 2 * NW, t1 - 1));
    }
    float p[8], mx = m_run;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      floatx4 d = floatx4{0, 0, 0, 0};
#pragma unroll
      for (int c = 0; c < NK; ++c) d = mfma16(k[s][c], qf[c], d);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = t * KT + hi * 8 + s * 4 + r;
        const float x = d[r] * mul + add;
        p[s * 4 + r] = key < len ? x : NEG;
        mx = fmaxf(mx, p[s * 4 + r]);
      }
    }
    if constexpr (SIG) {
#pragma unroll
      for (int i = 0; i < 8; ++i) p[i] = sigmoid2(p[i]);
    } else {
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      if (!__all(mx == m_run)) {
        const float corr = __builtin_amdgcn_exp2f(m_run - mx);
        l *= corr;
        m_run = mx;
#pragma unroll
        for (int d = 0; d < NV; ++d)
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[d][r] *= corr;
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        p[i] = __builtin_amdgcn_exp2f(p[i] - mx);
        l += p[i];
      }
    }
    const u16x8 pf = pack8(p);
#pragma unroll
    for (int d = 0; d < NV; ++d) acc[d] = mfma16(v[d], pf, acc[d]);
  }

  // the four waves together
  float* st = sh + NW * nh * PITCH;           // [NW][16] m, then l
  if constexpr (!SIG) {
    l += __shfl_xor(l, 16, WAVE);
    l += __shfl_xor(l, 32, WAVE);
    if (hi == 0) {
      st[wid * 16 + lo] = m_run;
      st[(NW + wid) * 16 + lo] = l;
    }
  }
  if (lo < nh)
#pragma unroll
    for (int d = 0; d < NV; ++d)
      *reinterpret_cast<floatx4*>(sh + (wid * nh + lo) * PITCH + d * 16 +
                                  hi * 4) = acc[d];
  __syncthreads();
  for (int i = tid; i < nh * half; i += NT) {
    const int n = i / half, pair = i % half;
    float f[NW], mm = 0.f, ll = 1.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) f[w] = 1.f;
    if constexpr (!SIG) {
      mm = NEG;
      ll = 0.f;
#pragma unroll
      for (int w = 0; w < NW; ++w) mm = fmaxf(mm, st[w * 16 + n]);
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        f[w] = __builtin_amdgcn_exp2f(st[w * 16 + n] - mm);
        ll += f[w] * st[(NW + w) * 16 + n];
      }
    }
    const int at = (pair >> 4) * 32 + (pair & 15);
    float a = 0.f, b = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      a += f[w] * sh[(w * nh + n) * PITCH + at];
      b += f[w] * sh[(w * nh + n) * PITCH + at + 16];
    }
    const int h = h0 + n;
    if (m.part != nullptr) {
      const int64_t r = ((int64_t)row * m.parts + part) * A.H + h;
      m.part[r * A.E + pair] = a;
      if (half + pair < A.E) m.part[r * A.E + half + pair] = b;
      if (pair == 0) m.ml[r] = make_float2(mm, ll);
      continue;
    }
    const float inv = A.out_scale / ll;
    turn_back(A, row, pair, a, b);
    store_pair(A, out, row, h, pair, half, a * inv, b * inv);
  }
}

// Partitions of a row into one: a thread per (row, head, pair).
__global__ __launch_bounds__(NT) void attn_merge_kernel(
    uint16_t* __restrict__ out, Rows m, bool sig, int64_t total) {
  const Attn& A = m.a;
  const int half = (A.E + 1) / 2;
  const int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x;
  if (i >= total) return;
  const int pair = (int)(i % half);
  const int h = (int)(i / half % A.H);
  const int64_t row = i / half / A.H;
  float mm = NEG, ll = 0.f, a = 0.f, b = 0.f;
  const bool two = half + pair < A.E;
  for (int p = 0; p < m.parts; ++p) {
    const int64_t r = (row * m.parts + p) * A.H + h;
    const float x = m.part[r * A.E + pair];
    const float y = two ? m.part[r * A.E + half + pair] : 0.f;
    if (sig) {
      a += x;
      b += y;
    } else {
      const float2 v = m.ml[r];
      const float top = fmaxf(mm, v.x);
      const float c = __builtin_amdgcn_exp2f(mm - top);
      const float f = __builtin_amdgcn_exp2f(v.x - top);
      ll = ll * c + v.y * f;
      a = a * c + x * f;
      b = b * c + y * f;
      mm = top;
    }
  }
  const float inv = A.out_scale / (sig ? 1.f : ll);
  turn_back(A, row, pair, a, b);
  store_pair(A, out, row, h, pair, half, a * inv, b * inv);
}

// Any size and type: a workgroup per (row, head), a thread per key, then a
// wave per group of value dimensions.
template <typename S, bool SIG>
__global__ __launch_bounds__(NT) void attn_plain_kernel(
    S* __restrict__ out, const S* __restrict__ q, const S* __restrict__ kc,
    const S* __restrict__ vc, Rows m) {
  extern __shared__ float sh[];               // q [Dp], weights [NT], o [E]
  __shared__ float red[16];
  const Attn& A = m.a;
  float *qs = sh, *ws = sh + A.Dp, *os = ws + NT;
  const int row = blockIdx.x, h = blockIdx.y, g = h / m.per;
  const int seq = m.row_seq != nullptr ? m.row_seq[row] : row;
  const int len = m.row_len[row], tid = threadIdx.x;
  const int wid = tid / WAVE, lane = tid & (WAVE - 1);
  const int* bt = A.bt + (int64_t)seq * A.max_blocks;
  for (int d = tid; d < A.Dp; d += NT)
    qs[d] = ld1(q + row * A.q_stride + h * A.Dp + d);
  for (int e = tid; e < A.E; e += NT) os[e] = 0.f;
  const float mul =
      A.scale * (A.temp != nullptr ? A.temp[h] : 1.f) * row_mul(A, row);
  const float add = A.bias != nullptr ? A.bias[h] : 0.f;
  float mm = NEG, ll = 0.f;
  for (int t = 0; t < len; t += NT) {
    __syncthreads();
    const int key = t + tid, n = min(NT, len - t);
    float x = NEG;
    if (key < len) {
      const S* k = kc + (((int64_t)bt[key / A.bs] * A.G + g) * A.bs +
                         key % A.bs) * A.Dp;
      float s = 0.f;
      for (int d = 0; d < A.Dp; d += 8) {
        float v[8];
        ldv<8>(k + d, v);
#pragma unroll
        for (int i = 0; i < 8; ++i) s += v[i] * qs[d + i];
      }
      x = s * mul + add;
    }
    float corr = 1.f;
    if constexpr (SIG) {
      ws[tid] = key < len ? sigmoid_s<S>(x) : 0.f;
      __syncthreads();
    } else {
      float top = wave_reduce_max(x);
      if (lane == 0) red[wid] = top;
      __syncthreads();
      for (int i = 0; i < NW; ++i) top = fmaxf(top, red[i]);
      top = fmaxf(top, mm);
      corr = exp_s<S>(mm - top);
      mm = top;
      const float w = exp_s<S>(x - top);
      ws[tid] = w;
      __syncthreads();
      ll = ll * corr + group_sum(w, red + 8);
    }
    for (int e = wid; e < A.E; e += NW) {
      float s = 0.f;
      for (int j = lane; j < n; j += WAVE) {
        const int k = t + j;
        s += ws[j] * ld1(vc + (((int64_t)bt[k / A.bs] * A.G + g) * A.E + e) *
                                  A.bs + k % A.bs);
      }
      s = wave_reduce_sum(s);
      if (lane == 0) os[e] = os[e] * corr + s;
    }
  }
  __syncthreads();
  const float inv = A.out_scale / (SIG ? 1.f : ll);
  const int half = (A.E + 1) / 2;
  for (int pair = tid; pair < half; pair += NT) {
    float a = os[pair], b = half + pair < A.E ? os[half + pair] : 0.f;
    turn_back(A, row, pair, a, b);
    store_pair(A, out, row, h, pair, half, a * inv, b * inv);
  }
}

Rows row_args(const torch::Tensor& q, const torch::Tensor& kc,
              const torch::Tensor& vc, const torch::Tensor& bt, OptT row_seq,
              const torch::Tensor& row_len, double scale, double out_scale,
              OptT temp, OptT bias, OptT vcs, OptT row_scale, OptT gate) {
  TORCH_CHECK(q.dim() == 3 && q.scalar_type() == kc.scalar_type());
  const int64_t R = q.size(0);
  Rows m{};
  m.a = attn_args(kc, vc, bt, R, q.size(1), scale, out_scale, temp, bias,
                  vcs, row_scale, gate);
  query_rows(m.a, q);
  TORCH_CHECK(row_len.scalar_type() == torch::kInt32 &&
              row_len.is_contiguous() && row_len.numel() == R);
  m.row_len = row_len.data_ptr<int>();
  if (row_seq.has_value()) {
    TORCH_CHECK(row_seq->scalar_type() == torch::kInt32 &&
                row_seq->is_contiguous() && row_seq->numel() == R);
    m.row_seq = row_seq->data_ptr<int>();
  } else {
    TORCH_CHECK(bt.size(0) >= R);
  }
  m.per = m.a.H / m.a.G;
  m.parts = 1;
  return m;
}

void set_out(Rows& m, const torch::Tensor& out, const torch::Tensor& q) {
  TORCH_CHECK(out.dim() == 2 && out.size(0) == q.size(0) &&
              out.size(1) == m.a.H * m.a.E && out.stride(1) == 1 &&
              out.scalar_type() == q.scalar_type());
  m.a.out_stride = out.stride(0);
}

template <bool SIG>
void launch_rows(uint16_t* out, torch::Tensor q, torch::Tensor kc,
                 torch::Tensor vc, Rows m) {
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(q.size(0), m.a.G * cdiv(m.per, 16), m.parts);
  const int nh = std::min(m.per, 16);
#define HELIX_ROWS(NK, NV)                                                   \
  do {                                                                       \
    static const hipError_t big = hipFuncSetAttribute(                       \
        (const void*)attn_rows_kernel<NK, NV, SIG>,                          \
        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);             \
    TORCH_CHECK(big == hipSuccess, "LDS size refused");                      \
    hipLaunchKernelGGL((attn_rows_kernel<NK, NV, SIG>), grid, dim3(NT),      \
                       (NW * nh * (NV * 16 + 4) + NW * 32) * 4, stream, out, \
                       (const uint16_t*)q.data_ptr(),                        \
                       (const uint16_t*)kc.data_ptr(),                       \
                       (const uint16_t*)vc.data_ptr(), m);                   \
  } while (0)
  const int half = (m.a.E + 1) / 2, D = m.a.Dp;
  if (D <= 32 && half <= 16) HELIX_ROWS(1, 2);
  else if (D <= 64 && half <= 32) HELIX_ROWS(2, 4);
  else if (D <= 128 && half <= 64) HELIX_ROWS(4, 8);
  else HELIX_ROWS(8, 16);
#undef HELIX_ROWS
}

}  // namespace

// bf16 heads of up to 256 dimensions.
bool attn_fits(torch::Tensor q, int64_t vdim) {
  return q.scalar_type() == torch::kBFloat16 && q.size(2) <= 256 &&
         vdim <= 256;
}

void attn_rows(OptT out, OptT part, OptT ml, torch::Tensor q,
               torch::Tensor kc, torch::Tensor vc, torch::Tensor bt,
               OptT row_seq, torch::Tensor row_len, double scale,
               double out_scale, bool sigmoid, OptT temp, OptT bias,
               OptT vcs, OptT row_scale, OptT gate) {
  Rows m = row_args(q, kc, vc, bt, row_seq, row_len, scale, out_scale, temp,
                    bias, vcs, row_scale, gate);
  TORCH_CHECK(attn_fits(q, m.a.E));
  TORCH_CHECK(out.has_value() != part.has_value());
  uint16_t* o = nullptr;
  if (out.has_value()) {
    set_out(m, *out, q);
    o = (uint16_t*)out->data_ptr();
  } else {
    TORCH_CHECK(part->dim() == 4 && part->is_contiguous() &&
                part->scalar_type() == torch::kFloat32 &&
                part->size(0) == q.size(0) && part->size(2) == m.a.H &&
                part->size(3) == m.a.E);
    m.parts = part->size(1);
    TORCH_CHECK(ml.has_value() && ml->is_contiguous() &&
                ml->scalar_type() == torch::kFloat32 &&
                ml->numel() == q.size(0) * m.parts * m.a.H * 2);
    m.part = part->data_ptr<float>();
    m.ml = (float2*)ml->data_ptr<float>();
  }
  if (q.size(0) == 0) return;
  if (sigmoid) launch_rows<true>(o, q, kc, vc, m);
  else launch_rows<false>(o, q, kc, vc, m);
}

void attn_merge(torch::Tensor out, torch::Tensor part, torch::Tensor ml,
                double out_scale, bool sigmoid, OptT vcs, OptT gate) {
  Rows m{};
  TORCH_CHECK(part.dim() == 4 && part.is_contiguous() && ml.is_contiguous() &&
              part.scalar_type() == torch::kFloat32 &&
              ml.scalar_type() == torch::kFloat32);
  const int64_t R = part.size(0);
  m.parts = part.size(1);
  m.a.H = part.size(2);
  m.a.E = part.size(3);
  TORCH_CHECK(ml.numel() == R * m.parts * m.a.H * 2);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == R &&
              out.size(1) == m.a.H * m.a.E && out.stride(1) == 1 &&
              out.scalar_type() == torch::kBFloat16);
  row_operands(m.a, R, torch::kBFloat16, vcs, gate);
  m.a.out_stride = out.stride(0);
  m.a.out_scale = (float)out_scale;
  m.part = part.data_ptr<float>();
  m.ml = (float2*)ml.data_ptr<float>();
  const int64_t total = R * m.a.H * ((m.a.E + 1) / 2);
  if (total == 0) return;
  hipLaunchKernelGGL(attn_merge_kernel, dim3((total + NT - 1) / NT),
                     dim3(NT), 0, at::hip::getCurrentHIPStream(),
                     (uint16_t*)out.data_ptr(), m, sigmoid, total);
}

void attn_plain(torch::Tensor out, torch::Tensor q, torch::Tensor kc,
                torch::Tensor vc, torch::Tensor bt, OptT row_seq,
                torch::Tensor row_len, double scale, double out_scale,
                bool sigmoid, OptT temp, OptT bias, OptT vcs,
                OptT row_scale, OptT gate) {
  Rows m = row_args(q, kc, vc, bt, row_seq, row_len, scale, out_scale, temp,
                    bias, vcs, row_scale, gate);
  set_out(m, out, q);
  if (q.size(0) == 0) return;
  const int lds = (m.a.Dp + NT + m.a.E) * sizeof(float);
  TORCH_CHECK(lds <= 60 * 1024, "heads of ", m.a.Dp, " + ", m.a.E);
  const dim3 grid(q.size(0), m.a.H);
#define HELIX_PLAIN(S, SIG)                                                  \
  hipLaunchKernelGGL((attn_plain_kernel<S, SIG>), grid, dim3(NT), lds,       \
                     at::hip::getCurrentHIPStream(), (S*)out.data_ptr(),     \
                     (const S*)q.data_ptr(), (const S*)kc.data_ptr(),        \
                     (const S*)vc.data_ptr(), m)
  if (q.scalar_type() == torch::kBFloat16) {
    if (sigmoid) HELIX_PLAIN(uint16_t, true);
    else HELIX_PLAIN(uint16_t, false);
  } else {
    TORCH_CHECK(q.scalar_type() == torch::kFloat32, "bf16 or fp32");
    if (sigmoid) HELIX_PLAIN(float, true);
    else HELIX_PLAIN(float, false);
  }
#undef HELIX_PLAIN
}
