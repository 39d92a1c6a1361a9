// Python bindings for helix_amd._C_hybrid: latent attention, Mamba-2 mixers
// and the fp32 residual stream of looped layers.
#include <torch/extension.h>

using OptT = c10::optional<torch::Tensor>;
using T = torch::Tensor;

void residual_norm(T h, OptT x, OptT y, OptT ls, double mult, OptT ids,
                   OptT embed, OptT step, T w, double eps, OptT x_out,
                   OptT tap);
void silu_mul(T out, T z, int64_t up_at);
void group_rms_norm(T out, T y, int64_t groups, T w, double eps);
void latent_epilogue(T z, int64_t q_at, int64_t heads, int64_t dim_pad,
                     int64_t head_cols, int64_t kv_at, int64_t rank,
                     int64_t rank_pad, int64_t rot_dim, OptT freqs,
                     double amp, T pos, T norm_w, double eps, T cache,
                     T slots);
void latent_absorb(T q, T z, int64_t q_at, int64_t head_cols,
                   int64_t dim_pad, T uk, T ukt, int64_t rank_pad);
bool latent_rows_fits(T q, int64_t rank_pad);
void latent_rows(OptT o, OptT part, OptT ml, T q, T cache, T block_tables,
                 OptT row_seq, T row_len, int64_t rank_pad, double scale,
                 int64_t window);
void latent_rows_plain(T o, T q, T cache, T block_tables, OptT row_seq,
                       T row_len, double scale, int64_t window);
void latent_merge(T o, T part, T ml);
void latent_out(T out, T o, T uv, OptT gate);
bool latent_prompt_fits(T z, int64_t dim_pad, int64_t rot_pad, int64_t vdim);
void latent_prompt(T out, T z, int64_t q_at, int64_t head_cols,
                   int64_t heads, T k, T kr, T vt, T cu, T start, T length,
                   int64_t max_q, double scale, int64_t window, OptT gate);
void ssm_step(T y, T z, OptT xbc, int64_t z_at, int64_t xbc_at,
              int64_t dt_at, T conv, T conv_b, T dt_bias, T A_log, T D,
              T ring, T state, T slots, T pos, OptT cu);
void conv_span(T out, T z, int64_t xbc_at, T conv, T conv_b, T ring, T slots,
               T pos, T cu, int64_t max_len);
bool ssm_chunks_fit(T z, int64_t vdim, int64_t state, int64_t taps);
void conv_chunks(T xt, T b, T bt, T c, T da, T z, int64_t xbc_at,
                 int64_t dt_at, int64_t vdim, int64_t state, T conv,
                 T conv_b, T dt_bias, T A_log, T ring, T slots, T pos, T cu,
                 T seq, T row, T count);
void ssm_chunks(T y, T z, int64_t z_at, int64_t vdim, int64_t state_size,
                T xt, T b, T bt, T c, T da, T D, T state, T slots, T pos,
                T cu, T first);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("residual_norm", &residual_norm,
        "fp32 residual add, loop entry and RMS norm");
  m.def("silu_mul", &silu_mul, "silu(gate) * up");
  m.def("group_rms_norm", &group_rms_norm, "RMS norm of equal parts");
  m.def("latent_epilogue", &latent_epilogue,
        "Rotation, latent norm, cache write");
  m.def("latent_absorb", &latent_absorb, "Queries in latent space");
  m.def("latent_rows_fits", &latent_rows_fits);
  m.def("latent_rows", &latent_rows,
        "Paged latent attention, single query rows (MFMA)");
  m.def("latent_rows_plain", &latent_rows_plain,
        "Paged latent attention, single query rows of any size");
  m.def("latent_merge", &latent_merge, "Partitions of a row into one");
  m.def("latent_out", &latent_out, "Values out of latent space, gate");
  m.def("latent_prompt_fits", &latent_prompt_fits);
  m.def("latent_prompt", &latent_prompt, "Latent attention of prompts (MFMA)");
  m.def("ssm_step", &ssm_step, "Mamba-2 recurrence, token by token");
  m.def("conv_span", &conv_span, "Causal convolution of prompt portions");
  m.def("ssm_chunks_fit", &ssm_chunks_fit);
  m.def("conv_chunks", &conv_chunks, "Operands of 64-token chunks");
  m.def("ssm_chunks", &ssm_chunks, "Mamba-2 over 64-token chunks (MFMA)");
}
