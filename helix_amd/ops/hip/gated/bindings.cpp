// Python bindings for helix_amd._C_gated: softmax and sigmoid attention over
// paged keys and values, linear attention (gated, or with a constant decay),
// and the fp32 stream of layers that norm before and after a sublayer.
#include <torch/extension.h>

using OptT = c10::optional<torch::Tensor>;
using T = torch::Tensor;

void stream_add(OptT h, T x, T y, T wy, T by, OptT w, OptT b, double eps,
                OptT x_out, OptT tap, OptT terms);
void stream_embed(OptT h, T ids, T embed, double scale, OptT w, OptT b,
                  double eps, OptT x_out, OptT terms);
void stream_enter(T h, T a, OptT a2, T e, double e_scale, OptT step, T w, T b,
                  double eps, OptT x_out);
void gated_mul(T out, T z, int64_t up_at, bool gelu);
void rotary_table(T cs, T pos, T freqs);
void query_temperature(T out, T pos, double coef, double every);
void attn_epilogue(OptT q, T kc, T vc, T z, int64_t q_at, int64_t k_at,
                   int64_t v_at, int64_t heads, int64_t dim, T slots, OptT cs,
                   OptT vcs, OptT qw, OptT kw, double eps, bool write_kv);
bool attn_fits(T q, int64_t vdim);
void attn_rows(OptT out, OptT part, OptT ml, T q, T kc, T vc, T bt,
               OptT row_seq, T row_len, double scale, double out_scale,
               bool sigmoid, OptT temp, OptT bias, OptT vcs, OptT row_scale,
               OptT gate);
void attn_merge(T out, T part, T ml, double out_scale, bool sigmoid,
                OptT vcs, OptT gate);
void attn_plain(T out, T q, T kc, T vc, T bt, OptT row_seq, T row_len,
                double scale, double out_scale, bool sigmoid, OptT temp,
                OptT bias, OptT vcs, OptT row_scale, OptT gate);
void attn_prompt(T out, T q, T kc, T vc, T bt, T cu, T seq_lens,
                 int64_t max_q, double scale, double out_scale, bool sigmoid,
                 OptT temp, OptT bias, OptT vcs, OptT row_scale, OptT gate);
void gla_step(T y, T z, int64_t q_at, int64_t k_at, int64_t v_at,
              int64_t g_at, int64_t a_at, int64_t vdim, int64_t rank, T a2,
              T a2_b, T norm, double tau, double q_scale, double out_scale, double eps,
              T state, T slots, T pos, OptT cu);
void decay_step(T y, T z, int64_t q_at, int64_t k_at, int64_t v_at,
                int64_t vdim, T decay, T state, T slots, T pos, OptT cu);
void decay_operands(T qe, T ke, T am, T vt, T ec, T z, int64_t q_at,
                    int64_t k_at, int64_t v_at, int64_t dim, int64_t vdim,
                    T log_decay, T row, T count);
void row_norm_gate(T y, T o, T g, T w, double eps);
bool gla_chunks_fit(T z, int64_t dim);
void gla_operands(T qe, T ke, T am, T vt, T ec, T z, int64_t q_at,
                  int64_t k_at, int64_t v_at, int64_t a_at, int64_t dim,
                  int64_t vdim, int64_t rank, T a2, T a2_b, double tau,
                  double q_scale, T row, T count);
void gla_chunks(T o, T qe, T ke, T am, T vt, T ec, int64_t vdim, T state,
                T slots, T pos, T cu, T first);
void head_norm_gate(T y, T o, T g, T w, double scale, double eps);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("stream_add", &stream_add, "x + norm(y), and its norm");
  m.def("stream_embed", &stream_embed, "Scaled embedding, and its norm");
  m.def("stream_enter", &stream_enter, "A loop pass begins, and its norm");
  m.def("gated_mul", &gated_mul, "act(gate) * up");
  m.def("rotary_table", &rotary_table, "Cosines and sines of positions");
  m.def("query_temperature", &query_temperature,
        "Factor of a query's scores by its position");
  m.def("attn_epilogue", &attn_epilogue, "Norms, rotation, cache write");
  m.def("attn_fits", &attn_fits);
  m.def("attn_rows", &attn_rows, "Paged attention of single rows (MFMA)");
  m.def("attn_merge", &attn_merge, "Partitions of a row into one");
  m.def("attn_plain", &attn_plain, "Paged attention of single rows");
  m.def("attn_prompt", &attn_prompt, "Paged attention of prompts (MFMA)");
  m.def("gla_step", &gla_step, "Gated linear attention, token by token");
  m.def("gla_chunks_fit", &gla_chunks_fit);
  m.def("gla_operands", &gla_operands, "Operands of 64-token chunks");
  m.def("gla_chunks", &gla_chunks, "Recurrence over chunks (MFMA)");
  m.def("decay_step", &decay_step,
        "Linear attention with a constant decay, token by token");
  m.def("decay_operands", &decay_operands,
        "Operands of 64-token chunks, constant decay");
  m.def("row_norm_gate", &row_norm_gate, "RMS norm of rows, sigmoid gate");
  m.def("head_norm_gate", &head_norm_gate, "RMS norm per head, gate");
}
