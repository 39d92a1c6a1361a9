// Python bindings for helix_amd._C_ext: kernels of the designs with paged
// talking-head attention and depth-averaged residual streams.
#include <torch/extension.h>

using OptT = c10::optional<torch::Tensor>;

void embed_norm(torch::Tensor h, torch::Tensor x, torch::Tensor ids,
                torch::Tensor embed, torch::Tensor w, double eps);
void depth_norm(torch::Tensor h, OptT x_out, torch::Tensor x,
                torch::Tensor y, torch::Tensor hist, int64_t n_prev,
                bool store_new, torch::Tensor coef, torch::Tensor w,
                double eps);
void unit_qkv_cache(torch::Tensor z, int64_t q_off, int64_t k_off,
                    int64_t v_off, torch::Tensor q_out, torch::Tensor k_cache,
                    torch::Tensor v_cache, torch::Tensor slots, OptT v_first,
                    OptT lam, bool first, int64_t head_dim, double eps);
void poly_norm(torch::Tensor out, torch::Tensor z, torch::Tensor coef,
               double eps);
void layer_epilogue(torch::Tensor z, int64_t q_off, int64_t k_off,
                    int64_t v_off, torch::Tensor q_out, torch::Tensor k_cache,
                    torch::Tensor v_cache, torch::Tensor slots, OptT v_first,
                    OptT lam, bool first, int64_t head_dim, double eps,
                    torch::Tensor ff_out, torch::Tensor ff_z,
                    torch::Tensor coef);
void talk_attn_rows(torch::Tensor out, torch::Tensor q, torch::Tensor kc,
                    torch::Tensor vc, torch::Tensor block_tables,
                    OptT row_seq, torch::Tensor row_len, int64_t max_keys,
                    double scale, double cap, int64_t window, OptT slopes,
                    OptT talk, OptT gate, torch::Tensor scores,
                    torch::Tensor ml, torch::Tensor tmp);
bool talk_prefill_fits(int64_t H, int64_t Dp, int64_t E);
void talk_attn_prefill(torch::Tensor out, torch::Tensor q, torch::Tensor kc,
                       torch::Tensor vc, torch::Tensor block_tables,
                       torch::Tensor cu_seqlens, torch::Tensor seq_lens,
                       int64_t max_q, double scale, double cap,
                       int64_t window, OptT slopes, torch::Tensor talk,
                       OptT gate, torch::Tensor lse);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_norm", &embed_norm,
        "Embedding gather into the fp32 stream + RMS norm");
  m.def("depth_norm", &depth_norm,
        "fp32 residual add + depth average + RMS norm");
  m.def("unit_qkv_cache", &unit_qkv_cache,
        "Unit-RMS q/k, value mixing, paged-cache write");
  m.def("poly_norm", &poly_norm, "PolyNorm activation");
  m.def("layer_epilogue", &layer_epilogue,
        "unit_qkv_cache and poly_norm in one launch");
  m.def("talk_attn_rows", &talk_attn_rows,
        "Paged talking-head attention, one query row at a time");
  m.def("talk_prefill_fits", &talk_prefill_fits);
  m.def("talk_attn_prefill", &talk_attn_prefill,
        "Paged talking-head prefill attention (MFMA)");
}
