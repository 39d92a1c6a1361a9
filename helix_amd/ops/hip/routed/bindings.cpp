// Python bindings for helix_amd._C_routed: mixtures of experts, residual
// streams side by side, and the selective scan.
#include <torch/extension.h>

using OptT = c10::optional<torch::Tensor>;
using T = torch::Tensor;

void hyper_embed(T h, T x, T ids, T pos, T embed, T places, T into, T alpha,
                 T w, T b);
void hyper_step(T h, T x, T y, T mix, T out, T into, T alpha, T w, T b,
                OptT tap);
void hyper_step_routed(T h, T x, T rows, T slot, T weight, T self, T mix,
                       T out, T into, T alpha, T w, T b, OptT tap);
void softcap(T x, double cap);
int64_t route_max_outputs();
void route(T ids, T weights, T rank, T hist, T z, T correction,
           int64_t experts, int64_t groups, int64_t keep, int64_t per);
void place(T order, T slot, T tiles, T ids, T rank, T hist, int64_t per,
           int64_t height);
bool experts_fit(T a, T w);
void expert_product(T out, T a, T w, T tiles, OptT order, int64_t choices,
                    int64_t height, const std::string& kind, bool relu2);
void conv_silu(T out, T z, int64_t x_at, T conv, T bias, T ring, T slots,
               T pos, OptT cu, int64_t max_len);
int64_t scan_max_state();
int64_t scan_columns(int64_t N);
void scan_step(T y, T x, T z, int64_t z_at, T dt, T bias, T bc, int64_t b_at,
               int64_t c_at, T A, T D, T state, T slots, T pos);
void scan_prompt(T y, T x, T z, int64_t z_at, T dt, T bias, T bc,
                 int64_t b_at, int64_t c_at, T A, T D, T state, T slots,
                 T pos, T cu, OptT row, OptT count, OptT first, OptT entry,
                 OptT sums);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("hyper_embed", &hyper_embed, "Embedding into all streams, and a norm");
  m.def("hyper_step", &hyper_step, "A result into the streams, and a norm");
  m.def("hyper_step_routed", &hyper_step_routed,
        "A mixture's rows into the streams, and a norm");
  m.def("softcap", &softcap, "cap * tanh(x / cap) in place");
  m.def("route_max_outputs", &route_max_outputs);
  m.def("route", &route, "Choice of experts per token");
  m.def("place", &place, "Experts' token lists and tiles");
  m.def("experts_fit", &experts_fit);
  m.def("expert_product", &expert_product, "All experts' matrix products");
  m.def("conv_silu", &conv_silu, "Short causal convolution and silu");
  m.def("scan_max_state", &scan_max_state);
  m.def("scan_columns", &scan_columns);
  m.def("scan_step", &scan_step, "Selective scan of single tokens");
  m.def("scan_prompt", &scan_prompt, "Selective scan of prompt portions");
}
