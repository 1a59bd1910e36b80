// Python bindings of the kernels of pre-norm blocks with windowed attention or a
// gated delta rule. A library of its own: a server of such a model needs nothing
// else compiled.
#include <torch/extension.h>

torch::Tensor gemv_bf16(
    torch::Tensor wt, torch::Tensor x, torch::Tensor workspace,
    c10::optional<torch::Tensor> residual, int64_t epilogue, int64_t splits_override,
    c10::optional<torch::Tensor> bias);
torch::Tensor batched_linear(torch::Tensor a, torch::Tensor w, bool out_f32, c10::optional<torch::Tensor> out);
torch::Tensor residual_norm(
    torch::Tensor x, c10::optional<torch::Tensor> y, c10::optional<torch::Tensor> bias,
    c10::optional<torch::Tensor> w, int64_t d, double eps, bool out_f32, double mult, int64_t groups);
void residual_sum(torch::Tensor partials, c10::optional<torch::Tensor> bias, torch::Tensor x, int64_t d, double mult);
torch::Tensor bias_relu2(torch::Tensor y, torch::Tensor bias);
torch::Tensor paged_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t kv_heads, int64_t dv, int64_t window,
    double scale, c10::optional<torch::Tensor> slopes, c10::optional<torch::Tensor> sink,
    c10::optional<torch::Tensor> gate, bool out_f32, int64_t splits);
torch::Tensor attn_prepare(
    torch::Tensor y, torch::Tensor bias, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner,
    torch::Tensor tables, int64_t heads, int64_t kv_heads, int64_t dk, int64_t dv, double temp_coef,
    int64_t temp_every, c10::optional<torch::Tensor> first, c10::optional<torch::Tensor> lambda, int64_t vdim);
torch::Tensor delta_prefill(
    torch::Tensor y, torch::Tensor a, torch::Tensor conv_w, torch::Tensor a_exp, torch::Tensor dt_bias,
    torch::Tensor tiles, torch::Tensor bounds, torch::Tensor pos, torch::Tensor owner, torch::Tensor slot,
    torch::Tensor delta, torch::Tensor conv, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim,
    std::vector<int64_t> cols);
torch::Tensor delta_norm(
    torch::Tensor o, torch::Tensor gate, torch::Tensor w, int64_t heads, int64_t width, bool f32, double eps);
bool delta_decodes(int64_t dim, int64_t vdim);
torch::Tensor delta_decode(
    torch::Tensor y, torch::Tensor conv_w, torch::Tensor a2, torch::Tensor g2, int64_t a1_col, int64_t g1_col,
    torch::Tensor a_exp, torch::Tensor dt_bias, torch::Tensor norm_w, torch::Tensor pos, torch::Tensor slot,
    torch::Tensor delta, torch::Tensor conv, int64_t heads, int64_t kv_heads, int64_t dim,
    int64_t vdim, std::vector<int64_t> cols, int64_t width, double eps);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("gemv_bf16", &gemv_bf16, "split-K bf16 gemv with fused epilogue",
        py::arg("wt"), py::arg("x"), py::arg("workspace"), py::arg("residual"), py::arg("epilogue"),
        py::arg("splits") = 0, py::arg("bias") = py::none());
  m.def("batched_linear", &batched_linear, "out[t,h,n] = sum_k a[t,h,k] w[h,n,k]",
        py::arg("a"), py::arg("w"), py::arg("out_f32"), py::arg("out") = py::none());
  m.def("residual_norm", &residual_norm, "x += mult (y + bias); RMS norm of x",
        py::arg("x"), py::arg("y"), py::arg("bias"), py::arg("w"), py::arg("d"), py::arg("eps"), py::arg("out_f32"),
        py::arg("mult") = 1.0, py::arg("groups") = 1);
  m.def("residual_sum", &residual_sum, "x += mult (split-K partial sums + bias)",
        py::arg("partials"), py::arg("bias"), py::arg("x"), py::arg("d"), py::arg("mult") = 1.0);
  m.def("bias_relu2", &bias_relu2, "relu(y + bias)^2 in place");
  m.def("paged_attention", &paged_attention, "windowed attention with distance bias, sink and gate over paged keys and values",
        py::arg("q"), py::arg("cache"), py::arg("pos"), py::arg("owner"), py::arg("tables"), py::arg("tiles"),
        py::arg("run_tokens"), py::arg("max_keys"), py::arg("kv_heads"), py::arg("dv"), py::arg("window"),
        py::arg("scale"), py::arg("slopes"), py::arg("sink"), py::arg("gate"), py::arg("out_f32"),
        py::arg("splits") = 0);
  m.def("attn_prepare", &attn_prepare, "bias, query temperature, value mixing; writes keys and values",
        py::arg("y"), py::arg("bias"), py::arg("cache"), py::arg("pos"), py::arg("owner"), py::arg("tables"),
        py::arg("heads"), py::arg("kv_heads"), py::arg("dk"), py::arg("dv"), py::arg("temp_coef"),
        py::arg("temp_every"), py::arg("first"), py::arg("lam"), py::arg("vdim"));
  m.def("delta_prefill", &delta_prefill, "gated delta rule over chunks of 16 tokens");
  m.def("delta_norm", &delta_norm, "norm and gate of the delta rule's result");
  m.def("delta_decodes", &delta_decodes, "whether delta_decode takes these head sizes");
  m.def("delta_decode", &delta_decode, "gated delta rule, one token per sequence");
}
