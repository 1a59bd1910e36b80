// Python bindings of the kernels of pre-norm blocks with gated linear attention or
// latent attention with a rotated key part. A library of its own: a server of such a
// model needs nothing else compiled.
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
torch::Tensor bias_xielu(torch::Tensor y, torch::Tensor bias, double pos, double neg);
torch::Tensor latent_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t window, double scale, int64_t splits,
    int64_t values, c10::optional<torch::Tensor> sink, c10::optional<torch::Tensor> factor);
std::vector<torch::Tensor> latent_rows(
    torch::Tensor y, int64_t at_q, torch::Tensor w_q, int64_t q_pad, bool q_f32, int64_t at_kv,
    c10::optional<torch::Tensor> w_kv, int64_t kv_pad, int64_t rot, torch::Tensor quarters, torch::Tensor cache,
    int64_t at_gate, int64_t heads, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables, double eps);
void rotate_queries(
    torch::Tensor y, int64_t first, int64_t rot_pad, torch::Tensor quarters, torch::Tensor pos, torch::Tensor q,
    int64_t offset);
torch::Tensor forget_prefill(
    torch::Tensor y, torch::Tensor bias, torch::Tensor lower, torch::Tensor tiles, torch::Tensor bounds,
    torch::Tensor pos, torch::Tensor owner, torch::Tensor slot, torch::Tensor state, int64_t heads, int64_t dim,
    int64_t vdim, std::vector<int64_t> cols);
torch::Tensor forget_decode(
    torch::Tensor y, torch::Tensor bias, torch::Tensor lower, torch::Tensor norm_w, torch::Tensor pos,
    torch::Tensor slot, torch::Tensor state, int64_t heads, int64_t dim, int64_t vdim, std::vector<int64_t> cols,
    int64_t width, double eps);
torch::Tensor ssm_prefill(
    torch::Tensor y, torch::Tensor conv_w, torch::Tensor conv_b, torch::Tensor a_exp, torch::Tensor dt_bias,
    torch::Tensor skip, torch::Tensor tiles, torch::Tensor bounds, torch::Tensor pos, torch::Tensor owner,
    torch::Tensor slot, torch::Tensor state, torch::Tensor conv, int64_t heads, int64_t groups, int64_t dim,
    int64_t vdim, int64_t o_conv, int64_t o_dt);
torch::Tensor ssm_decode(
    torch::Tensor y, torch::Tensor conv_w, torch::Tensor conv_b, torch::Tensor a_exp, torch::Tensor dt_bias,
    torch::Tensor skip, torch::Tensor pos, torch::Tensor slot, torch::Tensor state, torch::Tensor conv, int64_t heads,
    int64_t groups, int64_t dim, int64_t vdim, int64_t o_conv, int64_t o_dt);
torch::Tensor group_norm(
    torch::Tensor o, c10::optional<torch::Tensor> gate, torch::Tensor w, int64_t groups, int64_t width, bool f32,
    double eps);
bool linear_decodes(int64_t dim, int64_t vdim);

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
  m.def("bias_xielu", &bias_xielu, "xIELU of y + bias, in place or of split-K partial sums");
  m.def("latent_attention", &latent_attention, "latent attention over a paged cache",
        py::arg("q"), py::arg("cache"), py::arg("pos"), py::arg("owner"), py::arg("tables"), py::arg("tiles"),
        py::arg("run_tokens"), py::arg("max_keys"), py::arg("window"), py::arg("scale"), py::arg("splits") = 0,
        py::arg("values") = 0, py::arg("sink") = py::none(), py::arg("factor") = py::none());
  m.def("latent_rows", &latent_rows, "norms of the latents, rotated key part and gates; writes the cache");
  m.def("rotate_queries", &rotate_queries, "rotated part of the queries");
  m.def("forget_prefill", &forget_prefill, "linear attention with a forget gate over chunks of 16 tokens");
  m.def("forget_decode", &forget_decode, "linear attention with a forget gate, one token per sequence");
  m.def("ssm_prefill", &ssm_prefill, "state-space layer over chunks of 16 tokens");
  m.def("ssm_decode", &ssm_decode, "state-space layer, one token per sequence");
  m.def("group_norm", &group_norm, "gate and RMS norm in groups");
  m.def("linear_decodes", &linear_decodes, "whether the decoding kernels take these head sizes");
}
