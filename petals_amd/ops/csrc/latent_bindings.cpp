// Python bindings of the latent-attention / output-norm / routed-expert kernels.
// A library of its own: a server of such a model needs nothing else compiled.
#include <torch/extension.h>

torch::Tensor gemv_bf16(
    torch::Tensor wt, torch::Tensor x, torch::Tensor workspace,
    c10::optional<torch::Tensor> residual, int64_t epilogue, int64_t splits_override,
    c10::optional<torch::Tensor> bias);
torch::Tensor gemv_bf16_moe(
    torch::Tensor wt_all, torch::Tensor x, torch::Tensor sel, int64_t k_per_tok,
    torch::Tensor workspace, int64_t epilogue, int64_t splits_override, double limit, double alpha);
torch::Tensor moe_gemm(
    c10::optional<torch::Tensor> wt_all, c10::optional<torch::Tensor> packed_all,
    c10::optional<torch::Tensor> absmax_all, torch::Tensor x, torch::Tensor sorted_pairs,
    torch::Tensor tile_expert, int64_t k_per_tok, int64_t n_rows);
torch::Tensor latent_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t window, double scale, int64_t splits,
    int64_t values, c10::optional<torch::Tensor> sink, c10::optional<torch::Tensor> factor);
void latent_write(
    torch::Tensor y, int64_t offset, torch::Tensor w, torch::Tensor cache,
    torch::Tensor pos, torch::Tensor owner, torch::Tensor tables, double eps);
std::vector<torch::Tensor> sublayer_out(
    torch::Tensor y, c10::optional<torch::Tensor> slot_w, torch::Tensor norm_w, double eps,
    c10::optional<torch::Tensor> x, int64_t dp, bool want_bf16, c10::optional<torch::Tensor> router, int64_t top);
torch::Tensor batched_linear(torch::Tensor a, torch::Tensor w, bool out_f32, c10::optional<torch::Tensor> out);
torch::Tensor clamped_swiglu(torch::Tensor gu, double limit, double alpha);
std::vector<torch::Tensor> moe_group(torch::Tensor sel, int64_t experts, int64_t mt);
torch::Tensor moe_linear_f32(torch::Tensor w, torch::Tensor x, torch::Tensor sel, int64_t k);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("gemv_bf16", &gemv_bf16, "split-K bf16 gemv with fused epilogue",
        py::arg("wt"), py::arg("x"), py::arg("workspace"), py::arg("residual"), py::arg("epilogue"),
        py::arg("splits") = 0, py::arg("bias") = py::none());
  m.def("gemv_bf16_moe", &gemv_bf16_moe, "device-routed expert gemv (bf16 weights)",
        py::arg("wt_all"), py::arg("x"), py::arg("sel"), py::arg("k_per_tok"),
        py::arg("workspace"), py::arg("epilogue"), py::arg("splits") = 0,
        py::arg("limit") = 0.0, py::arg("alpha") = 0.0);
  m.def("moe_gemm", &moe_gemm, "grouped MFMA GEMM over expert-sorted pairs");
  m.def("latent_attention", &latent_attention, "sliding-window latent attention over a paged cache",
        py::arg("q"), py::arg("cache"), py::arg("pos"), py::arg("owner"), py::arg("tables"), py::arg("tiles"),
        py::arg("run_tokens"), py::arg("max_keys"), py::arg("window"), py::arg("scale"), py::arg("splits") = 0,
        py::arg("values") = 0, py::arg("sink") = py::none(), py::arg("factor") = py::none());
  m.def("latent_write", &latent_write, "RMS-normalise latents into their cache pages");
  m.def("sublayer_out", &sublayer_out, "output norm + 32-bit residual (+ router)");
  m.def("batched_linear", &batched_linear, "out[t,h,n] = sum_k a[t,h,k] w[h,n,k]",
        py::arg("a"), py::arg("w"), py::arg("out_f32"), py::arg("out") = py::none());
  m.def("clamped_swiglu", &clamped_swiglu, "g * sigmoid(alpha g) * (u + 1), clamped");
  m.def("moe_group", &moe_group, "expert-sorted, tile-padded pairs");
  m.def("moe_linear_f32", &moe_linear_f32, "expert products in 32-bit");
}
