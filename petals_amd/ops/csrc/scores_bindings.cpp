// Python bindings of the kernels of blocks whose attention caps its scores, subtracts
// one map from another or weighs keys by sigmoids, with a feed-forward beside it. A
// library of its own: a server of such a model needs nothing else compiled.
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
torch::Tensor prepare_rows(
    torch::Tensor y, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables, int64_t heads,
    int64_t kv_heads, int64_t dk, int64_t dim, int64_t values, c10::optional<torch::Tensor> bias,
    c10::optional<torch::Tensor> conv_w, c10::optional<torch::Tensor> norm, torch::Tensor quarters, double turn_factor,
    c10::optional<torch::Tensor> conv, c10::optional<torch::Tensor> slot, bool single,
    c10::optional<torch::Tensor> tiles, c10::optional<torch::Tensor> bounds, std::vector<double> poly, int64_t poly_at,
    int64_t ff, c10::optional<torch::Tensor> act, double eps);
void capped_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t kv_heads, int64_t dv, int64_t chunk,
    double scale, double cap, torch::Tensor out, int64_t splits);
void sigmoid_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t kv_heads, int64_t dv, int64_t chunk,
    double scale, torch::Tensor bias, torch::Tensor out, int64_t splits);
void paired_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t kv_heads, int64_t dv, int64_t chunk,
    double scale, double share, double factor, double eps, int64_t vdim, c10::optional<torch::Tensor> gate,
    torch::Tensor out, int64_t splits);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("gemv_bf16", &gemv_bf16, "split-K bf16 gemv with fused epilogue",
        py::arg("wt"), py::arg("x"), py::arg("workspace"), py::arg("residual"), py::arg("epilogue"),
        py::arg("splits") = 0, py::arg("bias") = py::none());
  m.def("batched_linear", &batched_linear, "out[t,h,n] = sum_k a[t,h,k] w[h,n,k]",
        py::arg("a"), py::arg("w"), py::arg("out_f32"), py::arg("out") = py::none());
  m.def("residual_norm", &residual_norm, "x += mult (y + bias); RMS norm of x in equal parts",
        py::arg("x"), py::arg("y"), py::arg("bias"), py::arg("w"), py::arg("d"), py::arg("eps"), py::arg("out_f32"),
        py::arg("mult") = 1.0, py::arg("groups") = 1);
  m.def("residual_sum", &residual_sum, "x += mult (split-K partial sums + bias)",
        py::arg("partials"), py::arg("bias"), py::arg("x"), py::arg("d"), py::arg("mult") = 1.0);
  m.def("prepare_rows", &prepare_rows,
        "bias, short convolution, norm and rotation of queries and keys, PolyNorm; writes keys and values",
        py::arg("y"), py::arg("cache"), py::arg("pos"), py::arg("owner"), py::arg("tables"), py::arg("heads"),
        py::arg("kv_heads"), py::arg("dk"), py::arg("dim"), py::arg("values"), py::arg("bias"), py::arg("conv_w"),
        py::arg("norm"), py::arg("quarters"), py::arg("turn_factor"), py::arg("conv"), py::arg("slot"),
        py::arg("single"), py::arg("tiles"), py::arg("bounds"), py::arg("poly"), py::arg("poly_at"), py::arg("ff"),
        py::arg("act"), py::arg("eps"));
#define ROWS                                                                                                   \
  py::arg("q"), py::arg("cache"), py::arg("pos"), py::arg("owner"), py::arg("tables"), py::arg("tiles"),       \
      py::arg("run_tokens"), py::arg("max_keys"), py::arg("kv_heads"), py::arg("dv"), py::arg("chunk"), py::arg("scale")
  m.def("capped_attention", &capped_attention, "softmax of capped scores over paged keys and values", ROWS,
        py::arg("cap"), py::arg("out"), py::arg("splits") = 0);
  m.def("sigmoid_attention", &sigmoid_attention, "sigmoid weights over paged keys and values", ROWS, py::arg("bias"),
        py::arg("out"), py::arg("splits") = 0);
  m.def("paired_attention", &paired_attention, "difference of two softmax maps over paged keys and values", ROWS,
        py::arg("share"), py::arg("factor"), py::arg("eps"), py::arg("vdim"), py::arg("gate"), py::arg("out"),
        py::arg("splits") = 0);
#undef ROWS
}
