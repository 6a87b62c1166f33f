// Python bindings of the ops every served model runs (norms, gated units,
// decode GEMM, sampling).

#include <torch/extension.h>

std::vector<at::Tensor> rmsnorm_fwd(at::Tensor x, at::Tensor w, double eps);
std::vector<at::Tensor> rmsnorm_fwd_dec(at::Tensor x, at::Tensor w, double eps);
std::vector<at::Tensor> rmsnorm_res_fwd_dec(at::Tensor x, at::Tensor res, at::Tensor w, double eps);
std::vector<at::Tensor> rmsnorm_res_slab_fwd_dec(at::Tensor x, at::Tensor slabs, at::Tensor w, double eps);
std::vector<at::Tensor> rmsnorm_res32(at::Tensor x, c10::optional<at::Tensor> delta, at::Tensor w, double eps, bool want_swz, double offset);
std::vector<at::Tensor> rmsnorm_bwd(at::Tensor x, at::Tensor w, at::Tensor dy,
                                    at::Tensor inv_rms);
std::vector<at::Tensor> layernorm_res32(at::Tensor x, c10::optional<at::Tensor> delta, at::Tensor w, at::Tensor b, double eps, bool want_swz);
std::vector<at::Tensor> join_res32(at::Tensor x, c10::optional<at::Tensor> delta, at::Tensor other, bool want_swz);
at::Tensor swiglu_packed(at::Tensor y);
at::Tensor geglu_packed(at::Tensor y);
std::vector<at::Tensor> swiglu_packed_dec(at::Tensor y);
std::vector<at::Tensor> geglu_packed_dec(at::Tensor y);
at::Tensor decode_gemm_raw(at::Tensor xs, at::Tensor ws, int64_t M, int64_t N, int64_t K, bool f32);
at::Tensor decode_gemm(at::Tensor xs, at::Tensor ws, int64_t M, int64_t N, int64_t K, int64_t force_split);
at::Tensor decode_swizzle_w(at::Tensor w);
at::Tensor decode_swizzle_x(at::Tensor x);
int64_t decode_gemm_split(int64_t N, int64_t K);
bool decode_gemm_supported(int64_t M, int64_t N, int64_t K);
at::Tensor sample_tokens(at::Tensor logits, double temperature, int64_t seed);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "runbooks_amd gfx950 HIP kernels: core serving ops";
  m.def("rmsnorm_fwd", &rmsnorm_fwd, "fused RMSNorm forward (bf16/f32)");
  m.def("rmsnorm_fwd_dec", &rmsnorm_fwd_dec,
        "RMSNorm forward + decode-GEMM operand swizzle in one pass");
  m.def("rmsnorm_res_fwd_dec", &rmsnorm_res_fwd_dec,
        "residual add + RMSNorm + decode operand swizzle in one pass");
  m.def("rmsnorm_res_slab_fwd_dec", &rmsnorm_res_slab_fwd_dec,
        "split-K slab combine + residual + RMSNorm + swizzle in one pass");
  m.def("rmsnorm_res32", &rmsnorm_res32,
        "fp32 residual += delta (or split-K slab), then RMSNorm");
  m.def("rmsnorm_bwd", &rmsnorm_bwd, "fused RMSNorm backward");
  m.def("layernorm_res32", &layernorm_res32,
        "fp32 residual += delta (or split-K slab), then LayerNorm");
  m.def("join_res32", &join_res32,
        "[fp32 residual + delta ; other] as a product's input");
  m.def("swiglu_packed", &swiglu_packed,
        "silu(y[:, :I]) * y[:, I:] from the fused gate/up GEMM output");
  m.def("geglu_packed", &geglu_packed,
        "packed GeGLU (tanh) epilogue [T,2I]->[T,I]");
  m.def("swiglu_packed_dec", &swiglu_packed_dec,
        "packed SwiGLU + decode-GEMM operand swizzle in one pass");
  m.def("geglu_packed_dec", &geglu_packed_dec,
        "packed GeGLU + decode-GEMM operand swizzle in one pass");
  m.def("decode_gemm_raw", &decode_gemm_raw,
        "decode GEMM returning the uncombined fp32 slab at split>1 (or always)",
        py::arg("xs"), py::arg("ws"), py::arg("M"), py::arg("N"),
        py::arg("K"), py::arg("f32") = false);
  m.def("decode_gemm", &decode_gemm,
        "v2 weight-stream decode GEMM over pre-swizzled operands: "
        "y[M<=32,N] = x @ W^T (bf16), 1KiB coalesced nt weight bursts",
        py::arg("xs"), py::arg("ws"), py::arg("M"), py::arg("N"),
        py::arg("K"), py::arg("force_split") = -1);
  m.def("decode_swizzle_w", &decode_swizzle_w,
        "one-time [N,K] -> fragment-lane-major weight layout");
  m.def("decode_swizzle_x", &decode_swizzle_x,
        "per-call x -> B-fragment lane order (zero-padded to M=32)");
  m.def("decode_gemm_split", &decode_gemm_split);
  m.def("decode_gemm_supported", &decode_gemm_supported);
  m.def("sample_tokens", &sample_tokens, "greedy / Gumbel-max sampling");
}
