// Python bindings of layers whose sublayers stand side by side, each behind a
// norm and an input convolution.

#include <torch/extension.h>

typedef c10::optional<at::Tensor> Opt;

void canon_norm(at::Tensor x, Opt delta, at::Tensor coef, at::Tensor tails,
                at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
                at::Tensor seq_of, bool single, int64_t n_seqs, double eps,
                std::vector<at::Tensor> out, std::vector<at::Tensor> operands,
                std::vector<bool> wants);
void qkv_conv(at::Tensor y, at::Tensor bias, at::Tensor conv, at::Tensor tails,
              at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
              at::Tensor seq_of, at::Tensor cache_slots, bool single,
              int64_t n_seqs, at::Tensor cache, int64_t kc, at::Tensor q);
at::Tensor power_sums(at::Tensor u, int64_t ff);
void poly_norm(at::Tensor u, int64_t ff, int64_t total, at::Tensor act,
               double eps, at::Tensor z, int64_t off, Opt swz, Opt sums);
void tanh_rows(at::Tensor y, int64_t off, at::Tensor out, Opt swz);
at::Tensor softcap(at::Tensor x, double cap);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "runbooks_amd gfx950 HIP kernels: input convolutions, PolyNorm";
  m.def("canon_norm", &canon_norm,
        "residual += pending; norm and input convolutions of the sublayers");
  m.def("qkv_conv", &qkv_conv,
        "biases and convolutions of queries, keys, values; cache write");
  m.def("power_sums", &power_sums, "sums of z^2, z^4, z^6 per token");
  m.def("poly_norm", &poly_norm, "polynomial of norms");
  m.def("tanh_rows", &tanh_rows, "tanh of some columns");
  m.def("softcap", &softcap, "cap tanh(logits / cap)");
}
