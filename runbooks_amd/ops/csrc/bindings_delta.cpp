// Python bindings of the gated and the generalized delta rule.

#include <torch/extension.h>

typedef c10::optional<at::Tensor> Opt;

void delta_step(at::Tensor y, at::Tensor y2, at::Tensor conv, at::Tensor decay,
                at::Tensor state, at::Tensor tails, at::Tensor positions,
                at::Tensor cu_q, at::Tensor slots, at::Tensor o,
                int64_t n_seqs, int64_t kv, int64_t dim);
void delta_chunk(at::Tensor y, at::Tensor y2, at::Tensor conv,
                 at::Tensor decay, at::Tensor state, at::Tensor tails,
                 at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
                 at::Tensor o, int64_t first_seq, int64_t n_seqs,
                 int64_t max_q, int64_t kv, int64_t dim);
void delta_out(at::Tensor o, at::Tensor w, at::Tensor gate, int64_t off_g,
               at::Tensor z, Opt swz, int64_t heads, int64_t vdim, double eps,
               at::Tensor y, Opt tails, at::Tensor positions, at::Tensor cu_q,
               at::Tensor slots, int64_t n_seqs, int64_t end);
void general_delta_step(at::Tensor y, at::Tensor y2, at::Tensor bias,
                        double scale, at::Tensor state, at::Tensor positions,
                        at::Tensor cu_q, at::Tensor slots, at::Tensor o,
                        int64_t n_seqs);
void general_delta_chunk(at::Tensor y, at::Tensor y2, at::Tensor bias,
                         double scale, at::Tensor state, at::Tensor positions,
                         at::Tensor cu_q, at::Tensor slots, at::Tensor o,
                         int64_t first_seq, int64_t n_seqs, int64_t max_q);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "runbooks_amd gfx950 HIP kernels: delta rules";
  m.def("delta_step", &delta_step, "gated delta rule, token after token");
  m.def("delta_chunk", &delta_chunk,
        "gated delta rule of long portions in chunks");
  m.def("delta_out", &delta_out,
        "norm per head times sigmoid gate; the convolutions' last inputs");
  m.def("general_delta_step", &general_delta_step,
        "generalized delta rule, token after token");
  m.def("general_delta_chunk", &general_delta_chunk,
        "generalized delta rule of long portions in chunks");
}
