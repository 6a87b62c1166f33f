// Python bindings of the lightning attention.

#include <torch/extension.h>

int64_t lightning_chunk_size();
void lightning_step(at::Tensor y, at::Tensor state, at::Tensor positions,
                    at::Tensor cu_q, at::Tensor slots, at::Tensor powers,
                    at::Tensor o, int64_t n_seqs);
void lightning_chunk(at::Tensor y, at::Tensor state, at::Tensor positions,
                     at::Tensor cu_q, at::Tensor slots, at::Tensor powers,
                     at::Tensor o, int64_t first_seq, int64_t n_seqs,
                     int64_t max_q);
void lightning_out(at::Tensor o, at::Tensor w, at::Tensor y, int64_t off_g,
                   c10::optional<at::Tensor> sums, at::Tensor z,
                   c10::optional<at::Tensor> swz, int64_t count, double eps);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "runbooks_amd gfx950 HIP kernels: lightning attention";
  m.def("lightning_chunk_size", &lightning_chunk_size);
  m.def("lightning_step", &lightning_step,
        "linear recurrence, token after token");
  m.def("lightning_chunk", &lightning_chunk,
        "linear recurrence of long portions in chunks");
  m.def("lightning_out", &lightning_out,
        "norm over all heads times sigmoid gate");
}
