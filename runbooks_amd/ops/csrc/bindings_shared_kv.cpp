// Python bindings of the attention over paged rows that hold a token's key and
// value at once.

#include <torch/extension.h>

void shared_kv_prep(at::Tensor y, at::Tensor cos, at::Tensor sin,
                    at::Tensor positions, at::Tensor slots, at::Tensor cache,
                    int64_t heads, int64_t rotc);
void shared_kv_attend(at::Tensor y, at::Tensor cache, at::Tensor block_tables,
                      at::Tensor cu_q, at::Tensor seq_lens, int64_t n_seqs,
                      int64_t t_seqs, int64_t max_q, int64_t nsplit,
                      double scale, int64_t window, int64_t heads,
                      int64_t hc, int64_t voff, at::Tensor z,
                      c10::optional<at::Tensor> swz, int64_t chunk,
                      c10::optional<at::Tensor> positions,
                      c10::optional<at::Tensor> sink, double out_scale,
                      c10::optional<at::Tensor> lam, int64_t count,
                      double eps);
void shared_kv_flash(at::Tensor y, at::Tensor cache, at::Tensor block_tables,
                     at::Tensor cu_q, at::Tensor seq_lens, int64_t first_seq,
                     int64_t n_seqs, int64_t max_q, double scale,
                     int64_t window, int64_t heads, int64_t hc, int64_t voff,
                     at::Tensor z, int64_t chunk,
                     c10::optional<at::Tensor> positions,
                     c10::optional<at::Tensor> sink, double out_scale,
                     c10::optional<at::Tensor> lam, int64_t count,
                     double eps);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "runbooks_amd gfx950 HIP kernels: attention over rows of keys "
            "and values";
  m.def("shared_kv_prep", &shared_kv_prep,
        "rotations and cache write of shared keys and values");
  m.def("shared_kv_attend", &shared_kv_attend,
        "attention of decoded tokens and short portions");
  m.def("shared_kv_flash", &shared_kv_flash,
        "flash attention of long portions over the paged cache");
}
