// Python bindings of the attention on shared keys and values and of the
// lightning attention.

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
                      c10::optional<at::Tensor> sink, double out_scale);
void shared_kv_flash(at::Tensor y, at::Tensor cache, at::Tensor block_tables,
                     at::Tensor cu_q, at::Tensor seq_lens, int64_t first_seq,
                     int64_t n_seqs, int64_t max_q, double scale,
                     int64_t window, int64_t heads, int64_t hc, int64_t voff,
                     at::Tensor z, int64_t chunk,
                     c10::optional<at::Tensor> positions,
                     c10::optional<at::Tensor> sink, double out_scale);
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
  m.doc() = "runbooks_amd gfx950 HIP kernels: attention on shared keys and "
            "values, lightning attention";
  m.def("shared_kv_prep", &shared_kv_prep,
        "rotations and cache write of shared keys and values");
  m.def("shared_kv_attend", &shared_kv_attend,
        "attention of decoded tokens and short portions");
  m.def("shared_kv_flash", &shared_kv_flash,
        "flash attention of long portions over the paged cache");
  m.def("lightning_chunk_size", &lightning_chunk_size);
  m.def("lightning_step", &lightning_step,
        "linear recurrence, token after token");
  m.def("lightning_chunk", &lightning_chunk,
        "linear recurrence of long portions in chunks");
  m.def("lightning_out", &lightning_out,
        "norm over all heads times sigmoid gate");
}
