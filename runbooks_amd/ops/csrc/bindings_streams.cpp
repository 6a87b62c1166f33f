// Python bindings of the residual streams, minGRU, mixture of experts and the
// preparation of queries, keys and values.

#include <torch/extension.h>

typedef c10::optional<at::Tensor> Opt;

std::vector<at::Tensor> streams_norm(at::Tensor x, Opt delta, Opt extra, Opt y,
                                     int64_t off, Opt join, at::Tensor inp,
                                     at::Tensor norm, bool bf16, bool operand);
std::vector<at::Tensor> squared_relu(at::Tensor y, int64_t n, bool operand);
void qkv_prep(at::Tensor y, at::Tensor cos, at::Tensor sin,
              at::Tensor positions, at::Tensor slots, at::Tensor cache,
              at::Tensor norms, int64_t heads, int64_t dim, int64_t hc,
              double eps);
void min_gru_step(at::Tensor y, int64_t off, at::Tensor bias, at::Tensor state,
                  at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
                  int64_t first_seq, int64_t n_seqs, at::Tensor z,
                  int64_t z_off, double scale, Opt swz);
void min_gru_scan(at::Tensor y, int64_t off, at::Tensor bias, at::Tensor state,
                  at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
                  int64_t first_seq, int64_t n_seqs, at::Tensor z,
                  int64_t z_off, double scale, int64_t max_q);
std::vector<at::Tensor> moe_route(at::Tensor logits, at::Tensor correction,
                                  int64_t top, int64_t groups, int64_t keep);
std::vector<at::Tensor> moe_plan(at::Tensor chosen, int64_t experts,
                                 int64_t tile);
at::Tensor moe_gemm(at::Tensor x, at::Tensor w, at::Tensor pairs,
                    at::Tensor tiles, at::Tensor weights, int64_t tile,
                    bool down);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "runbooks_amd gfx950 HIP kernels: residual streams, minGRU, "
            "mixture of experts";
  m.def("streams_norm", &streams_norm,
        "streams += pending result; next sublayer's normed input");
  m.def("squared_relu", &squared_relu, "relu(y[:, :n])^2");
  m.def("qkv_prep", &qkv_prep,
        "norms and rotations of queries and keys, cache write");
  m.def("min_gru_step", &min_gru_step, "minGRU, token after token");
  m.def("min_gru_scan", &min_gru_scan, "minGRU of long portions in segments");
  m.def("moe_route", &moe_route, "chosen experts and their weights");
  m.def("moe_plan", &moe_plan, "pairs sorted by expert, in tiles");
  m.def("moe_gemm", &moe_gemm, "one product per tile of pairs");
}
