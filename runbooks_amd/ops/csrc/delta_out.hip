// Output of the delta rules (gfx950): RMS norm per head, times weight and
// sigmoid gate; the workgroups after the tokens' move the convolutions' last
// inputs to the sequences' slots.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 256;

template <typename T> RB_DEV float sigmoid(float x) {
  if constexpr (sizeof(T) == 2)
    return __builtin_amdgcn_rcpf(1.0f + __expf(-x));
  else
    return 1.0f / (1.0f + expf(-x));
}

template <typename T> RB_DEV void load8(const T *p, float *f) {
  rb::VIO<T>::load(p, f);
  if constexpr (rb::VIO<T>::W == 4) rb::VIO<T>::load(p + 4, f + 4);
}
template <typename T> RB_DEV void store8(T *p, const float *f) {
  rb::VIO<T>::store(p, f);
  if constexpr (rb::VIO<T>::W == 4) rb::VIO<T>::store(p + 4, f + 4);
}

struct OutArgs {
  const float *o, *w;
  int64_t tokens, ny2, ny, nz;
  int heads, vc, vdim, off_g;
  int w_head, end;                     // w's step per head; z's zeros' end
  float eps;
  const void *y2, *y;
  void *z, *swz, *tails;
  const int *positions, *cu_q, *slots;
  int taps, channels, tail_blocks;
};

// L lanes per head with NV times 8 columns each; the convolutions' inputs are
// y's first columns
template <typename T, int L, int NV>
__global__ __launch_bounds__(BLOCK) void delta_out_kernel(OutArgs a) {
  if (blockIdx.x >= a.tokens) {
    const int i = blockIdx.x - (int)a.tokens, seq = i / a.tail_blocks;
    const int q0 = a.cu_q[seq], n = a.cu_q[seq + 1] - q0;
    if (n <= 0) return;
    const bool fresh = a.positions[q0] == 0;
    const int keep = a.taps - 1;
    T *tail = (T *)a.tails + (int64_t)a.slots[seq] * keep * a.channels;
    const int c = (i % a.tail_blocks * BLOCK + threadIdx.x) * 8;
    if (c >= a.channels) return;
    for (int j = 0; j < keep; ++j) {
      const int s = n - keep + j;              // token of the portion
      float v[8] = {};
      if (s >= 0)
        load8((const T *)a.y + (int64_t)(q0 + s) * a.ny + c, v);
      else if (!fresh)
        load8(tail + (int64_t)(keep + s) * a.channels + c, v);
      store8(tail + (int64_t)j * a.channels + c, v);
    }
    return;
  }
  constexpr int GROUPS = BLOCK / L;
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x % L, n = a.heads * a.vc;
  const float *orow = a.o + t * n;
  const T *g = (const T *)a.y2 + t * a.ny2 + a.off_g;
  T *zr = (T *)a.z + t * a.nz;
  auto put = [&](int col, const float *f) {
    store8(zr + col, f);
    if (a.swz != nullptr)
      store8((T *)a.swz + (int64_t)(col >> 4) * 512 + ((col >> 3) & 1) * 256 +
             t * 8, f);
  };
  for (int h0 = 0; h0 < a.heads; h0 += GROUPS) {
    const int h = h0 + threadIdx.x / L;
    float f[NV][8], sum = 0.0f;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int c = (v * L + lane) * 8;
      if (h < a.heads && c < a.vc) {
        load8(orow + h * a.vc + c, f[v]);
#pragma unroll
        for (int k = 0; k < 8; ++k) sum += f[v][k] * f[v][k];
      }
    }
#pragma unroll
    for (int o = L / 2; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
    const float inv = 1.0f / sqrtf(sum / a.vdim + a.eps);
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int c = (v * L + lane) * 8;
      if (h < a.heads && c < a.vc) {
        float gf[8], wf[8];
        load8(g + h * a.vc + c, gf);
        load8(a.w + h * a.w_head + c, wf);
#pragma unroll
        for (int k = 0; k < 8; ++k)
          f[v][k] = f[v][k] * inv * wf[k] * sigmoid<T>(gf[k]);
        put(h * a.vc + c, f[v]);
      }
    }
  }
  const float zero[8] = {};
  for (int c = n + threadIdx.x * 8; c < a.end; c += BLOCK * 8) put(c, zero);
}

}  // namespace

// z [T, nz] (and its decode operand) from o [T, heads * vc], w f32 of one head
// or all, gate logits in `gate` from column off_g; zeros in z from o's columns
// to `end`. The new `tails` of the n_seqs sequences, where there are some.
void delta_out(at::Tensor o, at::Tensor w, at::Tensor gate, int64_t off_g,
               at::Tensor z, c10::optional<at::Tensor> swz, int64_t heads,
               int64_t vdim, double eps, at::Tensor y,
               c10::optional<at::Tensor> tails, at::Tensor positions,
               at::Tensor cu_q, at::Tensor slots, int64_t n_seqs,
               int64_t end) {
  const auto dt = z.scalar_type();
  TORCH_CHECK(o.is_cuda() && o.dim() == 2 && o.is_contiguous() &&
              o.scalar_type() == at::kFloat && w.is_contiguous() &&
              w.scalar_type() == at::kFloat && gate.dim() == 2 &&
              gate.is_contiguous() && gate.scalar_type() == dt &&
              z.dim() == 2 && z.is_contiguous() && y.dim() == 2 &&
              y.is_contiguous() && y.scalar_type() == dt,
              "delta_out: tensors");
  const int64_t T = o.size(0), n = o.size(1), nz = z.size(1);
  TORCH_CHECK(heads >= 1 && n % heads == 0, "delta_out: heads");
  const int64_t vc = n / heads;
  TORCH_CHECK(gate.size(0) == T && z.size(0) == T && y.size(0) == T &&
              (w.numel() == vc || w.numel() == n) &&
              vc % 8 == 0 && vc >= 8 && vc <= 1024 &&
              nz % 8 == 0 && nz >= n && end >= n && end <= nz &&
              end % 8 == 0 && off_g % 8 == 0 && off_g >= 0 &&
              gate.size(1) % 8 == 0 && off_g + n <= gate.size(1) &&
              vdim >= 1 && vdim <= vc && y.size(1) % 8 == 0,
              "delta_out: layout");
  TORCH_CHECK(positions.scalar_type() == at::kInt &&
              positions.is_contiguous() && positions.numel() == T &&
              cu_q.scalar_type() == at::kInt && cu_q.is_contiguous() &&
              slots.scalar_type() == at::kInt && slots.is_contiguous() &&
              n_seqs >= 0 && cu_q.numel() > n_seqs && slots.numel() >= n_seqs,
              "delta_out: batch tensors");
  if (tails.has_value())
    TORCH_CHECK(tails->dim() == 3 && tails->is_contiguous() &&
                tails->scalar_type() == dt && tails->size(2) <= y.size(1) &&
                tails->size(2) % 8 == 0, "delta_out: tails");
  const bool bf16 = dt == at::kBFloat16;
  TORCH_CHECK(bf16 || dt == at::kFloat, "delta_out: dtype");
  if (swz.has_value())
    TORCH_CHECK(bf16 && T <= 32 && swz->is_contiguous() &&
                swz->scalar_type() == dt && nz % 16 == 0 &&
                swz->numel() == nz * 32, "delta_out: operand");
  if (T == 0) return;
  OutArgs a{};
  a.o = o.data_ptr<float>();
  a.w = w.data_ptr<float>();
  a.tokens = T;
  a.ny2 = gate.size(1);
  a.ny = y.size(1);
  a.nz = nz;
  a.heads = (int)heads;
  a.w_head = w.numel() == n ? (int)vc : 0;
  a.end = (int)end;
  a.vc = (int)vc;
  a.vdim = (int)vdim;
  a.off_g = (int)off_g;
  a.eps = (float)eps;
  a.y2 = gate.data_ptr();
  a.y = y.data_ptr();
  a.z = z.data_ptr();
  a.swz = swz ? swz->data_ptr() : nullptr;
  a.positions = positions.data_ptr<int>();
  a.cu_q = cu_q.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.tail_blocks = 0;
  if (tails.has_value()) {
    a.tails = tails->data_ptr();
    a.taps = (int)tails->size(1) + 1;
    a.channels = (int)tails->size(2);
    a.tail_blocks = (a.channels + BLOCK * 8 - 1) / (BLOCK * 8);
  }
  auto stream = at::hip::getCurrentHIPStream();
  auto launch = [&](auto tag, auto l, auto v) {
    using E = decltype(tag);
    hipLaunchKernelGGL(
        (delta_out_kernel<E, decltype(l)::value, decltype(v)::value>),
        dim3(T + n_seqs * a.tail_blocks), dim3(BLOCK), 0, stream, a);
  };
  constexpr std::integral_constant<int, 1> one{};
  auto pick = [&](auto tag) {
    if (vc <= 64) launch(tag, std::integral_constant<int, 8>{}, one);
    else if (vc <= 128) launch(tag, std::integral_constant<int, 16>{}, one);
    else if (vc <= 256) launch(tag, std::integral_constant<int, 32>{}, one);
    else launch(tag, std::integral_constant<int, 64>{},
                std::integral_constant<int, 2>{});
  };
  if (bf16) pick(uint16_t{});
  else pick(float{});
}
