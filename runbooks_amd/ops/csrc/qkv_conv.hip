// Queries, keys and values that pass a bias and a short causal convolution
// (gfx950): y's first columns [ q heads | k heads | v heads ] -> q, and rows
// [ keys | value ] of the paged cache (shared_kv.h). A sequence's slot keeps
// its last taps - 1 projections, without the bias; before a sequence's start
// there is neither.
//
// With single tokens a thread also moves its columns of the slot; after
// portions qkv_tails does.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "history.h"
#include "shared_kv.h"

namespace {

using rb::Ragged;

constexpr int BLOCK = 256;
constexpr int VECS = 32;               // column groups per workgroup
constexpr int MAX_TPT = 4;             // tokens per thread

struct Args {
  const void *y;
  int64_t ny, T;
  const float *bias, *conv;            // [n], [taps, n]
  void *tails;                         // [slots, taps - 1, n]
  Ragged b;
  const int *cache_slots;
  void *cache, *q;
  int n, off_k, off_v, kv, kc, vc;     // kc: keys of one kv head
};

template <typename T>
RB_DEV void put(const Args &a, int64_t t, int c, const float *f) {
  if (c < a.off_k) {
    rb::store_v<8>((T *)a.q + t * a.off_k + c, f);
    return;
  }
  const int slot = a.cache_slots[t], ec = a.kc + a.vc;
  const bool is_v = c >= a.off_v;
  const int i = c - (is_v ? a.off_v : a.off_k), size = is_v ? a.vc : a.kc;
  const int g = i / size, col = i - g * size + (is_v ? a.kc : 0);
  T *row = (T *)a.cache +
           (((int64_t)(slot / skv::PAGE) * a.kv + g) * skv::PAGE +
            slot % skv::PAGE) * ec;
  rb::store_v<8>(row + col, f);
}

template <typename T, int TPT, bool SINGLE>
__global__ __launch_bounds__(BLOCK) void qkv_conv_kernel(Args a) {
  const int c = (blockIdx.x * VECS + threadIdx.x % VECS) * 8;
  const int t0 = (blockIdx.y * (BLOCK / VECS) + threadIdx.x / VECS) * TPT;
  if (c >= a.n || t0 >= a.T) return;
  const int taps = a.b.taps;
  rb::Source src[TPT];
#pragma unroll
  for (int i = 0; i < TPT; ++i)
    src[i] = rb::source_of(a.b, min(t0 + i, (int)a.T - 1));
  float bias[8], out[TPT][8] = {};
  rb::load_v<8>(a.bias + c, bias);
  for (int j = 0; j < taps; ++j) {
    float w[8];
    rb::load_v<8>(a.conv + (int64_t)j * a.n + c, w);
#pragma unroll
    for (int i = 0; i < TPT; ++i) {
      const int t = min(t0 + i, (int)a.T - 1), at = src[i].at(t, j, taps);
      T *tail = (T *)a.tails + (int64_t)src[i].slot * (taps - 1) * a.n + c;
      float v[8] = {};
      const bool some = at != (int)0x80000000;
      if (some)
        rb::load_v<8>(at >= 0 ? (const T *)a.y + at * a.ny + c
                              : tail + (int64_t)~at * a.n, v);
      if (SINGLE && j > 0) rb::store_v<8>(tail + (int64_t)(j - 1) * a.n, v);
      if (some) {
#pragma unroll
        for (int k = 0; k < 8; ++k) out[i][k] += w[k] * (v[k] + bias[k]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < TPT; ++i)
    if (t0 + i < a.T) put<T>(a, t0 + i, c, out[i]);
}

template <typename T>
__global__ __launch_bounds__(BLOCK) void qkv_tails_kernel(Args a) {
  const int seq = blockIdx.y, keep = a.b.taps - 1;
  const int c = (blockIdx.x * BLOCK + threadIdx.x) * 8;
  const int first = a.b.cu_q[seq], end = a.b.cu_q[seq + 1];
  if (c >= a.n || end <= first) return;
  const rb::Source src{first, a.b.positions[first], a.b.slots[seq]};
  T *tail = (T *)a.tails + (int64_t)src.slot * keep * a.n + c;
  for (int j = 0; j < keep; ++j) {
    // the input that a token after the last one would read at tap j
    const int at = src.at(end, j, a.b.taps);
    float v[8] = {};
    if (at != (int)0x80000000)
      rb::load_v<8>(at >= 0 ? (const T *)a.y + at * a.ny + c
                            : tail + (int64_t)~at * a.n, v);
    rb::store_v<8>(tail + (int64_t)j * a.n, v);
  }
}

}  // namespace

void qkv_conv(at::Tensor y, at::Tensor bias, at::Tensor conv, at::Tensor tails,
              at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
              at::Tensor seq_of, at::Tensor cache_slots, bool single,
              int64_t n_seqs, at::Tensor cache, int64_t kc, at::Tensor q) {
  const auto dt = y.scalar_type();
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (dt == at::kBFloat16 || dt == at::kFloat) && y.size(1) % 8 == 0,
              "qkv_conv: y");
  const int64_t T = y.size(0), n = bias.numel();
  TORCH_CHECK(cache.is_cuda() && cache.dim() == 4 &&
              cache.size(2) == skv::PAGE && cache.is_contiguous() &&
              cache.scalar_type() == dt,
              "qkv_conv: cache [blocks, kv heads, 16, ec]");
  const int64_t G = cache.size(1), vc = cache.size(3) - kc;
  TORCH_CHECK(q.dim() == 2 && q.is_contiguous() && q.scalar_type() == dt &&
              q.size(0) == T, "qkv_conv: q");
  const int64_t off_k = q.size(1), off_v = off_k + G * kc;
  TORCH_CHECK(kc >= 8 && kc % 8 == 0 && vc >= 8 && vc % 8 == 0 &&
              off_k % 8 == 0 && n == off_v + G * vc && n <= y.size(1),
              "qkv_conv: layout");
  TORCH_CHECK(bias.scalar_type() == at::kFloat && bias.is_contiguous() &&
              conv.dim() == 2 && conv.scalar_type() == at::kFloat &&
              conv.is_contiguous() && conv.size(0) >= 1 && conv.size(1) == n &&
              tails.dim() == 3 && tails.is_contiguous() &&
              tails.scalar_type() == dt && tails.size(1) == conv.size(0) - 1 &&
              tails.size(2) == n, "qkv_conv: bias, taps, tails");
  auto ints = [](const at::Tensor &t, int64_t m) {
    return t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() &&
           t.numel() >= m;
  };
  TORCH_CHECK(ints(positions, T) && ints(cu_q, n_seqs + 1) &&
              ints(slots, n_seqs) && ints(seq_of, T) && ints(cache_slots, T) &&
              n_seqs <= 65535 && (!single || T == n_seqs),
              "qkv_conv: batch tensors");
  if (T == 0) return;
  Args a{};
  a.y = y.data_ptr();
  a.ny = y.size(1);
  a.T = T;
  a.bias = bias.data_ptr<float>();
  a.conv = conv.data_ptr<float>();
  a.tails = tails.data_ptr();
  a.b = Ragged{positions.data_ptr<int>(), cu_q.data_ptr<int>(),
               slots.data_ptr<int>(), seq_of.data_ptr<int>(),
               (int)conv.size(0)};
  a.cache_slots = cache_slots.data_ptr<int>();
  a.cache = cache.data_ptr();
  a.q = q.data_ptr();
  a.n = (int)n;
  a.off_k = (int)off_k;
  a.off_v = (int)off_v;
  a.kv = (int)G;
  a.kc = (int)kc;
  a.vc = (int)vc;
  auto stream = at::hip::getCurrentHIPStream();
  auto pick = [&](auto tag) {
    using E = decltype(tag);
    const int groups = (int)((n / 8 + VECS - 1) / VECS);
    auto tiles = [&](int tpt) {
      const int64_t per = BLOCK / VECS * tpt, m = (T + per - 1) / per;
      TORCH_CHECK(m <= 65535, "qkv_conv: ", T, " tokens");
      return dim3(groups, m);
    };
    if (single) {
      hipLaunchKernelGGL((qkv_conv_kernel<E, 1, true>), tiles(1), dim3(BLOCK),
                         0, stream, a);
      return;
    }
    hipLaunchKernelGGL((qkv_conv_kernel<E, MAX_TPT, false>), tiles(MAX_TPT),
                       dim3(BLOCK), 0, stream, a);
    if (a.b.taps > 1)
      hipLaunchKernelGGL((qkv_tails_kernel<E>),
                         dim3((n / 8 + BLOCK - 1) / BLOCK, n_seqs),
                         dim3(BLOCK), 0, stream, a);
  };
  if (dt == at::kBFloat16) pick(uint16_t{});
  else pick(float{});
}
