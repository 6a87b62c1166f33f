// Queries, keys and values that pass a bias and a short causal convolution
// (gfx950): y's first columns [ q heads | k heads | v heads ] -> q, and rows
// [ keys | value ] of the paged cache (shared_kv.h). A sequence's slot keeps
// its last taps - 1 projections, without the bias; before a sequence's start
// there is neither.
//
// With single tokens a thread also moves its columns of the slot; after
// portions qkv_tails does. With 2 to 4 taps a thread inside a portion reads
// every row once.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "history.h"
#include "shared_kv.h"

namespace {

using rb::Ragged;

constexpr int BLOCK = 256;
constexpr int VECS = 32;               // column groups per workgroup
constexpr int MAX_TPT = 4;             // tokens per thread
constexpr int MAX_TAPS = 4;            // taps that kernels are made for

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

template <typename T, int TPT, int TAPS, bool SINGLE>
__global__ __launch_bounds__(BLOCK) void qkv_conv_kernel(Args a) {
  const int c = (blockIdx.x * VECS + threadIdx.x % VECS) * 8;
  const int t0 = (blockIdx.y * (BLOCK / VECS) + threadIdx.x / VECS) * TPT;
  if (c >= a.n || t0 >= a.T) return;
  float bias[8];
  rb::load_v<8>(a.bias + c, bias);
  if constexpr (TAPS > 1 && !SINGLE) {
    const int end = t0 + TPT - 1;
    if (end < a.T && a.b.seq_of[end] == a.b.seq_of[t0] &&
        t0 - (TAPS - 1) >= a.b.cu_q[a.b.seq_of[t0]]) {
      // the rows of this thread and those before them are one portion's
      float u[TPT + TAPS - 1][8], w[TAPS][8];
#pragma unroll
      for (int i = 0; i < TPT + TAPS - 1; ++i)
        rb::load_v<8>((const T *)a.y + (t0 - (TAPS - 1) + i) * a.ny + c, u[i]);
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
        rb::load_v<8>(a.conv + (int64_t)j * a.n + c, w[j]);
#pragma unroll
      for (int i = 0; i < TPT + TAPS - 1; ++i)
#pragma unroll
        for (int k = 0; k < 8; ++k) u[i][k] += bias[k];
#pragma unroll
      for (int i = 0; i < TPT; ++i) {
        float out[8] = {};
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
#pragma unroll
          for (int k = 0; k < 8; ++k) out[k] += w[j][k] * u[i + j][k];
        put<T>(a, t0 + i, c, out);
      }
      return;
    }
  }
  const int taps = a.b.taps;
  for (int t = t0; t < min(t0 + TPT, (int)a.T); ++t) {
    const rb::Source src = rb::source_of(a.b, t);
    T *tail = (T *)a.tails + (int64_t)src.slot * (taps - 1) * a.n + c;
    float out[8] = {};
    for (int j = 0; j < taps; ++j) {
      const int at = src.at(t, j, taps);
      float v[8] = {};
      const bool some = at != (int)0x80000000;
      if (some)
        rb::load_v<8>(at >= 0 ? (const T *)a.y + at * a.ny + c
                              : tail + (int64_t)~at * a.n, v);
      if (SINGLE && j > 0) rb::store_v<8>(tail + (int64_t)(j - 1) * a.n, v);
      if (!some) continue;
      float w[8];
      rb::load_v<8>(a.conv + (int64_t)j * a.n + c, w);
#pragma unroll
      for (int k = 0; k < 8; ++k) out[k] += w[k] * (v[k] + bias[k]);
    }
    put<T>(a, t, c, out);
  }
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
      hipLaunchKernelGGL((qkv_conv_kernel<E, 1, 0, true>), tiles(1),
                         dim3(BLOCK), 0, stream, a);
      return;
    }
    auto go = [&](auto n) {
      hipLaunchKernelGGL(
          (qkv_conv_kernel<E, MAX_TPT, decltype(n)::value, false>),
          tiles(MAX_TPT), dim3(BLOCK), 0, stream, a);
    };
    if (a.b.taps == 2) go(std::integral_constant<int, 2>{});
    else if (a.b.taps == 3) go(std::integral_constant<int, 3>{});
    else if (a.b.taps == 4) go(std::integral_constant<int, MAX_TAPS>{});
    else go(std::integral_constant<int, 0>{});
    if (a.b.taps > 1)
      hipLaunchKernelGGL((qkv_tails_kernel<E>),
                         dim3((n / 8 + BLOCK - 1) / BLOCK, n_seqs),
                         dim3(BLOCK), 0, stream, a);
  };
  if (dt == at::kBFloat16) pick(uint16_t{});
  else pick(float{});
}
