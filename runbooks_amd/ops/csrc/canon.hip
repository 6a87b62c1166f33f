// RMS norm of a 32-bit residual and causal convolutions behind it (gfx950):
//
//   x += pending,  n_t = x_t / rms(x_t),  h_t = sum_j f_j n_(t - taps + 1 + j)
//
// for up to MAX_SUBS sublayers with coefficients f [sublayer][tap][column]
// (norm weight, convolution and the direct path in one). A sequence's slot
// keeps its last taps - 1 rows of n.
//
//  * canon_token: batches of single tokens, a workgroup per token (with up to
//    MAX_TAPS taps and one column group per thread everything is on its way
//    before the reduction)
//  * canon_rows, canon_conv, canon_tails: portions; the rows' factors first,
//    then the convolution (with up to MAX_TAPS taps a thread inside a portion
//    reads every row once), then the slots, which canon_conv has read

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "history.h"

namespace {

using rb::Ragged;

constexpr int BLOCK = 256;
constexpr int MAX_SUBS = 2;
constexpr int MAX_TAPS = 4;            // taps that kernels are made for
constexpr int TPT = 4;                 // tokens per thread
constexpr int VECS = 64;               // column groups per workgroup
constexpr int TILE = BLOCK / VECS * TPT;   // tokens per workgroup

struct Args {
  float *x;                            // [T, D]
  const void *delta;                   // [nd, T, D] or null
  const float *coef;                   // [subs, taps, D]
  float *tails;                        // [slots, taps - 1, D]
  float *inv;                          // [T], portions
  void *h[MAX_SUBS];                   // [T, width]
  void *swz[MAX_SUBS];
  Ragged b;
  int64_t T;
  int nd, subs, D, width, n_seqs;
  float eps;
};

// x += pending of V columns at c of row t; returns them in f
template <typename DT, int V>
RB_DEV void add_pending(const Args &a, int64_t t, int c, float *f) {
  float *xr = a.x + t * a.D + c;
  rb::load_v<V>(xr, f);
  for (int s = 0; s < a.nd; ++s) {
    float d[V];
    rb::load_v<V>((const DT *)a.delta + ((int64_t)s * a.T + t) * a.D + c, d);
#pragma unroll
    for (int k = 0; k < V; ++k) f[k] += d[k];
  }
  if (a.nd > 0) rb::store_v<V>(xr, f);
}

// writes V columns of a sublayer's input
template <typename T, int V>
RB_DEV void put(const Args &a, int i, int64_t t, int c, const float *f) {
  rb::store_v<V>((T *)a.h[i] + t * a.width + c, f);
  if (a.swz[i] != nullptr)
    rb::store_v<V>((T *)a.swz[i] + rb::operand_slot(c, (int)t), f);
}

// columns beyond D
template <typename T> RB_DEV void clear_padding(const Args &a, int64_t t) {
  const float zero[1] = {0.0f};
  for (int c = a.D + threadIdx.x; c < a.width; c += blockDim.x)
    for (int i = 0; i < a.subs; ++i) put<T, 1>(a, i, t, c, zero);
}

template <typename T, typename DT, int V>
__global__ __launch_bounds__(BLOCK) void canon_token_kernel(Args a) {
  __shared__ float red[BLOCK / RB_WAVE];
  const int64_t t = blockIdx.x;
  const int taps = a.b.taps, pos = a.b.positions[t];
  float *tail = a.tails + (int64_t)a.b.slots[t] * (taps - 1) * a.D;
  const int nvec = a.D / V;
  float ss = 0.0f;
  for (int i = threadIdx.x; i < nvec; i += BLOCK) {
    float f[V];
    add_pending<DT, V>(a, t, i * V, f);
#pragma unroll
    for (int k = 0; k < V; ++k) ss += f[k] * f[k];
  }
  ss = rb::block_reduce_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)a.D + a.eps);
  for (int i = threadIdx.x; i < nvec; i += BLOCK) {
    const int c = i * V;
    float n[V], out[MAX_SUBS][V] = {};
    rb::load_v<V>(a.x + t * a.D + c, n);       // this thread's own values
#pragma unroll
    for (int k = 0; k < V; ++k) n[k] *= inv;
    for (int j = 0; j < taps; ++j) {
      float v[V] = {};
      if (j == taps - 1) {
#pragma unroll
        for (int k = 0; k < V; ++k) v[k] = n[k];
      } else if (pos >= taps - 1 - j) {
        rb::load_v<V>(tail + (int64_t)j * a.D + c, v);
      }
      // every row moves up one place: this thread alone has these columns
      if (j > 0) rb::store_v<V>(tail + (int64_t)(j - 1) * a.D + c, v);
#pragma unroll
      for (int s = 0; s < MAX_SUBS; ++s) {
        if (s >= a.subs) break;
        float f[V];
        rb::load_v<V>(a.coef + ((int64_t)s * taps + j) * a.D + c, f);
#pragma unroll
        for (int k = 0; k < V; ++k) out[s][k] += f[k] * v[k];
      }
    }
#pragma unroll
    for (int s = 0; s < MAX_SUBS; ++s)
      if (s < a.subs) put<T, V>(a, s, t, c, out[s]);
  }
  clear_padding<T>(a, t);
}

// the same with one column group per thread
template <typename T, typename DT, int TAPS, int BLK>
__global__ __launch_bounds__(BLK) void canon_token_wide_kernel(Args a) {
  __shared__ float red[BLK / RB_WAVE];
  const int64_t t = blockIdx.x;
  const int c = threadIdx.x * 8, pos = a.b.positions[t];
  const bool ok = c < a.D;
  const int cc = ok ? c : 0;
  float *tail = a.tails + (int64_t)a.b.slots[t] * (TAPS - 1) * a.D + cc;
  float n[TAPS][8], f[MAX_SUBS][TAPS][8], ss = 0.0f;
#pragma unroll
  for (int j = 0; j < TAPS - 1; ++j)
    rb::load_v<8>(tail + (int64_t)j * a.D, n[j]);
#pragma unroll
  for (int s = 0; s < MAX_SUBS; ++s)
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
      rb::load_v<8>(a.coef + ((int64_t)min(s, a.subs - 1) * TAPS + j) * a.D +
                        cc, f[s][j]);
  if (ok) {
    add_pending<DT, 8>(a, t, c, n[TAPS - 1]);
#pragma unroll
    for (int k = 0; k < 8; ++k) ss += n[TAPS - 1][k] * n[TAPS - 1][k];
  }
  ss = rb::block_reduce_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)a.D + a.eps);
  if (ok) {
    float out[MAX_SUBS][8] = {};
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      const bool real = pos >= TAPS - 1 - j;
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        n[j][k] = j == TAPS - 1 ? n[j][k] * inv : real ? n[j][k] : 0.0f;
#pragma unroll
        for (int s = 0; s < MAX_SUBS; ++s) out[s][k] += f[s][j][k] * n[j][k];
      }
      if (j > 0) rb::store_v<8>(tail + (int64_t)(j - 1) * a.D, n[j]);
    }
#pragma unroll
    for (int s = 0; s < MAX_SUBS; ++s)
      if (s < a.subs) put<T, 8>(a, s, t, c, out[s]);
  }
  clear_padding<T>(a, t);
}

template <typename T, typename DT, int V>
__global__ __launch_bounds__(BLOCK) void canon_rows_kernel(Args a) {
  __shared__ float red[BLOCK / RB_WAVE];
  const int64_t t = blockIdx.x;
  float ss = 0.0f;
#pragma unroll 2
  for (int i = threadIdx.x; i < a.D / V; i += BLOCK) {
    float f[V];
    add_pending<DT, V>(a, t, i * V, f);
#pragma unroll
    for (int k = 0; k < V; ++k) ss += f[k] * f[k];
  }
  ss = rb::block_reduce_sum(ss, red);
  if (threadIdx.x == 0) a.inv[t] = 1.0f / sqrtf(ss / (float)a.D + a.eps);
  clear_padding<T>(a, t);
}

template <typename T, int V, int TAPS>
__global__ __launch_bounds__(BLOCK) void canon_conv_kernel(Args a) {
  const int c = (blockIdx.x * VECS + threadIdx.x % VECS) * V;
  const int t0 = blockIdx.y * TILE + threadIdx.x / VECS * TPT;
  if (c >= a.D || t0 >= a.T) return;
  if constexpr (TAPS > 1) {
    const int end = t0 + TPT - 1;
    if (end < a.T && a.b.seq_of[end] == a.b.seq_of[t0] &&
        t0 - (TAPS - 1) >= a.b.cu_q[a.b.seq_of[t0]]) {
      // the rows of this thread and those before them are one portion's
      float n[TPT + TAPS - 1][V], f[MAX_SUBS][TAPS][V];
#pragma unroll
      for (int i = 0; i < TPT + TAPS - 1; ++i)
        rb::load_v<V>(a.x + (int64_t)(t0 - (TAPS - 1) + i) * a.D + c, n[i]);
#pragma unroll
      for (int s = 0; s < MAX_SUBS; ++s)
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
          rb::load_v<V>(a.coef + ((int64_t)min(s, a.subs - 1) * TAPS + j) *
                            a.D + c, f[s][j]);
#pragma unroll
      for (int i = 0; i < TPT + TAPS - 1; ++i) {
        const float m = a.inv[t0 - (TAPS - 1) + i];
#pragma unroll
        for (int k = 0; k < V; ++k) n[i][k] *= m;
      }
#pragma unroll
      for (int i = 0; i < TPT; ++i)
#pragma unroll
        for (int s = 0; s < MAX_SUBS; ++s) {
          float out[V] = {};
#pragma unroll
          for (int j = 0; j < TAPS; ++j)
#pragma unroll
            for (int k = 0; k < V; ++k) out[k] += f[s][j][k] * n[i + j][k];
          if (s < a.subs) put<T, V>(a, s, t0 + i, c, out);
        }
      return;
    }
  }
  const int taps = a.b.taps;
  for (int t = t0; t < min(t0 + TPT, (int)a.T); ++t) {
    const rb::Source src = rb::source_of(a.b, t);
    float out[MAX_SUBS][V] = {};
    for (int j = 0; j < taps; ++j) {
      const int at = src.at(t, j, taps);
      if (at == (int)0x80000000) continue;
      const float m = at >= 0 ? a.inv[at] : 1.0f;
      float v[V];
      rb::load_v<V>((at >= 0 ? a.x + (int64_t)at * a.D
                             : a.tails + ((int64_t)src.slot * (taps - 1) +
                                          ~at) * a.D) + c, v);
#pragma unroll
      for (int s = 0; s < MAX_SUBS; ++s) {
        if (s >= a.subs) break;
        float f[V];
        rb::load_v<V>(a.coef + ((int64_t)s * taps + j) * a.D + c, f);
#pragma unroll
        for (int k = 0; k < V; ++k) out[s][k] += f[k] * (v[k] * m);
      }
    }
#pragma unroll
    for (int s = 0; s < MAX_SUBS; ++s)
      if (s < a.subs) put<T, V>(a, s, t, c, out[s]);
  }
}

// A thread owns V columns of a sequence's slot: rows that stay move up before
// they are overwritten.
template <int V>
__global__ __launch_bounds__(BLOCK) void canon_tails_kernel(Args a) {
  const int seq = blockIdx.y, keep = a.b.taps - 1;
  const int c = (blockIdx.x * BLOCK + threadIdx.x) * V;
  const int first = a.b.cu_q[seq], end = a.b.cu_q[seq + 1];
  if (c >= a.D || end <= first) return;
  const rb::Source src{first, a.b.positions[first], a.b.slots[seq]};
  float *tail = a.tails + (int64_t)src.slot * keep * a.D + c;
  for (int j = 0; j < keep; ++j) {
    // the input that a token after the last one would read at tap j
    const int at = src.at(end, j, a.b.taps);
    float v[V] = {};
    if (at >= 0) {
      rb::load_v<V>(a.x + (int64_t)at * a.D + c, v);
#pragma unroll
      for (int k = 0; k < V; ++k) v[k] *= a.inv[at];
    } else if (at != (int)0x80000000) {
      rb::load_v<V>(tail + (int64_t)~at * a.D, v);
    }
    rb::store_v<V>(tail + (int64_t)j * a.D, v);
  }
}

}  // namespace

// x [T, D] f32 += delta; out: the sublayers' inputs [T, width]; operands: one
// for every set entry of `wants`
void canon_norm(at::Tensor x, c10::optional<at::Tensor> delta, at::Tensor coef,
                at::Tensor tails, at::Tensor positions, at::Tensor cu_q,
                at::Tensor slots, at::Tensor seq_of, bool single,
                int64_t n_seqs, double eps, std::vector<at::Tensor> out,
                std::vector<at::Tensor> operands, std::vector<bool> wants) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() &&
              x.scalar_type() == at::kFloat, "canon_norm: x [T, D] f32");
  const int64_t T = x.size(0), D = x.size(1);
  const int64_t subs = (int64_t)out.size();
  TORCH_CHECK(subs >= 1 && subs <= MAX_SUBS && (int64_t)wants.size() == subs &&
              coef.dim() == 3 && coef.is_contiguous() &&
              coef.scalar_type() == at::kFloat && coef.size(0) == subs &&
              coef.size(1) >= 1 && coef.size(2) == D && tails.dim() == 3 &&
              tails.is_contiguous() && tails.scalar_type() == at::kFloat &&
              tails.size(1) == coef.size(1) - 1 && tails.size(2) == D,
              "canon_norm: coefficients, tails");
  auto ints = [](const at::Tensor &t, int64_t n) {
    return t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() &&
           t.numel() >= n;
  };
  TORCH_CHECK(ints(positions, T) && ints(cu_q, n_seqs + 1) &&
              ints(slots, n_seqs) && ints(seq_of, T) && n_seqs <= 65535 &&
              (!single || T == n_seqs), "canon_norm: batch tensors");
  const auto dt = out[0].scalar_type();
  const bool bf16 = dt == at::kBFloat16;
  TORCH_CHECK(bf16 || dt == at::kFloat, "canon_norm: dtype");
  Args a{};
  size_t next = 0;
  for (int64_t i = 0; i < subs; ++i) {
    const at::Tensor &h = out[i];
    TORCH_CHECK(h.is_cuda() && h.is_contiguous() && h.dim() == 2 &&
                h.size(0) == T && h.size(1) == out[0].size(1) &&
                h.size(1) >= D && h.size(1) % 32 == 0 &&
                h.scalar_type() == dt, "canon_norm: out");
    a.h[i] = h.data_ptr();
    if (!wants[i]) continue;
    TORCH_CHECK(next < operands.size(), "canon_norm: operands");
    const at::Tensor &s = operands[next++];
    TORCH_CHECK(bf16 && T <= 32 && s.is_contiguous() &&
                s.scalar_type() == dt && s.numel() == h.size(1) * 32,
                "canon_norm: operand");
    a.swz[i] = s.data_ptr();
  }
  bool d16 = false;
  if (delta.has_value()) {
    const at::Tensor &d = *delta;
    TORCH_CHECK(d.is_cuda() && d.is_contiguous() && d.size(-1) == D &&
                d.size(-2) == T && (d.dim() == 2 || d.dim() == 3),
                "canon_norm: delta shape");
    d16 = d.scalar_type() == at::kBFloat16;
    TORCH_CHECK(d16 || d.scalar_type() == at::kFloat, "canon_norm: delta");
    a.nd = d.dim() == 3 ? (int)d.size(0) : 1;
    a.delta = d.data_ptr();
  }
  if (T == 0) return;
  a.x = x.data_ptr<float>();
  a.coef = coef.data_ptr<float>();
  a.tails = tails.data_ptr<float>();
  a.b = Ragged{positions.data_ptr<int>(), cu_q.data_ptr<int>(),
               slots.data_ptr<int>(), seq_of.data_ptr<int>(),
               (int)coef.size(1)};
  a.T = T;
  a.subs = (int)subs;
  a.D = (int)D;
  a.width = (int)out[0].size(1);
  a.n_seqs = (int)n_seqs;
  a.eps = (float)eps;
  at::Tensor inv;
  if (!single) {
    inv = at::empty({T}, x.options());
    a.inv = inv.data_ptr<float>();
  }
  auto stream = at::hip::getCurrentHIPStream();
  auto with_taps = [&](auto f) {
    if (a.b.taps == 2) f(std::integral_constant<int, 2>{});
    else if (a.b.taps == 3) f(std::integral_constant<int, 3>{});
    else f(std::integral_constant<int, MAX_TAPS>{});
  };
  const bool made = D % 8 == 0 && a.b.taps >= 2 && a.b.taps <= MAX_TAPS;
  auto go = [&](auto tag, auto dtag, auto v) {
    using E = decltype(tag);
    using DT = decltype(dtag);
    constexpr int V = decltype(v)::value;
    if (single && made && D <= 8192) {
      with_taps([&](auto n) {
        constexpr int N = decltype(n)::value;
        if (D <= 2048)
          hipLaunchKernelGGL((canon_token_wide_kernel<E, DT, N, 256>), dim3(T),
                             dim3(256), 0, stream, a);
        else if (D <= 4096)
          hipLaunchKernelGGL((canon_token_wide_kernel<E, DT, N, 512>), dim3(T),
                             dim3(512), 0, stream, a);
        else
          hipLaunchKernelGGL((canon_token_wide_kernel<E, DT, N, 1024>),
                             dim3(T), dim3(1024), 0, stream, a);
      });
      return;
    }
    if (single) {
      hipLaunchKernelGGL((canon_token_kernel<E, DT, V>), dim3(T), dim3(BLOCK),
                         0, stream, a);
      return;
    }
    hipLaunchKernelGGL((canon_rows_kernel<E, DT, V>), dim3(T), dim3(BLOCK), 0,
                       stream, a);
    const int64_t tiles = (T + TILE - 1) / TILE;
    TORCH_CHECK(tiles <= 65535, "canon_norm: ", T, " tokens");
    const dim3 grid((D / V + VECS - 1) / VECS, tiles);
    if constexpr (V == 8) {
      if (made)
        with_taps([&](auto n) {
          hipLaunchKernelGGL((canon_conv_kernel<E, 8, decltype(n)::value>),
                             grid, dim3(BLOCK), 0, stream, a);
        });
    }
    if (!made)
      hipLaunchKernelGGL((canon_conv_kernel<E, V, 0>), grid, dim3(BLOCK), 0,
                         stream, a);
    if (a.b.taps > 1)
      hipLaunchKernelGGL((canon_tails_kernel<V>),
                         dim3((D / V + BLOCK - 1) / BLOCK, n_seqs),
                         dim3(BLOCK), 0, stream, a);
  };
  auto pick = [&](auto tag, auto dtag) {
    if (D % 8 == 0) go(tag, dtag, std::integral_constant<int, 8>{});
    else go(tag, dtag, std::integral_constant<int, 1>{});
  };
  if (bf16 && d16) pick(uint16_t{}, uint16_t{});
  else if (bf16) pick(uint16_t{}, float{});
  else if (d16) pick(float{}, uint16_t{});
  else pick(float{}, float{});
}
