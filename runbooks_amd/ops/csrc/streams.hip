// Residual streams with learned mixing, dynamic-tanh norm, squared ReLU
// (gfx950).
//
//   X_t <- sum_f mix[f, t] X_f + out[t] scale sigmoid(gate + b) y   (pending)
//   u = sum_s in[s] X_s,   h = tanh(alpha u) w + bias
//
// X [T, streams, D] fp32 is read and written once: the pending result, the
// next sublayer's input and its norm are one pass.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 256;
constexpr int MAX_STREAMS = 16;

struct Args {
  float *x;                            // [T, s, D]
  const float *delta, *extra;          // parts [n, T, D], or null
  int n_delta, n_extra;
  const void *y;                       // [T, ny]: gate logits from `off`
  int64_t ny;
  int off;
  const float *join;                   // scale, gate bias, out, mix; or null
  const float *inp;                    // [s]
  const float *norm;                   // weight, bias, alpha
  int64_t T;
  int s, D, Dp;
  void *h;                             // [T, Dp]
  void *swz;                           // decode operand, or null
};

// V columns of one token per thread; V = 4 needs D % 4 == 0
template <typename T, int S, int V>
__global__ __launch_bounds__(BLOCK) void streams_norm_kernel(Args a) {
  __shared__ float mix_s[S * S + 2 * S];     // mix [from][to], out, in
  for (int i = threadIdx.x; i < S * S; i += BLOCK) {
    const int f = i / S, t = i % S;
    mix_s[i] = a.join != nullptr && f < a.s && t < a.s
                   ? a.join[2 * a.D + a.s + f * a.s + t] : 0.0f;
  }
  if (threadIdx.x < S) {
    const bool ok = threadIdx.x < a.s;
    mix_s[S * S + threadIdx.x] =
        ok && a.join != nullptr ? a.join[2 * a.D + threadIdx.x] : 0.0f;
    mix_s[S * S + S + threadIdx.x] = ok ? a.inp[threadIdx.x] : 0.0f;
  }
  __syncthreads();
  const float *out_s = mix_s + S * S, *in_s = out_s + S;
  const float alpha = a.norm[2 * a.D];
  const int per_row = a.Dp / V;
  const int64_t total = a.T * per_row, part = a.T * a.D;
  auto load = [](const float *p, float *f) {
    if constexpr (V == 4) rb::VIO<float>::load(p, f);
    else f[0] = p[0];
  };
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < total;
       i += (int64_t)gridDim.x * BLOCK) {
    const int64_t t = i / per_row;
    const int c = (int)(i - t * per_row) * V;
    float r[V];
#pragma unroll
    for (int k = 0; k < V; ++k) r[k] = 0.0f;
    if (c < a.D) {
      float *xp = a.x + t * a.s * a.D + c;
      float x[S][V], u[V];
#pragma unroll
      for (int f = 0; f < S; ++f)
        if (f < a.s) {
          load(xp + (int64_t)f * a.D, x[f]);
        } else {
#pragma unroll
          for (int k = 0; k < V; ++k) x[f][k] = 0.0f;
        }
#pragma unroll
      for (int k = 0; k < V; ++k) u[k] = 0.0f;
      if (a.join != nullptr) {
        float y[V], sc[V], b[V];
        const int64_t at = t * a.D + c;
        load(a.delta + at, y);
        for (int n = 1; n < a.n_delta; ++n) {
          float p[V];
          load(a.delta + n * part + at, p);
#pragma unroll
          for (int k = 0; k < V; ++k) y[k] += p[k];
        }
        for (int n = 0; n < a.n_extra; ++n) {
          float p[V];
          load(a.extra + n * part + at, p);
#pragma unroll
          for (int k = 0; k < V; ++k) y[k] += p[k];
        }
        load(a.join + c, sc);
        load(a.join + a.D + c, b);
        const T *gp = (const T *)a.y + t * a.ny + a.off + c;
#pragma unroll
        for (int k = 0; k < V; ++k)
          y[k] *= sc[k] /
                  (1.0f + expf(-(rb::bf16_to_f32_or_id(gp[k]) + b[k])));
#pragma unroll
        for (int to = 0; to < S; ++to)
          if (to < a.s) {
            float n[V];
#pragma unroll
            for (int k = 0; k < V; ++k) n[k] = out_s[to] * y[k];
#pragma unroll
            for (int f = 0; f < S; ++f)
#pragma unroll
              for (int k = 0; k < V; ++k) n[k] += mix_s[f * S + to] * x[f][k];
#pragma unroll
            for (int k = 0; k < V; ++k) u[k] += in_s[to] * n[k];
            if constexpr (V == 4)
              rb::VIO<float>::store(xp + (int64_t)to * a.D, n);
            else
              xp[(int64_t)to * a.D] = n[0];
          }
      } else {
#pragma unroll
        for (int f = 0; f < S; ++f)
#pragma unroll
          for (int k = 0; k < V; ++k) u[k] += in_s[f] * x[f][k];
      }
      float w[V], b[V];
#pragma unroll
      for (int k = 0; k < V; ++k) {
        w[k] = a.norm[c + k];
        b[k] = a.norm[a.D + c + k];
        r[k] = tanhf(alpha * u[k]) * w[k] + b[k];
      }
    }
    T *hp = (T *)a.h + t * a.Dp + c;
    T *sp = a.swz == nullptr ? nullptr
                             : (T *)a.swz + (int64_t)(c >> 4) * 512 +
                                   ((c >> 3) & 1) * 256 + t * 8 + (c & 7);
    if constexpr (V == 4 && sizeof(T) == 2) {
      uint2 v;
      v.x = rb::pack_bf16x2(r[0], r[1]);
      v.y = rb::pack_bf16x2(r[2], r[3]);
      *reinterpret_cast<uint2 *>(hp) = v;
      if (sp != nullptr) *reinterpret_cast<uint2 *>(sp) = v;
    } else {
#pragma unroll
      for (int k = 0; k < V; ++k) {
        rb::store_scalar(hp + k, r[k]);
        if (sp != nullptr) rb::store_scalar(sp + k, r[k]);
      }
    }
  }
}

template <typename T>
__global__ __launch_bounds__(BLOCK) void squared_relu_kernel(
    const T *__restrict__ y, int64_t ny, T *__restrict__ z,
    T *__restrict__ swz, int64_t rows, int n) {
  constexpr int W = rb::VIO<T>::W;
  const int per_row = n / W;
  const int64_t total = rows * per_row;
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < total;
       i += (int64_t)gridDim.x * BLOCK) {
    const int64_t t = i / per_row;
    const int c = (int)(i - t * per_row) * W;
    float f[W];
    rb::VIO<T>::load(y + t * ny + c, f);
#pragma unroll
    for (int k = 0; k < W; ++k) {
      const float p = fmaxf(f[k], 0.0f);
      f[k] = p * p;
    }
    rb::VIO<T>::store(z + t * n + c, f);
    if constexpr (sizeof(T) == 2)
      if (swz != nullptr)
        rb::VIO<T>::store(swz + (int64_t)(c >> 4) * 512 +
                          ((c >> 3) & 1) * 256 + t * 8, f);
  }
}

int parts(const c10::optional<at::Tensor> &d, int64_t T, int64_t D) {
  if (!d.has_value()) return 0;
  TORCH_CHECK(d->is_cuda() && d->scalar_type() == at::kFloat &&
              d->is_contiguous() && (d->dim() == 2 || d->dim() == 3) &&
              d->size(-1) == D && d->size(-2) == T,
              "streams_norm: parts [n, T, D] f32");
  return d->dim() == 2 ? 1 : (int)d->size(0);
}

}  // namespace

std::vector<at::Tensor> streams_norm(
    at::Tensor x, c10::optional<at::Tensor> delta,
    c10::optional<at::Tensor> extra, c10::optional<at::Tensor> y, int64_t off,
    c10::optional<at::Tensor> join, at::Tensor inp, at::Tensor norm,
    bool bf16, bool operand) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 3 && x.is_contiguous() &&
              x.scalar_type() == at::kFloat, "streams_norm: x [T, s, D] f32");
  const int64_t T = x.size(0), s = x.size(1), D = x.size(2);
  TORCH_CHECK(s >= 1 && s <= MAX_STREAMS && inp.scalar_type() == at::kFloat &&
              inp.is_contiguous() && inp.numel() == s &&
              norm.scalar_type() == at::kFloat && norm.is_contiguous() &&
              norm.numel() == 2 * D + 1, "streams_norm: in, norm");
  Args a{};
  a.x = x.data_ptr<float>();
  a.n_delta = parts(delta, T, D);
  a.n_extra = parts(extra, T, D);
  TORCH_CHECK((a.n_delta > 0) == join.has_value() &&
              join.has_value() == y.has_value() &&
              (a.n_extra == 0 || a.n_delta > 0), "streams_norm: pending");
  const auto dt = bf16 ? at::kBFloat16 : at::kFloat;
  if (join.has_value()) {
    TORCH_CHECK(join->scalar_type() == at::kFloat && join->is_contiguous() &&
                join->numel() == 2 * D + s + s * s && y->is_cuda() &&
                y->dim() == 2 && y->is_contiguous() && y->size(0) == T &&
                y->scalar_type() == dt && off >= 0 && off + D <= y->size(1),
                "streams_norm: join, gate");
    a.delta = delta->data_ptr<float>();
    a.extra = extra ? extra->data_ptr<float>() : nullptr;
    a.y = y->data_ptr();
    a.ny = y->size(1);
    a.off = (int)off;
    a.join = join->data_ptr<float>();
  }
  a.inp = inp.data_ptr<float>();
  a.norm = norm.data_ptr<float>();
  a.T = T;
  a.s = (int)s;
  a.D = (int)D;
  a.Dp = (int)((D + 31) / 32 * 32);
  at::Tensor h = at::empty({T, (int64_t)a.Dp}, x.options().dtype(dt)), swz;
  a.h = h.data_ptr();
  if (operand) {
    TORCH_CHECK(bf16 && T <= 32, "streams_norm: operand");
    swz = at::empty({(int64_t)a.Dp * 32}, h.options());
    a.swz = swz.data_ptr();
  }
  if (T == 0) return {h, swz};
  auto stream = at::hip::getCurrentHIPStream();
  auto launch = [&](auto tag, auto n, auto v) {
    using E = decltype(tag);
    constexpr int S = decltype(n)::value, V = decltype(v)::value;
    const int64_t blocks = (T * (a.Dp / V) + BLOCK - 1) / BLOCK;
    hipLaunchKernelGGL((streams_norm_kernel<E, S, V>),
                       dim3((unsigned)std::min<int64_t>(blocks, 16384)),
                       dim3(BLOCK), 0, stream, a);
  };
  auto by_size = [&](auto tag, auto v) {
    if (s <= 1) launch(tag, std::integral_constant<int, 1>{}, v);
    else if (s <= 2) launch(tag, std::integral_constant<int, 2>{}, v);
    else if (s <= 3) launch(tag, std::integral_constant<int, 3>{}, v);
    else if (s <= 4) launch(tag, std::integral_constant<int, 4>{}, v);
    else if (s <= 8) launch(tag, std::integral_constant<int, 8>{}, v);
    else launch(tag, std::integral_constant<int, 16>{}, v);
  };
  auto by_width = [&](auto tag) {
    if (D % 4 == 0) by_size(tag, std::integral_constant<int, 4>{});
    else by_size(tag, std::integral_constant<int, 1>{});
  };
  if (bf16) by_width(uint16_t{});
  else by_width(float{});
  return {h, swz};
}

std::vector<at::Tensor> squared_relu(at::Tensor y, int64_t n, bool operand) {
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              n % 16 == 0 && n <= y.size(1) && y.size(1) % 8 == 0,
              "squared_relu: y [T, >= n]");
  const int64_t T = y.size(0);
  const bool bf16 = y.scalar_type() == at::kBFloat16;
  TORCH_CHECK(bf16 || y.scalar_type() == at::kFloat, "squared_relu: dtype");
  at::Tensor z = at::empty({T, n}, y.options()), swz;
  if (operand) {
    TORCH_CHECK(bf16 && T <= 32, "squared_relu: operand");
    swz = at::empty({n * 32}, y.options());
  }
  if (T == 0) return {z, swz};
  auto stream = at::hip::getCurrentHIPStream();
  auto launch = [&](auto tag) {
    using E = decltype(tag);
    const int64_t blocks = (T * (n / rb::VIO<E>::W) + BLOCK - 1) / BLOCK;
    hipLaunchKernelGGL((squared_relu_kernel<E>),
                       dim3((unsigned)std::min<int64_t>(blocks, 16384)),
                       dim3(BLOCK), 0, stream, (const E *)y.data_ptr(),
                       y.size(1), (E *)z.data_ptr(),
                       operand ? (E *)swz.data_ptr() : nullptr, T, (int)n);
  };
  if (bf16) launch(uint16_t{});
  else launch(float{});
  return {z, swz};
}
