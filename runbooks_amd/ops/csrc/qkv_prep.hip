// Queries and keys of attention with its own values, per-token step (gfx950):
// RMS norm per head, rotation of neighbouring pairs; q stays in y, the row
// [ key | value ] goes to the paged cache (shared_kv.h).
//
// y rows: [ q heads | k heads | v heads | .. ], sizes per head padded to 8.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "shared_kv.h"

namespace {

constexpr int BLOCK = 256;

struct PrepArgs {
  int64_t ny;
  int heads, kv, dim, hc, vc, half;    // half: rotated pairs
  float eps;
};

template <typename T> RB_DEV void load8(const T *p, float *f) {
  rb::VIO<T>::load(p, f);
  if constexpr (rb::VIO<T>::W == 4) rb::VIO<T>::load(p + 4, f + 4);
}
template <typename T> RB_DEV void store8(T *p, const float *f) {
  rb::VIO<T>::store(p, f);
  if constexpr (rb::VIO<T>::W == 4) rb::VIO<T>::store(p + 4, f + 4);
}

// One workgroup per token; L lanes per head with NV times 8 columns each.
template <typename T, int L, int NV>
__global__ __launch_bounds__(BLOCK) void qkv_prep_kernel(
    T *__restrict__ y, const float *__restrict__ cos,
    const float *__restrict__ sin, const int *__restrict__ positions,
    const int *__restrict__ slots, T *__restrict__ cache,
    const float *__restrict__ norms, PrepArgs a) {
  constexpr int GROUPS = BLOCK / L;
  const int64_t t = blockIdx.x;
  T *yr = y + t * a.ny;
  const int slot = slots[t], lane = threadIdx.x % L, ec = a.hc + a.vc;
  T *page = cache + ((int64_t)(slot / skv::PAGE) * a.kv * skv::PAGE +
                     slot % skv::PAGE) * ec;
  const int64_t page_head = (int64_t)skv::PAGE * ec;
  const float *cr = cos + (int64_t)positions[t] * a.half;
  const float *sr = sin + (int64_t)positions[t] * a.half;
  float cc[NV][4], ss[NV][4], wq[NV][8], wk[NV][8];
#pragma unroll
  for (int n = 0; n < NV; ++n) {
    const int c0 = (n * L + lane) * 8;
    const bool turns = c0 < 2 * a.half;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int p = c0 / 2 + k;
      cc[n][k] = turns ? cr[min(p, a.half - 1)] : 1.0f;
      ss[n][k] = turns ? sr[min(p, a.half - 1)] : 0.0f;
      if (p >= a.half) {
        cc[n][k] = 1.0f;
        ss[n][k] = 0.0f;
      }
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const int c = min(c0 + k, a.dim - 1);
      wq[n][k] = c0 + k < a.dim ? norms[c] : 0.0f;
      wk[n][k] = c0 + k < a.dim ? norms[a.dim + c] : 0.0f;
    }
  }
  const int n_heads = a.heads + a.kv;
  float ahead[NV][8];
  auto fetch = [&](int h) {
#pragma unroll
    for (int n = 0; n < NV; ++n) {
      const int c = (n * L + lane) * 8;
      // padding is zero; beyond it any address of the row
      load8(yr + (int64_t)min(h, n_heads - 1) * a.hc + (c < a.hc ? c : 0),
            ahead[n]);
    }
  };
  fetch(threadIdx.x / L);
  for (int h0 = 0; h0 < n_heads; h0 += GROUPS) {
    const int h = h0 + threadIdx.x / L;
    const bool ok = h < n_heads, is_k = h >= a.heads;
    T *src = yr + (int64_t)h * a.hc;
    float v[NV][8], sum = 0.0f;
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        v[n][k] = (n * L + lane) * 8 < a.hc ? ahead[n][k] : 0.0f;
        sum += v[n][k] * v[n][k];
      }
    if (h0 + GROUPS < n_heads) fetch(h + GROUPS);
#pragma unroll
    for (int o = L / 2; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
    const float inv = 1.0f / sqrtf(sum / a.dim + a.eps);
    if (!ok) continue;
#pragma unroll
    for (int n = 0; n < NV; ++n) {
      const int c = (n * L + lane) * 8;
      if (c >= a.hc) continue;
      float r[8];
#pragma unroll
      for (int k = 0; k < 8; ++k)
        r[k] = v[n][k] * inv * (is_k ? wk[n][k] : wq[n][k]);
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float p = r[2 * k], q = r[2 * k + 1];
        r[2 * k] = p * cc[n][k] - q * ss[n][k];
        r[2 * k + 1] = q * cc[n][k] + p * ss[n][k];
      }
      store8(is_k ? page + (h - a.heads) * page_head + c : src + c, r);
    }
  }
  const int vv = a.vc / 8;
  for (int i = threadIdx.x; i < a.kv * vv; i += BLOCK) {
    const int g = i / vv, c = (i - g * vv) * 8;
    float f[8];
    load8(yr + (int64_t)n_heads * a.hc + g * a.vc + c, f);
    store8(page + g * page_head + a.hc + c, f);
  }
}

}  // namespace

void qkv_prep(at::Tensor y, at::Tensor cos, at::Tensor sin,
              at::Tensor positions, at::Tensor slots, at::Tensor cache,
              at::Tensor norms, int64_t heads, int64_t dim, int64_t hc,
              double eps) {
  const auto dt = y.scalar_type();
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (dt == at::kBFloat16 || dt == at::kFloat) &&
              y.size(1) % 8 == 0, "qkv_prep: y");
  TORCH_CHECK(cache.is_cuda() && cache.dim() == 4 &&
              cache.size(2) == skv::PAGE && cache.is_contiguous() &&
              cache.scalar_type() == dt,
              "qkv_prep: cache [blocks, kv heads, 16, ec]");
  const int64_t T = y.size(0), G = cache.size(1), vc = cache.size(3) - hc;
  TORCH_CHECK(dim >= 1 && dim <= hc && hc % 8 == 0 && hc <= 1024 && vc >= 8 &&
              vc % 8 == 0 && heads >= 1 &&
              (heads + G) * hc + G * vc <= y.size(1), "qkv_prep: layout");
  TORCH_CHECK(cos.scalar_type() == at::kFloat && cos.is_contiguous() &&
              cos.dim() == 2 && cos.sizes() == sin.sizes() &&
              sin.scalar_type() == at::kFloat && sin.is_contiguous() &&
              2 * cos.size(1) <= dim, "qkv_prep: tables");
  TORCH_CHECK(positions.scalar_type() == at::kInt &&
              positions.is_contiguous() && positions.numel() == T &&
              slots.scalar_type() == at::kInt && slots.is_contiguous() &&
              slots.numel() == T && norms.scalar_type() == at::kFloat &&
              norms.is_contiguous() && norms.numel() == 2 * dim,
              "qkv_prep: positions, slots, norms");
  if (T == 0) return;
  const PrepArgs a{y.size(1), (int)heads, (int)G, (int)dim, (int)hc, (int)vc,
                   (int)cos.size(1), (float)eps};
  auto stream = at::hip::getCurrentHIPStream();
  auto launch = [&](auto tag, auto l, auto n) {
    using E = decltype(tag);
    hipLaunchKernelGGL(
        (qkv_prep_kernel<E, decltype(l)::value, decltype(n)::value>), dim3(T),
        dim3(BLOCK), 0, stream, (E *)y.data_ptr(), cos.data_ptr<float>(),
        sin.data_ptr<float>(), positions.data_ptr<int>(),
        slots.data_ptr<int>(), (E *)cache.data_ptr(), norms.data_ptr<float>(),
        a);
  };
  constexpr std::integral_constant<int, 1> one{};
  auto pick = [&](auto tag) {
    if (hc <= 64) launch(tag, std::integral_constant<int, 8>{}, one);
    else if (hc <= 128) launch(tag, std::integral_constant<int, 16>{}, one);
    else if (hc <= 256) launch(tag, std::integral_constant<int, 32>{}, one);
    else launch(tag, std::integral_constant<int, 64>{},
                std::integral_constant<int, 2>{});
  };
  if (dt == at::kBFloat16) pick(uint16_t{});
  else pick(float{});
}
