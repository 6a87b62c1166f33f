// Per-token activations of a feed-forward and a model's ends (gfx950):
//
//  * power_sums, poly_norm: a N(z) + b N(z^2) + c N(z^3) + e, N(v) = v / rms(v)
//  * tanh_rows: tanh of some columns, as the input of a product
//  * softcap: cap tanh(v / cap) of logits, a split-K slab's slices summed
//
// All in fp32 between a load and a store.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "history.h"

namespace {

constexpr int BLOCK = 256;

struct Sums { float s[3]; };

RB_DEV void add_powers(Sums &a, float z) {
  const float q = z * z, r = q * q;
  a.s[0] += q;
  a.s[1] += r;
  a.s[2] += r * q;
}

// The first ff columns of a row, 8 at a time; the first NV groups of a thread
// stay in `keep`.
template <typename T, int BLK, int NV>
RB_DEV Sums row_sums(const T *row, int ff, float (*red)[BLK / RB_WAVE],
                     float (*keep)[8]) {
  Sums a{};
#pragma unroll
  for (int n = 0; n < NV; ++n) {
    const int c = (n * BLK + threadIdx.x) * 8;
    if (c < ff) rb::load_v<8>(row + c, keep[n]);
  }
  auto add = [&](const float *f, int c) {
#pragma unroll
    for (int k = 0; k < 8; ++k)
      if (c + k < ff) add_powers(a, f[k]);
  };
#pragma unroll
  for (int n = 0; n < NV; ++n) add(keep[n], (n * BLK + threadIdx.x) * 8);
  for (int c = (NV * BLK + threadIdx.x) * 8; c < ff; c += BLK * 8) {
    float f[8];
    rb::load_v<8>(row + c, f);
    add(f, c);
  }
#pragma unroll
  for (int i = 0; i < 3; ++i) {
    a.s[i] = rb::wave_reduce_sum(a.s[i]);
    if ((threadIdx.x & 63) == 0) red[i][threadIdx.x >> 6] = a.s[i];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 3; ++i) {
    a.s[i] = 0.0f;
#pragma unroll
    for (int w = 0; w < BLK / RB_WAVE; ++w) a.s[i] += red[i][w];
  }
  return a;
}

template <typename T>
__global__ __launch_bounds__(BLOCK) void power_sums_kernel(
    const T *__restrict__ u, int64_t nu, int ff, float *__restrict__ out) {
  __shared__ float red[3][BLOCK / RB_WAVE];
  const int64_t t = blockIdx.x;
  float keep[1][8];
  const Sums s = row_sums<T, BLOCK, 1>(u + t * nu, ff, red, keep);
  if (threadIdx.x < 3) out[t * 3 + threadIdx.x] = s.s[threadIdx.x];
}

struct PolyArgs {
  int64_t nu, nz;
  int ff, off;
  float total, eps;
};

template <typename T, int BLK, int NV>
__global__ __launch_bounds__(BLK) void poly_norm_kernel(
    const T *__restrict__ u, const float *__restrict__ act,
    const float *__restrict__ sums, T *__restrict__ z, T *__restrict__ swz,
    PolyArgs a) {
  __shared__ float red[3][BLK / RB_WAVE];
  const int64_t t = blockIdx.x;
  const T *row = u + t * a.nu;
  float keep[NV][8];
  Sums s = row_sums<T, BLK, NV>(row, a.ff, red, keep);
  if (sums != nullptr) {                       // of all ranks
#pragma unroll
    for (int i = 0; i < 3; ++i) s.s[i] = sums[t * 3 + i];
  }
  float f[3];
#pragma unroll
  for (int i = 0; i < 3; ++i)
    f[i] = act[i] / sqrtf(s.s[i] / a.total + a.eps);
  const float e = act[3];
  const int n = (int)(a.nz - a.off);
  T *zr = z + t * a.nz + a.off;
  auto finish = [&](float *v, int c) {
#pragma unroll
    for (int k = 0; k < 8; ++k)
      v[k] = c + k < a.ff
                 ? v[k] * (f[0] + v[k] * (f[1] + v[k] * f[2])) + e : 0.0f;
    rb::store_v<8>(zr + c, v);
    if (swz != nullptr)
      rb::store_v<8>(swz + rb::operand_slot(a.off + c, (int)t), v);
  };
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * BLK + threadIdx.x) * 8;
    if (c < n) finish(keep[i], c);
  }
  for (int c = (NV * BLK + threadIdx.x) * 8; c < n; c += BLK * 8) {
    float v[8] = {};
    if (c < a.ff) rb::load_v<8>(row + c, v);
    finish(v, c);
  }
}

template <typename T>
__global__ __launch_bounds__(BLOCK) void tanh_rows_kernel(
    const T *__restrict__ y, int64_t ny, int n, T *__restrict__ out,
    T *__restrict__ swz, int64_t total) {
  const int64_t i = ((int64_t)blockIdx.x * BLOCK + threadIdx.x) * 8;
  if (i >= total) return;
  const int64_t t = i / n;
  const int c = (int)(i - t * n);
  float v[8];
  rb::load_v<8>(y + t * ny + c, v);
#pragma unroll
  for (int k = 0; k < 8; ++k) v[k] = tanhf(v[k]);
  rb::store_v<8>(out + i, v);
  if (swz != nullptr) rb::store_v<8>(swz + rb::operand_slot(c, (int)t), v);
}

template <int V>
__global__ __launch_bounds__(BLOCK) void softcap_kernel(
    const float *__restrict__ x, float *__restrict__ out, int64_t n, int parts,
    float cap) {
  const int64_t i = ((int64_t)blockIdx.x * BLOCK + threadIdx.x) * V;
  if (i >= n) return;
  float v[V] = {};
  for (int s = 0; s < parts; ++s) {
#pragma unroll
    for (int k = 0; k < V; ++k) v[k] += x[(int64_t)s * n + i + k];
  }
#pragma unroll
  for (int k = 0; k < V; ++k) out[i + k] = cap * tanhf(v[k] / cap);
}

void check_rows(const at::Tensor &u, int64_t ff, const char *who) {
  TORCH_CHECK(u.is_cuda() && u.dim() == 2 && u.is_contiguous() &&
              (u.scalar_type() == at::kBFloat16 ||
               u.scalar_type() == at::kFloat) && u.size(1) % 8 == 0 &&
              ff >= 1 && ff <= u.size(1), who, ": rows");
}

}  // namespace

at::Tensor power_sums(at::Tensor u, int64_t ff) {
  check_rows(u, ff, "power_sums");
  auto out = at::empty({u.size(0), 3}, u.options().dtype(at::kFloat));
  if (u.size(0) == 0) return out;
  auto stream = at::hip::getCurrentHIPStream();
  auto go = [&](auto tag) {
    using E = decltype(tag);
    hipLaunchKernelGGL((power_sums_kernel<E>), dim3(u.size(0)), dim3(BLOCK), 0,
                       stream, (const E *)u.data_ptr(), u.size(1), (int)ff,
                       out.data_ptr<float>());
  };
  if (u.scalar_type() == at::kBFloat16) go(uint16_t{});
  else go(float{});
  return out;
}

// z's columns from `off` on, and the same of its decode operand
void poly_norm(at::Tensor u, int64_t ff, int64_t total, at::Tensor act,
               double eps, at::Tensor z, int64_t off,
               c10::optional<at::Tensor> swz,
               c10::optional<at::Tensor> sums) {
  check_rows(u, ff, "poly_norm");
  const auto dt = u.scalar_type();
  const int64_t T = u.size(0);
  TORCH_CHECK(z.is_cuda() && z.dim() == 2 && z.is_contiguous() &&
              z.scalar_type() == dt && z.size(0) == T &&
              z.size(1) % 16 == 0 && off % 8 == 0 && off >= 0 &&
              off + ff <= z.size(1) && total >= ff && act.is_cuda() &&
              act.scalar_type() == at::kFloat && act.numel() == 4 &&
              act.is_contiguous(), "poly_norm: z, act");
  if (swz.has_value())
    TORCH_CHECK(dt == at::kBFloat16 && T <= 32 && swz->is_contiguous() &&
                swz->scalar_type() == dt && swz->numel() == z.size(1) * 32,
                "poly_norm: operand");
  if (sums.has_value())
    TORCH_CHECK(sums->is_cuda() && sums->scalar_type() == at::kFloat &&
                sums->is_contiguous() && sums->numel() == T * 3,
                "poly_norm: sums [T, 3] f32");
  if (T == 0) return;
  const PolyArgs a{u.size(1), z.size(1), (int)ff, (int)off, (float)total,
                   (float)eps};
  auto stream = at::hip::getCurrentHIPStream();
  auto go = [&](auto tag) {
    using E = decltype(tag);
    auto launch = [&](auto blk, auto nv) {
      constexpr int B = decltype(blk)::value, N = decltype(nv)::value;
      hipLaunchKernelGGL((poly_norm_kernel<E, B, N>), dim3(T), dim3(B), 0,
                         stream, (const E *)u.data_ptr(),
                         act.data_ptr<float>(),
                         sums ? sums->data_ptr<float>() : nullptr,
                         (E *)z.data_ptr(),
                         swz ? (E *)swz->data_ptr() : nullptr, a);
    };
    constexpr std::integral_constant<int, 256> few{};
    constexpr std::integral_constant<int, 1024> many{};
    if (ff <= 256 * 8 * 2) launch(few, std::integral_constant<int, 2>{});
    else if (T > 256 && ff <= 256 * 8 * 8)
      launch(few, std::integral_constant<int, 8>{});
    else launch(many, std::integral_constant<int, 2>{});
  };
  if (dt == at::kBFloat16) go(uint16_t{});
  else go(float{});
}

void tanh_rows(at::Tensor y, int64_t off, at::Tensor out,
               c10::optional<at::Tensor> swz) {
  const auto dt = y.scalar_type();
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (dt == at::kBFloat16 || dt == at::kFloat) && out.dim() == 2 &&
              out.is_contiguous() && out.scalar_type() == dt &&
              out.size(0) == y.size(0) && out.size(1) % 8 == 0 &&
              off % 8 == 0 && off >= 0 && y.size(1) % 8 == 0 &&
              off + out.size(1) <= y.size(1), "tanh_rows: layout");
  if (swz.has_value())
    TORCH_CHECK(dt == at::kBFloat16 && y.size(0) <= 32 &&
                swz->is_contiguous() && swz->scalar_type() == dt &&
                out.size(1) % 16 == 0 && swz->numel() == out.size(1) * 32,
                "tanh_rows: operand");
  const int64_t total = out.numel();
  if (total == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  auto go = [&](auto tag) {
    using E = decltype(tag);
    hipLaunchKernelGGL((tanh_rows_kernel<E>),
                       dim3((total / 8 + BLOCK - 1) / BLOCK), dim3(BLOCK), 0,
                       stream, (const E *)y.data_ptr() + off, y.size(1),
                       (int)out.size(1), (E *)out.data_ptr(),
                       swz ? (E *)swz->data_ptr() : nullptr, total);
  };
  if (dt == at::kBFloat16) go(uint16_t{});
  else go(float{});
}

at::Tensor softcap(at::Tensor x, double cap) {
  TORCH_CHECK(x.is_cuda() && x.is_contiguous() &&
              x.scalar_type() == at::kFloat && (x.dim() == 2 || x.dim() == 3)
              && cap > 0, "softcap: logits [n, V] or [split, n, V] f32");
  const int64_t rows = x.size(-2), V = x.size(-1), n = rows * V;
  auto out = at::empty({rows, V}, x.options());
  if (n == 0) return out;
  const int parts = x.dim() == 3 ? (int)x.size(0) : 1;
  auto stream = at::hip::getCurrentHIPStream();
  if (n % 4 == 0)
    hipLaunchKernelGGL((softcap_kernel<4>), dim3((n / 4 + BLOCK - 1) / BLOCK),
                       dim3(BLOCK), 0, stream, x.data_ptr<float>(),
                       out.data_ptr<float>(), n, parts, (float)cap);
  else
    hipLaunchKernelGGL((softcap_kernel<1>), dim3((n + BLOCK - 1) / BLOCK),
                       dim3(BLOCK), 0, stream, x.data_ptr<float>(),
                       out.data_ptr<float>(), n, parts, (float)cap);
  return out;
}
