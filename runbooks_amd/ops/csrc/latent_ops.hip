// Latent attention, per-token steps (gfx950): the epilogue of the wide
// projection and the per-head products between q/value space and latent
// space.
//
// y rows: [ q heads | latent, rotated key | head gates | mlp gate | mlp up ],
// z rows: [ gated heads | mlp activation ]; every section and head starts at
// a multiple of 8 elements (zero-padded weights), so all IO is 16 B/lane.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 256;
constexpr int ACT_VECS = BLOCK * 2;   // 8-wide activation vectors per block

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8v;
typedef __attribute__((ext_vector_type(4))) float f32x4v;

template <typename T> RB_DEV void load8(const T *p, float *f) {
  rb::VIO<T>::load(p, f);
  if constexpr (rb::VIO<T>::W == 4) rb::VIO<T>::load(p + 4, f + 4);
}
template <typename T> RB_DEV void store8(T *p, const float *f) {
  rb::VIO<T>::store(p, f);
  if constexpr (rb::VIO<T>::W == 4) rb::VIO<T>::store(p + 4, f + 4);
}

template <typename T> RB_DEV float sigmoidf(float v) {
  if constexpr (sizeof(T) == 2) return 1.0f / (1.0f + __expf(-v));
  else return 1.0f / (1.0f + expf(-v));
}

// decode-GEMM operand slot of 8 columns from k (k % 8 == 0)
RB_DEV int64_t operand_at(int k, int row) {
  return (int64_t)(k >> 4) * 512 + ((k >> 3) & 1) * 256 + row * 8;
}

template <typename T>
RB_DEV void rotate_pair(const T *in, T *out, float c, float s) {
  const float u = rb::bf16_to_f32_or_id(in[0]);
  const float v = rb::bf16_to_f32_or_id(in[1]);
  rb::store_scalar(out, u * c - v * s);
  rb::store_scalar(out + 1, v * c + u * s);
}

struct PrepArgs {
  int heads, dimc, rotc, rank, rc, off_kv, off_gate, off_up, fc, off_act;
  int ny, nz, half;
  float eps, limit, alpha, shift;
};

// block (token, 0): rotations, latent norm, cache write; blocks (token, 1..):
// the mlp activation, ACT_VECS vectors each
template <typename T>
__global__ __launch_bounds__(BLOCK) void latent_prep_kernel(
    T *__restrict__ y, const float *__restrict__ cos,
    const float *__restrict__ sin, const int *__restrict__ positions,
    const int *__restrict__ slots, T *__restrict__ cache,
    const T *__restrict__ w, T *__restrict__ z, T *__restrict__ swz,
    PrepArgs a) {
  const int t = blockIdx.x;
  T *yr = y + (int64_t)t * a.ny;
  if (blockIdx.y > 0) {
    const int base = (blockIdx.y - 1) * ACT_VECS;
    const int nvec = (a.nz - a.off_act) / 8;
    for (int i = base + threadIdx.x; i < min(nvec, base + ACT_VECS);
         i += BLOCK) {
      float o[8];
      if (i * 8 < a.fc) {
        float g[8], u[8];
        load8(yr + a.off_gate + i * 8, g);
        load8(yr + a.off_up + i * 8, u);
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          const float gg = fminf(g[k], a.limit);
          const float uu = fminf(fmaxf(u[k], -a.limit), a.limit);
          o[k] = gg * sigmoidf<T>(a.alpha * gg) * (uu + a.shift);
        }
      } else {
#pragma unroll
        for (int k = 0; k < 8; ++k) o[k] = 0.0f;
      }
      const int col = a.off_act + i * 8;
      store8(z + (int64_t)t * a.nz + col, o);
      if (swz != nullptr) store8(swz + operand_at(col, t), o);
    }
    return;
  }

  __shared__ float red[BLOCK / RB_WAVE];
  const int pos = positions[t];
  const float *cr = cos + (int64_t)pos * a.half;
  const float *sr = sin + (int64_t)pos * a.half;
  for (int p = threadIdx.x; p < a.heads * a.half; p += BLOCK) {
    const int h = p / a.half, i = p - h * a.half;
    T *q = yr + h * (a.dimc + a.rotc) + a.dimc + 2 * i;
    rotate_pair(q, q, cr[i], sr[i]);
  }
  if (cache == nullptr) return;
  const T *kv = yr + a.off_kv;
  T *row = cache + (int64_t)slots[t] * (a.rc + a.rotc);
  float ss = 0.0f;
  for (int i = threadIdx.x; i < a.rank; i += BLOCK) {
    const float v = rb::bf16_to_f32_or_id(kv[i]);
    ss += v * v;
  }
  ss = rb::block_reduce_sum(ss, red);
  const float ir = 1.0f / sqrtf(ss / (float)a.rank + a.eps);
  for (int i = threadIdx.x; i < a.rank; i += BLOCK)
    rb::store_scalar(row + i, rb::bf16_to_f32_or_id(kv[i]) * ir *
                                  rb::bf16_to_f32_or_id(w[i]));
  for (int i = threadIdx.x; i < a.half; i += BLOCK)
    rotate_pair(kv + a.rc + 2 * i, row + a.rc + 2 * i, cr[i], sr[i]);
  // dimensions beyond the rotated ones pass unchanged
  for (int i = 2 * a.half + threadIdx.x; i < a.rotc; i += BLOCK)
    row[a.rc + i] = kv[a.rc + i];
}

// ---------------------------------------------------------------------------
// RMS norms of two latents in y: blocks (token, 0) the queries' one, to `out`,
// blocks (token, 1) the cached one, both with zeros up to the row's end
// ---------------------------------------------------------------------------
struct NormsArgs {
  int64_t ny;
  int oq, nq, no, oc, nc, ec;
  float eps;
};

template <typename T>
__global__ __launch_bounds__(BLOCK) void latent_norms_kernel(
    const T *__restrict__ y, const float *__restrict__ wq,
    const float *__restrict__ wc, T *__restrict__ out, T *__restrict__ swz,
    T *__restrict__ cache, const int *__restrict__ slots, NormsArgs a) {
  __shared__ float red[BLOCK / RB_WAVE];
  constexpr int NV = 2;                        // 8-wide vectors kept
  const int64_t t = blockIdx.x;
  const bool cached = blockIdx.y > 0;
  const int n = cached ? a.nc : a.nq, width = cached ? a.ec : a.no;
  const T *row = y + t * a.ny + (cached ? a.oc : a.oq);
  const float *w = cached ? wc : wq;
  float v[NV][8], ss = 0.0f;
  auto add = [&](const float *f, int c) {
#pragma unroll
    for (int k = 0; k < 8; ++k) ss += c + k < n ? f[k] * f[k] : 0.0f;
  };
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * BLOCK + threadIdx.x) * 8;
    if (c < n) load8(row + c, v[i]);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) add(v[i], (i * BLOCK + threadIdx.x) * 8);
  for (int c = (NV * BLOCK + threadIdx.x) * 8; c < n; c += BLOCK * 8) {
    float f[8];
    load8(row + c, f);
    add(f, c);
  }
  ss = rb::block_reduce_sum(ss, red);
  const float ir = 1.0f / sqrtf(ss / (float)n + a.eps);
  T *dst = cached ? cache + (int64_t)slots[t] * a.ec : out + t * a.no;
  auto finish = [&](float *f, int c) {
#pragma unroll
    for (int k = 0; k < 8; ++k)
      f[k] = c + k < n ? f[k] * ir * w[c + k] : 0.0f;
    store8(dst + c, f);
    if (!cached && swz != nullptr) store8(swz + operand_at(c, (int)t), f);
  };
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * BLOCK + threadIdx.x) * 8;
    if (c < width) finish(v[i], c);
  }
  for (int c = (NV * BLOCK + threadIdx.x) * 8; c < width; c += BLOCK * 8) {
    float f[8] = {};
    if (c < n) load8(row + c, f);
    finish(f, c);
  }
}

// ---------------------------------------------------------------------------
// y_h = x_h @ w_h per head, optionally times sigmoid(gate).
//   x element (m, h, k): x[x_off + m * xs + h * xh + k], k < K (K % 8 == 0)
//   out element (m, h, n): out[o_off + m * os + h * oh + n], n < N
//   gate element: g[g_off + m * gs + h * oh + n], or one per head:
//                 g[g_off + m * gs + h]
// ---------------------------------------------------------------------------
struct HeadArgs {
  int64_t x_off, xs, o_off, os, g_off, gs;
  int xh, oh, K, N, T, head_gate;
};

// Weights in fragment order [H][N/16][K/32][lane][8]: each step of a wave is
// one contiguous 1 KiB read. The weight is the A operand, so a lane ends up
// with 4 consecutive columns of one row. Two row tiles (32 rows) per block.
// SPLITK: the block's waves share one column tile and split K; otherwise each
// wave has its own column tile.
template <bool SPLITK>
__global__ __launch_bounds__(BLOCK) void head_gemm_kernel(
    const uint16_t *__restrict__ x, const uint16_t *__restrict__ w,
    uint16_t *__restrict__ out, const uint16_t *__restrict__ gate,
    uint16_t *__restrict__ swz, HeadArgs a) {
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int l16 = lane & 15, grp = lane >> 4;
  const int ntiles = (a.N + 15) / 16, steps = (a.K + 31) / 32;
  const int nt = SPLITK ? blockIdx.x : blockIdx.x * 4 + wid;
  const int h = blockIdx.y, m0 = blockIdx.z * 32;
  if (!SPLITK && nt >= ntiles) return;

  const int per = SPLITK ? (steps + 3) / 4 : steps;
  const int s0 = SPLITK ? wid * per : 0;
  const int s1 = min(steps, s0 + per);
  const uint16_t *wp =
      w + ((int64_t)h * ntiles + nt) * steps * 512 + lane * 8;
  const uint16_t *xr[2];
  bool ok[2];
#pragma unroll
  for (int mt = 0; mt < 2; ++mt) {
    const int m = m0 + mt * 16 + l16;
    ok[mt] = m < a.T;
    xr[mt] = x + a.x_off + (int64_t)(ok[mt] ? m : 0) * a.xs +
             (int64_t)h * a.xh + grp * 8;
  }
  f32x4v acc[2] = {(f32x4v)(0.0f), (f32x4v)(0.0f)};
  const bf16x8v zero = (bf16x8v)(__bf16)0.0f;
#pragma unroll 4
  for (int s = s0; s < s1; ++s) {
    const bf16x8v wf = *reinterpret_cast<const bf16x8v *>(wp + s * 512);
    const bool in_k = s * 32 + grp * 8 < a.K;
#pragma unroll
    for (int mt = 0; mt < 2; ++mt) {
      const bf16x8v xf =
          (ok[mt] && in_k)
              ? *reinterpret_cast<const bf16x8v *>(xr[mt] + s * 32)
              : zero;
      acc[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, xf, acc[mt], 0, 0,
                                                        0);
    }
  }
  const int n = nt * 16 + grp * 4;
  auto finish = [&](int mt, f32x4v r4) {
    const int m = m0 + mt * 16 + l16;
    if (m >= a.T || n >= a.N) return;
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = r4[r];
    if (gate != nullptr) {
      const uint16_t *gp = gate + a.g_off + m * a.gs;
      uint2 gw;
      if (a.head_gate) gw.x = gw.y = gp[h] * 0x10001u;
      else gw = *reinterpret_cast<const uint2 *>(gp + (int64_t)h * a.oh + n);
      const uint32_t gu[2] = {gw.x, gw.y};
#pragma unroll
      for (int r = 0; r < 4; ++r)
        v[r] *= sigmoidf<uint16_t>(
            rb::bf16_to_f32((uint16_t)(gu[r >> 1] >> (16 * (r & 1)))));
    }
    uint2 o;
    o.x = rb::pack_bf16x2(v[0], v[1]);
    o.y = rb::pack_bf16x2(v[2], v[3]);
    *reinterpret_cast<uint2 *>(out + a.o_off + m * a.os + (int64_t)h * a.oh +
                               n) = o;
    if (swz != nullptr) {
      const int k = (int)a.o_off + h * a.oh + n;
      *reinterpret_cast<uint2 *>(swz + operand_at(k & ~7, m) + (k & 7)) = o;
    }
  };
  if constexpr (SPLITK) {
    __shared__ f32x4v red[4][2][64];
    red[wid][0][lane] = acc[0];
    red[wid][1][lane] = acc[1];
    __syncthreads();
    if (wid < 2)                        // waves 0, 1 finish row tiles 0, 1
      finish(wid, red[0][wid][lane] + red[1][wid][lane] + red[2][wid][lane] +
                      red[3][wid][lane]);
  } else {
    finish(0, acc[0]);
    finish(1, acc[1]);
  }
}

// fp32: weights [H][K][N], one thread per output
__global__ void head_gemm_f32_kernel(const float *__restrict__ x,
                                     const float *__restrict__ w,
                                     float *__restrict__ out,
                                     const float *__restrict__ gate,
                                     HeadArgs a) {
  const int n = blockIdx.x * 64 + threadIdx.x;
  const int h = blockIdx.y;
  const int64_t m = (int64_t)blockIdx.z * 4 + threadIdx.y;
  if (n >= a.N || m >= a.T) return;
  const float *xr = x + a.x_off + m * a.xs + (int64_t)h * a.xh;
  const float *wr = w + (int64_t)h * a.K * a.N + n;
  float acc = 0.0f;
  for (int k = 0; k < a.K; ++k) acc = fmaf(xr[k], wr[(int64_t)k * a.N], acc);
  if (gate != nullptr)
    acc *= sigmoidf<float>(gate[a.g_off + m * a.gs +
                                (a.head_gate ? h : (int64_t)h * a.oh + n)]);
  out[a.o_off + m * a.os + (int64_t)h * a.oh + n] = acc;
}

}  // namespace

void latent_prep(at::Tensor y, at::Tensor cos, at::Tensor sin,
                 at::Tensor positions, at::Tensor slots,
                 c10::optional<at::Tensor> cache, c10::optional<at::Tensor> w,
                 at::Tensor z, c10::optional<at::Tensor> swz, int64_t heads,
                 int64_t dimc, int64_t rotc, int64_t rank, int64_t rc,
                 int64_t off_kv, int64_t off_gate, int64_t off_up, int64_t fc,
                 int64_t off_act, double eps, double limit, double alpha,
                 double shift) {
  const int64_t T = y.size(0), ny = y.size(1), nz = z.size(1);
  const int64_t half = cos.size(1);
  TORCH_CHECK(y.is_cuda() && y.is_contiguous() && z.is_contiguous() &&
              z.size(0) == T && y.scalar_type() == z.scalar_type(),
              "latent_prep: y, z");
  TORCH_CHECK(dimc % 8 == 0 && rotc % 8 == 0 && rc % 8 == 0 && fc % 8 == 0 &&
              off_kv % 8 == 0 && off_gate % 8 == 0 && off_up % 8 == 0 &&
              off_act % 8 == 0 && ny % 8 == 0 && nz % 16 == 0 &&
              heads * (dimc + rotc) <= off_kv && off_kv <= off_gate &&
              off_gate + fc <= off_up && off_up + fc <= ny &&
              off_act + fc <= nz && 2 * half <= rotc && rank <= rc,
              "latent_prep: layout");
  TORCH_CHECK(cos.scalar_type() == at::kFloat && cos.is_contiguous() &&
              sin.is_contiguous() && sin.sizes() == cos.sizes() &&
              positions.scalar_type() == at::kInt && positions.numel() == T &&
              slots.scalar_type() == at::kInt && slots.numel() == T,
              "latent_prep: positions, tables");
  if (cache.has_value())
    TORCH_CHECK(w.has_value() && w->numel() == rank && w->is_contiguous() &&
                w->scalar_type() == y.scalar_type() && cache->is_contiguous() &&
                cache->scalar_type() == y.scalar_type() &&
                cache->size(-1) == rc + rotc && off_kv + rc + rotc <= off_gate,
                "latent_prep: cache");
  if (swz.has_value())
    TORCH_CHECK(T <= 32 && swz->numel() == nz * 32 && swz->is_contiguous() &&
                y.scalar_type() == at::kBFloat16, "latent_prep: operand");
  if (T == 0) return;
  PrepArgs a{(int)heads, (int)dimc, (int)rotc, (int)rank, (int)rc,
             (int)off_kv, (int)off_gate, (int)off_up, (int)fc, (int)off_act,
             (int)ny, (int)nz, (int)half,
             (float)eps, (float)limit, (float)alpha, (float)shift};
  const int nvec = (int)(nz - off_act) / 8;
  const dim3 grid(T, 1 + (nvec + ACT_VECS - 1) / ACT_VECS);
  auto stream = at::hip::getCurrentHIPStream();
  auto launch = [&](auto tag) {
    using E = decltype(tag);
    hipLaunchKernelGGL((latent_prep_kernel<E>), grid, dim3(BLOCK), 0, stream,
                       (E *)y.data_ptr(), cos.data_ptr<float>(),
                       sin.data_ptr<float>(), positions.data_ptr<int>(),
                       slots.data_ptr<int>(),
                       cache ? (E *)cache->data_ptr() : nullptr,
                       w ? (const E *)w->data_ptr() : nullptr,
                       (E *)z.data_ptr(), swz ? (E *)swz->data_ptr() : nullptr,
                       a);
  };
  if (y.scalar_type() == at::kBFloat16) launch(uint16_t{});
  else if (y.scalar_type() == at::kFloat) launch(float{});
  else TORCH_CHECK(false, "latent_prep: dtype");
}

void latent_norms(at::Tensor y, int64_t oq, int64_t nq, at::Tensor wq,
                  at::Tensor out, c10::optional<at::Tensor> swz, int64_t oc,
                  int64_t nc, at::Tensor wc, at::Tensor cache,
                  at::Tensor slots, double eps) {
  const auto dt = y.scalar_type();
  const int64_t T = y.size(0), no = out.size(1), ec = cache.size(-1);
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (dt == at::kBFloat16 || dt == at::kFloat) && out.dim() == 2 &&
              out.is_contiguous() && out.scalar_type() == dt &&
              out.size(0) == T && cache.is_contiguous() &&
              cache.scalar_type() == dt && slots.scalar_type() == at::kInt &&
              slots.is_contiguous() && slots.numel() == T,
              "latent_norms: tensors");
  // rows of both latents are padded to 8 columns in y
  TORCH_CHECK(nq >= 1 && nq <= no && nc >= 1 && nc <= ec && oq >= 0 &&
              oc >= 0 && oq % 8 == 0 && oc % 8 == 0 && no % 8 == 0 &&
              ec % 8 == 0 && y.size(1) % 8 == 0 &&
              oq + (nq + 7) / 8 * 8 <= y.size(1) &&
              oc + (nc + 7) / 8 * 8 <= y.size(1) &&
              wq.scalar_type() == at::kFloat && wq.is_contiguous() &&
              wq.numel() == nq && wc.scalar_type() == at::kFloat &&
              wc.is_contiguous() && wc.numel() == nc, "latent_norms: layout");
  if (swz.has_value())
    TORCH_CHECK(T <= 32 && no % 16 == 0 && swz->numel() == no * 32 &&
                swz->is_contiguous() && swz->scalar_type() == dt &&
                dt == at::kBFloat16, "latent_norms: operand");
  if (T == 0) return;
  const NormsArgs a{y.size(1), (int)oq, (int)nq, (int)no, (int)oc, (int)nc,
                    (int)ec, (float)eps};
  auto stream = at::hip::getCurrentHIPStream();
  auto launch = [&](auto tag) {
    using E = decltype(tag);
    hipLaunchKernelGGL((latent_norms_kernel<E>), dim3(T, 2), dim3(BLOCK), 0,
                       stream, (const E *)y.data_ptr(), wq.data_ptr<float>(),
                       wc.data_ptr<float>(), (E *)out.data_ptr(),
                       swz ? (E *)swz->data_ptr() : nullptr,
                       (E *)cache.data_ptr(), slots.data_ptr<int>(), a);
  };
  if (dt == at::kBFloat16) launch(uint16_t{});
  else launch(float{});
}

void head_gemm(at::Tensor x, int64_t x_off, int64_t xh, at::Tensor w,
               int64_t K, int64_t N, at::Tensor out, int64_t o_off, int64_t oh,
               c10::optional<at::Tensor> gate, int64_t g_off,
               c10::optional<at::Tensor> swz, int64_t T, int64_t H,
               bool head_gate) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && out.dim() == 2 &&
              x.stride(1) == 1 && out.stride(1) == 1 && w.is_contiguous() &&
              T <= x.size(0) && T <= out.size(0), "head_gemm: tensors");
  TORCH_CHECK(K % 8 == 0 && N % 8 == 0 && xh % 8 == 0 && oh % 8 == 0 &&
              x_off % 8 == 0 && o_off % 8 == 0 && g_off % 8 == 0 &&
              x.stride(0) % 8 == 0 && out.stride(0) % 8 == 0 &&
              x_off + (H - 1) * xh + K <= x.size(1) &&
              o_off + (H - 1) * oh + N <= out.size(1), "head_gemm: layout");
  const bool bf16 = x.scalar_type() == at::kBFloat16;
  TORCH_CHECK((bf16 || x.scalar_type() == at::kFloat) &&
              out.scalar_type() == x.scalar_type() &&
              w.scalar_type() == x.scalar_type(), "head_gemm: dtype");
  if (gate.has_value())
    TORCH_CHECK(gate->dim() == 2 && gate->stride(1) == 1 &&
                gate->stride(0) % 8 == 0 && T <= gate->size(0) &&
                g_off + (head_gate ? H : (H - 1) * oh + N) <=
                    gate->size(1) &&
                gate->scalar_type() == x.scalar_type(), "head_gemm: gate");
  if (swz.has_value())
    TORCH_CHECK(bf16 && T <= 32 && swz->is_contiguous() &&
                swz->numel() == out.size(1) * 32, "head_gemm: operand");
  if (T == 0) return;
  HeadArgs a{x_off, x.stride(0), o_off, out.stride(0), g_off,
             gate ? gate->stride(0) : 0, (int)xh, (int)oh, (int)K, (int)N,
             (int)T, (int)head_gate};
  auto stream = at::hip::getCurrentHIPStream();
  if (!bf16) {
    TORCH_CHECK(w.numel() == H * K * N, "head_gemm: weight");
    hipLaunchKernelGGL(head_gemm_f32_kernel,
                       dim3((N + 63) / 64, H, (T + 3) / 4), dim3(64, 4), 0,
                       stream, x.data_ptr<float>(), w.data_ptr<float>(),
                       out.data_ptr<float>(),
                       gate ? gate->data_ptr<float>() : nullptr, a);
    return;
  }
  const int64_t steps = (K + 31) / 32, nt = (N + 15) / 16;
  TORCH_CHECK(w.numel() == H * nt * steps * 512, "head_gemm: weight");
  const dim3 block(BLOCK);
  auto xp = (const uint16_t *)x.data_ptr();
  auto wp = (const uint16_t *)w.data_ptr();
  auto op = (uint16_t *)out.data_ptr();
  auto gp = gate ? (const uint16_t *)gate->data_ptr() : nullptr;
  auto sp = swz ? (uint16_t *)swz->data_ptr() : nullptr;
  const int mz = (int)(T + 31) / 32;
  if (steps >= 8)
    hipLaunchKernelGGL((head_gemm_kernel<true>), dim3(nt, H, mz), block, 0,
                       stream, xp, wp, op, gp, sp, a);
  else
    hipLaunchKernelGGL((head_gemm_kernel<false>), dim3((nt + 3) / 4, H, mz),
                       block, 0, stream, xp, wp, op, gp, sp, a);
}
