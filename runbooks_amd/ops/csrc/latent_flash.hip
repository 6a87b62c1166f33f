// Flash attention of long prompt portions for latent attention (gfx950).
//
// Keys and values were expanded from the context's latents by one product:
// kv[key][h] = [ unrotated key (dimc) | value (vc) ]; the rotated key part,
// shared by all heads, is read from the context rows themselves
// (ctx[key][rc..]). Queries lie in y ([dimc | rotc] per head). The sigmoid
// output gate, per value column or per head, is applied to the result, which
// goes to z.
//
// 4 waves, each 32 query rows of one head; 64-key tiles in LDS (next tile
// prefetched to registers), scores transposed (key x query) so a query's
// softmax lives on a lane pair; values are read transposed from row-major
// LDS (ds_read_b64_tr_b16). Query i of a portion sits at key index rel + i
// and sees keys j with 0 <= rel + i - j < window (window 0: all earlier).
//
// Blocks of one head are 'heads' apart in launch order, so with a head count
// divisible by the XCDs a head's keys and values stay in one L2.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 256;
constexpr int QB = 128;                // query rows per workgroup
constexpr int KB = 64;                 // keys per tile

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8v;
typedef __attribute__((ext_vector_type(16))) float f32x16v;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4v;

struct FlashArgs {
  const uint16_t *y;                   // [T, ny]
  const uint16_t *kv;                  // [Tk, H, dimc + vc]
  const uint16_t *ctx;                 // [Tk, ec]
  const int *meta;                     // [n, 5]
  uint16_t *z;                         // [T, nz]
  const uint16_t *gate;                // [T, ng], from column off_g
  int64_t ny, nz, ng;
  int heads, dimc, rotc, vc, rc, ec, off_g, head_gate, window;
  float scale_log2e;
};

RB_DEV unsigned pack2(float lo, float hi) {
  union { __bf16 b[2]; unsigned u; } c;
  c.b[0] = (__bf16)lo;
  c.b[1] = (__bf16)hi;
  return c.u;
}

template <int DQ, int DV>
__global__ __launch_bounds__(BLOCK, 2) void latent_flash_kernel(FlashArgs a) {
  constexpr int QSTEPS = DQ / 16;
  constexpr int DT = DV / 32;
  constexpr int KSTRIDE = DQ * 2 + 16;         // bytes
  constexpr int VSTRIDE = DV * 2 + 64;
  constexpr int KC = DQ / 64, VC = DV / 64;    // chunks per lane and key

  extern __shared__ __attribute__((aligned(16))) char smem[];
  char *k_s = smem;                            // [KB][KSTRIDE]
  char *v_s = smem + KB * KSTRIDE;             // [KB][VSTRIDE]

  const int *mt = a.meta + blockIdx.z * 5;
  const int q_row0 = mt[0], nq = mt[1], k_row0 = mt[2], nk = mt[3],
            rel = mt[4];
  // the blocks with the most keys first
  const int q0 = (gridDim.y - 1 - blockIdx.y) * QB;
  if (q0 >= nq) return;
  const int h = blockIdx.x;
  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int hi = lane >> 5, col = lane & 31;
  const int qi = q0 + wid * 32 + col;          // this lane's query
  const bool q_ok = qi < nq;
  const int qpos = rel + qi;
  const int win = a.window > 0 ? a.window : (1 << 30);
  const u32x4v zero4 = (u32x4v)(0u);

  bf16x8v qf[QSTEPS];
  {
    const uint16_t *qp = a.y + (int64_t)(q_row0 + (q_ok ? qi : 0)) * a.ny +
                         h * (a.dimc + a.rotc);
#pragma unroll
    for (int s = 0; s < QSTEPS; ++s) {
      const int d = s * 16 + hi * 8;
      union { u32x4v u; bf16x8v v; } c;
      c.u = (q_ok && d < a.dimc + a.rotc)
                ? *reinterpret_cast<const u32x4v *>(qp + d) : zero4;
      qf[s] = c.v;
    }
  }

  // key range of the workgroup, and of this wave's queries
  const int wg_hi = min(nk, rel + min(nq, q0 + QB));
  const int wg_lo = max(0, rel + q0 - win + 1);
  const int first = rel + q0 + wid * 32;       // wave's first query position
  const int last = rel + min(nq, q0 + wid * 32 + 32) - 1;
  const int tile0 = wg_lo / KB, tile1 = (wg_hi + KB - 1) / KB;

  const int lkey = tid >> 3, lchunk = tid & 7;
  const int kvrow = a.heads * (a.dimc + a.vc);
  u32x4v kr[2][KC], vr[2][VC];
  // Branch-free: keys beyond the last one repeat it (masked), columns beyond
  // the real ones hold finite values (q is zero there, or they are not kept).
  auto fetch = [&](int t) {
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int64_t krow = k_row0 + min(t * KB + p * 32 + lkey, wg_hi - 1);
      const uint16_t *kvp = a.kv + krow * kvrow + h * (a.dimc + a.vc);
      const uint16_t *cp = a.ctx + krow * a.ec + a.rc - a.dimc;
#pragma unroll
      for (int i = 0; i < KC; ++i) {
        const int d = (lchunk + i * 8) * 8;
        kr[p][i] = *reinterpret_cast<const u32x4v *>(
            d < a.dimc ? kvp + d : d < a.dimc + a.rotc ? cp + d : kvp);
      }
#pragma unroll
      for (int i = 0; i < VC; ++i) {
        const int d = (lchunk + i * 8) * 8;
        vr[p][i] = *reinterpret_cast<const u32x4v *>(
            kvp + a.dimc + (d < a.vc ? d : 0));
      }
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int key = p * 32 + lkey;
#pragma unroll
      for (int i = 0; i < KC; ++i) {
        const int d = (lchunk + i * 8) * 8;
        *reinterpret_cast<u32x4v *>(k_s + key * KSTRIDE + d * 2) = kr[p][i];
      }
#pragma unroll
      for (int i = 0; i < VC; ++i) {
        const int d = (lchunk + i * 8) * 8;
        *reinterpret_cast<u32x4v *>(v_s + key * VSTRIDE + d * 2) = vr[p][i];
      }
    }
  };

  f32x16v acc[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) acc[d] = (f32x16v)(0.0f);
  float m_run = -INFINITY, l_run = 0.0f;

  fetch(tile0);
  for (int t = tile0; t < tile1; ++t) {
    __syncthreads();
    stage();
    __syncthreads();
    if (t + 1 < tile1) fetch(t + 1);

#pragma unroll
    for (int it = 0; it < 2; ++it) {
      const int k0 = t * KB + it * 32;
      if (k0 > last || k0 + 31 < first - win + 1) continue;   // wave-uniform
      f32x16v s = (f32x16v)(0.0f);
#pragma unroll
      for (int ks = 0; ks < QSTEPS; ++ks) {
        const bf16x8v kf = *reinterpret_cast<const bf16x8v *>(
            k_s + (it * 32 + col) * KSTRIDE + (ks * 16 + hi * 8) * 2);
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[ks], s, 0, 0, 0);
      }
      float p[16];
#pragma unroll
      for (int r = 0; r < 16; ++r) p[r] = s[r] * a.scale_log2e;
      if (k0 + 31 > first || k0 < last - win + 1) {
        // some key of this sub-tile is hidden from some query
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int d = qpos - (k0 + (r & 3) + 8 * (r >> 2) + 4 * hi);
          if (d < 0 || d >= win) p[r] = -INFINITY;
        }
      }
      float mx = p[0];
#pragma unroll
      for (int r = 1; r < 16; ++r) mx = fmaxf(mx, p[r]);
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m_run, mx);
      // rows that have seen no key yet keep a finite reference
      const float ref = mn == -INFINITY ? 0.0f : mn;
      if (__any(mn > m_run)) {
        const float alpha = exp2f(m_run - ref);
        l_run *= alpha;
#pragma unroll
        for (int d = 0; d < DT; ++d)
#pragma unroll
          for (int r = 0; r < 16; ++r) acc[d][r] *= alpha;
        m_run = mn;
      }
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        p[r] = __builtin_amdgcn_exp2f(p[r] - ref);
        l_run += p[r];
      }
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const int r0 = ks * 8;
        const unsigned w0 = pack2(p[r0], p[r0 + 1]);
        const unsigned w1 = pack2(p[r0 + 2], p[r0 + 3]);
        const unsigned w2 = pack2(p[r0 + 4], p[r0 + 5]);
        const unsigned w3 = pack2(p[r0 + 6], p[r0 + 7]);
        auto x02 = __builtin_amdgcn_permlane32_swap(w0, w2, false, false);
        auto x13 = __builtin_amdgcn_permlane32_swap(w1, w3, false, false);
        union { unsigned u[4]; bf16x8v v; } pf;
        pf.u[0] = x02[0];
        pf.u[1] = x13[0];
        pf.u[2] = x02[1];
        pf.u[3] = x13[1];
        const int g = lane >> 4, i = lane & 15;
        const char *vp =
            v_s + (it * 32 + ks * 16 + 8 * (g >> 1) + (i >> 2)) * VSTRIDE +
            (16 * (g & 1) + (i & 3) * 4) * 2;
#pragma unroll
        for (int d = 0; d < DT; ++d) {
          const bf16x8v vf = rb::lds_column8(vp + d * 64, vp + d * 64 + 4 * VSTRIDE);
          acc[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf.v, acc[d],
                                                           0, 0, 0);
        }
      }
    }
  }

  if (!q_ok) return;
  const float l = l_run + __shfl_xor(l_run, 32, 64);
  const float inv = l > 0.0f ? 1.0f / l : 0.0f;
  const int64_t t = q_row0 + qi;
  const uint16_t *gp = a.gate + t * a.ng + a.off_g;
  const uint32_t one = a.head_gate ? gp[h] * 0x10001u : 0;
  gp += h * a.vc;
  uint16_t *zp = a.z + t * a.nz + h * a.vc;
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int rq = 0; rq < 4; ++rq) {
      const int c = d * 32 + 8 * rq + 4 * hi;
      if (c >= a.vc) continue;
      uint2 gw = make_uint2(one, one);
      if (!a.head_gate) gw = *reinterpret_cast<const uint2 *>(gp + c);
      const uint32_t gu[2] = {gw.x, gw.y};
      float o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float g =
            rb::bf16_to_f32((uint16_t)(gu[e >> 1] >> (16 * (e & 1))));
        o[e] = acc[d][rq * 4 + e] * inv / (1.0f + __expf(-g));
      }
      uint2 w;
      w.x = rb::pack_bf16x2(o[0], o[1]);
      w.y = rb::pack_bf16x2(o[2], o[3]);
      *reinterpret_cast<uint2 *>(zp + c) = w;
    }
}

template <int DQ, int DV>
void launch_flash(const FlashArgs &a, dim3 grid, hipStream_t stream) {
  constexpr size_t shmem = KB * (DQ * 2 + 16) + KB * (DV * 2 + 64);
  static bool once = [] {
    return hipFuncSetAttribute(
               reinterpret_cast<const void *>(&latent_flash_kernel<DQ, DV>),
               hipFuncAttributeMaxDynamicSharedMemorySize,
               (int)shmem) == hipSuccess;
  }();
  TORCH_CHECK(once, "latent_flash: LDS size");
  hipLaunchKernelGGL((latent_flash_kernel<DQ, DV>), grid, dim3(BLOCK), shmem,
                     stream, a);
}

}  // namespace

void latent_flash(at::Tensor y, at::Tensor kv, at::Tensor ctx, at::Tensor meta,
                  at::Tensor z, int64_t heads, int64_t dimc, int64_t rotc,
                  int64_t vc, int64_t rc, at::Tensor gate, int64_t off_g,
                  bool head_gate, int64_t max_q, double scale,
                  int64_t window) {
  TORCH_CHECK(y.is_cuda() && y.is_contiguous() && kv.is_contiguous() &&
              ctx.is_contiguous() && z.is_contiguous() &&
              meta.is_contiguous() && y.dim() == 2 && z.dim() == 2,
              "latent_flash: contiguous GPU tensors");
  TORCH_CHECK(y.scalar_type() == at::kBFloat16 &&
              kv.scalar_type() == at::kBFloat16 &&
              ctx.scalar_type() == at::kBFloat16 &&
              z.scalar_type() == at::kBFloat16 &&
              meta.scalar_type() == at::kInt, "latent_flash: dtypes");
  TORCH_CHECK(dimc % 8 == 0 && rotc % 8 == 0 && vc % 8 == 0 && rc % 8 == 0 &&
              off_g % 8 == 0 && y.size(1) % 8 == 0 && z.size(1) % 8 == 0 &&
              heads * (dimc + rotc) <= y.size(1) &&
              heads * vc <= z.size(1) &&
              kv.size(-1) == heads * (dimc + vc) && kv.size(0) == ctx.size(0) &&
              ctx.dim() == 2 && ctx.size(1) == rc + rotc &&
              y.size(0) == z.size(0) && meta.dim() == 2 && meta.size(1) == 5,
              "latent_flash: layout");
  TORCH_CHECK(gate.dim() == 2 && gate.is_contiguous() &&
              gate.scalar_type() == at::kBFloat16 &&
              gate.size(0) == y.size(0) && gate.size(1) % 8 == 0 &&
              off_g >= 0 && off_g + heads * (head_gate ? 1 : vc) <=
              gate.size(1), "latent_flash: gate");
  FlashArgs a{(const uint16_t *)y.data_ptr(), (const uint16_t *)kv.data_ptr(),
              (const uint16_t *)ctx.data_ptr(), meta.data_ptr<int>(),
              (uint16_t *)z.data_ptr(), (const uint16_t *)gate.data_ptr(),
              y.size(1), z.size(1), gate.size(1), (int)heads, (int)dimc,
              (int)rotc, (int)vc, (int)rc, (int)ctx.size(1), (int)off_g,
              (int)head_gate, (int)window,
              (float)(scale * 1.4426950408889634)};
  const dim3 grid(heads, (max_q + QB - 1) / QB, meta.size(0));
  auto stream = at::hip::getCurrentHIPStream();
  const int64_t dq = dimc + rotc;
  if (dq <= 64 && vc <= 64) launch_flash<64, 64>(a, grid, stream);
  else if (dq <= 128 && vc <= 64) launch_flash<128, 64>(a, grid, stream);
  else if (dq <= 128 && vc <= 128) launch_flash<128, 128>(a, grid, stream);
  else if (dq <= 192 && vc <= 128) launch_flash<192, 128>(a, grid, stream);
  else if (dq <= 256 && vc <= 256) launch_flash<256, 256>(a, grid, stream);
  else TORCH_CHECK(false, "latent_flash: head sizes ", dq, ", ", vc);
}
