// Attention over the paged rows of shared_kv.h: long portions (gfx950, bf16).
//
// 128 query rows of one kv head per workgroup, 32 per wave; tiles of 64 keys
// (four pages, one per wave to load) in LDS, the next one on its way in
// registers. Scores are transposed (key x query) so a query's softmax lives
// on a lane pair; the same LDS rows serve as keys, read by rows, and as
// values, read by columns (ds_read_b64_tr_b16).
//
// With two maps 64 (token, head) pairs per workgroup: two waves take the first
// key's scores, two the second's, over the same tiles; the latter hand their
// result to the former through LDS, which subtract it and norm.
//
// Blocks of one kv head are `kv` apart in launch order, so with a head count
// divisible by the XCDs a head's keys stay in one L2.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "shared_kv.h"

namespace {

using namespace skv;

constexpr int BLOCK = 256;
constexpr int QB = 128;                // query rows per workgroup
constexpr int KB = 4 * PAGE;           // keys per tile
constexpr int SLACK = 512;             // LDS bytes past the tile

RB_DEV unsigned pack2(float lo, float hi) {
  union { __bf16 b[2]; unsigned u; } c;
  c.b[0] = (__bf16)lo;
  c.b[1] = (__bf16)hi;
  return c.u;
}

template <typename SZ>
__global__ __launch_bounds__(BLOCK, SZ::HCP > 128 ? 1 : 2)
void shared_kv_flash_kernel(Args a, int first_seq) {
  constexpr int HCP = SZ::HCP, NI = SZ::NI, MAPS = SZ::MAPS;
  constexpr int QSTEPS = SZ::HCK / 16;
  constexpr int DT = HCP / 32;
  constexpr int QR = QB / MAPS;                // (token, head) pairs

  extern __shared__ __attribute__((aligned(16))) char smem[];

  const int seq = first_seq + blockIdx.z;
  const int q_tok0 = a.cu_q[seq], nq = a.cu_q[seq + 1] - q_tok0;
  const int rows = nq * a.group;
  // the blocks with the most keys first
  const int q0 = (gridDim.y - 1 - blockIdx.y) * QR;
  if (q0 >= rows) return;
  const int rel = a.seq_lens[seq] - nq;        // retained position of query 0
  const int g = blockIdx.x;
  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int hi = lane >> 5, col = lane & 31;
  const int map = MAPS == 2 ? wid / 2 : 0;
  const int wrow = q0 + wid % (4 / MAPS) * 32;
  const int qi = wrow + col;                   // this lane's query row
  const bool q_ok = qi < rows;
  const int tok = (q_ok ? qi : 0) / a.group;
  const int head = g * a.group + (q_ok ? qi : 0) % a.group;
  const int qpos = rel + tok;
  const int dropped = dropped_of(a, q_tok0, rel);
  const u32x4v zero4 = (u32x4v)(0u);
  const int stride = row_stride(a.ec);

  // key range of the workgroup, and of this wave's queries
  const int wg_hi = rel + (min(rows, q0 + QR) - 1) / a.group + 1;
  const int wg_lo = max(0, first_key(a, rel + q0 / a.group, dropped));
  const int first = rel + wrow / a.group;
  const int last =
      wrow < rows ? rel + (min(rows, wrow + 32) - 1) / a.group : -1;
  // the first keys of the wave's first and last query, and of this lane's
  const int lo_first = first_key(a, first, dropped);
  const int lo_last = first_key(a, max(last, 0), dropped);
  const int kmin = first_key(a, qpos, dropped);
  const int tile0 = wg_lo / KB, tile1 = (wg_hi + KB - 1) / KB;
  const int page_hi = (wg_hi - 1) / PAGE;

  const int *table = a.tables + (int64_t)seq * a.table_width;
  const int64_t page_size = (int64_t)PAGE * a.ec;
  const uint16_t *cache = (const uint16_t *)a.cache + g * page_size;
  const PageCopy<NI> copy(lane, a.ec);
  u32x4v reg[NI];
  auto page_of = [&](int t) {
    return table[__builtin_amdgcn_readfirstlane(min(t * 4 + wid, page_hi))];
  };
  auto fetch = [&](int page) {
    copy.load(reg, cache + (int64_t)page * a.kv * page_size);
  };
  fetch(page_of(tile0));
  int next_page = page_of(tile0 + 1);

  bf16x8v qf[QSTEPS];
  {
    const uint16_t *qp = (const uint16_t *)a.y + (q_tok0 + tok) * a.ny +
                         (head * MAPS + map) * a.hc;
#pragma unroll
    for (int s = 0; s < QSTEPS; ++s) {
      const int d = s * 16 + hi * 8;
      union { u32x4v u; bf16x8v v; } c;
      c.u = (q_ok && d < a.hc) ? *reinterpret_cast<const u32x4v *>(qp + d)
                               : zero4;
      qf[s] = c.v;
    }
  }
  // columns past a row's end are read (times zero, or into columns that are
  // not kept): they must be finite
  for (int i = tid * 16; i < KB * stride + SLACK; i += BLOCK * 16)
    *reinterpret_cast<u32x4v *>(smem + i) = zero4;

  f32x16v acc[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) acc[d] = (f32x16v)(0.0f);
  float m_run = -INFINITY, l_run = 0.0f;
  if (a.sink != nullptr) {
    m_run = a.sink[head] * 1.4426950408889634f;
    l_run = hi == 0 ? 1.0f : 0.0f;             // the halves are added up
  }

  for (int t = tile0; t < tile1; ++t) {
    __syncthreads();
    copy.store(smem + wid * PAGE * stride, reg);
    __syncthreads();
    if (t + 1 < tile1) {
      fetch(next_page);
      next_page = page_of(t + 2);
    }

#pragma unroll
    for (int it = 0; it < 2; ++it) {
      const int k0 = t * KB + it * 32;
      if (k0 > last || k0 + 31 < lo_first) continue;          // wave-uniform
      f32x16v s = (f32x16v)(0.0f);
      const char *kp = smem + (it * 32 + col) * stride + hi * 16 +
                       map * a.hc * 2;
#pragma unroll
      for (int ks = 0; ks < QSTEPS; ++ks) {
        const bf16x8v kf = *reinterpret_cast<const bf16x8v *>(kp + ks * 32);
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[ks], s, 0, 0, 0);
      }
      float p[16];
#pragma unroll
      for (int r = 0; r < 16; ++r) p[r] = s[r] * a.scale;
      if (k0 + 31 > first || k0 < lo_last) {
        // some key of this sub-tile is hidden from some query
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = k0 + (r & 3) + 8 * (r >> 2) + 4 * hi;
          if (key > qpos || key < kmin) p[r] = -INFINITY;
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
        const float alpha = __builtin_amdgcn_exp2f(m_run - ref);
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
        // the order of the summed keys is free: the transposed reads of the
        // values follow the order of the scores
        union { unsigned u[4]; bf16x8v v; } pf;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          pf.u[i] = pack2(p[r0 + 2 * i], p[r0 + 2 * i + 1]);
        const int i = lane & 15;
        const char *vp =
            smem + (it * 32 + ks * 16 + 4 * hi + (i >> 2)) * stride +
            (a.voff + 16 * ((lane >> 4) & 1) + (i & 3) * 4) * 2;
#pragma unroll
        for (int d = 0; d < DT; ++d) {
          const bf16x8v vf =
              rb::lds_column8(vp + d * 64, vp + d * 64 + 8 * stride);
          acc[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf.v, acc[d],
                                                           0, 0, 0);
        }
      }
    }
  }

  const float l = l_run + __shfl_xor(l_run, 32, 64);
  float inv = a.out_scale / l;
  if constexpr (MAPS == 2) {
    f32x4v *ex = reinterpret_cast<f32x4v *>(smem) + wid % 2 * DT * 4 * 64 +
                 lane;
    __syncthreads();                           // the tile has been read
    if (map == 1) {
      const float f = a.lam[0] / l;
#pragma unroll
      for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int rq = 0; rq < 4; ++rq)
          ex[(d * 4 + rq) * 64] =
              (f32x4v){acc[d][rq * 4] * f, acc[d][rq * 4 + 1] * f,
                       acc[d][rq * 4 + 2] * f, acc[d][rq * 4 + 3] * f};
    }
    __syncthreads();
    if (map == 1) return;
    inv = 1.0f / l;
    float sum = 0.0f;
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
      for (int rq = 0; rq < 4; ++rq) {
        const f32x4v o2 = ex[(d * 4 + rq) * 64];
        const bool real = d * 32 + 8 * rq + 4 * hi < a.vc;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float o = acc[d][rq * 4 + e] * inv - o2[e];
          acc[d][rq * 4 + e] = o;
          sum += real ? o * o : 0.0f;
        }
      }
    sum += __shfl_xor(sum, 32, 64);
    inv = a.out_scale / sqrtf(sum / (float)a.count + a.eps);
  }
  if (!q_ok) return;
  uint16_t *zp = (uint16_t *)a.z + (q_tok0 + tok) * a.nz + head * a.vc;
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int rq = 0; rq < 4; ++rq) {
      const int c = d * 32 + 8 * rq + 4 * hi;
      if (c >= a.vc) continue;
      uint2 w;
      w.x = rb::pack_bf16x2(acc[d][rq * 4] * inv, acc[d][rq * 4 + 1] * inv);
      w.y = rb::pack_bf16x2(acc[d][rq * 4 + 2] * inv,
                            acc[d][rq * 4 + 3] * inv);
      *reinterpret_cast<uint2 *>(zp + c) = w;
    }
}

template <typename SZ>
void launch_flash(const Args &a, int first_seq, dim3 grid,
                  hipStream_t stream) {
  // a tile, or two waves' results
  constexpr size_t merge = SZ::MAPS == 1 ? 0 : (size_t)2 * SZ::HCP * 128;
  constexpr size_t most = std::max(
      merge, (size_t)KB * row_stride(SZ::MAPS == 1 ? 2 * SZ::HCP
                                     : 2 * SZ::HCK + SZ::HCP) + SLACK);
  static bool once = [] {
    return hipFuncSetAttribute(
               reinterpret_cast<const void *>(
                   &shared_kv_flash_kernel<SZ>),
               hipFuncAttributeMaxDynamicSharedMemorySize,
               (int)most) == hipSuccess;
  }();
  const size_t shmem =
      std::max(merge, (size_t)KB * row_stride(a.ec) + SLACK);
  TORCH_CHECK(once && shmem <= most, "shared_kv_flash: LDS size");
  hipLaunchKernelGGL((shared_kv_flash_kernel<SZ>), grid, dim3(BLOCK),
                     shmem, stream, a, first_seq);
}

}  // namespace

void check_mask(const at::Tensor &y, int64_t window, int64_t chunk,
                const c10::optional<at::Tensor> &positions,
                const c10::optional<at::Tensor> &sink, int64_t heads);
void check_maps(const c10::optional<at::Tensor> &lam, int64_t count,
                int64_t hc, int64_t voff, int64_t vc,
                const c10::optional<at::Tensor> &sink);

// Attention of the sequences first_seq .. first_seq + n_seqs - 1.
void shared_kv_flash(at::Tensor y, at::Tensor cache, at::Tensor block_tables,
                     at::Tensor cu_q, at::Tensor seq_lens, int64_t first_seq,
                     int64_t n_seqs, int64_t max_q, double scale,
                     int64_t window, int64_t heads, int64_t hc, int64_t voff,
                     at::Tensor z, int64_t chunk,
                     c10::optional<at::Tensor> positions,
                     c10::optional<at::Tensor> sink, double out_scale,
                     c10::optional<at::Tensor> lam, int64_t count,
                     double eps) {
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              y.scalar_type() == at::kBFloat16 && z.dim() == 2 &&
              z.is_contiguous() && z.size(0) == y.size(0) &&
              z.scalar_type() == at::kBFloat16, "shared_kv_flash: y, z");
  TORCH_CHECK(cache.dim() == 4 && cache.size(2) == PAGE &&
              cache.is_contiguous() && cache.scalar_type() == at::kBFloat16,
              "shared_kv_flash: cache [blocks, kv heads, 16, ec]");
  const int64_t G = cache.size(1), ec = cache.size(3), vc = ec - voff;
  const int64_t maps = lam.has_value() ? 2 : 1;
  TORCH_CHECK(heads % G == 0 && voff >= 0 && hc >= 8 && hc <= 256 &&
              hc % 8 == 0 && voff % 8 == 0 && voff <= maps * hc && hc <= ec &&
              vc >= 8 && vc <= 256 && ec % 8 == 0 &&
              y.size(1) % 8 == 0 && z.size(1) % 8 == 0 &&
              heads * maps * hc <= y.size(1) && heads * vc <= z.size(1),
              "shared_kv_flash: layout");
  check_mask(y, window, chunk, positions, sink, heads);
  check_maps(lam, count, hc, voff, vc, sink);
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.is_contiguous() &&
              block_tables.scalar_type() == at::kInt &&
              cu_q.scalar_type() == at::kInt && cu_q.is_contiguous() &&
              seq_lens.scalar_type() == at::kInt && seq_lens.is_contiguous() &&
              first_seq >= 0 && n_seqs <= 65535 &&
              block_tables.size(0) >= first_seq + n_seqs &&
              cu_q.numel() > first_seq + n_seqs &&
              seq_lens.numel() >= first_seq + n_seqs,
              "shared_kv_flash: batch tensors");
  if (n_seqs <= 0 || max_q == 0) return;
  Args a{};
  a.y = y.data_ptr();
  a.ny = y.size(1);
  a.cache = cache.data_ptr();
  a.tables = block_tables.data_ptr<int>();
  a.cu_q = cu_q.data_ptr<int>();
  a.seq_lens = seq_lens.data_ptr<int>();
  a.table_width = (int)block_tables.size(1);
  a.heads = (int)heads;
  a.kv = (int)G;
  a.group = (int)(heads / G);
  a.hc = (int)hc;
  a.vc = (int)vc;
  a.voff = (int)voff;
  a.ec = (int)ec;
  a.window = (int)window;
  a.chunk = (int)chunk;
  a.positions = chunk > 0 ? positions->data_ptr<int>() : nullptr;
  a.sink = sink ? sink->data_ptr<float>() : nullptr;
  a.out_scale = (float)out_scale;
  a.lam = lam ? lam->data_ptr<float>() : nullptr;
  a.count = (int)count;
  a.eps = (float)eps;
  a.scale = (float)(scale * 1.4426950408889634);
  a.z = z.data_ptr();
  a.nz = z.size(1);
  const int64_t rows = QB / maps;
  const int64_t blocks = (max_q * a.group + rows - 1) / rows;
  TORCH_CHECK(blocks <= 65535, "shared_kv_flash: portion of ", max_q);
  const dim3 grid(G, blocks, n_seqs);
  auto stream = at::hip::getCurrentHIPStream();
  auto go = [&](auto size) {
    launch_flash<decltype(size)>(a, (int)first_seq, grid, stream);
  };
  if (maps > 1) pick_sizes2((int)hc, (int)vc, go);
  else pick_sizes((int)std::max(hc, vc), (int)ec, go);
}
