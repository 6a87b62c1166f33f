// Attention over the paged rows of shared_kv.h: decoding and short portions
// (gfx950).
//
// MFMA kernel (bf16): 16 query rows of one kv head per workgroup. Each of the
// 4 waves walks tiles of 32 keys (two pages) of its own, through its own LDS,
// without barriers: S^T = K Q^T leaves a lane 8 scores of one query row,
// which are, exponentiated and packed, the lane's operand of O^T += V^T P^T
// as they stand (the order of the summed keys is free, so the transposed
// reads of V follow the order of the scores). The waves' partial results are
// merged at the end; `nsplit` workgroups may share a sequence's keys, merged
// by shared_kv_combine. With two maps a row's query stands in its own key's
// columns, zeros in the other's, so rows of both share a tile; their results
// meet in shared_kv_diff_combine.
//
// The scalar kernel covers fp32 and head sizes beyond 256: one workgroup per
// row, a wave per key, lanes across the columns.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "shared_kv.h"

namespace {

using namespace skv;

constexpr int BLOCK = 256;
constexpr int WAVES = 4;
constexpr int TK = 2 * PAGE;           // keys per tile
constexpr int M = 16;                  // query rows per workgroup
constexpr int SLACK = 512;             // LDS bytes past a wave's tile
constexpr size_t MAX_LDS = 158 * 1024;

__host__ __device__ constexpr int wave_bytes(int ec) {
  return TK * row_stride(ec) + SLACK;
}

// orders a wave's own LDS accesses
RB_DEV void wave_fence() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

template <typename SZ>
__global__ __launch_bounds__(BLOCK) void shared_kv_attend_kernel(Args a) {
  constexpr int HCP = SZ::HCP, NI = SZ::NI;
  constexpr int KS = SZ::MAPS * SZ::HCK / 32;  // QK steps
  constexpr int DT = HCP / 16;                 // column tiles of the result
  constexpr int OSTRIDE = HCP + 4;             // floats

  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float ml_s[WAVES][M][2];
  __shared__ float out_s[M][2];                // m, l of the workgroup

  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int l16 = lane & 15, grp = lane >> 4;
  const int split = blockIdx.x, seq = blockIdx.z;
  const int g = blockIdx.y % a.kv, row0 = blockIdx.y / a.kv * M;
  const int q0 = a.cu_q[seq], nq = a.cu_q[seq + 1] - q0;
  const int n_keys = a.seq_lens[seq];
  const int rows = nq * a.group;
  if (row0 >= rows) return;
  const int v0 = n_keys - nq;                  // retained position of query 0
  const int tok_lo = row0 / a.group;
  const int tok_hi = (min(row0 + M, rows) - 1) / a.group;
  const int key_hi = v0 + tok_hi + 1;
  const int dropped = dropped_of(a, q0, v0);
  const int key_lo = max(0, first_key(a, v0 + tok_lo, dropped));
  const int page_lo = key_lo / PAGE, page_hi = (key_hi - 1) / PAGE;
  const int tiles = (page_hi - page_lo + 2) / 2;
  // short contexts use fewer splits: at least a tile per wave
  const int per = max(WAVES, (tiles + a.nsplit - 1) / a.nsplit);
  const int t0 = split * per, t1 = min(tiles, t0 + per);

  // global row (token * heads + head) of this workgroup's row m
  auto global_row = [&](int m) {
    const int r = row0 + m;
    return (int64_t)(q0 + r / a.group) * a.heads + g * a.group + r % a.group;
  };
  if (t0 >= t1) {                              // nothing left for this split
    if (a.part_o != nullptr && tid < min(M, rows - row0)) {
      float *ml =
          a.part_ml + ((int64_t)split * a.total_rows + global_row(tid)) * 2;
      ml[0] = -INFINITY;
      ml[1] = 0.0f;
    }
    return;
  }

  const int stride = row_stride(a.ec);
  char *tile = smem + wid * wave_bytes(a.ec);
  const int *table = a.tables + (int64_t)seq * a.table_width;
  const int64_t page_size = (int64_t)PAGE * a.ec;
  const uint16_t *cache = (const uint16_t *)a.cache + g * page_size;
  const PageCopy<NI> copy(lane, a.ec);
  u32x4v reg[2][NI];
  auto fetch = [&](int t) {
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int i = min(page_lo + t * 2 + p, page_hi);
      const int page = table[__builtin_amdgcn_readfirstlane(i)];
      copy.load(reg[p], cache + (int64_t)page * a.kv * page_size);
    }
  };
  int t = t0 + wid;
  if (t < t1) fetch(t);

  // columns past a row's end are read (times zero, or into columns that are
  // not kept): they must be finite
  for (int i = lane * 16; i < wave_bytes(a.ec); i += 64 * 16)
    *reinterpret_cast<u32x4v *>(tile + i) = (u32x4v)(0u);

  // this lane's query row
  const int row = row0 + l16;
  const bool row_ok = row < rows;
  const int qpos = row_ok ? v0 + row / a.group : -1;
  const int kmin = first_key(a, max(qpos, 0), dropped);
  bf16x8v qf[KS];
  {
    const int64_t gr = global_row(row_ok ? l16 : 0);
    const uint16_t *qp = (const uint16_t *)a.y + gr / a.heads * a.ny +
                         gr % a.heads * a.hc;
    const int at = SZ::MAPS > 1 ? (int)(gr % SZ::MAPS) * a.hc : 0;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int c = s * 32 + grp * 8 - at;
      union { u32x4v u; bf16x8v v; } q;
      q.u = row_ok && c >= 0 && c < a.hc
                ? *reinterpret_cast<const u32x4v *>(qp + c) : (u32x4v)(0u);
      qf[s] = q.v;
    }
  }

  f32x4v acc[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) acc[d] = (f32x4v)(0.0f);
  float m_run = -INFINITY, l_run = 0.0f;
  if (a.sink != nullptr && split == 0 && wid == 0 && row_ok) {
    // counts once: l_run is summed over the lane groups
    m_run = a.sink[g * a.group + row % a.group] * 1.4426950408889634f;
    l_run = grp == 0 ? 1.0f : 0.0f;
  }

  for (; t < t1; t += WAVES) {
    wave_fence();                              // the last tile has been read
    copy.store(tile, reg[0]);
    copy.store(tile + PAGE * stride, reg[1]);
    if (t + WAVES < t1) fetch(t + WAVES);
    wave_fence();

    f32x4v s[2] = {(f32x4v)(0.0f), (f32x4v)(0.0f)};
    const char *kp = tile + l16 * stride + grp * 16;
#pragma unroll
    for (int k = 0; k < KS; ++k)
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const bf16x8v kf = *reinterpret_cast<const bf16x8v *>(
            kp + h * PAGE * stride + k * 64);
        s[h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[k], s[h], 0, 0,
                                                       0);
      }
    float p[8], mx = -INFINITY;
    const int key0 = (page_lo + t * 2) * PAGE + grp * 4;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int key = key0 + (i >> 2) * PAGE + (i & 3);
      p[i] = key <= qpos && key >= kmin ? s[i >> 2][i & 3] * a.scale
                                        : -INFINITY;
      mx = fmaxf(mx, p[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx);
    // rows that have seen no key yet keep a finite reference
    const float ref = m_new == -INFINITY ? 0.0f : m_new;
    const float alpha = __builtin_amdgcn_exp2f(m_run - ref);
    float sum = 0.0f;
    union { uint32_t u[4]; bf16x8v v; } pf;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      p[i] = __builtin_amdgcn_exp2f(p[i] - ref);
      sum += p[i];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      pf.u[i] = rb::pack_bf16x2(p[2 * i], p[2 * i + 1]);
    l_run = l_run * alpha + sum;
    m_run = m_new;
    const char *vp = tile + (grp * 4 + (l16 >> 2)) * stride +
                     (a.voff + (l16 & 3) * 4) * 2;
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      const bf16x8v vf =
          rb::lds_column8(vp + d * 32, vp + PAGE * stride + d * 32);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[d][r] *= alpha;
      acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf.v, acc[d], 0, 0,
                                                       0);
    }
  }

  // ---- merge the waves ----------------------------------------------------
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (grp == 0) {
    ml_s[wid][l16][0] = m_run;
    ml_s[wid][l16][1] = l_run;
  }
  __syncthreads();                             // the tiles are free, too
  float mx = -INFINITY, l = 0.0f;
#pragma unroll
  for (int w = 0; w < WAVES; ++w) mx = fmaxf(mx, ml_s[w][l16][0]);
  const float ref = mx == -INFINITY ? 0.0f : mx;
#pragma unroll
  for (int w = 0; w < WAVES; ++w)
    l += ml_s[w][l16][1] * __builtin_amdgcn_exp2f(ml_s[w][l16][0] - ref);
  const float f = __builtin_amdgcn_exp2f(m_run - ref);
  float *o_s = reinterpret_cast<float *>(smem);  // [WAVES][M][OSTRIDE]
#pragma unroll
  for (int d = 0; d < DT; ++d) {
    f32x4v o;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] = acc[d][r] * f;
    *reinterpret_cast<f32x4v *>(o_s + (wid * M + l16) * OSTRIDE + d * 16 +
                                grp * 4) = o;
  }
  if (wid == 0 && grp == 0) {
    out_s[l16][0] = mx;
    out_s[l16][1] = l;
    if (a.part_o != nullptr && row_ok) {
      float *ml =
          a.part_ml + ((int64_t)split * a.total_rows + global_row(l16)) * 2;
      ml[0] = mx;
      ml[1] = l;
    }
  }
  __syncthreads();
  const int quads = a.vc / 4;
  for (int i = tid; i < M * quads; i += BLOCK) {
    const int m = i / quads, c = (i - m * quads) * 4;
    if (row0 + m >= rows) break;
    f32x4v o = (f32x4v)(0.0f);
#pragma unroll
    for (int w = 0; w < WAVES; ++w)
      o += *reinterpret_cast<const f32x4v *>(o_s + (w * M + m) * OSTRIDE + c);
    const int64_t gr = global_row(m);
    if (a.part_o != nullptr) {
      *reinterpret_cast<f32x4v *>(
          a.part_o + ((int64_t)split * a.total_rows + gr) * a.vc + c) = o;
    } else {
      const float inv = a.out_scale / out_s[m][1];
      const float v[4] = {o[0] * inv, o[1] * inv, o[2] * inv, o[3] * inv};
      store4(a, gr / a.heads, (int)(gr % a.heads) * a.vc + c, v);
    }
  }
}

// One block per row merges the splits (at most 64); splits without keys get
// weight 0.
__global__ __launch_bounds__(64) void shared_kv_combine_kernel(Args a) {
  const int64_t row = blockIdx.x;
  const int lane = threadIdx.x;
  float m = -INFINITY, l = 0.0f;
  if (lane < a.nsplit) {
    const float2 ml = *reinterpret_cast<const float2 *>(
        a.part_ml + ((int64_t)lane * a.total_rows + row) * 2);
    m = ml.x;
    l = ml.y;
  }
  const float mx = rb::wave_reduce_max(m);
  float w = l > 0.0f ? __builtin_amdgcn_exp2f(m - mx) : 0.0f;
  w *= a.out_scale / rb::wave_reduce_sum(l * w);
  __shared__ float w_s[64];
  w_s[lane] = w;
  __syncthreads();
  for (int c = lane * 4; c < a.vc; c += 256) {
    float o[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int s = 0; s < a.nsplit; ++s) {
      const float ws = w_s[s];
      if (ws == 0.0f) continue;                // its part was not written
      const f32x4v p = *reinterpret_cast<const f32x4v *>(
          a.part_o + ((int64_t)s * a.total_rows + row) * a.vc + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] += ws * p[e];
    }
    store4(a, row / a.heads, (int)(row % a.heads) * a.vc + c, o);
  }
}

// One block per token and head merges the splits of its two maps, subtracts the
// second one's result and norms.
__global__ __launch_bounds__(64) void shared_kv_diff_combine_kernel(Args a) {
  constexpr int NV = 4;                        // vc <= 1024
  const int64_t row = blockIdx.x * (int64_t)2;
  const int lane = threadIdx.x;
  __shared__ float w_s[2][64];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    float m = -INFINITY, l = 0.0f;
    if (lane < a.nsplit) {
      const float2 ml = *reinterpret_cast<const float2 *>(
          a.part_ml + ((int64_t)lane * a.total_rows + row + i) * 2);
      m = ml.x;
      l = ml.y;
    }
    const float mx = rb::wave_reduce_max(m);
    float w = l > 0.0f ? __builtin_amdgcn_exp2f(m - mx) : 0.0f;
    w /= rb::wave_reduce_sum(l * w);
    w_s[i][lane] = i == 0 ? w : -a.lam[0] * w;
  }
  __syncthreads();
  float o[NV][4] = {}, sum = 0.0f;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int c = (v * 64 + lane) * 4;
    if (c >= a.vc) continue;
    for (int s = 0; s < a.nsplit; ++s)
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const float ws = w_s[i][s];
        if (ws == 0.0f) continue;              // its part may be unwritten
        const f32x4v p = *reinterpret_cast<const f32x4v *>(
            a.part_o + ((int64_t)s * a.total_rows + row + i) * a.vc + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) o[v][e] += ws * p[e];
      }
#pragma unroll
    for (int e = 0; e < 4; ++e) sum += o[v][e] * o[v][e];
  }
  sum = rb::wave_reduce_sum(sum);
  const float f = a.out_scale / sqrtf(sum / (float)a.count + a.eps);
  const int64_t t = row / a.heads;
  const int col = (int)(row % a.heads) / 2 * a.vc;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int c = (v * 64 + lane) * 4;
    if (c >= a.vc) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[v][e] *= f;
    if (a.f32)
      *reinterpret_cast<f32x4v *>((float *)a.z + t * a.nz + col + c) =
          (f32x4v){o[v][0], o[v][1], o[v][2], o[v][3]};
    else
      store4(a, t, col + c, o[v]);
  }
}

// ---------------------------------------------------------------------------
// scalar kernel: block = one (token, head) row, wave = every fourth key
// ---------------------------------------------------------------------------
template <typename T, int NE>
__global__ __launch_bounds__(BLOCK) void shared_kv_rows_kernel(Args a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float *o_s = reinterpret_cast<float *>(smem);        // [4][vc]
  __shared__ float ml_s[4][2];
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int seq = blockIdx.y;
  const int q0 = a.cu_q[seq], nq = a.cu_q[seq + 1] - q0;
  if ((int)blockIdx.x >= nq * a.heads) return;
  const int tok = blockIdx.x / a.heads, head = blockIdx.x % a.heads;
  const int g = head / a.group;
  const int qpos = a.seq_lens[seq] - nq + tok;
  const int v0 = a.seq_lens[seq] - nq;
  const int lo = max(0, first_key(a, qpos, dropped_of(a, q0, v0)));
  const T *qp = (const T *)a.y + (q0 + tok) * a.ny + head * a.hc;
  const int koff = a.lam != nullptr ? head % 2 * a.hc : 0;
  const int *table = a.tables + (int64_t)seq * a.table_width;

  float q[NE], o[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + i * 64;
    q[i] = e < a.hc ? rb::bf16_to_f32_or_id(qp[e]) : 0.0f;
    o[i] = 0.0f;
  }
  float m = -INFINITY, l = 0.0f;
  if (a.sink != nullptr && wid == 0) {
    m = a.sink[head];
    l = 1.0f;
  }
  for (int key = lo + wid; key <= qpos; key += 4) {
    const T *c = (const T *)a.cache +
                 (((int64_t)table[key / PAGE] * a.kv + g) * PAGE + key % PAGE) *
                     a.ec;
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = lane + i * 64;
      if (e < a.hc) s = fmaf(q[i], rb::bf16_to_f32_or_id(c[koff + e]), s);
    }
    s = rb::wave_reduce_sum(s) * a.scale;
    const float mn = fmaxf(m, s);
    const float al = expf(m - mn), p = expf(s - mn);
    l = l * al + p;
    m = mn;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = lane + i * 64;
      if (e < a.vc)
        o[i] = o[i] * al + p * rb::bf16_to_f32_or_id(c[a.voff + e]);
    }
  }
  if (lane == 0) {
    ml_s[wid][0] = m;
    ml_s[wid][1] = l;
  }
#pragma unroll
  for (int i = 0; i < NE; ++i)
    if (lane + i * 64 < a.vc) o_s[wid * a.vc + lane + i * 64] = o[i];
  __syncthreads();
  float mx = -INFINITY, lt = 0.0f, w[4];
#pragma unroll
  for (int k = 0; k < 4; ++k) mx = fmaxf(mx, ml_s[k][0]);
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    w[k] = ml_s[k][1] > 0.0f ? expf(ml_s[k][0] - mx) : 0.0f;
    lt += w[k] * ml_s[k][1];
  }
  const int64_t gr = (int64_t)(q0 + tok) * a.heads + head;
  if (a.part_o != nullptr && threadIdx.x == 0) {
    a.part_ml[gr * 2] = mx;
    a.part_ml[gr * 2 + 1] = lt;
  }
  for (int e = threadIdx.x; e < a.vc; e += BLOCK) {
    float v = 0.0f;
#pragma unroll
    for (int k = 0; k < 4; ++k) v += w[k] * o_s[k * a.vc + e];
    if (a.part_o != nullptr) {
      a.part_o[gr * a.vc + e] = v;
      continue;
    }
    v *= a.out_scale / lt;
    const int col = head * a.vc + e;
    rb::store_scalar((T *)a.z + (q0 + tok) * a.nz + col, v);
    if constexpr (sizeof(T) == 2) {
      if (a.swz != nullptr)
        a.swz[operand_at(col & ~7, q0 + tok) + (col & 7)] = rb::f32_to_bf16(v);
    }
  }
}

template <typename SZ>
void launch_attend(const Args &a, dim3 grid, hipStream_t stream) {
  constexpr int HCP = SZ::HCP;
  const size_t tiles = (size_t)WAVES * wave_bytes(a.ec);
  const size_t merge = (size_t)WAVES * M * (HCP + 4) * sizeof(float);
  const size_t shmem = std::max(tiles, merge);
  constexpr size_t most = std::min(
      MAX_LDS, std::max((size_t)WAVES * wave_bytes(SZ::MAPS == 1 ? 2 * HCP
                                                   : 2 * SZ::HCK + HCP),
                        (size_t)WAVES * M * (HCP + 4) * sizeof(float)));
  static bool once = [] {
    return hipFuncSetAttribute(
               reinterpret_cast<const void *>(
                   &shared_kv_attend_kernel<SZ>),
               hipFuncAttributeMaxDynamicSharedMemorySize,
               (int)most) == hipSuccess;
  }();
  TORCH_CHECK(once && shmem <= most, "shared_kv_attend: LDS size");
  hipLaunchKernelGGL((shared_kv_attend_kernel<SZ>), grid, dim3(BLOCK),
                     shmem, stream, a);
}

}  // namespace

// The mask and the sink as both entry points take them.
void check_mask(const at::Tensor &y, int64_t window, int64_t chunk,
                const c10::optional<at::Tensor> &positions,
                const c10::optional<at::Tensor> &sink, int64_t heads) {
  TORCH_CHECK(window >= 0 && chunk >= 0 && (window == 0 || chunk == 0),
              "shared_kv: window ", window, ", chunk ", chunk);
  if (chunk > 0)
    TORCH_CHECK(positions.has_value() && positions->is_cuda() &&
                positions->scalar_type() == at::kInt &&
                positions->is_contiguous() &&
                positions->numel() == y.size(0), "shared_kv: positions");
  if (sink.has_value())
    TORCH_CHECK(sink->is_cuda() && sink->scalar_type() == at::kFloat &&
                sink->is_contiguous() && sink->numel() == heads,
                "shared_kv: sink [heads] f32");
}

// Two maps: their norm's columns and the row's layout.
void check_maps(const c10::optional<at::Tensor> &lam, int64_t count,
                int64_t hc, int64_t voff, int64_t vc,
                const c10::optional<at::Tensor> &sink) {
  if (!lam.has_value()) return;
  TORCH_CHECK(lam->is_cuda() && lam->scalar_type() == at::kFloat &&
              lam->numel() == 1 && voff == 2 * hc && count >= 1 &&
              count <= vc && !sink.has_value(), "shared_kv: two maps");
}

// Attention of the first n_seqs sequences, whose t_seqs tokens are the first
// ones of y; the heads' results go to z's first columns, and to the decode
// operand `swz` when given.
void shared_kv_attend(at::Tensor y, at::Tensor cache, at::Tensor block_tables,
                      at::Tensor cu_q, at::Tensor seq_lens, int64_t n_seqs,
                      int64_t t_seqs, int64_t max_q, int64_t nsplit,
                      double scale, int64_t window, int64_t heads,
                      int64_t hc, int64_t voff, at::Tensor z,
                      c10::optional<at::Tensor> swz, int64_t chunk,
                      c10::optional<at::Tensor> positions,
                      c10::optional<at::Tensor> sink, double out_scale,
                      c10::optional<at::Tensor> lam, int64_t count,
                      double eps) {
  const auto dt = y.scalar_type();
  const bool bf16 = dt == at::kBFloat16;
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (bf16 || dt == at::kFloat) && z.dim() == 2 &&
              z.is_contiguous() && z.size(0) == y.size(0) &&
              z.scalar_type() == dt, "shared_kv_attend: y, z");
  TORCH_CHECK(cache.dim() == 4 && cache.size(2) == PAGE &&
              cache.is_contiguous() && cache.scalar_type() == dt,
              "shared_kv_attend: cache [blocks, kv heads, 16, ec]");
  const int64_t T = y.size(0), G = cache.size(1), ec = cache.size(3);
  const int64_t vc = ec - voff, wide = std::max(hc, vc);
  const int64_t maps = lam.has_value() ? 2 : 1;
  TORCH_CHECK(heads % G == 0 && voff >= 0 && hc >= 8 && hc % 8 == 0 &&
              voff % 8 == 0 && voff <= maps * hc && hc <= ec && vc >= 8 &&
              ec % 8 == 0 && y.size(1) % 8 == 0 &&
              z.size(1) % 8 == 0 && heads * maps * hc <= y.size(1) &&
              heads * vc <= z.size(1), "shared_kv_attend: layout");
  check_mask(y, window, chunk, positions, sink, heads);
  check_maps(lam, count, hc, voff, vc, sink);
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.is_contiguous() &&
              block_tables.scalar_type() == at::kInt &&
              cu_q.scalar_type() == at::kInt && cu_q.is_contiguous() &&
              seq_lens.scalar_type() == at::kInt && seq_lens.is_contiguous() &&
              block_tables.size(0) >= n_seqs && cu_q.numel() > n_seqs &&
              seq_lens.numel() >= n_seqs, "shared_kv_attend: batch tensors");
  TORCH_CHECK(T * heads * maps < (1 << 30) && n_seqs <= 65535 && t_seqs <= T,
              "shared_kv_attend: rows");
  if (swz.has_value())
    TORCH_CHECK(bf16 && T <= 32 && swz->is_contiguous() &&
                swz->numel() == z.size(1) * 32, "shared_kv_attend: operand");
  if (t_seqs == 0 || n_seqs == 0 || max_q == 0) return;

  Args a{};
  a.y = y.data_ptr();
  a.ny = y.size(1);
  a.cache = cache.data_ptr();
  a.tables = block_tables.data_ptr<int>();
  a.cu_q = cu_q.data_ptr<int>();
  a.seq_lens = seq_lens.data_ptr<int>();
  a.table_width = (int)block_tables.size(1);
  a.heads = (int)(heads * maps);       // a map counts as a head
  a.kv = (int)G;
  a.group = (int)(heads * maps / G);
  a.hc = (int)hc;
  a.vc = (int)vc;
  a.voff = (int)voff;
  a.ec = (int)ec;
  a.window = (int)window;
  a.chunk = (int)chunk;
  a.positions = chunk > 0 ? positions->data_ptr<int>() : nullptr;
  a.sink = sink ? sink->data_ptr<float>() : nullptr;
  a.out_scale = (float)out_scale;
  a.total_rows = (int)(t_seqs * heads * maps);
  a.lam = lam ? lam->data_ptr<float>() : nullptr;
  a.count = (int)count;
  a.eps = (float)eps;
  a.f32 = !bf16;
  a.z = z.data_ptr();
  a.nz = z.size(1);
  a.swz = swz ? (uint16_t *)swz->data_ptr() : nullptr;
  a.nsplit = 1;
  auto stream = at::hip::getCurrentHIPStream();

  const bool scalar = !bf16 || wide > 256 ||
                      (size_t)WAVES * wave_bytes((int)ec) > MAX_LDS;
  if (!scalar)
    a.nsplit = (int)std::min<int64_t>(64, std::max<int64_t>(1, nsplit));
  at::Tensor po, pml;
  if (a.nsplit > 1 || maps > 1) {
    const auto f32 = y.options().dtype(at::kFloat);
    po = at::empty({a.nsplit, a.total_rows, vc}, f32);
    pml = at::empty({a.nsplit, a.total_rows, 2}, f32);
    a.part_o = po.data_ptr<float>();
    a.part_ml = pml.data_ptr<float>();
  }
  auto combine = [&]() {
    if (maps > 1)
      hipLaunchKernelGGL(shared_kv_diff_combine_kernel, dim3(a.total_rows / 2),
                         dim3(64), 0, stream, a);
    else if (a.nsplit > 1)
      hipLaunchKernelGGL(shared_kv_combine_kernel, dim3(a.total_rows),
                         dim3(64), 0, stream, a);
  };
  if (scalar) {
    TORCH_CHECK(wide <= 1024, "shared_kv_attend: heads of ", wide);
    a.scale = (float)scale;
    const dim3 grid(max_q * a.heads, n_seqs);
    const size_t shmem = 4 * vc * sizeof(float);
    auto pick = [&](auto tag) {
      using E = decltype(tag);
      auto go = [&](auto n) {
        hipLaunchKernelGGL((shared_kv_rows_kernel<E, decltype(n)::value>),
                           grid, dim3(BLOCK), shmem, stream, a);
      };
      if (wide <= 64) go(std::integral_constant<int, 1>{});
      else if (wide <= 128) go(std::integral_constant<int, 2>{});
      else if (wide <= 256) go(std::integral_constant<int, 4>{});
      else go(std::integral_constant<int, 16>{});
    };
    if (bf16) pick(uint16_t{});
    else pick(float{});
    combine();
    return;
  }

  a.scale = (float)(scale * 1.4426950408889634);
  const int64_t tiles = (max_q * a.group + M - 1) / M;
  TORCH_CHECK(tiles * G <= 65535, "shared_kv_attend: portion of ", max_q);
  const dim3 grid(a.nsplit, tiles * G, n_seqs);
  auto go = [&](auto size) {
    launch_attend<decltype(size)>(a, grid, stream);
  };
  if (maps > 1) pick_sizes2((int)hc, (int)vc, go);
  else pick_sizes((int)wide, (int)ec, go);
  combine();
}
