// Attention over the paged latent cache (gfx950).
//
// All heads of a layer attend to the same cached row per token: the latent
// (which is key and value at once, after q was moved into latent space) and
// one rotated key part. Query rows are (token, head) pairs of one sequence,
// heads fastest, so a workgroup reads each cache row once for 16-64 rows:
// single decoded tokens and short prompt portions are the same kernel.
//
//   score(row, key) = scale * (q_lat . c[key] + q_rot . k_rot[key])
//   out(row)        = softmax(score) . c         (still in latent space)
//
// A query at retained position i sees keys j with 0 <= i - j < window
// (window 0: all earlier keys).
//
// MFMA kernel (bf16): 4 waves, 64-key tiles staged once into LDS (next tile
// prefetched to registers). QK: each wave scores 16 keys for all rows, one
// fp32 exchange through LDS for the row-wise online softmax, PV: each wave
// owns a quarter of the latent columns and reads the same LDS rows
// transposed (ds_read_b64_tr_b16). `nsplit` workgroups share a sequence's
// keys; latent_combine merges their partial sums.
//
// The scalar kernel covers fp32 and sizes beyond the MFMA tiles: one
// workgroup per row, a wave per key, lanes across the cache row.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 256;
constexpr int TK = 64;                 // keys per tile
constexpr int ROTP = 64;               // padded rotated part
constexpr int PAGE = 16;               // tokens per cache block
constexpr int SSTRIDE = 68;            // floats per score row

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8v;
typedef __attribute__((ext_vector_type(4))) float f32x4v;
typedef __attribute__((ext_vector_type(4))) short s16x4v;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4v;

struct AttendArgs {
  const void *q_lat;                   // [T, H, rc]
  const void *q_rot;                   // y at the first rotated q element
  int64_t q_row;                       // y row stride
  int q_head;                          // y head stride
  const void *cache;                   // [blocks, PAGE, ec]
  const int *tables, *cu_q, *seq_lens;
  int table_width, heads, rc, rotc, ec, window, nsplit, total_rows;
  float scale;
  void *out;                           // [T, H, rc]
  float *part_o;                       // [nsplit, T*H, rc]
  float *part_ml;                      // [nsplit, T*H, 2]
};

// 8 values down a column of row-major 16-bit LDS rows: lane i of each 16-lane
// group gets column i of the 4 rows its group addresses, twice (rows +0..3
// and +4..7). `p` is this lane's 8-byte piece of the first 4 rows.
RB_DEV bf16x8v read_column8(const char *p, int stride4) {
  typedef __attribute__((address_space(3))) s16x4v *lds4;
  union { s16x4v h[2]; bf16x8v v; } r;
  r.h[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4)p);
  r.h[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4)(p + stride4));
  return r.v;
}

template <int RP, int MT>
__global__ __launch_bounds__(BLOCK, 1) void latent_attend_kernel(AttendArgs a) {
  constexpr int M = MT * 16;
  constexpr int COLS = RP + ROTP;
  constexpr int STRIDE = (COLS + 8) * 2;       // LDS row bytes
  constexpr int STEPS = COLS / 32;
  constexpr int CPP = COLS / 64;               // 16 B chunks per lane and key
  constexpr int CT = RP / 64;                  // column tiles per wave
  constexpr int TPR = BLOCK / M;               // softmax threads per row
  constexpr int KPT = TK / TPR;                // their keys

  extern __shared__ __attribute__((aligned(16))) char smem[];
  char *kv_s = smem;                           // [TK][STRIDE]
  char *q_s = kv_s + TK * STRIDE;              // [M][STRIDE]
  float *s_s = reinterpret_cast<float *>(q_s + M * STRIDE);  // [M][SSTRIDE]
  float *alpha_s = s_s + M * SSTRIDE;          // [M]
  float *l_s = alpha_s + M;                    // [M]

  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int l16 = lane & 15, grp = lane >> 4;
  const int split = blockIdx.x, seq = blockIdx.z;
  const int q0 = a.cu_q[seq], nq = a.cu_q[seq + 1] - q0;
  const int rows = nq * a.heads, row0 = blockIdx.y * M;
  if (row0 >= rows) return;
  const int n_keys = a.seq_lens[seq];
  const int v0 = n_keys - nq;                  // retained position of query 0
  const int tok_lo = row0 / a.heads;
  const int tok_hi = (min(row0 + M, rows) - 1) / a.heads;
  const int key_hi = v0 + tok_hi + 1;
  const int key_lo = a.window > 0 ? max(0, v0 + tok_lo - a.window + 1) : 0;
  const int base = key_lo & ~(PAGE - 1);
  const int tiles = (key_hi - base + TK - 1) / TK;
  const int per = (tiles + a.nsplit - 1) / a.nsplit;
  const int t0 = split * per, t1 = min(tiles, t0 + per);
  const int64_t grow0 = (int64_t)q0 * a.heads + row0;   // first global row

  if (t0 >= t1) {                              // nothing left for this split
    if (a.nsplit > 1)
      for (int m = tid; m < min(M, rows - row0); m += BLOCK) {
        float *ml = a.part_ml + ((int64_t)split * a.total_rows + grow0 + m) * 2;
        ml[0] = -INFINITY;
        ml[1] = 0.0f;
      }
    return;
  }

  const uint16_t *cache = (const uint16_t *)a.cache;
  const int *table = a.tables + (int64_t)seq * a.table_width;
  const u32x4v zero4 = (u32x4v)(0u);

  // ---- q rows (zero-padded) and the padding columns of the key tile -----
  for (int c = tid; c < M * (COLS / 8); c += BLOCK) {
    const int m = c / (COLS / 8), col = (c % (COLS / 8)) * 8;
    u32x4v v = zero4;
    if (row0 + m < rows) {
      const int64_t g = grow0 + m;
      if (col < RP) {
        if (col < a.rc)
          v = *reinterpret_cast<const u32x4v *>(
              (const uint16_t *)a.q_lat + g * a.rc + col);
      } else if (col - RP < a.rotc) {
        v = *reinterpret_cast<const u32x4v *>(
            (const uint16_t *)a.q_rot + (g / a.heads) * a.q_row +
            (g % a.heads) * a.q_head + col - RP);
      }
    }
    *reinterpret_cast<u32x4v *>(q_s + m * STRIDE + col * 2) = v;
  }
  for (int c = tid; c < TK * (COLS / 8); c += BLOCK) {
    const int key = c / (COLS / 8), col = (c % (COLS / 8)) * 8;
    if (col < RP ? col >= a.rc : col - RP >= a.rotc)
      *reinterpret_cast<u32x4v *>(kv_s + key * STRIDE + col * 2) = zero4;
  }

  // ---- tile loader: 8 lanes per key, 32 keys per pass, 2 passes ---------
  const int lkey = tid >> 3, lchunk = tid & 7;
  const int chunks = a.ec / 8;
  u32x4v reg[2][CPP];
  int page[2];
  auto fetch_pages = [&](int t) {
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int key = base + t * TK + p * 32 + lkey;
      page[p] = key < key_hi ? table[key / PAGE] : 0;
    }
  };
  auto fetch = [&](int t) {
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int key = base + t * TK + p * 32 + lkey;
      const bool ok = key < key_hi;
      const uint16_t *src =
          cache + ((int64_t)page[p] * PAGE + key % PAGE) * a.ec;
#pragma unroll
      for (int i = 0; i < CPP; ++i) {
        const int c = lchunk + i * 8;
        reg[p][i] = (ok && c < chunks)
                        ? *reinterpret_cast<const u32x4v *>(src + c * 8)
                        : zero4;
      }
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int p = 0; p < 2; ++p)
#pragma unroll
      for (int i = 0; i < CPP; ++i) {
        const int c = lchunk + i * 8;
        if (c < chunks) {
          const int col = c * 8 < a.rc ? c * 8 : RP + c * 8 - a.rc;
          *reinterpret_cast<u32x4v *>(kv_s + (p * 32 + lkey) * STRIDE +
                                      col * 2) = reg[p][i];
        }
      }
  };

  // ---- softmax role of this thread --------------------------------------
  const int srow = tid / TPR, spart = tid % TPR;
  const int qpos =
      row0 + srow < rows ? v0 + (row0 + srow) / a.heads : -1;
  const int kmin = a.window > 0 ? qpos - a.window + 1 : 0;
  float m_run = -INFINITY, l_run = 0.0f;

  f32x4v acc[CT][MT];
#pragma unroll
  for (int c = 0; c < CT; ++c)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[c][m] = (f32x4v)(0.0f);

  fetch_pages(t0);
  fetch(t0);
  if (t0 + 1 < t1) fetch_pages(t0 + 1);

  for (int t = t0; t < t1; ++t) {
    __syncthreads();                           // last tile fully read
    stage();
    __syncthreads();
    if (t + 1 < t1) {
      fetch(t + 1);
      if (t + 2 < t1) fetch_pages(t + 2);
    }

    // ---- scores: wave's 16 keys x all rows ------------------------------
    f32x4v sc[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) sc[m] = (f32x4v)(0.0f);
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
      const int off = (s * 32 + grp * 8) * 2;
      const bf16x8v kf = *reinterpret_cast<const bf16x8v *>(
          kv_s + (wid * 16 + l16) * STRIDE + off);
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        const bf16x8v qf = *reinterpret_cast<const bf16x8v *>(
            q_s + (m * 16 + l16) * STRIDE + off);
        sc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, kf, sc[m], 0, 0, 0);
      }
    }
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        s_s[(m * 16 + grp * 4 + r) * SSTRIDE + wid * 16 + l16] =
            sc[m][r] * a.scale;
    __syncthreads();

    // ---- online softmax; P replaces the scores of its row ---------------
    {
      float p[KPT];
      float mx = -INFINITY;
      const float *sr = s_s + srow * SSTRIDE + spart * KPT;
      const int k0 = base + t * TK + spart * KPT;
#pragma unroll
      for (int j = 0; j < KPT; ++j) {
        const bool vis = k0 + j <= qpos && k0 + j >= kmin;
        p[j] = vis ? sr[j] : -INFINITY;
        mx = fmaxf(mx, p[j]);
      }
#pragma unroll
      for (int o = TPR / 2; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
      const float m_new = fmaxf(m_run, mx);
      float alpha = 1.0f;
      if (m_new != -INFINITY) {
        alpha = __expf(m_run - m_new);         // 0 on the first visible tile
        float sum = 0.0f;
#pragma unroll
        for (int j = 0; j < KPT; ++j) {
          p[j] = __expf(p[j] - m_new);
          sum += p[j];
        }
        l_run = l_run * alpha + sum;
        m_run = m_new;
      } else {
#pragma unroll
        for (int j = 0; j < KPT; ++j) p[j] = 0.0f;
      }
      // a row's threads are lanes of one wave: all have read their scores
      uint32_t *pr = reinterpret_cast<uint32_t *>(s_s + srow * SSTRIDE) +
                     spart * (KPT / 2);
#pragma unroll
      for (int j = 0; j < KPT; j += 2)
        pr[j / 2] = rb::f32_to_bf16(p[j]) |
                    ((uint32_t)rb::f32_to_bf16(p[j + 1]) << 16);
      if (spart == 0) alpha_s[srow] = alpha;
    }
    __syncthreads();

    // ---- O^T += C^T P^T on the wave's latent columns --------------------
    bf16x8v pf[2][MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const float al = alpha_s[m * 16 + l16];
#pragma unroll
      for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[c][m][r] *= al;
#pragma unroll
      for (int ks = 0; ks < 2; ++ks)
        pf[ks][m] = *reinterpret_cast<const bf16x8v *>(
            reinterpret_cast<const char *>(s_s + (m * 16 + l16) * SSTRIDE) +
            (ks * 32 + grp * 8) * 2);
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const char *vrow = kv_s + (ks * 32 + grp * 8 + (l16 >> 2)) * STRIDE +
                         (wid * (RP / 4) + (l16 & 3) * 4) * 2;
#pragma unroll
      for (int c = 0; c < CT; ++c) {
        const bf16x8v vf = read_column8(vrow + c * 32, 4 * STRIDE);
#pragma unroll
        for (int m = 0; m < MT; ++m)
          acc[c][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[ks][m],
                                                              acc[c][m], 0, 0, 0);
      }
    }
  }

  // ---- row sums, then O^T: lane holds 4 consecutive columns of one row ---
#pragma unroll
  for (int o = TPR / 2; o > 0; o >>= 1) l_run += __shfl_xor(l_run, o, 64);
  if (spart == 0) {
    l_s[srow] = l_run;
    if (a.nsplit > 1 && row0 + srow < rows) {
      float *ml =
          a.part_ml + ((int64_t)split * a.total_rows + grow0 + srow) * 2;
      ml[0] = m_run;
      ml[1] = l_run;
    }
  }
  __syncthreads();
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int row = m * 16 + l16;
    if (row0 + row >= rows) continue;
    const float l = l_s[row];
    const float inv = l > 0.0f ? 1.0f / l : 0.0f;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      const int col = wid * (RP / 4) + c * 16 + grp * 4;
      if (col >= a.rc) continue;
      if (a.nsplit > 1) {
        *reinterpret_cast<f32x4v *>(
            a.part_o + ((int64_t)split * a.total_rows + grow0 + row) * a.rc +
            col) = acc[c][m];
      } else {
        uint2 o;
        o.x = rb::f32_to_bf16(acc[c][m][0] * inv) |
              ((uint32_t)rb::f32_to_bf16(acc[c][m][1] * inv) << 16);
        o.y = rb::f32_to_bf16(acc[c][m][2] * inv) |
              ((uint32_t)rb::f32_to_bf16(acc[c][m][3] * inv) << 16);
        *reinterpret_cast<uint2 *>((uint16_t *)a.out + (grow0 + row) * a.rc +
                                   col) = o;
      }
    }
  }
}

// one block per row: merge the splits
__global__ __launch_bounds__(128) void latent_combine_kernel(
    const float *__restrict__ part_o, const float *__restrict__ part_ml,
    uint16_t *__restrict__ out, int nsplit, int total_rows, int rc) {
  const int64_t row = blockIdx.x;
  float mx = -INFINITY;
  for (int s = 0; s < nsplit; ++s)
    mx = fmaxf(mx, part_ml[((int64_t)s * total_rows + row) * 2]);
  float l = 0.0f;
  for (int s = 0; s < nsplit; ++s) {
    const float *ml = part_ml + ((int64_t)s * total_rows + row) * 2;
    if (ml[1] > 0.0f) l += ml[1] * __expf(ml[0] - mx);
  }
  const float inv = l > 0.0f ? 1.0f / l : 0.0f;
  for (int c = threadIdx.x * 4; c < rc; c += blockDim.x * 4) {
    f32x4v o = (f32x4v)(0.0f);
    for (int s = 0; s < nsplit; ++s) {
      const float *ml = part_ml + ((int64_t)s * total_rows + row) * 2;
      if (!(ml[1] > 0.0f)) continue;
      const float w = __expf(ml[0] - mx) * inv;
      const f32x4v p = *reinterpret_cast<const f32x4v *>(
          part_o + ((int64_t)s * total_rows + row) * rc + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] += w * p[e];
    }
    uint2 w2;
    w2.x = rb::f32_to_bf16(o[0]) | ((uint32_t)rb::f32_to_bf16(o[1]) << 16);
    w2.y = rb::f32_to_bf16(o[2]) | ((uint32_t)rb::f32_to_bf16(o[3]) << 16);
    *reinterpret_cast<uint2 *>(out + row * rc + c) = w2;
  }
}

// ---------------------------------------------------------------------------
// scalar kernel: block = one (token, head) row, wave = every fourth key
// ---------------------------------------------------------------------------
template <typename T, int NE>
__global__ __launch_bounds__(BLOCK) void latent_attend_rows_kernel(
    AttendArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float *o_s = reinterpret_cast<float *>(smem);        // [4][ec]
  __shared__ float ml_s[4][2];
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int row = blockIdx.x, seq = blockIdx.y;
  const int q0 = a.cu_q[seq], nq = a.cu_q[seq + 1] - q0;
  if (row >= nq * a.heads) return;
  const int qpos = a.seq_lens[seq] - nq + row / a.heads;
  const int lo = a.window > 0 ? max(0, qpos - a.window + 1) : 0;
  const int64_t g = (int64_t)q0 * a.heads + row;
  const T *ql = (const T *)a.q_lat + g * a.rc;
  const T *qr = (const T *)a.q_rot + (g / a.heads) * a.q_row +
                (g % a.heads) * a.q_head;
  const int *table = a.tables + (int64_t)seq * a.table_width;

  float q[NE], o[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + i * 64;
    q[i] = e < a.rc ? rb::bf16_to_f32_or_id(ql[e])
           : e < a.ec ? rb::bf16_to_f32_or_id(qr[e - a.rc]) : 0.0f;
    o[i] = 0.0f;
  }
  float m = -INFINITY, l = 0.0f;
  for (int key = lo + wid; key <= qpos; key += 4) {
    const T *c = (const T *)a.cache +
                 ((int64_t)table[key / PAGE] * PAGE + key % PAGE) * a.ec;
    float v[NE], s = 0.0f;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = lane + i * 64;
      v[i] = e < a.ec ? rb::bf16_to_f32_or_id(c[e]) : 0.0f;
      s = fmaf(q[i], v[i], s);
    }
    s = rb::wave_reduce_sum(s) * a.scale;
    const float mn = fmaxf(m, s);
    const float al = expf(m - mn), p = expf(s - mn);
    l = l * al + p;
    m = mn;
#pragma unroll
    for (int i = 0; i < NE; ++i) o[i] = o[i] * al + p * v[i];
  }
  if (lane == 0) {
    ml_s[wid][0] = m;
    ml_s[wid][1] = l;
  }
#pragma unroll
  for (int i = 0; i < NE; ++i)
    if (lane + i * 64 < a.ec) o_s[wid * a.ec + lane + i * 64] = o[i];
  __syncthreads();
  float mx = -INFINITY, lt = 0.0f, w[4];
#pragma unroll
  for (int k = 0; k < 4; ++k) mx = fmaxf(mx, ml_s[k][0]);
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    w[k] = ml_s[k][1] > 0.0f ? expf(ml_s[k][0] - mx) : 0.0f;
    lt += w[k] * ml_s[k][1];
  }
  for (int e = threadIdx.x; e < a.rc; e += BLOCK) {
    float v = 0.0f;
#pragma unroll
    for (int k = 0; k < 4; ++k) v += w[k] * o_s[k * a.ec + e];
    rb::store_scalar((T *)a.out + g * a.rc + e, v / lt);
  }
}

bool mfma_sizes(int64_t rc, int64_t rotc) { return rc <= 512 && rotc <= ROTP; }
int padded_rank(int64_t rc) {
  return rc <= 64 ? 64 : rc <= 128 ? 128 : rc <= 256 ? 256 : 512;
}

template <int RP, int MT>
void launch_attend(const AttendArgs &a, dim3 grid, hipStream_t stream) {
  constexpr size_t shmem = (size_t)(TK + MT * 16) * ((RP + ROTP + 8) * 2) +
                           (size_t)MT * 16 * (SSTRIDE + 2) * sizeof(float);
  static_assert(shmem <= 160 * 1024, "LDS");
  static bool once = [] {
    return hipFuncSetAttribute(
               reinterpret_cast<const void *>(&latent_attend_kernel<RP, MT>),
               hipFuncAttributeMaxDynamicSharedMemorySize,
               (int)shmem) == hipSuccess;
  }();
  TORCH_CHECK(once, "latent_attend: LDS size");
  hipLaunchKernelGGL((latent_attend_kernel<RP, MT>), grid, dim3(BLOCK), shmem,
                     stream, a);
}

}  // namespace

int64_t latent_attend_rows(int64_t rows, int64_t rc, int64_t rotc, bool bf16) {
  if (!bf16 || !mfma_sizes(rc, rotc)) return 1;
  if (rows <= 16) return 16;
  return rows <= 32 || padded_rank(rc) == 512 ? 32 : 64;
}

at::Tensor latent_attend(at::Tensor q_lat, at::Tensor y, int64_t q_off,
                         int64_t q_head, at::Tensor cache,
                         at::Tensor block_tables, at::Tensor cu_q,
                         at::Tensor seq_lens, int64_t n_seqs, int64_t max_q,
                         int64_t nsplit, double scale, int64_t window,
                         int64_t rc) {
  TORCH_CHECK(q_lat.is_cuda() && q_lat.dim() == 3 && q_lat.is_contiguous() &&
              q_lat.size(2) == rc, "latent_attend: q_lat [T, H, rc]");
  const int64_t T = q_lat.size(0), H = q_lat.size(1);
  const auto dt = q_lat.scalar_type();
  const bool bf16 = dt == at::kBFloat16;
  TORCH_CHECK(bf16 || dt == at::kFloat, "latent_attend: dtype");
  TORCH_CHECK(cache.dim() == 3 && cache.size(1) == PAGE &&
              cache.is_contiguous() && cache.scalar_type() == dt,
              "latent_attend: cache [blocks, 16, ec]");
  const int64_t ec = cache.size(2), rotc = ec - rc;
  TORCH_CHECK(rc % 8 == 0 && rotc >= 8 && rotc % 8 == 0 && q_off % 8 == 0 &&
              q_head % 8 == 0 && y.size(1) % 8 == 0, "latent_attend: layout");
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && y.scalar_type() == dt &&
              y.size(0) >= T && q_off + (H - 1) * q_head + rotc <= y.size(1),
              "latent_attend: y");
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.is_contiguous() &&
              block_tables.scalar_type() == at::kInt &&
              cu_q.scalar_type() == at::kInt && cu_q.is_contiguous() &&
              seq_lens.scalar_type() == at::kInt && seq_lens.is_contiguous() &&
              block_tables.size(0) >= n_seqs && cu_q.numel() > n_seqs &&
              seq_lens.numel() >= n_seqs, "latent_attend: batch tensors");
  TORCH_CHECK(T * H < (1 << 30) && n_seqs <= 65535, "latent_attend: rows");
  auto out = at::empty_like(q_lat);
  if (T == 0 || n_seqs == 0) return out;

  const size_t esz = bf16 ? 2 : 4;
  AttendArgs a{};
  a.q_lat = q_lat.data_ptr();
  a.q_rot = (const char *)y.data_ptr() + q_off * esz;
  a.q_row = y.size(1);
  a.q_head = (int)q_head;
  a.cache = cache.data_ptr();
  a.tables = block_tables.data_ptr<int>();
  a.cu_q = cu_q.data_ptr<int>();
  a.seq_lens = seq_lens.data_ptr<int>();
  a.table_width = (int)block_tables.size(1);
  a.heads = (int)H;
  a.rc = (int)rc;
  a.rotc = (int)rotc;
  a.ec = (int)ec;
  a.window = (int)window;
  a.scale = (float)scale;
  a.total_rows = (int)(T * H);
  a.nsplit = 1;
  a.out = out.data_ptr();
  auto stream = at::hip::getCurrentHIPStream();
  const int64_t rows = max_q * H;
  const int64_t M = latent_attend_rows(rows, rc, rotc, bf16);

  if (M == 1) {
    TORCH_CHECK(ec <= 2048, "latent_attend: cache rows of ", ec);
    const dim3 grid(rows, n_seqs);
    const size_t shmem = 4 * ec * sizeof(float);
    const int ne = ec <= 128 ? 2 : ec <= 320 ? 5 : ec <= 640 ? 10 : 32;
    auto go = [&](auto tag, auto n) {
      using E = decltype(tag);
      hipLaunchKernelGGL((latent_attend_rows_kernel<E, decltype(n)::value>),
                         grid, dim3(BLOCK), shmem, stream, a);
    };
    auto pick = [&](auto tag) {
      if (ne == 2) go(tag, std::integral_constant<int, 2>{});
      else if (ne == 5) go(tag, std::integral_constant<int, 5>{});
      else if (ne == 10) go(tag, std::integral_constant<int, 10>{});
      else go(tag, std::integral_constant<int, 32>{});
    };
    if (bf16) pick(uint16_t{});
    else pick(float{});
    return out;
  }

  a.nsplit = (int)std::max<int64_t>(1, nsplit);
  at::Tensor po, pml;
  if (a.nsplit > 1) {
    const auto f32 = q_lat.options().dtype(at::kFloat);
    po = at::empty({a.nsplit, T * H, rc}, f32);
    pml = at::empty({a.nsplit, T * H, 2}, f32);
    a.part_o = po.data_ptr<float>();
    a.part_ml = pml.data_ptr<float>();
  }
  const dim3 grid(a.nsplit, (rows + M - 1) / M, n_seqs);
  const int rp = padded_rank(rc);
#define RB_ATTEND(RP)                                     \
  do {                                                    \
    if (M == 16) launch_attend<RP, 1>(a, grid, stream);   \
    else if (M == 32) launch_attend<RP, 2>(a, grid, stream); \
    else if constexpr (RP < 512) launch_attend<RP, 4>(a, grid, stream); \
  } while (0)
  if (rp == 64) RB_ATTEND(64);
  else if (rp == 128) RB_ATTEND(128);
  else if (rp == 256) RB_ATTEND(256);
  else RB_ATTEND(512);
#undef RB_ATTEND
  if (a.nsplit > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3(T * H), dim3(128), 0,
                       stream, a.part_o, a.part_ml, (uint16_t *)a.out,
                       a.nsplit, a.total_rows, a.rc);
  return out;
}
