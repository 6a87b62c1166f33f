// Attention over the paged latent cache (gfx950).
//
// All heads of a layer attend to the same cached row per token: the latent
// (which is key and value at once, after q was moved into latent space) and
// one rotated key part (or none). Query rows are (token, head) pairs of one sequence,
// heads fastest, so a workgroup reads each cache row once for 16-64 rows:
// single decoded tokens and short prompt portions are the same kernel.
//
//   score(row, key) = scale * (q_lat . c[key] + q_rot . k_rot[key])
//   out(row)        = softmax(score) . c         (still in latent space)
//
// A query at retained position i sees keys j with 0 <= i - j < window
// (window 0: all earlier keys).
//
// MFMA kernel (bf16): 8 waves, 64-key tiles staged once into double-buffered
// LDS (the tile after next is in registers). QK: each wave scores 16 keys for
// one part of the rows, whose q it keeps in registers (with 16 rows, for one
// half of the columns); one fp32 exchange through LDS for the row-wise online
// softmax; PV: each wave owns an eighth of the latent columns and reads the
// same LDS rows transposed (ds_read_b64_tr_b16). Two barriers per tile: one
// interval holds softmax(t) and the staging of tile t+1, the other PV(t) and
// QK(t+1). `nsplit` workgroups share a sequence's keys; latent_combine merges
// their partial sums.
//
// The scalar kernel covers fp32 and sizes beyond the MFMA tiles: one
// workgroup per row, a wave per key, lanes across the cache row.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 512;             // MFMA kernel
constexpr int ROWS_BLOCK = 256;        // scalar kernel
constexpr int TK = 64;                 // keys per tile
constexpr int MAX_ROT = 64;            // padded rotated part
constexpr int PAGE = 16;               // tokens per cache block
constexpr int SSTRIDE = 68;            // floats per score row
constexpr int PSTRIDE = 72;            // 16-bit weights per row

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8v;
typedef __attribute__((ext_vector_type(4))) float f32x4v;
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

// The key tile's rows are unpadded; 16-byte chunk c of key k lies at chunk
// c ^ (k & 7), which spreads both the row-wise reads (16 keys, one chunk) and
// the column-wise ones (8 keys, two chunks) over the banks.
RB_DEV int tile_chunk(int key, int chunk) { return (chunk ^ (key & 7)) * 16; }

// maximum over aligned groups of N lanes (N = 8, 16, 32)
template <int N> RB_DEV float group_max(float v) {
  auto dpp = [](float x, auto ctrl) {
    return __int_as_float(__builtin_amdgcn_update_dpp(
        0, __float_as_int(x), decltype(ctrl)::value, 0xf, 0xf, true));
  };
  v = fmaxf(v, dpp(v, std::integral_constant<int, 0xB1>{}));   // lane ^ 1
  v = fmaxf(v, dpp(v, std::integral_constant<int, 0x4E>{}));   // lane ^ 2
  v = fmaxf(v, dpp(v, std::integral_constant<int, 0x141>{}));  // 7 - lane
  if constexpr (N >= 16)
    v = fmaxf(v, dpp(v, std::integral_constant<int, 0x140>{}));  // 15 - lane
  if constexpr (N >= 32) v = fmaxf(v, __shfl_xor(v, 16, 64));
  return v;
}

template <int RP, int MT, int ROTP>
__global__ __launch_bounds__(BLOCK, 1) void latent_attend_kernel(AttendArgs a) {
  constexpr int M = MT * 16;
  constexpr int COLS = RP + ROTP;
  constexpr int STRIDE = COLS * 2;             // LDS row bytes
  constexpr int KH = MT == 1 ? 2 : 1;          // column halves in QK
  constexpr int QT = MT == 4 ? 2 : 1;          // row tiles per wave in QK
  constexpr int NS = COLS / 32 / KH;           // QK steps per wave
  constexpr int CPP = COLS / 64;               // 16 B chunks per lane and key
  constexpr int CG = RP / 16 < 8 ? RP / 16 : 8;  // waves that own columns
  constexpr int CT = RP / 16 / CG;             // their column tiles
  constexpr int TPR = BLOCK / M;               // softmax threads per row
  constexpr int KPT = TK / TPR;                // their keys

  extern __shared__ __attribute__((aligned(16))) char smem[];
  char *kv_s = smem;                           // [2][TK][STRIDE]
  float *s_s = reinterpret_cast<float *>(kv_s + 2 * TK * STRIDE);
                                               // [KH][M][SSTRIDE]
  uint16_t *p_s = reinterpret_cast<uint16_t *>(s_s + KH * M * SSTRIDE);
                                               // [M][PSTRIDE]
  float *alpha_s = reinterpret_cast<float *>(p_s + M * PSTRIDE);  // [M]
  float *l_s = alpha_s + M;                    // [M]

  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int l16 = lane & 15, grp = lane >> 4;
  const int kg = wid & 3, part = wid >> 2;     // QK role: keys, rows/columns
  const int split = blockIdx.x, seq = blockIdx.z;
  const int q0 = a.cu_q[seq], nq = a.cu_q[seq + 1] - q0;
  const int n_keys = a.seq_lens[seq];
  const int rows = nq * a.heads, row0 = blockIdx.y * M;
  if (row0 >= rows) return;
  const int v0 = n_keys - nq;                  // retained position of query 0
  const int tok_lo = row0 / a.heads;
  const int tok_hi = (min(row0 + M, rows) - 1) / a.heads;
  const int key_hi = v0 + tok_hi + 1;
  const int key_lo = a.window > 0 ? max(0, v0 + tok_lo - a.window + 1) : 0;
  const int base = key_lo & ~(PAGE - 1);
  const int tiles = (key_hi - base + TK - 1) / TK;
  // short contexts use fewer splits: at least two tiles each
  const int per = max(2, (tiles + a.nsplit - 1) / a.nsplit);
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

  // ---- tile loader: 8 lanes per key ---------------------------------------
  // Branch-free: keys beyond the last one repeat it (their scores are masked),
  // lanes beyond the row's last chunk repeat that chunk.
  const int lkey = tid >> 3, lchunk = tid & 7;
  const int last_chunk = a.ec / 8 - 1, split_chunk = a.rc / 8;
  u32x4v reg[CPP], reg0[CPP];
  auto page_of = [&](int t) {
    return table[min(base + t * TK + lkey, key_hi - 1) / PAGE];
  };
  auto fetch = [&](u32x4v *dst, int t, int page) {
    const int key = min(base + t * TK + lkey, key_hi - 1);
    const uint16_t *src = cache + ((int64_t)page * PAGE + key % PAGE) * a.ec;
#pragma unroll
    for (int i = 0; i < CPP; ++i)
      dst[i] = *reinterpret_cast<const u32x4v *>(
          src + min(lchunk + i * 8, last_chunk) * 8);
  };
  auto stage = [&](char *dst, const u32x4v *src) {
#pragma unroll
    for (int i = 0; i < CPP; ++i) {
      const int c = min(lchunk + i * 8, last_chunk);
      *reinterpret_cast<u32x4v *>(
          dst + lkey * STRIDE +
          tile_chunk(lkey, c < split_chunk ? c : c - split_chunk + RP / 8)) =
          src[i];
    }
  };
  // the first two tiles and q are on their way before anything else
  const int page0 = page_of(t0), page1 = page_of(t0 + 1);
  int page = page_of(t0 + 2);
  fetch(reg0, t0, page0);

  // q rows come once per workgroup, through the second key buffer
  constexpr int QCHUNKS = M * (COLS / 8), QN = (QCHUNKS + BLOCK - 1) / BLOCK;
  u32x4v qreg[QN];
#pragma unroll
  for (int i = 0; i < QN; ++i) {
    const int c = min(tid + i * BLOCK, QCHUNKS - 1);
    const int m = c / (COLS / 8), col = (c % (COLS / 8)) * 8;
    const bool ok = row0 + m < rows &&
                    (col < RP ? col < a.rc : col - RP < a.rotc);
    const int row = ok ? row0 + m : 0;
    const int tok = q0 + row / a.heads, head = row % a.heads;
    const uint16_t *src =
        ok && col >= RP
            ? (const uint16_t *)a.q_rot + tok * a.q_row + head * a.q_head +
                  col - RP
            : (const uint16_t *)a.q_lat +
                  ((int64_t)tok * a.heads + head) * a.rc + (ok ? col : 0);
    const u32x4v v = *reinterpret_cast<const u32x4v *>(src);
    qreg[i] = ok ? v : zero4;
  }
  if (t0 + 1 < t1) fetch(reg, t0 + 1, page1);

  // padding columns of the key tiles
  auto clear_padding = [&](char *tile) {
    if (a.rc == RP && a.rotc == ROTP) return;
    for (int c = tid; c < TK * (COLS / 8); c += BLOCK) {
      const int key = c / (COLS / 8), col = (c % (COLS / 8)) * 8;
      if (col < RP ? col >= a.rc : col - RP >= a.rotc)
        *reinterpret_cast<u32x4v *>(tile + key * STRIDE +
                                    tile_chunk(key, col / 8)) = zero4;
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

  bf16x8v qf[QT][NS];                  // this wave's q fragments

  // ---- scores of a staged tile: 16 keys x this wave's rows ---------------
  auto scores = [&](const char *tile) {
    // key fragments come in groups, one group of LDS reads ahead of the
    // products; two accumulators per row tile shorten the dependent chain
    constexpr int G = NS == 18 && MT > 1 ? 3 : NS % 6 == 0 ? 6 :
                      NS % 5 == 0 ? 5 : NS % 4 == 0 ? 4 :
                      NS % 3 == 0 ? 3 : NS;
    static_assert(NS % G == 0, "QK groups");
    f32x4v sc[QT][2];
#pragma unroll
    for (int q = 0; q < QT; ++q) sc[q][0] = sc[q][1] = (f32x4v)(0.0f);
    const char *krow = tile + (kg * 16 + l16) * STRIDE;
    const int s_first = KH == 2 ? part * NS : 0;
    auto fragment = [&](int s) {
      return *reinterpret_cast<const bf16x8v *>(
          krow + tile_chunk(l16, (s_first + s) * 4 + grp));
    };
    bf16x8v kf[2][G];
#pragma unroll
    for (int s = 0; s < G; ++s) kf[0][s] = fragment(s);
#pragma unroll
    for (int g = 0; g < NS / G; ++g) {
      if (g + 1 < NS / G) {
#pragma unroll
        for (int s = 0; s < G; ++s)
          kf[(g + 1) & 1][s] = fragment((g + 1) * G + s);
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int s = 0; s < G; ++s)
#pragma unroll
        for (int q = 0; q < QT; ++q)
          sc[q][s & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              qf[q][g * G + s], kf[g & 1][s], sc[q][s & 1], 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int q = 0; q < QT; ++q) {
      const int m0 = KH == 2 ? part * M : (part * QT + q) * 16;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        s_s[(m0 + grp * 4 + r) * SSTRIDE + kg * 16 + l16] =
            (sc[q][0][r] + sc[q][1][r]) * a.scale;
    }
  };

  // ---- O^T += C^T P^T on the wave's latent columns ------------------------
  auto accumulate = [&](const char *tile) {
    if (wid >= CG) return;
    bf16x8v pf[2][MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks)
        pf[ks][m] = *reinterpret_cast<const bf16x8v *>(
            p_s + (m * 16 + l16) * PSTRIDE + ks * 32 + grp * 8);
      const float al = alpha_s[m * 16 + l16];
#pragma unroll
      for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[c][m][r] *= al;
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const char *vrow = tile + (ks * 32 + grp * 8 + (l16 >> 2)) * STRIDE +
                         (l16 & 1) * 8;
      const int vchunk = wid * (CT * 2) + ((l16 >> 1) & 1);
      bf16x8v vf[CT];
#pragma unroll
      for (int c = 0; c < CT; ++c)
        vf[c] = rb::lds_column8(
            vrow + tile_chunk(l16 >> 2, vchunk + c * 2),
            vrow + 4 * STRIDE + tile_chunk((l16 >> 2) + 4, vchunk + c * 2));
#pragma unroll
      for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int m = 0; m < MT; ++m)
          acc[c][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              vf[c], pf[ks][m], acc[c][m], 0, 0, 0);
    }
  };

  clear_padding(kv_s);
  stage(kv_s, reg0);
  char *q_s = kv_s + TK * STRIDE;
#pragma unroll
  for (int i = 0; i < QN; ++i) {
    const int c = min(tid + i * BLOCK, QCHUNKS - 1);
    const int m = c / (COLS / 8);
    *reinterpret_cast<u32x4v *>(
        q_s + m * STRIDE + tile_chunk(m, c % (COLS / 8))) = qreg[i];
  }
  __syncthreads();
#pragma unroll
  for (int q = 0; q < QT; ++q) {
    const int m = (KH == 2 ? 0 : (part * QT + q) * 16) + l16;
#pragma unroll
    for (int s = 0; s < NS; ++s)
      qf[q][s] = *reinterpret_cast<const bf16x8v *>(
          q_s + m * STRIDE +
          tile_chunk(m, ((KH == 2 ? part * NS : 0) + s) * 4 + grp));
  }
  scores(kv_s);
  if (t0 + 1 < t1 && (a.rc < RP || a.rotc < ROTP)) {
    __syncthreads();                   // q has been read by all waves
    clear_padding(q_s);
  }

  for (int t = t0; t < t1; ++t) {
    char *tile = kv_s + ((t - t0) & 1) * TK * STRIDE;
    char *next = kv_s + ((t - t0 + 1) & 1) * TK * STRIDE;
    __syncthreads();                   // scores(t) written, PV(t-1) done
    // ---- online softmax ---------------------------------------------------
    {
      float p[KPT];
      float mx = -INFINITY;
      const float *sr = s_s + srow * SSTRIDE + spart * KPT;
      const int k0 = base + t * TK + spart * KPT;
#pragma unroll
      for (int j = 0; j < KPT; ++j) {
        p[j] = sr[j];
        if constexpr (KH == 2) p[j] += sr[M * SSTRIDE + j];
      }
#pragma unroll
      for (int j = 0; j < KPT; ++j) {
        const bool vis = k0 + j <= qpos && k0 + j >= kmin;
        p[j] = vis ? p[j] : -INFINITY;
        mx = fmaxf(mx, p[j]);
      }
      const float m_new = fmaxf(m_run, group_max<TPR>(mx));
      // rows that have seen no key yet keep a finite reference
      const float ref = m_new == -INFINITY ? 0.0f : m_new;
      const float alpha = __expf(m_run - ref);   // 0 before the first key
      float sum = 0.0f;
#pragma unroll
      for (int j = 0; j < KPT; ++j) {
        p[j] = __expf(p[j] - ref);
        sum += p[j];
      }
      l_run = l_run * alpha + sum;
      m_run = m_new;
      uint32_t *pr =
          reinterpret_cast<uint32_t *>(p_s + srow * PSTRIDE + spart * KPT);
#pragma unroll
      for (int j = 0; j < KPT; j += 2)
        pr[j / 2] = rb::pack_bf16x2(p[j], p[j + 1]);
      if (spart == 0) alpha_s[srow] = alpha;
    }
    if (t + 1 < t1) {
      stage(next, reg);
      if (t + 2 < t1) fetch(reg, t + 2, page);
      if (t + 3 < t1) page = page_of(t + 3);
    }
    __syncthreads();                   // P(t) and tile t+1 are there
    accumulate(tile);
    if (t + 1 < t1) scores(next);
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
  if (wid >= CG) return;
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int row = m * 16 + l16;
    if (row0 + row >= rows) continue;
    const float l = l_s[row];
    const float inv = l > 0.0f ? 1.0f / l : 0.0f;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      const int col = wid * (CT * 16) + c * 16 + grp * 4;
      if (col >= a.rc) continue;
      if (a.nsplit > 1) {
        *reinterpret_cast<f32x4v *>(
            a.part_o + ((int64_t)split * a.total_rows + grow0 + row) * a.rc +
            col) = acc[c][m];
      } else {
        uint2 o;
        o.x = rb::pack_bf16x2(acc[c][m][0] * inv, acc[c][m][1] * inv);
        o.y = rb::pack_bf16x2(acc[c][m][2] * inv, acc[c][m][3] * inv);
        *reinterpret_cast<uint2 *>((uint16_t *)a.out + (grow0 + row) * a.rc +
                                   col) = o;
      }
    }
  }
}

// One block per row merges the splits (at most 64). Each wave reads all
// splits' statistics at once; splits without keys get weight 0 and the
// address of one that has some, so every load is unconditional.
__global__ __launch_bounds__(128) void latent_combine_kernel(
    const float *__restrict__ part_o, const float *__restrict__ part_ml,
    uint16_t *__restrict__ out, int nsplit, int total_rows, int rc) {
  const int64_t row = blockIdx.x;
  const int lane = threadIdx.x & 63;
  float m = -INFINITY, l = 0.0f;
  if (lane < nsplit) {
    const float2 ml = *reinterpret_cast<const float2 *>(
        part_ml + ((int64_t)lane * total_rows + row) * 2);
    m = ml.x;
    l = ml.y;
  }
  const bool has = l > 0.0f;
  const int first = __ffsll((unsigned long long)__ballot(has)) - 1;
  const float mx = rb::wave_reduce_max(m);
  float w = has ? __expf(m - mx) : 0.0f;
  w /= rb::wave_reduce_sum(l * w);
  // through LDS: not every lane takes part in the loop below
  __shared__ float w_s[64];
  __shared__ int src_s[64];
  if (threadIdx.x < 64) {
    w_s[lane] = w;
    src_s[lane] = has ? lane : max(first, 0);
  }
  __syncthreads();
  for (int c = threadIdx.x * 4; c < rc; c += blockDim.x * 4) {
    f32x4v o = (f32x4v)(0.0f);
#pragma unroll 8
    for (int s = 0; s < nsplit; ++s) {
      const float ws = w_s[s];
      const f32x4v p = *reinterpret_cast<const f32x4v *>(
          part_o + ((int64_t)src_s[s] * total_rows + row) * rc + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] += ws * p[e];
    }
    uint2 w2;
    w2.x = rb::pack_bf16x2(o[0], o[1]);
    w2.y = rb::pack_bf16x2(o[2], o[3]);
    *reinterpret_cast<uint2 *>(out + row * rc + c) = w2;
  }
}

// ---------------------------------------------------------------------------
// scalar kernel: block = one (token, head) row, wave = every fourth key
// ---------------------------------------------------------------------------
template <typename T, int NE>
__global__ __launch_bounds__(ROWS_BLOCK) void latent_attend_rows_kernel(
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
  for (int e = threadIdx.x; e < a.rc; e += ROWS_BLOCK) {
    float v = 0.0f;
#pragma unroll
    for (int k = 0; k < 4; ++k) v += w[k] * o_s[k * a.ec + e];
    rb::store_scalar((T *)a.out + g * a.rc + e, v / lt);
  }
}

bool mfma_sizes(int64_t rc, int64_t rotc) {
  return rc <= 512 && rotc <= MAX_ROT;
}
int padded_rank(int64_t rc) {
  return rc <= 64 ? 64 : rc <= 128 ? 128 : rc <= 256 ? 256 : 512;
}

template <int RP, int MT, int ROTP>
void launch_attend(const AttendArgs &a, dim3 grid, hipStream_t stream) {
  constexpr int planes = MT == 1 ? 2 : 1;
  constexpr size_t shmem =
      (size_t)2 * TK * ((RP + ROTP) * 2) +
      (size_t)MT * 16 * ((planes * SSTRIDE + 2) * sizeof(float) + PSTRIDE * 2);
  static_assert(shmem <= 160 * 1024, "LDS");
  static bool once = [] {
    return hipFuncSetAttribute(
               reinterpret_cast<const void *>(&latent_attend_kernel<RP, MT, ROTP>),
               hipFuncAttributeMaxDynamicSharedMemorySize,
               (int)shmem) == hipSuccess;
  }();
  TORCH_CHECK(once, "latent_attend: LDS size");
  hipLaunchKernelGGL((latent_attend_kernel<RP, MT, ROTP>), grid, dim3(BLOCK), shmem,
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
  TORCH_CHECK(rc % 8 == 0 && rc >= 8 && rotc >= 0 && rotc % 8 == 0 && q_off % 8 == 0 &&
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
                         grid, dim3(ROWS_BLOCK), shmem, stream, a);
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

  a.nsplit = (int)std::min<int64_t>(64, std::max<int64_t>(1, nsplit));
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
  auto launch = [&](auto r, auto rot) {
    constexpr int RP = decltype(r)::value, ROT = decltype(rot)::value;
    if (M == 16) launch_attend<RP, 1, ROT>(a, grid, stream);
    else if (M == 32) launch_attend<RP, 2, ROT>(a, grid, stream);
    else if constexpr (RP < 512) launch_attend<RP, 4, ROT>(a, grid, stream);
  };
  auto pick = [&](auto rot) {
    if (rp == 64) launch(std::integral_constant<int, 64>{}, rot);
    else if (rp == 128) launch(std::integral_constant<int, 128>{}, rot);
    else if (rp == 256) launch(std::integral_constant<int, 256>{}, rot);
    else launch(std::integral_constant<int, 512>{}, rot);
  };
  if (rotc > 0) pick(std::integral_constant<int, MAX_ROT>{});
  else pick(std::integral_constant<int, 0>{});
  if (a.nsplit > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3(T * H), dim3(128), 0,
                       stream, a.part_o, a.part_ml, (uint16_t *)a.out,
                       a.nsplit, a.total_rows, a.rc);
  return out;
}
