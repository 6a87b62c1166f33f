// Generalized delta rule with a decay w and a removal rate a per head and key
// channel (gfx950):
//
//   S <- diag(w) S - (a u)(u^T S) + k v^T,   o = S^T r,   u = k / |k|
//
// S [dc, vc] fp32 per sequence (its slot) and head; both terms read the old S.
// log w = scale sigmoid(logit + bias), a = sigmoid(logit + bias). A portion
// that starts at position 0 starts from zero, whatever its slot holds.
//
// y rows: [ r heads | k heads | v heads | a logits | .. ], y2 rows: [ decay
// logits ]; sizes per head are padded to 8 (zero columns). o rows: [ heads ]
// in fp32.
//
//  * general_delta_step: token after token, decoding and short portions, fp32
//    or bf16. A workgroup holds 32 columns of one state in registers.
//  * general_delta_chunk: long portions, bf16, in chunks of C = 32 tokens. With
//    alpha = a u, G_t the sum of log w over the chunk's tokens up to t and
//
//      A[t, s]  = sum_d u_t alpha_s exp(G_(t-1) - G_s)   (s < t)
//      B[t, s]  = sum_d u_t k_s     exp(G_(t-1) - G_s)   (s < t)
//      Pa[t, s] = sum_d r_t alpha_s exp(G_t - G_s)       (s <= t)
//      Pk[t, s] = sum_d r_t k_s     exp(G_t - G_s)       (s <= t)
//
//    what is removed, P_t = u_t^T S_(t-1), and the rest follow from the state
//    before the chunk:
//
//      (I + A) P = (exp(G_(t-1)) u) S + B V
//      O = (exp(G) r) S + Pk V - Pa P
//      S <- exp(G_C) S + (exp(G_C - G) k)^T V - (exp(G_C - G) alpha)^T P
//
//    A step's decay is bounded (|scale| <= 2), so the exponentials split into
//    two factors around the chunk's middle, G_m. With
//
//      R_t = exp(G_t - G_m) r_t,   U_t = exp(G_(t-1) - G_m) u_t,
//      K_s = exp(G_m - G_s) k_s,   N_s = exp(G_m - G_s) alpha_s
//
//    all four matrices are plain products of these rows, and so is the rest,
//    on the state Z = exp(G_m) S:
//
//      P = (I + A)^-1 (U Z + B V),   O = R Z + Pk V - Pa P
//      Z <- Z + K^T V - N^T P,       S <- exp(G_C - G_m) Z
//
//    general_delta_prep, parallel over chunks, inverts I + A (two triangular
//    blocks, then the one below them) and leaves everything that multiplies Z,
//    V or P as MFMA operands in lane order; general_delta_scan walks the
//    chunks, 16 state columns per four waves, in registers. An fp32 factor
//    enters a product as two bf16 parts (split.h), so the recurrence keeps
//    fp32's quality; k, r and v are bf16 as they come.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "split.h"

namespace {

using namespace split;

constexpr int BLOCK = 256;
constexpr int STEP_COLS = 32;          // state columns per workgroup, step
constexpr int C = 32;                  // tokens per chunk
constexpr int PREP = 512;              // threads of general_delta_prep
constexpr float UNIT_EPS = 1e-6f;      // under the root of a unit vector
constexpr float LOG2E = 1.4426950408889634f;

struct Args {
  const void *y, *y2;
  int64_t ny, ny2;
  int heads, dc, vc, off_k, off_v, off_a;
  const float *bias;                   // [2, heads * dc]: decay, removal
  float scale;                         // of log2 w
  float *state;                        // [slots, heads, dc, vc]
  const int *positions, *cu_q, *slots;
  float *o;                            // [T, heads * vc]
  int first_seq;
  int chunk0, chunks;                  // this launch's chunks of a sequence
  char *scratch;                       // [sequences, chunks, heads, bytes]
  int64_t entry;
};

RB_DEV float sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---------------------------------------------------------------------------
// token after token
// ---------------------------------------------------------------------------
template <typename T, int RPT>
__global__ __launch_bounds__(BLOCK) void general_delta_step_kernel(Args a) {
  constexpr int DP = RPT * 32;                 // rows held
  __shared__ float r_s[2][DP], k_s[2][DP], a_s[2][DP], w_s[2][DP];
  __shared__ float v_s[2][STEP_COLS];
  __shared__ f32x4v red[2][BLOCK / RB_WAVE][8];
  const int tid = threadIdx.x, cl = tid & 7, rg = tid >> 3;
  const int h = blockIdx.y, seq = a.first_seq + blockIdx.z;
  const int col0 = blockIdx.x * STEP_COLS, col = col0 + cl * 4;
  const bool col_ok = col < a.vc;
  const int q0 = a.cu_q[seq], q1 = a.cu_q[seq + 1];
  if (q0 >= q1) return;
  float *st = a.state + ((int64_t)a.slots[seq] * a.heads + h) * a.dc * a.vc;
  const bool fresh = a.positions[q0] == 0;
  f32x4v S[RPT];
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    const int r = rg * RPT + j;
    S[j] = !fresh && col_ok && r < a.dc
               ? *reinterpret_cast<const f32x4v *>(st + (int64_t)r * a.vc + col)
               : (f32x4v)(0.0f);
  }
  for (int t = q0; t < q1; ++t) {
    const int buf = t & 1;                     // two: a wave may run ahead
    const T *y = (const T *)a.y + (int64_t)t * a.ny + h * a.dc;
    const T *y2 = (const T *)a.y2 + (int64_t)t * a.ny2 + h * a.dc;
    for (int i = tid; i < 4 * DP + STEP_COLS; i += BLOCK) {
      const int which = i / DP, d = i - which * DP;
      if (which >= 4) {
        const int c = col0 + i - 4 * DP;
        v_s[buf][i - 4 * DP] =
            c < a.vc ? rb::bf16_to_f32_or_id(
                           ((const T *)a.y)[(int64_t)t * a.ny + a.off_v +
                                            h * a.vc + c])
                     : 0.0f;
        continue;
      }
      float f = 0.0f;
      if (d < a.dc) {
        const float *b = a.bias + h * a.dc + d;
        if (which == 0) f = rb::bf16_to_f32_or_id(y[d]);
        else if (which == 1) f = rb::bf16_to_f32_or_id(y[a.off_k + d]);
        else if (which == 2)
          f = sigmoid(rb::bf16_to_f32_or_id(y[a.off_a + d]) +
                      b[a.heads * a.dc]);
        else
          f = __builtin_amdgcn_exp2f(
              a.scale * sigmoid(rb::bf16_to_f32_or_id(y2[d]) + b[0]));
      }
      (which == 0 ? r_s : which == 1 ? k_s : which == 2 ? a_s : w_s)[buf][d] =
          f;
    }
    __syncthreads();
    const float *ks = k_s[buf];
    float nk = 0.0f;
    for (int d = tid & 63; d < DP; d += 64) nk += ks[d] * ks[d];
    nk = 1.0f / sqrtf(rb::wave_reduce_sum(nk) + UNIT_EPS);
    f32x4v p = (f32x4v)(0.0f), o = (f32x4v)(0.0f), v;
    float k[RPT];
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      k[j] = ks[rg * RPT + j];
#pragma unroll
      for (int e = 0; e < 4; ++e) p[e] += S[j][e] * (k[j] * nk);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      p[e] += __shfl_xor(p[e], 8, 64);
      p[e] += __shfl_xor(p[e], 16, 64);
      p[e] += __shfl_xor(p[e], 32, 64);
    }
    if ((tid & 63) < 8) red[0][tid >> 6][cl] = p;
    __syncthreads();
    p = red[0][0][cl] + red[0][1][cl] + red[0][2][cl] + red[0][3][cl];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = v_s[buf][cl * 4 + e];
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      const int d = rg * RPT + j;
      const float w = w_s[buf][d], r = r_s[buf][d];
      const float al = a_s[buf][d] * (k[j] * nk);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[j][e] = w * S[j][e] - al * p[e] + k[j] * v[e];
        o[e] += S[j][e] * r;
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      o[e] += __shfl_xor(o[e], 8, 64);
      o[e] += __shfl_xor(o[e], 16, 64);
      o[e] += __shfl_xor(o[e], 32, 64);
    }
    if ((tid & 63) < 8) red[1][tid >> 6][cl] = o;
    __syncthreads();
    if (tid < 8 && col_ok)
      *reinterpret_cast<f32x4v *>(a.o + (int64_t)t * a.heads * a.vc +
                                  h * a.vc + col) =
          red[1][0][cl] + red[1][1][cl] + red[1][2][cl] + red[1][3][cl];
  }
  if (!col_ok) return;
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    const int r = rg * RPT + j;
    if (r < a.dc)
      *reinterpret_cast<f32x4v *>(st + (int64_t)r * a.vc + col) = S[j];
  }
}

// ---------------------------------------------------------------------------
// chunks: operands
// ---------------------------------------------------------------------------
// One chunk and head in scratch. An operand has its big and its small part
// behind each other; V, exact in bf16, only the one.
template <int DCP> struct Entry {
  static constexpr int KS = DCP / 32, TD = DCP / 16, OP = 2048;
  static constexpr int W = 0;                  // -(I + A)^-1 U, [2 tiles][KS]
  static constexpr int R = W + 2 * KS * OP;    // [2 token tiles][KS]
  static constexpr int TB = R + 2 * KS * OP;   // -(I + A)^-1 B, [2 tiles]
  static constexpr int PK = TB + 2 * OP;       // [2 token tiles]
  static constexpr int PA = PK + 2 * OP;       // [2 token tiles]
  static constexpr int K = PA + 2 * OP;        // [TD]
  static constexpr int N = K + TD * OP;        // [TD]
  static constexpr int F = N + TD * OP;        // exp(G_m), exp(G_C - G_m) fp32
  static constexpr int V = F + DCP * 8;        // [vc / 16][64 lanes]
  static __host__ __device__ int64_t bytes(int vc) {
    return V + (int64_t)((vc + 15) / 16) * 1024;
  }
};

constexpr int AS = C + 4;              // floats per row of a token matrix
template <int DCP> struct Lds {
  static constexpr int RB = DCP + 8;   // 16-bit elements per row
  static constexpr int RS = DCP + 4;   // floats per row
  // four kinds of rows in two parts; before them, in their place, G and V
  static constexpr int rows = 8 * C * RB * 2;
  static constexpr int g = C * RS * 4;
  static constexpr int bytes = rows + 2 * C * AS * 4;
  static_assert(g + C * RB * 2 <= rows, "G and V");
};

// element k of a lane of group grp: the summed index within 32
RB_DEV constexpr int index_of(int grp, int k) {
  return grp * 4 + (k & 3) + (k >> 2) * 16;
}
// orders a wave's own LDS accesses
RB_DEV void wave_fence() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}
// a lane's elements of 32 columns of a row
RB_DEV void row8(const float *row, int grp, float *f) {
  const f32x4v lo = *reinterpret_cast<const f32x4v *>(row + grp * 4);
  const f32x4v hi = *reinterpret_cast<const f32x4v *>(row + grp * 4 + 16);
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    f[k] = lo[k];
    f[k + 4] = hi[k];
  }
}
RB_DEV void row8(const uint16_t *row, int grp, Frag &f) {
  const uint2 lo = *reinterpret_cast<const uint2 *>(row + grp * 4);
  const uint2 hi = *reinterpret_cast<const uint2 *>(row + grp * 4 + 16);
  f.u = (u32x4v){lo.x, lo.y, hi.x, hi.y};
}
// its elements of a column (l16) of 32 rows
template <int RB> RB_DEV void column8(const uint16_t *rows, int lane, Frag &f) {
  const int l16 = lane & 15, grp = lane >> 4;
  const uint16_t *p = rows + (grp * 4 + (l16 >> 2)) * RB + (l16 & 3) * 4;
  f.v = rb::lds_column8((const char *)p, (const char *)(p + 16 * RB));
}
RB_DEV void split_frag(const float *f, Frag *out) {
  split8(f, out[0].u, out[1].u);
}
// c += a b of split operands
RB_DEV f32x4v product(const Frag *a, const Frag *b, f32x4v c) {
#pragma unroll
  for (int i = 0; i < 3; ++i) c = part(i, a, b[0], b[1], c);
  return c;
}

template <int DCP>
__global__ __launch_bounds__(PREP, DCP > 128 ? 2 : 4)
void general_delta_prep_kernel(Args a, int vcp) {
  using E = Entry<DCP>;
  using T = uint16_t;
  constexpr int RB = Lds<DCP>::RB, RS = Lds<DCP>::RS, KS = E::KS;
  constexpr int L = DCP / 8;                   // threads per token
  constexpr int NV = (C * L + PREP - 1) / PREP;
  constexpr int PART = C * RB;                 // elements of a part
  enum { R = 0, U = 2, K = 4, N = 6 };         // first part of a kind of rows
  extern __shared__ __attribute__((aligned(16))) char lds[];
  uint16_t *rows = reinterpret_cast<uint16_t *>(lds);     // [8][C][RB]
  float *g_s = reinterpret_cast<float *>(lds);            // [C][RS]
  uint16_t *v_s = reinterpret_cast<uint16_t *>(lds + Lds<DCP>::g);  // [C][RB]
  float *a_s = reinterpret_cast<float *>(lds + Lds<DCP>::rows);
  float *b_s = a_s + C * AS;                   // A (then its inverse), B

  const int tid = threadIdx.x;
  const int lane = tid & 63, l16 = lane & 15, grp = lane >> 4;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, chunk = a.chunk0 + blockIdx.y;
  const int seq = a.first_seq + blockIdx.z;
  const int q0 = a.cu_q[seq], n = a.cu_q[seq + 1] - q0;
  const int t0 = chunk * C;
  if (t0 >= n) return;
  const int len = min(C, n - t0);
  char *entry = a.scratch + (((int64_t)blockIdx.z * a.chunks + blockIdx.y) *
                             a.heads + h) * a.entry;
  auto put = [&](int at, const Frag *x) {
    *reinterpret_cast<u32x4v *>(entry + at + lane * 16) = x[0].u;
    *reinterpret_cast<u32x4v *>(entry + at + 1024 + lane * 16) = x[1].u;
  };

  // ---- this thread's columns of r, k, a; log2 w and v to LDS ---------------
  const T *y = (const T *)a.y + (int64_t)(q0 + t0) * a.ny;
  const T *y2 = (const T *)a.y2 + (int64_t)(q0 + t0) * a.ny2;
  float r[NV][8], k[NV][8], al[NV][8], nk[NV];
  // vector i of this thread: token and first column; false where there is none
  auto vec = [&](int i, int &t, int &d) {
    const int v = tid + i * PREP;
    t = v / L;
    d = v % L * 8;
    return v < C * L;
  };
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    int t, d;
    const bool mine = vec(i, t, d), ok = mine && t < len && d < a.dc;
    const int64_t tt = ok ? t : 0;
    const int c = h * a.dc + (ok ? d : 0);
    float z[8], b[2][8];
    rb::VIO<T>::load(y + tt * a.ny + c, r[i]);
    rb::VIO<T>::load(y + tt * a.ny + a.off_k + c, k[i]);
    rb::VIO<T>::load(y + tt * a.ny + a.off_a + c, al[i]);
    rb::VIO<T>::load(y2 + tt * a.ny2 + c, z);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      b[0][e] = a.bias[c + e];
      b[1][e] = a.bias[a.heads * a.dc + c + e];
    }
    float s = 0.0f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      if (!ok) r[i][e] = k[i][e] = 0.0f;
      al[i][e] = sigmoid(al[i][e] + b[1][e]);
      z[e] = ok ? a.scale * sigmoid(z[e] + b[0][e]) : 0.0f;
      s += k[i][e] * k[i][e];
    }
#pragma unroll
    for (int o = L / 2; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
    nk[i] = 1.0f / sqrtf(s + UNIT_EPS);
    if (mine) rb::VIO<float>::store(g_s + t * RS + d, z);
    if (mine) rb::VIO<float>::store(g_s + t * RS + d + 4, z + 4);
  }
  for (int i = tid; i < C * (vcp / 8); i += PREP) {
    const int t = i / (vcp / 8), c = i % (vcp / 8) * 8;
    u32x4v v = (u32x4v)(0u);
    if (t < len && c < a.vc)
      v = *reinterpret_cast<const u32x4v *>(y + (int64_t)t * a.ny + a.off_v +
                                            h * a.vc + c);
    *reinterpret_cast<u32x4v *>(v_s + t * RB + c) = v;
  }
  __syncthreads();
  // ---- G: sums of log2 w over tokens; the other waves write V -------------
  constexpr int SUMS = (DCP + RB_WAVE - 1) / RB_WAVE;      // waves
  if (wid < SUMS) {
    const int d = tid;
    if (d < DCP) {
      float s[C];
#pragma unroll
      for (int t = 0; t < C; ++t) s[t] = g_s[t * RS + d];
#pragma unroll
      for (int t = 1; t < C; ++t) s[t] += s[t - 1];
#pragma unroll
      for (int t = 1; t < C; ++t) g_s[t * RS + d] = s[t];
      float *f = reinterpret_cast<float *>(entry + E::F);
      f[d] = __builtin_amdgcn_exp2f(s[C / 2 - 1]);
      f[DCP + d] = __builtin_amdgcn_exp2f(s[C - 1] - s[C / 2 - 1]);
    }
  } else {
    for (int i = wid - SUMS; i < vcp / 16; i += PREP / RB_WAVE - SUMS) {
      Frag x;
      column8<RB>(v_s + i * 16, lane, x);
      *reinterpret_cast<u32x4v *>(entry + E::V + i * 1024 + lane * 16) = x.u;
    }
  }
  __syncthreads();
  // ---- the four kinds of rows, in two parts each ----------------------------
  u32x4v part_r[NV][2], part_u[NV][2], part_k[NV][2], part_n[NV][2];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    int t, d;
    if (!vec(i, t, d)) t = d = 0;
    float g[8], before[8], mid[8], u[8], x[8];
    const float *gp = g_s + t * RS + d;
    const float *bp = gp - (t > 0 ? RS : 0), *mp = g_s + (C / 2 - 1) * RS + d;
#pragma unroll
    for (int e = 0; e < 8; e += 4) {
      rb::VIO<float>::load(gp + e, g + e);
      rb::VIO<float>::load(bp + e, before + e);
      rb::VIO<float>::load(mp + e, mid + e);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      u[e] = k[i][e] * nk[i];
      x[e] = r[i][e] * __builtin_amdgcn_exp2f(g[e] - mid[e]);
    }
    split8(x, part_r[i][0], part_r[i][1]);
#pragma unroll
    for (int e = 0; e < 8; ++e)
      x[e] = u[e] *
             __builtin_amdgcn_exp2f((t > 0 ? before[e] : 0.0f) - mid[e]);
    split8(x, part_u[i][0], part_u[i][1]);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      g[e] = __builtin_amdgcn_exp2f(mid[e] - g[e]);
      x[e] = k[i][e] * g[e];
    }
    split8(x, part_k[i][0], part_k[i][1]);
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = al[i][e] * u[e] * g[e];
    split8(x, part_n[i][0], part_n[i][1]);
  }
  __syncthreads();                             // G and V have been read
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    int t, d;
    if (!vec(i, t, d)) continue;
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      uint16_t *at = rows + p * PART + t * RB + d;
      *reinterpret_cast<u32x4v *>(at + R * PART) = part_r[i][p];
      *reinterpret_cast<u32x4v *>(at + U * PART) = part_u[i][p];
      *reinterpret_cast<u32x4v *>(at + K * PART) = part_k[i][p];
      *reinterpret_cast<u32x4v *>(at + N * PART) = part_n[i][p];
    }
  }
  __syncthreads();
  // ---- the four token matrices: a wave has 16 rows (tokens t) of one. The
  // lane's results, row t = l16 and four neighbouring s per tile, are, packed,
  // an operand. ----------------------------------------------------------------
  {
    const int with_r = wid >> 2, m = (wid >> 1) & 1, with_k = wid & 1;
    const int t = m * 16 + l16;
    const uint16_t *tp = rows + (with_r ? R : U) * PART + t * RB;
    const uint16_t *sp = rows + (with_k ? K : N) * PART + l16 * RB;
    f32x4v acc[2] = {(f32x4v)(0.0f), (f32x4v)(0.0f)};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      Frag row[2], col[2];
#pragma unroll
      for (int p = 0; p < 2; ++p) row8(tp + p * PART + ks * 32, grp, row[p]);
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        if (j > m) break;                      // above the diagonal
#pragma unroll
        for (int p = 0; p < 2; ++p)
          row8(sp + p * PART + j * 16 * RB + ks * 32, grp, col[p]);
        acc[j] = product(col, row, acc[j]);
      }
      if (with_r && with_k)                    // these rows multiply Z, too
        put(E::R + (m * KS + ks) * E::OP, row);
    }
    float f[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int s = index_of(grp, e);
      f[e] = s < t || (with_r && s == t) ? acc[e >> 2][e & 3] : 0.0f;
    }
    if (with_r) {
      Frag x[2];
      split_frag(f, x);
      put((with_k ? E::PK : E::PA) + m * E::OP, x);
    } else {
      float *dst = (with_k ? b_s : a_s) + t * AS + grp * 4;
      *reinterpret_cast<f32x4v *>(dst) = (f32x4v){f[0], f[1], f[2], f[3]};
      *reinterpret_cast<f32x4v *>(dst + 16) = (f32x4v){f[4], f[5], f[6], f[7]};
    }
  }
  __syncthreads();
  if (wid == 0) {
    // ---- (I + A)^-1 in A's place: column l16 of a 16 x 16 block per lane,
    // then the block below the diagonal, -T22 (A21 T11) ---------------------
    const int b0 = (lane >> 4 & 1) * 16;
    float x[16], f[8] = {}, z[8] = {};
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      x[i] = i == l16 ? 1.0f : 0.0f;
#pragma unroll
      for (int j = 0; j < i; ++j)
        x[i] -= a_s[(b0 + i) * AS + b0 + j] * x[j];
    }
    wave_fence();
    if (lane < 32) {
#pragma unroll
      for (int i = 0; i < 16; ++i)
        a_s[(b0 + i) * AS + b0 + l16] = x[i];
    }
    wave_fence();
    Frag fa[2], fb[2];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      f[e] = a_s[(16 + l16) * AS + grp * 4 + e];
      z[e] = a_s[(grp * 4 + e) * AS + l16];
    }
    split_frag(f, fa);
    split_frag(z, fb);
    f32x4v c = product(fa, fb, (f32x4v)(0.0f));
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      f[e] = a_s[(16 + l16) * AS + 16 + grp * 4 + e];
      z[e] = c[e];
    }
    split_frag(f, fa);
    split_frag(z, fb);
    c = product(fa, fb, (f32x4v)(0.0f));
    wave_fence();
#pragma unroll
    for (int e = 0; e < 4; ++e)
      a_s[(16 + grp * 4 + e) * AS + l16] = -c[e];
  } else {
    // ---- the keys and alphas of a state row ---------------------------------
    for (int i = wid - 1; i < 2 * E::TD; i += PREP / RB_WAVE - 1) {
      const int tile = i >> 1;
      const uint16_t *p = rows + (i & 1 ? N : K) * PART + tile * 16;
      Frag x[2];
      column8<RB>(p, lane, x[0]);
      column8<RB>(p + PART, lane, x[1]);
      put((i & 1 ? E::N : E::K) + tile * E::OP, x);
    }
  }
  __syncthreads();
  // ---- what the inverse multiplies: U, and B. A result's rows are the other
  // factor's columns, so that it is an operand, too. ---------------------------
  for (int i = wid; i < 2 * KS + 2; i += PREP / RB_WAVE) {
    const int m = i < 2 * KS ? i / KS : i - 2 * KS;
    float f[8], out[8];
    Frag inv[2], x[2];
    row8(a_s + (m * 16 + l16) * AS, grp, f);
    split_frag(f, inv);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      if (i < 2 * KS) {
        const uint16_t *p = rows + U * PART + i % KS * 32 + j * 16;
        column8<RB>(p, lane, x[0]);
        column8<RB>(p + PART, lane, x[1]);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          f[e] = b_s[index_of(grp, e) * AS + j * 16 + l16];
        split_frag(f, x);
      }
      const f32x4v c = product(x, inv, (f32x4v)(0.0f));
#pragma unroll
      for (int e = 0; e < 4; ++e) out[j * 4 + e] = -c[e];
    }
    split_frag(out, x);
    put(i < 2 * KS ? E::W + i * E::OP : E::TB + m * E::OP, x);
  }
}

// ---------------------------------------------------------------------------
// chunks: the recurrence. Four waves own 16 state columns, a quarter of the
// rows each, as MFMA result tiles; packed, two stacked ones are an operand.
// They exchange Z, packed, through LDS. Two waves (one per tile of 16 tokens)
// make -P, the two others O; all four bring their rows up to date.
// ---------------------------------------------------------------------------
template <int DCP>
__global__ __launch_bounds__(4 * RB_WAVE, 1)
void general_delta_scan_kernel(Args a) {
  using E = Entry<DCP>;
  constexpr int KS = E::KS, HT = E::TD < 4 ? 1 : E::TD / 4;
  __shared__ u32x4v s_s[2][KS][64], u_s[2][64];
  const int lane = threadIdx.x & 63, l16 = lane & 15, grp = lane >> 4;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int m = wid & 1;                       // token tile
  const bool out = wid >= 2;                   // makes O
  const bool owns = wid * HT < E::TD;          // has state tiles
  const int first = owns ? wid * HT : 0;
  const int h = blockIdx.x % a.heads, cb = blockIdx.x / a.heads;
  const int seq = a.first_seq + blockIdx.z;
  const int q0 = a.cu_q[seq], n = a.cu_q[seq + 1] - q0;
  const int nc = min(a.chunks, (n + C - 1) / C - a.chunk0);
  if (nc <= 0) return;
  const int col = cb * 16 + l16;
  const bool col_ok = col < a.vc;
  float *st = a.state + ((int64_t)a.slots[seq] * a.heads + h) * a.dc * a.vc;
  const bool zero = a.chunk0 == 0 && a.positions[q0] == 0;
  f32x4v S[HT];
#pragma unroll
  for (int d = 0; d < HT; ++d)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int dim = (first + d) * 16 + grp * 4 + r;
      S[d][r] = !zero && owns && col_ok && dim < a.dc
                    ? st[(int64_t)dim * a.vc + col] : 0.0f;
    }
  const int64_t stride = a.heads * a.entry;
  const char *base = a.scratch +
                     ((int64_t)blockIdx.z * a.chunks * a.heads + h) * a.entry;
  const int64_t orow = (int64_t)a.heads * a.vc;
  const int tok = a.chunk0 * C + m * 16 + grp * 4;
  float *op = a.o + (int64_t)(q0 + tok) * orow + h * a.vc + col;
  int left = n - tok;                          // tokens from this lane's on

  // what multiplies Z, V (TB or Pk; the keys) and P (Pa; the alphas)
  struct Operands {
    Frag ff[KS][2], tf[2], pf[2], kf[HT][2], af[HT][2], vf;
    f32x4v f0[HT], f1[HT];                     // S to Z and back
  };
  auto get = [&](Frag *f, const char *e) __attribute__((always_inline)) {
    f[0].u = *reinterpret_cast<const u32x4v *>(e + lane * 16);
    f[1].u = *reinterpret_cast<const u32x4v *>(e + 1024 + lane * 16);
  };
  auto load = [&](Operands &o, int c) __attribute__((always_inline)) {
    const char *e = base + min(c, nc - 1) * stride;
    o.vf.u = *reinterpret_cast<const u32x4v *>(e + E::V + cb * 1024 +
                                               lane * 16);
#pragma unroll
    for (int d = 0; d < HT; ++d) {
      const char *f = e + E::F + ((first + d) * 16 + grp * 4) * 4;
      o.f0[d] = *reinterpret_cast<const f32x4v *>(f);
      o.f1[d] = *reinterpret_cast<const f32x4v *>(f + DCP * 4);
      get(o.kf[d], e + E::K + (first + d) * E::OP);
    }
    get(o.tf, e + (out ? E::PK : E::TB) + m * E::OP);
    const char *f = e + (out ? E::R : E::W) + m * KS * E::OP;
#pragma unroll
    for (int i = 0; i < KS; ++i) get(o.ff[i], f + i * E::OP);
#pragma unroll
    for (int d = 0; d < HT; ++d) get(o.af[d], e + E::N + (first + d) * E::OP);
    if (out) get(o.pf, e + E::PA + m * E::OP);
  };
  auto step = [&](const Operands &o) __attribute__((always_inline)) {
#pragma unroll
    for (int d = 0; d < HT; ++d)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[d][r] *= o.f0[d][r];
    if (owns) {
#pragma unroll
      for (int d = 0; d < HT; ++d) {
        const int t = first + d;
        uint2 big, small;
        split2(S[d][0], S[d][1], big.x, small.x);
        split2(S[d][2], S[d][3], big.y, small.y);
        reinterpret_cast<uint2 *>(&s_s[0][t >> 1][lane])[t & 1] = big;
        reinterpret_cast<uint2 *>(&s_s[1][t >> 1][lane])[t & 1] = small;
      }
    }
    // meanwhile: what V gives to the state and to the tokens
    f32x4v x[2];
    x[0] = mfma(o.tf[0], o.vf, (f32x4v)(0.0f));
    x[1] = mfma(o.tf[1], o.vf, (f32x4v)(0.0f));
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int d = 0; d < HT; ++d) S[d] = mfma(o.kf[d][i], o.vf, S[d]);
    __syncthreads();                           // Z; P has been read
    Frag sf[KS][2];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      sf[ks][0].u = s_s[0][ks][lane];
      sf[ks][1].u = s_s[1][ks][lane];
    }
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int i = 0; i < 3; ++i)
        x[(ks * 3 + i) & 1] = part(i, o.ff[ks], sf[ks][0], sf[ks][1],
                                   x[(ks * 3 + i) & 1]);
    f32x4v y = x[0] + x[1];
    if (!out) {
      uint2 big, small;
      split2(y[0], y[1], big.x, small.x);
      split2(y[2], y[3], big.y, small.y);
      reinterpret_cast<uint2 *>(&u_s[0][lane])[m] = big;
      reinterpret_cast<uint2 *>(&u_s[1][lane])[m] = small;
    }
    __syncthreads();                           // P; Z has been read
    Frag u[2];
    u[0].u = u_s[0][lane];
    u[1].u = u_s[1][lane];
#pragma unroll
    for (int i = 0; i < 3; ++i)
#pragma unroll
      for (int d = 0; d < HT; ++d) S[d] = part(i, o.af[d], u[0], u[1], S[d]);
#pragma unroll
    for (int d = 0; d < HT; ++d)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[d][r] *= o.f1[d][r];
    if (out) {
      y = product(o.pf, u, y);
      if (col_ok) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (r < left) op[r * orow] = y[r];
      }
    }
    op += C * orow;
    left -= C;
  };
  // a chunk's operands are on their way while the one before it is walked
  Operands even, odd;
  load(even, 0);
  for (int c = 0; c < nc; c += 2) {
    load(odd, c + 1);
    __builtin_amdgcn_sched_barrier(0);
    step(even);
    if (c + 1 >= nc) break;
    load(even, c + 2);
    __builtin_amdgcn_sched_barrier(0);
    step(odd);
  }
  if (!col_ok || !owns) return;
#pragma unroll
  for (int d = 0; d < HT; ++d)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int dim = (first + d) * 16 + grp * 4 + r;
      if (dim < a.dc) st[(int64_t)dim * a.vc + col] = S[d][r];
    }
}

Args check(const at::Tensor &y, const at::Tensor &y2, const at::Tensor &bias,
           double scale, const at::Tensor &state, const at::Tensor &positions,
           const at::Tensor &cu_q, const at::Tensor &slots,
           const at::Tensor &o, int64_t first_seq, int64_t n_seqs,
           const char *who) {
  const auto dt = y.scalar_type();
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (dt == at::kBFloat16 || dt == at::kFloat) && y2.dim() == 2 &&
              y2.is_contiguous() && y2.scalar_type() == dt &&
              y2.size(0) == y.size(0) && state.dim() == 4 &&
              state.is_contiguous() && state.scalar_type() == at::kFloat,
              who, ": y, y2, state [slots, heads, dc, vc] f32");
  const int64_t H = state.size(1), dc = state.size(2), vc = state.size(3);
  const int64_t off_a = H * (2 * dc + vc);
  TORCH_CHECK(dc >= 8 && dc % 8 == 0 && dc <= 256 && vc >= 8 && vc % 8 == 0 &&
              H <= 65535 && y.size(1) % 8 == 0 &&
              off_a + H * dc <= y.size(1) && y2.size(1) % 8 == 0 &&
              H * dc <= y2.size(1) && bias.is_contiguous() &&
              bias.scalar_type() == at::kFloat && bias.numel() == 2 * H * dc,
              who, ": layout");
  TORCH_CHECK(scale <= 0.0 && scale >= -2.0, who, ": decay scale ", scale);
  TORCH_CHECK(o.scalar_type() == at::kFloat && o.is_contiguous() &&
              o.dim() == 2 && o.size(0) == y.size(0) && o.size(1) == H * vc,
              who, ": o [T, heads * vc] f32");
  TORCH_CHECK(positions.scalar_type() == at::kInt &&
              positions.is_contiguous() && positions.numel() == y.size(0) &&
              cu_q.scalar_type() == at::kInt && cu_q.is_contiguous() &&
              slots.scalar_type() == at::kInt && slots.is_contiguous() &&
              first_seq >= 0 && n_seqs >= 0 && n_seqs <= 65535 &&
              cu_q.numel() > first_seq + n_seqs &&
              slots.numel() >= first_seq + n_seqs, who, ": batch tensors");
  Args a{};
  a.y = y.data_ptr();
  a.y2 = y2.data_ptr();
  a.ny = y.size(1);
  a.ny2 = y2.size(1);
  a.heads = (int)H;
  a.dc = (int)dc;
  a.vc = (int)vc;
  a.off_k = (int)(H * dc);
  a.off_v = (int)(2 * H * dc);
  a.off_a = (int)off_a;
  a.bias = bias.data_ptr<float>();
  a.scale = (float)(scale * LOG2E);
  a.state = state.data_ptr<float>();
  a.positions = positions.data_ptr<int>();
  a.cu_q = cu_q.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.o = o.data_ptr<float>();
  a.first_seq = (int)first_seq;
  return a;
}

template <int DCP>
void launch_chunk(Args a, int64_t n_seqs, int64_t max_q,
                  const at::TensorOptions &options, hipStream_t stream) {
  const int vcp = (a.vc + 15) / 16 * 16;
  constexpr int shmem = Lds<DCP>::bytes;
  static_assert(shmem <= 159 * 1024, "LDS");
  static bool once = [] {
    return hipFuncSetAttribute(
               reinterpret_cast<const void *>(&general_delta_prep_kernel<DCP>),
               hipFuncAttributeMaxDynamicSharedMemorySize,
               shmem) == hipSuccess;
  }();
  TORCH_CHECK(once && vcp <= DCP, "general_delta_chunk: LDS size");
  a.entry = Entry<DCP>::bytes(a.vc);
  // as many chunks at once as keep the entries in the last-level cache
  const int64_t all = (max_q + C - 1) / C;
  const int64_t fit = ((int64_t)192 << 20) / (n_seqs * a.heads * a.entry);
  a.chunks = (int)std::min<int64_t>(all, std::max<int64_t>(fit, 16));
  TORCH_CHECK(a.chunks <= 65535, "general_delta_chunk: portion of ", max_q);
  auto scratch = at::empty({n_seqs * a.chunks * a.heads * a.entry}, options);
  a.scratch = (char *)scratch.data_ptr();
  const dim3 scan(a.heads * (vcp / 16), 1, n_seqs);
  for (int64_t c = 0; c < all; c += a.chunks) {
    a.chunk0 = (int)c;
    hipLaunchKernelGGL((general_delta_prep_kernel<DCP>),
                       dim3(a.heads, a.chunks, n_seqs), dim3(PREP), shmem,
                       stream, a, vcp);
    hipLaunchKernelGGL((general_delta_scan_kernel<DCP>), scan,
                       dim3(4 * RB_WAVE), 0, stream, a);
  }
}

}  // namespace

// o and the new state of the first n_seqs sequences
void general_delta_step(at::Tensor y, at::Tensor y2, at::Tensor bias,
                        double scale, at::Tensor state, at::Tensor positions,
                        at::Tensor cu_q, at::Tensor slots, at::Tensor o,
                        int64_t n_seqs) {
  const Args a = check(y, y2, bias, scale, state, positions, cu_q, slots, o, 0,
                       n_seqs, "general_delta_step");
  if (n_seqs == 0) return;
  const dim3 grid((a.vc + STEP_COLS - 1) / STEP_COLS, a.heads, n_seqs);
  auto stream = at::hip::getCurrentHIPStream();
  auto pick = [&](auto tag) {
    using E = decltype(tag);
    auto go = [&](auto rpt) {
      hipLaunchKernelGGL((general_delta_step_kernel<E, decltype(rpt)::value>),
                         grid, dim3(BLOCK), 0, stream, a);
    };
    if (a.dc <= 32) go(std::integral_constant<int, 1>{});
    else if (a.dc <= 64) go(std::integral_constant<int, 2>{});
    else if (a.dc <= 128) go(std::integral_constant<int, 4>{});
    else go(std::integral_constant<int, 8>{});
  };
  if (y.scalar_type() == at::kBFloat16) pick(uint16_t{});
  else pick(float{});
}

// the same for the sequences first_seq .. first_seq + n_seqs - 1, the
// longest of which has max_q tokens in y
void general_delta_chunk(at::Tensor y, at::Tensor y2, at::Tensor bias,
                         double scale, at::Tensor state, at::Tensor positions,
                         at::Tensor cu_q, at::Tensor slots, at::Tensor o,
                         int64_t first_seq, int64_t n_seqs, int64_t max_q) {
  const Args a = check(y, y2, bias, scale, state, positions, cu_q, slots, o,
                       first_seq, n_seqs, "general_delta_chunk");
  TORCH_CHECK(y.scalar_type() == at::kBFloat16 && a.vc <= 256,
              "general_delta_chunk: bf16, values up to 256");
  if (n_seqs == 0 || max_q == 0) return;
  const auto bytes = y.options().dtype(at::kByte);
  auto stream = at::hip::getCurrentHIPStream();
  const int wide = std::max(a.dc, a.vc);
  if (wide <= 32) launch_chunk<32>(a, n_seqs, max_q, bytes, stream);
  else if (wide <= 64) launch_chunk<64>(a, n_seqs, max_q, bytes, stream);
  else if (wide <= 128) launch_chunk<128>(a, n_seqs, max_q, bytes, stream);
  else launch_chunk<256>(a, n_seqs, max_q, bytes, stream);
}
