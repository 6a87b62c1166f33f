// Gated delta rule with one decay per head and key channel (gfx950):
//
//   S <- g S,  u = beta (v - S^T k),  S <- S + k u^T,  o = S^T q
//
// S [dc, vc] fp32 per sequence (its slot) and head. q, k, v pass a causal
// convolution over time and silu; q and k are then unit vectors, q also times
// dim^-1/2. log g = -exp(a_log) softplus(logit + bias). A portion that starts
// at position 0 starts from zero, whatever its slot holds.
//
// y rows: [ q heads | k heads | v heads | beta | .. ], y2 rows: [ decay logits
// | gate logits ]; sizes per head are padded to 8 (zero columns). o rows:
// [ heads ] in fp32.
//
//  * delta_step: token after token, decoding and short portions, fp32 or
//    bf16. A workgroup holds 32 columns of one state in registers.
//  * delta_chunk: long portions, bf16, in chunks of C = 32 tokens. With
//    G_t the sum of log g over the chunk's tokens up to t,
//
//      A[t, s] = beta_t sum_d k_t k_s exp(G_t - G_s)    (s < t)
//      P[t, s] =        sum_d q_t k_s exp(G_t - G_s)    (s <= t)
//      (I + A) U = beta V - (beta exp(G) K) S
//      O = (exp(G) Q) S + P U,   S <- exp(G_C) S + (exp(G_C - G) K)^T U
//
//    delta_prep, parallel over chunks, solves for both right sides and leaves
//    what multiplies S or U as MFMA operands in lane order; delta_scan walks
//    the chunks, 16 state columns per two waves, in registers. Exponents are
//    differences that are never positive. An fp32 factor enters a product as
//    two bf16 parts, so the recurrence keeps fp32's quality.
//
// delta_out.hip norms and gates o and moves the convolutions' last inputs to
// the sequences' slots.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "split.h"

namespace {

constexpr int BLOCK = 256;
constexpr int STEP_COLS = 32;          // state columns per workgroup, step
constexpr int C = 32;                  // tokens per chunk
constexpr int PREP = 512;              // threads of delta_prep
constexpr int VB = 256;                // value columns staged at once
constexpr float UNIT_EPS = 1e-6f;
constexpr float LOG2E = 1.4426950408889634f;

using namespace split;

typedef __attribute__((ext_vector_type(2))) float f32x2v;

struct Args {
  const void *y, *y2;
  int64_t ny, ny2;
  int heads, kv, dim, dc, vc, taps, off_k, off_v, off_b;
  const float *conv;                   // [taps, off_b]
  const float *decay;                  // [heads, dc] biases, [heads] factors
  float *state;                        // [slots, heads, dc, vc]
  void *tails;                         // [slots, taps - 1, off_b]
  const int *positions, *cu_q, *slots;
  float *o;                            // [T, heads * vc]
  float qscale;
  int first_seq;
  int chunk0, chunks;                  // this launch's chunks of a sequence
  char *scratch;                       // [sequences, chunks, heads, bytes]
  int64_t entry;
};

template <typename T> RB_DEV float sigmoid(float x) {
  if constexpr (sizeof(T) == 2)
    return __builtin_amdgcn_rcpf(1.0f + __expf(-x));
  else
    return 1.0f / (1.0f + expf(-x));
}
RB_DEV float gate(float x) { return 1.0f / (1.0f + expf(-x)); }
template <typename T> RB_DEV float softplus(float x) {
  if constexpr (sizeof(T) == 2) {
    const float e = __expf(-fabsf(x));
    return fmaxf(x, 0.0f) +
           (e < 1e-3f ? e - 0.5f * e * e : __logf(1.0f + e));
  }
  return fmaxf(x, 0.0f) + log1pf(expf(-fabsf(x)));
}

// N neighbouring values of T or fp32
template <int N, typename E> RB_DEV void load_n(const E *p, float *f) {
  if constexpr (N == 8) {
    rb::VIO<E>::load(p, f);
    if constexpr (rb::VIO<E>::W == 4) rb::VIO<E>::load(p + 4, f + 4);
  } else {
#pragma unroll
    for (int k = 0; k < N; ++k) f[k] = rb::bf16_to_f32_or_id(p[k]);
  }
}

// Convolution and silu of N neighbouring channels at token t of the portion
// that starts at row q0.
template <typename T, int N>
RB_DEV void conv(const Args &a, int q0, int t, bool fresh, int slot, int ch,
                 float *out) {
#pragma unroll
  for (int k = 0; k < N; ++k) out[k] = 0.0f;
  const T *now = (const T *)a.y + (int64_t)(q0 + t) * a.ny + ch;
  for (int j0 = 0; j0 < a.taps; j0 += 4) {
    float f[4][N], w[4][N];
    // a tap that does not count reads the current token
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int j = j0 + i, back = a.taps - 1 - j, s = t - back;
      const T *p = now - (int64_t)back * a.ny;
      if (s < 0)
        p = (const T *)a.tails +
            ((int64_t)slot * (a.taps - 1) + a.taps - 1 + s) * a.off_b + ch;
      if (j >= a.taps || (s < 0 && fresh)) p = now;
      load_n<N>(p, f[i]);
      load_n<N>(a.conv + (int64_t)min(j, a.taps - 1) * a.off_b + ch, w[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int j = j0 + i;
      const bool ok = j < a.taps && (t - (a.taps - 1) + j >= 0 || !fresh);
#pragma unroll
      for (int k = 0; k < N; ++k) out[k] += ok ? f[i][k] * w[i][k] : 0.0f;
    }
  }
#pragma unroll
  for (int k = 0; k < N; ++k) out[k] *= sigmoid<T>(out[k]);
}

// log2 g of N neighbouring channels of one head
template <typename T, int N>
RB_DEV void log_decay(const Args &a, int64_t row, int h, int d, float *out) {
  float x[N], b[N];
  load_n<N>((const T *)a.y2 + row * a.ny2 + h * a.dc + d, x);
  load_n<N>(a.decay + h * a.dc + d, b);
  const float f = LOG2E * a.decay[a.heads * a.dc + h];
#pragma unroll
  for (int k = 0; k < N; ++k) out[k] = f * softplus<T>(x[k] + b[k]);
}

// ---------------------------------------------------------------------------
// token after token
// ---------------------------------------------------------------------------
template <typename T, int RPT>
__global__ __launch_bounds__(BLOCK) void delta_step_kernel(Args a) {
  constexpr int DP = RPT * 32;                 // rows held
  __shared__ float qk_s[2][2 * DP], g_s[2][DP], v_s[2][STEP_COLS], b_s[2];
  __shared__ f32x4v red[2][BLOCK / RB_WAVE][8];
  const int tid = threadIdx.x, cl = tid & 7, rg = tid >> 3;
  const int h = blockIdx.y, seq = a.first_seq + blockIdx.z;
  const int col0 = blockIdx.x * STEP_COLS, col = col0 + cl * 4;
  const bool col_ok = col < a.vc;
  const int q0 = a.cu_q[seq], q1 = a.cu_q[seq + 1];
  if (q0 >= q1) return;
  const int slot = a.slots[seq], kh = h / (a.heads / a.kv);
  float *st = a.state + ((int64_t)slot * a.heads + h) * a.dc * a.vc;
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
    for (int i = tid; i < 3 * DP + STEP_COLS + 1; i += BLOCK) {
      if (i < 2 * DP) {
        const int which = i / DP, d = i - which * DP;
        float f = 0.0f;
        if (d < a.dc)
          conv<T, 1>(a, q0, t - q0, fresh, slot,
                     which * a.off_k + kh * a.dc + d, &f);
        qk_s[buf][i] = f;
      } else if (i < 3 * DP) {
        const int d = i - 2 * DP;
        float f = -INFINITY;
        if (d < a.dc) log_decay<T, 1>(a, t, h, d, &f);
        g_s[buf][d] = __builtin_amdgcn_exp2f(f);
      } else if (i < 3 * DP + STEP_COLS) {
        const int c = i - 3 * DP;
        float f = 0.0f;
        if (col0 + c < a.vc)
          conv<T, 1>(a, q0, t - q0, fresh, slot,
                     a.off_v + h * a.vc + col0 + c, &f);
        v_s[buf][c] = f;
      } else {
        b_s[buf] = gate(rb::bf16_to_f32_or_id(
            ((const T *)a.y)[(int64_t)t * a.ny + a.off_b + h]));
      }
    }
    __syncthreads();
    const float *qs = qk_s[buf], *ks = qs + DP;
    float nq = 0.0f, nk = 0.0f;
    for (int d = tid & 63; d < DP; d += 64) {
      nq += qs[d] * qs[d];
      nk += ks[d] * ks[d];
    }
    nq = a.qscale / sqrtf(rb::wave_reduce_sum(nq) + UNIT_EPS);
    nk = 1.0f / sqrtf(rb::wave_reduce_sum(nk) + UNIT_EPS);
    f32x4v p = (f32x4v)(0.0f), o = (f32x4v)(0.0f), u;
    float k[RPT];
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      const int r = rg * RPT + j;
      const float g = g_s[buf][r];
      k[j] = ks[r] * nk;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[j][e] *= g;
        p[e] += S[j][e] * k[j];
      }
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
    const float beta = b_s[buf];
#pragma unroll
    for (int e = 0; e < 4; ++e) u[e] = beta * (v_s[buf][cl * 4 + e] - p[e]);
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      const float q = qs[rg * RPT + j] * nq;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[j][e] += k[j] * u[e];
        o[e] += S[j][e] * q;
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
// One chunk and head in scratch. An operand is 64 lanes x 16 bytes, its big
// and its small part behind each other. Its summed index runs, in lane l,
// 4 (l / 16) + {0..3} and 16 + that.
template <int DCP> struct Entry {
  static constexpr int KS = DCP / 32, TD = DCP / 16, OP = 2048;
  static constexpr int W = 0;                  // -(beta exp(G) K), solved:
  static constexpr int Q = W + 2 * KS * OP;    // [2 token tiles][KS]
  static constexpr int P = Q + 2 * KS * OP;    // [2 token tiles]
  static constexpr int K = P + 2 * OP;         // [TD]
  static constexpr int G = K + TD * OP;        // exp(G_C), [DCP] fp32
  static constexpr int U = G + DCP * 4;        // [vc / 16][2][64][4] fp32
  static __host__ __device__ int64_t bytes(int vc) {
    return U + (int64_t)((vc + 15) / 16) * 2048;
  }
};

template <int DCP> constexpr int prep_lds(int vb) {
  return (3 * C * (DCP + 4) + C * (vb + 4) + 2 * C * (C + 4) + C) * 4;
}

template <int DCP>
__global__ __launch_bounds__(PREP, 2) void delta_prep_kernel(Args a, int vb) {
  using E = Entry<DCP>;
  using T = uint16_t;
  constexpr int RS = DCP + 4, AS = C + 4;      // floats per LDS row
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float *q_s = lds, *k_s = q_s + C * RS, *g_s = k_s + C * RS;
  float *a_s = g_s + C * RS;                   // A transposed
  float *p_s = a_s + C * AS, *b_s = p_s + C * AS;
  float *v_s = b_s + C;
  const int VS = vb + 4;

  const int tid = threadIdx.x;
  const int h = blockIdx.x, chunk = a.chunk0 + blockIdx.y;
  const int seq = a.first_seq + blockIdx.z;
  const int q0 = a.cu_q[seq], n = a.cu_q[seq + 1] - q0;
  const int t0 = chunk * C;
  if (t0 >= n) return;
  const int len = min(C, n - t0);
  const int slot = a.slots[seq], kh = h / (a.heads / a.kv);
  const bool fresh = a.positions[q0] == 0;
  char *entry = a.scratch + (((int64_t)blockIdx.z * a.chunks + blockIdx.y) *
                             a.heads + h) * a.entry;

  auto stage_v = [&](int c0) {
#pragma unroll 2
    for (int i = tid; i < C * (vb / 8); i += PREP) {
      const int t = i / (vb / 8), c = i % (vb / 8) * 8;
      float f[8] = {};
      if (t < len && c0 + c < a.vc)
        conv<T, 8>(a, q0, t0 + t, fresh, slot, a.off_v + h * a.vc + c0 + c, f);
#pragma unroll
      for (int k = 0; k < 8; ++k) v_s[t * VS + c + k] = f[k];
    }
  };
  // ---- q, k, log g, beta, v ----------------------------------------------
#pragma unroll 2
  for (int i = tid; i < 2 * C * (DCP / 8); i += PREP) {
    const int which = i / (C * (DCP / 8)), r = i % (C * (DCP / 8));
    const int t = r / (DCP / 8), d = r % (DCP / 8) * 8;
    float f[8] = {};
    if (t < len && d < a.dc)
      conv<T, 8>(a, q0, t0 + t, fresh, slot,
                 which * a.off_k + kh * a.dc + d, f);
    float *dst = (which ? k_s : q_s) + t * RS + d;
#pragma unroll
    for (int k = 0; k < 8; ++k) dst[k] = f[k];
  }
#pragma unroll 2
  for (int i = tid; i < C * (DCP / 8); i += PREP) {
    const int t = i / (DCP / 8), d = i % (DCP / 8) * 8;
    float f[8] = {};
    if (t < len && d < a.dc) log_decay<T, 8>(a, q0 + t0 + t, h, d, f);
#pragma unroll
    for (int k = 0; k < 8; ++k) g_s[t * RS + d + k] = f[k];
  }
  if (tid < C)
    b_s[tid] = tid < len
        ? gate(rb::bf16_to_f32(((const T *)a.y)[(int64_t)(q0 + t0 + tid) *
                                                a.ny + a.off_b + h]))
        : 0.0f;
  stage_v(0);
  __syncthreads();
  // ---- unit vectors (8 lanes per token); sums of log g --------------------
  {
    const int t = tid >> 4, l = tid & 15;
    float sq = 0.0f, sk = 0.0f;
    for (int d = l; d < DCP; d += 16) {
      sq += q_s[t * RS + d] * q_s[t * RS + d];
      sk += k_s[t * RS + d] * k_s[t * RS + d];
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) {
      sq += __shfl_xor(sq, o, 64);
      sk += __shfl_xor(sk, o, 64);
    }
    sq = a.qscale / sqrtf(sq + UNIT_EPS);
    sk = 1.0f / sqrtf(sk + UNIT_EPS);
    for (int d = l; d < DCP; d += 16) {
      q_s[t * RS + d] *= sq;
      k_s[t * RS + d] *= sk;
    }
  }
  for (int d = tid; d < DCP; d += PREP) {
    float s[C];
#pragma unroll
    for (int t = 0; t < C; ++t) s[t] = g_s[t * RS + d];
#pragma unroll
    for (int t = 1; t < C; ++t) s[t] += s[t - 1];
#pragma unroll
    for (int t = 1; t < C; ++t) g_s[t * RS + d] = s[t];
  }
  __syncthreads();
  // ---- A and P: tiles of 4 x 4 tokens, 8 lanes share a tile's channels.
  // Below the diagonal the exponents go through the tile's first token. -----
  {
    const int part = tid & 7;
    const bool off_diag = tid < 224, diag = tid >= 256 && tid < 320;
    int ti = 0, tj = 0;
    if (off_diag) {
      int i = tid >> 3;                        // 28 tiles
      ti = 1;
      while (i >= ti) i -= ti++;
      tj = i;
    } else if (diag) {
      ti = tj = (tid - 256) >> 3;
    }
    float A[4][4] = {}, P[4][4] = {};
    if (off_diag || diag) {
      const float *qp = q_s + ti * 4 * RS, *kp = k_s + ti * 4 * RS;
      const float *gp = g_s + ti * 4 * RS;
      const float *kj = k_s + tj * 4 * RS, *gj = g_s + tj * 4 * RS;
      for (int d0 = part * 2; d0 < DCP; d0 += 16) {
        f32x2v q[4], k[4], g[4], k2[4], g2[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          q[r] = *reinterpret_cast<const f32x2v *>(qp + r * RS + d0);
          k[r] = *reinterpret_cast<const f32x2v *>(kp + r * RS + d0);
          g[r] = *reinterpret_cast<const f32x2v *>(gp + r * RS + d0);
          k2[r] = *reinterpret_cast<const f32x2v *>(kj + r * RS + d0);
          g2[r] = *reinterpret_cast<const f32x2v *>(gj + r * RS + d0);
        }
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          if (off_diag) {
            float x[4];
#pragma unroll
            for (int s = 0; s < 4; ++s)
              x[s] = k2[s][e] * __builtin_amdgcn_exp2f(g[0][e] - g2[s][e]);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const float f = __builtin_amdgcn_exp2f(g[r][e] - g[0][e]);
              const float kf = k[r][e] * f, qf = q[r][e] * f;
#pragma unroll
              for (int s = 0; s < 4; ++s) {
                A[r][s] += kf * x[s];
                P[r][s] += qf * x[s];
              }
            }
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r)
#pragma unroll
              for (int s = 0; s <= r; ++s) {
                const float x =
                    k[s][e] * __builtin_amdgcn_exp2f(g[r][e] - g[s][e]);
                if (s < r) A[r][s] += k[r][e] * x;
                P[r][s] += q[r][e] * x;
              }
          }
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        A[r][s] += __shfl_xor(A[r][s], 1, 64);
        A[r][s] += __shfl_xor(A[r][s], 2, 64);
        A[r][s] += __shfl_xor(A[r][s], 4, 64);
        P[r][s] += __shfl_xor(P[r][s], 1, 64);
        P[r][s] += __shfl_xor(P[r][s], 2, 64);
        P[r][s] += __shfl_xor(P[r][s], 4, 64);
      }
    for (int i = tid; i < C * C; i += PREP)   // above the diagonal
      if (i % C / 4 > i / C / 4) p_s[(i / C) * AS + i % C] = 0.0f;
    if ((off_diag || diag) && part == 0) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float *b = b_s + ti * 4;
        *reinterpret_cast<f32x4v *>(a_s + (tj * 4 + r) * AS + ti * 4) =
            (f32x4v){A[0][r] * b[0], A[1][r] * b[1], A[2][r] * b[2],
                     A[3][r] * b[3]};
        *reinterpret_cast<f32x4v *>(p_s + (ti * 4 + r) * AS + tj * 4) =
            (f32x4v){P[r][0], P[r][1], P[r][2], P[r][3]};
      }
    }
  }
  __syncthreads();
  // ---- operands that need no solving --------------------------------------
  auto put = [&](int at, int lane, const float *f) {
    u32x4v big, small;
    split8(f, big, small);
    *reinterpret_cast<u32x4v *>(entry + at + lane * 16) = big;
    *reinterpret_cast<u32x4v *>(entry + at + 1024 + lane * 16) = small;
  };
  const int lane = tid & 63, wid = tid >> 6, l16 = lane & 15, grp = lane >> 4;
  for (int i = wid; i < 2 * E::KS + 2 + E::TD; i += PREP / RB_WAVE) {
    float f[8];
    if (i < 2 * E::KS) {
      const int t = i / E::KS * 16 + l16, d = i % E::KS * 32 + grp * 4;
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        const int at = t * RS + d + (k & 3) + (k >> 2) * 16;
        f[k] = q_s[at] * __builtin_amdgcn_exp2f(g_s[at]);
      }
      put(E::Q + i * E::OP, lane, f);
    } else if (i < 2 * E::KS + 2) {
      const int m = i - 2 * E::KS, t = m * 16 + l16;
#pragma unroll
      for (int k = 0; k < 8; ++k)
        f[k] = p_s[t * AS + grp * 4 + (k & 3) + (k >> 2) * 16];
      put(E::P + m * E::OP, lane, f);
    } else {
      const int m = i - 2 * E::KS - 2, d = m * 16 + l16;
      const float last = g_s[(C - 1) * RS + d];
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        const int t = grp * 4 + (k & 3) + (k >> 2) * 16;
        f[k] = k_s[t * RS + d] *
               __builtin_amdgcn_exp2f(last - g_s[t * RS + d]);
      }
      put(E::K + m * E::OP, lane, f);
    }
  }
  for (int d = tid; d < DCP; d += PREP)
    reinterpret_cast<float *>(entry + E::G)[d] =
        __builtin_amdgcn_exp2f(g_s[(C - 1) * RS + d]);
  __syncthreads();                             // q_s is free
  // ---- (I + A)^-1 of both right sides, a column per thread ----------------
  float x[C];
  auto solve = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < C - 1; ++j) {
      // A is read when it is needed: it does not fit the registers
      if (j % 4 == 0) asm volatile("" ::: "memory");
#pragma unroll
      for (int i = 0; i < C / 4; ++i) {
        if (i * 4 + 3 <= j) continue;
        const f32x4v f = *reinterpret_cast<const f32x4v *>(a_s + j * AS +
                                                           i * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (i * 4 + e > j) x[i * 4 + e] -= f[e] * x[j];
      }
    }
  };
  auto solve_v = [&](int c, int c0) __attribute__((always_inline)) {
    // staged column c
#pragma unroll
    for (int t = 0; t < C; ++t) x[t] = b_s[t] * v_s[t * VS + c];
    solve();
    float *u = reinterpret_cast<float *>(entry + E::U) +
               (int64_t)((c0 + c) / 16) * 512 + ((c0 + c) & 15) * 4;
#pragma unroll
    for (int i = 0; i < 8; ++i)
      *reinterpret_cast<f32x4v *>(u + (i >> 2) * 256 + (i & 3) * 64) =
          (f32x4v){x[4 * i], x[4 * i + 1], x[4 * i + 2], x[4 * i + 3]};
  };
  const int vround = (a.vc + 15) / 16 * 16;
  for (int i = tid; i < DCP + min(vb, vround); i += PREP) {
    if (i < DCP) {
#pragma unroll
      for (int t = 0; t < C; ++t)
        x[t] = b_s[t] * __builtin_amdgcn_exp2f(g_s[t * RS + i]) *
               k_s[t * RS + i];
      solve();
#pragma unroll
      for (int t = 0; t < C; ++t) q_s[t * RS + i] = -x[t];
    } else {
      solve_v(i - DCP, 0);
    }
  }
  __syncthreads();
  for (int i = wid; i < 2 * E::KS; i += PREP / RB_WAVE) {
    float f[8];
    const int t = i / E::KS * 16 + l16, d = i % E::KS * 32 + grp * 4;
#pragma unroll
    for (int k = 0; k < 8; ++k)
      f[k] = q_s[t * RS + d + (k & 3) + (k >> 2) * 16];
    put(E::W + i * E::OP, lane, f);
  }
  for (int c0 = vb; c0 < vround; c0 += vb) {   // value columns beyond vb
    __syncthreads();
    stage_v(c0);
    __syncthreads();
    for (int c = tid; c < min(vb, vround - c0); c += PREP) solve_v(c, c0);
  }
}

// ---------------------------------------------------------------------------
// chunks: the recurrence. Two waves own 16 state columns, half of the rows
// each, as MFMA result tiles: tile d, register r of a lane is
// S[16 d + 4 (lane / 16) + r][lane % 16]; two stacked tiles are, packed, an
// operand with the entries' order of the summed index. So is U. The waves give
// each other their packed halves through LDS; the first one makes U, the
// second one O.
// ---------------------------------------------------------------------------
template <int DCP>
__global__ __launch_bounds__(2 * RB_WAVE, 1) void delta_scan_kernel(Args a) {
  using E = Entry<DCP>;
  constexpr int KS = E::KS, HT = E::TD / 2;    // state tiles per wave
  __shared__ u32x4v s_s[2][KS][64], u_s[2][64];
  const int lane = threadIdx.x & 63, l16 = lane & 15, grp = lane >> 4;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
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
      const int dim = (wid * HT + d) * 16 + grp * 4 + r;
      S[d][r] = !zero && col_ok && dim < a.dc
                    ? st[(int64_t)dim * a.vc + col] : 0.0f;
    }
  const int64_t stride = a.heads * a.entry;
  const char *base = a.scratch +
                     ((int64_t)blockIdx.z * a.chunks * a.heads + h) * a.entry;
  const int64_t orow = (int64_t)a.heads * a.vc;
  float *op = a.o + (int64_t)(q0 + a.chunk0 * C + grp * 4) * orow + h * a.vc +
              col;
  int left = n - a.chunk0 * C - grp * 4;       // tokens from this lane's on

  // what multiplies S (-W and U, or Q), and what multiplies U
  Frag ff[2 * KS][2], pf[2][2], kf[HT][2];
  f32x4v gf[HT], uf[2];
  auto get = [&](Frag *f, const char *e) __attribute__((always_inline)) {
    f[0].u = *reinterpret_cast<const u32x4v *>(e + lane * 16);
    f[1].u = *reinterpret_cast<const u32x4v *>(e + 1024 + lane * 16);
  };
  auto get_f = [&](const char *e) __attribute__((always_inline)) {
    const char *f = e + (wid == 0 ? E::W : E::Q);
#pragma unroll
    for (int i = 0; i < 2 * KS; ++i) get(ff[i], f + i * E::OP);
#pragma unroll
    for (int i = 0; i < 2; ++i)
      uf[i] = *reinterpret_cast<const f32x4v *>(e + E::U + cb * 2048 +
                                                i * 1024 + lane * 16);
  };
  auto get_k = [&](const char *e) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < 2; ++i) get(pf[i], e + E::P + i * E::OP);
#pragma unroll
    for (int d = 0; d < HT; ++d) {
      const int t = wid * HT + d;
      get(kf[d], e + E::K + t * E::OP);
      gf[d] = *reinterpret_cast<const f32x4v *>(e + E::G +
                                                (t * 16 + grp * 4) * 4);
    }
  };
  get_f(base);
  get_k(base);
  for (int c = 0; c < nc; ++c) {
    const char *next = base + min(c + 1, nc - 1) * stride;
#pragma unroll
    for (int d = 0; d < HT; ++d) {
      const int t = wid * HT + d;
      uint2 big, small;
      split2(S[d][0], S[d][1], big.x, small.x);
      split2(S[d][2], S[d][3], big.y, small.y);
      reinterpret_cast<uint2 *>(&s_s[0][t >> 1][lane])[t & 1] = big;
      reinterpret_cast<uint2 *>(&s_s[1][t >> 1][lane])[t & 1] = small;
    }
    __syncthreads();                           // S; U has been read
    Frag sh[KS], sl[KS];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      sh[ks].u = s_s[0][ks][lane];
      sl[ks].u = s_s[1][ks][lane];
    }
    f32x4v x[2];                               // U, or what S gives to O
#pragma unroll
    for (int m = 0; m < 2; ++m) x[m] = wid == 0 ? uf[m] : (f32x4v)(0.0f);
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int i = 0; i < 3; ++i)
#pragma unroll
        for (int m = 0; m < 2; ++m)
          x[m] = part(i, ff[m * KS + ks], sh[ks], sl[ks], x[m]);
    __builtin_amdgcn_sched_barrier(0);
    get_f(next);
    __builtin_amdgcn_sched_barrier(0);
    if (wid == 0) {
      u32x4v big, small;
      const float f[8] = {x[0][0], x[0][1], x[0][2], x[0][3],
                          x[1][0], x[1][1], x[1][2], x[1][3]};
      split8(f, big, small);
      u_s[0][lane] = big;
      u_s[1][lane] = small;
    }
#pragma unroll
    for (int d = 0; d < HT; ++d)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[d][r] *= gf[d][r];
    __syncthreads();                           // U; S has been read
    Frag uh, ul;
    uh.u = u_s[0][lane];
    ul.u = u_s[1][lane];
#pragma unroll
    for (int i = 0; i < 3; ++i)
#pragma unroll
      for (int d = 0; d < HT; ++d) S[d] = part(i, kf[d], uh, ul, S[d]);
    if (wid == 1) {
#pragma unroll
      for (int i = 0; i < 3; ++i)
#pragma unroll
        for (int m = 0; m < 2; ++m) x[m] = part(i, pf[m], uh, ul, x[m]);
    }
    __builtin_amdgcn_sched_barrier(0);
    get_k(next);
    __builtin_amdgcn_sched_barrier(0);
    if (wid == 1 && col_ok) {
#pragma unroll
      for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (m * 16 + r < left) op[(m * 16 + r) * orow] = x[m][r];
    }
    op += C * orow;
    left -= C;
  }
  if (!col_ok) return;
#pragma unroll
  for (int d = 0; d < HT; ++d)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int dim = (wid * HT + d) * 16 + grp * 4 + r;
      if (dim < a.dc) st[(int64_t)dim * a.vc + col] = S[d][r];
    }
}

Args check(const at::Tensor &y, const at::Tensor &y2, const at::Tensor &conv,
           const at::Tensor &decay, const at::Tensor &state,
           const at::Tensor &tails, const at::Tensor &positions,
           const at::Tensor &cu_q, const at::Tensor &slots,
           const at::Tensor &o, int64_t first_seq, int64_t n_seqs, int64_t kv,
           int64_t dim, const char *who) {
  const auto dt = y.scalar_type();
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (dt == at::kBFloat16 || dt == at::kFloat) && y2.dim() == 2 &&
              y2.is_contiguous() && y2.scalar_type() == dt &&
              y2.size(0) == y.size(0) && state.dim() == 4 &&
              state.is_contiguous() && state.scalar_type() == at::kFloat,
              who, ": y, y2, state [slots, heads, dc, vc] f32");
  const int64_t H = state.size(1), dc = state.size(2), vc = state.size(3);
  TORCH_CHECK(kv >= 1 && H % kv == 0 && dc % 8 == 0 && vc % 8 == 0 &&
              dim >= 1 && dim <= dc, who, ": sizes");
  const int64_t off_b = 2 * kv * dc + H * vc;
  TORCH_CHECK(tails.dim() == 3 && tails.is_contiguous() &&
              tails.scalar_type() == dt && tails.size(0) == state.size(0) &&
              tails.size(2) == off_b && conv.dim() == 2 &&
              conv.is_contiguous() && conv.scalar_type() == at::kFloat &&
              conv.size(1) == off_b && conv.size(0) == tails.size(1) + 1 &&
              decay.is_contiguous() && decay.scalar_type() == at::kFloat &&
              decay.numel() == H * (dc + 1) && y.size(1) % 8 == 0 &&
              off_b + H <= y.size(1) && y2.size(1) % 8 == 0 &&
              H * dc <= y2.size(1), who, ": layout");
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
  a.kv = (int)kv;
  a.dim = (int)dim;
  a.dc = (int)dc;
  a.vc = (int)vc;
  a.taps = (int)conv.size(0);
  a.off_k = (int)(kv * dc);
  a.off_v = (int)(2 * kv * dc);
  a.off_b = (int)off_b;
  a.conv = conv.data_ptr<float>();
  a.decay = decay.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.tails = tails.data_ptr();
  a.positions = positions.data_ptr<int>();
  a.cu_q = cu_q.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.o = o.data_ptr<float>();
  a.qscale = 1.0f / sqrtf((float)dim);
  a.first_seq = (int)first_seq;
  return a;
}

template <int DCP>
void launch_chunk(Args a, int64_t n_seqs, int64_t max_q,
                  const at::TensorOptions &options, hipStream_t stream) {
  using E = Entry<DCP>;
  const int vb = std::min(VB, (a.vc + 15) / 16 * 16);
  const int shmem = prep_lds<DCP>(vb);
  static_assert(prep_lds<DCP>(VB) <= 159 * 1024, "LDS");
  static bool once = [] {
    return hipFuncSetAttribute(
               reinterpret_cast<const void *>(&delta_prep_kernel<DCP>),
               hipFuncAttributeMaxDynamicSharedMemorySize,
               prep_lds<DCP>(VB)) == hipSuccess;
  }();
  TORCH_CHECK(once, "delta_chunk: LDS size");
  a.entry = E::bytes(a.vc);
  // as many chunks at once as keep the entries in the last-level cache
  const int64_t all = (max_q + C - 1) / C;
  const int64_t fit = ((int64_t)160 << 20) / (n_seqs * a.heads * a.entry);
  a.chunks = (int)std::min<int64_t>(all, std::max<int64_t>(fit, 16));
  TORCH_CHECK(a.chunks <= 65535 && a.heads <= 65535, "delta_chunk: portion of ",
              max_q);
  auto scratch = at::empty({n_seqs * a.chunks * a.heads * a.entry}, options);
  a.scratch = (char *)scratch.data_ptr();
  const dim3 scan(a.heads * ((a.vc + 15) / 16), 1, n_seqs);
  for (int64_t c = 0; c < all; c += a.chunks) {
    a.chunk0 = (int)c;
    hipLaunchKernelGGL((delta_prep_kernel<DCP>),
                       dim3(a.heads, a.chunks, n_seqs), dim3(PREP), shmem,
                       stream, a, vb);
    hipLaunchKernelGGL((delta_scan_kernel<DCP>), scan, dim3(2 * RB_WAVE), 0,
                       stream, a);
  }
}

}  // namespace

// o and the new state of the first n_seqs sequences
void delta_step(at::Tensor y, at::Tensor y2, at::Tensor conv, at::Tensor decay,
                at::Tensor state, at::Tensor tails, at::Tensor positions,
                at::Tensor cu_q, at::Tensor slots, at::Tensor o,
                int64_t n_seqs, int64_t kv, int64_t dim) {
  const Args a = check(y, y2, conv, decay, state, tails, positions, cu_q,
                       slots, o, 0, n_seqs, kv, dim, "delta_step");
  TORCH_CHECK(a.dc <= 256 && a.heads <= 65535, "delta_step: dim ", a.dc);
  if (n_seqs == 0) return;
  const dim3 grid((a.vc + STEP_COLS - 1) / STEP_COLS, a.heads, n_seqs);
  auto stream = at::hip::getCurrentHIPStream();
  auto pick = [&](auto tag) {
    using E = decltype(tag);
    auto go = [&](auto rpt) {
      hipLaunchKernelGGL((delta_step_kernel<E, decltype(rpt)::value>), grid,
                         dim3(BLOCK), 0, stream, a);
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
void delta_chunk(at::Tensor y, at::Tensor y2, at::Tensor conv,
                 at::Tensor decay, at::Tensor state, at::Tensor tails,
                 at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
                 at::Tensor o, int64_t first_seq, int64_t n_seqs,
                 int64_t max_q, int64_t kv, int64_t dim) {
  const Args a = check(y, y2, conv, decay, state, tails, positions, cu_q,
                       slots, o, first_seq, n_seqs, kv, dim, "delta_chunk");
  TORCH_CHECK(y.scalar_type() == at::kBFloat16 && a.dc <= 256,
              "delta_chunk: bf16, dim <= 256");
  if (n_seqs == 0 || max_q == 0) return;
  const auto bytes = y.options().dtype(at::kByte);
  auto stream = at::hip::getCurrentHIPStream();
  if (a.dc <= 32) launch_chunk<32>(a, n_seqs, max_q, bytes, stream);
  else if (a.dc <= 64) launch_chunk<64>(a, n_seqs, max_q, bytes, stream);
  else if (a.dc <= 128) launch_chunk<128>(a, n_seqs, max_q, bytes, stream);
  else launch_chunk<256>(a, n_seqs, max_q, bytes, stream);
}
