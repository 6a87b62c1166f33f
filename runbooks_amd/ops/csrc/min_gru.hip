// minGRU (gfx950): z = sigmoid(y_z + b_z), u = y_x + b_x, candidate c = u + 1/2
// where u >= 0, else sigmoid(u); S <- (1 - z) S + z c; result
// scale S silu(y_g). Columns [ z | x | gate ] of y from `off` on, R each.
//
//  * min_gru_step: token after token.
//  * min_gru_scan: long portions. A segment of tokens maps the state before
//    it to A S + B; a first pass leaves (A, B) of every segment, from which
//    the second starts each one.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 64;
constexpr int V = 2;                   // columns per thread
constexpr int U = 8;                   // tokens loaded ahead

struct Args {
  const void *y;
  int64_t ny;
  int off, R;
  const float *bias;                   // [2, R]
  float *state;                        // [slots, R]
  const int *positions, *cu_q, *slots;
  int first_seq, seg_tokens, max_seg;
  float scale;
  void *z;                             // [T, nz], columns from z_off on
  int64_t nz;
  int z_off;
  void *swz;
  float *scratch;                      // [sequences, max_seg, 2, R]
};

template <typename T> RB_DEV float sigmoid(float x) {
  if constexpr (sizeof(T) == 2) return 1.0f / (1.0f + __expf(-x));
  else return 1.0f / (1.0f + expf(-x));
}

template <typename T> RB_DEV void load2(const T *p, float *f) {
  if constexpr (sizeof(T) == 2) {
    const uint32_t w = *reinterpret_cast<const uint32_t *>(p);
    f[0] = rb::bf16_to_f32((uint16_t)w);
    f[1] = rb::bf16_to_f32((uint16_t)(w >> 16));
  } else {
    const float2 w = *reinterpret_cast<const float2 *>(p);
    f[0] = w.x;
    f[1] = w.y;
  }
}

// tokens t0 .. t1 - 1 from state S; PASS 0: only A and S (= B)
template <typename T, bool OUT>
RB_DEV void run(const Args &a, int t0, int t1, int c, const float (*b)[V],
                float *S, float *A) {
  const T *base = (const T *)a.y + a.off + c;
  for (int t = t0; t < t1; t += U) {
    float yz[U][V], yx[U][V], yg[U][V];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const T *p = base + (int64_t)min(t + i, t1 - 1) * a.ny;
      load2(p, yz[i]);
      load2(p + a.R, yx[i]);
      if constexpr (OUT) load2(p + 2 * a.R, yg[i]);
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (t + i >= t1) break;
      float o[V];
#pragma unroll
      for (int k = 0; k < V; ++k) {
        const float zt = sigmoid<T>(yz[i][k] + b[0][k]);
        const float u = yx[i][k] + b[1][k];
        const float cand = u >= 0.0f ? u + 0.5f : sigmoid<T>(u);
        S[k] = (1.0f - zt) * S[k] + zt * cand;
        if constexpr (OUT)
          o[k] = a.scale * S[k] * yg[i][k] * sigmoid<T>(yg[i][k]);
        else
          A[k] *= 1.0f - zt;
      }
      if constexpr (OUT) {
        const int64_t row = t + i;
        const int col = a.z_off + c;
        T *zp = (T *)a.z + row * a.nz + col;
        if constexpr (sizeof(T) == 2) {
          const uint32_t w = rb::pack_bf16x2(o[0], o[1]);
          *reinterpret_cast<uint32_t *>(zp) = w;
          if (a.swz != nullptr)
            *reinterpret_cast<uint32_t *>(
                (uint16_t *)a.swz + (int64_t)(col >> 4) * 512 +
                ((col >> 3) & 1) * 256 + row * 8 + (col & 7)) = w;
        } else {
          *reinterpret_cast<float2 *>(zp) = make_float2(o[0], o[1]);
        }
      }
    }
  }
}

// PASS 0: token after token; 1: a segment's (A, B); 2: the segments' results
template <typename T, int PASS>
__global__ __launch_bounds__(BLOCK) void min_gru_kernel(Args a) {
  const int c = (blockIdx.x * BLOCK + threadIdx.x) * V;
  const int seq = a.first_seq + blockIdx.z;
  const int q0 = a.cu_q[seq], q1 = a.cu_q[seq + 1];
  if (c >= a.R || q0 >= q1) return;
  float b[2][V], S[V], A[V];
#pragma unroll
  for (int k = 0; k < V; ++k) {
    b[0][k] = a.bias[c + k];
    b[1][k] = a.bias[a.R + c + k];
    S[k] = 0.0f;
    A[k] = 1.0f;
  }
  float *slot = a.state + (int64_t)a.slots[seq] * a.R + c;
  const bool fresh = a.positions[q0] == 0;
  if constexpr (PASS == 0) {
    if (!fresh) load2(slot, S);
    run<T, true>(a, q0, q1, c, b, S, A);
    *reinterpret_cast<float2 *>(slot) = make_float2(S[0], S[1]);
    return;
  }
  const int seg = blockIdx.y;
  const int nseg = (q1 - q0 + a.seg_tokens - 1) / a.seg_tokens;
  if (seg >= nseg) return;
  const int t0 = q0 + seg * a.seg_tokens, t1 = min(q1, t0 + a.seg_tokens);
  float *part = a.scratch + (int64_t)blockIdx.z * a.max_seg * 2 * a.R + c;
  if constexpr (PASS == 1) {
    if (seg == 0) {                    // from the slot: A = 0
      if (!fresh) load2(slot, S);
      A[0] = A[1] = 0.0f;
    }
    run<T, false>(a, t0, t1, c, b, S, A);
    *reinterpret_cast<float2 *>(part + (int64_t)seg * 2 * a.R) =
        make_float2(A[0], A[1]);
    *reinterpret_cast<float2 *>(part + ((int64_t)seg * 2 + 1) * a.R) =
        make_float2(S[0], S[1]);
  } else {
    // the slot's own state is read only where no other workgroup writes it
    if (nseg == 1) {
      if (!fresh) load2(slot, S);
    } else if (seg > 0) {
#pragma unroll 4
      for (int e = 0; e < seg; ++e) {
        float pa[V], pb[V];
        load2(part + (int64_t)e * 2 * a.R, pa);
        load2(part + ((int64_t)e * 2 + 1) * a.R, pb);
#pragma unroll
        for (int k = 0; k < V; ++k) S[k] = pa[k] * S[k] + pb[k];
      }
    } else {
      load2(part + (int64_t)(a.max_seg - 1) * 2 * a.R, S);
    }
    run<T, true>(a, t0, t1, c, b, S, A);
    if (seg == nseg - 1)
      *reinterpret_cast<float2 *>(slot) = make_float2(S[0], S[1]);
  }
}

// segment 0 of pass 2 starts from a copy of the slot: the last entry of the
// sequence's scratch, which no segment uses
__global__ __launch_bounds__(BLOCK) void min_gru_start_kernel(Args a) {
  const int c = blockIdx.x * BLOCK + threadIdx.x;
  const int seq = a.first_seq + blockIdx.z;
  const int q0 = a.cu_q[seq];
  if (c >= a.R || q0 >= a.cu_q[seq + 1]) return;
  a.scratch[((int64_t)blockIdx.z * a.max_seg + a.max_seg - 1) * 2 * a.R + c] =
      a.positions[q0] == 0 ? 0.0f
                           : a.state[(int64_t)a.slots[seq] * a.R + c];
}

Args check(const at::Tensor &y, int64_t off, const at::Tensor &bias,
           const at::Tensor &state, const at::Tensor &positions,
           const at::Tensor &cu_q, const at::Tensor &slots, int64_t first_seq,
           int64_t n_seqs, const at::Tensor &z, int64_t z_off, double scale) {
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
              (y.scalar_type() == at::kBFloat16 ||
               y.scalar_type() == at::kFloat) &&
              state.dim() == 2 && state.is_contiguous() &&
              state.scalar_type() == at::kFloat, "min_gru: y, state");
  const int64_t R = state.size(1);
  TORCH_CHECK(R % 8 == 0 && off % 8 == 0 && off >= 0 &&
              off + 3 * R <= y.size(1) && y.size(1) % 8 == 0 &&
              bias.scalar_type() == at::kFloat && bias.is_contiguous() &&
              bias.numel() == 2 * R, "min_gru: layout");
  TORCH_CHECK(z.dim() == 2 && z.is_contiguous() && z.size(0) == y.size(0) &&
              z.scalar_type() == y.scalar_type() && z.size(1) % 8 == 0 &&
              z_off % 8 == 0 && z_off >= 0 && z_off + R <= z.size(1),
              "min_gru: z");
  TORCH_CHECK(positions.scalar_type() == at::kInt &&
              positions.is_contiguous() && positions.numel() == y.size(0) &&
              cu_q.scalar_type() == at::kInt && cu_q.is_contiguous() &&
              slots.scalar_type() == at::kInt && slots.is_contiguous() &&
              first_seq >= 0 && n_seqs >= 0 && n_seqs <= 65535 &&
              cu_q.numel() > first_seq + n_seqs &&
              slots.numel() >= first_seq + n_seqs, "min_gru: batch tensors");
  Args a{};
  a.y = y.data_ptr();
  a.ny = y.size(1);
  a.off = (int)off;
  a.R = (int)R;
  a.bias = bias.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.positions = positions.data_ptr<int>();
  a.cu_q = cu_q.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.first_seq = (int)first_seq;
  a.scale = (float)scale;
  a.z = z.data_ptr();
  a.nz = z.size(1);
  a.z_off = (int)z_off;
  return a;
}

template <int PASS>
void launch(const Args &a, bool bf16, dim3 grid, hipStream_t stream) {
  if (bf16)
    hipLaunchKernelGGL((min_gru_kernel<uint16_t, PASS>), grid, dim3(BLOCK), 0,
                       stream, a);
  else
    hipLaunchKernelGGL((min_gru_kernel<float, PASS>), grid, dim3(BLOCK), 0,
                       stream, a);
}

}  // namespace

void min_gru_step(at::Tensor y, int64_t off, at::Tensor bias, at::Tensor state,
                  at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
                  int64_t first_seq, int64_t n_seqs, at::Tensor z,
                  int64_t z_off, double scale,
                  c10::optional<at::Tensor> swz) {
  Args a = check(y, off, bias, state, positions, cu_q, slots, first_seq,
                 n_seqs, z, z_off, scale);
  if (swz.has_value()) {
    TORCH_CHECK(z.scalar_type() == at::kBFloat16 && z.size(0) <= 32 &&
                swz->scalar_type() == at::kBFloat16 && swz->is_contiguous() &&
                swz->numel() >= (z_off + a.R + 15) / 16 * 512,
                "min_gru: operand");
    a.swz = swz->data_ptr();
  }
  if (n_seqs == 0) return;
  launch<0>(a, y.scalar_type() == at::kBFloat16,
            dim3((a.R / V + BLOCK - 1) / BLOCK, 1, n_seqs),
            at::hip::getCurrentHIPStream());
}

void min_gru_scan(at::Tensor y, int64_t off, at::Tensor bias, at::Tensor state,
                  at::Tensor positions, at::Tensor cu_q, at::Tensor slots,
                  int64_t first_seq, int64_t n_seqs, at::Tensor z,
                  int64_t z_off, double scale, int64_t max_q) {
  Args a = check(y, off, bias, state, positions, cu_q, slots, first_seq,
                 n_seqs, z, z_off, scale);
  if (n_seqs == 0 || max_q == 0) return;
  TORCH_CHECK(max_q >= 1 && max_q <= y.size(0), "min_gru_scan: max_q");
  const bool bf16 = y.scalar_type() == at::kBFloat16;
  a.seg_tokens = 32;                   // and at most 64 segments
  while (a.seg_tokens * 64 < max_q) a.seg_tokens *= 2;
  const int64_t segs = (max_q + a.seg_tokens - 1) / a.seg_tokens;
  a.max_seg = (int)segs + 1;
  auto scratch = at::empty({n_seqs, (int64_t)a.max_seg, 2, (int64_t)a.R},
                           state.options());
  a.scratch = scratch.data_ptr<float>();
  auto stream = at::hip::getCurrentHIPStream();
  const unsigned gx = (a.R / V + BLOCK - 1) / BLOCK;
  if (segs > 1) {
    hipLaunchKernelGGL(min_gru_start_kernel,
                       dim3((a.R + BLOCK - 1) / BLOCK, 1, n_seqs),
                       dim3(BLOCK), 0, stream, a);
    launch<1>(a, bf16, dim3(gx, segs, n_seqs), stream);
  }
  launch<2>(a, bf16, dim3(gx, segs, n_seqs), stream);
}
