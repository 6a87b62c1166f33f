// Mixture of squared-ReLU experts (gfx950).
//
//  * moe_route: softmax scores, the `top` largest of score + correction out of
//    the `keep` best groups; a wave per token.
//  * moe_plan: (token, choice) pairs sorted by expert, in tiles of at most
//    `tile` pairs of one expert; the list of tiles has a fixed length, its
//    unused entries are empty, and the last one counts the used ones.
//  * moe_gemm: one product per tile with its expert's weight. First product:
//    relu^2, rows by pair number. Second: times the pair's weight, fp32, one
//    part [T, N] per choice.
//      tile 16: decoding, bound by reading weights; K split over the waves
//      tile 128: bf16, 128 x 128 through LDS

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

namespace {

constexpr int BLOCK = 256;
constexpr int MAX_EXPERTS = 1024;
constexpr int MAX_TOP = 64;
// a tile: expert, first pair, pairs, the expert's first tile, its tiles
constexpr int TILE_INTS = 5;

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8v;
typedef __attribute__((ext_vector_type(4))) float f32x4v;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4v;

// ---------------------------------------------------------------------------
// routing
// ---------------------------------------------------------------------------
// largest (value, smallest index on a tie) over the wave
RB_DEV void wave_argmax(float &v, int &i) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(v, o, 64);
    const int oi = __shfl_xor(i, o, 64);
    if (ov > v || (ov == v && oi < i)) {
      v = ov;
      i = oi;
    }
  }
}

template <int EPL>
__global__ __launch_bounds__(BLOCK) void moe_route_kernel(
    const float *__restrict__ logits, int parts, int64_t T, int ld,
    const float *__restrict__ correction, int experts, int top, int groups,
    int keep, int *__restrict__ chosen, float *__restrict__ weights) {
  __shared__ float choice_s[BLOCK / RB_WAVE][EPL * 64];
  __shared__ float group_s[BLOCK / RB_WAVE][EPL * 64];
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int64_t token = (int64_t)blockIdx.x * (BLOCK / RB_WAVE) + wid;
  const int64_t t = min(token, T - 1);
  float s[EPL], c[EPL], m = -INFINITY, sum = 0.0f;
#pragma unroll
  for (int i = 0; i < EPL; ++i) {
    const int e = lane + i * 64;
    s[i] = -INFINITY;
    if (e < experts) {
      s[i] = 0.0f;
      for (int p = 0; p < parts; ++p) s[i] += logits[(p * T + t) * ld + e];
    }
    m = fmaxf(m, s[i]);
  }
  m = rb::wave_reduce_max(m);
#pragma unroll
  for (int i = 0; i < EPL; ++i) {
    s[i] = expf(s[i] - m);
    sum += s[i];
  }
  sum = rb::wave_reduce_sum(sum);
#pragma unroll
  for (int i = 0; i < EPL; ++i) {
    const int e = lane + i * 64;
    s[i] /= sum;
    c[i] = e < experts ? s[i] + correction[e] : -INFINITY;
  }
  if (keep < groups) {                         // the same in every wave
    const int size = experts / groups;
    float *ch = choice_s[wid], *gr = group_s[wid];
#pragma unroll
    for (int i = 0; i < EPL; ++i) ch[lane + i * 64] = c[i];
    __syncthreads();
    float best[EPL];
#pragma unroll
    for (int i = 0; i < EPL; ++i) {
      const int g = lane + i * 64;
      best[i] = -INFINITY;
      if (g < groups) {
        for (int k = 0; k < size; ++k)
          best[i] = fmaxf(best[i], ch[g * size + k]);
        gr[g] = 0.0f;
      }
    }
    __syncthreads();
    for (int r = 0; r < keep; ++r) {
      float v = -INFINITY;
      int at = INT_MAX;
#pragma unroll
      for (int i = 0; i < EPL; ++i)
        if (lane + i * 64 < groups && best[i] > v) {
          v = best[i];
          at = lane + i * 64;
        }
      wave_argmax(v, at);
#pragma unroll
      for (int i = 0; i < EPL; ++i)
        if (lane + i * 64 == at) {
          best[i] = -INFINITY;
          gr[at] = 1.0f;
        }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < EPL; ++i) {
      const int e = lane + i * 64;
      if (e < experts && gr[e / size] == 0.0f) c[i] = -INFINITY;
    }
  }
  if (token >= T) return;
  for (int r = 0; r < top; ++r) {
    float v = -INFINITY;
    int at = INT_MAX;
#pragma unroll
    for (int i = 0; i < EPL; ++i)
      if (c[i] > v) {
        v = c[i];
        at = lane + i * 64;
      }
    wave_argmax(v, at);
    if (at == INT_MAX) {                       // not a number: any expert
      if (lane == 0) {
        chosen[t * top + r] = 0;
        weights[t * top + r] = s[0];
      }
      continue;
    }
#pragma unroll
    for (int i = 0; i < EPL; ++i)
      if (lane + i * 64 == at) {
        chosen[t * top + r] = at;
        weights[t * top + r] = s[i];
        c[i] = -INFINITY;
      }
  }
}

// ---------------------------------------------------------------------------
// pairs by expert: one workgroup
// ---------------------------------------------------------------------------
__global__ __launch_bounds__(1024) void moe_plan_kernel(
    const int *__restrict__ chosen, int n, int experts, int tile,
    int *__restrict__ pairs, int *__restrict__ tiles, int n_tiles) {
  __shared__ int count[MAX_EXPERTS], at[2][MAX_EXPERTS], tl[2][MAX_EXPERTS];
  const int i = threadIdx.x;
  count[i] = 0;
  __syncthreads();
  for (int p = i; p < n; p += 1024) atomicAdd(&count[chosen[p]], 1);
  __syncthreads();
  const int mine = count[i], mine_t = (mine + tile - 1) / tile;
  at[0][i] = mine;
  tl[0][i] = mine_t;
  int src = 0;
  for (int o = 1; o < MAX_EXPERTS; o *= 2) {
    __syncthreads();
    at[src ^ 1][i] = at[src][i] + (i >= o ? at[src][i - o] : 0);
    tl[src ^ 1][i] = tl[src][i] + (i >= o ? tl[src][i - o] : 0);
    src ^= 1;
  }
  __syncthreads();
  const int first = at[src][i] - mine, first_t = tl[src][i] - mine_t;
  const int used = tl[src][MAX_EXPERTS - 1];
  for (int k = 0; k < mine_t; ++k) {
    int *e = tiles + (first_t + k) * TILE_INTS;
    e[0] = i;
    e[1] = first + k * tile;
    e[2] = min(tile, mine - k * tile);
    e[3] = first_t;
    e[4] = mine_t;
  }
  for (int k = used + i; k < n_tiles; k += 1024) {
    int *e = tiles + k * TILE_INTS;
    e[0] = k == n_tiles - 1 ? used : 0;
    e[1] = e[2] = e[3] = e[4] = 0;
  }
  count[i] = first;
  __syncthreads();
  for (int p = i; p < n; p += 1024) pairs[atomicAdd(&count[chosen[p]], 1)] = p;
}

// ---------------------------------------------------------------------------
// products
// ---------------------------------------------------------------------------
struct Args {
  const void *x, *w;                   // [rows, K], [experts, N, K]
  const int *pairs, *tiles;
  const float *weights;
  void *out;                           // [pairs, N], or [top, T, N] fp32
  int top, N, K;
  int64_t T;
};

// four results from column n of one pair
template <typename T, bool DOWN>
RB_DEV void put(const Args &a, int pair, int n, f32x4v v) {
  if constexpr (DOWN) {
    const int t = pair / a.top, c = pair - t * a.top;
    const float w = a.weights[pair];
    float *p = (float *)a.out + ((int64_t)c * a.T + t) * a.N + n;
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] *= w;
    if (a.N % 4 == 0) {
      *reinterpret_cast<f32x4v *>(p) = v;
    } else {
      for (int r = 0; r < 4; ++r)
        if (n + r < a.N) p[r] = v[r];
    }
  } else {                             // N % 8 == 0
    T *p = (T *)a.out + (int64_t)pair * a.N + n;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float x = fmaxf(v[r], 0.0f);
      v[r] = x * x;
    }
    if constexpr (sizeof(T) == 2) {
      uint2 o;
      o.x = rb::pack_bf16x2(v[0], v[1]);
      o.y = rb::pack_bf16x2(v[2], v[3]);
      *reinterpret_cast<uint2 *>(p) = o;
    } else {
      *reinterpret_cast<f32x4v *>(p) = v;
    }
  }
}

// 16 columns of one step: 32 values of K for 16-bit, 16 for fp32
template <typename T> struct Step;
template <> struct Step<uint16_t> {
  static constexpr int K = 32, W = 8;
  typedef bf16x8v V;
  RB_DEV static f32x4v mul(V w, V x, f32x4v c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, x, c, 0, 0, 0);
  }
};
template <> struct Step<float> {
  static constexpr int K = 16, W = 4;
  typedef f32x4v V;
  RB_DEV static f32x4v mul(V w, V x, f32x4v c) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      c = __builtin_amdgcn_mfma_f32_16x16x4f32(w[i], x[i], c, 0, 0, 0);
    return c;
  }
};

// A tile of 16 pairs and 32 columns per workgroup, K split over its waves.
template <typename T, bool DOWN>
__global__ __launch_bounds__(BLOCK) void moe_rows_kernel(Args a) {
  using S = Step<T>;
  using V = typename S::V;
  constexpr int U = 4;
  __shared__ f32x4v red[BLOCK / RB_WAVE][2][64];
  const int *tile = a.tiles + blockIdx.y * TILE_INTS;
  const int expert = tile[0], first = tile[1], count = tile[2];
  if (count <= 0) return;
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int l16 = lane & 15, grp = lane >> 4;
  const int n0 = blockIdx.x * 32;
  const int pair = a.pairs[first + min(l16, count - 1)];
  const T *x = (const T *)a.x +
               (int64_t)(DOWN ? pair : pair / a.top) * a.K + grp * S::W;
  const T *w[2];
#pragma unroll
  for (int m = 0; m < 2; ++m)
    w[m] = (const T *)a.w +
           ((int64_t)expert * a.N + min(n0 + m * 16 + l16, a.N - 1)) * a.K +
           grp * S::W;
  const int steps = a.K / S::K, per = (steps + 3) / 4;
  int s = wid * per;
  const int s1 = min(steps, s + per);
  f32x4v acc[2] = {(f32x4v)(0.0f), (f32x4v)(0.0f)};
  auto load = [](const T *p) { return *reinterpret_cast<const V *>(p); };
  for (; s + U <= s1; s += U) {
    V xv[U], wv[2][U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      xv[u] = load(x + (s + u) * S::K);
      wv[0][u] = load(w[0] + (s + u) * S::K);
      wv[1][u] = load(w[1] + (s + u) * S::K);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      acc[0] = S::mul(wv[0][u], xv[u], acc[0]);
      acc[1] = S::mul(wv[1][u], xv[u], acc[1]);
    }
  }
  for (; s < s1; ++s) {
    const V xv = load(x + s * S::K);
    acc[0] = S::mul(load(w[0] + s * S::K), xv, acc[0]);
    acc[1] = S::mul(load(w[1] + s * S::K), xv, acc[1]);
  }
  red[wid][0][lane] = acc[0];
  red[wid][1][lane] = acc[1];
  __syncthreads();
  if (wid >= 2 || l16 >= count) return;
  const f32x4v v = red[0][wid][lane] + red[1][wid][lane] + red[2][wid][lane] +
                   red[3][wid][lane];
  const int n = n0 + wid * 16 + grp * 4;
  if (n < a.N) put<T, DOWN>(a, pair, n, v);
}

// 128 pairs x 128 columns per workgroup, 4 waves of 64 x 64, K in steps of 64
// straight to LDS; the workgroups of a CU fill each other's waits. A row's
// eight 16-byte chunks are stored in an order that depends on the row, so that
// 16 rows are read without bank conflicts.
constexpr int BK = 64, ROW = BK * 2;           // LDS bytes per row

RB_DEV int chunk_at(int row, int c) { return c ^ ((row >> 1) & 7); }

template <bool DOWN>
__global__ __launch_bounds__(BLOCK, 4) void moe_tile_kernel(Args a, int nb,
                                                            int n_tiles) {
  __shared__ __attribute__((aligned(16))) char smem[2 * 128 * ROW];
  // neighbouring workgroups are on one XCD and share an expert's columns,
  // so that a weight is read once
  const int total = a.tiles[(n_tiles - 1) * TILE_INTS] * nb;
  const int q8 = total / 8, r8 = total % 8;
  const int xcd = blockIdx.x % 8, pos = blockIdx.x / 8;
  if (pos >= q8 + (xcd < r8)) return;
  const int wg = xcd * q8 + min(xcd, r8) + pos;
  const int *own = a.tiles + wg / nb * TILE_INTS;
  const int local = wg - own[3] * nb;
  const int *tile = a.tiles + (own[3] + local % own[4]) * TILE_INTS;
  const int expert = tile[0], first = tile[1], count = tile[2];
  const int n0 = local / own[4] * 128;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  const int l16 = lane & 15, grp = lane >> 4;
  const int wn = (wid & 1) * 64, wm = (wid >> 1) * 64;

  // a lane's 16 bytes of eight rows at a time
  const uint16_t *xp[4], *wp[4];
  int kc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = (wid * 4 + i) * 8 + (lane >> 3);
    const int pair = a.pairs[first + min(row, count - 1)];
    xp[i] = (const uint16_t *)a.x +
            (int64_t)(DOWN ? pair : pair / a.top) * a.K;
    wp[i] = (const uint16_t *)a.w +
            ((int64_t)expert * a.N + min(n0 + row, a.N - 1)) * a.K;
    kc[i] = chunk_at(row, lane & 7) * 8;
  }
  auto to_lds = [](const uint16_t *p, char *dst) {
    __builtin_amdgcn_global_load_lds(
        (const __attribute__((address_space(1))) uint32_t *)(const void *)p,
        (__attribute__((address_space(3))) uint32_t *)(void *)dst, 16, 0, 0);
  };
  f32x4v acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = (f32x4v)(0.0f);
  for (int k0 = 0; k0 < a.K; k0 += BK) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      // beyond K any address of the row: those chunks are not read
      const int k = k0 + kc[i] < a.K ? k0 + kc[i] : 0;
      char *dst = smem + (wid * 4 + i) * 8 * ROW;
      to_lds(xp[i] + k, dst);
      to_lds(wp[i] + k, dst + 128 * ROW);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    const char *xs = smem, *ws = smem + 128 * ROW;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      if (k0 + ks * 32 >= a.K) break;
      bf16x8v xf[4], wf[4];
      const int at = chunk_at(l16, ks * 4 + grp) * 16;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        xf[i] = *reinterpret_cast<const bf16x8v *>(
            xs + (wm + i * 16 + l16) * ROW + at);
        wf[i] = *reinterpret_cast<const bf16x8v *>(
            ws + (wn + i * 16 + l16) * ROW + at);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              wf[i], xf[j], acc[i][j], 0, 0, 0);
    }
    __syncthreads();
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int row = wm + j * 16 + l16;
    if (row >= count) continue;
    const int pair = a.pairs[first + row];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = n0 + wn + i * 16 + grp * 4;
      if (n < a.N) put<uint16_t, DOWN>(a, pair, n, acc[i][j]);
    }
  }
}

template <bool DOWN> void launch_tile(const Args &a, int n_tiles,
                                      hipStream_t stream) {
  const int nb = (a.N + 127) / 128;
  const int total = (nb * n_tiles + 7) / 8 * 8;
  hipLaunchKernelGGL((moe_tile_kernel<DOWN>), dim3(total), dim3(BLOCK),
                     0, stream, a, nb, n_tiles);
}

}  // namespace

// chosen [T, top] i32, weights [T, top] f32
std::vector<at::Tensor> moe_route(at::Tensor logits, at::Tensor correction,
                                  int64_t top, int64_t groups, int64_t keep) {
  TORCH_CHECK(logits.is_cuda() && (logits.dim() == 2 || logits.dim() == 3) &&
              logits.is_contiguous() && logits.scalar_type() == at::kFloat &&
              correction.is_contiguous() &&
              correction.scalar_type() == at::kFloat,
              "moe_route: logits [(n,) T, >= experts] f32");
  const int64_t E = correction.numel(), T = logits.size(-2);
  TORCH_CHECK(E >= 1 && E <= MAX_EXPERTS && logits.size(-1) >= E && top >= 1 &&
              top <= MAX_TOP && groups >= 1 && E % groups == 0 && keep >= 1 &&
              keep <= groups && top <= E / groups * keep,
              "moe_route: top ", top, " of ", E, " in ", groups, " groups");
  auto chosen = at::empty({T, top}, logits.options().dtype(at::kInt));
  auto weights = at::empty({T, top}, logits.options());
  if (T == 0) return {chosen, weights};
  auto stream = at::hip::getCurrentHIPStream();
  auto go = [&](auto n) {
    hipLaunchKernelGGL((moe_route_kernel<decltype(n)::value>),
                       dim3((T + 3) / 4), dim3(BLOCK), 0, stream,
                       logits.data_ptr<float>(),
                       logits.dim() == 3 ? (int)logits.size(0) : 1, T,
                       (int)logits.size(-1), correction.data_ptr<float>(),
                       (int)E, (int)top, (int)groups, (int)keep,
                       chosen.data_ptr<int>(), weights.data_ptr<float>());
  };
  if (E <= 64) go(std::integral_constant<int, 1>{});
  else if (E <= 128) go(std::integral_constant<int, 2>{});
  else if (E <= 256) go(std::integral_constant<int, 4>{});
  else go(std::integral_constant<int, 16>{});
  return {chosen, weights};
}

std::vector<at::Tensor> moe_plan(at::Tensor chosen, int64_t experts,
                                 int64_t tile) {
  TORCH_CHECK(chosen.is_cuda() && chosen.is_contiguous() &&
              chosen.scalar_type() == at::kInt && experts >= 1 &&
              experts <= MAX_EXPERTS && tile >= 1, "moe_plan: chosen i32");
  const int64_t n = chosen.numel();
  TORCH_CHECK(n < (1 << 30), "moe_plan: pairs");
  const int64_t n_tiles = (n + tile - 1) / tile + std::min(n, experts) + 1;
  auto pairs = at::empty({n}, chosen.options());
  auto tiles = at::empty({n_tiles, TILE_INTS}, chosen.options());
  if (n == 0) return {pairs, tiles};
  hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), 0,
                     at::hip::getCurrentHIPStream(), chosen.data_ptr<int>(),
                     (int)n, (int)experts, (int)tile, pairs.data_ptr<int>(),
                     tiles.data_ptr<int>(), (int)n_tiles);
  return {pairs, tiles};
}

// down False: x [T, K] -> relu^2, [pairs, N]; True: x [pairs, K] -> fp32
// [top, T, N] times weights [T, top]. w [experts, N, K].
at::Tensor moe_gemm(at::Tensor x, at::Tensor w, at::Tensor pairs,
                    at::Tensor tiles, at::Tensor weights, int64_t tile,
                    bool down) {
  const auto dt = x.scalar_type();
  const bool bf16 = dt == at::kBFloat16;
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() &&
              (bf16 || dt == at::kFloat) && w.dim() == 3 &&
              w.is_contiguous() && w.scalar_type() == dt, "moe_gemm: x, w");
  TORCH_CHECK(weights.dim() == 2 && weights.is_contiguous() &&
              weights.scalar_type() == at::kFloat && pairs.is_contiguous() &&
              pairs.scalar_type() == at::kInt &&
              pairs.numel() == weights.numel() && tiles.dim() == 2 &&
              tiles.size(1) == TILE_INTS && tiles.size(0) >= 1 && tiles.is_contiguous() &&
              tiles.scalar_type() == at::kInt, "moe_gemm: plan");
  const int64_t T = weights.size(0), top = weights.size(1), N = w.size(1),
                K = w.size(2), n = pairs.numel();
  TORCH_CHECK(x.size(1) == K && K % 32 == 0 && K >= 32 &&
              x.size(0) == (down ? n : T) && (down || N % 8 == 0) && N >= 1,
              "moe_gemm: layout");
  TORCH_CHECK(tile == 16 || (tile == 128 && bf16), "moe_gemm: tile ", tile);
  const int64_t n_tiles = tiles.size(0);
  TORCH_CHECK(n_tiles <= 65535 || tile == 128, "moe_gemm: tiles");
  TORCH_CHECK(n_tiles * ((N + 127) / 128) < (1ll << 31), "moe_gemm: grid");
  auto out = down ? at::empty({top, T, N}, x.options().dtype(at::kFloat))
                  : at::empty({n, N}, x.options());
  if (n == 0) return out;
  Args a{x.data_ptr(), w.data_ptr(), pairs.data_ptr<int>(),
         tiles.data_ptr<int>(), weights.data_ptr<float>(), out.data_ptr(),
         (int)top, (int)N, (int)K, T};
  auto stream = at::hip::getCurrentHIPStream();
  if (tile == 128) {
    if (down) launch_tile<true>(a, (int)n_tiles, stream);
    else launch_tile<false>(a, (int)n_tiles, stream);
    return out;
  }
  const dim3 grid((N + 31) / 32, n_tiles - 1);
  auto launch = [&](auto tag, auto d) {
    hipLaunchKernelGGL((moe_rows_kernel<decltype(tag), decltype(d)::value>),
                       grid, dim3(BLOCK), 0, stream, a);
  };
  auto pick = [&](auto tag) {
    if (down) launch(tag, std::true_type{});
    else launch(tag, std::false_type{});
  };
  if (bf16) pick(uint16_t{});
  else pick(float{});
  return out;
}
