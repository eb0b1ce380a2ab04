// Routed experts (mixture of experts): routing, grouping of the step's (token, choice) entries
// by expert, the grouped products, and the weighted sum.  Everything stays on the device: no
// count ever travels to the host, so a step's launches depend on its number of tokens only.
//
// Routing, per token, from float32 router logits z [E]:
//   s = softmax(z), or sigmoid(z) of each on its own;
//   with groups > 1: the experts are cut into `groups` runs of equal length, ranked by their best s, and
//   those outside the first `keep` runs leave the choice;
//   the `top` allowed experts with the largest s are chosen, weights = their s (as they are,
//   or divided by their sum + renorm_eps when `renorm`).  Equal scores: the lower index wins.
//   With a `correction` [E] the choice (of groups and of experts) goes by s + correction; the
//   weights stay the scores themselves.
// Experts from `num_real` on are identity experts: they have no matrices, make no tiles, and the
// weighted sum takes the token's own activations for them.
#include "common.h"

#define RE_MAX_EXPERTS 1024
#define RE_TILE 64          // rows of a tile of the general grouped product (the most it takes)

// (value, index) arg max over a wave; equal values: the lower index
__device__ inline void wave_argmax(float& v, int& idx) {
#pragma unroll
  for (int off = PI_WAVE / 2; off > 0; off >>= 1) {
    const float ov = __shfl_xor(v, off, PI_WAVE);
    const int oi = __shfl_xor(idx, off, PI_WAVE);
    if (ov > v || (ov == v && oi < idx)) {
      v = ov;
      idx = oi;
    }
  }
}

__global__ __launch_bounds__(PI_WAVE) void route_kernel(int* __restrict__ ids, float* __restrict__ weights, const float* __restrict__ logits,
                                                        long logits_stride, int splits, long plane, int E, int top, int groups, int keep, int renorm,
                                                        const float* __restrict__ correction, float renorm_eps, int sigmoid) {
  __shared__ float s[RE_MAX_EXPERTS];
  __shared__ float c[RE_MAX_EXPERTS];      // what the choice goes by
  __shared__ unsigned char allowed[RE_MAX_EXPERTS];
  __shared__ float gscore[RE_MAX_EXPERTS];
  const long t = blockIdx.x;
  const int lane = threadIdx.x;
  // the logits, or the pieces of their product (`splits` planes), added in split order
  __shared__ float z[RE_MAX_EXPERTS];
  for (int e = lane; e < E; e += PI_WAVE) z[e] = split_sum(logits, splits, plane, t * logits_stride + e);
  if (sigmoid) {
    // the sigmoid grows with z, so without a correction the choice goes by z itself: large logits whose scores round
    // to the same number keep their order
    for (int e = lane; e < E; e += PI_WAVE) {
      s[e] = 1.0f / (1.0f + expf(-z[e]));
      c[e] = correction ? s[e] + correction[e] : z[e];
      allowed[e] = (groups <= 1) ? 1 : 0;
    }
  } else {
    float mx = -INFINITY;
    for (int e = lane; e < E; e += PI_WAVE) mx = fmaxf(mx, z[e]);
    mx = wave_max(mx);
    float sum = 0.f;
    for (int e = lane; e < E; e += PI_WAVE) {
      const float v = expf(z[e] - mx);
      s[e] = v;
      sum += v;
    }
    sum = wave_sum(sum);
    const float inv = 1.0f / sum;
    for (int e = lane; e < E; e += PI_WAVE) {
      s[e] *= inv;
      c[e] = correction ? s[e] + correction[e] : s[e];
      allowed[e] = (groups <= 1) ? 1 : 0;
    }
  }
  __syncthreads();
  if (groups > 1) {
    const int per = E / groups;
    for (int g = lane; g < groups; g += PI_WAVE) {
      float best = -INFINITY;
      for (int e = g * per; e < (g + 1) * per; ++e) best = fmaxf(best, c[e]);
      gscore[g] = best;
    }
    __syncthreads();
    for (int j = 0; j < keep; ++j) {
      float v = -INFINITY;
      int idx = 0x7fffffff;
      for (int g = lane; g < groups; g += PI_WAVE)
        if (gscore[g] > v) {
          v = gscore[g];
          idx = g;
        }
      wave_argmax(v, idx);
      if (idx < groups) {
        for (int e = idx * per + lane; e < (idx + 1) * per; e += PI_WAVE) allowed[e] = 1;
        if (lane == 0) gscore[idx] = -INFINITY;
      }
      __syncthreads();
    }
  }
  float wsum = 0.f;
  for (int j = 0; j < top; ++j) {
    float v = -INFINITY;
    int idx = 0x7fffffff;
    for (int e = lane; e < E; e += PI_WAVE)
      if (allowed[e] && c[e] > v) {
        v = c[e];
        idx = e;
      }
    wave_argmax(v, idx);
    if (idx >= E) {          // fewer allowed experts than choices: the entry counts nothing
      idx = 0;
      v = 0.f;
    } else {
      v = s[idx];
      if (lane == 0) allowed[idx] = 0;
    }
    wsum += v;
    if (lane == 0) {
      ids[t * top + j] = idx;
      weights[t * top + j] = v;
    }
    __syncthreads();
  }
  if (renorm && lane == 0) {
    const float r = 1.0f / (wsum + renorm_eps);
    for (int j = 0; j < top; ++j) weights[t * top + j] *= r;
  }
}

extern "C" int pi_route(int* ids, float* weights, const float* logits, long logits_stride, int splits, int T, int E, int top, int groups,
                        int keep, int renorm, const float* correction, float renorm_eps, int sigmoid, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && E > 0 && E <= RE_MAX_EXPERTS, "routing: %d experts (at most %d)", E, RE_MAX_EXPERTS);
  PI_REQUIRE(splits >= 1 && logits_stride >= E, "routing: bad logits (%d pieces, rows of %ld)", splits, logits_stride);
  PI_REQUIRE(top > 0 && top <= E, "routing: %d choices among %d experts", top, E);
  PI_REQUIRE(groups <= 1 || (E % groups == 0 && keep > 0 && keep <= groups), "routing: %d experts in %d groups, %d kept", E, groups, keep);
  PI_REQUIRE(groups <= 1 || (long)keep * (E / groups) >= top, "routing: %d kept groups of %d experts hold fewer than %d choices", keep, groups > 0 ? E / groups : 0, top);
  if (T == 0) return 0;
  hipLaunchKernelGGL(route_kernel, dim3(T), dim3(PI_WAVE), 0, stream, ids, weights, logits, logits_stride, splits, (long)T * logits_stride, E, top, groups, keep, renorm, correction, renorm_eps, sigmoid);
  return pi_check_launch("route");
}

// ---------------------------------------------------------------- entries grouped by expert
// N entries (entry = token * top + choice) with their expert ids -> rows in expert order:
//   row_entry[row] = entry, entry_row[entry] = row (entries of one expert keep their order),
//   tiles of up to `tile` rows that never straddle two experts: tile_expert[i] (-1: unused),
//   tile_row0[i], tile_rows[i]; max_tiles = ceil(N / tile) + E bounds their number.
// Entries whose id is not in 0 .. E - 1 (identity experts) own no row: their entry_row is 0, and the rows
// that stay empty behind the last expert's name entry 0, so that whoever walks all N rows stays in bounds.
// One block of 1024 threads.  Wave w owns the w-th sixteenth of the entries and a row of counters [experts] in LDS: it
// counts its entries per expert, the counters become every wave's first row per expert, and it places its entries in
// order.  The lanes of a wave that hold the same expert find each other by votes on the bits of its number.
#define RE_WAVES 16
#define RE_AHEAD 8          // rounds of 64 entries whose ids are asked for together

// calls use(entry, expert or -1, lanes with the same expert) for the wave's entries, 64 at a time and in order
template <typename Use>
__device__ inline void walk_entries(const int* __restrict__ ids, int first, int last, int E, int bits, int lane, Use&& use) {
  for (int i0 = first; i0 < last; i0 += RE_AHEAD * PI_WAVE) {
    int id[RE_AHEAD];
#pragma unroll
    for (int u = 0; u < RE_AHEAD; ++u) {
      const int i = i0 + u * PI_WAVE + lane;
      id[u] = i < last ? ids[i] : -1;
    }
#pragma unroll
    for (int u = 0; u < RE_AHEAD; ++u) {
      if (i0 + u * PI_WAVE >= last) break;
      const int e = id[u] >= 0 && id[u] < E ? id[u] : -1;
      unsigned long long same = __ballot(e >= 0);
      for (int b = 0; b < bits; ++b) {
        const unsigned long long ones = __ballot((e >> b) & 1);
        same &= (e >> b) & 1 ? ones : ~ones;
      }
      use(i0 + u * PI_WAVE + lane, e, same);
    }
  }
}

__global__ __launch_bounds__(1024) void group_entries_kernel(const int* __restrict__ ids, int N, int E, int* __restrict__ row_entry,
                                                             int* __restrict__ entry_row, int* __restrict__ tile_expert,
                                                             int* __restrict__ tile_row0, int* __restrict__ tile_rows, int max_tiles,
                                                             int tile, int bits) {
  extern __shared__ int counters[];              // [waves][E]
  __shared__ int rows_to[2][RE_MAX_EXPERTS];     // running sums over the experts, two buffers in turn: rows ...
  __shared__ int tiles_to[2][RE_MAX_EXPERTS];    // ... and tiles
  const int tid = threadIdx.x, lane = tid % PI_WAVE, wave = tid / PI_WAVE;
  const int per = ((N + RE_WAVES - 1) / RE_WAVES + PI_WAVE - 1) / PI_WAVE * PI_WAVE;
  const int first = min(N, wave * per), last = min(N, first + per);
  volatile int* mine = counters + wave * E;      // read by all lanes of the wave before one of them changes it
  for (int i = tid; i < RE_WAVES * E; i += 1024) counters[i] = 0;
  __syncthreads();
  walk_entries(ids, first, last, E, bits, lane, [&](int, int e, unsigned long long same) {
    if (e >= 0 && lane == __ffsll(same) - 1) mine[e] = mine[e] + __popcll(same);
  });
  __syncthreads();
  int rows = 0;                                  // thread e: expert e (RE_MAX_EXPERTS is the block's size)
  if (tid < E)
    for (int w = 0; w < RE_WAVES; ++w) rows += counters[w * E + tid];
  const int tiles = (rows + tile - 1) / tile;
  rows_to[0][tid] = rows;
  tiles_to[0][tid] = tiles;
  int b = 0;
  for (int off = 1; off < E; off *= 2, b ^= 1) {
    __syncthreads();
    rows_to[b ^ 1][tid] = rows_to[b][tid] + (tid >= off ? rows_to[b][tid - off] : 0);
    tiles_to[b ^ 1][tid] = tiles_to[b][tid] + (tid >= off ? tiles_to[b][tid - off] : 0);
  }
  __syncthreads();
  const int all_rows = rows_to[b][E - 1], all_tiles = tiles_to[b][E - 1];
  if (tid < E) {
    int at = rows_to[b][tid] - rows;
    for (int w = 0; w < RE_WAVES; ++w) {         // every wave's first row of this expert
      const int n = counters[w * E + tid];
      counters[w * E + tid] = at;
      at += n;
    }
  }
  for (int i = all_rows + tid; i < N; i += 1024) row_entry[i] = 0;
  for (int i = all_tiles + tid; i < max_tiles; i += 1024) {
    tile_expert[i] = -1;
    tile_row0[i] = 0;
    tile_rows[i] = 0;
  }
  for (int e = wave; e < E; e += RE_WAVES) {
    const int end = rows_to[b][e], row0 = e ? rows_to[b][e - 1] : 0, t0 = e ? tiles_to[b][e - 1] : 0;
    for (int i = lane; t0 + i < tiles_to[b][e]; i += PI_WAVE) {
      tile_expert[t0 + i] = e;
      tile_row0[t0 + i] = row0 + i * tile;
      tile_rows[t0 + i] = min(tile, end - row0 - i * tile);
    }
  }
  __syncthreads();
  walk_entries(ids, first, last, E, bits, lane, [&](int i, int e, unsigned long long same) {
    const int at = e >= 0 ? mine[e] : 0;
    if (e >= 0) {
      const int row = at + __popcll(same & ((1ull << lane) - 1ull));
      row_entry[row] = i;
      entry_row[i] = row;
      if (lane == __ffsll(same) - 1) mine[e] = at + __popcll(same);
    } else if (i < last) {
      entry_row[i] = 0;
    }
  });
}

extern "C" int pi_group_entries(const int* ids, int N, int E, int* row_entry, int* entry_row, int* tile_expert, int* tile_row0,
                                int* tile_rows, int max_tiles, int tile, hipStream_t stream) {
  PI_REQUIRE(N >= 0 && E > 0 && E <= RE_MAX_EXPERTS && tile > 0, "grouping: bad sizes N=%d E=%d tile=%d", N, E, tile);
  PI_REQUIRE(max_tiles >= (N + tile - 1) / tile + E, "grouping: room for %d tiles is too little", max_tiles);
  if (N == 0) return 0;
  int bits = 0;
  while ((1 << bits) < E) ++bits;
  const size_t lds = (size_t)RE_WAVES * E * sizeof(int);
  static bool configured = false;
  if (!configured) {
    hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(group_entries_kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                                         RE_WAVES * RE_MAX_EXPERTS * (int)sizeof(int));
    if (err != hipSuccess) return pi_fail("grouping: cannot reserve LDS: %s", hipGetErrorString(err));
    configured = true;
  }
  hipLaunchKernelGGL(group_entries_kernel, dim3(1), dim3(1024), lds, stream, ids, N, E, row_entry, entry_row, tile_expert, tile_row0,
                     tile_rows, max_tiles, tile, bits);
  return pi_check_launch("group_entries");
}

extern "C" int pi_group_tile_rows() { return RE_TILE; }

// rows[row, :] = src[row_entry[row] / top, :]   (activations copied into expert order), times the entry's weight when
// weights are given (routing that weighs an expert's input instead of its output)
template <typename T>
__global__ void gather_rows_kernel(T* __restrict__ out, const T* __restrict__ src, const int* __restrict__ row_entry, int top, int D,
                                   const float* __restrict__ weights) {
  const long row = blockIdx.x;
  const long t = row_entry[row] / top;
  if (weights) {
    const float w = weights[row_entry[row]];
    for (int d = threadIdx.x; d < D; d += blockDim.x) out[row * D + d] = from_float<T>(to_float(src[t * D + d]) * w);
    return;
  }
  for (int d = threadIdx.x; d < D; d += blockDim.x) out[row * D + d] = src[t * D + d];
}

// The same for rows of whole 16-byte groups.
template <typename T>
__global__ void gather_rows_wide_kernel(T* __restrict__ out, const T* __restrict__ src, const int* __restrict__ row_entry, int top, int groups,
                                        const float* __restrict__ weights) {
  const long row = blockIdx.x;
  const int entry = row_entry[row];
  const uint4* from = reinterpret_cast<const uint4*>(src) + (long)(entry / top) * groups;
  uint4* to = reinterpret_cast<uint4*>(out) + row * groups;
  const float w = weights ? weights[entry] : 1.f;
  for (int g = threadIdx.x; g < groups; g += blockDim.x) {
    uint4 v = from[g];
    if (weights) {
      uint32_t* p = reinterpret_cast<uint32_t*>(&v);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (sizeof(T) == 4) p[i] = __float_as_uint(__uint_as_float(p[i]) * w);
        else p[i] = f32x2_to_bf16x2_bits(__uint_as_float(p[i] << 16) * w, __uint_as_float(p[i] & 0xffff0000u) * w);
      }
    }
    to[g] = v;
  }
}

extern "C" int pi_gather_rows(void* out, const void* src, int dtype, const int* row_entry, int N, int top, int D, const float* weights,
                              hipStream_t stream) {
  PI_REQUIRE(N >= 0 && top > 0 && D > 0, "gather: bad sizes");
  PI_REQUIRE(dtype == PI_F32 || dtype == PI_BF16, "gather: unsupported dtype %d", dtype);
  if (N == 0) return 0;
  const int per = dtype == PI_F32 ? 4 : 8;
  if (D % per == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)src % 16 == 0) {
    const int groups = D / per, threads = groups >= 256 ? 256 : ceil_div(groups, PI_WAVE) * PI_WAVE;
    if (dtype == PI_F32)
      hipLaunchKernelGGL(gather_rows_wide_kernel<float>, dim3(N), dim3(threads), 0, stream, (float*)out, (const float*)src, row_entry, top, groups, weights);
    else
      hipLaunchKernelGGL(gather_rows_wide_kernel<bf16_t>, dim3(N), dim3(threads), 0, stream, (bf16_t*)out, (const bf16_t*)src, row_entry, top, groups, weights);
    return pi_check_launch("gather_rows_wide");
  }
  if (dtype == PI_F32)
    hipLaunchKernelGGL(gather_rows_kernel<float>, dim3(N), dim3(256), 0, stream, (float*)out, (const float*)src, row_entry, top, D, weights);
  else
    hipLaunchKernelGGL(gather_rows_kernel<bf16_t>, dim3(N), dim3(256), 0, stream, (bf16_t*)out, (const bf16_t*)src, row_entry, top, D, weights);
  return pi_check_launch("gather_rows");
}

// ---------------------------------------------------------------- grouped product, any size and type
// C[row, :] = A[row, :] . W[expert of row]^T for the rows of every tile; W is [E, N, K].  float32
// multiply-add, each output accumulating over k in ascending order: a row's result does not
// depend on the rows around it.
#define RG_T 64
#define RG_K 16
template <typename TA, typename TW, typename TC>
__global__ __launch_bounds__(256) void grouped_gemm_general_kernel(TC* __restrict__ C, long ldc, const TA* __restrict__ A, long lda,
                                                                   const TW* __restrict__ W, long ldw, long w_expert_stride,
                                                                   const int* __restrict__ tile_expert, const int* __restrict__ tile_row0,
                                                                   const int* __restrict__ tile_rows, int N, int K) {
  const int e = tile_expert[blockIdx.y];
  if (e < 0) return;
  __shared__ float As[RG_K][RG_T + 4];
  __shared__ float Ws[RG_K][RG_T + 4];
  const int tid = threadIdx.x;
  const int tx = tid % 16, ty = tid / 16;
  const long n0 = (long)blockIdx.x * RG_T;
  const TW* We = W + (long)e * w_expert_stride;
  // a tile of more than RG_T rows (lists made for the matrix-core kernel) is walked in pieces
  for (int sub = 0; sub < tile_rows[blockIdx.y]; sub += RG_T) {
    const long m0 = tile_row0[blockIdx.y] + sub;
    const int M = min(RG_T, tile_rows[blockIdx.y] - sub);
    float acc[4][4] = {};
    for (int k0 = 0; k0 < K; k0 += RG_K) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int idx = tid + i * 256;
        const int row = idx / RG_K, kk = idx % RG_K;
        const long n = n0 + row;
        const int k = k0 + kk;
        As[kk][row] = (row < M && k < K) ? to_float(A[(m0 + row) * lda + k]) : 0.f;
        Ws[kk][row] = (n < N && k < K) ? to_float(We[n * ldw + k]) : 0.f;
      }
      __syncthreads();
#pragma unroll
      for (int kk = 0; kk < RG_K; ++kk) {
        float a[4], w[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) a[i] = As[kk][ty * 4 + i];
#pragma unroll
        for (int j = 0; j < 4; ++j) w[j] = Ws[kk][tx * 4 + j];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], w[j], acc[i][j]);
      }
      __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = ty * 4 + i;
      if (r >= M) continue;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const long n = n0 + tx * 4 + j;
        if (n < N) C[(m0 + r) * ldc + n] = from_float<TC>(acc[i][j]);
      }
    }
  }
}

extern "C" int pi_grouped_gemm_general(void* C, int c_dtype, long ldc, const void* A, int a_dtype, long lda, const void* W, int w_dtype,
                                       long ldw, long w_expert_stride, const int* tile_expert, const int* tile_row0,
                                       const int* tile_rows, int tiles, int N, int K, hipStream_t stream) {
  PI_REQUIRE(tiles >= 0 && N > 0 && K > 0 && lda >= K && ldw >= K && ldc >= N, "grouped product: bad sizes");
  PI_REQUIRE(tiles <= 65535, "grouped product: too many tiles (%d)", tiles);
  PI_REQUIRE(a_dtype == w_dtype, "grouped product: activations and weights must have one type");
  if (tiles == 0) return 0;
  const dim3 grid(ceil_div(N, RG_T), tiles), block(256);
#define RG_GO(TA, TC) hipLaunchKernelGGL((grouped_gemm_general_kernel<TA, TA, TC>), grid, block, 0, stream, (TC*)C, ldc, (const TA*)A, lda, \
                                         (const TA*)W, ldw, w_expert_stride, tile_expert, tile_row0, tile_rows, N, K)
  if (a_dtype == PI_F32 && c_dtype == PI_F32) RG_GO(float, float);
  else if (a_dtype == PI_BF16 && c_dtype == PI_F32) RG_GO(bf16_t, float);
  else if (a_dtype == PI_BF16 && c_dtype == PI_BF16) RG_GO(bf16_t, bf16_t);
  else return pi_fail("grouped product: unsupported dtypes a=%d c=%d", a_dtype, c_dtype);
#undef RG_GO
  return pi_check_launch("grouped_gemm_general");
}

// out[t, :] (+)= sum_j weights[t, j] * y[entry_row[t * top + j], :], choices in order (float32); a choice whose
// id is num_real or more (ids given) stands for the token's own activations h[t, :] instead; weights null: a plain sum
template <typename TH>
__global__ void combine_choices_kernel(float* __restrict__ out, const float* __restrict__ y, const float* __restrict__ weights,
                                       const int* __restrict__ entry_row, int top, int D, int accumulate, const int* __restrict__ ids,
                                       int num_real, const TH* __restrict__ h) {
  const long t = blockIdx.x;
  const int d = blockIdx.y * blockDim.x + threadIdx.x;
  if (d >= D) return;
  float acc = 0.f;
  for (int j = 0; j < top; ++j) {
    const bool own = ids && ids[t * top + j] >= num_real;
    const float v = own ? to_float(h[t * D + d]) : y[(long)entry_row[t * top + j] * D + d];
    acc = weights ? fmaf(weights[t * top + j], v, acc) : acc + v;
  }
  out[t * D + d] = accumulate ? out[t * D + d] + acc : acc;
}

extern "C" int pi_combine_choices(float* out, const float* y, const float* weights, const int* entry_row, int T, int top, int D,
                                  int accumulate, const int* ids, int num_real, const void* h, int h_dtype, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && top > 0 && D > 0, "combine: bad sizes");
  PI_REQUIRE(!ids || h, "combine: identity experts need the tokens' activations");
  if (T == 0) return 0;
  PI_REQUIRE((D + 255) / 256 <= 65535, "combine: rows of %d are too long", D);
  const dim3 grid(T, (D + 255) / 256), block(256);
  if (ids && h_dtype == PI_BF16)
    hipLaunchKernelGGL(combine_choices_kernel<bf16_t>, grid, block, 0, stream, out, y, weights, entry_row, top, D, accumulate, ids, num_real, (const bf16_t*)h);
  else if (!ids || h_dtype == PI_F32)
    hipLaunchKernelGGL(combine_choices_kernel<float>, grid, block, 0, stream, out, y, weights, entry_row, top, D, accumulate, ids, num_real, (const float*)h);
  else
    return pi_fail("combine: unsupported activation dtype %d", h_dtype);
  return pi_check_launch("combine_choices");
}
