// A recurrence of one number per feature whose gate and candidate do not look at the state (minGRU):
//   z = sigmoid(zp + bz),  u = up + bu,  c = u + 1/2 where u >= 0, sigmoid(u) where u < 0
//   S <- (1 - z) S + z c;   out = S * silu(g)
// from float32 projection rows [zp: W | up: W | g: W] (a tensor, or the pieces of a product split over k), from and
// into the requests' state rows.  Everything is float32; 1 - z is made as sigmoid(-(zp + bz)), so that a gate that is
// nearly shut loses nothing to cancellation.
//
// The recurrence is linear in S: a run of tokens takes S to A S + B with A the product of its (1 - z) and B its walk
// from zero.  A request's tokens are cut into chunks; a first kernel makes every chunk's (A, B), a second one runs
// over the earlier chunks' (A, B) to its own start and walks its chunk, all chunks side by side.  All terms are
// positive and A is at most 1, so the cut changes nothing but the rounding.  The first chunk's record is (the state
// before it, the state behind it): the state row is read by the first kernel alone and written by the second alone.
// Short portions and single tokens are one chunk and need the second kernel only.
#include "common.h"

#define GR_THREADS 256

struct GruArgs {
  const float* proj;      // [T, >= 3W], or null: the pieces
  long proj_stride;
  const float* part;      // [splits, T, proj_stride]
  int splits;
  long plane;
  const float* bias;      // bz [W], bu [W]
  const int* q_start;
  const int* slots;
  float* state;           // [slots, >= W]
  long state_stride;
  int num_slots, W, chunk;
  float* ab;              // [T / chunk + R, 2, W]: the chunks' records; null: every request is one chunk
};

__device__ inline float gr_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }

// the step's two numbers for (token, feature): keep = 1 - z, add = z c
__device__ inline void gr_terms(float zp, float up, float& keep, float& add) {
  const float e = expf(-fabsf(zp));                 // no overflow: the two sigmoids from one exponential
  const float small = e / (1.0f + e), big = 1.0f / (1.0f + e);
  const float z = zp >= 0.f ? big : small;
  keep = zp >= 0.f ? small : big;
  add = z * (up >= 0.f ? up + 0.5f : gr_sigmoid(up));
}

template <bool PIECES>
__device__ inline float gr_column(const GruArgs& a, long t, int col) {
  return PIECES ? split_sum(a.part, a.splits, a.plane, t * a.proj_stride + col) : a.proj[t * a.proj_stride + col];
}

// (request, chunk) of this block and its tokens; false: there is no such chunk
__device__ inline bool gr_range(const GruArgs& a, int& t0, int& t1, long& row) {
  const int r = blockIdx.z, q0 = a.q_start[r], q1 = a.q_start[r + 1];
  t0 = q0 + blockIdx.y * a.chunk;
  t1 = min(q1, t0 + a.chunk);
  row = q0 / a.chunk + r;                           // the request's first row of `ab`: chunks of different requests never share one
  return t0 < q1;
}

#define GR_AHEAD 8        // tokens whose loads are in flight together
#define GR_RECORDS 16     // the same of the chunks' records

// The tokens t0 .. t1 - 1 of feature c, in order: use(t, keep, add, gate) for each; GATE: with the gate's column.
template <bool PIECES, bool GATE, typename Use>
__device__ inline void gr_walk(const GruArgs& a, int c, int t0, int t1, Use&& use) {
  const float bz = a.bias[c], bu = a.bias[a.W + c];
  int t = t0;
  for (; t + GR_AHEAD <= t1; t += GR_AHEAD) {
    float zp[GR_AHEAD], up[GR_AHEAD], g[GR_AHEAD];
#pragma unroll
    for (int i = 0; i < GR_AHEAD; ++i) {
      zp[i] = gr_column<PIECES>(a, t + i, c);
      up[i] = gr_column<PIECES>(a, t + i, a.W + c);
      g[i] = GATE ? gr_column<PIECES>(a, t + i, 2 * a.W + c) : 0.f;
    }
#pragma unroll
    for (int i = 0; i < GR_AHEAD; ++i) {
      float keep, add;
      gr_terms(zp[i] + bz, up[i] + bu, keep, add);
      use(t + i, keep, add, g[i]);
    }
  }
  for (; t < t1; ++t) {
    float keep, add;
    const float g = GATE ? gr_column<PIECES>(a, t, 2 * a.W + c) : 0.f;
    gr_terms(gr_column<PIECES>(a, t, c) + bz, gr_column<PIECES>(a, t, a.W + c) + bu, keep, add);
    use(t, keep, add, g);
  }
}

template <bool PIECES>
__global__ __launch_bounds__(GR_THREADS) void gru_chunk_kernel(GruArgs a) {
  int t0, t1;
  long row;
  if (!gr_range(a, t0, t1, row)) return;
  const int c = blockIdx.x * GR_THREADS + threadIdx.x;
  if (c >= a.W) return;
  float A = 1.f, B = 0.f, S0 = 0.f;
  if (blockIdx.y == 0) {
    const int slot = a.slots[blockIdx.z];
    S0 = slot >= 0 && slot < a.num_slots ? a.state[(long)slot * a.state_stride + c] : 0.f;
  }
  gr_walk<PIECES, false>(a, c, t0, t1, [&](int, float keep, float add, float) {
    A *= keep;
    B = fmaf(keep, B, add);
  });
  float* ab = a.ab + (row + blockIdx.y) * 2 * a.W + c;
  ab[0] = blockIdx.y == 0 ? S0 : A;
  ab[a.W] = blockIdx.y == 0 ? fmaf(A, S0, B) : B;
}

template <typename T, bool PIECES>
__global__ __launch_bounds__(GR_THREADS) void gru_walk_kernel(GruArgs a, T* __restrict__ out, long out_stride) {
  int t0, t1;
  long row;
  if (!gr_range(a, t0, t1, row)) return;
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= a.W) return;
  const int slot = a.slots[blockIdx.z];
  const bool has_state = slot >= 0 && slot < a.num_slots;
  float* st = a.state + (long)slot * a.state_stride + c;
  float S;
  if (!a.ab) {
    S = has_state ? *st : 0.f;
  } else if (blockIdx.y == 0) {
    S = a.ab[row * 2 * a.W + c];
  } else {
    const float* ab = a.ab + row * 2 * a.W + c;
    S = ab[a.W];
    const int before = blockIdx.y;
    for (int j = 1; j < before; j += GR_RECORDS) {
      float A[GR_RECORDS], B[GR_RECORDS];
#pragma unroll
      for (int i = 0; i < GR_RECORDS; ++i) {
        const bool in = j + i < before;
        A[i] = in ? ab[(long)(j + i) * 2 * a.W] : 1.f;
        B[i] = in ? ab[(long)(j + i) * 2 * a.W + a.W] : 0.f;
      }
#pragma unroll
      for (int i = 0; i < GR_RECORDS; ++i) S = fmaf(A[i], S, B[i]);
    }
  }
  gr_walk<PIECES, true>(a, c, t0, t1, [&](int t, float keep, float add, float g) {
    S = fmaf(keep, S, add);
    out[(long)t * out_stride + c] = from_float<T>(S * g / (1.0f + expf(-g)));
  });
  if (has_state && t1 == a.q_start[blockIdx.z + 1]) *st = S;
}

// A step of single tokens: a thread per (request, feature), nothing ahead.
template <typename T, bool PIECES>
__global__ __launch_bounds__(GR_THREADS) void gru_step_kernel(GruArgs a, T* __restrict__ out, long out_stride) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x, r = blockIdx.z;
  const long t = a.q_start[r];
  const int slot = a.slots[r];
  if (c >= a.W) return;
  const bool has_state = slot >= 0 && slot < a.num_slots;
  float* st = a.state + (long)slot * a.state_stride + c;
  const float S0 = has_state ? *st : 0.f;
  const float zp = gr_column<PIECES>(a, t, c) + a.bias[c], up = gr_column<PIECES>(a, t, a.W + c) + a.bias[a.W + c], g = gr_column<PIECES>(a, t, 2 * a.W + c);
  float keep, add;
  gr_terms(zp, up, keep, add);
  const float S = fmaf(keep, S0, add);
  out[t * out_stride + c] = from_float<T>(S * g / (1.0f + expf(-g)));
  if (has_state) *st = S;
}

// Tokens per chunk for a step whose longest request brings `longest` tokens.
static int gru_chunk(int longest) {
  int chunk = 32;
  while (chunk < 512 && longest > 64 * chunk) chunk *= 2;      // no more than 64 chunks to run over (long portions: more)
  return chunk;
}

// Floats of the chunks' records that pi_min_gru wants for such a step (0: every request is one chunk).
extern "C" long pi_min_gru_work_floats(int T, int R, int longest, int W) {
  const int chunk = gru_chunk(longest);
  return longest <= chunk ? 0 : ((long)T / chunk + R) * 2 * W;
}

extern "C" int pi_min_gru(void* out, int out_dtype, long out_stride, const float* proj, long proj_stride, const float* part, int splits,
                          const float* bias, const int* q_start, const int* slots, int R, int T, int longest, float* state,
                          long state_stride, int num_slots, int W, float* work, long work_floats, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && R >= 0 && W > 0 && longest >= 0 && longest <= T, "min gru: bad sizes T=%d R=%d W=%d longest=%d", T, R, W, longest);
  PI_REQUIRE((proj != nullptr) != (part != nullptr) && (!part || splits >= 1) && proj_stride >= 3L * W, "min gru: bad projection");
  PI_REQUIRE(out && out_stride >= W && bias && q_start && slots && state && state_stride >= W, "min gru: bad arguments");
  PI_REQUIRE(out_dtype == PI_F32 || out_dtype == PI_BF16, "min gru: unsupported dtype %d", out_dtype);
  PI_REQUIRE(R <= 65535, "min gru: too many requests (%d)", R);
  if (T == 0 || R == 0) return 0;
  GruArgs a{proj, proj_stride, part, splits, (long)T * proj_stride, bias, q_start, slots, state, state_stride, num_slots, W, gru_chunk(longest), nullptr};
  const int threads = W >= 4 * GR_THREADS && longest > 1 ? GR_THREADS : PI_WAVE;
#define GR_GO(K, GRID)                                                                                                     \
  do {                                                                                                                     \
    if (out_dtype == PI_F32) {                                                                                             \
      if (part) hipLaunchKernelGGL((K<float, true>), GRID, dim3(threads), 0, stream, a, (float*)out, out_stride);          \
      else hipLaunchKernelGGL((K<float, false>), GRID, dim3(threads), 0, stream, a, (float*)out, out_stride);              \
    } else {                                                                                                               \
      if (part) hipLaunchKernelGGL((K<bf16_t, true>), GRID, dim3(threads), 0, stream, a, (bf16_t*)out, out_stride);        \
      else hipLaunchKernelGGL((K<bf16_t, false>), GRID, dim3(threads), 0, stream, a, (bf16_t*)out, out_stride);            \
    }                                                                                                                      \
  } while (0)
  if (longest == 1) {
    const dim3 grid(ceil_div(W, threads), 1, R);
    GR_GO(gru_step_kernel, grid);
    return pi_check_launch("gru_step");
  }
  const int chunks = ceil_div(longest, a.chunk);
  PI_REQUIRE(chunks <= 65535, "min gru: a portion of %d tokens is too long", longest);
  if (chunks > 1) {
    PI_REQUIRE(work && work_floats >= pi_min_gru_work_floats(T, R, longest, W), "min gru: the chunks' records do not fit");
    a.ab = work;
    const dim3 grid(ceil_div(W, GR_THREADS), chunks, R);
    if (part) hipLaunchKernelGGL(gru_chunk_kernel<true>, grid, dim3(GR_THREADS), 0, stream, a);
    else hipLaunchKernelGGL(gru_chunk_kernel<false>, grid, dim3(GR_THREADS), 0, stream, a);
    if (pi_check_launch("gru_chunk")) return -1;
  }
  const dim3 grid(ceil_div(W, threads), chunks, R);
  GR_GO(gru_walk_kernel, grid);
#undef GR_GO
  return pi_check_launch("gru_walk");
}
