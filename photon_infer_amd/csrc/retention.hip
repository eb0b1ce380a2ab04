// Retention, a linear attention whose state decays by a constant of its head (Sun et al., "Retentive Network: A
// Successor to Transformer for Large Language Models").  Per head, with state S [d, dv] (float32, zero at the start):
//   q' = rotate(q);  k' = rotate(k) * k_scale;   S <- decay S + k' v^T;   o = S^T q'
//   y = o / sqrt(mean(o^2) + eps) * silu(gate)
// A token's row of the projection (float32) holds [q: H*d | k: H*d | v: H*dv | gates: H*dv].  A request's state row
// (state[slots[r]], laid out [H, d, dv]) is read at the start of a step and left ready for the next, so a prompt may be cut
// anywhere.  Everything is float32 in both compute modes, the matrix products too (v_mfma_f32_16x16x4_f32); only y is rounded.
//
// A step of single tokens is one kernel: rotation, state, norm and gate.  Longer portions are cut into chunks of 64 tokens,
// counted from a request's first token of the step, that run side by side in three kernels:
//   sums    U_c  = sum over the chunk's tokens j of decay^(len - 1 - j) k'_j v_j^T
//   states  S_c  = the state in front of chunk c:  S_(c+1) = decay^len S_c + U_c  (one thread per element walks the chunks)
//   out     o_i  = decay^(i+1) S_c^T q'_i + sum over j <= i of decay^(i-j) <q'_i, k'_j> v_j,  then norm and gate
// Powers of the decay are taken as 2^(n log2 decay), never by dividing one by another.
#include "mfma.h"

#define RT_CHUNK 64
#define RT_THREADS 256
#define RT_SLAB 64              // features staged at a time
#define RT_QK_LD (RT_SLAB + 4)  // row length in LDS: rows fall four banks apart, and four rows on sixteen

struct RetentionArgs {
  const float* proj;        // [T, stride], or null: the pieces (single tokens only)
  long stride;
  const float* part;        // [splits, T, stride]
  int splits;
  long plane;
  const float* table;       // [T, rd]: cosines, then sines
  int rd, interleaved;
  const float* decay;       // [H]: the decay, then [H]: its log2
  float k_scale, eps;
  const int* q_start;
  const int* slots;
  float* state;
  long state_stride;
  int num_slots;
  int H, d, dv;
  int vec;                  // rows and heads are whole 16-byte groups
  float* work;              // chunk records, [records, H, d, dv]
  int col_tiles;            // `out`: blocks per (chunk, head)
};

__device__ inline float* state_row(const RetentionArgs& a, int r) {
  const int slot = a.slots[r];
  return slot >= 0 && slot < a.num_slots ? a.state + (long)slot * a.state_stride : nullptr;      // the host checks slots
}
__device__ inline float power2(float n, float log2_decay) { return __builtin_amdgcn_exp2f(n * log2_decay); }
__device__ inline float silu_full(float z) { return z / (1.0f + expf(-z)); }

// where feature i's rotation partner lies and which pair it is (i < rd)
__device__ inline int partner_of(const RetentionArgs& a, int i) { return a.interleaved ? i ^ 1 : (i < a.rd / 2 ? i + a.rd / 2 : i - a.rd / 2); }
__device__ inline float rotated(const RetentionArgs& a, const float* cs, int i, float x, float other) {
  const int half = a.rd / 2;
  const bool low = a.interleaved ? (i & 1) == 0 : i < half;
  const int j = a.interleaved ? i / 2 : (low ? i : i - half);
  float lo, hi;
  rope_pair(low ? x : other, low ? other : x, cs[j], cs[half + j], lo, hi);
  return low ? lo : hi;
}

// ------------------------------------------------------------------ single tokens
// One block per (head, request).  A thread owns VEC neighbouring value columns of the rows rg, rg + row groups, ..
template <typename TY, int VEC>
__global__ __launch_bounds__(1024) void retention_step_kernel(RetentionArgs a, TY* __restrict__ y) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float scratch[16];
  const int h = blockIdx.x, r = blockIdx.y, tid = threadIdx.x, NT = blockDim.x;
  const int d = a.d, dv = a.dv;
  const long t = r;                                  // token r is request r's
  float* const q = lds;
  float* const k = q + d;
  float* const v = k + d;
  float* const gate = v + dv;
  float* const o = gate + dv;
  float* const sums = lds + ((2 * d + 3 * dv + 3) & ~3);
  float* const row = state_row(a, r);
  if (!row) return;                                  // the same for the whole block
  float* const S = row + (long)h * d * dv;
  const float g = a.decay[h];
  const int groups = dv / VEC;                       // column groups; VEC divides dv
  int lanes_c = 1;
  while (lanes_c < groups && lanes_c < NT) lanes_c *= 2;
  const int rg = tid / lanes_c, nrg = NT / lanes_c;
  constexpr int U = 8;                               // rows in flight
  float s[U][VEC];
  auto fetch = [&](int cg, int c0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + u * nrg;
      const bool ok = cg < groups && c < d;
      const float* src = S + (long)(ok ? c : 0) * dv + (ok ? cg : 0) * VEC;
      if constexpr (VEC == 4) {
        const float4 f = *reinterpret_cast<const float4*>(src);
        s[u][0] = f.x; s[u][1] = f.y; s[u][2] = f.z; s[u][3] = f.w;
      } else {
        s[u][0] = *src;
      }
    }
  };
  fetch(tid % lanes_c, rg);                          // the first rows, on their way while the token's vectors are made
  auto at = [&](long col) { return a.part ? split_sum(a.part, a.splits, a.plane, t * a.stride + col) : a.proj[t * a.stride + col]; };
  const long k_col = (long)a.H * d, v_col = 2 * k_col, g_col = v_col + (long)a.H * dv;
  const float* cs = a.table + t * a.rd;
  const int half = a.rd / 2;
  const float cos0 = tid < half ? cs[tid] : 1.f, sin0 = tid < half ? cs[half + tid] : 0.f;
  for (int i = tid; i < 2 * d + 2 * dv; i += NT) {   // q, k, v and gate lie in a row in LDS
    const long col = i < d ? (long)h * d + i : i < 2 * d ? k_col + (long)h * d + (i - d)
                     : i < 2 * d + dv ? v_col + (long)h * dv + (i - 2 * d) : g_col + (long)h * dv + (i - 2 * d - dv);
    const float x = at(col);
    lds[i] = i >= d && i < 2 * d ? x * a.k_scale : x;
  }
  __syncthreads();
  for (int j = tid; j < half; j += NT) {             // a thread owns a pair
    const int lo_i = a.interleaved ? 2 * j : j, hi_i = a.interleaved ? 2 * j + 1 : j + half;
    const float c = j == tid ? cos0 : cs[j], s1 = j == tid ? sin0 : cs[half + j];
    float lo, hi;
    rope_pair(q[lo_i], q[hi_i], c, s1, lo, hi);
    q[lo_i] = lo; q[hi_i] = hi;
    rope_pair(k[lo_i], k[hi_i], c, s1, lo, hi);
    k[lo_i] = lo; k[hi_i] = hi;
  }
  __syncthreads();
  for (int cb = 0; cb < groups; cb += lanes_c) {
    const int cg = cb + tid % lanes_c;
    const bool in = cg < groups;
    float acc[VEC], vv[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) { acc[e] = 0.f; vv[e] = in ? v[cg * VEC + e] : 0.f; }
    for (int c0 = rg; c0 < d; c0 += U * nrg) {
      if (cb > 0 || c0 > rg) fetch(cg, c0);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int c = c0 + u * nrg;
        if (!(in && c < d)) continue;
        const float kc = k[c], qc = q[c];
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          s[u][e] = fmaf(g, s[u][e], kc * vv[e]);
          acc[e] = fmaf(qc, s[u][e], acc[e]);
        }
        float* dst = S + (long)c * dv + cg * VEC;
        if constexpr (VEC == 4) *reinterpret_cast<float4*>(dst) = make_float4(s[u][0], s[u][1], s[u][2], s[u][3]);
        else *dst = s[u][0];
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) sums[(rg * lanes_c + tid % lanes_c) * VEC + e] = acc[e];
    __syncthreads();
    for (int e = tid; e < lanes_c * VEC; e += NT) {
      const int col = cb * VEC + e;
      if (col < dv) {
        float x = 0.f;
        for (int p = 0; p < nrg; ++p) x += sums[p * lanes_c * VEC + e];
        o[col] = x;
      }
    }
    __syncthreads();
  }
  float ss = 0.f;
  for (int e = tid; e < dv; e += NT) ss = fmaf(o[e], o[e], ss);
  const float rinv = 1.0f / sqrtf(block_sum(ss, scratch) / dv + a.eps);
  for (int e = tid; e < dv; e += NT)
    y[t * a.H * dv + (long)h * dv + e] = from_float<TY>(o[e] * rinv * silu_full(gate[e]));
}

// ------------------------------------------------------------------ chunks
// v_mfma_f32_16x16x4_f32: lane l holds A[l % 16][k], B[k][l % 16] with k = l / 16, and D[(l / 16) * 4 + i][l % 16], i = 0..3.
// Four instructions contract sixteen k; instruction v takes the k = 4 (l / 16) + v of them, in both operands, so that a
// lane's share of a row is four neighbouring numbers and a result tile can be the next product's operand as it is.
__device__ inline f32x4_t mfma_f32(float a, float b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// first record of request r's chunks: requests never meet, whatever their lengths
__device__ inline long first_record(const RetentionArgs& a, int r) { return a.q_start[r] / RT_CHUNK + r; }

// 64 tokens' features f0 .. f0 + SLAB - 1 of q or k of head h (`col`: the head's first column), rotated, into LDS; token j times
// `factor(j)`.  Tokens from len on and features from d on are zero.
template <int SLAB, int THREADS, class Factor>
__device__ inline void stage_rotated(const RetentionArgs& a, float* dst, long t0, int len, long col, int f0, Factor&& factor) {
  if (a.vec) {
    const bool by_fours = !a.interleaved && (a.rd / 2) % 4 == 0 && (uintptr_t)a.table % 16 == 0;
#pragma unroll
    for (int it = 0; it < RT_CHUNK * (SLAB / 4) / THREADS; ++it) {
      const int i = threadIdx.x + it * THREADS;
      const int j = i / (SLAB / 4), f = (i % (SLAB / 4)) * 4, c = f0 + f;
      float x[4] = {0.f, 0.f, 0.f, 0.f};
      if (j < len && c < a.d) {
        const float* src = a.proj + (t0 + j) * a.stride + col;
        const float4 own = *reinterpret_cast<const float4*>(src + c);
        x[0] = own.x; x[1] = own.y; x[2] = own.z; x[3] = own.w;
        if (c < a.rd) {
          const float* cs = a.table + (t0 + j) * a.rd;
          if (by_fours) {                            // four features on one side, their partners side by side on the other
            const int half = a.rd / 2;
            const bool low = c < half;
            const float4 p = *reinterpret_cast<const float4*>(src + (low ? c + half : c - half));
            const float4 cv = *reinterpret_cast<const float4*>(cs + (low ? c : c - half)), sv = *reinterpret_cast<const float4*>(cs + (low ? c + half : c));
            const float o[4] = {p.x, p.y, p.z, p.w}, cc[4] = {cv.x, cv.y, cv.z, cv.w}, ss[4] = {sv.x, sv.y, sv.z, sv.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              float lo, hi;
              rope_pair(low ? x[e] : o[e], low ? o[e] : x[e], cc[e], ss[e], lo, hi);
              x[e] = low ? lo : hi;
            }
          } else {
            float other[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) other[e] = c + e < a.rd ? src[partner_of(a, c + e)] : 0.f;
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (c + e < a.rd) x[e] = rotated(a, cs, c + e, x[e], other[e]);
          }
        }
        const float w = factor(j);
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] *= w;
      }
      *reinterpret_cast<float4*>(dst + j * (SLAB + 4) + f) = make_float4(x[0], x[1], x[2], x[3]);
    }
    return;
  }
  for (int i = threadIdx.x; i < RT_CHUNK * SLAB; i += THREADS) {
    const int j = i / SLAB, f = i % SLAB, c = f0 + f;
    float x = 0.f;
    if (j < len && c < a.d) {
      const float* src = a.proj + (t0 + j) * a.stride + col;
      x = src[c];
      if (c < a.rd) x = rotated(a, a.table + (t0 + j) * a.rd, c, x, src[partner_of(a, c)]);
      x *= factor(j);
    }
    dst[j * (SLAB + 4) + f] = x;
  }
}

// ROWS rows of `ld_src` floats apart, COLS columns from column e0 on, on their way into LDS rows of COLS + 4; rows from n on and
// columns from `cols` on are zero.  Fetching and storing are two steps, so that the next rows can be in flight while the
// ones before them are used (rows that are no whole 16-byte groups are copied by store()).
template <int ROWS, int COLS, int THREADS>
struct StagedRows {
  static constexpr int N = ROWS * (COLS / 4), IT = (N + THREADS - 1) / THREADS;
  float4 v[IT];
  const float* src;
  long ld;
  int n, e0, cols;
  bool vec;
  __device__ inline void fetch(const float* __restrict__ from, long ld_src, int rows, int first_col, int num_cols, bool wide) {
    src = from; ld = ld_src; n = rows; e0 = first_col; cols = num_cols; vec = wide;
    if (!vec) return;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int i = threadIdx.x + it * THREADS, j = i / (COLS / 4), e = (i % (COLS / 4)) * 4;
      v[it] = (j < n && j < ROWS && e0 + e < cols) ? *reinterpret_cast<const float4*>(src + j * ld + e0 + e) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
  }
  __device__ inline void store(float* dst) const {
    if (vec) {
#pragma unroll
      for (int it = 0; it < IT; ++it) {
        const int i = threadIdx.x + it * THREADS, j = i / (COLS / 4), e = (i % (COLS / 4)) * 4;
        if (N % THREADS == 0 || j < ROWS) *reinterpret_cast<float4*>(dst + j * (COLS + 4) + e) = v[it];
      }
      return;
    }
    for (int i = threadIdx.x; i < ROWS * COLS; i += THREADS) {
      const int j = i / COLS, e = i % COLS;
      dst[j * (COLS + 4) + e] = (j < n && e0 + e < cols) ? src[j * ld + e0 + e] : 0.f;
    }
  }
};

// U of one chunk and head: blocks of NW waves, 16 * NW key features x 16 * NT value columns; a wave has 16 features.
template <int NT, int NW>
__global__ __launch_bounds__(NW * PI_WAVE) void retention_sums_kernel(RetentionArgs a) {
  constexpr int COLS = 16 * NT, SLAB = 16 * NW, KLD = SLAB + 4;
  __shared__ __attribute__((aligned(16))) float Ks[RT_CHUNK * KLD];
  __shared__ __attribute__((aligned(16))) float Vs[RT_CHUNK * (COLS + 4)];
  const int tiles_e = (a.dv + COLS - 1) / COLS, tiles = tiles_e * ((a.d + SLAB - 1) / SLAB);
  const int chunk = blockIdx.x / tiles, tile = blockIdx.x % tiles, h = blockIdx.y, r = blockIdx.z;
  const int f0 = tile / tiles_e * SLAB, e0 = tile % tiles_e * COLS;
  const int qs = a.q_start[r], n = a.q_start[r + 1] - qs;
  if (chunk * RT_CHUNK >= n) return;
  const long t0 = qs + chunk * RT_CHUNK;
  const int len = min(RT_CHUNK, n - chunk * RT_CHUNK);
  const int lane = threadIdx.x % PI_WAVE, wave = threadIdx.x / PI_WAVE, lr = lane % 16, lg = lane / 16;
  const float l2 = a.decay[a.H + h];
  StagedRows<RT_CHUNK, COLS, NW * PI_WAVE> values;
  values.fetch(a.proj + t0 * a.stride + 2L * a.H * a.d + (long)h * a.dv, a.stride, len, e0, a.dv, a.vec != 0);
  stage_rotated<SLAB, NW * PI_WAVE>(a, Ks, t0, len, (long)(a.H + h) * a.d, f0, [&](int j) { return a.k_scale * power2((float)(len - 1 - j), l2); });
  values.store(Vs);
  __syncthreads();
  f32x4_t u[NT];
#pragma unroll
  for (int e = 0; e < NT; ++e) u[e] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int used = (len + 15) / 16;                  // later tokens are zero
  for (int jt = 0; jt < used; ++jt) {
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int j = jt * 16 + lg * 4 + v;
      const float kf = Ks[j * KLD + wave * 16 + lr];
#pragma unroll
      for (int e = 0; e < NT; ++e) u[e] = mfma_f32(kf, Vs[j * (COLS + 4) + e * 16 + lr], u[e]);
    }
  }
  float* U = a.work + ((first_record(a, r) + chunk) * a.H + h) * (long)a.d * a.dv;
#pragma unroll
  for (int v = 0; v < 4; ++v) {
    const int c = f0 + wave * 16 + lg * 4 + v;
    if (c >= a.d) continue;
#pragma unroll
    for (int e = 0; e < NT; ++e) {
      const int col = e0 + e * 16 + lr;
      if (col < a.dv) U[(long)c * a.dv + col] = u[e][v];
    }
  }
}

// Records: what each chunk adds becomes the state in front of it; the state row becomes the state behind the last chunk.
template <int VEC>
__global__ __launch_bounds__(RT_THREADS) void retention_states_kernel(RetentionArgs a) {
  const long size = (long)a.d * a.dv;
  const long i = ((long)blockIdx.x * RT_THREADS + threadIdx.x) * VEC;
  const int h = blockIdx.y, r = blockIdx.z;
  if (i >= size) return;
  const int n = a.q_start[r + 1] - a.q_start[r];
  float* row = state_row(a, r);
  if (n <= 0 || !row) return;
  const int chunks = (n + RT_CHUNK - 1) / RT_CHUNK;
  float* st = row + h * size + i;
  float* rec = a.work + (first_record(a, r) * a.H + h) * size + i;
  const long step = (long)a.H * size;
  const float l2 = a.decay[a.H + h], whole = power2((float)RT_CHUNK, l2), last = power2((float)(n - (chunks - 1) * RT_CHUNK), l2);
  float s[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) s[e] = st[e];
  constexpr int U = 8;                               // records in flight
  for (int c0 = 0; c0 < chunks; c0 += U) {
    float u[U][VEC];
#pragma unroll
    for (int x = 0; x < U; ++x) {
      const float* src = rec + (c0 + x < chunks ? c0 + x : 0) * step;
      if constexpr (VEC == 4) {
        const float4 f = *reinterpret_cast<const float4*>(src);
        u[x][0] = f.x; u[x][1] = f.y; u[x][2] = f.z; u[x][3] = f.w;
      } else {
        u[x][0] = *src;
      }
    }
#pragma unroll
    for (int x = 0; x < U; ++x) {
      if (c0 + x >= chunks) break;
      float* dst = rec + (c0 + x) * step;
      if constexpr (VEC == 4) *reinterpret_cast<float4*>(dst) = make_float4(s[0], s[1], s[2], s[3]);
      else *dst = s[0];
      const float g = c0 + x + 1 < chunks ? whole : last;
#pragma unroll
      for (int e = 0; e < VEC; ++e) s[e] = fmaf(g, s[e], u[x][e]);
    }
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) st[e] = s[e];
}

// The results of one chunk and head, value columns e0 .. e0 + 16 * VT * CW - 1.  A wave has 16 queries and 16 * VT columns
// (CW waves share the queries, and the tiles of scores, which they exchange through LDS); everything is transposed (value columns or keys as rows, queries as columns), so that the tile of decayed scores is the operand of the product with
// the values as it lies, and a query's results lie in the four lanes l, l + 16, l + 32, l + 48.  A wave's queries
// meet the key tiles up to their own only.  With all columns in one block (col_tiles 1) the head's norm and the gate
// follow on the spot into y; otherwise the results go to o as float32.
template <typename TY, int VT, int CW>
__global__ __launch_bounds__(RT_THREADS * CW) __attribute__((amdgpu_waves_per_eu(VT <= 4 ? 4 : 2))) void retention_out_kernel(RetentionArgs a, TY* __restrict__ y, float* __restrict__ o_out) {
  constexpr int COLS = 16 * VT * CW, LD = COLS + 4, BR = COLS > 128 ? 16 : 32;      // BR: rows of the state, or of values, staged at a time
  static_assert(CW == 1 || CW == 2, "one or two waves share their queries");
  __shared__ __attribute__((aligned(16))) float Qs[RT_CHUNK * RT_QK_LD];
  __shared__ __attribute__((aligned(16))) float Ks[RT_CHUNK * RT_QK_LD];
  __shared__ __attribute__((aligned(16))) float Bs[BR * LD];
  const int chunk = blockIdx.x / a.col_tiles, e0 = blockIdx.x % a.col_tiles * COLS, h = blockIdx.y, r = blockIdx.z;
  const int qs = a.q_start[r], n = a.q_start[r + 1] - qs;
  if (chunk * RT_CHUNK >= n) return;
  const long t0 = qs + chunk * RT_CHUNK;
  const int len = min(RT_CHUNK, n - chunk * RT_CHUNK);
  const int lane = threadIdx.x % PI_WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / PI_WAVE) % 4, lr = lane % 16, lg = lane / 16;
  const int cw = CW == 1 ? 0 : __builtin_amdgcn_readfirstlane(threadIdx.x / RT_THREADS), w0 = cw * 16 * VT;      // the wave's first column
  __shared__ float squares[CW][RT_CHUNK];
  const float l2 = a.decay[a.H + h];
  const float* S = a.work + ((first_record(a, r) + chunk) * a.H + h) * (long)a.d * a.dv;
  const long k_col = (long)(a.H + h) * a.d, v_col = 2L * a.H * a.d + (long)h * a.dv;
  const bool live = wave * 16 < len;                 // the wave has queries
  const int i = wave * 16 + lr;                      // this lane's query
  f32x4_t o[VT], p[4];
#pragma unroll
  for (int e = 0; e < VT; ++e) o[e] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kt = 0; kt < 4; ++kt) p[kt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  // the rows of the state, then the values, BR at a time; the next ones are fetched while the present ones are used
  const int state_parts = (a.d + BR - 1) / BR;
  StagedRows<BR, COLS, RT_THREADS * CW> rows;
  auto fetch_rows = [&](int part) {
    if (part < state_parts) rows.fetch(S + (long)part * BR * a.dv, a.dv, a.d - part * BR, e0, a.dv, a.vec != 0);
    else rows.fetch(a.proj + (t0 + (part - state_parts) * BR) * a.stride + v_col, a.stride, len - (part - state_parts) * BR, e0, a.dv, a.vec != 0);
  };
  fetch_rows(0);
  int part = 0;
  for (int f0 = 0; f0 < a.d; f0 += RT_SLAB) {
    if (f0 > 0) __syncthreads();
    stage_rotated<RT_SLAB, RT_THREADS * CW>(a, Qs, t0, len, (long)h * a.d, f0, [](int) { return 1.0f; });
    stage_rotated<RT_SLAB, RT_THREADS * CW>(a, Ks, t0, len, k_col, f0, [&](int) { return a.k_scale; });
    for (int b0 = 0; b0 < RT_SLAB && f0 + b0 < a.d; b0 += BR) {
      if (b0 > 0) __syncthreads();
      rows.store(Bs);
      __syncthreads();
      fetch_rows(++part);
      if (live) {
#pragma unroll
        for (int kk = 0; kk < BR / 16; ++kk) {
          const int f = kk * 16 + lg * 4;
          const f32x4_t qf = *reinterpret_cast<const f32x4_t*>(Qs + i * RT_QK_LD + b0 + f);
#pragma unroll
          for (int kt = 0; kt < 4; ++kt) {
            if (kt > wave || (CW == 2 && (kt & 1) != cw)) continue;
            const f32x4_t kf = *reinterpret_cast<const f32x4_t*>(Ks + (kt * 16 + lr) * RT_QK_LD + b0 + f);
#pragma unroll
            for (int v = 0; v < 4; ++v) p[kt] = mfma_f32(kf[v], qf[v], p[kt]);
          }
#pragma unroll
          for (int v = 0; v < 4; ++v)
#pragma unroll
            for (int e = 0; e < VT; ++e) o[e] = mfma_f32(Bs[(f + v) * LD + w0 + e * 16 + lr], qf[v], o[e]);
        }
      }
    }
  }
  // the state's share decays from in front of the chunk to the query; a key's from the key to the query
  const float carried = power2((float)(i + 1), l2);
#pragma unroll
  for (int e = 0; e < VT; ++e) o[e] *= carried;
#pragma unroll
  for (int kt = 0; kt < 4; ++kt)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int j = kt * 16 + lg * 4 + v;
      p[kt][v] = j <= i ? p[kt][v] * power2((float)(i - j), l2) : 0.f;
    }
  if constexpr (CW == 2) {                           // each of the two waves has every second tile
    f32x4_t* const shared = reinterpret_cast<f32x4_t*>(Qs) + wave * 4 * PI_WAVE + lane;
    static_assert(sizeof(Qs) >= 4 * 4 * PI_WAVE * sizeof(f32x4_t), "the tiles of scores take the queries' place");
    __syncthreads();
#pragma unroll
    for (int kt = 0; kt < 4; ++kt)
      if ((kt & 1) == cw) shared[kt * PI_WAVE] = p[kt];
    __syncthreads();
#pragma unroll
    for (int kt = 0; kt < 4; ++kt)
      if ((kt & 1) != cw) p[kt] = shared[kt * PI_WAVE];
  }
#pragma unroll
  for (int jb = 0; jb < RT_CHUNK / BR; ++jb) {
    if (jb * BR >= len) break;
    __syncthreads();
    rows.store(Bs);
    __syncthreads();
    if ((jb + 1) * BR < len) fetch_rows(++part);
    if (!live) continue;
#pragma unroll
    for (int k2 = 0; k2 < BR / 16; ++k2) {
      const int kt = jb * (BR / 16) + k2;
      if (kt > wave) continue;
#pragma unroll
      for (int v = 0; v < 4; ++v)
#pragma unroll
        for (int e = 0; e < VT; ++e) o[e] = mfma_f32(Bs[(k2 * 16 + lg * 4 + v) * LD + w0 + e * 16 + lr], p[kt][v], o[e]);
    }
  }
  // o[e][v] is column e0 + w0 + 16 e + 4 lg + v of query i; columns beyond dv are zero
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < VT; ++e)
#pragma unroll
    for (int v = 0; v < 4; ++v) ss = fmaf(o[e][v], o[e][v], ss);
  ss = column_sum(ss);
  if constexpr (CW == 2) {
    if (lg == 0) squares[cw][i] = ss;
    __syncthreads();
    ss = squares[0][i] + squares[1][i];
  }
  if (i >= len) return;
  const long t = t0 + i;
  if (o_out) {
#pragma unroll
    for (int e = 0; e < VT; ++e)
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int col = e0 + w0 + e * 16 + lg * 4 + v;
        if (col < a.dv) o_out[(t * a.H + h) * a.dv + col] = o[e][v];
      }
    return;
  }
  const float rinv = 1.0f / sqrtf(ss / a.dv + a.eps);
  const float* gates = a.proj + t * a.stride + v_col + (long)a.H * a.dv;
  TY* yr = y + (t * a.H + h) * a.dv;
#pragma unroll
  for (int e = 0; e < VT; ++e) {
    const int col = w0 + e * 16 + lg * 4;
    if (a.vec) {
      if (col >= a.dv) continue;
      const float4 g = *reinterpret_cast<const float4*>(gates + col);
      const float w[4] = {o[e][0] * rinv * silu_full(g.x), o[e][1] * rinv * silu_full(g.y), o[e][2] * rinv * silu_full(g.z),
                          o[e][3] * rinv * silu_full(g.w)};
      if constexpr (sizeof(TY) == 2)
        *reinterpret_cast<uint2*>(yr + col) = make_uint2(f32x2_to_bf16x2_bits(w[0], w[1]), f32x2_to_bf16x2_bits(w[2], w[3]));
      else
        *reinterpret_cast<float4*>(yr + col) = make_float4(w[0], w[1], w[2], w[3]);
    } else {
#pragma unroll
      for (int v = 0; v < 4; ++v)
        if (col + v < a.dv) yr[col + v] = from_float<TY>(o[e][v] * rinv * silu_full(gates[col + v]));
    }
  }
}

// heads too wide for one block: norm and gate behind the results; one wave per (token, head)
template <typename TY>
__global__ __launch_bounds__(PI_WAVE) void retention_finish_kernel(TY* __restrict__ y, const float* __restrict__ o, const float* __restrict__ gates,
                                                                   long gate_stride, float eps, int H, int dv) {
  const long t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x;
  const float* x = o + (t * H + h) * dv;
  float ss = 0.f;
  for (int e = lane; e < dv; e += PI_WAVE) ss = fmaf(x[e], x[e], ss);
  const float rinv = 1.0f / sqrtf(wave_sum(ss) / dv + eps);
  for (int e = lane; e < dv; e += PI_WAVE) y[(t * H + h) * dv + e] = from_float<TY>(x[e] * rinv * silu_full(gates[t * gate_stride + (long)h * dv + e]));
}

#define RT_MAX_TILES 16          // value columns of one block of `out`: up to 16 tiles of 16

// Floats of scratch memory for a step of T tokens in R requests, the longest of `longest` tokens (0: single tokens, none).
extern "C" long pi_retention_work_floats(int T, int R, int longest, int H, int d, int dv) {
  if (longest <= 1) return 0;
  const long records = (long)(T / RT_CHUNK + R) * H * d * dv;
  return ((records + 3) & ~3L) + (dv > 16 * RT_MAX_TILES ? (long)T * H * dv : 0);
}

// y [T, H * dv] in y_dtype.  `proj` or `part` (pieces only in a step of single tokens, longest <= 1, in which token r is
// request r's).  decay: [2, H], the decays and their base-2 logarithms (no infinities).
extern "C" int pi_retention(void* y, int y_dtype, const float* proj, long stride, const float* part, int splits, const float* table, int rd,
                            int interleaved, const float* decay, float k_scale, float eps, const int* q_start, const int* slots, int R, int T,
                            int longest, float* state, long state_stride, int num_slots, int H, int d, int dv, float* work, long work_floats,
                            hipStream_t stream) {
  PI_REQUIRE(T >= 0 && R >= 0 && R <= 65535 && H > 0 && H <= 65535 && d > 0 && dv > 0, "retention: bad sizes T=%d R=%d heads=%d dim=%d vdim=%d", T, R, H, d, dv);
  PI_REQUIRE((proj != nullptr) != (part != nullptr) && (!part || (splits >= 1 && longest <= 1)), "retention: give the projection as a tensor, or single tokens as pieces");
  PI_REQUIRE(stride >= 2L * H * d + 2L * H * dv, "retention: rows of %ld hold no queries, keys, values and gates", stride);
  PI_REQUIRE(rd >= 0 && rd <= d && rd % 2 == 0 && (rd == 0 || table), "retention: rotation of %d features of %d", rd, d);
  PI_REQUIRE(y && decay && q_start && slots && state && num_slots > 0 && state_stride >= (long)H * d * dv, "retention: a state row of %ld floats cannot hold %d x %d x %d", state_stride, H, d, dv);
  PI_REQUIRE(y_dtype == PI_F32 || y_dtype == PI_BF16, "retention: unsupported dtype %d", y_dtype);
  PI_REQUIRE(work_floats >= pi_retention_work_floats(T, R, longest, H, d, dv), "retention: %ld floats of scratch memory are too few", work_floats);
  if (T == 0 || R == 0) return 0;
  RetentionArgs a{proj, stride, part, splits, (long)T * stride, table, rd, interleaved, decay, k_scale, eps, q_start, slots, state, state_stride,
                  num_slots, H, d, dv, 0, work, 1};
  const bool wide_state = dv % 4 == 0 && state_stride % 4 == 0 && (uintptr_t)state % 16 == 0;
  if (longest <= 1) {
    PI_REQUIRE(T == R, "retention: %d single tokens for %d requests", T, R);
    const int per = wide_state ? 4 : 1;
    int threads = 256;
    while (threads < 1024 && (long)threads * per * 8 < (long)d * dv) threads *= 2;
    const size_t lds = (size_t)(((2 * d + 3 * dv + 3) & ~3) + threads * per) * sizeof(float);
    PI_REQUIRE(lds <= 60000, "retention: heads of %d and %d features do not fit the staging memory", d, dv);
#define RT_STEP(TY, V) hipLaunchKernelGGL((retention_step_kernel<TY, V>), dim3(H, R), dim3(threads), lds, stream, a, (TY*)y)
    if (y_dtype == PI_F32) { if (per == 4) RT_STEP(float, 4); else RT_STEP(float, 1); }
    else { if (per == 4) RT_STEP(bf16_t, 4); else RT_STEP(bf16_t, 1); }
#undef RT_STEP
    return pi_check_launch("retention_step");
  }
  PI_REQUIRE(work, "retention: scratch memory is missing");
  a.vec = wide_state && d % 4 == 0 && stride % 4 == 0 && (uintptr_t)proj % 16 == 0 && (uintptr_t)work % 16 == 0 && (uintptr_t)y % 16 == 0;
  const int chunks = ceil_div(longest, RT_CHUNK);
#define RT_SUMS1(N_, W_) hipLaunchKernelGGL((retention_sums_kernel<N_, W_>), dim3(chunks * ceil_div(d, 16 * W_) * ceil_div(dv, 16 * N_), H, R), dim3(W_ * PI_WAVE), 0, stream, a)
#define RT_SUMS(N_) do { if (d <= 64) RT_SUMS1(N_, 4); else RT_SUMS1(N_, 8); } while (0)
  if (dv <= 32) RT_SUMS(2); else if (dv <= 64) RT_SUMS(4); else RT_SUMS(8);
#undef RT_SUMS
#undef RT_SUMS1
  if (pi_check_launch("retention_sums")) return -1;
  const long size = (long)d * dv;
  if (a.vec)
    hipLaunchKernelGGL((retention_states_kernel<4>), dim3(ceil_div(size, 4 * RT_THREADS), H, R), dim3(RT_THREADS), 0, stream, a);
  else
    hipLaunchKernelGGL((retention_states_kernel<1>), dim3(ceil_div(size, RT_THREADS), H, R), dim3(RT_THREADS), 0, stream, a);
  if (pi_check_launch("retention_states")) return -1;
  float* o = nullptr;
  if (dv > 16 * RT_MAX_TILES) {
    a.col_tiles = ceil_div(dv, 128);
    o = work + ((((long)(T / RT_CHUNK + R) * H * size) + 3) & ~3L);
  }
#define RT_OUT(TY, V_, C_) hipLaunchKernelGGL((retention_out_kernel<TY, V_, C_>), dim3(chunks * a.col_tiles, H, R), dim3(RT_THREADS * C_), 0, stream, a, (TY*)y, o)
#define RT_OUT_PICK(TY)                      \
  do {                                       \
    if (dv <= 32) RT_OUT(TY, 2, 1);          \
    else if (dv <= 64) RT_OUT(TY, 2, 2);     \
    else if (dv <= 128 || o) RT_OUT(TY, 4, 2); \
    else RT_OUT(TY, 8, 2);                   \
  } while (0)
  if (y_dtype == PI_F32) RT_OUT_PICK(float); else RT_OUT_PICK(bf16_t);
#undef RT_OUT_PICK
#undef RT_OUT
  if (pi_check_launch("retention_out")) return -1;
  if (o) {
    const float* gates = proj + 2L * H * d + (long)H * dv;
    if (y_dtype == PI_F32)
      hipLaunchKernelGGL(retention_finish_kernel<float>, dim3(T, H), dim3(PI_WAVE), 0, stream, (float*)y, o, gates, stride, eps, H, dv);
    else
      hipLaunchKernelGGL(retention_finish_kernel<bf16_t>, dim3(T, H), dim3(PI_WAVE), 0, stream, (bf16_t*)y, o, gates, stride, eps, H, dv);
    return pi_check_launch("retention_finish");
  }
  return 0;
}
