// Several residual streams side by side (hyper-connections), X [T, n, D] float32.  Around a sublayer:
//   u = sum_s in[s] X_s;   h = u / sqrt(mean(u^2) + eps) * w       (what the sublayer reads, in the activation type)
//   X_t <- sum_s mix[s, t] X_s + out[t] * y                        (no new stream is read while any is made)
// and, for a sublayer that also sees the token before its own,
//   h <- h + (h_before - h) * share                                (per feature; h_before: the neighbour's h, itself unshifted)
// with h_before of a request's first token of the step taken from the request's state row, which then takes the
// request's last h.
//
// One kernel does any of: the update of the streams with a sublayer's result y (a tensor, or the float32 pieces of a
// product split over k), then the next sublayer's h from the new streams.  A block holds a whole row in registers: the
// streams are read once and written once, everything is float32 until h is stored.  In a step of single tokens the token
// before is the state row's, and the shift is part of that kernel; in other steps h is left in float32 and a second
// kernel shifts it.
#include "common.h"

#define HS_MAX_THREADS 1024     // a block whose threads hold one group each
#define HS_THREADS 512          // ... or several
#define HS_MAX_STREAMS 16

struct HyperArgs {
  float* x;               // [T, n, D]
  int n, D, T;
  // the update (POST)
  const float* y;         // [T, D], or null: the pieces
  const float* part;      // [splits, T, D]
  int splits;
  const float* post;      // out [n], then mix [n, n] (from, to)
  int write_x;
  // what the next sublayer reads (h null: nothing)
  void* h;
  int h_bf16;
  const float* in;        // [n]
  const float* w;         // [D]
  float eps;
  const int* rows;        // the rows to make h of (null: all)
  // the token before (SHIFT)
  const float* share;     // [D]
  float* state;           // [slots, >= D]
  long state_stride;
  int num_slots;
  const int* slots;
  const int* req_of_token;
};

template <int V> struct Lanes { float v[V]; };
template <int V> __device__ inline Lanes<V> load_lanes(const float* p);
template <> __device__ inline Lanes<4> load_lanes<4>(const float* p) {
  const float4 t = *reinterpret_cast<const float4*>(p);
  return Lanes<4>{{t.x, t.y, t.z, t.w}};
}
template <> __device__ inline Lanes<1> load_lanes<1>(const float* p) { return Lanes<1>{{*p}}; }
template <int V> __device__ inline void store_lanes(float* p, const Lanes<V>& l);
template <> __device__ inline void store_lanes<4>(float* p, const Lanes<4>& l) { *reinterpret_cast<float4*>(p) = make_float4(l.v[0], l.v[1], l.v[2], l.v[3]); }
template <> __device__ inline void store_lanes<1>(float* p, const Lanes<1>& l) { *p = l.v[0]; }
template <int V> __device__ inline void store_lanes(bf16_t* p, const Lanes<V>& l);
template <> __device__ inline void store_lanes<4>(bf16_t* p, const Lanes<4>& l) {
  *reinterpret_cast<uint2*>(p) = make_uint2(f32x2_to_bf16x2_bits(l.v[0], l.v[1]), f32x2_to_bf16x2_bits(l.v[2], l.v[3]));
}
template <> __device__ inline void store_lanes<1>(bf16_t* p, const Lanes<1>& l) { *p = from_float<bf16_t>(l.v[0]); }

// Row `row` of the streams: updated with y and written back (POST), then summed into u and normalised into h.
// S is the number of streams, or the most there may be (FIT false: a.n says how many there are).
template <int S, int V, int VPT, bool POST, bool FIT>
__device__ inline void hyper_row(const HyperArgs& a, long row, Lanes<V> (&h)[VPT], float* scratch) {
  const int n = FIT ? S : a.n, D = a.D, groups = D / V;
  Lanes<V> x[S][VPT];
  float* xr = a.x + row * n * D;
#pragma unroll
  for (int s = 0; s < S; ++s)
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
      const int g = threadIdx.x + k * blockDim.x;
      if (g < groups && s < n) x[s][k] = load_lanes<V>(xr + (long)s * D + g * V);
      else
#pragma unroll
        for (int e = 0; e < V; ++e) x[s][k].v[e] = 0.f;
    }
  if (POST) {
    Lanes<V> y[VPT];
#pragma unroll
    for (int k = 0; k < VPT; ++k)
#pragma unroll
      for (int e = 0; e < V; ++e) y[k].v[e] = 0.f;
    if (a.y) {
#pragma unroll
      for (int k = 0; k < VPT; ++k) {
        const int g = threadIdx.x + k * blockDim.x;
        if (g < groups) y[k] = load_lanes<V>(a.y + row * D + g * V);
      }
    } else {
      // several pieces' loads go out together, the adds keep the split order
      constexpr int U = VPT <= 2 ? 8 : 2;
      const long plane = (long)a.T * D;
      for (int s0 = 0; s0 < a.splits; s0 += U) {
        Lanes<V> t[U][VPT];
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int k = 0; k < VPT; ++k) {
            const int g = threadIdx.x + k * blockDim.x;
            if (s0 + u < a.splits && g < groups) t[u][k] = load_lanes<V>(a.part + (s0 + u) * plane + row * D + g * V);
            else
#pragma unroll
              for (int e = 0; e < V; ++e) t[u][k].v[e] = 0.f;
          }
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int k = 0; k < VPT; ++k)
#pragma unroll
            for (int e = 0; e < V; ++e) y[k].v[e] += t[u][k].v[e];
      }
    }
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
      Lanes<V> z[S];
#pragma unroll
      for (int t = 0; t < S; ++t) {
        if (t >= n) continue;
        const float o = a.post[t];
#pragma unroll
        for (int e = 0; e < V; ++e) z[t].v[e] = o * y[k].v[e];
#pragma unroll
        for (int s = 0; s < S; ++s) {
          if (s >= n) continue;
          const float m = a.post[n + s * n + t];
#pragma unroll
          for (int e = 0; e < V; ++e) z[t].v[e] = fmaf(m, x[s][k].v[e], z[t].v[e]);
        }
      }
      const int g = threadIdx.x + k * blockDim.x;
#pragma unroll
      for (int t = 0; t < S; ++t) {
        if (t >= n) continue;
        x[t][k] = z[t];
        if (a.write_x && g < groups) store_lanes<V>(xr + (long)t * D + g * V, z[t]);
      }
    }
  }
  if (!a.h) return;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
#pragma unroll
    for (int e = 0; e < V; ++e) h[k].v[e] = 0.f;
#pragma unroll
    for (int s = 0; s < S; ++s) {
      if (s >= n) continue;
      const float c = a.in[s];
#pragma unroll
      for (int e = 0; e < V; ++e) h[k].v[e] = fmaf(c, x[s][k].v[e], h[k].v[e]);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(h[k].v[e], h[k].v[e], ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)D + a.eps);
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int g = threadIdx.x + k * blockDim.x;
    if (g >= groups) continue;
    const Lanes<V> w = load_lanes<V>(a.w + g * V);
#pragma unroll
    for (int e = 0; e < V; ++e) h[k].v[e] = w.v[e] * (h[k].v[e] * inv);
  }
}

__device__ inline float shifted(float h, float before, float share) { return fmaf(before - h, share, h); }

template <int V, int VPT>
__device__ inline void store_h(const HyperArgs& a, long row, const Lanes<V> (&h)[VPT]) {
  const int groups = a.D / V;
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int g = threadIdx.x + k * blockDim.x;
    if (g >= groups) continue;
    if (a.h_bf16) store_lanes<V>(reinterpret_cast<bf16_t*>(a.h) + row * a.D + g * V, h[k]);
    else store_lanes<V>(reinterpret_cast<float*>(a.h) + row * a.D + g * V, h[k]);
  }
}

template <int S, int V, int VPT, bool POST, bool SHIFT, bool FIT>
__global__ __launch_bounds__(VPT == 1 ? HS_MAX_THREADS : HS_THREADS) void hyper_streams_kernel(HyperArgs a) {
  __shared__ float scratch[16];
  [[maybe_unused]] const int groups = a.D / V;
  if (!SHIFT) {
    const long m = blockIdx.x;
    const long r = a.rows ? a.rows[m] : m;
    Lanes<V> h[VPT];
    hyper_row<S, V, VPT, POST, FIT>(a, r, h, scratch);
    if (a.h) store_h<V, VPT>(a, m, h);
    return;
  }
  const int t = blockIdx.x, slot = a.slots[a.req_of_token[t]];
  const bool has_state = slot >= 0 && slot < a.num_slots;
  float* st = a.state + (long)slot * a.state_stride;
  Lanes<V> before[VPT], cur[VPT], share[VPT];
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int g = threadIdx.x + k * blockDim.x;
    if (g < groups) share[k] = load_lanes<V>(a.share + g * V);
    if (g < groups && has_state) before[k] = load_lanes<V>(st + g * V);
    else
#pragma unroll
      for (int e = 0; e < V; ++e) before[k].v[e] = 0.f;
  }
  hyper_row<S, V, VPT, POST, FIT>(a, t, cur, scratch);
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int g = threadIdx.x + k * blockDim.x;
    if (g >= groups) continue;
    if (has_state) store_lanes<V>(st + g * V, cur[k]);
#pragma unroll
    for (int e = 0; e < V; ++e) cur[k].v[e] = shifted(cur[k].v[e], before[k].v[e], share[k].v[e]);
  }
  store_h<V, VPT>(a, t, cur);
}

template <int S, int V, int VPT, bool FIT>
static int launch_hyper(const HyperArgs& a, int blocks, int threads, bool post, bool shift, hipStream_t stream) {
  if (post && shift) hipLaunchKernelGGL((hyper_streams_kernel<S, V, VPT, true, true, FIT>), dim3(blocks), dim3(threads), 0, stream, a);
  else if (post) hipLaunchKernelGGL((hyper_streams_kernel<S, V, VPT, true, false, FIT>), dim3(blocks), dim3(threads), 0, stream, a);
  else if (shift) hipLaunchKernelGGL((hyper_streams_kernel<S, V, VPT, false, true, FIT>), dim3(blocks), dim3(threads), 0, stream, a);
  else hipLaunchKernelGGL((hyper_streams_kernel<S, V, VPT, false, false, FIT>), dim3(blocks), dim3(threads), 0, stream, a);
  return pi_check_launch("hyper_streams");
}

// y or part: the sublayer's result to add (both null: no update).  h null: no next sublayer.  share null: no shift.
// M: rows of h (with `rows`; else M == T).  single: every request of the step holds one token (a shift is for such steps).
extern "C" int pi_hyper_streams(float* x, int n, int D, int T, const float* y, const float* part, int splits, const float* post, int write_x,
                                void* h, int h_dtype, const float* in, const float* w, float eps, const int* rows, int M, const float* share,
                                float* state, long state_stride, int num_slots, const int* slots, const int* req_of_token,
                                int single, hipStream_t stream) {
  PI_REQUIRE(x && n > 0 && n <= HS_MAX_STREAMS && D > 0 && T >= 0 && M >= 0, "hyper streams: bad sizes streams=%d D=%d T=%d", n, D, T);
  const bool has_post = y || part, shift = share != nullptr;
  PI_REQUIRE(has_post || h, "hyper streams: nothing to do");
  PI_REQUIRE(!has_post || (post && !(y && part) && (!part || splits >= 1)), "hyper streams: bad description of the sublayer's result");
  PI_REQUIRE(!h || (in && w && (h_dtype == PI_F32 || h_dtype == PI_BF16)), "hyper streams: bad description of the next sublayer");
  PI_REQUIRE(!shift || (h && !rows && state && slots && req_of_token && state_stride >= D), "hyper streams: bad description of the shift");
  PI_REQUIRE(!shift || single, "hyper streams: the shift in the same kernel is for steps of single tokens");
  PI_REQUIRE(rows || M == T, "hyper streams: %d rows of %d", M, T);
  PI_REQUIRE(!rows || !write_x, "hyper streams: chosen rows are read, not written");
  if (M == 0 || T == 0) return 0;
  HyperArgs a{x, n, D, T, y, part, splits, post, has_post ? write_x : 0, h, h_dtype == PI_BF16, in, w, eps, rows, share, state, state_stride,
              num_slots, slots, req_of_token};
  bool wide = D % 4 == 0 && state_stride % 4 == 0;
  for (const void* p : {(const void*)x, (const void*)y, (const void*)part, (const void*)h, (const void*)w, (const void*)share, (const void*)state})
    wide = wide && (uintptr_t)p % 16 == 0;
  const int groups = wide ? D / 4 : D;
  // a thread per 16-byte group as far as a block goes (measured at 2,048 rows of 2,048 x 4: 27 us, two groups per thread 30)
  int threads = ((groups + PI_WAVE - 1) / PI_WAVE) * PI_WAVE;
  if (threads > (wide ? HS_MAX_THREADS : HS_THREADS)) threads = HS_THREADS;
  const int vpt = (groups + threads - 1) / threads;
  PI_REQUIRE(vpt <= 8 && (n <= 4 || !wide || vpt <= 4), "hyper streams: rows of %d features in %d streams are too wide", D, n);
#define HS_GO(S_, V_, N_, F_) return launch_hyper<S_, V_, N_, F_>(a, M, threads, has_post, shift, stream)
  if (!wide) HS_GO(HS_MAX_STREAMS, 1, 8, false);
#define HS_PICK(S_)               \
  do {                            \
    if (vpt <= 1) HS_GO(S_, 4, 1, true); \
    if (vpt <= 2) HS_GO(S_, 4, 2, true); \
    if (vpt <= 4) HS_GO(S_, 4, 4, true); \
    HS_GO(S_, 4, 8, true);        \
  } while (0)
  switch (n) {
    case 1: HS_PICK(1);
    case 2: HS_PICK(2);
    case 3: HS_PICK(3);
    case 4: HS_PICK(4);
  }
  if (n <= 8) {
    if (vpt <= 1) HS_GO(8, 4, 1, false);
    if (vpt <= 2) HS_GO(8, 4, 2, false);
    HS_GO(8, 4, 4, false);
  }
  if (vpt <= 1) HS_GO(16, 4, 1, false);
  if (vpt <= 2) HS_GO(16, 4, 2, false);
  HS_GO(16, 4, 4, false);
#undef HS_PICK
#undef HS_GO
}

// ---------------------------------------------------------------- the shift on its own, any number of tokens per request
// out[t] = h[t] + (h of the request's token before - h[t]) * share.  The first token's predecessor is the request's
// state row, which then takes the request's last h: read and written by the threads of the first token only.
template <typename TO, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(TO* __restrict__ out, const float* __restrict__ h, const float* __restrict__ share,
                                                          float* __restrict__ state, long state_stride, int num_slots,
                                                          const int* __restrict__ q_start, const int* __restrict__ slots,
                                                          const int* __restrict__ req_of_token, int D) {
  const long t = blockIdx.x;
  const int d = (blockIdx.y * 256 + threadIdx.x) * V;
  if (d >= D) return;
  const int r = req_of_token[t];
  const Lanes<V> cur = load_lanes<V>(h + t * D + d), w = load_lanes<V>(share + d);
  Lanes<V> before;
  if (t == q_start[r]) {
    const int slot = slots[r];
    const bool has_state = slot >= 0 && slot < num_slots;
    float* st = state + (long)slot * state_stride + d;
    if (has_state) {
      before = load_lanes<V>(st);
      store_lanes<V>(st, load_lanes<V>(h + (long)(q_start[r + 1] - 1) * D + d));
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) before.v[e] = 0.f;
    }
  } else {
    before = load_lanes<V>(h + (t - 1) * D + d);
  }
  Lanes<V> o;
#pragma unroll
  for (int e = 0; e < V; ++e) o.v[e] = shifted(cur.v[e], before.v[e], w.v[e]);
  store_lanes<V>(out + t * D + d, o);
}

extern "C" int pi_token_shift(void* out, int out_dtype, const float* h, const float* share, float* state, long state_stride, int num_slots,
                              const int* q_start, const int* slots, const int* req_of_token, int T, int D, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && D > 0 && out && h && share && state && state_stride >= D && q_start && slots && req_of_token && out != (const void*)h,
             "token shift: bad arguments T=%d D=%d", T, D);
  PI_REQUIRE(out_dtype == PI_F32 || out_dtype == PI_BF16, "token shift: unsupported dtype %d", out_dtype);
  if (T == 0) return 0;
  bool wide = D % 4 == 0 && state_stride % 4 == 0;
  for (const void* p : {(const void*)out, (const void*)h, (const void*)share, (const void*)state}) wide = wide && (uintptr_t)p % 16 == 0;
  const int per_block = 256 * (wide ? 4 : 1);
  PI_REQUIRE((D + per_block - 1) / per_block <= 65535, "token shift: rows of %d features are too wide", D);
  const dim3 grid(T, (D + per_block - 1) / per_block), block(256);
#define TS_GO(TO, V_) hipLaunchKernelGGL((token_shift_kernel<TO, V_>), grid, block, 0, stream, (TO*)out, h, share, state, state_stride, num_slots, q_start, slots, req_of_token, D)
  if (out_dtype == PI_F32) { if (wide) TS_GO(float, 4); else TS_GO(float, 1); }
  else { if (wide) TS_GO(bf16_t, 4); else TS_GO(bf16_t, 1); }
#undef TS_GO
  return pi_check_launch("token_shift");
}
