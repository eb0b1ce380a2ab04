// Kernels around a residual stream whose sublayers are normalised on the way OUT:
//   x <- x + mult * norm(y; w),   y = a                               (one branch)
//                                 y = (norm(a; wa) + norm(b; wb)) / 2 (two branches side by side)
// with norm(v; w) = v / sqrt(mean(v^2) + eps) * w.  One block per token row does the branch
// norms, their mean, the outer norm, the scaled add into the float32 stream and, when asked,
// the copy of the new stream in the activation type that the next sublayer's products read.
// Sums of squares, roots and the stream are float32 throughout.  Weights are float32 (a weight
// stored around zero is handed over as 1 + w).
#include "common.h"

template <typename TH>
__global__ __launch_bounds__(256) void branch_norm_add_kernel(float* __restrict__ x, TH* __restrict__ h, const float* __restrict__ a,
                                                              const float* __restrict__ wa, const float* __restrict__ b,
                                                              const float* __restrict__ wb, const float* __restrict__ wo,
                                                              float eps, float mult, int D) {
  extern __shared__ float y[];          // D floats
  __shared__ float scratch[16];
  const long row = blockIdx.x;
  const float* ar = a + row * D;
  const float* br = b ? b + row * D : nullptr;
  float sa = 0.f, sb = 0.f;
  for (int d = threadIdx.x; d < D; d += blockDim.x) {
    const float va = ar[d];
    sa = fmaf(va, va, sa);
    if (br) {
      const float vb = br[d];
      sb = fmaf(vb, vb, sb);
    }
  }
  float sy = 0.f;
  if (wa) {
    const float ra = 1.0f / sqrtf(block_sum(sa, scratch) / D + eps);
    const float rb = br ? 1.0f / sqrtf(block_sum(sb, scratch) / D + eps) : 0.f;
    for (int d = threadIdx.x; d < D; d += blockDim.x) {
      float v = ar[d] * ra * wa[d];
      if (br) v = 0.5f * (v + br[d] * rb * wb[d]);
      y[d] = v;
      sy = fmaf(v, v, sy);
    }
  } else {
    for (int d = threadIdx.x; d < D; d += blockDim.x) y[d] = ar[d];
    sy = sa;
  }
  const float ry = 1.0f / sqrtf(block_sum(sy, scratch) / D + eps);
  float* xr = x + row * D;
  for (int d = threadIdx.x; d < D; d += blockDim.x) {
    const float v = xr[d] + mult * (y[d] * ry * wo[d]);
    xr[d] = v;
    if (h) h[row * D + d] = from_float<TH>(v);
  }
}

// The same for rows of whole 16-byte groups, at most VPT groups per thread: a thread keeps its
// values in registers between the passes, both branches' sums of squares share one reduction,
// and every access is 16 bytes wide.  Few rows (decode steps) are a matter of latency: as many
// threads per row as the row has groups.
template <typename TH, int VPT>
__global__ __launch_bounds__(1024) void branch_norm_add_wide_kernel(float* __restrict__ x, TH* __restrict__ h, const float* __restrict__ a,
                                                                    const float* __restrict__ wa, const float* __restrict__ b,
                                                                    const float* __restrict__ wb, const float* __restrict__ wo,
                                                                    float eps, float mult, int D) {
  __shared__ float scratch[32];
  const long row = blockIdx.x;
  const int groups = D / 4;
  float4 va[VPT], vb[VPT], xo[VPT];
  float sa = 0.f, sb = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int g = threadIdx.x + v * blockDim.x;
    const bool in = g < groups;
    va[v] = in ? reinterpret_cast<const float4*>(a + row * D)[g] : make_float4(0.f, 0.f, 0.f, 0.f);
    vb[v] = (in && b) ? reinterpret_cast<const float4*>(b + row * D)[g] : make_float4(0.f, 0.f, 0.f, 0.f);
    xo[v] = in ? reinterpret_cast<const float4*>(x + row * D)[g] : make_float4(0.f, 0.f, 0.f, 0.f);
    sa = fmaf(va[v].x, va[v].x, sa); sa = fmaf(va[v].y, va[v].y, sa); sa = fmaf(va[v].z, va[v].z, sa); sa = fmaf(va[v].w, va[v].w, sa);
    sb = fmaf(vb[v].x, vb[v].x, sb); sb = fmaf(vb[v].y, vb[v].y, sb); sb = fmaf(vb[v].z, vb[v].z, sb); sb = fmaf(vb[v].w, vb[v].w, sb);
  }
  float sy = sa, unused = 0.f;
  if (wa) {
    block_sum2(sa, sb, scratch);
    const float ra = 1.0f / sqrtf(sa / D + eps);
    const float rb = b ? 1.0f / sqrtf(sb / D + eps) : 0.f;
    sy = 0.f;
#pragma unroll
    for (int v = 0; v < VPT; ++v) {
      const int g = threadIdx.x + v * blockDim.x;
      if (g >= groups) continue;
      const float4 w1 = reinterpret_cast<const float4*>(wa)[g];
      float y[4] = {va[v].x * ra * w1.x, va[v].y * ra * w1.y, va[v].z * ra * w1.z, va[v].w * ra * w1.w};
      if (b) {
        const float4 w2 = reinterpret_cast<const float4*>(wb)[g];
        y[0] = 0.5f * (y[0] + vb[v].x * rb * w2.x);
        y[1] = 0.5f * (y[1] + vb[v].y * rb * w2.y);
        y[2] = 0.5f * (y[2] + vb[v].z * rb * w2.z);
        y[3] = 0.5f * (y[3] + vb[v].w * rb * w2.w);
      }
      va[v] = make_float4(y[0], y[1], y[2], y[3]);
      sy = fmaf(y[0], y[0], sy); sy = fmaf(y[1], y[1], sy); sy = fmaf(y[2], y[2], sy); sy = fmaf(y[3], y[3], sy);
    }
  }
  block_sum2(sy, unused, scratch);
  const float ry = 1.0f / sqrtf(sy / D + eps);
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int g = threadIdx.x + v * blockDim.x;
    if (g >= groups) continue;
    const float4 w3 = reinterpret_cast<const float4*>(wo)[g];
    const float4 r = make_float4(xo[v].x + mult * (va[v].x * ry * w3.x), xo[v].y + mult * (va[v].y * ry * w3.y),
                                 xo[v].z + mult * (va[v].z * ry * w3.z), xo[v].w + mult * (va[v].w * ry * w3.w));
    reinterpret_cast<float4*>(x + row * D)[g] = r;
    if (h) {
      TH* hp = h + row * D + 4 * (long)g;
      hp[0] = from_float<TH>(r.x); hp[1] = from_float<TH>(r.y); hp[2] = from_float<TH>(r.z); hp[3] = from_float<TH>(r.w);
    }
  }
}

// x (float32 stream) += mult * norm(...); h (optional, h_dtype) = the new stream.
// wa == null: a is taken as it is (one branch, no inner norm); b == null: one branch.
extern "C" int pi_branch_norm_add(float* x, void* h, int h_dtype, const float* a, const float* wa, const float* b,
                                  const float* wb, const float* wo, float eps, float mult, int T, int D, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && D > 0 && D <= 40000, "branch norm: bad sizes T=%d D=%d", T, D);
  PI_REQUIRE(x && a && wo, "branch norm: the stream, a branch and the outer weight are needed");
  PI_REQUIRE(!b || (wa && wb), "branch norm: two branches need both their weights");
  if (T == 0) return 0;
  PI_REQUIRE(!h || h_dtype == PI_BF16 || h_dtype == PI_F32, "branch norm: unsupported activation dtype %d", h_dtype);
  const bool aligned = D % 4 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)a % 16 == 0 && (!b || (uintptr_t)b % 16 == 0) &&
                       (uintptr_t)wo % 16 == 0 && (!wa || (uintptr_t)wa % 16 == 0) && (!wb || (uintptr_t)wb % 16 == 0);
  if (aligned && D / 4 <= 4 * 1024) {
    const int groups = D / 4;
    // few rows: a thread per group (latency); many rows: fewer, fatter threads
    int threads = T <= 512 ? groups : (groups + 3) / 4;
    threads = threads > 1024 ? 1024 : ((threads + PI_WAVE - 1) / PI_WAVE) * PI_WAVE;
    const int vpt = (groups + threads - 1) / threads;
#define BN_GO(TH, V) hipLaunchKernelGGL((branch_norm_add_wide_kernel<TH, V>), dim3(T), dim3(threads), 0, stream, x, (TH*)h, a, wa, b, wb, wo, eps, mult, D)
#define BN_PICK(TH)            \
  do {                         \
    if (vpt <= 1) BN_GO(TH, 1); \
    else if (vpt <= 2) BN_GO(TH, 2); \
    else BN_GO(TH, 4);         \
  } while (0)
    if (h && h_dtype == PI_BF16) BN_PICK(bf16_t);
    else BN_PICK(float);
#undef BN_PICK
#undef BN_GO
    return pi_check_launch("branch_norm_add_wide");
  }
  const size_t lds = (size_t)D * sizeof(float);
  if (h && h_dtype == PI_BF16)
    hipLaunchKernelGGL(branch_norm_add_kernel<bf16_t>, dim3(T), dim3(256), lds, stream, x, (bf16_t*)h, a, wa, b, wb, wo, eps, mult, D);
  else if (!h || h_dtype == PI_F32)
    hipLaunchKernelGGL(branch_norm_add_kernel<float>, dim3(T), dim3(256), lds, stream, x, (float*)h, a, wa, b, wb, wo, eps, mult, D);
  else
    return pi_fail("branch norm: unsupported activation dtype %d", h_dtype);
  return pi_check_launch("branch_norm_add");
}

// ---------------------------------------------------------------- layer norm with weight and bias
// LN(v; w, b) = (v - mean) / sqrt(mean of squared deviations + eps) * w + b, all float32.  The row sits in
// LDS between the passes: the mean first, then the deviations' squares, so that nothing is cancelled.
__device__ inline void layer_norm_stats(const float* row, int D, float eps, float* scratch, float& mean, float& rinv) {
  float s = 0.f;
  for (int d = threadIdx.x; d < D; d += blockDim.x) s += row[d];
  mean = block_sum(s, scratch) / D;
  float q = 0.f;
  for (int d = threadIdx.x; d < D; d += blockDim.x) {
    const float dev = row[d] - mean;
    q = fmaf(dev, dev, q);
  }
  rinv = 1.0f / sqrtf(block_sum(q, scratch) / D + eps);
}

// out[m, :] = LN(x[rows[m] or m, :]; w, b) in the activation type
template <typename TO>
__global__ __launch_bounds__(256) void layer_norm_kernel(TO* __restrict__ out, const float* __restrict__ x, const int* __restrict__ rows,
                                                         const float* __restrict__ w, const float* __restrict__ b, float eps, int D,
                                                         int x_rows) {
  extern __shared__ float row[];
  __shared__ float scratch[16];
  const long m = blockIdx.x;
  const long r = rows ? rows[m] : m;
  const bool ok = r >= 0 && r < x_rows;          // a row outside the stream gives NaN, no fault
  for (int d = threadIdx.x; d < D; d += blockDim.x) row[d] = ok ? x[r * D + d] : NAN;
  __syncthreads();
  float mean, rinv;
  layer_norm_stats(row, D, eps, scratch, mean, rinv);
  for (int d = threadIdx.x; d < D; d += blockDim.x) out[m * D + d] = from_float<TO>((row[d] - mean) * rinv * w[d] + b[d]);
}

// The same for rows of whole 16-byte groups, at most VPT groups per thread: a thread keeps its values in registers
// between the passes and every access is 16 bytes wide.  Few rows (decode steps) are a matter of latency: as many
// threads per row as the row has groups.
__device__ inline float sum4(const float4& v) { return (v.x + v.y) + (v.z + v.w); }
__device__ inline float4 sub4(const float4& v, float m) { return make_float4(v.x - m, v.y - m, v.z - m, v.w - m); }
__device__ inline float dot4(const float4& v) { return fmaf(v.w, v.w, fmaf(v.z, v.z, fmaf(v.y, v.y, v.x * v.x))); }
__device__ inline float4 affine4(const float4& d, float r, const float4& w, const float4& b) {
  return make_float4(fmaf(d.x * r, w.x, b.x), fmaf(d.y * r, w.y, b.y), fmaf(d.z * r, w.z, b.z), fmaf(d.w * r, w.w, b.w));
}
template <typename TO> __device__ inline void store4(TO* p, const float4& v);
template <> __device__ inline void store4<float>(float* p, const float4& v) { *reinterpret_cast<float4*>(p) = v; }
template <> __device__ inline void store4<bf16_t>(bf16_t* p, const float4& v) {
  *reinterpret_cast<uint2*>(p) = make_uint2(f32x2_to_bf16x2_bits(v.x, v.y), f32x2_to_bf16x2_bits(v.z, v.w));
}

// mean and 1 / sqrt(variance + eps) of a row whose groups sit in v[VPT] (groups beyond the row are zero and not counted);
// v becomes the deviations from the mean
template <int VPT>
__device__ inline float centre_and_scale(float4 (&v)[VPT], int groups, int D, float eps, float* scratch) {
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) s += sum4(v[i]);
  const float mean = block_sum(s, scratch) / D;
  float q = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const bool in = (int)(threadIdx.x + i * blockDim.x) < groups;
    v[i] = in ? sub4(v[i], mean) : make_float4(0.f, 0.f, 0.f, 0.f);
    q += dot4(v[i]);
  }
  return 1.0f / sqrtf(block_sum(q, scratch) / D + eps);
}

template <typename TO, int VPT>
__global__ __launch_bounds__(1024) void layer_norm_wide_kernel(TO* __restrict__ out, const float* __restrict__ x, const int* __restrict__ rows,
                                                               const float* __restrict__ w, const float* __restrict__ b, float eps, int D,
                                                               int x_rows) {
  __shared__ float scratch[16];
  const long m = blockIdx.x;
  const long r = rows ? rows[m] : m;
  const bool ok = r >= 0 && r < x_rows;
  const int groups = D / 4;
  float4 v[VPT], wv[VPT], bv[VPT];
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int g = threadIdx.x + i * blockDim.x;
    const bool in = g < groups;
    v[i] = !in ? make_float4(0.f, 0.f, 0.f, 0.f) : ok ? reinterpret_cast<const float4*>(x + r * D)[g] : make_float4(NAN, NAN, NAN, NAN);
    wv[i] = in ? reinterpret_cast<const float4*>(w)[g] : make_float4(0.f, 0.f, 0.f, 0.f);
    bv[i] = in ? reinterpret_cast<const float4*>(b)[g] : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const float rinv = centre_and_scale<VPT>(v, groups, D, eps, scratch);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int g = threadIdx.x + i * blockDim.x;
    if (g < groups) store4<TO>(out + m * D + 4 * (long)g, affine4(v[i], rinv, wv[i], bv[i]));
  }
}

// threads per row and groups per thread for the wide kernels: few rows, a thread per group (latency); many rows, fewer, fatter threads
static inline bool wide_row_shape(int T, int D, int& threads, int& vpt) {
  if (D % 4) return false;
  const int groups = D / 4;
  threads = T <= 512 ? groups : (groups + 3) / 4;
  threads = threads > 1024 ? 1024 : ((threads + PI_WAVE - 1) / PI_WAVE) * PI_WAVE;
  vpt = (groups + threads - 1) / threads;
  return vpt <= 4;
}

extern "C" int pi_layer_norm(void* out, int out_dtype, const float* x, const int* rows, const float* w, const float* b, float eps,
                             int M, int D, int x_rows, hipStream_t stream) {
  PI_REQUIRE(M >= 0 && D > 0 && D <= 16000 && x_rows >= 0, "layer norm: bad sizes M=%d D=%d", M, D);
  PI_REQUIRE(out && x && w && b, "layer norm: output, input, weight and bias are needed");
  PI_REQUIRE(out_dtype == PI_F32 || out_dtype == PI_BF16, "layer norm: unsupported dtype %d", out_dtype);
  if (M == 0) return 0;
  int wide_threads = 0, vpt = 0;
  const bool aligned = (uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)b % 16 == 0 && (uintptr_t)out % 16 == 0;
  if (aligned && wide_row_shape(M, D, wide_threads, vpt)) {
#define LN_GO(TO, V) hipLaunchKernelGGL((layer_norm_wide_kernel<TO, V>), dim3(M), dim3(wide_threads), 0, stream, (TO*)out, x, rows, w, b, eps, D, x_rows)
#define LN_PICK(TO) do { if (vpt <= 1) LN_GO(TO, 1); else if (vpt <= 2) LN_GO(TO, 2); else LN_GO(TO, 4); } while (0)
    if (out_dtype == PI_F32) LN_PICK(float); else LN_PICK(bf16_t);
#undef LN_PICK
#undef LN_GO
    return pi_check_launch("layer_norm_wide");
  }
  const int threads = D >= 1024 ? 256 : (D >= 256 ? 128 : 64);
  const size_t lds = (size_t)D * sizeof(float);
  if (out_dtype == PI_F32)
    hipLaunchKernelGGL(layer_norm_kernel<float>, dim3(M), dim3(threads), lds, stream, (float*)out, x, rows, w, b, eps, D, x_rows);
  else
    hipLaunchKernelGGL(layer_norm_kernel<bf16_t>, dim3(M), dim3(threads), lds, stream, (bf16_t*)out, x, rows, w, b, eps, D, x_rows);
  return pi_check_launch("layer_norm");
}

// A sublayer's result joins the stream through a layer norm, and the next sublayer's input is made on the way:
//   y = a (+ a_bias)                                                      (one branch)
//   y = (rms(a (+ a_bias); wa) + rms(b; wb)) / 2                           (two branches side by side)
//   x <- x + LN(y; pw, pb);   h = LN(x; nw, nb)   (nw null: no h)
// with rms(v; w) = v / sqrt(mean(v^2) + eps) * w.  One block per token; the row stays in LDS throughout.
template <typename TH>
__global__ __launch_bounds__(256) void sandwich_norm_add_kernel(float* __restrict__ x, TH* __restrict__ h, const float* __restrict__ a,
                                                                const float* __restrict__ a_bias, const float* __restrict__ wa,
                                                                const float* __restrict__ b, const float* __restrict__ wb,
                                                                const float* __restrict__ pw, const float* __restrict__ pb,
                                                                const float* __restrict__ nw, const float* __restrict__ nb, float eps,
                                                                int D) {
  extern __shared__ float row[];
  __shared__ float scratch[32];
  const long t = blockIdx.x;
  const float* ar = a + t * D;
  const float* br = b ? b + t * D : nullptr;
  if (wa) {
    float sa = 0.f, sb = 0.f;
    for (int d = threadIdx.x; d < D; d += blockDim.x) {
      const float va = ar[d] + (a_bias ? a_bias[d] : 0.f);
      row[d] = va;
      sa = fmaf(va, va, sa);
      if (br) {
        const float vb = br[d];
        sb = fmaf(vb, vb, sb);
      }
    }
    block_sum2(sa, sb, scratch);
    const float ra = 1.0f / sqrtf(sa / D + eps), rb = br ? 1.0f / sqrtf(sb / D + eps) : 0.f;
    for (int d = threadIdx.x; d < D; d += blockDim.x) {
      float v = row[d] * ra * wa[d];
      if (br) v = 0.5f * (v + br[d] * rb * wb[d]);
      row[d] = v;
    }
  } else {
    for (int d = threadIdx.x; d < D; d += blockDim.x) row[d] = ar[d] + (a_bias ? a_bias[d] : 0.f);
  }
  __syncthreads();
  float mean, rinv;
  layer_norm_stats(row, D, eps, scratch, mean, rinv);
  float* xr = x + t * D;
  for (int d = threadIdx.x; d < D; d += blockDim.x) {
    const float v = xr[d] + ((row[d] - mean) * rinv * pw[d] + pb[d]);
    xr[d] = v;
    row[d] = v;
  }
  if (!nw) return;
  __syncthreads();
  layer_norm_stats(row, D, eps, scratch, mean, rinv);
  for (int d = threadIdx.x; d < D; d += blockDim.x) h[t * D + d] = from_float<TH>((row[d] - mean) * rinv * nw[d] + nb[d]);
}

// The same with the row in registers and 16-byte accesses (see layer_norm_wide_kernel).
template <typename TH, int VPT>
__global__ __launch_bounds__(1024) void sandwich_norm_add_wide_kernel(float* __restrict__ x, TH* __restrict__ h, const float* __restrict__ a,
                                                                      const float* __restrict__ a_bias, const float* __restrict__ wa,
                                                                      const float* __restrict__ b, const float* __restrict__ wb,
                                                                      const float* __restrict__ pw, const float* __restrict__ pb,
                                                                      const float* __restrict__ nw, const float* __restrict__ nb,
                                                                      float eps, int D) {
  __shared__ float scratch[32];
  const long t = blockIdx.x;
  const int groups = D / 4;
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 y[VPT], xo[VPT];
  float sa = 0.f, sb = 0.f;
  {
    float4 vb[VPT];
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int g = threadIdx.x + i * blockDim.x;
      const bool in = g < groups;
      y[i] = in ? reinterpret_cast<const float4*>(a + t * D)[g] : zero;
      if (in && a_bias) {
        const float4 ab = reinterpret_cast<const float4*>(a_bias)[g];
        y[i] = make_float4(y[i].x + ab.x, y[i].y + ab.y, y[i].z + ab.z, y[i].w + ab.w);
      }
      vb[i] = (in && b) ? reinterpret_cast<const float4*>(b + t * D)[g] : zero;
      xo[i] = in ? reinterpret_cast<const float4*>(x + t * D)[g] : zero;
      sa += dot4(y[i]);
      sb += dot4(vb[i]);
    }
    if (wa) {
      block_sum2(sa, sb, scratch);
      const float ra = 1.0f / sqrtf(sa / D + eps), rb = b ? 1.0f / sqrtf(sb / D + eps) : 0.f;
#pragma unroll
      for (int i = 0; i < VPT; ++i) {
        const int g = threadIdx.x + i * blockDim.x;
        if (g >= groups) continue;
        const float4 w1 = reinterpret_cast<const float4*>(wa)[g];
        float4 v = make_float4(y[i].x * ra * w1.x, y[i].y * ra * w1.y, y[i].z * ra * w1.z, y[i].w * ra * w1.w);
        if (b) {
          const float4 w2 = reinterpret_cast<const float4*>(wb)[g];
          v = make_float4(0.5f * (v.x + vb[i].x * rb * w2.x), 0.5f * (v.y + vb[i].y * rb * w2.y), 0.5f * (v.z + vb[i].z * rb * w2.z),
                          0.5f * (v.w + vb[i].w * rb * w2.w));
        }
        y[i] = v;
      }
    }
  }
  float rinv = centre_and_scale<VPT>(y, groups, D, eps, scratch);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int g = threadIdx.x + i * blockDim.x;
    if (g >= groups) continue;
    const float4 l = affine4(y[i], rinv, reinterpret_cast<const float4*>(pw)[g], reinterpret_cast<const float4*>(pb)[g]);
    xo[i] = make_float4(xo[i].x + l.x, xo[i].y + l.y, xo[i].z + l.z, xo[i].w + l.w);
    reinterpret_cast<float4*>(x + t * D)[g] = xo[i];
  }
  if (!nw) return;
  rinv = centre_and_scale<VPT>(xo, groups, D, eps, scratch);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int g = threadIdx.x + i * blockDim.x;
    if (g < groups)
      store4<TH>(h + t * D + 4 * (long)g, affine4(xo[i], rinv, reinterpret_cast<const float4*>(nw)[g], reinterpret_cast<const float4*>(nb)[g]));
  }
}

extern "C" int pi_sandwich_norm_add(float* x, void* h, int h_dtype, const float* a, const float* a_bias, const float* wa,
                                    const float* b, const float* wb, const float* pw, const float* pb, const float* nw,
                                    const float* nb, float eps, int T, int D, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && D > 0 && D <= 16000, "norm and add: bad sizes T=%d D=%d", T, D);
  PI_REQUIRE(x && a && pw && pb, "norm and add: the stream, a result and the norm's weight and bias are needed");
  PI_REQUIRE(!b || (wa && wb), "norm and add: two branches need both their weights");
  PI_REQUIRE(!nw || (nb && h), "norm and add: the next norm needs its bias and a place for its result");
  PI_REQUIRE(!nw || h_dtype == PI_F32 || h_dtype == PI_BF16, "norm and add: unsupported activation dtype %d", h_dtype);
  if (T == 0) return 0;
  const bool f32 = !nw || h_dtype == PI_F32;
  int wide_threads = 0, vpt = 0;
  bool aligned = true;
  for (const void* p : {(const void*)x, (const void*)h, (const void*)a, (const void*)a_bias, (const void*)wa, (const void*)b, (const void*)wb,
                        (const void*)pw, (const void*)pb, (const void*)nw, (const void*)nb})
    aligned = aligned && (uintptr_t)p % 16 == 0;
  if (aligned && wide_row_shape(T, D, wide_threads, vpt)) {
#define SW_GO(TH, V) hipLaunchKernelGGL((sandwich_norm_add_wide_kernel<TH, V>), dim3(T), dim3(wide_threads), 0, stream, x, (TH*)h, a, a_bias, wa, b, wb, pw, pb, nw, nb, eps, D)
#define SW_PICK(TH) do { if (vpt <= 1) SW_GO(TH, 1); else if (vpt <= 2) SW_GO(TH, 2); else SW_GO(TH, 4); } while (0)
    if (f32) SW_PICK(float); else SW_PICK(bf16_t);
#undef SW_PICK
#undef SW_GO
    return pi_check_launch("sandwich_norm_add_wide");
  }
  const int threads = D >= 1024 ? 256 : (D >= 256 ? 128 : 64);
  const size_t lds = (size_t)D * sizeof(float);
  if (f32)
    hipLaunchKernelGGL(sandwich_norm_add_kernel<float>, dim3(T), dim3(threads), lds, stream, x, (float*)h, a, a_bias, wa, b, wb, pw, pb, nw, nb, eps, D);
  else
    hipLaunchKernelGGL(sandwich_norm_add_kernel<bf16_t>, dim3(T), dim3(threads), lds, stream, x, (bf16_t*)h, a, a_bias, wa, b, wb, pw, pb, nw, nb, eps, D);
  return pi_check_launch("sandwich_norm_add");
}

// ---------------------------------------------------------------- a sublayer's result between two RMS norms
// A sublayer's result joins the stream through an RMS norm, and the next sublayer's input is made on the way:
//   x <- x + rms(y; pw);   h = rms(x; nw)       (nw null: no h),   rms(v; w) = v / sqrt(mean(v^2) + eps) * w
// y is a tensor [T, D]; or the float32 pieces of a product split over k, added here in split order; or the sum over a
// token's `top` choices of weight * (the row of `a` that the choice got), in choice order (routed experts).
// With `rows` only those rows of h are made (h row m from stream row rows[m]) and the stream is not written back.
struct JoinArgs {
  float* x;
  const float* a;          // the result, or the experts' rows
  const float* part;       // pieces [splits, T, D]
  int splits;
  const int* entry_row;    // [T, top]: where each choice's row lies
  const float* weights;    // [T, top]
  int top;
  const int* rows;
  const float* pw;
  float post_eps;
  const float* nw;
  float next_eps;
  int T, D, entries;
};

__device__ inline float4 fma4(float w, const float4& v, const float4& s) { return make_float4(fmaf(w, v.x, s.x), fmaf(w, v.y, s.y), fmaf(w, v.z, s.z), fmaf(w, v.w, s.w)); }
__device__ inline float4 add4(const float4& a, const float4& b) { return make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w); }

// columns 4 g .. 4 g + 3 of the result's row t
__device__ inline float4 join_value4(const JoinArgs& j, long t, int g) {
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
  if (j.part) {
    const float4* p = reinterpret_cast<const float4*>(j.part + t * j.D) + g;
    const long plane = (long)j.T * j.D / 4;
    for (int s0 = 0; s0 < j.splits; s0 += 8) {
      float4 l[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) l[u] = s0 + u < j.splits ? p[(s0 + u) * plane] : make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
      for (int u = 0; u < 8; ++u) v = add4(v, l[u]);
    }
    return v;
  }
  if (j.entry_row) {
    for (int c0 = 0; c0 < j.top; c0 += 4) {
      float4 l[4];
      float w[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int row = c0 + u < j.top ? j.entry_row[t * j.top + c0 + u] : -1;
        const bool ok = row >= 0 && row < j.entries;
        w[u] = ok ? j.weights[t * j.top + c0 + u] : 0.f;
        l[u] = ok ? reinterpret_cast<const float4*>(j.a + (long)row * j.D)[g] : make_float4(0.f, 0.f, 0.f, 0.f);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) v = fma4(w[u], l[u], v);
    }
    return v;
  }
  return reinterpret_cast<const float4*>(j.a + t * j.D)[g];
}

__device__ inline float join_value(const JoinArgs& j, long t, int d) {
  if (j.part) return split_sum(j.part, j.splits, (long)j.T * j.D, t * j.D + d);
  if (j.entry_row) {
    float v = 0.f;
    for (int c = 0; c < j.top; ++c) {
      const int row = j.entry_row[t * j.top + c];
      if (row >= 0 && row < j.entries) v = fmaf(j.weights[t * j.top + c], j.a[(long)row * j.D + d], v);
    }
    return v;
  }
  return j.a[t * j.D + d];
}

template <typename TH, int VPT>
__global__ __launch_bounds__(1024) void rms_join_wide_kernel(JoinArgs j, TH* __restrict__ h) {
  __shared__ float scratch[16];
  const long m = blockIdx.x, t = j.rows ? j.rows[m] : m;
  const int groups = j.D / 4;
  const bool ok = t >= 0 && t < j.T;                // a row outside the stream gives NaN, no fault
  float4 y[VPT], xo[VPT], w[VPT];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int g = threadIdx.x + i * blockDim.x;
    const bool in = g < groups;
    const float4 none = make_float4(0.f, 0.f, 0.f, 0.f), nan = make_float4(NAN, NAN, NAN, NAN);
    y[i] = !in ? none : ok ? join_value4(j, t, g) : nan;
    xo[i] = !in ? none : ok ? reinterpret_cast<const float4*>(j.x + t * j.D)[g] : nan;
    w[i] = in ? reinterpret_cast<const float4*>(j.pw)[g] : none;
    ss += dot4(y[i]);
  }
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / j.D + j.post_eps);
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int g = threadIdx.x + i * blockDim.x;
    xo[i] = make_float4(fmaf(y[i].x * r, w[i].x, xo[i].x), fmaf(y[i].y * r, w[i].y, xo[i].y), fmaf(y[i].z * r, w[i].z, xo[i].z),
                        fmaf(y[i].w * r, w[i].w, xo[i].w));
    ss += dot4(xo[i]);
    if (g >= groups) continue;
    if (!j.rows) reinterpret_cast<float4*>(j.x + t * j.D)[g] = xo[i];
    if (j.nw) w[i] = reinterpret_cast<const float4*>(j.nw)[g];
  }
  if (!j.nw) return;
  const float rn = 1.0f / sqrtf(block_sum(ss, scratch) / j.D + j.next_eps);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int g = threadIdx.x + i * blockDim.x;
    if (g < groups)
      store4<TH>(h + m * j.D + 4 * (long)g, make_float4(xo[i].x * rn * w[i].x, xo[i].y * rn * w[i].y, xo[i].z * rn * w[i].z, xo[i].w * rn * w[i].w));
  }
}

// the same for any width: the row stays in LDS
template <typename TH>
__global__ __launch_bounds__(256) void rms_join_kernel(JoinArgs j, TH* __restrict__ h) {
  extern __shared__ float row[];
  __shared__ float scratch[16];
  const long m = blockIdx.x, t = j.rows ? j.rows[m] : m;
  const bool ok = t >= 0 && t < j.T;
  float ss = 0.f;
  for (int d = threadIdx.x; d < j.D; d += blockDim.x) {
    const float v = ok ? join_value(j, t, d) : NAN;
    row[d] = v;
    ss = fmaf(v, v, ss);
  }
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / j.D + j.post_eps);
  ss = 0.f;
  for (int d = threadIdx.x; d < j.D; d += blockDim.x) {       // a thread meets its own entries only
    const float v = fmaf(row[d] * r, j.pw[d], ok ? j.x[t * j.D + d] : NAN);
    row[d] = v;
    if (ok && !j.rows) j.x[t * j.D + d] = v;
    ss = fmaf(v, v, ss);
  }
  if (!j.nw) return;
  const float rn = 1.0f / sqrtf(block_sum(ss, scratch) / j.D + j.next_eps);
  for (int d = threadIdx.x; d < j.D; d += blockDim.x) h[m * j.D + d] = from_float<TH>(row[d] * rn * j.nw[d]);
}

extern "C" int pi_rms_join(float* x, void* h, int h_dtype, const float* a, const float* part, int splits, const int* entry_row,
                           const float* weights, int top, int entries, const int* rows, int M, const float* pw, float post_eps,
                           const float* nw, float next_eps, int T, int D, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && M >= 0 && D > 0 && D <= 16000, "rms join: bad sizes T=%d M=%d D=%d", T, M, D);
  PI_REQUIRE(x && pw && (a != nullptr) != (part != nullptr), "rms join: the stream, the norm's weight and one result (a tensor or pieces) are needed");
  PI_REQUIRE(!part || (splits >= 1 && !entry_row), "rms join: %d pieces", splits);
  PI_REQUIRE(!entry_row || (weights && top > 0 && entries >= 0), "rms join: choices need their weights");
  PI_REQUIRE(!nw || (h && (h_dtype == PI_F32 || h_dtype == PI_BF16)), "rms join: the next norm needs a place for its result (dtype %d)", h_dtype);
  PI_REQUIRE(rows ? nw != nullptr : M == T, "rms join: %d rows of %d", M, T);
  if (M == 0) return 0;
  const JoinArgs j{x, a, part, splits, entry_row, weights, top, rows, pw, post_eps, nw, next_eps, T, D, entries};
  const bool f32 = !nw || h_dtype == PI_F32;
  int wide_threads = 0, vpt = 0;
  bool aligned = true;
  for (const void* p : {(const void*)x, (const void*)h, (const void*)a, (const void*)part, (const void*)pw, (const void*)nw}) aligned = aligned && (uintptr_t)p % 16 == 0;
  if (aligned && wide_row_shape(M, D, wide_threads, vpt)) {
#define RJ_GO(TH, V) hipLaunchKernelGGL((rms_join_wide_kernel<TH, V>), dim3(M), dim3(wide_threads), 0, stream, j, (TH*)h)
#define RJ_PICK(TH) do { if (vpt <= 1) RJ_GO(TH, 1); else if (vpt <= 2) RJ_GO(TH, 2); else RJ_GO(TH, 4); } while (0)
    if (f32) RJ_PICK(float); else RJ_PICK(bf16_t);
#undef RJ_PICK
#undef RJ_GO
    return pi_check_launch("rms_join_wide");
  }
  const int threads = D >= 1024 ? 256 : (D >= 256 ? 128 : 64);
  const size_t lds = (size_t)D * sizeof(float);
  if (f32) hipLaunchKernelGGL(rms_join_kernel<float>, dim3(M), dim3(threads), lds, stream, j, (float*)h);
  else hipLaunchKernelGGL(rms_join_kernel<bf16_t>, dim3(M), dim3(threads), lds, stream, j, (bf16_t*)h);
  return pi_check_launch("rms_join");
}

// ---------------------------------------------------------------- two attention maps into one head
// Differential attention: head n of kv group g holds the results a1 and a2 of two softmax maps over the same
// values.  In `attn` the maps are heads of their own, and a head's value vector may come in `split` equal pieces
// (each attended as a head of its own, so that heads whose values are a multiple of their keys' width fit kernels
// that want both alike): heads are ordered [g][map][piece][head within group], so that piece p of map m of group g
// is kv head (2 g + m) * split + p of the attention.  out[t, n, :] = mult * o / sqrt(mean(o^2) + eps),
// o = a1 - lam * a2, float32; one wave per (token, head).
template <typename TO, typename TI>
__global__ __launch_bounds__(PI_WAVE) void diff_combine_kernel(TO* __restrict__ out, const TI* __restrict__ attn, float lam, float eps,
                                                               float mult, int H, int G, int dv, int split) {
  const long t = blockIdx.x;
  const int n = blockIdx.y, lane = threadIdx.x;
  const int per = H / G, g = n / per, i = n % per, w = dv / split;      // w: a piece's width
  const TI* row = attn + t * 2 * H * dv;
  const long map_step = (long)split * per * w;                          // from map 1 to map 2 of a group
  float ss = 0.f;
  for (int c = lane; c < dv; c += PI_WAVE) {
    const long at = (((long)(2 * g) * split + c / w) * per + i) * w + c % w;
    const float o = fmaf(-lam, to_float(row[at + map_step]), to_float(row[at]));
    ss = fmaf(o, o, ss);
  }
  const float r = mult / sqrtf(wave_sum(ss) / dv + eps);
  for (int c = lane; c < dv; c += PI_WAVE) {
    const long at = (((long)(2 * g) * split + c / w) * per + i) * w + c % w;
    out[(t * H + n) * dv + c] = from_float<TO>(fmaf(-lam, to_float(row[at + map_step]), to_float(row[at])) * r);
  }
}

extern "C" int pi_diff_combine(void* out, int out_dtype, const void* attn, int in_dtype, float lam, float eps, float mult, int T, int H,
                               int G, int dv, int split, hipStream_t stream) {
  PI_REQUIRE(T >= 0 && H > 0 && H <= 65535 && G > 0 && H % G == 0 && dv > 0, "two maps: bad sizes heads=%d kv_heads=%d vdim=%d", H, G, dv);
  PI_REQUIRE(split >= 1 && dv % split == 0, "two maps: values of %d do not come in %d equal pieces", dv, split);
  if (T == 0) return 0;
  const dim3 grid(T, H), block(PI_WAVE);
#define DC_GO(TO, TI) hipLaunchKernelGGL((diff_combine_kernel<TO, TI>), grid, block, 0, stream, (TO*)out, (const TI*)attn, lam, eps, mult, H, G, dv, split)
  if (out_dtype == PI_F32 && in_dtype == PI_F32) DC_GO(float, float);
  else if (out_dtype == PI_BF16 && in_dtype == PI_BF16) DC_GO(bf16_t, bf16_t);
  else if (out_dtype == PI_BF16 && in_dtype == PI_F32) DC_GO(bf16_t, float);
  else return pi_fail("two maps: unsupported dtypes out=%d in=%d", out_dtype, in_dtype);
#undef DC_GO
  return pi_check_launch("diff_combine");
}

template <typename TO>
__global__ void cast_stream_kernel(TO* __restrict__ out, const float* __restrict__ x, long n) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) out[i] = from_float<TO>(x[i]);
}

// out = the float32 stream in the activation type (for sublayers that read the stream itself)
extern "C" int pi_cast_stream(void* out, int out_dtype, const float* x, long n, hipStream_t stream) {
  PI_REQUIRE(n >= 0 && out_dtype == PI_BF16, "cast: only float32 -> bfloat16 is a copy worth making (dtype %d)", out_dtype);
  if (n == 0) return 0;
  hipLaunchKernelGGL(cast_stream_kernel<bf16_t>, dim3(ceil_div(n, 256)), dim3(256), 0, stream, (bf16_t*)out, x, n);
  return pi_check_launch("cast_stream");
}

// ---------------------------------------------------------------- queries and keys normalised, then into the cache
// One block per token.  The projection row (float32) holds [q: nh*hd | k: nkv*hd | v: nkv*vd | gate: ng]
// (without the k and v columns when has_kv is 0: a layer that reads another layer's keys and values).
//   per_head 0:  q <- q / sqrt(mean over ALL nh*hd entries + eps) * wq     (wq / wk null: no norm of that projection)
//                k <- k / sqrt(mean over all nkv*hd entries + eps) * wk
//   per_head 1:  every head of q and of k divided by the root mean square of its own hd entries (+ eps inside the
//                root), times wq / wk where they are given
//   q times the token's temperature 1 + coef * ln(floor((p + 1) / every) + 1)           (coef 0: none)
//   k -> key pages [page, kv head, slot, hd];   v -> value pages [page, kv head, vd, slot]
//   gate <- 1 / (1 + exp(-gate))                              -> float32 [T, ng]
// `part` (with `splits` planes of `part_stride` floats, rows of proj_stride columns): the projection as the float32
// pieces of a product split over k, instead of `proj`.
template <typename T>
__global__ __launch_bounds__(1024) void qk_norm_kv_write_kernel(
    T* __restrict__ q_out, long q_stride, float* __restrict__ gate_out, const float* __restrict__ proj, long proj_stride,
    const float* __restrict__ wq, const float* __restrict__ wk, const int* __restrict__ positions, const int* __restrict__ req_of_token,
    float eps, float temp_coef, int temp_every, int nh, int nkv, int hd, int vd, int ng, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const int* __restrict__ block_table, int table_width, int page_size, long num_pages,
    const float* __restrict__ part, int splits, long part_stride, int per_head, int has_kv) {
  __shared__ float scratch[32];
  extern __shared__ float staged[];              // the token's row, when it comes in pieces
  const long t = blockIdx.x;
  const float* row = proj + t * proj_stride;
  const int QN = nh * hd, KN = has_kv ? nkv * hd : 0, VN = has_kv ? nkv * vd : 0;
  if (part) {
    // the projection is still split over k: its float32 pieces are added here, in split order, once per element
    for (int i = threadIdx.x; i < QN + KN + VN + ng; i += blockDim.x) staged[i] = split_sum(part, splits, part_stride, t * proj_stride + i);
    __syncthreads();
    row = staged;
  }
  const int p = positions[t];
  const float temp = temp_coef != 0.f ? 1.0f + temp_coef * logf((float)((p + 1) / temp_every) + 1.0f) : 1.0f;
  T* qr = q_out + t * q_stride;
  for (int i = threadIdx.x; i < ng; i += blockDim.x) gate_out[t * ng + i] = 1.0f / (1.0f + expf(-row[QN + KN + VN + i]));
  long page = -1;
  int slot = 0;
  if (k_cache && has_kv) {
    const int blk = p / page_size;
    slot = p % page_size;
    page = blk < table_width ? block_table[(long)req_of_token[t] * table_width + blk] : -1;
    if (page >= num_pages) page = -1;              // no page for this position: nothing is written
  }
  if (per_head) {
    // a wave per head: query heads first, then key heads; the sum of squares runs over the head's own entries
    const int wave = threadIdx.x / PI_WAVE, lane = threadIdx.x % PI_WAVE, nwaves = blockDim.x / PI_WAVE;
    for (int u = wave; u < nh + (has_kv ? nkv : 0); u += nwaves) {
      const bool is_q = u < nh;
      const float* src = row + (is_q ? u * hd : QN + (u - nh) * hd);
      float ss = 0.f;
      for (int d = lane; d < hd; d += PI_WAVE) ss = fmaf(src[d], src[d], ss);
      ss = wave_sum(ss);
      const float r = 1.0f / sqrtf(ss / hd + eps);
      if (is_q) {
        for (int d = lane; d < hd; d += PI_WAVE) {
          float v = src[d] * r;
          if (wq) v *= wq[u * hd + d];
          qr[u * hd + d] = from_float<T>(v * temp);
        }
      } else if (page >= 0) {
        const int g = u - nh;
        for (int d = lane; d < hd; d += PI_WAVE) {
          float v = src[d] * r;
          if (wk) v *= wk[g * hd + d];
          k_cache[((page * nkv + g) * page_size + slot) * hd + d] = from_float<T>(v);
        }
      }
    }
  } else {
    float sq = 0.f, sk = 0.f;
    for (int i = threadIdx.x; i < QN; i += blockDim.x) sq = fmaf(row[i], row[i], sq);
    for (int i = threadIdx.x; i < KN; i += blockDim.x) sk = fmaf(row[QN + i], row[QN + i], sk);
    block_sum2(sq, sk, scratch);                   // both sums of squares in one trip through LDS
    const float rq = wq ? 1.0f / sqrtf(sq / QN + eps) : 1.0f;
    const float rk = wk && KN ? 1.0f / sqrtf(sk / KN + eps) : 1.0f;
    for (int i = threadIdx.x; i < QN; i += blockDim.x) {
      float v = row[i];
      if (wq) v = v * rq * wq[i];
      qr[i] = from_float<T>(v * temp);
    }
    if (page >= 0) {
      for (int i = threadIdx.x; i < KN; i += blockDim.x) {
        float v = row[QN + i];
        if (wk) v = v * rk * wk[i];
        const int g = i / hd, d = i % hd;
        k_cache[((page * nkv + g) * page_size + slot) * hd + d] = from_float<T>(v);
      }
    }
  }
  if (page < 0) return;
  for (int i = threadIdx.x; i < VN; i += blockDim.x) {
    const int g = i / vd, d = i % vd;
    v_cache[((page * nkv + g) * vd + d) * page_size + slot] = from_float<T>(row[QN + KN + i]);
  }
}

extern "C" int pi_qk_norm_kv_write(void* q_out, long q_stride, float* gate_out, int dtype, const float* proj, long proj_stride,
                                   const float* wq, const float* wk, const int* positions, const int* req_of_token, float eps,
                                   float temp_coef, int temp_every, int T, int nh, int nkv, int hd, int vd, int ng,
                                   void* k_cache, void* v_cache, const int* block_table, int table_width, int page_size,
                                   long num_pages, const float* part, int splits, long part_stride, int per_head, int has_kv,
                                   hipStream_t stream) {
  PI_REQUIRE(T >= 0 && nh > 0 && nkv > 0 && hd > 0 && vd > 0 && ng >= 0, "qk norm: bad sizes");
  const long row_floats = (long)nh * hd + (has_kv ? (long)nkv * (hd + vd) : 0) + ng;
  PI_REQUIRE(proj_stride >= row_floats, "qk norm: projection rows of %ld hold no q, k, v and gates", proj_stride);
  PI_REQUIRE(temp_coef == 0.f || temp_every > 0, "qk norm: the temperature's period must be positive, got %d", temp_every);
  PI_REQUIRE(!k_cache || (has_kv && v_cache && block_table && req_of_token && table_width > 0 && page_size > 0 && num_pages > 0),
             "qk norm: bad cache geometry");
  PI_REQUIRE(ng == 0 || gate_out, "qk norm: gates without a place for them");
  PI_REQUIRE((proj != nullptr) != (part != nullptr), "qk norm: give the projection as a tensor or as pieces");
  PI_REQUIRE(!part || (splits >= 1 && part_stride >= (long)T * proj_stride), "qk norm: bad pieces (%d planes of %ld floats)", splits, part_stride);
  PI_REQUIRE(!part || row_floats * 4 <= 60000, "qk norm: rows of %ld floats in pieces do not fit the staging memory", row_floats);
  const size_t lds = part ? (size_t)row_floats * sizeof(float) : 0;
  if (T == 0) return 0;
  const int threads = T <= 64 ? 1024 : 256;      // few tokens (decode steps): the row's passes are a matter of latency
#define QKN_GO(TT) hipLaunchKernelGGL(qk_norm_kv_write_kernel<TT>, dim3(T), dim3(threads), lds, stream, (TT*)q_out, q_stride, gate_out, proj, \
                                      proj_stride, wq, wk, positions, req_of_token, eps, temp_coef, temp_every, nh, nkv, hd, vd, ng,  \
                                      (TT*)k_cache, (TT*)v_cache, block_table, table_width, page_size, num_pages, part, splits, part_stride, \
                                      per_head, has_kv)
  if (dtype == PI_F32) QKN_GO(float);
  else if (dtype == PI_BF16) QKN_GO(bf16_t);
  else return pi_fail("qk norm: unsupported dtype %d", dtype);
#undef QKN_GO
  return pi_check_launch("qk_norm_kv_write");
}

// ---------------------------------------------------------------- queries and keys rotated, then normalised per head
// Projection rows (float32, a tensor or the pieces of a product split over k) hold [q: nh*hd | k: nkv*hd | v: nkv*vd | gates: ng],
// or no v: values are then the keys (vd = hd, v_col = the keys' first column).
//   q, k <- + bias (by column; null: none), rotated by the token's angles on the first rd features of each head
//           (halves paired, or neighbours), then every head divided by the root mean square of its hd entries, times
//           wq / wk (one weight of hd for all heads; null: none)
//   values: their columns (with their bias), neither rotated nor normalised
// Queries go to q_out, keys to the key pages [page, kv head, slot, hd], values to the value pages [page, kv head, vd, slot].
// Pieces only: the gates' columns are summed into gate_out (float32 [T, ng]) as they are, for whoever applies them.
// Everything is float32 until the one rounding on store.
struct QkRopeArgs {
  const float* proj;       // [T, stride], or null: the pieces
  long stride;
  const float* part;       // [splits, T, stride]
  int splits;
  long plane;
  const float* bias;       // one per column of q, k and v, or null
  const float* wq;         // [hd] or null
  const float* wk;
  int v_col, vd, g_col;    // where the values and the gates start in a row; a value head's width
  const float* table;      // [T, rd]: cosines, then sines
  int rd, interleaved;
  float eps;
  int T, nh, nkv, hd, ng;
  const int* positions;
  const int* req_of_token;
  const int* block_table;
  int table_width, page_size;
  long num_pages;
  float* gate_out;
};

__device__ inline float qkr_value(const QkRopeArgs& a, long t, int col) {
  const float v = a.part ? split_sum(a.part, a.splits, a.plane, t * a.stride + col) : a.proj[t * a.stride + col];
  return a.bias ? v + a.bias[col] : v;
}

// four neighbouring columns; rows and columns are whole 16-byte groups
__device__ inline float4 qkr_value4(const QkRopeArgs& a, long t, int col, bool with_bias) {
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
  if (a.part) {
    const float* p = a.part + t * a.stride + col;
    for (int s0 = 0; s0 < a.splits; s0 += 8) {       // eight pieces' loads in flight, added in split order
      float4 l[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) l[u] = s0 + u < a.splits ? *reinterpret_cast<const float4*>(p + (s0 + u) * a.plane) : make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
      for (int u = 0; u < 8; ++u) { v.x += l[u].x; v.y += l[u].y; v.z += l[u].z; v.w += l[u].w; }
    }
  } else {
    v = *reinterpret_cast<const float4*>(a.proj + t * a.stride + col);
  }
  if (with_bias && a.bias) {
    const float4 b = *reinterpret_cast<const float4*>(a.bias + col);
    v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w;
  }
  return v;
}

// page and slot of a token's position; false: no page (the host checks tables; nothing is written outside the pool)
__device__ inline bool qkr_place(const QkRopeArgs& a, long t, long& page, int& slot) {
  const int pos = a.positions[t], blk = pos / a.page_size;
  slot = pos % a.page_size;
  page = blk < a.table_width ? a.block_table[(long)a.req_of_token[t] * a.table_width + blk] : -1;
  return page >= 0 && page < a.num_pages;
}

// Blocks [0, head_blocks): heads of queries and keys, LANES lanes per (token, head) with four features each (LANES 0:
// a wave per (token, head), features 64 apart, for sizes that are no whole 16-byte groups); then value_blocks: a
// thread per (PT neighbouring tokens, kv head, feature); then the gates of pieces, four columns per thread.
template <typename T, int LANES, int PT>
__global__ __launch_bounds__(256) void qk_rope_norm_write_kernel(QkRopeArgs a, T* __restrict__ q_out, long q_stride, T* __restrict__ k_cache,
                                                                 T* __restrict__ v_cache, int head_blocks, int value_blocks) {
  const int hd = a.hd, half = a.rd / 2;
  if ((int)blockIdx.x < head_blocks) {
    constexpr int L = LANES ? LANES : PI_WAVE;
    const long item = ((long)blockIdx.x * 256 + threadIdx.x) / L;
    const int lane = threadIdx.x % L, heads = a.nh + a.nkv;
    const int u = (int)(item % heads);
    const long t = item / heads;
    if (t >= a.T) return;                            // whole groups of lanes leave together
    const int col = u * hd;                          // key heads follow the query heads in the row
    T* dst;
    if (u < a.nh) {
      dst = q_out + t * q_stride + col;
    } else {
      long page;
      int slot;
      if (!qkr_place(a, t, page, slot)) return;
      dst = k_cache + ((page * a.nkv + (u - a.nh)) * a.page_size + slot) * hd;
    }
    const float* cs = a.table + t * a.rd;
    const float* wn = u < a.nh ? a.wq : a.wk;
    if constexpr (LANES > 0) {
      const int d = 4 * lane;
      const bool in = d < hd;
      const float4 v4 = in ? qkr_value4(a, t, col + d, true) : make_float4(0.f, 0.f, 0.f, 0.f);
      float v[4] = {v4.x, v4.y, v4.z, v4.w}, o[4];
      float ss = fmaf(v[3], v[3], fmaf(v[2], v[2], fmaf(v[1], v[1], v[0] * v[0])));      // a rotation keeps it
#pragma unroll
      for (int off = L / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, PI_WAVE);
      const float r = 1.0f / sqrtf(ss / hd + a.eps);
      const bool by_lanes = !a.interleaved && half % 4 == 0;      // a feature's partner is the same feature of another lane
      float other[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) other[e] = 0.f;
      if (by_lanes && a.rd > 0) {
        const int partner = (int)(threadIdx.x % PI_WAVE) + (d < half ? half / 4 : (d < a.rd ? -half / 4 : 0));
#pragma unroll
        for (int e = 0; e < 4; ++e) other[e] = __shfl(v[e], partner, PI_WAVE);
      }
      if (!in) return;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = d + e;
        o[e] = v[e];
        if (i < a.rd) {
          const int j = a.interleaved ? i / 2 : (i < half ? i : i - half);
          const bool low = a.interleaved ? (i & 1) == 0 : i < half;
          const float b = a.interleaved ? v[e ^ 1] : (by_lanes ? other[e] : qkr_value(a, t, col + (low ? i + half : i - half)));
          float lo, hi;
          rope_pair(low ? v[e] : b, low ? b : v[e], cs[j], cs[half + j], lo, hi);
          o[e] = low ? lo : hi;
        }
        o[e] *= r;
        if (wn) o[e] *= wn[i];
      }
      store4<T>(dst + d, make_float4(o[0], o[1], o[2], o[3]));
    } else {
      float ss = 0.f;
      for (int i = lane; i < hd; i += PI_WAVE) {
        const float v = qkr_value(a, t, col + i);
        ss = fmaf(v, v, ss);
      }
      const float r = 1.0f / sqrtf(wave_sum(ss) / hd + a.eps);
      for (int i = lane; i < hd; i += PI_WAVE) {
        float v = qkr_value(a, t, col + i);
        if (i < a.rd) {
          const int j = a.interleaved ? i / 2 : (i < half ? i : i - half);
          const bool low = a.interleaved ? (i & 1) == 0 : i < half;
          const float b = qkr_value(a, t, col + (a.interleaved ? i ^ 1 : (low ? i + half : i - half)));
          float lo, hi;
          rope_pair(low ? v : b, low ? b : v, cs[j], cs[half + j], lo, hi);
          v = low ? lo : hi;
        }
        v *= r;
        dst[i] = from_float<T>(wn ? v * wn[i] : v);
      }
    }
    return;
  }
  if ((int)blockIdx.x < head_blocks + value_blocks) {
    const long idx = ((long)blockIdx.x - head_blocks) * 256 + threadIdx.x;
    const int vd = a.vd, row = a.nkv * vd;
    const int c = (int)(idx % row), g = c / vd, d = c % vd;
    const long t0 = idx / row * PT;
    if (t0 >= a.T) return;
    const int n = (int)min((long)PT, a.T - t0);
    T val[PT];
    int pos[PT], req[PT];
#pragma unroll
    for (int i = 0; i < PT; ++i) {
      const long t = t0 + (i < n ? i : 0);
      val[i] = from_float<T>(qkr_value(a, t, a.v_col + c));
      pos[i] = a.positions[t];
      req[i] = a.req_of_token[t];
    }
    if constexpr (PT == 4 && sizeof(T) == 2) {
      // four neighbours in one page: one 8-byte store
      if (n == 4 && a.page_size % 4 == 0 && pos[0] % 4 == 0 && req[1] == req[0] && req[2] == req[0] && req[3] == req[0] &&
          pos[1] == pos[0] + 1 && pos[2] == pos[0] + 2 && pos[3] == pos[0] + 3) {
        long page;
        int slot;
        if (!qkr_place(a, t0, page, slot)) return;
        const uint16_t* b = reinterpret_cast<const uint16_t*>(val);
        *reinterpret_cast<uint2*>(v_cache + ((page * a.nkv + g) * vd + d) * a.page_size + slot) =
            make_uint2((uint32_t)b[0] | ((uint32_t)b[1] << 16), (uint32_t)b[2] | ((uint32_t)b[3] << 16));
        return;
      }
    }
#pragma unroll
    for (int i = 0; i < PT; ++i) {
      long page;
      int slot;
      if (i < n && qkr_place(a, t0 + i, page, slot)) v_cache[((page * a.nkv + g) * vd + d) * a.page_size + slot] = val[i];
    }
    return;
  }
  const long idx = ((long)blockIdx.x - head_blocks - value_blocks) * 256 + threadIdx.x;
  const int per = (a.ng + 3) / 4;
  const long t = idx / per;
  const int c = (int)(idx % per) * 4;
  if (t >= a.T) return;
  const int col = a.g_col + c;
  if constexpr (LANES > 0) {
    if (a.ng % 4 == 0 && a.g_col % 4 == 0) {
      *reinterpret_cast<float4*>(a.gate_out + t * a.ng + c) = qkr_value4(a, t, col, false);
      return;
    }
  }
  for (int e = 0; e < 4 && c + e < a.ng; ++e) a.gate_out[t * a.ng + c + e] = split_sum(a.part, a.splits, a.plane, t * a.stride + col + e);
}

extern "C" int pi_qk_rope_norm_write(void* q_out, long q_stride, int dtype, const float* proj, long stride, const float* part, int splits,
                                     const float* bias, const float* table, int rd, int interleaved, float eps, const float* wq,
                                     const float* wk, int T, int nh, int nkv, int hd, int vd, int ng, float* gate_out, const int* positions, const int* req_of_token, void* k_cache,
                                     void* v_cache, const int* block_table, int table_width, int page_size, long num_pages,
                                     hipStream_t stream) {
  PI_REQUIRE(T >= 0 && nh > 0 && nkv > 0 && hd > 0 && hd <= 640 && ng >= 0, "qk rope norm: bad sizes T=%d heads=%d kv_heads=%d head_dim=%d", T, nh, nkv, hd);
  PI_REQUIRE((proj != nullptr) != (part != nullptr) && (!part || splits >= 1), "qk rope norm: give the projection as a tensor or as pieces");
  // vd == 0: the values are the keys
  const int g_col = (nh + nkv) * hd + (vd > 0 ? nkv * vd : 0), v_col = vd > 0 ? (nh + nkv) * hd : nh * hd;
  if (vd == 0) vd = hd;
  PI_REQUIRE(vd > 0 && vd <= 640, "qk rope norm: values of %d", vd);
  PI_REQUIRE(stride >= (long)g_col + (part ? ng : 0), "qk rope norm: rows of %ld hold no queries, keys and gates", stride);
  PI_REQUIRE(rd >= 0 && rd <= hd && rd % 2 == 0 && (rd == 0 || table), "qk rope norm: rotation of %d features", rd);
  PI_REQUIRE(q_out && positions && req_of_token && k_cache && v_cache && block_table && table_width > 0 && page_size > 0 && num_pages > 0,
             "qk rope norm: bad cache geometry");
  PI_REQUIRE(!part || ng == 0 || gate_out, "qk rope norm: gates in pieces need a place");
  PI_REQUIRE(dtype == PI_F32 || dtype == PI_BF16, "qk rope norm: unsupported dtype %d", dtype);
  if (T == 0) return 0;
  QkRopeArgs a{proj, stride, part, splits, (long)T * stride, bias, wq, wk, v_col, vd, g_col, table, rd, interleaved, eps, T, nh, nkv, hd, ng, positions, req_of_token,
               block_table, table_width, page_size, num_pages, gate_out};
  const int bytes = dtype == PI_F32 ? 16 : 8;
  bool wide = hd % 4 == 0 && hd <= 256 && stride % 4 == 0 && q_stride % 4 == 0 && (uintptr_t)q_out % bytes == 0 && (uintptr_t)k_cache % bytes == 0;
  for (const void* p : {(const void*)proj, (const void*)part, (const void*)bias, (const void*)gate_out}) wide = wide && (uintptr_t)p % 16 == 0;
  const int lanes = !wide ? 0 : (hd <= 64 ? 16 : (hd <= 128 ? 32 : 64));
  const bool four = T >= 16 && (uintptr_t)v_cache % 8 == 0;
  const long items = (long)T * (nh + nkv), values = (long)ceil_div(T, four ? 4 : 1) * nkv * vd, gates = part ? (long)T * ceil_div(ng, 4) : 0;
  const long hb = (items * (lanes ? lanes : PI_WAVE) + 255) / 256, vb = (values + 255) / 256, gb = (gates + 255) / 256;
  PI_REQUIRE(hb + vb + gb < 2147483647L, "qk rope norm: too many tokens (%d)", T);
  const dim3 grid((unsigned)(hb + vb + gb)), block(256);
#define QR_GO(TT, L_, P_) hipLaunchKernelGGL((qk_rope_norm_write_kernel<TT, L_, P_>), grid, block, 0, stream, a, (TT*)q_out, q_stride, (TT*)k_cache, (TT*)v_cache, (int)hb, (int)vb)
#define QR_PICK(TT)                                                            \
  do {                                                                         \
    if (lanes == 0) { if (four) QR_GO(TT, 0, 4); else QR_GO(TT, 0, 1); }       \
    else if (lanes == 16) { if (four) QR_GO(TT, 16, 4); else QR_GO(TT, 16, 1); } \
    else if (lanes == 32) { if (four) QR_GO(TT, 32, 4); else QR_GO(TT, 32, 1); } \
    else { if (four) QR_GO(TT, 64, 4); else QR_GO(TT, 64, 1); }                \
  } while (0)
  if (dtype == PI_F32) QR_PICK(float); else QR_PICK(bf16_t);
#undef QR_PICK
#undef QR_GO
  return pi_check_launch("qk_rope_norm_write");
}
