// bfloat16 matrix product on the matrix cores for many rows (prompts):
//   C[M, N] (+)= A[M, K] . W[N, K]^T, float32 accumulation.
// Block tile 128 x 128, reduction slab 64, four waves in 2 x 2, each wave 64 x 64 as 2 x 2
// tiles of v_mfma_f32_32x32x16_bf16.  Slabs go from memory straight into LDS (buffer loads
// with the LDS as their destination, double buffered): no registers and no LDS store
// instructions in between.  Such a load writes its 64 lanes' 16 bytes one after the other, so
// rows cannot be padded; instead the 16-byte pieces of a row are turned by (row / 2) % 8, which
// puts the fragment reads of sixteen neighbouring rows on all 64 banks.  (Through registers
// and padded rows, which this kernel did first, the q/k/v product of a 2,048-token prompt took
// 40 us instead of 34 and the 256 x 256 kernel below 133 us instead of 120 on the gate / up
// product: 230 instead of 180 registers, eight LDS stores per slab and thread.)
//
// Epilogues: store bfloat16, store float32, add into float32 (the residual stream), or
// SwiGLU: with gate and up rows interleaved in blocks of 16 in W, the gate and the up value of
// the same (row, feature) sit 16 lanes apart; one row swap brings them together and
// silu(gate) * up is stored directly.
//
// Any M and N (edges read zeros and are skipped on store); K must be a multiple of
// 8 and row strides multiples of 8 so that 16-byte loads stay aligned.  Each output row
// accumulates over k in the same order whatever the other rows are.
#include <type_traits>

#include "addressing.h"
#include "mfma.h"

PI_DEFINE_MODULE(bf16)

#define BM 128
#define BN 128
#define BK 64
#define TILE_ELEMS (BM * BK)                // a tile's slab in LDS: rows of 128 bytes

enum { EPI_BF16 = 0, EPI_F32 = 1, EPI_ACCUM = 2, EPI_SWIGLU = 3, EPI_CLAMPED_GLU = 4, EPI_RELU2 = 5, EPI_GELU = 6, EPI_GATE = 7 };

// results that leave as bfloat16, one per input column: as they are, through max(c, 0)^2, through the exact gelu, or times
// the sigmoid of a gate of their own
#define EPI_HALF(E) ((E) == EPI_BF16 || (E) == EPI_RELU2 || (E) == EPI_GELU || (E) == EPI_GATE)

// the gated epilogues store one output column per pair of input columns, in bfloat16
#define EPI_GATED(E) ((E) == EPI_SWIGLU || (E) == EPI_CLAMPED_GLU)

// What the clamped gated unit needs beside the products: biases in the order of W's rows (gate and up
// interleaved by 16), the clamp and the sigmoid's factor.  For EPI_GATE, `bias` points at the gates (float32, before
// their sigmoid, one per output; rows gate_stride apart).
struct GluArgs {
  const float* bias;
  float limit, alpha;
  long gate_stride;
};

// g' = min(g + bg, limit), u' = clamp(u + bu, -limit, limit): g' * sigmoid(alpha * g') * (u' + 1)
__device__ inline float clamped_glu_mul(float g, float u, float bg, float bu, float limit, float alpha) {
  g = fminf(g + bg, limit);
  u = fminf(fmaxf(u + bu, -limit), limit);
  return g * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * alpha * g)) * (u + 1.0f);
}

// silu(g) * u for a bfloat16 result: the hardware exponential and reciprocal (1 ulp each) are
// far inside the rounding of the store
__device__ inline float silu_mul(float g, float u) {
  return g * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * g)) * u;
}

__device__ inline float sigmoid_fast(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }

// x Phi(x) for a bfloat16 result, the error function by formula 7.1.26 of Abramowitz and Stegun's Handbook of
// Mathematical Functions (absolute error of Phi below 1e-7): with q(|x|) = 1 - Phi(|x|) it is x (1 - q) above zero and
// x q below, so that nothing cancels where x is far below zero.
__device__ inline float gelu_mul(float x) {
  const float a = fabsf(x) * 0.70710678118654752f;
  const float t = __builtin_amdgcn_rcpf(fmaf(0.3275911f, a, 1.0f));
  const float poly = t * fmaf(t, fmaf(t, fmaf(t, fmaf(t, 1.061405429f, -1.453152027f), 1.421413741f), -0.284496736f), 0.254829592f);
  const float q = 0.5f * poly * __builtin_amdgcn_exp2f(-1.4426950408889634f * a * a);
  return x * (x >= 0.f ? 1.0f - q : q);
}

// The epilogue of both kernels: 32 rows x 64 columns of a wave's result, held as two 32 x 32
// accumulator tiles (lane = column, register = row), go through a patch of LDS that belongs to
// the wave alone and come back with eight (bfloat16) or four (float32) neighbouring columns in
// one lane, so that a row leaves as whole 16-byte stores instead of 2- or 4-byte ones.
// `C` points at the corner's first element (for SwiGLU: of the halved output); rows_left and
// cols_left (input columns) may be <= 0 or ragged; `wide` says that 16-byte stores are aligned.
#define PATCH_LD 72                      // floats per patch row: rows r and r + 4 fall on different bank halves
#define PATCH_FLOATS (32 * PATCH_LD)

__device__ inline uint32_t pack2(float a, float b) { return f32x2_to_bf16x2_bits(a, b); }

template <int EPI>
__device__ inline void store_rows32(float* patch, const f32x16_t& acc0, const f32x16_t& acc1, void* C, int ld, int row0,
                                    int rows_left, int cols_left, int lane, bool wide, GluArgs glu = GluArgs{nullptr, 0.f, 0.f, 0},
                                    long col0 = 0) {
  const int half = lane / 32, ccol = lane % 32;
#pragma unroll
  for (int v = 0; v < 16; ++v) {
    const int r = 8 * (v / 4) + 4 * half + v % 4;
    patch[r * PATCH_LD + ccol] = acc0[v];
    patch[r * PATCH_LD + 32 + ccol] = acc1[v];
  }
  // the wave reads what its own lanes wrote: LDS serves one wave's accesses in order
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  if (EPI_GATED(EPI)) {
    // columns 0..15 of a tile are gate rows of W, 16..31 the up rows of the same features
    bf16_t* out = reinterpret_cast<bf16_t*>(C);
#pragma unroll
    for (int pass = 0; pass < 2; ++pass) {
      const int id = pass * 64 + lane, r = id / 4, j = (id % 4) / 2, q = id % 2;
      const float* g = patch + r * PATCH_LD + j * 32 + q * 8;
      const int oc = j * 16 + q * 8;                       // output column; its up column in the input is j*32 + 16 + q*8 (+7)
      if (row0 + r >= rows_left || j * 32 + 16 + q * 8 >= cols_left) continue;
      const f32x4_t g0 = *reinterpret_cast<const f32x4_t*>(g), g1 = *reinterpret_cast<const f32x4_t*>(g + 4);
      const f32x4_t u0 = *reinterpret_cast<const f32x4_t*>(g + 16), u1 = *reinterpret_cast<const f32x4_t*>(g + 20);
      float o[8];
      if (EPI == EPI_CLAMPED_GLU) {
        const bool biased = glu.bias != nullptr;
        const float* bg = glu.bias + (biased ? col0 + j * 32 + q * 8 : 0);      // col0: the corner's first input column
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          o[e] = clamped_glu_mul(g0[e], u0[e], biased ? bg[e] : 0.f, biased ? bg[16 + e] : 0.f, glu.limit, glu.alpha);
          o[4 + e] = clamped_glu_mul(g1[e], u1[e], biased ? bg[4 + e] : 0.f, biased ? bg[20 + e] : 0.f, glu.limit, glu.alpha);
        }
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) { o[e] = silu_mul(g0[e], u0[e]); o[4 + e] = silu_mul(g1[e], u1[e]); }
      }
      bf16_t* dst = out + (row0 + r) * ld + oc;
      if (wide && j * 32 + 16 + q * 8 + 8 <= cols_left) {
        *reinterpret_cast<u32x4_t*>(dst) = u32x4_t{pack2(o[0], o[1]), pack2(o[2], o[3]), pack2(o[4], o[5]), pack2(o[6], o[7])};
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (j * 32 + 16 + q * 8 + e < cols_left) dst[e] = from_float<bf16_t>(o[e]);
      }
    }
  } else if (EPI_HALF(EPI)) {
    bf16_t* out = reinterpret_cast<bf16_t*>(C);
#pragma unroll
    for (int pass = 0; pass < 4; ++pass) {
      const int id = pass * 64 + lane, r = id / 8, c = (id % 8) * 8;
      if (row0 + r >= rows_left || c >= cols_left) continue;
      const float* src = patch + r * PATCH_LD + c;
      f32x4_t a = *reinterpret_cast<const f32x4_t*>(src), b = *reinterpret_cast<const f32x4_t*>(src + 4);
      if (EPI == EPI_RELU2) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          a[e] = fmaxf(a[e], 0.f); a[e] *= a[e];
          b[e] = fmaxf(b[e], 0.f); b[e] *= b[e];
        }
      }
      if (EPI == EPI_GELU) {
#pragma unroll
        for (int e = 0; e < 4; ++e) { a[e] = gelu_mul(a[e]); b[e] = gelu_mul(b[e]); }
      }
      if (EPI == EPI_GATE) {
        const float* g = glu.bias + (row0 + r) * glu.gate_stride + c;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float f = c + e < cols_left ? sigmoid_fast(g[e]) : 0.f;
          if (e < 4) a[e] *= f; else b[e - 4] *= f;
        }
      }
      bf16_t* dst = out + (row0 + r) * ld + c;
      if (wide && c + 8 <= cols_left) {
        *reinterpret_cast<u32x4_t*>(dst) = u32x4_t{pack2(a[0], a[1]), pack2(a[2], a[3]), pack2(b[0], b[1]), pack2(b[2], b[3])};
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (c + e < cols_left) dst[e] = from_float<bf16_t>(e < 4 ? a[e] : b[e - 4]);
      }
    }
  } else {
    float* out = reinterpret_cast<float*>(C);
#pragma unroll
    for (int pass = 0; pass < 8; ++pass) {
      const int id = pass * 64 + lane, r = id / 16, c = (id % 16) * 4;
      if (row0 + r >= rows_left || c >= cols_left) continue;
      f32x4_t a = *reinterpret_cast<const f32x4_t*>(patch + r * PATCH_LD + c);
      float* dst = out + (row0 + r) * ld + c;
      if (wide && c + 4 <= cols_left) {
        if (EPI == EPI_ACCUM) a += *reinterpret_cast<const f32x4_t*>(dst);
        *reinterpret_cast<f32x4_t*>(dst) = a;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c + e < cols_left) dst[e] = EPI == EPI_ACCUM ? dst[e] + a[e] : a[e];
      }
    }
  }
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

// Global loads go through buffer descriptors: a scalar base (the block's first row at its first
// k), a byte length, and per-lane 32-bit offsets.  An offset at or beyond the length reads
// zeros, which is how rows beyond the matrix and k beyond the range are filled, without a branch.
#if defined(__HIP_DEVICE_COMPILE__)
__device__ inline __amdgpu_buffer_rsrc_t operand_descriptor(const bf16_t* operand, addressing::Descriptor d) {
  // made scalar by hand so that the loads take the descriptor from scalar registers
  const long bytes = d.bytes;
  const uint64_t v = reinterpret_cast<uint64_t>(operand + d.base);
  const uint32_t lo = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(v));
  const uint32_t hi = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(v >> 32));
  void* p = reinterpret_cast<void*>((static_cast<uint64_t>(hi) << 32) | lo);
  return __builtin_amdgcn_make_buffer_rsrc(p, 0, __builtin_amdgcn_readfirstlane((int)bytes), 0x00020000);
}
#endif

template <int EPI>
__global__ __launch_bounds__(256) void gemm_mfma_kernel(void* __restrict__ Cv, long ldc, const bf16_t* __restrict__ A, long lda,
                                                        const bf16_t* __restrict__ W, long ldw, int M, int N, int K,
                                                        int tiles_n, int k_per_split, const int* __restrict__ group_of_tile,
                                                        const int* __restrict__ tile_row0, const int* __restrict__ tile_rows,
                                                        long group_stride, long group_a_step, long group_c_step, GluArgs glu) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  constexpr int ROW = BK;                   // rows of 128 bytes, no padding (see the large-tile kernel)
  constexpr int TILE = BM * ROW;
  uint16_t* As = lds;                       // [2][BM][ROW], 16-byte pieces of a row turned by (row / 2) % 8
  uint16_t* Ws = lds + 2 * TILE;            // [2][BN][ROW]
  const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64;
  const int wm = wave / 2, wn = wave % 2;
  // k split over blocks (gridDim.y > 1, float32 store only): split s owns k in
  // [s * k_per_split, (s + 1) * k_per_split) and writes its piece to C + s * M * N.
  const int k_lo = blockIdx.y * k_per_split;
  const int k_hi = min(K, k_lo + k_per_split);
  if (gridDim.y > 1) Cv = reinterpret_cast<float*>(Cv) + (long)blockIdx.y * M * ldc;
  // Consecutive blocks go to the chip's 8 dies in turn, each with an L2 of its own.  Give every
  // die a contiguous range of weight tiles (columns) and let it walk the row tiles of a column
  // before the next column: a die then streams its slice of W once and re-reads only A.
  const int tiles_m = gridDim.x / tiles_n;
  int tile_m, tile_n;
  if (tiles_n % 8 == 0) {
    const int die = blockIdx.x % 8, local = blockIdx.x / 8;
    tile_n = die * (tiles_n / 8) + local / tiles_m;
    tile_m = local % tiles_m;
  } else {
    tile_m = blockIdx.x / tiles_n;
    tile_n = blockIdx.x % tiles_n;
  }
  // Grouped: the rows are sorted by group (a routed feed-forward's experts) and cut into tiles of
  // up to 128 rows of one group; tile t multiplies rows tile_row0[t] .. + tile_rows[t] - 1 with the
  // matrix of group group_of_tile[t] (W + group * group_stride).  The list lives on the device
  // and is as long as the worst case; unused entries (-1) end their blocks at once.  A group may also sit
  // at columns of its own in A and C (group * group_a_step, group * group_c_step elements into a row): a product
  // per head, whose heads lie side by side in the rows.
  if (group_of_tile) {
    const int t = blockIdx.x / tiles_n;
    const int grp = group_of_tile[t];
    if (grp < 0) return;
    const long r0 = tile_row0[t];
    tile_m = 0;
    tile_n = blockIdx.x % tiles_n;
    M = tile_rows[t];
    A += r0 * lda + grp * group_a_step;
    W += (long)grp * group_stride;
    Cv = reinterpret_cast<char*>(Cv) + (r0 * ldc + grp * group_c_step) * (EPI_HALF(EPI) || EPI_GATED(EPI) ? 2 : 4);
    if (EPI == EPI_GATE) glu.bias += r0 * glu.gate_stride + grp * group_c_step;       // a gate per column of the result's rows
  }
  const long m0 = (long)tile_m * BM, n0 = (long)tile_n * BN;

  // global -> LDS without registers in between: load instruction p of wave w fills rows
  // (4 w + p) * 8 .. + 7 of a tile, lane l the 16-byte piece l % 8 of row l / 8, which is piece
  // (l % 8) ^ ((row / 2) % 8) of the row in memory.  Rows beyond the matrix and k beyond the
  // range take an offset outside the descriptor and arrive as zeros.
  const int a_rows = (int)min((long)BM, M - m0), w_rows = (int)min((long)BN, N - n0);
#if defined(__HIP_DEVICE_COMPILE__)
  const __amdgpu_buffer_rsrc_t a_src = operand_descriptor(A, addressing::tile_descriptor(m0, lda, k_lo, k_hi, a_rows));
  const __amdgpu_buffer_rsrc_t w_src = operand_descriptor(W, addressing::tile_descriptor(n0, ldw, k_lo, k_hi, w_rows));
#endif
  unsigned a_off[4], w_off[4];
  int piece_k[4];                           // the piece (8 k) of a slab's row that this lane fetches
#pragma unroll
  for (int p = 0; p < 4; ++p) {
    const int row = (wave * 4 + p) * 8 + lane / 8;
    const int piece = addressing::tile_piece(lane, row);
    piece_k[p] = piece;
    a_off[p] = addressing::tile_lane_offset(row, a_rows, lda, piece);
    w_off[p] = addressing::tile_lane_offset(row, w_rows, ldw, piece);
  }
  typedef __attribute__((address_space(3))) void* lds_ptr_t;
  auto load_slab = [&](int k0, int buf) {
    // k0 is relative to k_lo; a lane's 8 k of the slab may lie beyond the range (last slab)
#if defined(__HIP_DEVICE_COMPILE__)
#pragma unroll
    for (int p = 0; p < 4; ++p) {
      __builtin_amdgcn_raw_ptr_buffer_load_lds(a_src, (lds_ptr_t)(As + buf * TILE + (wave * 4 + p) * 8 * ROW), 16,
                                               addressing::tile_slab_offset(a_off[p], k0, piece_k[p], k_hi - k_lo), 0, 0, 0);
      __builtin_amdgcn_raw_ptr_buffer_load_lds(w_src, (lds_ptr_t)(Ws + buf * TILE + (wave * 4 + p) * 8 * ROW), 16,
                                               addressing::tile_slab_offset(w_off[p], k0, piece_k[p], k_hi - k_lo), 0, 0, 0);
    }
#endif
  };

  f32x16_t acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[i][j][v] = 0.f;

  const int slabs = (k_hi - k_lo + BK - 1) / BK;
  // 32 x 32 x 16 instruction: a lane reads row lane % 32, the 16 bytes of k = (lane / 32) * 8 of
  // every 16 k, at the place its row's turn puts them
  const int frow = lane % 32;
  int place[4];
#pragma unroll
  for (int ks = 0; ks < 4; ++ks) place[ks] = ((ks * 2 + lane / 32) ^ ((frow >> 1) & 7)) * 8;
  Frag fa[2][2], fb[2][2];
  auto read_frags = [&](int which, int buf, int ks) {   // ks: which 16 k of the slab
    const uint16_t* a_base = As + buf * TILE + (wm * 64 + frow) * ROW + place[ks];
    const uint16_t* w_base = Ws + buf * TILE + (wn * 64 + frow) * ROW + place[ks];
#pragma unroll
    for (int i = 0; i < 2; ++i) fa[which][i].n = *reinterpret_cast<const u32x4_t*>(a_base + i * 32 * ROW);
#pragma unroll
    for (int j = 0; j < 2; ++j) fb[which][j].n = *reinterpret_cast<const u32x4_t*>(w_base + j * 32 * ROW);
  };
  auto products = [&](int which) {
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i][j] = mfma32(fa[which][i], fb[which][j], acc[i][j]);
  };
  // The loop has no branch: a slab beyond the range loads zeros (offsets out of the
  // descriptor's range) into the buffer nobody reads.  Fragments of the next 16 k are read
  // while the matrix instructions of these 16 run; the hints deal one memory instruction of
  // each kind named after every matrix instruction.
  // The loop has no branch: a slab beyond the range arrives as zeros in the buffer nobody reads.
  // Fragments of the next 16 k are read while the matrix instructions of these 16 run; the hints
  // deal one memory instruction of each kind named after every matrix instruction.
#define PI_SCHED_MFMA 0x008
#define PI_SCHED_VMEM_READ 0x020
#define PI_SCHED_DS_READ 0x100
#define PI_SCHED_DS_WRITE 0x200
#define PI_DEAL4(kind_a, kind_b)                                                     \
  _Pragma("unroll") for (int d_ = 0; d_ < 4; ++d_) {                                 \
    __builtin_amdgcn_sched_group_barrier(PI_SCHED_MFMA, 1, 0);                       \
    if (kind_a) __builtin_amdgcn_sched_group_barrier(kind_a, 1, 0);                  \
    if (kind_b) __builtin_amdgcn_sched_group_barrier(kind_b, 2, 0);                  \
  }
  load_slab(0, 0);
  __builtin_amdgcn_s_waitcnt(0x0F70);       // vmcnt(0): this wave's pieces of the slab are in LDS
  __syncthreads();
  load_slab(BK, 1);
  read_frags(0, 0, 0);
  for (int s = 0; s < slabs; ++s) {
    const int buf = s & 1;
    read_frags(1, buf, 1);
    products(0);
    PI_DEAL4(PI_SCHED_DS_READ, 0)
    read_frags(0, buf, 2);
    products(1);
    PI_DEAL4(PI_SCHED_DS_READ, 0)
    read_frags(1, buf, 3);
    products(0);
    PI_DEAL4(PI_SCHED_DS_READ, 0)
    __builtin_amdgcn_s_waitcnt(0x0F70);     // slab s + 1 has landed (asked for a whole slab ago)
    __syncthreads();
    load_slab((s + 2) * BK, buf);           // into the buffer everybody has just left; beyond the range: zeros, unused
    read_frags(0, buf ^ 1, 0);
    products(1);
    PI_DEAL4(PI_SCHED_DS_READ, PI_SCHED_VMEM_READ)
  }
  __builtin_amdgcn_s_waitcnt(0x0F70);       // nothing may still be on its way into LDS when the patches take it over
#undef PI_DEAL4
  __syncthreads();                  // the fragments read last belong to no slab; LDS is free for the patches

  // acc[i][j][v] is C[m0 + wm*64 + i*32 + 8*(v/4) + 4*(lane/32) + v%4][n0 + wn*64 + j*32 + lane%32].
  // Offsets inside the wave's corner are 32-bit (the host checks that 128 * ldc fits).
  {
    const long mw = m0 + wm * 64, nw = n0 + wn * 64;
    const int rows_left = (int)min((long)64, M - mw), cols_left = (int)min((long)64, N - nw);   // may be <= 0
    if (EPI == EPI_GATE) glu.bias += mw * glu.gate_stride + nw;
    float* patch = reinterpret_cast<float*>(lds) + wave * PATCH_FLOATS;
    const int esize = EPI_HALF(EPI) || EPI_GATED(EPI) ? 2 : 4;
    char* corner = reinterpret_cast<char*>(Cv) + (mw * ldc + (EPI_GATED(EPI) ? nw / 2 : nw)) * esize;
    const bool wide = (ldc * esize) % 16 == 0 && reinterpret_cast<uintptr_t>(corner) % 16 == 0;
#pragma unroll
    for (int i = 0; i < 2; ++i) store_rows32<EPI>(patch, acc[i][0], acc[i][1], corner, (int)ldc, i * 32, rows_left, cols_left, lane, wide, glu, nw);
  }
}

// ---------------------------------------------------------------------------------------------
// The same product with block tile 256 x 256 for problems that have enough of them to fill the
// chip and a k that is a multiple of the slab: eight waves in 2 x 4 (two per SIMD), each
// 128 x 64 as 4 x 2 tiles of v_mfma_f32_32x32x16_bf16.  Per 16 k a wave reads 6 fragments from
// LDS for 8 matrix-core instructions, three quarters of the LDS traffic per flop of the
// 128 x 128 kernel, and a block asks L2 for half the bytes per flop.  With one wave per SIMD
// (four waves of 128 x 128, the first form of this kernel) every barrier and every wait left
// the matrix pipe idle.  No branch in the loop (rows beyond the matrix are clamped on load and
// skipped on store), loads through a buffer descriptor (a scalar base that moves with k plus
// fixed 32-bit lane offsets, no vector arithmetic per slab) straight into the other LDS
// buffer, issued at the top of a slab and awaited at its one barrier, and scheduling hints that
// deal the memory instructions out between the matrix-core ones.
// Per output element the sum over k runs in ascending k, as in the small kernel.
#define GM 256
#define GN 256
#define BIG_TILE_ELEMS (GM * BK)

template <int EPI>
__global__ __launch_bounds__(512) void gemm_mfma_big_kernel(void* __restrict__ Cv, long ldc, const bf16_t* __restrict__ A, long lda,
                                                            const bf16_t* __restrict__ W, long ldw, int M, int N, int K,
                                                            int tiles_n, int k_per_split, GluArgs glu) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  constexpr int ROW = BK;                       // rows of 128 bytes, no padding: the loads write LDS themselves, lane after lane
  constexpr int TILE = GM * ROW;
  uint16_t* As = lds;                           // [2][GM][ROW], 16-byte pieces of a row turned by (row / 2) % 8
  uint16_t* Ws = lds + 2 * TILE;                // [2][GN][ROW]
  const int tid = threadIdx.x, lane = tid % 64;
  const int wave = __builtin_amdgcn_readfirstlane(tid / 64);
  const int wm = wave / 4, wn = wave % 4;       // a wave's corner: 128 rows x 64 columns
  const int k_lo = blockIdx.y * k_per_split;
  const int k_hi = min(K, k_lo + k_per_split);
  if (gridDim.y > 1) Cv = reinterpret_cast<float*>(Cv) + (long)blockIdx.y * M * ldc;
  const int tiles_m = gridDim.x / tiles_n;
  int tile_m, tile_n;
  if (tiles_n % 8 == 0) {                       // a die streams its own slice of W, see above
    const int die = blockIdx.x % 8, local = blockIdx.x / 8;
    tile_n = die * (tiles_n / 8) + local / tiles_m;
    tile_m = local % tiles_m;
  } else {
    tile_m = blockIdx.x / tiles_n;
    tile_n = blockIdx.x % tiles_n;
  }
  const long m0 = (long)tile_m * GM, n0 = (long)tile_n * GN;

  // global -> LDS without registers in between: load instruction p of wave w fills rows
  // (4 w + p) * 8 .. + 7 of a tile, lane l the 16-byte piece l % 8 of row l / 8.  Which piece of
  // the row in memory that is depends on the row: piece c of row r lies at place c ^ ((r / 2) % 8),
  // so that the fragment reads of sixteen neighbouring rows fall on all 64 banks.
  const int a_rows = (int)min((long)GM, M - m0), w_rows = (int)min((long)GN, N - n0);
#if defined(__HIP_DEVICE_COMPILE__)
  const __amdgpu_buffer_rsrc_t a_src = operand_descriptor(A, addressing::tile_descriptor(m0, lda, k_lo, k_hi, a_rows));
  const __amdgpu_buffer_rsrc_t w_src = operand_descriptor(W, addressing::tile_descriptor(n0, ldw, k_lo, k_hi, w_rows));
#endif
  unsigned a_off[4], w_off[4];
#pragma unroll
  for (int p = 0; p < 4; ++p) {
    const int row = (wave * 4 + p) * 8 + lane / 8;
    const int piece = addressing::tile_piece(lane, row);
    a_off[p] = addressing::big_lane_offset(row, a_rows, lda, piece);
    w_off[p] = addressing::big_lane_offset(row, w_rows, ldw, piece);
  }
  const int slabs = (k_hi - k_lo) / BK;
  typedef __attribute__((address_space(3))) void* lds_ptr_t;
  auto load_slab = [&](int s, int buf) {
    const int kbytes = addressing::big_slab_bytes(s, slabs);     // past the last slab: read it again, unused
#if defined(__HIP_DEVICE_COMPILE__)
#pragma unroll
    for (int p = 0; p < 4; ++p) {
      __builtin_amdgcn_raw_ptr_buffer_load_lds(a_src, (lds_ptr_t)(As + buf * TILE + (wave * 4 + p) * 8 * ROW), 16, a_off[p], kbytes, 0, 0);
      __builtin_amdgcn_raw_ptr_buffer_load_lds(w_src, (lds_ptr_t)(Ws + buf * TILE + (wave * 4 + p) * 8 * ROW), 16, w_off[p], kbytes, 0, 0);
    }
#endif
  };

  f32x16_t acc[4][2];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[i][j][v] = 0.f;

  const int frow = lane % 32;
  int place[4];                                  // where this lane's piece of each 16 k lies in its rows
#pragma unroll
  for (int ks = 0; ks < 4; ++ks) place[ks] = ((ks * 2 + lane / 32) ^ ((frow >> 1) & 7)) * 8;
  Frag fa[2][4], fb[2][2];
  auto read_frags = [&](int which, int buf, int ks) {   // ks: which 16 k of the slab
    const uint16_t* a_base = As + buf * TILE + (wm * 128 + frow) * ROW + place[ks];
    const uint16_t* w_base = Ws + buf * TILE + (wn * 64 + frow) * ROW + place[ks];
#pragma unroll
    for (int i = 0; i < 4; ++i) fa[which][i].n = *reinterpret_cast<const u32x4_t*>(a_base + i * 32 * ROW);
#pragma unroll
    for (int j = 0; j < 2; ++j) fb[which][j].n = *reinterpret_cast<const u32x4_t*>(w_base + j * 32 * ROW);
  };
  auto products = [&](int which) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i][j] = mfma32(fa[which][i], fb[which][j], acc[i][j]);
  };

  load_slab(0, 0);
  __builtin_amdgcn_s_waitcnt(0x0F70);           // vmcnt(0): this wave's pieces of the slab are in LDS
  __syncthreads();
  read_frags(0, 0, 0);
  // the order wanted inside one scheduling region: one matrix-core instruction, then one of
  // each kind of memory instruction named, `n` times; the rest of the 8 after that
#define PI_DEAL(n, kind_a, kind_b)                                                   \
  _Pragma("unroll") for (int d_ = 0; d_ < n; ++d_) {                                 \
    __builtin_amdgcn_sched_group_barrier(PI_SCHED_MFMA, 1, 0);                       \
    if (kind_a) __builtin_amdgcn_sched_group_barrier(kind_a, 1, 0);                  \
    if (kind_b) __builtin_amdgcn_sched_group_barrier(kind_b, 1, 0);                  \
  }
  load_slab(1, 1);
  for (int s = 0; s < slabs; ++s) {
    const int buf = s & 1;
    read_frags(1, buf, 1);
    products(0);
    PI_DEAL(6, PI_SCHED_DS_READ, 0)
    PI_DEAL(2, 0, 0)
    read_frags(0, buf, 2);
    products(1);
    PI_DEAL(6, PI_SCHED_DS_READ, 0)
    PI_DEAL(2, 0, 0)
    read_frags(1, buf, 3);
    products(0);
    PI_DEAL(6, PI_SCHED_DS_READ, 0)
    PI_DEAL(2, 0, 0)
    __builtin_amdgcn_s_waitcnt(0x0F70);     // slab s + 1 has landed (asked for a whole slab ago)
    __syncthreads();
    load_slab(s + 2, buf);          // into the buffer everybody has just left
    read_frags(0, buf ^ 1, 0);
    products(1);
    PI_DEAL(6, PI_SCHED_DS_READ, PI_SCHED_VMEM_READ)
    PI_DEAL(2, PI_SCHED_VMEM_READ, 0)
  }
  __builtin_amdgcn_s_waitcnt(0x0F70);       // nothing may still be on its way into LDS when the patches take it over
#undef PI_DEAL

  // acc[i][j][v] is C[m0 + wm*128 + i*32 + 8*(v/4) + 4*(lane/32) + v%4][n0 + wn*64 + j*32 + lane%32].
  // Offsets inside the wave's corner are 32-bit (the host checks that 128 * ldc fits).
  __syncthreads();                              // LDS is free for the waves' patches
  {
    const long mw = m0 + wm * 128, nw = n0 + wn * 64;
    const int rows_left = (int)min((long)128, M - mw), cols_left = (int)min((long)64, N - nw);   // may be <= 0
    if (EPI == EPI_GATE) glu.bias += mw * glu.gate_stride + nw;
    float* patch = reinterpret_cast<float*>(lds) + wave * PATCH_FLOATS;
    const int esize = EPI_HALF(EPI) || EPI_GATED(EPI) ? 2 : 4;
    char* corner = reinterpret_cast<char*>(Cv) + (mw * ldc + (EPI_GATED(EPI) ? nw / 2 : nw)) * esize;
    const bool wide = (ldc * esize) % 16 == 0 && reinterpret_cast<uintptr_t>(corner) % 16 == 0;
#pragma unroll
    for (int i = 0; i < 4; ++i) store_rows32<EPI>(patch, acc[i][0], acc[i][1], corner, (int)ldc, i * 32, rows_left, cols_left, lane, wide, glu, nw);
  }
}

static const size_t kBigLdsBytes = 4 * BIG_TILE_ELEMS * sizeof(uint16_t);   // 131,072 bytes
// enough 256 x 256 tiles (times k pieces) to occupy most of the chip: three quarters of its compute units
static int big_min_tiles() {
  static int units = 0;
  if (units == 0) {
    int device = 0, count = 0;
    if (hipGetDevice(&device) != hipSuccess || hipDeviceGetAttribute(&count, hipDeviceAttributeMultiprocessorCount, device) != hipSuccess || count <= 0)
      count = 256;
    units = count;
  }
  return units * 3 / 4;
}

static const size_t kLdsBytes = 4 * TILE_ELEMS * sizeof(uint16_t);   // 65,536 bytes

template <int EPI>
static int launch(void* C, long ldc, const void* A, long lda, const void* W, long ldw, int M, int N, int K, int splits,
                  hipStream_t stream, GluArgs glu = GluArgs{nullptr, 0.f, 0.f, 0}) {
  static bool configured = false;
  if (!configured) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(gemm_mfma_kernel<EPI>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsBytes);
    if (e != hipSuccess) return pi_fail("gemm_mfma: cannot reserve %zu bytes of LDS: %s", kLdsBytes, hipGetErrorString(e));
    configured = true;
  }
  const addressing::KSplit cut = addressing::cut_k(K, splits, BK);
  const int kps = cut.k_per_block;
  splits = cut.splits;
  const long big_tiles = (long)ceil_div(M, GM) * ceil_div(N, GN);
  if (big_tiles * splits >= big_min_tiles() && big_tiles < 2147483647L && K % BK == 0) {
    static bool big_configured = false;
    if (!big_configured) {
      hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(gemm_mfma_big_kernel<EPI>),
                                         hipFuncAttributeMaxDynamicSharedMemorySize, (int)kBigLdsBytes);
      if (e != hipSuccess) return pi_fail("gemm_mfma: cannot reserve %zu bytes of LDS: %s", kBigLdsBytes, hipGetErrorString(e));
      big_configured = true;
    }
    hipLaunchKernelGGL((gemm_mfma_big_kernel<EPI>), dim3((unsigned)big_tiles, splits), dim3(512), kBigLdsBytes, stream, C, ldc,
                       (const bf16_t*)A, lda, (const bf16_t*)W, ldw, M, N, K, ceil_div(N, GN), kps, glu);
    return pi_check_launch("gemm_mfma_big");
  }
  const int tiles_m = ceil_div(M, BM), tiles_n = ceil_div(N, BN);
  hipLaunchKernelGGL((gemm_mfma_kernel<EPI>), dim3((unsigned)tiles_m * tiles_n, splits), dim3(256), kLdsBytes, stream, C, ldc,
                     (const bf16_t*)A, lda, (const bf16_t*)W, ldw, M, N, K, tiles_n, kps, (const int*)nullptr, (const int*)nullptr,
                     (const int*)nullptr, 0L, 0L, 0L, glu);
  return pi_check_launch("gemm_mfma");
}

// Rows of a grouped product's tiles (the 128 x 128 kernel's block tile).
extern "C" int pi_gemm_mfma_group_tile_rows() { return BM; }

// C[row, :] = A[row, :] . W[group of row]^T over a device-side list of `tiles` row tiles (see the
// kernel); W is [groups, N, K] with `group_stride` elements from one group's matrix to the next.
// epilogue: 0 store bf16, 1 store f32, 3 SwiGLU (every group's rows interleaved by 16; C is [rows, N / 2] bf16), 4 the clamped
// gated unit without biases (rows as for 3; `limit` and `alpha`), 5 max(c, 0)^2 as bf16, 7 c * sigmoid(gate) as bf16 (`gate`
// float32, rows `gate_stride` apart, a gate per column of C's rows).
template <int EPI>
static int launch_grouped(void* C, long ldc, const void* A, long lda, const void* W, long ldw, long group_stride,
                          const int* group_of_tile, const int* tile_row0, const int* tile_rows, int tiles, int N, int K,
                          long group_a_step, long group_c_step, hipStream_t stream, GluArgs glu = GluArgs{nullptr, 0.f, 0.f, 0}) {
  static bool configured = false;
  if (!configured) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(gemm_mfma_kernel<EPI>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsBytes);
    if (e != hipSuccess) return pi_fail("gemm_mfma: cannot reserve %zu bytes of LDS: %s", kLdsBytes, hipGetErrorString(e));
    configured = true;
  }
  const int tiles_n = ceil_div(N, BN);
  hipLaunchKernelGGL((gemm_mfma_kernel<EPI>), dim3((unsigned)tiles * tiles_n, 1), dim3(256), kLdsBytes, stream, C, ldc,
                     (const bf16_t*)A, lda, (const bf16_t*)W, ldw, BM, N, K, tiles_n, K, group_of_tile, tile_row0, tile_rows,
                     group_stride, group_a_step, group_c_step, glu);
  return pi_check_launch("gemm_mfma_grouped");
}

extern "C" int pi_gemm_mfma_grouped(void* C, int epilogue, long ldc, const void* A, long lda, const void* W, long ldw,
                                    long group_stride, const int* group_of_tile, const int* tile_row0, const int* tile_rows,
                                    int tiles, int N, int K, long group_a_step, long group_c_step, float limit, float alpha,
                                    const float* gate, long gate_stride, hipStream_t stream) {
  PI_REQUIRE(tiles >= 0 && N > 0 && K > 0, "gemm_mfma_grouped: bad sizes tiles=%d N=%d K=%d", tiles, N, K);
  PI_REQUIRE(group_a_step >= 0 && group_c_step >= 0 && group_a_step % 8 == 0 && group_c_step % 8 == 0,
             "gemm_mfma_grouped: a group's columns in the rows (%ld, %ld) must start at multiples of 8", group_a_step, group_c_step);
  PI_REQUIRE(group_c_step == 0 || epilogue == EPI_BF16 || epilogue == EPI_F32 || epilogue == EPI_GATE, "gemm_mfma_grouped: groups side by side in the result's rows store plainly");
  PI_REQUIRE(K % 8 == 0 && lda % 8 == 0 && ldw % 8 == 0 && group_stride % 8 == 0, "gemm_mfma_grouped: K (%d) and strides must be multiples of 8", K);
  PI_REQUIRE(256 * lda < (1L << 29) && 256 * ldw < (1L << 29), "gemm_mfma_grouped: row strides (%ld, %ld) are too long", lda, ldw);
  PI_REQUIRE(ldc > 0 && ldc < (1L << 23), "gemm_mfma_grouped: the result's row stride (%ld) is too long", ldc);
  PI_REQUIRE(((uintptr_t)A % 16 == 0) && ((uintptr_t)W % 16 == 0), "gemm_mfma_grouped: operands must be 16-byte aligned");
  PI_REQUIRE(!EPI_GATED(epilogue) || N % 32 == 0, "gemm_mfma_grouped: the gated epilogues need N (%d) to be a multiple of 32", N);
  PI_REQUIRE((long)tiles * ceil_div(N, BN) < 2147483647L, "gemm_mfma_grouped: too many tiles");
  PI_REQUIRE(group_of_tile && tile_row0 && tile_rows, "gemm_mfma_grouped: the tile list is missing");
  PI_REQUIRE(epilogue != EPI_GATE || (gate && gate_stride > 0), "gemm_mfma_grouped: the gates are missing");
  if (tiles == 0) return 0;
  switch (epilogue) {
    case EPI_BF16: return launch_grouped<EPI_BF16>(C, ldc, A, lda, W, ldw, group_stride, group_of_tile, tile_row0, tile_rows, tiles, N, K, group_a_step, group_c_step, stream);
    case EPI_F32: return launch_grouped<EPI_F32>(C, ldc, A, lda, W, ldw, group_stride, group_of_tile, tile_row0, tile_rows, tiles, N, K, group_a_step, group_c_step, stream);
    case EPI_CLAMPED_GLU: return launch_grouped<EPI_CLAMPED_GLU>(C, ldc, A, lda, W, ldw, group_stride, group_of_tile, tile_row0, tile_rows, tiles, N, K, group_a_step, group_c_step, stream, GluArgs{nullptr, limit, alpha, 0});
    case EPI_GATE: return launch_grouped<EPI_GATE>(C, ldc, A, lda, W, ldw, group_stride, group_of_tile, tile_row0, tile_rows, tiles, N, K, group_a_step, group_c_step, stream, GluArgs{gate, 0.f, 0.f, gate_stride});
    case EPI_RELU2: return launch_grouped<EPI_RELU2>(C, ldc, A, lda, W, ldw, group_stride, group_of_tile, tile_row0, tile_rows, tiles, N, K, group_a_step, group_c_step, stream);
    case EPI_SWIGLU: return launch_grouped<EPI_SWIGLU>(C, ldc, A, lda, W, ldw, group_stride, group_of_tile, tile_row0, tile_rows, tiles, N, K, group_a_step, group_c_step, stream);
  }
  return pi_fail("gemm_mfma_grouped: unknown epilogue %d", epilogue);
}

// Pieces a k-split into `splits` makes (the kernel rounds a split's range up to whole slabs).
extern "C" int pi_gemm_mfma_pieces(int K, int splits) {
  if (splits < 1 || K < 1) return 0;
  return addressing::cut_k(K, splits, BK).splits;
}

// epilogue: 0 store bf16, 1 store f32, 2 add into f32, 3 SwiGLU (W rows interleaved by 16; C is [M, N / 2] bf16),
// 5 store max(c, 0)^2 as bf16, 6 store the exact gelu of c as bf16
extern "C" int pi_gemm_mfma(void* C, int epilogue, long ldc, const void* A, long lda, const void* W, long ldw, int M,
                            int N, int K, int splits, hipStream_t stream) {
  PI_REQUIRE(M > 0 && N > 0 && K > 0, "gemm_mfma: bad sizes M=%d N=%d K=%d", M, N, K);
  // splits > 1: C is a float32 workspace [splits, M, N] (ldc = N) that receives the pieces; the
  // number of pieces is ceil(K / (ceil(K / splits) rounded up to 64))
  PI_REQUIRE(splits >= 1 && splits <= 64 && (splits == 1 || (epilogue == EPI_F32 && ldc == N)),
             "gemm_mfma: a k-split (%d) needs the float32 store into a [splits, M, N] workspace", splits);
  PI_REQUIRE(K % 8 == 0 && lda % 8 == 0 && ldw % 8 == 0, "gemm_mfma: K (%d) and row strides (%ld, %ld) must be multiples of 8", K, lda, ldw);
  PI_REQUIRE(256 * lda < (1L << 29) && 256 * ldw < (1L << 29), "gemm_mfma: row strides (%ld, %ld) are too long for 32-bit offsets inside a tile", lda, ldw);
  PI_REQUIRE(ldc > 0 && ldc < (1L << 23), "gemm_mfma: the result's row stride (%ld) is too long for 32-bit offsets inside a tile", ldc);
  PI_REQUIRE(((uintptr_t)A % 16 == 0) && ((uintptr_t)W % 16 == 0), "gemm_mfma: operands must be 16-byte aligned");
  PI_REQUIRE(epilogue != EPI_SWIGLU || N % 32 == 0, "gemm_mfma: the SwiGLU epilogue needs N (%d) to be a multiple of 32", N);
  PI_REQUIRE((long)ceil_div(M, BM) * ceil_div(N, BN) < 2147483647L, "gemm_mfma: too many tiles");
  switch (epilogue) {
    case EPI_BF16: return launch<EPI_BF16>(C, ldc, A, lda, W, ldw, M, N, K, splits, stream);
    case EPI_F32: return launch<EPI_F32>(C, ldc, A, lda, W, ldw, M, N, K, splits, stream);
    case EPI_ACCUM: return launch<EPI_ACCUM>(C, ldc, A, lda, W, ldw, M, N, K, splits, stream);
    case EPI_RELU2: return launch<EPI_RELU2>(C, ldc, A, lda, W, ldw, M, N, K, splits, stream);
    case EPI_GELU: return launch<EPI_GELU>(C, ldc, A, lda, W, ldw, M, N, K, splits, stream);
    case EPI_SWIGLU: return launch<EPI_SWIGLU>(C, ldc, A, lda, W, ldw, M, N, K, splits, stream);
  }
  return pi_fail("gemm_mfma: unknown epilogue %d", epilogue);
}

// C[M, N / 2] (bfloat16) = the clamped gated unit of A . W^T: W's rows and `bias` (float32 [N]) hold gate and up
// interleaved by 16; g' = min(g + bg, limit), u' = clamp(u + bu, -limit, limit), g' * sigmoid(alpha * g') * (u' + 1).
extern "C" int pi_gemm_mfma_clamped_glu(void* C, long ldc, const void* A, long lda, const void* W, long ldw, int M, int N, int K,
                                        const float* bias, float limit, float alpha, hipStream_t stream) {
  PI_REQUIRE(M > 0 && N > 0 && K > 0 && bias, "gemm_mfma: bad sizes M=%d N=%d K=%d", M, N, K);
  PI_REQUIRE(K % 8 == 0 && lda % 8 == 0 && ldw % 8 == 0, "gemm_mfma: K (%d) and row strides (%ld, %ld) must be multiples of 8", K, lda, ldw);
  PI_REQUIRE(256 * lda < (1L << 29) && 256 * ldw < (1L << 29), "gemm_mfma: row strides (%ld, %ld) are too long for 32-bit offsets inside a tile", lda, ldw);
  PI_REQUIRE(ldc > 0 && ldc < (1L << 23), "gemm_mfma: the result's row stride (%ld) is too long for 32-bit offsets inside a tile", ldc);
  PI_REQUIRE(((uintptr_t)A % 16 == 0) && ((uintptr_t)W % 16 == 0), "gemm_mfma: operands must be 16-byte aligned");
  PI_REQUIRE(N % 32 == 0, "gemm_mfma: the gated epilogue needs N (%d) to be a multiple of 32", N);
  PI_REQUIRE((long)ceil_div(M, BM) * ceil_div(N, BN) < 2147483647L, "gemm_mfma: too many tiles");
  return launch<EPI_CLAMPED_GLU>(C, ldc, A, lda, W, ldw, M, N, K, 1, stream, GluArgs{bias, limit, alpha, 0});
}
