// gemm_bf16.hpp -- rows x bfloat16 weights on the matrix cores: the prompt-time linear of the hybrid decoder.
//
//   C[row][n] = sum_k A[row][k] W[n][k]     A: bf16 planes, W: bf16 rows, f32 accumulation (v_mfma_f32_16x16x32_bf16)
//
// One plane of A is bf16 arithmetic.  Three planes are a row of f32 numbers cut into its upper, middle and lower eight significand
// bits (split3): every f32 is the exact sum of its planes and every plane times a bf16 weight is exact in f32, so three planes give
// true f32 products with f32 sums -- the weights ARE bf16 numbers -- at a fifth of the time the f32 matrix instruction would take.
//
// Mapping: BM x 128 output tile per workgroup (BM = 256: eight waves; else four), k in steps of 64.  A step's tiles go from memory
// straight into LDS (global_load_lds, 16 bytes per lane); three or four steps are in LDS or on their way, and a wave waits for the oldest
// only (s_waitcnt vmcnt(n)).  LDS holds rows of 128 bytes whose 16-byte chunks are permuted by (row / 2) % 8 -- on the SOURCE side, the LDS side of the instruction
// being linear -- so that the 16 rows a fragment read touches spread over all 64 banks.  Operands are padded by their owners (k to 64,
// weight rows to 256, activation rows to 256), so the loop has no bounds checks; stores have.  Short launches cut k into pieces (the
// last workgroup of a tile adds them).  Workgroups are dealt to the eight XCDs
// in contiguous runs of the tile order, row tiles fastest: an XCD's L2 keeps the weight tile that its row tiles share.
//
// The row operations around a linear are folded into it.  In: an RMS norm with a single gain is a factor per row, applied to the
// accumulators (the producers leave each row's sum of squares in 64-column pieces); a gain per column is in the planes already.  Out:
// activations by column range, xIELU, a gated unit, soft cap, or the residual add (of one stream or of several that mix), which also
// leaves the new row's bf16 planes and square sums for the next linear.
#pragma once
#include "gemv_bf16.hpp"

namespace crabml_hip {

typedef unsigned short u16x4 __attribute__((ext_vector_type(4)));

enum {
  GEMM_OUT_ACT_BF16 = 0,   // rows of bf16 (ActRanges)
  GEMM_OUT_ACT_F32 = 1,    // rows of f32 (ActRanges)
  GEMM_OUT_RESIDUAL = 2,   // x += acc (+ add_rows + add_vec); planes of x; square sums
  GEMM_OUT_XIELU = 3,      // planes of xielu(acc)
  GEMM_OUT_SOFTCAP = 4,    // f32 rows
  GEMM_OUT_STREAMS = 5,    // the residual streams take acc (+ bias); planes of gain_next * what the next linear reads; its square sums
  GEMM_OUT_GLU = 6,        // weight rows 2 j, 2 j + 1 are gate j and up j: planes of gelu(gate) * up
};

// an f32 as bf16 planes: 1 plane = rounded to nearest even; 3 planes = upper / middle / lower bits, their sum exact
template <int P>
__device__ __forceinline__ void split_store(float v, unsigned short* p, size_t plane_stride) {
  if constexpr (P == 1) {
    *p = f2bf(v);
  } else {
    const float hi = __builtin_bit_cast(float, __builtin_bit_cast(unsigned, v) & 0xffff0000u);
    const float r = v - hi;  // exact: the low 16 bits of the significand
    const float mid = __builtin_bit_cast(float, __builtin_bit_cast(unsigned, r) & 0xffff0000u);
    p[0] = (unsigned short)(__builtin_bit_cast(unsigned, hi) >> 16);
    p[plane_stride] = (unsigned short)(__builtin_bit_cast(unsigned, mid) >> 16);
    p[2 * plane_stride] = f2bf(r - mid);
  }
}

// four neighbouring columns at once (p: 8-byte aligned)
template <int P>
__device__ __forceinline__ void split_store4(const float (&v)[4], unsigned short* p, size_t plane_stride) {
  unsigned short t[P][4];
#pragma unroll
  for (int e = 0; e < 4; e++) split_store<P>(v[e], &t[0][e], 4);
#pragma unroll
  for (int i = 0; i < P; i++) __builtin_memcpy(p + i * plane_stride, t[i], 8);
}

// eight of them (p: 16-byte aligned)
template <int P>
__device__ __forceinline__ void split_store8(const float (&v)[8], unsigned short* p, size_t plane_stride) {
  unsigned short t[P][8];
#pragma unroll
  for (int e = 0; e < 8; e++) split_store<P>(v[e], &t[0][e], 8);
#pragma unroll
  for (int i = 0; i < P; i++) {
    i32x4 w;
    __builtin_memcpy(&w, t[i], 16);
    *(i32x4*)(p + i * plane_stride) = w;
  }
}
__device__ __forceinline__ void read8(const float* p, float (&o)[8]) {
  const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
#pragma unroll
  for (int e = 0; e < 4; e++) {
    o[e] = a[e];
    o[e + 4] = b[e];
  }
}

struct GemmBf16 {
  const unsigned short* a = nullptr;  // [planes][rows padded][k]
  size_t a_plane = 0;                 // elements between planes
  const unsigned short* w = nullptr;  // [N padded][k]
  int M = 0, N = 0, K = 0;            // K % 64 == 0
  // row factor (nullable sq): gain (nullable: 1) / sqrt(sum_i sq[row][i] / mean_n + eps)
  const float* sq_in = nullptr;
  int n_sq = 0, mean_n = 1;
  float eps = 0.f;
  const float* gain = nullptr;
  // outputs
  void* out = nullptr;  // ACT / SOFTCAP rows
  int ldo = 0;
  ActRanges act;
  const float* xielu = nullptr;
  float cap = 0.f;
  const float* bias = nullptr;  // [N padded to 8], nullable (ACT, STREAMS)
  float* x = nullptr;           // RESIDUAL; STREAMS: stream 0
  StreamMix sm;
  const float* gain_next = nullptr;  // STREAMS: a gain per column of the next RMS norm
  int ldx = 0;
  const float *add_rows = nullptr, *add_vec = nullptr;
  unsigned short* planes = nullptr;  // RESIDUAL / STREAMS / XIELU / GLU: [planes][rows padded][ldp]
  size_t p_plane = 0;
  int ldp = 0;
  float* sq_out = nullptr;  // [row][n_sq_out]: square sums by 64 columns
  int n_sq_out = 0;
};

// room for k pieces: partial tiles, and a zeroed counter per tile
#define GEMM_TICKS 4096
struct GemmScratch {
  float* partials = nullptr;
  size_t floats = 0;
  unsigned* ticks = nullptr;
};
// planes: 1 or 3 (GEMM_OUT_ACT_BF16 goes with one, GEMM_OUT_ACT_F32 with three)
void launch_gemm_bf16(crabml_hip_device* dev, crabml_hip_device::ProfRec* rec, int planes, int out, const GemmBf16& g, const GemmScratch& w);

}  // namespace crabml_hip
