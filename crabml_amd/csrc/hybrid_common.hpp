// hybrid_common.hpp -- what the prompt pass (hybrid_rows.hpp) and the decode step (hybrid_step.hpp) of the hybrid decoder share:
// the per-sequence state's layout, a layer's geometry, the embedding.
//
// Mixers:
//   softmax attention inside chunks or a sliding window: grouped queries, and, each optional, an RMS norm over all of a token's queries
//   (keys), a log-distance penalty per head, a sink logit per head, an output gate per element or per head, values mixed with those of an
//   earlier layer
//   its latent form: keys and values are products of one normed latent row per token (and one rotated key part shared by all heads),
//   which is all that is cached (hybrid_latent.hpp)
//   linear attention with decay: S <- d S + k v^T, o = S^T q, one f32 state per head; usable beside attention in the same layer
#pragma once
#include "gemm_bf16.hpp"

namespace crabml_hip {

// KV cache element: f32, or bf16 rounded to nearest even
template <typename T>
__device__ __forceinline__ T kv_from(float f);
template <>
__device__ __forceinline__ float kv_from<float>(float f) { return f; }
template <>
__device__ __forceinline__ unsigned short kv_from<unsigned short>(float f) { return f2bf(f); }
__device__ __forceinline__ float kv_to(float v) { return v; }
__device__ __forceinline__ float kv_to(unsigned short v) { return bf2f(v); }
// eight consecutive elements (16-byte aligned rows)
__device__ __forceinline__ void kv_load8(const float* p, float (&o)[8]) { read8(p, o); }
__device__ __forceinline__ void kv_load8(const unsigned short* p, float (&o)[8]) {
  const i32x4 a = *(const i32x4*)p;
#pragma unroll
  for (int e = 0; e < 4; e++) {
    o[2 * e] = __builtin_bit_cast(float, (unsigned)a[e] << 16);
    o[2 * e + 1] = __builtin_bit_cast(float, (unsigned)a[e] & 0xffff0000u);
  }
}

template <typename T>
struct Oct {  // eight elements on their way from memory to LDS
  i32x4 d[sizeof(T) / 2];
};
template <typename T>
__device__ __forceinline__ Oct<T> oct_zero() {
  Oct<T> o;
#pragma unroll
  for (unsigned i = 0; i < sizeof(T) / 2; i++) o.d[i] = i32x4{0, 0, 0, 0};
  return o;
}
template <typename T>
__device__ __forceinline__ Oct<T> oct_load(const T* p) {
  Oct<T> o;
#pragma unroll
  for (unsigned i = 0; i < sizeof(T) / 2; i++) o.d[i] = ((const i32x4*)p)[i];
  return o;
}
template <typename T>
__device__ __forceinline__ void oct_store(T* p, const Oct<T>& o) {
#pragma unroll
  for (unsigned i = 0; i < sizeof(T) / 2; i++) ((i32x4*)p)[i] = o.d[i];
}
template <typename T>
__device__ __forceinline__ void oct_scatter(T* p, int stride, const Oct<T>& o) {  // element e -> p[e * stride]
  T v[8];
  __builtin_memcpy(v, &o, sizeof v);
#pragma unroll
  for (int e = 0; e < 8; e++) p[e * stride] = v[e];
}
template <typename T>
__device__ __forceinline__ void oct_floats(const Oct<T>& o, float (&f)[8]) {
  if constexpr (sizeof(T) == 4) {
    __builtin_memcpy(f, &o, sizeof f);
  } else {
#pragma unroll
    for (int e = 0; e < 4; e++) {
      f[2 * e] = __builtin_bit_cast(float, (unsigned)o.d[0][e] << 16);
      f[2 * e + 1] = __builtin_bit_cast(float, (unsigned)o.d[0][e] & 0xffff0000u);
    }
  }
}

// One layer's mixers.  Head widths are padded to multiples of 8 (zero weight rows make the padding zero), so every head starts on a
// 16-byte boundary of its row; D / V / ... below are the padded widths.
enum { GATE_NONE = 0, GATE_ELEMENT = 1, GATE_HEAD = 2 };
enum { VMIX_NONE = 0, VMIX_KEEP = 1, VMIX_MIX = 2 };  // KEEP: this layer's values are the ones that later layers mix into theirs
struct AttnGeom {
  int H = 0, G = 0, D = 0, V = 0;
  int span = 0;     // positions per chunk, or of the window (a token itself and the span - 1 before it)
  int window = 0;   // 0: chunks counted from the sequence's start
  int rows = 0;     // cache rows per sequence: position p lives in row p % span, so min(span, longest sequence) of them
  int gate = GATE_NONE, vmix = VMIX_NONE;
  int q_mean = 0, k_mean = 0;  // unpadded widths that the norms of q and k average over
  float eps = 0.f;
  const float *q_norm = nullptr, *k_norm = nullptr;  // [H * D], [G * D] (nullable): gains of the norms
  const float* lambda = nullptr;                     // VMIX_MIX: v <- (1 - lambda) v + lambda v_kept
  float scale = 0.f, out_scale = 1.f;
  int cq = 0, ck = 0, cv = 0, cg = 0;  // columns of the projected row
  const float *amp = nullptr, *rate = nullptr, *sink = nullptr;  // per head (nullable): penalty amp ln(1 + rate d), sink logit
};
// first position that a query sees
__host__ __device__ inline int attn_first(const AttnGeom& g, int pos) {
  if (g.window) return pos >= g.span ? pos - g.span + 1 : 0;
  return pos - pos % g.span;
}
// Latent attention (beside an AttnGeom with G = H, D = dim + rot): per head q = [dim, rot], the key's first part and the value are
// products of the latent, its second part is shared.  A cache row is [rank, rot].
struct LatGeom {
  int rank = 0, dim = 0, rot = 0;  // padded to 8
  int rank_true = 0;               // what the latent's norm averages over
  int ldl = 0;                     // rank padded to 64: the latent as a row operand
  int cc = 0, cr = 0;              // columns of the projected row: latent, shared key part
  const float* norm = nullptr;     // [rank]
  const double* freq = nullptr;    // [rot / 2]: pair (2 i, 2 i + 1) turns by position * freq[i]
  const unsigned short* w_q = nullptr;   // [H][rank][dim]: the key matrix transposed, for queries that read latents
  const unsigned short* w_kv = nullptr;  // [H * dim + H * V][ldl]: keys, then values
};
struct LinGeom {
  int H = 0, D = 0, V = 0;
  int v_true = 0;  // unpadded value width: what the norm averages over is H * v_true
  float out_scale = 1.f;
  int cq = 0, ck = 0, cv = 0, cg = 0;
  int slices = 0;                // value columns are independent: slices of 32 per workgroup
  const float* decay = nullptr;  // [H][LIN_POW] decay^n
  const float* norm = nullptr;   // [H * V]
};
#define LIN_POW 65
#define LIN_SLICE 32
// where a layer run keeps its share of a sequence's state (byte offsets into the sequence's slab)
struct RunState {
  size_t k = 0, v = 0, s = 0;
};

__device__ __forceinline__ float reduced_angle(int pos, double freq) {  // pos * freq inside [-pi, pi]
  const double turns = (double)pos * freq * 0.15915494309189533577;
  return (float)((turns - rint(turns)) * 6.28318530717958647692);
}
// ---- embedding: row * scale, plus interleaved sin / cos of the position where the design has them (freq nullable) -----------------
// freq[c / 2] in f64: the angle is formed and reduced in f64, its sine taken in f32
__device__ __forceinline__ float position_entry(int pos, int c, const double* __restrict__ freq) {
  if (!freq) return 0.f;
  const float r = reduced_angle(pos, freq[c >> 1]);
  return (c & 1) ? cosf(r) : sinf(r);
}

}  // namespace crabml_hip
