// gemv_bf16.hpp -- bfloat16 weight rows x f32 activations for up to 8 rows of the rhs at a time, with the neighbouring row
// operations folded into its two ends: the decode-time linear of the hybrid decoder (hybrid_step.hpp), and matmul_vec on BF16.
//
// Mapping: a wave owns R consecutive output rows and strides k 512 elements at a time (8 per lane = one aligned 16-byte request per
// row); the rhs rows sit in LDS as f32 in two half-octet planes, so the two ds_read_b128 a lane needs are contiguous across the wave.
// Weights become f32 by a shift / mask, products and sums are f32 fmas: the rhs is never rounded.  The weight requests of a block
// of steps go out before the activations are staged (the first block) or while the previous block is multiplied.  One pass over the
// weights serves NB rhs rows; more rows are further grid rows (blockIdx.y) that hit the same weights in L2 / Infinity Cache.
#pragma once
#include "devutil.hpp"
#include "kernels.hpp"

namespace crabml_hip {

// what happens to an rhs row on the way in
enum {
  GEMV_IN_PLAIN = 0,
  GEMV_IN_RMS = 1,    // the row is RMS-normalized with a single gain.  The row factor is taken from the staged row itself and
                      // applied to the finished dots: W (s x) = s (W x)
  GEMV_IN_SPLIT = 2,  // elements from k_split on still want their RMS normalization; their sum of squares arrives in pieces (ss)
  GEMV_IN_RMSV = 3,   // GEMV_IN_RMS with a gain per element (gain: K numbers), applied while the row is staged
};
// what happens to a dot product on the way out
enum {
  GEMV_OUT_STORE = 0,
  GEMV_OUT_ACT = 1,      // (+ bias) column ranges with their own activation (ActRanges)
  GEMV_OUT_RESIDUAL = 2, // out += dot (+ add_rows[b] + add_vec)
  GEMV_OUT_XIELU = 3,    // xielu(dot)
  GEMV_OUT_SOFTCAP = 4,  // cap * tanh(dot / cap)
  GEMV_OUT_STREAMS = 5,  // (+ bias) into the residual streams; what the next linear reads goes to u
  GEMV_OUT_GLU = 6,      // weight rows 2 j, 2 j + 1 are gate j and up j: out[j] = gelu(gate) * up
};
enum { ACT_NONE = 0, ACT_SIGMOID = 1, ACT_SILU = 2 };
struct ActRanges {  // columns [end[i-1], end[i]) take activation kind[i]
  int end[4] = {0, 0, 0, 0};
  int kind[4] = {0, 0, 0, 0};
};

// Residual streams: a sublayer's result y turns the n streams x_s into x_t = sum_s mix[s][t] x_s + out[t] y, and the next linear reads
// u = sum_t in[t] x_t.  All of it is local to an element, so it is the epilogue of the sublayer's last linear.
#define HC_MAX 8
#define HC_ROW (HC_MAX + 1)
struct StreamMix {
  int n = 0;
  size_t stride = 0;            // floats between the streams
  const float* coef = nullptr;  // [HC_MAX][HC_ROW]: row t = mix[0 .. HC_MAX)[t], out[t]; zeros from n on, both ways
  const float* in = nullptr;    // [HC_MAX]: of the sublayer that comes next
};
// (constant address space: scalar loads, which no store can be taken to change)
typedef const float __attribute__((address_space(4))) const_f32;
// x: an element (or a vector of neighbours) of stream 0
template <typename V>
__device__ __forceinline__ void stream_load(const StreamMix& m, const float* x, V (&old)[HC_MAX]) {
  // (four at a time without a branch each -- past the last stream the first one again, with a zero coefficient)
#pragma unroll
  for (int s = 0; s < 4; s++) old[s] = *(const V*)(x + (s < m.n ? s : 0) * m.stride);
#pragma unroll
  for (int s = 4; s < HC_MAX; s++) old[s] = V{};
  if (m.n > 4) {
#pragma unroll
    for (int s = 4; s < HC_MAX; s++) old[s] = *(const V*)(x + (s < m.n ? s : 0) * m.stride);
  }
}
template <typename V>
__device__ __forceinline__ V stream_apply(const StreamMix& m, float* x, const V (&old)[HC_MAX], V y) {
  const_f32 *coef = (const_f32*)(size_t)m.coef, *in = (const_f32*)(size_t)m.in;
  V u = V{};
  if (m.n <= 4) {  // (all coefficients in one go)
    V v[4];
#pragma unroll
    for (int t = 0; t < 4; t++) {
      v[t] = coef[t * HC_ROW + HC_MAX] * y;
#pragma unroll
      for (int s = 0; s < 4; s++) v[t] += coef[t * HC_ROW + s] * old[s];
      u += in[t] * v[t];
    }
#pragma unroll
    for (int t = 0; t < 4; t++)
      if (t < m.n) *(V*)(x + t * m.stride) = v[t];
    return u;
  }
#pragma unroll 1
  for (int t = 0; t < m.n; t++) {
    const_f32* c = coef + t * HC_ROW;
    V v = c[HC_MAX] * y;
#pragma unroll
    for (int s = 0; s < HC_MAX; s++) v += c[s] * old[s];
    *(V*)(x + t * m.stride) = v;
    u += in[t] * v;
  }
  return u;
}

struct GemvBf16 {
  const unsigned short* w = nullptr;  // [N][ldw]
  const float* x = nullptr;           // [nb][ldx]
  float* out = nullptr;               // [nb][ldo]
  int N = 0, K = 0, ldw = 0, ldx = 0, ldo = 0, nb = 1;  // K % 8 == 0
  // GEMV_IN_RMS: elements the mean is over, eps, the gain (device); GEMV_IN_SPLIT: the same for the tail, with ss[b][n_ss] pieces
  int mean_n = 1;
  float eps = 0.f;
  const float* gain = nullptr;
  int k_split = 0, n_ss = 0;
  const float* ss = nullptr;
  ActRanges act;
  const float* xielu = nullptr;  // {softplus(p), 1/2 + softplus(q)}
  const float *add_rows = nullptr, *add_vec = nullptr;
  int ld_add = 0;
  float cap = 0.f;
  const float* bias = nullptr;  // [N], nullable (ACT, STREAMS)
  StreamMix sm;                 // STREAMS: out = stream 0, u[b][ldo] = what the next linear reads
  float* u = nullptr;
};

__device__ __forceinline__ float act_sigmoid(float z) { return 1.0f / (1.0f + __expf(-z)); }
__device__ __forceinline__ float act_apply(float z, int kind) {
  if (kind == ACT_NONE) return z;
  const float s = act_sigmoid(z);
  return kind == ACT_SILU ? z * s : s;
}
__device__ __forceinline__ float act_ranges(float z, int col, const ActRanges& a) {
  const int kind = col < a.end[0] ? a.kind[0] : col < a.end[1] ? a.kind[1] : col < a.end[2] ? a.kind[2] : a.kind[3];
  return act_apply(z, kind);
}
// e^z - 1 - z for z <= 0 without the cancellation near zero: its own series below 1/4
__device__ __forceinline__ float exp_minus_line(float z) {
  if (z > -0.25f) {
    float s = 1.0f / 40320.0f;
    s = __builtin_fmaf(s, z, 1.0f / 5040.0f);
    s = __builtin_fmaf(s, z, 1.0f / 720.0f);
    s = __builtin_fmaf(s, z, 1.0f / 120.0f);
    s = __builtin_fmaf(s, z, 1.0f / 24.0f);
    s = __builtin_fmaf(s, z, 1.0f / 6.0f);
    s = __builtin_fmaf(s, z, 0.5f);
    return s * z * z;
  }
  return __expf(z) - 1.0f - z;
}
__device__ __forceinline__ float xielu_apply(float z, float right, float left) {
  const float curved = z > 0.0f ? right * z * z : left * exp_minus_line(z);
  return __builtin_fmaf(0.5f, z, curved);
}
// z / 2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), the bracket's half being a logistic function of twice the argument
__device__ __forceinline__ float gelu_tanh(float z) {
  const float t = 1.5957691216057308f * __builtin_fmaf(0.044715f * z, z * z, z);
  return z / (1.0f + __expf(-t));
}
__device__ __forceinline__ float soft_cap(float z, float cap) { return cap > 0.0f ? cap * tanhf(z / cap) : z; }

template <int OUT>
__device__ __forceinline__ void gemv_out(const GemvBf16& a, int row, int b, float v) {
  float* o = a.out + (size_t)b * a.ldo + row;
  if constexpr (OUT == GEMV_OUT_STORE) *o = v;
  if constexpr (OUT == GEMV_OUT_ACT) *o = act_ranges(a.bias ? v + a.bias[row] : v, row, a.act);
  if constexpr (OUT == GEMV_OUT_RESIDUAL) {
    float s = *o + v;
    if (a.add_rows) s += a.add_rows[(size_t)b * a.ld_add + row];
    if (a.add_vec) s += a.add_vec[row];
    *o = s;
  }
  if constexpr (OUT == GEMV_OUT_XIELU) *o = xielu_apply(v, a.xielu[0], a.xielu[1]);
  if constexpr (OUT == GEMV_OUT_SOFTCAP) *o = soft_cap(v, a.cap);
}

// GEMV_OUT_STREAMS: what the thread that will have (row, b) needs, requested ahead of the products
struct StreamElem {
  float old[HC_MAX], bias = 0.f;
};
__device__ __forceinline__ void stream_elem_load(const GemvBf16& a, int row, int b, StreamElem& e) {
  stream_load(a.sm, a.out + (size_t)b * a.ldo + row, e.old);
  if (a.bias) e.bias = a.bias[row];
}
__device__ __forceinline__ void stream_elem_out(const GemvBf16& a, int row, int b, const StreamElem& e, float v) {
  a.u[(size_t)b * a.ldo + row] = stream_apply(a.sm, a.out + (size_t)b * a.ldo + row, e.old, v + e.bias);
}

#define GEMV_BF16_LDS_FLOATS 8192  // rhs elements staged at a time, all rows together: a cut segment is a multiple of the steps in flight

template <int NB, int R, int IN, int OUT>
__global__ __launch_bounds__(256) void k_gemv_bf16(const GemvBf16 a) {
  extern __shared__ __attribute__((aligned(16))) float gemv_lds[];  // [NB][2][seg / 2]
  __shared__ float red[4][NB];
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg();
  const int row0 = (blockIdx.x * 4 + wave) * R, b0 = blockIdx.y * NB;
  const int seg = a.K < GEMV_BF16_LDS_FLOATS / NB ? a.K : GEMV_BF16_LDS_FLOATS / NB;  // elements per staged segment (512-multiple if cut)
  const int half = seg / 2;                                                           // floats per half-octet plane
  constexpr int UN = R >= 4 || NB >= 8 ? 2 : 4;  // steps of 512 in flight
  const unsigned short* wr[R];
#pragma unroll
  for (int r = 0; r < R; r++) {
    const int row = row0 + r < a.N ? row0 + r : a.N - 1;
    wr[r] = a.w + (size_t)row * a.ldw;
  }
  i32x4 wv[UN][R];
  auto request = [&](int k0) {
#pragma unroll
    for (int u = 0; u < UN; u++) {
      int k = k0 + u * 512 + lane * 8;
      k = k < a.K ? k : 0;  // (a lane past the end requests the row's start and never uses it)
#pragma unroll
      for (int r = 0; r < R; r++) wv[u][r] = __builtin_nontemporal_load((const i32x4*)(wr[r] + k));
    }
  };
  request(0);
  StreamElem elem;  // of lane r NB + b
  const int my_row = row0 + lane / NB, my_b = b0 + lane % NB;
  const bool mine = OUT == GEMV_OUT_STREAMS && lane < R * NB && my_row < a.N && my_b < a.nb;
  if constexpr (OUT == GEMV_OUT_STREAMS) {
    static_assert(R * NB <= 64, "a lane per result");
    if (mine) stream_elem_load(a, my_row, my_b, elem);
  }
  float acc[R][NB];
#pragma unroll
  for (int r = 0; r < R; r++)
#pragma unroll
    for (int b = 0; b < NB; b++) acc[r][b] = 0.f;
  float tail[NB], sq[NB];
#pragma unroll
  for (int b = 0; b < NB; b++) {
    sq[b] = 0.f;
    tail[b] = 1.f;
  }
  if constexpr (IN == GEMV_IN_SPLIT) {
#pragma unroll
    for (int b = 0; b < NB; b++) {
      const int bb = b0 + b < a.nb ? b0 + b : a.nb - 1;
      float s = 0.f;
      for (int i = lane; i < a.n_ss; i += 64) s += a.ss[(size_t)bb * a.n_ss + i];
      s = wave_sum_f32(s);
      tail[b] = 1.0f / sqrtf(s / (float)a.mean_n + a.eps);
    }
  }
  for (int s0 = 0; s0 < a.K; s0 += seg) {
    const int n = a.K - s0 < seg ? a.K - s0 : seg;
    if (s0 > 0) __syncthreads();  // the previous segment has been read by every wave
#pragma unroll
    for (int b = 0; b < NB; b++) {
      const int bb = b0 + b < a.nb ? b0 + b : a.nb - 1;
      const float* xr = a.x + (size_t)bb * a.ldx + s0;
      float* lo = gemv_lds + b * 2 * half;
      for (int q = tid; q < n / 8; q += 256) {
        f32x4 v0 = *(const f32x4*)(xr + q * 8), v1 = *(const f32x4*)(xr + q * 8 + 4);
        if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) {
#pragma unroll
          for (int e = 0; e < 4; e++) sq[b] = __builtin_fmaf(v0[e], v0[e], __builtin_fmaf(v1[e], v1[e], sq[b]));
        }
        if constexpr (IN == GEMV_IN_RMSV) {
          v0 *= *(const f32x4*)(a.gain + s0 + q * 8);
          v1 *= *(const f32x4*)(a.gain + s0 + q * 8 + 4);
        }
        if constexpr (IN == GEMV_IN_SPLIT) {
          if (s0 + q * 8 >= a.k_split) {
            v0 *= tail[b];
            v1 *= tail[b];
          }
        }
        *(f32x4*)(lo + q * 4) = v0;
        *(f32x4*)(lo + half + q * 4) = v1;
      }
    }
    if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) {
      if (s0 + seg >= a.K) {
#pragma unroll
        for (int b = 0; b < NB; b++) {
          const float s = wave_sum_f32(sq[b]);
          if (lane == 0) red[wave][b] = s;
        }
      }
    }
    __syncthreads();
    for (int k0 = 0; k0 < n; k0 += UN * 512) {
      i32x4 cur[UN][R];
#pragma unroll
      for (int u = 0; u < UN; u++)
#pragma unroll
        for (int r = 0; r < R; r++) cur[u][r] = wv[u][r];
      if (s0 + k0 + UN * 512 < a.K) request(s0 + k0 + UN * 512);  // (also across a segment's end: seg % (UN * 512) == 0 then)
#pragma unroll
      for (int u = 0; u < UN; u++) {
        const int k = k0 + u * 512 + lane * 8;
        if (k < n) {
#pragma unroll
          for (int b = 0; b < NB; b++) {
            const float* lo = gemv_lds + b * 2 * half + (k >> 1);
            const f32x4 x0 = *(const f32x4*)lo, x1 = *(const f32x4*)(lo + half);
#pragma unroll
            for (int r = 0; r < R; r++) {
              float s = acc[r][b];
#pragma unroll
              for (int e = 0; e < 2; e++) {
                const unsigned p = (unsigned)cur[u][r][e], p2 = (unsigned)cur[u][r][e + 2];
                s = __builtin_fmaf(__builtin_bit_cast(float, p << 16), x0[2 * e], s);
                s = __builtin_fmaf(__builtin_bit_cast(float, p & 0xffff0000u), x0[2 * e + 1], s);
                s = __builtin_fmaf(__builtin_bit_cast(float, p2 << 16), x1[2 * e], s);
                s = __builtin_fmaf(__builtin_bit_cast(float, p2 & 0xffff0000u), x1[2 * e + 1], s);
              }
              acc[r][b] = s;
            }
          }
        }
      }
    }
  }
  float scale[NB];
#pragma unroll
  for (int b = 0; b < NB; b++) {
    scale[b] = 1.f;
    if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) {
      const float s = (red[0][b] + red[1][b]) + (red[2][b] + red[3][b]);
      scale[b] = (IN == GEMV_IN_RMS ? *a.gain : 1.0f) / sqrtf(s / (float)a.mean_n + a.eps);
    }
  }
  if constexpr (OUT == GEMV_OUT_GLU) {
    static_assert(R % 2 == 0, "a wave holds both rows of a pair");
#pragma unroll
    for (int r = 0; r < R; r += 2)
#pragma unroll
      for (int b = 0; b < NB; b++) {
        const float gate = wave_sum_f32(acc[r][b]) * scale[b], up = wave_sum_f32(acc[r + 1][b]) * scale[b];
        const int row = row0 + r, bb = b0 + b;
        if (lane == ((r / 2 * NB + b) & 63) && row < a.N && bb < a.nb) a.out[(size_t)bb * a.ldo + row / 2] = gelu_tanh(gate) * up;
      }
    return;
  }
  if constexpr (OUT == GEMV_OUT_STREAMS) {
    float y = 0.f;
#pragma unroll
    for (int r = 0; r < R; r++)
#pragma unroll
      for (int b = 0; b < NB; b++) {
        const float v = wave_sum_f32(acc[r][b]) * scale[b];
        y = lane == r * NB + b ? v : y;
      }
    if (mine) stream_elem_out(a, my_row, my_b, elem, y);
    return;
  }
#pragma unroll
  for (int r = 0; r < R; r++)
#pragma unroll
    for (int b = 0; b < NB; b++) {
      const float v = wave_sum_f32(acc[r][b]) * scale[b];
      const int row = row0 + r, bb = b0 + b;
      if (lane == ((r * NB + b) & 63) && row < a.N && bb < a.nb) {
        gemv_out<OUT>(a, row, bb, v);
      }
    }
}

// ---- the same linear for 3 .. 16 rhs rows: one pass over the weights on the matrix cores ---------------------------------------------
// A 512-thread workgroup owns 16 RT weight rows; its eight waves take the 64-element pieces of k in turn and their tiles are added
// through LDS at the end.  Both operands come straight from memory in fragment order (16 rows x 64 bytes per request; the rhs, a few
// hundred KB, lives in L2), the next piece's requests out before the current one is multiplied.  The rhs becomes bf16 on the way:
// rounded (SPL = 1), or as three exact pieces (SPL = 3; see split_store in gemm_bf16.hpp).  K is a multiple of 64.
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
// f32 -> its upper, middle and lower eight significand bits as bf16: their sum is exact
__device__ __forceinline__ void split3(const float (&v)[8], bf16x8& hi, bf16x8& mid, bf16x8& lo) {
  unsigned short h[8], m[8], l[8];
#pragma unroll
  for (int e = 0; e < 8; e++) {
    const float a = __builtin_bit_cast(float, __builtin_bit_cast(unsigned, v[e]) & 0xffff0000u), r = v[e] - a;
    const float b = __builtin_bit_cast(float, __builtin_bit_cast(unsigned, r) & 0xffff0000u);
    h[e] = (unsigned short)(__builtin_bit_cast(unsigned, a) >> 16);
    m[e] = (unsigned short)(__builtin_bit_cast(unsigned, b) >> 16);
    l[e] = f2bf(r - b);
  }
  __builtin_memcpy(&hi, h, 16);
  __builtin_memcpy(&mid, m, 16);
  __builtin_memcpy(&lo, l, 16);
}
__device__ __forceinline__ f32x4 mfma_bf16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

template <int RT, int SPL, int IN, int OUT>
__global__ __launch_bounds__(512) void k_gemv16_bf16(const GemvBf16 a) {
  constexpr int W = 8, LD = 20;
  __shared__ __attribute__((aligned(16))) float tile[W][RT][16 * LD];
  __shared__ float sums[W][16], scale[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg(), fr = lane & 15, fk = lane >> 4;
  const int row0 = blockIdx.x * 16 * RT;
  const unsigned short* wr[RT];
#pragma unroll
  for (int t = 0; t < RT; t++) {
    const int row = row0 + t * 16 + fr;
    wr[t] = a.w + (size_t)(row < a.N ? row : a.N - 1) * a.ldw + fk * 8;
  }
  const float* xr = a.x + (size_t)(fr < a.nb ? fr : a.nb - 1) * a.ldx + fk * 8;
  bf16x8 wv[2][RT];
  f32x4 xv[2][2], gv[2][2];
  auto request = [&](int k) {
#pragma unroll
    for (int u = 0; u < 2; u++) {
#pragma unroll
      for (int t = 0; t < RT; t++) wv[u][t] = *(const bf16x8*)(wr[t] + k + u * 32);
      xv[u][0] = *(const f32x4*)(xr + k + u * 32);
      xv[u][1] = *(const f32x4*)(xr + k + u * 32 + 4);
      if constexpr (IN == GEMV_IN_RMSV) {
        gv[u][0] = *(const f32x4*)(a.gain + k + u * 32 + fk * 8);
        gv[u][1] = *(const f32x4*)(a.gain + k + u * 32 + fk * 8 + 4);
      }
    }
  };
  const int n = a.K / 64;
  if (wave < n) request(wave * 64);
  StreamElem elem[(RT + 1) / 2];  // of this thread's results: element tid + 512 i of the tile
  if constexpr (OUT == GEMV_OUT_STREAMS) {
#pragma unroll
    for (int i = 0; i < (RT + 1) / 2; i++) {
      const int j = tid + i * 512, b = (j >> 4) & 15, row = row0 + (j >> 8) * 16 + (j & 15);
      if (j < RT * 256 && b < a.nb && row < a.N) stream_elem_load(a, row, b, elem[i]);
    }
  }
  float tail = 1.f, sq = 0.f;
  if constexpr (IN == GEMV_IN_SPLIT) {
    float s = 0.f;
    for (int i = fk; i < a.n_ss; i += 4) s += a.ss[(size_t)(fr < a.nb ? fr : a.nb - 1) * a.n_ss + i];
    s += __shfl_xor(s, 16, 64);
    s += __shfl_xor(s, 32, 64);
    tail = 1.0f / sqrtf(s / (float)a.mean_n + a.eps);
  }
  f32x4 acc[RT];
#pragma unroll
  for (int t = 0; t < RT; t++) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int i = wave; i < n; i += W) {
    bf16x8 wc[2][RT];
    f32x4 xc[2][2], gc[2][2];
#pragma unroll
    for (int u = 0; u < 2; u++) {
#pragma unroll
      for (int t = 0; t < RT; t++) wc[u][t] = wv[u][t];
      xc[u][0] = xv[u][0];
      xc[u][1] = xv[u][1];
      if constexpr (IN == GEMV_IN_RMSV) {
        gc[u][0] = gv[u][0];
        gc[u][1] = gv[u][1];
      }
    }
    if (i + W < n) request((i + W) * 64);
#pragma unroll
    for (int u = 0; u < 2; u++) {
      float v[8] = {xc[u][0][0], xc[u][0][1], xc[u][0][2], xc[u][0][3], xc[u][1][0], xc[u][1][1], xc[u][1][2], xc[u][1][3]};
      if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) {
#pragma unroll
        for (int e = 0; e < 8; e++) sq = __builtin_fmaf(v[e], v[e], sq);
      }
      if constexpr (IN == GEMV_IN_RMSV) {
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] *= gc[u][e >> 2][e & 3];
      }
      if constexpr (IN == GEMV_IN_SPLIT) {
        const float f = i * 64 >= a.k_split ? tail : 1.f;  // (k_split is a multiple of 64)
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] *= f;
      }
      if constexpr (SPL == 1) {
        bf16x8 b;
#pragma unroll
        for (int e = 0; e < 8; e++) b[e] = (__bf16)v[e];
#pragma unroll
        for (int t = 0; t < RT; t++) acc[t] = mfma_bf16(wc[u][t], b, acc[t]);
      } else {
        bf16x8 h, m, l;
        split3(v, h, m, l);
#pragma unroll
        for (int t = 0; t < RT; t++) acc[t] = mfma_bf16(wc[u][t], h, mfma_bf16(wc[u][t], m, mfma_bf16(wc[u][t], l, acc[t])));
      }
    }
  }
  // lane: weight rows 4 fk .. of rhs row fr
#pragma unroll
  for (int t = 0; t < RT; t++) *(f32x4*)&tile[wave][t][fr * LD + fk * 4] = acc[t];
  if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) {
    sq += __shfl_xor(sq, 16, 64);
    sq += __shfl_xor(sq, 32, 64);
    if (fk == 0) sums[wave][fr] = sq;
  }
  __syncthreads();
  if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) {
    if (tid < 16) {
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < W; w++) s += sums[w][tid];
      scale[tid] = (IN == GEMV_IN_RMS ? *a.gain : 1.0f) / sqrtf(s / (float)a.mean_n + a.eps);
    }
    __syncthreads();
  }
  if constexpr (OUT == GEMV_OUT_GLU) {
    for (int i = tid; i < RT * 128; i += 512) {
      const int t = i >> 7, b = (i >> 3) & 15, r = (i & 7) * 2, row = row0 + t * 16 + r;
      float gate = 0.f, up = 0.f;
#pragma unroll
      for (int w = 0; w < W; w++) {
        gate += tile[w][t][b * LD + r];
        up += tile[w][t][b * LD + r + 1];
      }
      if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) {
        gate *= scale[b];
        up *= scale[b];
      }
      if (b < a.nb && row < a.N) a.out[(size_t)b * a.ldo + row / 2] = gelu_tanh(gate) * up;
    }
    return;
  }
  if constexpr (OUT == GEMV_OUT_STREAMS) {
#pragma unroll
    for (int i = 0; i < (RT + 1) / 2; i++) {
      const int j = tid + i * 512, t = j >> 8, b = (j >> 4) & 15, r = j & 15, row = row0 + t * 16 + r;
      if (j < RT * 256 && b < a.nb && row < a.N) {
        float v = 0.f;
#pragma unroll
        for (int w = 0; w < W; w++) v += tile[w][t][b * LD + r];
        stream_elem_out(a, row, b, elem[i], v);
      }
    }
    return;
  }
  for (int i = tid; i < RT * 256; i += 512) {
    const int t = i >> 8, b = (i >> 4) & 15, r = i & 15, row = row0 + t * 16 + r;
    float v = 0.f;
#pragma unroll
    for (int w = 0; w < W; w++) v += tile[w][t][b * LD + r];
    if constexpr (IN == GEMV_IN_RMS || IN == GEMV_IN_RMSV) v *= scale[b];
    if (b < a.nb && row < a.N) gemv_out<OUT>(a, row, b, v);
  }
}

template <int IN, int OUT>
inline void launch_gemv16_bf16(hipStream_t st, crabml_hip_device::ProfRec* rec, const GemvBf16& a, bool exact) {
  const bool two = a.N >= 16384;
  const dim3 grid((a.N + (two ? 31 : 15)) / (two ? 32 : 16));
  if (exact)
    launch_k(st, rec, two ? k_gemv16_bf16<2, 3, IN, OUT> : k_gemv16_bf16<1, 3, IN, OUT>, grid, dim3(512), 0, a);
  else
    launch_k(st, rec, two ? k_gemv16_bf16<2, 1, IN, OUT> : k_gemv16_bf16<1, 1, IN, OUT>, grid, dim3(512), 0, a);
}

template <int NB, int R, int IN, int OUT>
inline void launch_gemv_bf16_t(hipStream_t st, crabml_hip_device::ProfRec* rec, const GemvBf16& a) {
  const int cap = GEMV_BF16_LDS_FLOATS / NB, seg = a.K < cap ? a.K : cap;
  launch_k(st, rec, k_gemv_bf16<NB, R, IN, OUT>, dim3((a.N + 4 * R - 1) / (4 * R), (a.nb + NB - 1) / NB), dim3(256),
           (size_t)NB * seg * sizeof(float), a);
}
// rows of the rhs that share one pass over the weights: as many as there are, up to 8
template <int IN, int OUT>
inline void launch_gemv_bf16(hipStream_t st, crabml_hip_device::ProfRec* rec, const GemvBf16& a) {
  const bool wide = a.N >= 16384;  // enough rows to give a wave four and still fill the chip
  if (a.nb <= 1) {
    if (wide)
      launch_gemv_bf16_t<1, 4, IN, OUT>(st, rec, a);
    else if (a.N >= 2048 || OUT == GEMV_OUT_GLU)
      launch_gemv_bf16_t<1, 2, IN, OUT>(st, rec, a);
    else if constexpr (OUT != GEMV_OUT_GLU)
      launch_gemv_bf16_t<1, 1, IN, OUT>(st, rec, a);
  } else if (a.nb <= 2) {
    launch_gemv_bf16_t<2, 2, IN, OUT>(st, rec, a);
  } else if (a.nb <= 4) {
    launch_gemv_bf16_t<4, 2, IN, OUT>(st, rec, a);
  } else {
    launch_gemv_bf16_t<8, 2, IN, OUT>(st, rec, a);
  }
}

}  // namespace crabml_hip
