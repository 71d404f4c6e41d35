// hybrid_rows.hpp -- the hybrid decoder's prompt pass: any number of tokens of any number of sequences as one batch of rows
//   k_gemm_bf16<ACT>       norm 1 + every projection of both mixers + their activations
//   k_attn_rows            softmax attention, 64 query rows of one head per workgroup, on the matrix cores
//   k_linear_rows          linear attention in blocks of rows: inside a block as a masked product, across blocks through the state
//   k_mix_rows             the linear branch's norm and gate, the cache append
//   k_gemm_bf16<RESIDUAL>, k_gemm_bf16<XIELU>, k_gemm_bf16<RESIDUAL>
// Keys of this pass are read from its own projected rows, earlier ones from the cache; the cache is appended only after the attention
// launch, with the rows that later tokens can see.
//
// T = unsigned short: bf16 operands.  T = float: every operand f32 (v_mfma_f32_16x16x4_f32), activations in three exact planes.
#pragma once
#include "hybrid_common.hpp"

namespace crabml_hip {

struct PassSeq {
  int row0, n, pos0;  // rows row0 .. row0 + n - 1 of the pass are the sequence's positions pos0 ..
  int hist_end;       // earlier positions that latent layers read again, as rows: position p < pos0 is row hist_end - (pos0 - p)
  char* slab;
};
struct PassRow {
  int seq, pos;
};
struct PassTile {  // up to 64 (times AttnTile::RT) consecutive rows of one sequence
  int seq, row, pos, n;
};

// ---- operand fragments of 16x16 matrix products out of LDS rows with k contiguous ------------------------------------------------
// lane: row lane % 16 of the operand, k group lane / 16
// acc += A B^T over k < K; a / b: this lane's rows.  K is a multiple of 32.
__device__ __forceinline__ f32x4 mma_rows(const unsigned short* a, const unsigned short* b, int K, f32x4 acc) {
  const int o = (threadIdx.x >> 4 & 3) * 8;
  for (int k = 0; k < K; k += 32) acc = mfma_bf16(*(const bf16x8*)(a + k + o), *(const bf16x8*)(b + k + o), acc);
  return acc;
}
// one side f32: three exact bf16 pieces of it.  w (nullable, LDS): a factor per k
__device__ __forceinline__ f32x4 mma_rows(const float* a, const unsigned short* b, int K, f32x4 acc) {
  const int o = (threadIdx.x >> 4 & 3) * 8;
  for (int k = 0; k < K; k += 32) {
    float v[8];
    kv_load8(a + k + o, v);
    bf16x8 h, m, l;
    split3(v, h, m, l);
    const bf16x8 fb = *(const bf16x8*)(b + k + o);
    acc = mfma_bf16(h, fb, mfma_bf16(m, fb, mfma_bf16(l, fb, acc)));
  }
  return acc;
}
__device__ __forceinline__ f32x4 mma_rows(const unsigned short* a, const float* b, int K, f32x4 acc) {
  const int o = (threadIdx.x >> 4 & 3) * 8;
  for (int k = 0; k < K; k += 32) {
    float v[8];
    kv_load8(b + k + o, v);
    bf16x8 h, m, l;
    split3(v, h, m, l);
    const bf16x8 fa = *(const bf16x8*)(a + k + o);
    acc = mfma_bf16(fa, h, mfma_bf16(fa, m, mfma_bf16(fa, l, acc)));
  }
  return acc;
}
__device__ __forceinline__ f32x4 mma_rows(const float* a, const float* b, int K, f32x4 acc) {
  const int o = threadIdx.x >> 4 & 3;
#pragma unroll 8
  for (int k = 0; k < K; k += 4) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[k + o], b[k + o], acc, 0, 0, 0);
  return acc;
}
// the same with a factor w[k] (LDS) on A's elements
__device__ __forceinline__ f32x4 mma_rows_w(const unsigned short* a, const float* w, const unsigned short* b, int K, f32x4 acc) {
  const int o = (threadIdx.x >> 4 & 3) * 8;
  for (int k = 0; k < K; k += 32) {
    float v[8], f[8];
    kv_load8(a + k + o, v);
    kv_load8(w + k + o, f);
#pragma unroll
    for (int e = 0; e < 8; e++) v[e] *= f[e];
    bf16x8 h, m, l;
    split3(v, h, m, l);
    const bf16x8 fb = *(const bf16x8*)(b + k + o);
    acc = mfma_bf16(h, fb, mfma_bf16(m, fb, mfma_bf16(l, fb, acc)));
  }
  return acc;
}
__device__ __forceinline__ f32x4 mma_rows_w(const float* a, const float* w, const float* b, int K, f32x4 acc) {
  const int o = threadIdx.x >> 4 & 3;
#pragma unroll 8
  for (int k = 0; k < K; k += 4) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[k + o] * w[k + o], b[k + o], acc, 0, 0, 0);
  return acc;
}

// ---- embedding of the pass's rows: x, its planes, its square sum (piece 0; the others are cleared) --------------------------------
template <int P>
__global__ __launch_bounds__(256) void k_embed_rows(const unsigned short* __restrict__ table, const int* __restrict__ tokens,
                                                    const PassRow* __restrict__ rows, int width, int ldx, float scale,
                                                    const double* __restrict__ freq, float* __restrict__ x, float* __restrict__ emb,
                                                    const float* __restrict__ add_vec, unsigned short* __restrict__ planes, size_t p_plane,
                                                    float* __restrict__ sq_out, int n_sq, const StreamMix sm, const float* __restrict__ gain) {
  __shared__ float red[4];
  const int r = blockIdx.x, tok = tokens[r], pos = rows[r].pos;
  float s = 0.f;
  for (int c = threadIdx.x; c < width; c += 256) {
    float v = __builtin_fmaf(bf2f(table[(size_t)tok * width + c]), scale, position_entry(pos, c, freq));
    if (sm.n) {  // every stream starts as the embedding
      float u = 0.f;
      for (int t = 0; t < sm.n; t++) {
        x[t * sm.stride + (size_t)r * ldx + c] = v;
        u = __builtin_fmaf(sm.in[t], v, u);
      }
      v = u;
    } else {
      if (emb) emb[(size_t)r * ldx + c] = v;
      if (add_vec) v += add_vec[c];
      x[(size_t)r * ldx + c] = v;
    }
    split_store<P>(gain ? v * gain[c] : v, planes + (size_t)r * ldx + c, p_plane);
    s = __builtin_fmaf(v, v, s);
  }
  s = wave_sum_f32(s);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = s;
  __syncthreads();
  for (int i = threadIdx.x; i < n_sq; i += 256) sq_out[(size_t)r * n_sq + i] = i ? 0.f : (red[0] + red[1]) + (red[2] + red[3]);
}

// rows[i] of x (the weighted sum of its streams) -> dense rows of f32 (P = 0) or planes, with their square sums in piece 0
template <int P>
__global__ __launch_bounds__(256) void k_gather_rows(const float* __restrict__ x, int ldx, int width, const int* __restrict__ which,
                                                     float* __restrict__ dst, unsigned short* __restrict__ planes, size_t p_plane,
                                                     float* __restrict__ sq_out, int n_sq, const StreamMix sm, const float* __restrict__ gain) {
  __shared__ float red[4];
  const int r = blockIdx.x;
  const float* src = x + (size_t)which[r] * ldx;
  float s = 0.f;
  for (int c = threadIdx.x; c < width; c += 256) {
    float v = src[c];
    if (sm.n) {
      v *= sm.in[0];
      for (int t = 1; t < sm.n; t++) v = __builtin_fmaf(sm.in[t], src[t * sm.stride + c], v);
    }
    if constexpr (P == 0) {
      dst[(size_t)r * ldx + c] = v;
    } else {
      split_store<P>(gain ? v * gain[c] : v, planes + (size_t)r * ldx + c, p_plane);
      s = __builtin_fmaf(v, v, s);
    }
  }
  if constexpr (P != 0) {
    s = wave_sum_f32(s);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = s;
    __syncthreads();
    for (int i = threadIdx.x; i < n_sq; i += 256) sq_out[(size_t)r * n_sq + i] = i ? 0.f : (red[0] + red[1]) + (red[2] + red[3]);
  }
}

// ---- softmax attention ------------------------------------------------------------------------------------------------------------
template <typename T>
struct MixRows {
  AttnGeom at;
  LinGeom li;
  LatGeom la;
  RunState rs;
  const PassSeq* seqs = nullptr;
  const PassTile* tiles = nullptr;
  const PassRow* rows = nullptr;
  const T* proj = nullptr;  // [rows][ldp]
  unsigned short* cat = nullptr;
  size_t cat_plane = 0;
  float* lin = nullptr;  // [rows][H * V] raw outputs of the linear branch
  int n_tiles = 0, ldp = 0, ldc = 0, lin_off = 0;
  T* v_kept = nullptr;  // [rows][ld_vk] values that VMIX_KEEP leaves
  int ld_vk = 0;
  // latent attention: rows of this pass, then the earlier ones (PassSeq::hist_end)
  unsigned short* lat = nullptr;  // [planes][rows][la.ldl] normed latents
  size_t lat_plane = 0;
  T* rot = nullptr;       // [rows][la.rot] rotated key parts
  const T* kv = nullptr;  // [rows][H * (la.dim + V)] keys of all heads, values of all heads
  int M = 0;              // rows of this pass
};

// Shape of the attention kernel for keys up to KC and values up to VC wide: KT keys per tile; RT times 16 query rows per wave.
template <typename T, int KC, int VC>
struct AttnTile {
  static constexpr int PAD = 16 / sizeof(T), KT = sizeof(T) == 2 ? (KC > 128 ? 32 : 64) : 4096 / KC;
  static constexpr int RT = sizeof(T) == 2 && KC <= 192 && VC <= 128 ? 2 : 1;
};

// One workgroup: 64 RT query rows of one head, four waves of 16 RT.  Keys come in tiles through LDS (K as rows, V transposed), the next
// tile's rows already on their way into registers while the current one is multiplied.
// Everything is transposed -- S^T = K Q^T, O^T = V^T P^T -- so that a lane owns one query row (its column): the softmax statistics are
// one number per lane, and the accumulators of S^T, exponentiated, ARE the operand of the second product: k slot (lane / 16, i) of the
// matrix instruction stands for key 4 (lane / 16) + i of a 16-key group, and V^T is read from LDS in the same order.  Scores live in
// the log2 domain.
template <typename T, int KC, int VC, int P, bool LAT>
__global__ __launch_bounds__(256, sizeof(T) == 2 ? 2 : 1) void k_attn_rows(const MixRows<T> a) {
  typedef AttnTile<T, KC, VC> A;
  constexpr int KT = A::KT, RT = A::RT, LK = KC + A::PAD, LV = KT + A::PAD, VT = VC / 16, ST = KT / 16;
  constexpr int NK = KT * KC / 8 / 256, NV = KT * VC / 8 / 256;  // octets of K and of V per thread and tile
  static_assert(NK >= 1 && NV >= 2 && NV % 2 == 0, "V octets are handled in pairs of keys");
  __shared__ __attribute__((aligned(16))) T ks[KT * LK];
  __shared__ __attribute__((aligned(16))) T vs[VC * LV];
  const AttnGeom& g = a.at;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg(), fr = lane & 15, fk = lane >> 4;
  const PassTile t = a.tiles[a.n_tiles - 1 - blockIdx.x];  // (a sequence's last tiles see the most keys: first)
  const PassSeq sq = a.seqs[t.seq];
  const int h = blockIdx.y, kvh = h / (g.H / g.G);
  const int DK = (g.D + 31) & ~31;
  const int lo = attn_first(g, t.pos), hi = t.pos + t.n;  // keys [lo, hi); those before pos0 are cache rows from that of `lo` on
  const int ring = lo % g.span;
  const T* kc = (const T*)(sq.slab + a.rs.k) + (size_t)kvh * g.rows * g.D;
  const T* vc = (const T*)(sq.slab + a.rs.v) + (size_t)kvh * g.rows * g.V;
  const T* pk = a.proj + (size_t)sq.row0 * a.ldp + g.ck + kvh * g.D;
  const T* pv = a.proj + (size_t)sq.row0 * a.ldp + g.cv + kvh * g.V;
  const int ldkv = LAT ? g.H * (a.la.dim + g.V) : 0;
  // position p, column c -> the octet of its key / value
  auto k_at = [&](int p, int c) -> const T* {
    if constexpr (LAT) {
      const size_t row = (size_t)((p >= sq.pos0 ? sq.row0 : sq.hist_end) + (p - sq.pos0));
      return c < a.la.dim ? a.kv + row * ldkv + h * a.la.dim + c : a.rot + row * a.la.rot + (c - a.la.dim);
    } else {
      if (p >= sq.pos0) return pk + (size_t)(p - sq.pos0) * a.ldp + c;
      const int r = ring + (p - lo);
      return kc + (size_t)(r < g.span ? r : r - g.span) * g.D + c;
    }
  };
  auto v_at = [&](int p, int c) -> const T* {
    if constexpr (LAT) {
      const size_t row = (size_t)((p >= sq.pos0 ? sq.row0 : sq.hist_end) + (p - sq.pos0));
      return a.kv + row * ldkv + g.H * a.la.dim + h * g.V + c;
    } else {
      if (p >= sq.pos0) return pv + (size_t)(p - sq.pos0) * a.ldp + c;
      const int r = ring + (p - lo);
      return vc + (size_t)(r < g.span ? r : r - g.span) * g.V + c;
    }
  };
  // this wave's rows, and the keys any of them sees
  const int w0 = wave * 16 * RT, wn = min(16 * RT, t.n - w0);
  const int wfirst = t.pos + w0, wlast = wfirst + wn - 1, wlo = attn_first(g, wfirst), wlast_lo = attn_first(g, wlast > 0 ? wlast : 0);
  bf16x8 q16[RT][sizeof(T) == 2 ? KC / 32 : 1];
  float q32[RT][sizeof(T) == 4 ? KC / 4 : 1];
  int pos[RT], first[RT];
#pragma unroll
  for (int r = 0; r < RT; r++) {
    const int row = w0 + r * 16 + fr;
    const T* qp = a.proj + (size_t)(t.row + (row < t.n ? row : t.n - 1)) * a.ldp + g.cq + h * g.D;
    pos[r] = t.pos + row;
    first[r] = attn_first(g, pos[r]);
    if constexpr (sizeof(T) == 2) {
#pragma unroll
      for (int i = 0; i < KC / 32; i++) {
        const int k = i * 32 + fk * 8;
        const Oct<T> o = k < g.D ? oct_load(qp + k) : oct_zero<T>();
        __builtin_memcpy(&q16[r][i], &o, 16);
      }
    } else {
#pragma unroll
      for (int i = 0; i < KC / 4; i++) q32[r][i] = i * 4 + fk < g.D ? (float)qp[i * 4 + fk] : 0.f;
    }
  }
  float m[RT], l[RT];
  f32x4 o[RT][VT];
#pragma unroll
  for (int r = 0; r < RT; r++) {
    m[r] = -INFINITY;
    l[r] = 0.f;
#pragma unroll
    for (int j = 0; j < VT; j++) o[r][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float amp = g.amp ? g.amp[h] : 0.f, rate = g.amp ? g.rate[h] : 0.f, scale2 = g.scale * 1.44269504f;
  Oct<T> rk[NK], rv[NV];
  auto request = [&](int j0) {
#pragma unroll
    for (int u = 0; u < NK; u++) {
      const int i = u * 256 + tid, c = i % (KC / 8) * 8, p = j0 + i / (KC / 8);
      rk[u] = oct_zero<T>();
      if (p < hi && c < g.D) rk[u] = oct_load(k_at(p, c));
    }
#pragma unroll
    for (int u = 0; u < NV; u++) {  // octets u, u + 1: the same columns of two neighbouring keys
      const int i = (u >> 1) * 256 + tid, c = i / (KT / 2) * 8, p = j0 + i % (KT / 2) * 2 + (u & 1);
      rv[u] = oct_zero<T>();
      if (p < hi && c < g.V) rv[u] = oct_load(v_at(p, c));
    }
  };
  request(lo);
  for (int j0 = lo; j0 < hi; j0 += KT) {
    __syncthreads();
#pragma unroll
    for (int u = 0; u < NK; u++) {
      const int i = u * 256 + tid;
      oct_store(ks + i / (KC / 8) * LK + i % (KC / 8) * 8, rk[u]);
    }
#pragma unroll
    for (int u = 0; u < NV; u += 2) {
      const int i = (u >> 1) * 256 + tid, c = i / (KT / 2) * 8, key = i % (KT / 2) * 2;
      T v0[8], v1[8];
      __builtin_memcpy(v0, &rv[u], sizeof v0);
      __builtin_memcpy(v1, &rv[u + 1], sizeof v1);
#pragma unroll
      for (int e = 0; e < 8; e++) {
        T two[2] = {v0[e], v1[e]};
        __builtin_memcpy(vs + (c + e) * LV + key, two, sizeof two);
      }
    }
    __syncthreads();
    if (j0 + KT < hi) request(j0 + KT);
    if (wn <= 0 || j0 > wlast || j0 + KT <= wlo) continue;  // (wave-uniform: nothing here for this wave's rows)
    const bool edge = j0 + KT - 1 > wfirst || j0 < wlast_lo;
    f32x4 s[RT][ST];
#pragma unroll
    for (int j = 0; j < ST; j++) {
      const T* kr = ks + (j * 16 + fr) * LK;
#pragma unroll
      for (int r = 0; r < RT; r++) s[r][j] = f32x4{0.f, 0.f, 0.f, 0.f};
      if constexpr (sizeof(T) == 2) {
#pragma unroll
        for (int i = 0; i < KC / 32; i++)
          if (i * 32 < DK) {
            const bf16x8 kf = *(const bf16x8*)(kr + i * 32 + fk * 8);
#pragma unroll
            for (int r = 0; r < RT; r++) s[r][j] = mfma_bf16(kf, q16[r][i], s[r][j]);
          }
      } else {
#pragma unroll
        for (int i = 0; i < KC / 4; i++)
          if (i * 4 < DK) {
            const float kf = kr[i * 4 + fk];
#pragma unroll
            for (int r = 0; r < RT; r++) s[r][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf, q32[r][i], s[r][j], 0, 0, 0);
          }
      }
    }
#pragma unroll
    for (int r = 0; r < RT; r++) {
      const float d0 = (float)(pos[r] - j0 - fk * 4);  // distance to this lane's first key of the tile
      float mx = -INFINITY;
#pragma unroll
      for (int j = 0; j < ST; j++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
          float v = s[r][j][e] * scale2;
          if (g.amp) v = __builtin_fmaf(-amp, __builtin_amdgcn_logf(__builtin_fmaf(rate, d0 - (float)(j * 16 + e), 1.0f)), v);
          if (edge) {
            const int p = j0 + j * 16 + fk * 4 + e;
            v = p <= pos[r] && p >= first[r] ? v : -INFINITY;
          }
          s[r][j][e] = v;
          mx = fmaxf(mx, v);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      mx = fmaxf(m[r], mx);
      const float ref = mx == -INFINITY ? 0.f : mx, w = __builtin_amdgcn_exp2f(m[r] - ref);
      m[r] = mx;
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < ST; j++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
          const float pe = __builtin_amdgcn_exp2f(s[r][j][e] - ref);
          s[r][j][e] = pe;
          sum += pe;
        }
      l[r] = __builtin_fmaf(l[r], w, sum);  // (this lane's keys; the four lanes of a row are added at the end)
#pragma unroll
      for (int j = 0; j < VT; j++) o[r][j] *= w;
    }
    if constexpr (sizeof(T) == 2) {
#pragma unroll
      for (int jj = 0; jj < ST; jj += 2) {
        bf16x8 pf[RT];
#pragma unroll
        for (int r = 0; r < RT; r++)
#pragma unroll
          for (int e = 0; e < 4; e++) {
            pf[r][e] = (__bf16)s[r][jj][e];
            pf[r][e + 4] = (__bf16)s[r][jj + 1][e];
          }
#pragma unroll
        for (int j = 0; j < VT; j++)
          if (j * 16 < g.V) {
            const T* vr = vs + (j * 16 + fr) * LV + jj * 16 + fk * 4;
            bf16x8 vf;
            __builtin_memcpy(&vf, vr, 8);
            __builtin_memcpy((char*)&vf + 8, vr + 16, 8);
#pragma unroll
            for (int r = 0; r < RT; r++) o[r][j] = mfma_bf16(vf, pf[r], o[r][j]);
          }
      }
    } else {
#pragma unroll
      for (int jj = 0; jj < ST; jj++)
#pragma unroll
        for (int j = 0; j < VT; j++)
          if (j * 16 < g.V) {
            const f32x4 vf = *(const f32x4*)(vs + (j * 16 + fr) * LV + jj * 16 + fk * 4);
#pragma unroll
            for (int r = 0; r < RT; r++)
#pragma unroll
              for (int e = 0; e < 4; e++) o[r][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(vf[e], s[r][jj][e], o[r][j], 0, 0, 0);
          }
    }
  }
#pragma unroll
  for (int r = 0; r < RT; r++) {
    float den = l[r];
    den += __shfl_xor(den, 16, 64);
    den += __shfl_xor(den, 32, 64);
    const int row = w0 + r * 16 + fr;
    if (row >= t.n) continue;
    float w = 1.f;
    if (g.sink) {
      const float s2 = g.sink[h] * 1.44269504f, top = fmaxf(m[r], s2);
      w = __builtin_amdgcn_exp2f(m[r] - top);
      den = __builtin_fmaf(den, w, __builtin_amdgcn_exp2f(s2 - top));
    }
    w *= g.out_scale / den;
    const size_t at = (size_t)(t.row + row);
#pragma unroll
    for (int j = 0; j < VT; j++) {
      const int c = j * 16 + fk * 4;
      if (c < g.V) {  // (widths are multiples of 8: four columns at a time)
        const int col = h * g.V + c;
        const T* gp = a.proj + at * a.ldp + g.cg + (g.gate == GATE_HEAD ? h : col);
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] = o[r][j][e] * (g.gate == GATE_NONE ? w : w * kv_to(gp[g.gate == GATE_HEAD ? 0 : e]));
        split_store4<P>(v, a.cat + at * a.ldc + col, a.cat_plane);
      }
    }
  }
}

// ---- linear attention with decay --------------------------------------------------------------------------------------------------
// One workgroup: one head of one sequence, LIN_SLICE value columns, blocks of C rows in order.  With i, j inside a block of n rows:
//   o_i = d^(i+1) S^T q_i + sum_{j <= i} d^(i-j) (q_i . k_j) v_j          S <- d^n S + sum_j d^(n-1-j) k_j v_j^T
// The state lives in the accumulators (transposed: value columns are matrix rows) and passes through LDS once per block for the first
// term.  Decay powers, products with the state and the masked weights are f32 (mma_rows on an f32 side).
template <typename T, int CLS>
struct LinTile {
  static constexpr int C = sizeof(T) == 2 ? 64 : 32, PAD = 16 / sizeof(T);
  static constexpr int LD = CLS + PAD, LC = C + PAD, LP = C + 4, LS = CLS + 4;
  static constexpr size_t T_ELEMS = (size_t)2 * C * LD + (size_t)CLS * LC + LIN_SLICE * LC;
  static constexpr size_t F_ELEMS = (size_t)C * LP + LIN_SLICE * LS + C + LIN_POW + 7;
  static constexpr size_t LDS = T_ELEMS * sizeof(T) + F_ELEMS * sizeof(float);
};
template <typename T, int CLS>
__global__ __launch_bounds__(256) void k_linear_rows(const MixRows<T> a) {
  typedef LinTile<T, CLS> L;
  constexpr int C = L::C, LD = L::LD, LC = L::LC, LP = L::LP, LS = L::LS, MT = C / 16, NG = 4 / MT, ND = CLS / 64;
  constexpr int NQ = C * CLS / 8 / 256;  // octets of Q (and of K) per thread
  extern __shared__ __attribute__((aligned(16))) char lin_lds[];
  T* qs = (T*)lin_lds;          // [C][LD]
  T* ks = qs + C * LD;          // [C][LD]
  T* kt = ks + C * LD;          // [CLS][LC]
  T* vt = kt + CLS * LC;        // [LIN_SLICE][LC]
  float* p = (float*)(vt + LIN_SLICE * LC);  // [C][LP]
  float* st = p + C * LP;                    // [LIN_SLICE][LS]
  float* wj = st + LIN_SLICE * LS;           // [C] d^(n-1-j)
  float* pow = wj + C;                       // [LIN_POW]
  const LinGeom& g = a.li;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg(), fr = lane & 15, fk = lane >> 4;
  const int slice = blockIdx.x % g.slices, h = blockIdx.x / g.slices;
  const PassSeq sq = a.seqs[blockIdx.y];
  const int c0 = slice * LIN_SLICE;
  float* S = (float*)(sq.slab + a.rs.s) + (size_t)h * g.D * g.V;
  const T* base = a.proj + (size_t)sq.row0 * a.ldp;
  for (int i = tid; i < LIN_POW; i += 256) pow[i] = g.decay[h * LIN_POW + i];
  // state tile (value columns c0 + 16 i + 4 fk .., key column 16 (wave + 4 n) + fr)
  f32x4 s[2][ND];
#pragma unroll
  for (int i = 0; i < 2; i++)
#pragma unroll
    for (int n = 0; n < ND; n++) {
      const int c = c0 + i * 16 + fk * 4, d = (wave + 4 * n) * 16 + fr;
      s[i][n] = sq.pos0 > 0 && c < g.V && d < g.D ? *(const f32x4*)(S + (size_t)d * g.V + c) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
  Oct<T> rq[NQ], rk[NQ], rv;
  auto request = [&](int r0) {
#pragma unroll
    for (int u = 0; u < NQ; u++) {
      const int i = u * 256 + tid, r = r0 + i % C, c = i / C * 8;
      const bool in = r < sq.n && c < g.D;
      const T* row = base + (size_t)r * a.ldp + h * g.D + c;
      rq[u] = in ? oct_load(row + g.cq) : oct_zero<T>();
      rk[u] = in ? oct_load(row + g.ck) : oct_zero<T>();
    }
    const int r = r0 + tid % C, c = c0 + tid / C * 8;
    rv = tid < C * (LIN_SLICE / 8) && r < sq.n && c < g.V ? oct_load(base + (size_t)r * a.ldp + g.cv + h * g.V + c) : oct_zero<T>();
  };
  request(0);
  for (int r0 = 0; r0 < sq.n; r0 += C) {
    const int n = sq.n - r0 < C ? sq.n - r0 : C;
    __syncthreads();  // the previous block's products are done with LDS (and pow is there)
#pragma unroll
    for (int u = 0; u < NQ; u++) {
      const int i = u * 256 + tid, r = i % C, c = i / C * 8;
      oct_store(qs + r * LD + c, rq[u]);
      oct_store(ks + r * LD + c, rk[u]);
      oct_scatter(kt + c * LC + r, LC, rk[u]);
    }
    if (tid < C * (LIN_SLICE / 8)) oct_scatter(vt + (tid / C * 8) * LC + tid % C, LC, rv);
    if (tid < C) wj[tid] = tid < n ? pow[n - 1 - tid] : 0.f;
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
      for (int nn = 0; nn < ND; nn++)
#pragma unroll
        for (int e = 0; e < 4; e++) st[(i * 16 + fk * 4 + e) * LS + (wave + 4 * nn) * 16 + fr] = s[i][nn][e];
    __syncthreads();
    if (r0 + C < sq.n) request(r0 + C);
    const int mt = wave % MT;
    // masked, decayed products of the block's rows
    for (int j = wave / MT; j < MT; j += NG) {
      f32x4 v = {0.f, 0.f, 0.f, 0.f};
      if (j <= mt) v = mma_rows(qs + (mt * 16 + fr) * LD, ks + (j * 16 + fr) * LD, CLS, v);
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const int i = mt * 16 + fk * 4 + e, d = i - (j * 16 + fr);
        p[i * LP + j * 16 + fr] = d >= 0 ? v[e] * pow[d] : 0.f;
      }
    }
    __syncthreads();
    for (int j = wave / MT; j < 2; j += NG) {
      f32x4 v = mma_rows(qs + (mt * 16 + fr) * LD, st + (j * 16 + fr) * LS, CLS, f32x4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
      for (int e = 0; e < 4; e++) v[e] *= pow[mt * 16 + fk * 4 + e + 1];
      v = mma_rows(p + (mt * 16 + fr) * LP, vt + (j * 16 + fr) * LC, C, v);
      const int c = c0 + j * 16 + fr;
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const int i = mt * 16 + fk * 4 + e;
        if (i < n && c < g.V) a.lin[(size_t)(sq.row0 + r0 + i) * (g.H * g.V) + h * g.V + c] = v[e];
      }
    }
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
      for (int nn = 0; nn < ND; nn++) {
        s[i][nn] *= pow[n];
        s[i][nn] = mma_rows_w(vt + (i * 16 + fr) * LC, wj, kt + ((wave + 4 * nn) * 16 + fr) * LC, C, s[i][nn]);
      }
  }
#pragma unroll
  for (int i = 0; i < 2; i++)
#pragma unroll
    for (int nn = 0; nn < ND; nn++) {
      const int c = c0 + i * 16 + fk * 4, d = (wave + 4 * nn) * 16 + fr;
      if (c < g.V && d < g.D) *(f32x4*)(S + (size_t)d * g.V + c) = s[i][nn];
    }
}

// ---- in front of attention: the norms over all of a row's queries (keys), the values of an earlier layer ------------------------------
template <typename T>
__device__ __forceinline__ void octet_scale(T* p, float f, const float* gain) {
  float v[8], n[8];
  kv_load8(p, v);
  read8(gain, n);
#pragma unroll
  for (int e = 0; e < 8; e++) p[e] = kv_from<T>(v[e] * (f * n[e]));
}
template <typename T>
__global__ __launch_bounds__(256) void k_qkv_rows(const MixRows<T> a) {
  __shared__ float red[8];
  const AttnGeom& g = a.at;
  const int r = blockIdx.x, tid = threadIdx.x, nq = g.H * g.D, nk = g.G * g.D, nv = g.G * g.V;
  T* pr = const_cast<T*>(a.proj) + (size_t)r * a.ldp;
  if (g.q_norm) {
    float sq = 0.f, sk = 0.f, v[8];
    for (int i = tid * 8; i < nq; i += 2048) {
      kv_load8(pr + g.cq + i, v);
#pragma unroll
      for (int e = 0; e < 8; e++) sq = __builtin_fmaf(v[e], v[e], sq);
    }
    for (int i = tid * 8; i < nk; i += 2048) {
      kv_load8(pr + g.ck + i, v);
#pragma unroll
      for (int e = 0; e < 8; e++) sk = __builtin_fmaf(v[e], v[e], sk);
    }
    sq = wave_sum_f32(sq);
    sk = wave_sum_f32(sk);
    if ((tid & 63) == 0) {
      red[tid >> 6] = sq;
      red[4 + (tid >> 6)] = sk;
    }
    __syncthreads();
    const float fq = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)g.q_mean + g.eps);
    const float fk = 1.0f / sqrtf(((red[4] + red[5]) + (red[6] + red[7])) / (float)g.k_mean + g.eps);
    for (int i = tid * 8; i < nq; i += 2048) octet_scale(pr + g.cq + i, fq, g.q_norm + i);
    for (int i = tid * 8; i < nk; i += 2048) octet_scale(pr + g.ck + i, fk, g.k_norm + i);
  }
  T* vk = a.v_kept + (size_t)r * a.ld_vk;
  if (g.vmix == VMIX_KEEP)
    for (int i = tid; i < nv; i += 256) vk[i] = pr[g.cv + i];
  if (g.vmix == VMIX_MIX) {
    const float la = *g.lambda;
    for (int i = tid; i < nv; i += 256) pr[g.cv + i] = kv_from<T>(__builtin_fmaf(la, kv_to(vk[i]), (1.0f - la) * kv_to(pr[g.cv + i])));
  }
}

// ---- behind both: the linear branch's norm and gate; the cache rows of the chunk each sequence's part of the pass ends in ----------
template <typename T, int P>
__global__ __launch_bounds__(256) void k_mix_rows(const MixRows<T> a, float eps) {
  __shared__ float red[4];
  const int r = blockIdx.x, tid = threadIdx.x;
  const PassRow rw = a.rows[r];
  const T* pr = a.proj + (size_t)r * a.ldp;
  if (a.li.H) {
    const LinGeom& g = a.li;
    const int n = g.H * g.V;
    const float* o = a.lin + (size_t)r * n;
    float s = 0.f;
    for (int i = tid; i < n; i += 256) s = __builtin_fmaf(o[i], o[i], s);
    s = wave_sum_f32(s);
    if ((tid & 63) == 0) red[tid >> 6] = s;
    __syncthreads();
    const float f = g.out_scale / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)(g.H * g.v_true) + eps);
    for (int i = tid; i < n; i += 256)
      split_store<P>(o[i] * (f * g.norm[i] * kv_to(pr[g.cg + i])), a.cat + (size_t)r * a.ldc + a.lin_off + i, a.cat_plane);
  }
  if (a.at.H) {
    const AttnGeom& g = a.at;
    const PassSeq sq = a.seqs[rw.seq];
    const int last = sq.pos0 + sq.n - 1;
    if (rw.pos < attn_first(g, last)) return;
    T* kc = (T*)(sq.slab + a.rs.k);
    T* vc = (T*)(sq.slab + a.rs.v);
    const size_t at = (size_t)(rw.pos % g.span);
    for (int i = tid; i < g.G * g.D; i += 256) kc[((size_t)(i / g.D) * g.rows + at) * g.D + i % g.D] = pr[g.ck + i];
    for (int i = tid; i < g.G * g.V; i += 256) vc[((size_t)(i / g.V) * g.rows + at) * g.V + i % g.V] = pr[g.cv + i];
  }
}

}  // namespace crabml_hip
