// hybrid_latent.hpp -- latent attention of the hybrid decoder: a token leaves one row, its normed latent and one rotated key part, and
// every head's keys and values are products of the latent.
//
// Prompt pass: the products are formed (keys and values of all heads, one k_gemm_bf16 over the pass's rows and the earlier rows still
// visible) and k_attn_rows reads them.
//   k_latent_rows    norm of the latents, rotation of queries and keys; earlier rows are taken from the cache
//   k_latent_append  the cache rows that later tokens can see
// Decode step: queries are taken to the latent instead, so a step reads the cache once, whatever the number of heads.
//   k_latent_query   the same norm and rotation, the cache append; per head W_k^T q
//   k_latent_attn    16 heads of one sequence over a split of its cached rows, on the matrix cores
//   k_latent_value   merge of the splits; per head W_v times the averaged latent
#pragma once
#include "hybrid_rows.hpp"
#include "hybrid_step.hpp"

namespace crabml_hip {

// ---- prompt pass ---------------------------------------------------------------------------------------------------------------------
template <typename T, int P>
__device__ __forceinline__ T latent_elem(const MixRows<T>& a, size_t row, int i) {  // as the cache holds it
  const unsigned short* p = a.lat + row * a.la.ldl + i;
  if constexpr (P == 1)
    return *p;
  else
    return bf2f(p[0]) + (bf2f(p[a.lat_plane]) + bf2f(p[2 * a.lat_plane]));
}

template <typename T, int P>
__global__ __launch_bounds__(256) void k_latent_rows(const MixRows<T> a) {
  __shared__ float red[4], turn[256];  // cos, sin per pair
  const AttnGeom& g = a.at;
  const LatGeom& l = a.la;
  const int r = blockIdx.x, tid = threadIdx.x;
  const PassRow rw = a.rows[r];
  unsigned short* lat = a.lat + (size_t)r * l.ldl;
  T* rot = a.rot + (size_t)r * l.rot;
  const PassSeq sq = a.seqs[rw.seq];
  if (r >= a.M) {  // an earlier position: zero where this layer no longer sees it (and no longer has it)
    const bool seen = rw.pos >= attn_first(g, sq.pos0);
    const T* c = (const T*)(sq.slab + a.rs.k) + (size_t)(rw.pos % g.span) * (l.rank + l.rot);
    for (int i = tid; i < l.rank; i += 256) {
      const T v = seen ? c[i] : kv_from<T>(0.f);
      if constexpr (P == 1)
        lat[i] = v;
      else
        split_store<P>(v, lat + i, a.lat_plane);
    }
    for (int i = tid; i < l.rot; i += 256) rot[i] = seen ? c[l.rank + i] : kv_from<T>(0.f);
    return;
  }
  T* pr = const_cast<T*>(a.proj) + (size_t)r * a.ldp;
  if (tid < l.rot / 2) {
    const float ang = reduced_angle(rw.pos, l.freq[tid]);
    turn[2 * tid] = cosf(ang);
    turn[2 * tid + 1] = sinf(ang);
  }
  float s = 0.f;
  for (int i = tid; i < l.rank; i += 256) {
    const float v = kv_to(pr[l.cc + i]);
    s = __builtin_fmaf(v, v, s);
  }
  s = wave_sum_f32(s);
  if ((tid & 63) == 0) red[tid >> 6] = s;
  __syncthreads();
  const float f = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)l.rank_true + g.eps);
  for (int i = tid; i < l.rank; i += 256) split_store<P>(kv_to(pr[l.cc + i]) * (f * l.norm[i]), lat + i, a.lat_plane);
  const int np = l.rot / 2;
  for (int i = tid; i < np * (g.H + 1); i += 256) {  // head H: the shared key part
    const int h = i / np, p = i % np;
    const T* src = h < g.H ? pr + g.cq + h * g.D + l.dim + 2 * p : pr + l.cr + 2 * p;
    T* dst = h < g.H ? const_cast<T*>(src) : rot + 2 * p;
    const float u = kv_to(src[0]), v = kv_to(src[1]), c = turn[2 * p], sn = turn[2 * p + 1];
    dst[0] = kv_from<T>(u * c - v * sn);
    dst[1] = kv_from<T>(v * c + u * sn);
  }
}

template <typename T, int P>
__global__ __launch_bounds__(256) void k_latent_append(const MixRows<T> a) {
  const LatGeom& l = a.la;
  const int r = blockIdx.x, tid = threadIdx.x;
  const PassRow rw = a.rows[r];
  const PassSeq sq = a.seqs[rw.seq];
  if (rw.pos < attn_first(a.at, sq.pos0 + sq.n - 1)) return;
  T* c = (T*)(sq.slab + a.rs.k) + (size_t)(rw.pos % a.at.span) * (l.rank + l.rot);
  for (int i = tid; i < l.rank; i += 256) c[i] = latent_elem<T, P>(a, r, i);
  for (int i = tid; i < l.rot; i += 256) c[l.rank + i] = a.rot[(size_t)r * l.rot + i];
}

// ---- decode step ---------------------------------------------------------------------------------------------------------------------
#define LAT_HEADS 16       // query heads per workgroup: the rows of a matrix instruction
#define LAT_SPLITS 16      // most workgroups that share a sequence's cached rows
#define LAT_SLICE 64       // latent columns per workgroup of k_latent_query
#define LAT_MAX_ROW 768    // rank + rot
template <typename T>
struct LatTile {
  static constexpr int KT = sizeof(T) == 2 ? 64 : 32, PAD = 16 / sizeof(T), LP = KT + 4;
};
struct LatStep {
  AttnGeom at;
  LatGeom la;
  RunState rs;
  const StepSeq* seq = nullptr;
  const float* proj = nullptr;  // [B][ldp]
  float* q = nullptr;           // [B][H][rank + rot]
  float* part = nullptr;        // [B][H][LAT_SPLITS][rank + 2]: unnormalized sums, maximum, denominator
  float* cat = nullptr;         // [B][ldc]
  int B = 0, ldp = 0, ldc = 0;
  int splits = LAT_SPLITS;
};
// rows that are there, rows per split
struct LatRange {
  int n, per;
};
template <typename T>
__device__ __forceinline__ LatRange latent_range(const AttnGeom& g, int splits, int pos) {
  constexpr int KT = LatTile<T>::KT;
  LatRange r;
  r.n = g.window && pos >= g.span ? g.span : pos % g.span + 1;
  const int tiles = (r.n + KT - 1) / KT;
  r.per = (tiles + splits - 1) / splits * KT;
  return r;
}

// grid: H * slices workgroups of one head's latent columns (all rows of the batch), then one per row for everything else
template <typename T>
__global__ __launch_bounds__(256) void k_latent_query(const LatStep a) {
  extern __shared__ __attribute__((aligned(16))) float lat_lds[];  // [16][ldq]; the last workgroups: cos, sin per pair
  __shared__ float red[4];
  const AttnGeom& g = a.at;
  const LatGeom& l = a.la;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg();
  const int slices = (l.rank + LAT_SLICE - 1) / LAT_SLICE, row_w = l.rank + l.rot;
  if ((int)blockIdx.x >= g.H * slices) {
    const int b = blockIdx.x - g.H * slices, np = l.rot / 2;
    const StepSeq sq = a.seq[b];
    const float* pr = a.proj + (size_t)b * a.ldp;
    T* c = (T*)(sq.slab + a.rs.k) + (size_t)(sq.pos % g.span) * row_w;
    if (tid < np) {
      const float ang = reduced_angle(sq.pos, l.freq[tid]);
      lat_lds[2 * tid] = cosf(ang);
      lat_lds[2 * tid + 1] = sinf(ang);
    }
    float s = 0.f;
    for (int i = tid; i < l.rank; i += 256) s = __builtin_fmaf(pr[l.cc + i], pr[l.cc + i], s);
    s = wave_sum_f32(s);
    if (lane == 0) red[wave] = s;
    __syncthreads();
    const float f = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)l.rank_true + g.eps);
    for (int i = tid; i < l.rank; i += 256) c[i] = kv_from<T>(pr[l.cc + i] * (f * l.norm[i]));
    for (int i = tid; i < np * (g.H + 1); i += 256) {  // head H: the shared key part
      const int h = i / np, p = i % np;
      const float* src = h < g.H ? pr + g.cq + h * g.D + l.dim + 2 * p : pr + l.cr + 2 * p;
      const float cs = lat_lds[2 * p], sn = lat_lds[2 * p + 1];
      const float u = src[0] * cs - src[1] * sn, v = src[1] * cs + src[0] * sn;
      if (h < g.H) {
        float* d = a.q + ((size_t)b * g.H + h) * row_w + l.rank + 2 * p;
        d[0] = u;
        d[1] = v;
      } else {
        c[l.rank + 2 * p] = kv_from<T>(u);
        c[l.rank + 2 * p + 1] = kv_from<T>(v);
      }
    }
    return;
  }
  const int h = blockIdx.x / slices, r0 = blockIdx.x % slices * LAT_SLICE;
  const int r1 = r0 + LAT_SLICE < l.rank ? r0 + LAT_SLICE : l.rank;
  // a wave: 16 latent columns of every row of the batch.  (The last weight row's reads run past its end into zeros: dim is padded to 32
  // here by zero queries, and the matrix has 32 elements to spare.)
  const int k32 = (l.dim + 31) & ~31, ldq = k32 + 4, fr = lane & 15, fk = lane >> 4;
  const int rr = r0 + wave * 16 + fr;
  const unsigned short* w = l.w_q + ((size_t)h * l.rank + (rr < r1 ? rr : r1 - 1)) * l.dim + fk * 8;
  bf16x8 wf[8];  // (dim is at most 256)
#pragma unroll
  for (int i = 0; i < 8; i++)
    if (i * 32 < l.dim) __builtin_memcpy(&wf[i], w + i * 32, 16);
  for (int i = tid; i < 16 * (k32 / 4); i += 256) {
    const int b = i / (k32 / 4), c = i % (k32 / 4) * 4;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (b < a.B && c < l.dim) v = *(const f32x4*)(a.proj + (size_t)b * a.ldp + g.cq + h * g.D + c);
    *(f32x4*)(lat_lds + b * ldq + c) = v;
  }
  __syncthreads();
  if (r0 + wave * 16 >= r1) return;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 8; i++)
    if (i * 32 < l.dim) {
      float v[8];
      read8(lat_lds + fr * ldq + i * 32 + fk * 8, v);
      bf16x8 hi, mid, lo;
      split3(v, hi, mid, lo);
      acc = mfma_bf16(hi, wf[i], mfma_bf16(mid, wf[i], mfma_bf16(lo, wf[i], acc)));
    }
  if (rr < r1) {
#pragma unroll
    for (int e = 0; e < 4; e++)
      if (fk * 4 + e < a.B) a.q[((size_t)(fk * 4 + e) * g.H + h) * row_w + rr] = acc[e];
  }
}

// out += P V over one tile: P [16][KT] f32 (LDS), V [KT][ld] (LDS rows of the cache); this lane's column of V
__device__ __forceinline__ f32x4 latent_pv(const float* p, const unsigned short* v, int ld, f32x4 acc) {
  const int fr = threadIdx.x & 15, fk = threadIdx.x >> 4 & 3;
#pragma unroll
  for (int k = 0; k < LatTile<unsigned short>::KT; k += 32) {
    float w[8];
    read8(p + fr * LatTile<unsigned short>::LP + k + fk * 8, w);
    bf16x8 fa, fb;
    unsigned short t[8];
#pragma unroll
    for (int e = 0; e < 8; e++) {
      fa[e] = (__bf16)w[e];
      t[e] = v[(size_t)(k + fk * 8 + e) * ld];
    }
    __builtin_memcpy(&fb, t, 16);
    acc = mfma_bf16(fa, fb, acc);
  }
  return acc;
}
__device__ __forceinline__ f32x4 latent_pv(const float* p, const float* v, int ld, f32x4 acc) {
  const int fr = threadIdx.x & 15, fk = threadIdx.x >> 4 & 3;
#pragma unroll
  for (int k = 0; k < LatTile<float>::KT; k += 4)
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(p[fr * LatTile<float>::LP + k + fk], v[(size_t)(k + fk) * ld], acc, 0, 0, 0);
  return acc;
}

// NT: latent columns up to 64 NT
template <typename T, int NT>
__global__ __launch_bounds__(256) void k_latent_attn(const LatStep a) {
  constexpr int KT = LatTile<T>::KT, LP = LatTile<T>::LP;
  extern __shared__ __attribute__((aligned(16))) char latt_lds[];
  __shared__ float alpha[LAT_HEADS];
  const AttnGeom& g = a.at;
  const LatGeom& l = a.la;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg(), fr = lane & 15, fk = lane >> 4;
  const int split = blockIdx.x, h0 = blockIdx.y * LAT_HEADS, b = blockIdx.z;
  const int row_w = l.rank + l.rot, w32 = (row_w + 31) & ~31, ld = w32 + LatTile<T>::PAD, cpr = w32 / 8;
  T* q_s = (T*)latt_lds;               // [16][ld]
  T* k_s = q_s + LAT_HEADS * ld;       // [KT][ld]
  float* p_s = (float*)(k_s + KT * ld);  // [16][LP]
  const int nh = g.H - h0 < LAT_HEADS ? g.H - h0 : LAT_HEADS;
  const float* q = a.q + ((size_t)b * g.H + h0) * row_w;
  const StepSeq sq = a.seq[b];
  const LatRange rg = latent_range<T>(g, a.splits, sq.pos);
  const int lo = split * rg.per, hi = lo + rg.per < rg.n ? lo + rg.per : rg.n;
  if (lo >= hi) return;  // (whole workgroup)
  const T* cache = (const T*)(sq.slab + a.rs.k);
  // a tile's octets in row order, 256 at a time: thread t starts at (row tr0, octet tc0) and goes on by (dr, dc)
  const int tr0 = tid / cpr, tc0 = tid % cpr, dr = 256 / cpr, dc = 256 % cpr;
  constexpr int UN = sizeof(T) == 2 ? 9 : 5;  // octets in flight per thread
  auto stage = [&](int t0, int n, int rows, const T* src, T* dst) {  // rows of LDS; those from n on are zero
    int r = tr0, c = tc0;
    while (true) {
      Oct<T> v[UN];
      int at[UN];
#pragma unroll
      for (int u = 0; u < UN; u++) {
        at[u] = r < rows ? r * ld + c * 8 : -1;
        v[u] = oct_zero<T>();
        if (r < n && r < rows && c * 8 < row_w) v[u] = oct_load(src + (size_t)(t0 + r) * row_w + c * 8);
        r += dr;
        c += dc;
        if (c >= cpr) {
          c -= cpr;
          r++;
        }
      }
#pragma unroll
      for (int u = 0; u < UN; u++)
        if (at[u] >= 0) oct_store(dst + at[u], v[u]);
      if (__all(r >= rows)) return;
    }
  };
  {
    constexpr int UQ = LAT_HEADS * LAT_MAX_ROW / 8 / 256;
    int r = tr0, c = tc0, at[UQ];
    float v[UQ][8];
#pragma unroll
    for (int u = 0; u < UQ; u++) {
      at[u] = r < LAT_HEADS ? r * ld + c * 8 : -1;
#pragma unroll
      for (int e = 0; e < 8; e++) v[u][e] = 0.f;
      if (r < nh && c * 8 < row_w) read8(q + (size_t)r * row_w + c * 8, v[u]);
      r += dr;
      c += dc;
      if (c >= cpr) {
        c -= cpr;
        r++;
      }
    }
#pragma unroll
    for (int u = 0; u < UQ; u++)
      if (at[u] >= 0) {
        T t[8];
#pragma unroll
        for (int e = 0; e < 8; e++) t[e] = kv_from<T>(v[u][e]);
        __builtin_memcpy(q_s + at[u], t, sizeof t);
      }
  }
  f32x4 o[NT];
#pragma unroll
  for (int j = 0; j < NT; j++) o[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m[4], den[4];  // of heads 4 wave .. 4 wave + 3
#pragma unroll
  for (int i = 0; i < 4; i++) {
    m[i] = -INFINITY;
    den[i] = 0.f;
  }
  for (int t0 = lo; t0 < hi; t0 += KT) {
    __syncthreads();  // the previous tile has been read
    stage(t0, hi - t0, KT, cache, k_s);
    __syncthreads();
    if (wave < KT / 16) {
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < w32; k += 32) s = mma_rows(q_s + fr * ld + k, k_s + (wave * 16 + fr) * ld + k, 32, s);
#pragma unroll
      for (int e = 0; e < 4; e++) p_s[(fk * 4 + e) * LP + wave * 16 + fr] = t0 + wave * 16 + fr < hi ? s[e] * g.scale : -INFINITY;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int h = wave * 4 + i;
      const float s = lane < KT ? p_s[h * LP + lane] : -INFINITY;
      const float mx = fmaxf(m[i], wave_max_f32(s));  // (a tile has at least one row: finite)
      const float e = __expf(s - mx), w = __expf(m[i] - mx);
      den[i] = __builtin_fmaf(den[i], w, wave_sum_f32(e));
      m[i] = mx;
      if (lane < KT) p_s[h * LP + lane] = e;
      if (lane == 0) alpha[h] = w;
    }
    __syncthreads();
    const f32x4 w = *(const f32x4*)&alpha[fk * 4];
#pragma unroll
    for (int j = 0; j < NT; j++) {
      const int c = (wave + 4 * j) * 16;
      if (c < l.rank) o[j] = latent_pv(p_s, k_s + c + fr, ld, o[j] * w);
    }
  }
  const int pw = l.rank + 2;
  float* part = a.part + (((size_t)b * g.H + h0) * LAT_SPLITS + split) * pw;
#pragma unroll
  for (int j = 0; j < NT; j++) {
    const int c = (wave + 4 * j) * 16 + fr;
    if (c < l.rank) {
#pragma unroll
      for (int e = 0; e < 4; e++)
        if (fk * 4 + e < nh) part[(size_t)(fk * 4 + e) * LAT_SPLITS * pw + c] = o[j][e];
    }
  }
#pragma unroll
  for (int i = 0; i < 4; i++) {
    const int h = wave * 4 + i;
    if (lane == 0 && h < nh) {
      part[(size_t)h * LAT_SPLITS * pw + l.rank] = m[i];
      part[(size_t)h * LAT_SPLITS * pw + l.rank + 1] = den[i];
    }
  }
}

// grid: (H * slices of VS value columns, B); SP: splits
template <typename T, int SP, int VS>
__global__ __launch_bounds__(256) void k_latent_value(const LatStep a) {
  __shared__ __attribute__((aligned(16))) float x[LAT_MAX_ROW];
  const AttnGeom& g = a.at;
  const LatGeom& l = a.la;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg(), b = blockIdx.y;
  const int slices = (g.V + VS - 1) / VS, h = blockIdx.x / slices, v0 = blockIdx.x % slices * VS;
  const int v1 = v0 + VS < g.V ? v0 + VS : g.V;
  const LatRange rg = latent_range<T>(g, SP, a.seq[b].pos);
  const int active = (rg.n + rg.per - 1) / rg.per, pw = l.rank + 2;
  const float* part = a.part + ((size_t)b * g.H + h) * LAT_SPLITS * pw;
  int lpr = 1;  // lanes per weight row
  while (lpr < 64 && lpr * 8 < l.rank) lpr <<= 1;
  const int rows = 64 / lpr, sub = lane / lpr, k0 = lane % lpr * 8;
  const unsigned short* wv = l.w_kv + (size_t)(g.H * l.dim + h * g.V) * l.ldl;
  // a wave's VS / 4 rows, `rows` at a time: their first octets are on their way while the splits are merged
  constexpr int RW = VS / 4;
  i32x4 wf[RW];
  const int kf = k0 < l.ldl ? k0 : 0;
#pragma unroll
  for (int j = 0; j < RW; j++) {
    const int v = v0 + wave * RW + j * rows + sub;
    if (j * rows < RW) wf[j] = *(const i32x4*)(wv + (size_t)(v < v1 ? v : v1 - 1) * l.ldl + kf);
  }
  float w[SP], ds[SP], top = -INFINITY, den = 0.f;
#pragma unroll
  for (int s = 0; s < SP; s++) {  // (requests without branches; a split that is not there counts nothing)
    const float* p = part + (size_t)s * pw + l.rank;
    w[s] = p[0];
    ds[s] = p[1];
  }
#pragma unroll
  for (int s = 0; s < SP; s++) {
    w[s] = s < active ? w[s] : -INFINITY;
    top = fmaxf(top, w[s]);
  }
#pragma unroll
  for (int s = 0; s < SP; s++) {
    w[s] = __expf(w[s] - top);
    den = __builtin_fmaf(s < active ? ds[s] : 0.f, w[s], den);
  }
  const float inv = 1.0f / den;
  for (int i = tid; i < l.ldl; i += 256) {
    float p[SP], o = 0.f;
#pragma unroll
    for (int s = 0; s < SP; s++) p[s] = part[(size_t)s * pw + (i < l.rank ? i : 0)];
#pragma unroll
    for (int s = 0; s < SP; s++) o = __builtin_fmaf(s < active ? p[s] : 0.f, w[s], o);
    x[i] = i < l.rank ? o * inv : 0.f;
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < RW; j++) {
    if (j * rows >= RW) break;
    const int v = v0 + wave * RW + j * rows + sub;
    float s = 0.f;
    for (int k = k0; k < l.ldl; k += lpr * 8) {  // (one round up to 512 latent columns; the padding is zero on both sides)
      if (k != k0) wf[j] = *(const i32x4*)(wv + (size_t)(v < v1 ? v : v1 - 1) * l.ldl + k);
      float xv[8];
      read8(x + k, xv);
#pragma unroll
      for (int e = 0; e < 4; e++) {
        s = __builtin_fmaf(__builtin_bit_cast(float, (unsigned)wf[j][e] << 16), xv[2 * e], s);
        s = __builtin_fmaf(__builtin_bit_cast(float, (unsigned)wf[j][e] & 0xffff0000u), xv[2 * e + 1], s);
      }
    }
    if (lpr == 64)
      s = wave_sum_f32(s);
    else
      for (int o = 1; o < lpr; o <<= 1) s += __shfl_xor(s, o, 64);
    if (k0 == 0 && v < v1 && j * rows + sub < RW) a.cat[(size_t)b * a.ldc + h * g.V + v] = s * g.out_scale;
  }
}

// half as many splits once the chip is full: every split's sums pass through memory
inline int latent_splits(int B, int H) { return B * H >= 512 ? LAT_SPLITS / 2 : LAT_SPLITS; }
template <typename T>
inline size_t latent_attn_lds(const LatGeom& l) {
  const size_t ld = align_up((size_t)(l.rank + l.rot), 32) + LatTile<T>::PAD;
  return (LAT_HEADS + LatTile<T>::KT) * ld * sizeof(T) + (size_t)LAT_HEADS * LatTile<T>::LP * sizeof(float);
}
template <typename T, int NT>
inline int launch_latent_attn_t(crabml_hip_device* dev, crabml_hip_device::ProfRec* rec, const LatStep& a) {
  const size_t lds = latent_attn_lds<T>(a.la);
  CH_HIP(dev, raise_dyn_lds(dev, (const void*)k_latent_attn<T, NT>, (int)lds));
  launch_k(dev->stream, rec, k_latent_attn<T, NT>, dim3(a.splits, (a.at.H + LAT_HEADS - 1) / LAT_HEADS, a.B), dim3(256), lds, a);
  return 0;
}
template <typename T>
inline int launch_latent_attn(crabml_hip_device* dev, crabml_hip_device::ProfRec* rec, const LatStep& a) {
  if (a.la.rank <= 128) return launch_latent_attn_t<T, 2>(dev, rec, a);
  if (a.la.rank <= 256) return launch_latent_attn_t<T, 4>(dev, rec, a);
  if (a.la.rank <= 512) return launch_latent_attn_t<T, 8>(dev, rec, a);
  return launch_latent_attn_t<T, 12>(dev, rec, a);
}
template <typename T>
inline void launch_latent_query(hipStream_t st, crabml_hip_device::ProfRec* rec, const LatStep& a) {
  const size_t fl = 16 * (align_up((size_t)a.la.dim, 32) + 4);  // (at least the 256 of a whole turn table)
  launch_k(st, rec, k_latent_query<T>, dim3(a.at.H * ((a.la.rank + LAT_SLICE - 1) / LAT_SLICE) + a.B), dim3(256), fl * sizeof(float), a);
}
template <typename T>
inline void launch_latent_value(hipStream_t st, crabml_hip_device::ProfRec* rec, const LatStep& a) {
  if (a.splits == LAT_SPLITS)
    launch_k(st, rec, k_latent_value<T, LAT_SPLITS, 32>, dim3(a.at.H * ((a.at.V + 31) / 32), a.B), dim3(256), 0, a);
  else
    launch_k(st, rec, k_latent_value<T, LAT_SPLITS / 2, 64>, dim3(a.at.H * ((a.at.V + 63) / 64), a.B), dim3(256), 0, a);
}

}  // namespace crabml_hip
