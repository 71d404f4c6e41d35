// gemm_bf16.hip -- the kernel behind gemm_bf16.hpp
#include <cmath>
#include <cstdlib>

#include "gemm_bf16.hpp"

namespace crabml_hip {

// 16 bytes per lane from memory into LDS at l + 16 lane (l: wave-uniform).  As assembly, because the compiler would wait for ALL of them
// in front of the next LDS read (it cannot tell the buffers apart); who waits for what is landed_barrier's business.
// (m0, the LDS address of such a load, needs one wait state behind its write; nothing else here uses it.)
__device__ __forceinline__ void lds_dma16(const void* g, const void* l) {
  const unsigned at = (unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)(size_t)(const __attribute__((address_space(3))) void*)l);
  asm volatile("s_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, off" ::"v"(g), "s"(at) : "memory");
}
// four values as f32 / as bf16 planes (16- and 8-byte stores)
__device__ __forceinline__ void store4(float* p, const float (&v)[4]) { *(f32x4*)p = f32x4{v[0], v[1], v[2], v[3]}; }

// S > 1: k is cut into S pieces, one workgroup each.  A workgroup leaves its accumulators in ws (write-through) and counts itself in; the
// one that comes last adds the others' pieces to its own, in piece order, and goes on to the epilogue.  The counter is left at zero.
// waits until at most N of this wave's memory requests are outstanding, then for the workgroup.  (__syncthreads would drain them all.)
template <int N>
__device__ __forceinline__ void landed_barrier() {
  asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(N) : "memory");
}

// (NS: GEMM_OUT_STREAMS with up to that many streams)
template <int BM, int BN, int WGM, int WGN, int ST, int P, int OUT, int NS>
__global__ __launch_bounds__(64 * WGM * WGN) void k_gemm_bf16(const GemmBf16 g, int S, float* __restrict__ ws, unsigned* __restrict__ tick) {
  constexpr int WM = BM / WGM, WN = BN / WGN, TM = WM / 16, TN = WN / 16;
  constexpr int HR = BM < 64 ? BM : 64, LC = BN + 4;  // the epilogue's slab of rows in LDS
  constexpr int NT = 64 * WGM * WGN, FA = BM * 8 / NT, FB = BN * 8 / NT;  // threads; a step's requests per thread
  static_assert(WN == 64 && HR % WM == 0 && BM * 8 % NT == 0 && BN * 8 % NT == 0, "a wave's columns are one square-sum piece; its rows lie in one slab");
  __shared__ __attribute__((aligned(16))) unsigned short lds[ST][(BM + BN) * 64];
  static_assert(sizeof(lds) >= (HR * LC + BM) * sizeof(float), "the epilogue reuses the tiles' LDS");
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg();
  const int wm = wave / WGN, wn = wave % WGN;
  const int mt = (g.M + BM - 1) / BM, nt = (g.N + BN - 1) / BN, total = mt * nt * S;
  int id = blockIdx.x;
  {  // XCD x (= id % 8) takes a contiguous run of tiles
    const int x = id & 7, i = id >> 3, q = total >> 3, r = total & 7;
    id = x * q + (x < r ? x : r) + i;
  }
  const int piece = id / mt % S, tile = id / mt / S * mt + id % mt;  // row tiles fastest, then pieces: a weight tile's readers are neighbours
  const int row0 = (tile % mt) * BM, col0 = (tile / mt) * BN;
  f32x4 acc[TM][TN];
#pragma unroll
  for (int i = 0; i < TM; i++)
#pragma unroll
    for (int j = 0; j < TN; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int steps = g.K / 64, all = steps * P;
  const int s_lo = (int)((long long)all * piece / S), s_hi = (int)((long long)all * (piece + 1) / S);
  auto fetch = [&](int s, int buf) {
    const int p = P == 1 ? 0 : s / steps, k0 = (P == 1 ? s : s - p * steps) * 64;
    const unsigned short* ap = g.a + (P == 1 ? 0 : (size_t)(P - 1 - p) * g.a_plane) + k0;  // (the smallest plane first)
#pragma unroll
    for (int it = 0; it < FA; it++) {
      const int slot = it * NT + tid, r = slot >> 3, c = (slot & 7) ^ ((r >> 1) & 7);
      lds_dma16(ap + (size_t)(row0 + r) * g.K + c * 8, &lds[buf][(it * NT + wave * 64) * 8]);
    }
#pragma unroll
    for (int it = 0; it < FB; it++) {
      const int slot = it * NT + tid, r = slot >> 3, c = (slot & 7) ^ ((r >> 1) & 7);
      lds_dma16(g.w + (size_t)(col0 + r) * g.K + k0 + c * 8, &lds[buf][BM * 64 + (it * NT + wave * 64) * 8]);
    }
  };
  float factor = 1.f;  // of row tid, waiting for the epilogue
  if (g.sq_in != nullptr && tid < BM) {
    const float* q = g.sq_in + (size_t)(row0 + tid < g.M ? row0 + tid : g.M - 1) * g.n_sq;
    float s = 0.f;
#pragma unroll 8
    for (int i = 0; i < g.n_sq; i++) s += q[i];
    factor = (g.gain ? *g.gain : 1.0f) / sqrtf(s / (float)g.mean_n + g.eps);
  }
  const int fr = lane & 15, fk = lane >> 4;
#pragma unroll
  for (int i = 0; i < ST - 1; i++)
    if (s_lo + i < s_hi) fetch(s_lo + i, i);
  int buf = 0;
  for (int s = s_lo; s < s_hi; s++) {
    // step s has landed -- this wave's part (later steps' requests stay out), then everybody's -- and step s - 1 has been read by all
    if (s + ST - 2 < s_hi)
      landed_barrier<(ST - 2) * (FA + FB)>();
    else
      landed_barrier<0>();
    if (s + ST - 1 < s_hi) fetch(s + ST - 1, buf == 0 ? ST - 1 : buf - 1);
    const unsigned short* la = &lds[buf][0];
    const unsigned short* lb = la + BM * 64;
#pragma unroll
    for (int kk = 0; kk < 2; kk++) {
      bf16x8 fa[TM], fb[TN];
#pragma unroll
      for (int i = 0; i < TM; i++) {
        const int r = wm * WM + i * 16 + fr;
        fa[i] = *(const bf16x8*)(la + r * 64 + (((kk * 4 + fk) ^ ((r >> 1) & 7)) * 8));
      }
#pragma unroll
      for (int j = 0; j < TN; j++) {
        const int r = wn * WN + j * 16 + fr;
        fb[j] = *(const bf16x8*)(lb + r * 64 + (((kk * 4 + fk) ^ ((r >> 1) & 7)) * 8));
      }
#pragma unroll
      for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++) acc[i][j] = mfma_bf16(fa[i], fb[j], acc[i][j]);
    }
    buf = buf + 1 == ST ? 0 : buf + 1;
  }
  if (S > 1) {
    constexpr int FRAG = TM * TN * 2;  // 8-byte halves of a lane's accumulators
    unsigned long long* base = (unsigned long long*)ws + (size_t)tile * S * NT * FRAG + tid;
    unsigned long long* mine = base + (size_t)piece * NT * FRAG;
#pragma unroll
    for (int i = 0; i < TM; i++)
#pragma unroll
      for (int j = 0; j < TN; j++)
#pragma unroll
        for (int e = 0; e < 2; e++) {
          const f32x2 v = {acc[i][j][2 * e], acc[i][j][2 * e + 1]};
          __hip_atomic_store(mine + ((i * TN + j) * 2 + e) * NT, __builtin_bit_cast(unsigned long long, v), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this thread's write-through stores have been acknowledged
    __shared__ unsigned s_last;
    __syncthreads();
    if (tid == 0) s_last = __hip_atomic_fetch_add(tick + tile, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (unsigned)(S - 1);
    __syncthreads();
    if (!s_last) return;
    if (tid == 0) __hip_atomic_store(tick + tile, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
#pragma unroll
    for (int i = 0; i < TM; i++)
#pragma unroll
      for (int j = 0; j < TN; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int q = 0; q < S; q++) {  // (its own piece from memory as well: one order of addition, whoever is last)
      const unsigned long long* p = base + (size_t)q * NT * FRAG;
#pragma unroll
      for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++)
#pragma unroll
          for (int e = 0; e < 2; e++) {
            const f32x2 v = __builtin_bit_cast(f32x2, __hip_atomic_load(p + ((i * TN + j) * 2 + e) * NT, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT));
            acc[i][j][2 * e] += v[0];
            acc[i][j][2 * e + 1] += v[1];
          }
    }
  }
  // epilogue: the tile goes through LDS in slabs of HR rows, so that a thread has eight neighbouring columns of a row
  float* lc = (float*)lds;            // [HR][LC]
  float* lf = lc + HR * LC;           // [BM] row factors
  float xr = 0.f, xl = 0.f;
  if constexpr (OUT == GEMM_OUT_XIELU) {
    xr = g.xielu[0];
    xl = g.xielu[1];
  }
  if constexpr (OUT == GEMM_OUT_STREAMS && NS == 4) {
    // Up to four streams: a slab's rows of all of them are requested, two units of eight columns at a time, before the accumulators take
    // their way through LDS, so that a thread has sixteen requests out.
    constexpr int UNITS = HR * BN / 8 / NT, UG = 2;
    static_assert(UNITS % UG == 0, "units come in pairs");
    const_f32 *coef = (const_f32*)(size_t)g.sm.coef, *inw = (const_f32*)(size_t)g.sm.in;
#pragma unroll 1
    for (int h = 0; h < BM / HR; h++) {
#pragma unroll
      for (int u0 = 0; u0 < UNITS; u0 += UG) {
        f32x4 old[UG][2][4];
        float* xs[UG];
        int row[UG], col[UG], lr[UG];
        bool in[UG];
#pragma unroll
        for (int u = 0; u < UG; u++) {
          const int unit = (u0 + u) * NT + tid, r = unit / (BN / 8), c = unit % (BN / 8) * 8;
          row[u] = row0 + h * HR + r;
          col[u] = col0 + c;
          lr[u] = r * LC + c;
          in[u] = row[u] < g.M && col[u] < g.N;
          xs[u] = g.x + (size_t)row[u] * g.ldx + col[u];
          if (in[u]) {
#pragma unroll
            for (int s = 0; s < 4; s++) {
              const float* p = xs[u] + (s < g.sm.n ? s : 0) * g.sm.stride;
              old[u][0][s] = *(const f32x4*)p;
              old[u][1][s] = *(const f32x4*)(p + 4);
            }
          }
        }
        if (u0 == 0) {  // (LDS hand-overs that leave the requests out)
          asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
          if (h == 0 && tid < BM) lf[tid] = factor;
          if (wm * WM / HR == h) {
#pragma unroll
            for (int i = 0; i < TM; i++)
#pragma unroll
              for (int j = 0; j < TN; j++)
#pragma unroll
                for (int e = 0; e < 4; e++) lc[(wm * WM % HR + i * 16 + fk * 4 + e) * LC + wn * WN + j * 16 + fr] = acc[i][j][e];
          }
          asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        }
#pragma unroll
        for (int u = 0; u < UG; u++) {
          float sq = 0.f;
          if (in[u]) {
            const float f = lf[h * HR + lr[u] / LC];
            f32x4 y[2], n[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int k = 0; k < 2; k++) {
              y[k] = *(const f32x4*)(lc + lr[u] + 4 * k) * f;
              if (g.bias) y[k] += *(const f32x4*)(g.bias + col[u] + 4 * k);
            }
#pragma unroll
            for (int t = 0; t < 4; t++) {
              const_f32* c = coef + t * HC_ROW;
#pragma unroll
              for (int k = 0; k < 2; k++) {
                f32x4 v = c[HC_MAX] * y[k];
#pragma unroll
                for (int s = 0; s < 4; s++) v += c[s] * old[u][k][s];
                if (t < g.sm.n) *(f32x4*)(xs[u] + t * g.sm.stride + 4 * k) = v;
                n[k] += inw[t] * v;
              }
            }
            float v[8];
#pragma unroll
            for (int k = 0; k < 2; k++) {
              const f32x4 gain = *(const f32x4*)(g.gain_next + col[u] + 4 * k);
#pragma unroll
              for (int e = 0; e < 4; e++) {
                sq = __builtin_fmaf(n[k][e], n[k][e], sq);
                v[4 * k + e] = n[k][e] * gain[e];
              }
            }
            split_store8<P>(v, g.planes + (size_t)row[u] * g.ldp + col[u], g.p_plane);
          }
          sq += dpp_f<0xB1>(sq);  // eight lanes hold a row's 64 columns
          sq += dpp_f<0x4E>(sq);
          sq += dpp_f<0x141>(sq);
          if (in[u] && (tid & 7) == 0) g.sq_out[(size_t)row[u] * g.n_sq_out + col[u] / 64] = sq;
        }
      }
    }
    return;
  }
  for (int h = 0; h < BM / HR; h++) {
    __syncthreads();
    if (h == 0 && tid < BM) lf[tid] = factor;
    if (wm * WM / HR == h) {
#pragma unroll
      for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++)
#pragma unroll
          for (int e = 0; e < 4; e++) lc[(wm * WM % HR + i * 16 + fk * 4 + e) * LC + wn * WN + j * 16 + fr] = acc[i][j][e];
    }
    __syncthreads();
    constexpr int UNITS = HR * BN / 8 / NT;
    if constexpr (OUT == GEMM_OUT_STREAMS) {  // four columns of all streams in registers at a time
#pragma unroll 1
      for (int unit = tid; unit < HR * BN / 8; unit += NT) {
        const int r = unit / (BN / 8), c = unit % (BN / 8) * 8, row = row0 + h * HR + r, col = col0 + c;
        const bool in = row < g.M && col < g.N;
        float sq = 0.f;
        if (in) {
          const float f = lf[h * HR + r];
          float v[8];
#pragma unroll
          for (int k = 0; k < 8; k += 4) {
            f32x4 y = *(const f32x4*)(lc + r * LC + c + k) * f;
            if (g.bias) y += *(const f32x4*)(g.bias + col + k);
            f32x4 old[HC_MAX];
            float* xs = g.x + (size_t)row * g.ldx + col + k;
            stream_load(g.sm, xs, old);
            const f32x4 n = stream_apply(g.sm, xs, old, y), gain = *(const f32x4*)(g.gain_next + col + k);
#pragma unroll
            for (int e = 0; e < 4; e++) {
              sq = __builtin_fmaf(n[e], n[e], sq);
              v[k + e] = n[e] * gain[e];
            }
          }
          split_store8<P>(v, g.planes + (size_t)row * g.ldp + col, g.p_plane);
        }
        sq += dpp_f<0xB1>(sq);  // eight lanes hold a row's 64 columns
        sq += dpp_f<0x4E>(sq);
        sq += dpp_f<0x141>(sq);
        if (in && (tid & 7) == 0) g.sq_out[(size_t)row * g.n_sq_out + col / 64] = sq;
      }
      continue;
    }
    int row[UNITS], col[UNITS];
    bool in[UNITS];
    float v[UNITS][8], x[UNITS][8];
#pragma unroll
    for (int u = 0; u < UNITS; u++) {
      const int unit = u * NT + tid, r = unit / (BN / 8), c = unit % (BN / 8) * 8;
      row[u] = row0 + h * HR + r;
      col[u] = col0 + c;
      in[u] = row[u] < g.M && col[u] < g.N;
      if constexpr (OUT == GEMM_OUT_RESIDUAL) {  // (rows are padded past N: eight columns from any col < N lie inside)
#pragma unroll
        for (int e = 0; e < 8; e++) x[u][e] = 0.f;
        if (in[u]) read8(g.x + (size_t)row[u] * g.ldx + col[u], x[u]);
      }
      const f32x4 a = *(const f32x4*)(lc + r * LC + c), b = *(const f32x4*)(lc + r * LC + c + 4);
      const float f = lf[h * HR + r];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        v[u][e] = a[e] * f;
        v[u][e + 4] = b[e] * f;
      }
    }
    if constexpr (OUT == GEMM_OUT_RESIDUAL) {
      if (g.add_rows) {
#pragma unroll
        for (int u = 0; u < UNITS; u++) {
          float t[8];
          if (in[u]) {
            read8(g.add_rows + (size_t)row[u] * g.ldx + col[u], t);
#pragma unroll
            for (int e = 0; e < 8; e++) x[u][e] += t[e];
          }
        }
      }
      if (g.add_vec) {
#pragma unroll
        for (int u = 0; u < UNITS; u++)
#pragma unroll
          for (int e = 0; e < 8; e++)
            if (in[u] && col[u] + e < g.N) x[u][e] += g.add_vec[col[u] + e];
      }
    }
#pragma unroll
    for (int u = 0; u < UNITS; u++) {
      float sq = 0.f;
      if constexpr (OUT == GEMM_OUT_SOFTCAP) {
        if (in[u]) {
#pragma unroll
          for (int e = 0; e < 8; e++)
            if (col[u] + e < g.N) ((float*)g.out)[(size_t)row[u] * g.ldo + col[u] + e] = soft_cap(v[u][e], g.cap);
        }
        continue;
      }
      if constexpr (OUT == GEMM_OUT_ACT_BF16 || OUT == GEMM_OUT_ACT_F32) {
        if (g.bias && in[u]) {
          float t[8];
          read8(g.bias + col[u], t);
#pragma unroll
          for (int e = 0; e < 8; e++) v[u][e] += t[e];
        }
      }
      if constexpr (OUT == GEMM_OUT_GLU) {
        if (!in[u]) continue;
        float t[4];
#pragma unroll
        for (int e = 0; e < 4; e++) t[e] = gelu_tanh(v[u][2 * e]) * v[u][2 * e + 1];
        split_store4<P>(t, g.planes + (size_t)row[u] * g.ldp + col[u] / 2, g.p_plane);
        continue;
      }
#pragma unroll
      for (int e = 0; e < 8; e++) {
        if constexpr (OUT == GEMM_OUT_ACT_BF16 || OUT == GEMM_OUT_ACT_F32) v[u][e] = act_ranges(v[u][e], col[u], g.act);  // (ranges end on multiples of 8)
        if constexpr (OUT == GEMM_OUT_XIELU) v[u][e] = xielu_apply(v[u][e], xr, xl);
        if constexpr (OUT == GEMM_OUT_RESIDUAL) {
          v[u][e] += x[u][e];
          sq = __builtin_fmaf(v[u][e], v[u][e], sq);
        }
      }
      float lo[4], hi[4];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        lo[e] = v[u][e];
        hi[e] = v[u][e + 4];
      }
      if constexpr (OUT == GEMM_OUT_RESIDUAL) {  // eight lanes hold a row's 64 columns
        sq = in[u] ? sq : 0.f;
        sq += dpp_f<0xB1>(sq);
        sq += dpp_f<0x4E>(sq);
        sq += dpp_f<0x141>(sq);
        if (in[u] && (tid & 7) == 0) g.sq_out[(size_t)row[u] * g.n_sq_out + col[u] / 64] = sq;
      }
      if (!in[u]) continue;
      if constexpr (OUT == GEMM_OUT_ACT_F32) {
        store4((float*)g.out + (size_t)row[u] * g.ldo + col[u], lo);
        store4((float*)g.out + (size_t)row[u] * g.ldo + col[u] + 4, hi);
      } else if constexpr (OUT == GEMM_OUT_ACT_BF16) {
        split_store8<1>(v[u], (unsigned short*)g.out + (size_t)row[u] * g.ldo + col[u], 0);
      } else {
        if constexpr (OUT == GEMM_OUT_RESIDUAL) {
          store4(g.x + (size_t)row[u] * g.ldx + col[u], lo);
          store4(g.x + (size_t)row[u] * g.ldx + col[u] + 4, hi);
        }
        split_store8<P>(v[u], g.planes + (size_t)row[u] * g.ldp + col[u], g.p_plane);
      }
    }
  }
}

// Tile and k pieces.  A CU's time for a step of 64 (tile by tile, one workgroup after the other or side by side) and a workgroup's own
// chain of steps are what was measured; a cut of k costs the hand-over of the pieces.
struct GemmPlan {
  int bm, S;
};
struct TileCost {
  int bm, resident;     // workgroups of this tile a CU holds
  double step, chain;   // us per step of 64: a workgroup's share of a busy CU; the latency of one alone
};
static GemmPlan plan(const GemmBf16& g, int planes, int n_cu, size_t ws_floats) {
  static const TileCost costs[] = {{256, 1, 1.03, 1.03}, {128, 1, 0.68, 0.68}, {64, 2, 0.42, 0.51}, {32, 2, 0.41, 0.41}};
  GemmPlan best{128, 1};
  double best_cost = 1e30;
  const int steps = g.K / 64 * planes;
  for (const TileCost& t : costs) {
    if (t.bm > 32 && g.M <= t.bm / 2) continue;
    const int tiles = ((g.M + t.bm - 1) / t.bm) * ((g.N + 127) / 128);
    for (int S : {1, 2, 3, 4, 6, 8}) {
      if (S > 1 && (steps / S < 6 || (size_t)tiles * S * t.bm * 128 > ws_floats || tiles > GEMM_TICKS)) break;
      const double per = (double)steps / S, wgs = (double)tiles * S, rounds = ceil(wgs / (n_cu * t.resident));
      const double busy = ceil(wgs / n_cu) * per * t.step, chain = rounds * per * t.chain;
      const double cost = (busy > chain ? busy : chain) + 6.0 * rounds + (S > 1 ? 8.0 + 1.3 * S * t.bm / 128 : 0.0);
      if (cost < best_cost) {
        best_cost = cost;
        best = {t.bm, S};
      }
    }
  }
  static const int force = [] {  // lab hook (CRABML_HIP_TEST_HOOKS=1 CRABML_HIP_GEMM_BF16_PLAN=rows*100+pieces)
    const char* h = getenv("CRABML_HIP_TEST_HOOKS");
    const char* e = getenv("CRABML_HIP_GEMM_BF16_PLAN");
    return h && h[0] == '1' && e ? atoi(e) : 0;
  }();
  if (force) {
    const int bm = force / 100, S = force % 100, tiles = ((g.M + bm - 1) / bm) * ((g.N + 127) / 128);
    if ((bm == 256 || bm == 128 || bm == 64 || bm == 32) && S >= 1 && S <= steps && (S == 1 || ((size_t)tiles * S * bm * 128 <= ws_floats && tiles <= GEMM_TICKS))) return {bm, S};
  }
  return best;
}

template <int P, int OUT, int NS = 0>
static void launch_t(hipStream_t st, crabml_hip_device::ProfRec* rec, const GemmBf16& g, int n_cu, const GemmScratch& w) {
  const GemmPlan p = plan(g, P, n_cu, w.floats);
  const dim3 grid(((g.M + p.bm - 1) / p.bm) * ((g.N + 127) / 128) * p.S);
  if (p.bm == 256)
    launch_k(st, rec, k_gemm_bf16<256, 128, 4, 2, 3, P, OUT, NS>, grid, dim3(512), 0, g, p.S, w.partials, w.ticks);
  else if (p.bm == 128)
    launch_k(st, rec, k_gemm_bf16<128, 128, 2, 2, 4, P, OUT, NS>, grid, dim3(256), 0, g, p.S, w.partials, w.ticks);
  else if (p.bm == 64)
    launch_k(st, rec, k_gemm_bf16<64, 128, 2, 2, 3, P, OUT, NS>, grid, dim3(256), 0, g, p.S, w.partials, w.ticks);
  else
    launch_k(st, rec, k_gemm_bf16<32, 128, 2, 2, 4, P, OUT, NS>, grid, dim3(256), 0, g, p.S, w.partials, w.ticks);
}

void launch_gemm_bf16(crabml_hip_device* dev, crabml_hip_device::ProfRec* rec, int planes, int out, const GemmBf16& g, const GemmScratch& w) {
  const int n = dev->n_cu;
  hipStream_t st = dev->stream;
  if (planes == 1) {
    switch (out) {
      case GEMM_OUT_ACT_BF16: launch_t<1, GEMM_OUT_ACT_BF16>(st, rec, g, n, w); break;
      case GEMM_OUT_RESIDUAL: launch_t<1, GEMM_OUT_RESIDUAL>(st, rec, g, n, w); break;
      case GEMM_OUT_XIELU: launch_t<1, GEMM_OUT_XIELU>(st, rec, g, n, w); break;
      case GEMM_OUT_STREAMS:
        if (g.sm.n <= 4)
          launch_t<1, GEMM_OUT_STREAMS, 4>(st, rec, g, n, w);
        else
          launch_t<1, GEMM_OUT_STREAMS, HC_MAX>(st, rec, g, n, w);
        break;
      case GEMM_OUT_GLU: launch_t<1, GEMM_OUT_GLU>(st, rec, g, n, w); break;
      default: launch_t<1, GEMM_OUT_SOFTCAP>(st, rec, g, n, w); break;
    }
  } else {
    switch (out) {
      case GEMM_OUT_ACT_F32: launch_t<3, GEMM_OUT_ACT_F32>(st, rec, g, n, w); break;
      case GEMM_OUT_RESIDUAL: launch_t<3, GEMM_OUT_RESIDUAL>(st, rec, g, n, w); break;
      case GEMM_OUT_XIELU: launch_t<3, GEMM_OUT_XIELU>(st, rec, g, n, w); break;
      case GEMM_OUT_STREAMS:
        if (g.sm.n <= 4)
          launch_t<3, GEMM_OUT_STREAMS, 4>(st, rec, g, n, w);
        else
          launch_t<3, GEMM_OUT_STREAMS, HC_MAX>(st, rec, g, n, w);
        break;
      case GEMM_OUT_GLU: launch_t<3, GEMM_OUT_GLU>(st, rec, g, n, w); break;
      default: launch_t<3, GEMM_OUT_SOFTCAP>(st, rec, g, n, w); break;
    }
  }
}

}  // namespace crabml_hip
