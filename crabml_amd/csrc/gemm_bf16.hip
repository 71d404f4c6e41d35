// gemm_bf16.hip -- the kernel behind gemm_bf16.hpp
#include "gemm_bf16.hpp"

namespace crabml_hip {

__device__ __forceinline__ void lds_dma16(const void* g, void* l) {
  __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)g, (__attribute__((address_space(3))) void*)l, 16, 0, 0);
}

template <int BM, int BN, int WGM, int WGN, int P, int OUT>
__global__ __launch_bounds__(256) void k_gemm_bf16(const GemmBf16 g) {
  constexpr int WM = BM / WGM, WN = BN / WGN, TM = WM / 16, TN = WN / 16;
  static_assert(WGM * WGN == 4 && WN == 64, "a wave's columns are one square-sum piece");
  __shared__ __attribute__((aligned(16))) unsigned short lds[2][(BM + BN) * 64];
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg();
  const int wm = wave / WGN, wn = wave % WGN;
  const int mt = (g.M + BM - 1) / BM, nt = (g.N + BN - 1) / BN, total = mt * nt;
  int id = blockIdx.x;
  {  // XCD x (= id % 8) takes a contiguous run of tiles
    const int x = id & 7, i = id >> 3, q = total >> 3, r = total & 7;
    id = x * q + (x < r ? x : r) + i;
  }
  const int row0 = (id % mt) * BM, col0 = (id / mt) * BN;
  f32x4 acc[TM][TN];
#pragma unroll
  for (int i = 0; i < TM; i++)
#pragma unroll
    for (int j = 0; j < TN; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int steps = g.K / 64;
  auto fetch = [&](int s, int buf) {
    const int p = P == 1 ? 0 : s / steps, k0 = (P == 1 ? s : s - p * steps) * 64;
    const unsigned short* ap = g.a + (P == 1 ? 0 : (size_t)(P - 1 - p) * g.a_plane) + k0;  // (the smallest plane first)
#pragma unroll
    for (int it = 0; it < BM / 32; it++) {
      const int slot = it * 256 + tid, r = slot >> 3, c = (slot & 7) ^ ((r >> 1) & 7);
      lds_dma16(ap + (size_t)(row0 + r) * g.K + c * 8, &lds[buf][(it * 256 + wave * 64) * 8]);
    }
#pragma unroll
    for (int it = 0; it < BN / 32; it++) {
      const int slot = it * 256 + tid, r = slot >> 3, c = (slot & 7) ^ ((r >> 1) & 7);
      lds_dma16(g.w + (size_t)(col0 + r) * g.K + k0 + c * 8, &lds[buf][BM * 64 + (it * 256 + wave * 64) * 8]);
    }
  };
  fetch(0, 0);
  const int n_steps = steps * P;
  const int fr = lane & 15, fk = lane >> 4;
  for (int s = 0; s < n_steps; s++) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this wave's part of step s has landed ...
    __syncthreads();                                  // ... and everybody's; and step s - 1 has been read by every wave
    if (s + 1 < n_steps) fetch(s + 1, (s + 1) & 1);
    const unsigned short* la = &lds[s & 1][0];
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
        for (int j = 0; j < TN; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
    }
  }
  // C layout: lane holds rows 4 (lane / 16) .. + 3 of column lane % 16
  float xr = 0.f, xl = 0.f;
  if constexpr (OUT == GEMM_OUT_XIELU) {
    xr = g.xielu[0];
    xl = g.xielu[1];
  }
#pragma unroll
  for (int i = 0; i < TM; i++) {
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const int row = row0 + wm * WM + i * 16 + fk * 4 + e;
      const bool live = row < g.M;
      const int rr = live ? row : g.M - 1;
      float f = 1.f;
      if (g.sq_in != nullptr) {
        float s = 0.f;
        for (int q = fr; q < g.n_sq; q += 16) s += g.sq_in[(size_t)rr * g.n_sq + q];
        f = *g.gain / sqrtf(row16_sum_f32(s) / (float)g.mean_n + g.eps);
      }
      float sq = 0.f;
#pragma unroll
      for (int j = 0; j < TN; j++) {
        const int col = col0 + wn * WN + j * 16 + fr;
        const bool in = live && col < g.N;
        const float v = acc[i][j][e] * f;
        if constexpr (OUT == GEMM_OUT_ACT_BF16) {
          if (in) ((unsigned short*)g.out)[(size_t)row * g.ldo + col] = f2bf(act_ranges(v, col, g.act));
        } else if constexpr (OUT == GEMM_OUT_ACT_F32) {
          if (in) ((float*)g.out)[(size_t)row * g.ldo + col] = act_ranges(v, col, g.act);
        } else if constexpr (OUT == GEMM_OUT_SOFTCAP) {
          if (in) ((float*)g.out)[(size_t)row * g.ldo + col] = soft_cap(v, g.cap);
        } else if constexpr (OUT == GEMM_OUT_XIELU) {
          if (in) split_store<P>(xielu_apply(v, xr, xl), g.planes + (size_t)row * g.ldp + col, g.p_plane);
        } else {
          if (in) {
            float* px = g.x + (size_t)row * g.ldx + col;
            float s = *px + v;
            if (g.add_rows) s += g.add_rows[(size_t)row * g.ldx + col];
            if (g.add_vec) s += g.add_vec[col];
            *px = s;
            split_store<P>(s, g.planes + (size_t)row * g.ldp + col, g.p_plane);
            sq = __builtin_fmaf(s, s, sq);
          }
        }
      }
      if constexpr (OUT == GEMM_OUT_RESIDUAL) {
        sq = row16_sum_f32(sq);
        const int piece = (col0 + wn * WN) / 64;
        if (fr == 0 && live && piece < g.n_sq_out) g.sq_out[(size_t)row * g.n_sq_out + piece] = sq;
      }
    }
  }
}

// the tile that covers the chip: 128 x 128 when that makes enough workgroups, smaller row tiles below
template <int P, int OUT>
static void launch_t(hipStream_t st, crabml_hip_device::ProfRec* rec, const GemmBf16& g, int n_cu) {
  auto tiles = [&](int bm, int bn) { return ((g.M + bm - 1) / bm) * ((g.N + bn - 1) / bn); };
  if (g.M > 64 && tiles(128, 128) >= n_cu)
    launch_k(st, rec, k_gemm_bf16<128, 128, 2, 2, P, OUT>, dim3(tiles(128, 128)), dim3(256), 0, g);
  else if (g.M > 32 && (tiles(64, 128) >= n_cu || g.M > 512))
    launch_k(st, rec, k_gemm_bf16<64, 128, 2, 2, P, OUT>, dim3(tiles(64, 128)), dim3(256), 0, g);
  else
    launch_k(st, rec, k_gemm_bf16<32, 128, 2, 2, P, OUT>, dim3(tiles(32, 128)), dim3(256), 0, g);
}

void launch_gemm_bf16(crabml_hip_device* dev, crabml_hip_device::ProfRec* rec, int planes, int out, const GemmBf16& g) {
  const int n = dev->n_cu;
  hipStream_t st = dev->stream;
  if (planes == 1) {
    switch (out) {
      case GEMM_OUT_ACT_BF16: launch_t<1, GEMM_OUT_ACT_BF16>(st, rec, g, n); break;
      case GEMM_OUT_RESIDUAL: launch_t<1, GEMM_OUT_RESIDUAL>(st, rec, g, n); break;
      case GEMM_OUT_XIELU: launch_t<1, GEMM_OUT_XIELU>(st, rec, g, n); break;
      default: launch_t<1, GEMM_OUT_SOFTCAP>(st, rec, g, n); break;
    }
  } else {
    switch (out) {
      case GEMM_OUT_ACT_F32: launch_t<3, GEMM_OUT_ACT_F32>(st, rec, g, n); break;
      case GEMM_OUT_RESIDUAL: launch_t<3, GEMM_OUT_RESIDUAL>(st, rec, g, n); break;
      case GEMM_OUT_XIELU: launch_t<3, GEMM_OUT_XIELU>(st, rec, g, n); break;
      default: launch_t<3, GEMM_OUT_SOFTCAP>(st, rec, g, n); break;
    }
  }
}

}  // namespace crabml_hip
