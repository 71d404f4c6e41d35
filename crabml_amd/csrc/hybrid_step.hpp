// hybrid_step.hpp -- the hybrid decoder's decode step: one token of each of up to HYB_STEP_ROWS sequences, five launches per layer
//   k_gemv_bf16<RMS, ACT>         norm 1 + every projection of both mixers + their activations
//   k_mix_step                    both mixers: cache append + attention (split over cached rows, merged by the last workgroup to
//                                 finish) and the linear-attention state update, side by side in one grid
//   k_gemv_bf16<SPLIT, RESIDUAL>  both output projections (one matrix) + the linear branch's norm + residual (+ what a pass adds)
//   k_gemv_bf16<RMS, XIELU>       norm 2 + up projection + activation
//   k_gemv_bf16<PLAIN, RESIDUAL>  down projection + residual (+ what a pass adds)
// Tokens, positions and the sequences' state pointers are read from device memory, so a captured graph serves every step.
#pragma once
#include "hybrid_common.hpp"
#include "sampler.hpp"

namespace crabml_hip {

#define HYB_STEP_ROWS 16
#define MIX_KEYS 64   // cached rows per attention workgroup
#define MIX_HEADS 8   // query heads per attention workgroup

struct StepSeq {
  int token, pos;
  char* slab;
};

__global__ __launch_bounds__(256) void k_embed_step(const unsigned short* __restrict__ table, const StepSeq* __restrict__ seq, int width, int ldx,
                                                    float scale, const double* __restrict__ freq, float* __restrict__ x, float* __restrict__ emb,
                                                    const float* __restrict__ add_vec, const StreamMix sm, float* __restrict__ u) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (c >= width) return;
  const StepSeq s = seq[b];
  const float v = __builtin_fmaf(bf2f(table[(size_t)s.token * width + c]), scale, position_entry(s.pos, c, freq));
  if (sm.n) {  // every stream starts as the embedding
    float r = 0.f;
    for (int t = 0; t < sm.n; t++) {
      x[t * sm.stride + (size_t)b * ldx + c] = v;
      r = __builtin_fmaf(sm.in[t], v, r);
    }
    u[(size_t)b * ldx + c] = r;
    return;
  }
  if (emb) emb[(size_t)b * ldx + c] = v;
  x[(size_t)b * ldx + c] = add_vec ? v + add_vec[c] : v;
}

struct MixStep {
  AttnGeom at;
  LinGeom li;
  RunState rs;
  const StepSeq* seq = nullptr;
  const float* proj = nullptr;  // [B][ldp]
  float* cat = nullptr;         // [B][ldc]: attention columns from 0, linear columns from lin_off
  float* ss = nullptr;          // [B][H * slices] square sums of the linear branch
  float* part = nullptr;        // attention partials
  float* v_kept = nullptr;      // [B][ld_vk] values that VMIX_KEEP leaves
  int ld_vk = 0;
  unsigned* tick = nullptr;     // arrivals per (sequence, kv head, head block); the last one puts it back to zero
  int B = 0, ldp = 0, ldc = 0, lin_off = 0, splits = 0, head_blocks = 0;
};
// floats of one partial: per head its V sums, the running maximum and the denominator
__host__ __device__ inline int mix_part_floats(int V) { return MIX_HEADS * (V + 2); }

// One workgroup: up to MIX_HEADS query heads of one kv head over MIX_KEYS cached rows; heads up to CLS wide.  Everything it needs from
// memory is requested up front; the rest is register and LDS work.  (The launch runs cold: its code is kept short.)
template <typename T, int CLS>
__device__ __forceinline__ void mix_attention(const MixStep& a, int blk, float* lds) {
  constexpr int NU = CLS / 32;                             // K: four lanes per row, their octets interleaved
  constexpr int CP = CLS / 8, GR = 256 / CP, NV = MIX_KEYS / GR;  // V: CP lanes across the columns, GR groups of rows
  const AttnGeom& g = a.at;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg();
  const int split = blk % a.splits;
  int rest = blk / a.splits;
  const int hb = rest % a.head_blocks;
  rest /= a.head_blocks;
  const int kvh = rest % g.G, b = rest / g.G;
  const StepSeq sq = a.seq[b];
  const int hpg = g.H / g.G, h0 = kvh * hpg + hb * MIX_HEADS;
  const int nh = hpg - hb * MIX_HEADS < MIX_HEADS ? hpg - hb * MIX_HEADS : MIX_HEADS;
  const float* pr = a.proj + (size_t)b * a.ldp;
  float* ml = lds;                          // [MIX_HEADS][2]: maximum, denominator
  float* hp_s = ml + 2 * MIX_HEADS;         // [3][MIX_HEADS]: penalty factor, its rate, sink; then the waves' square sums of q and k
  T* kn_s = (T*)(hp_s + 5 * MIX_HEADS);     // [CLS], [CLS]: the new token's row as the cache holds it
  T* vn_s = kn_s + CLS;
  float* g_s = (float*)(vn_s + CLS);        // [MIX_HEADS][V]: gates
  float* q_s = g_s + MIX_HEADS * g.V;       // [MIX_HEADS][D]
  float* p_s = q_s + MIX_HEADS * g.D;       // [MIX_HEADS][MIX_KEYS]
  float* o_s = p_s + MIX_HEADS * MIX_KEYS;  // [4 waves][MIX_HEADS][V]
  // what does not depend on the position: on its way together with it
  float q_f = g.scale, k_f = 1.f;
  if (g.q_norm) {  // (the same for the whole workgroup)
    float sq2 = 0.f, sk2 = 0.f;
    for (int i = tid; i < g.H * g.D; i += 256) sq2 = __builtin_fmaf(pr[g.cq + i], pr[g.cq + i], sq2);
    for (int i = tid; i < g.G * g.D; i += 256) sk2 = __builtin_fmaf(pr[g.ck + i], pr[g.ck + i], sk2);
    sq2 = wave_sum_f32(sq2);
    sk2 = wave_sum_f32(sk2);
    float* red = hp_s + 3 * MIX_HEADS;
    if (lane == 0) {
      red[wave] = sq2;
      red[4 + wave] = sk2;
    }
    __syncthreads();
    q_f *= 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)g.q_mean + g.eps);
    k_f = 1.0f / sqrtf(((red[4] + red[5]) + (red[6] + red[7])) / (float)g.k_mean + g.eps);
  }
  for (int i = tid; i < nh * g.D; i += 256) q_s[i] = pr[g.cq + h0 * g.D + i] * (g.q_norm ? q_f * g.q_norm[h0 * g.D + i] : q_f);
  for (int i = tid; i < nh * g.V; i += 256)
    g_s[i] = (g.gate == GATE_ELEMENT ? pr[g.cg + h0 * g.V + i] : g.gate == GATE_HEAD ? pr[g.cg + h0 + i / g.V] : 1.f) * g.out_scale;
  if (tid < g.D) kn_s[tid] = kv_from<T>(pr[g.ck + kvh * g.D + tid] * (g.k_norm ? k_f * g.k_norm[kvh * g.D + tid] : 1.f));
  float v_raw = 0.f;
  if (tid < g.V) {
    v_raw = pr[g.cv + kvh * g.V + tid];
    float v = v_raw;
    if (g.vmix == VMIX_MIX) {
      const float la = *g.lambda;
      v = __builtin_fmaf(la, a.v_kept[(size_t)b * a.ld_vk + kvh * g.V + tid], (1.0f - la) * v);
    }
    vn_s[tid] = kv_from<T>(v);
  }
  if (tid < nh) {
    hp_s[tid] = g.amp ? g.amp[h0 + tid] : 0.f;
    hp_s[MIX_HEADS + tid] = g.amp ? g.rate[h0 + tid] : 0.f;
    hp_s[2 * MIX_HEADS + tid] = g.sink ? g.sink[h0 + tid] : -INFINITY;
  }
  // the new token's row, and the rows it sees: its chunk's up to itself, or the whole ring once the window has gone round
  const int in_chunk = sq.pos % g.span, n_rows = g.window && sq.pos >= g.span ? g.span : in_chunk + 1;
  const int r0 = split * MIX_KEYS;
  if (r0 >= n_rows) return;  // (whole workgroup)
  const int active = (n_rows + MIX_KEYS - 1) / MIX_KEYS;
  const int nk = n_rows - r0 < MIX_KEYS ? n_rows - r0 : MIX_KEYS;
  T* kc = (T*)(sq.slab + a.rs.k) + (size_t)kvh * g.rows * g.D;
  T* vc = (T*)(sq.slab + a.rs.v) + (size_t)kvh * g.rows * g.V;
  const bool own_new = in_chunk >= r0 && in_chunk < r0 + MIX_KEYS;
  const int key = tid >> 2, part = tid & 3, vcol = tid % CP * 8, vgrp = tid / CP;
  Oct<T> kr[NU], vr[NV];
#pragma unroll
  for (int u = 0; u < NU; u++) {
    const int c = part * 8 + u * 32;
    kr[u] = oct_zero<T>();
    if (c < g.D && key < nk && r0 + key != in_chunk) kr[u] = oct_load(kc + (size_t)(r0 + key) * g.D + c);
  }
#pragma unroll
  for (int u = 0; u < NV; u++) {
    const int k = vgrp + u * GR;
    vr[u] = oct_zero<T>();
    if (k < nk && vcol < g.V && r0 + k != in_chunk) vr[u] = oct_load(vc + (size_t)(r0 + k) * g.V + vcol);
  }
  __syncthreads();
  if (own_new) {  // the new row: appended to the cache by one head block, taken from LDS by all
    if (hb == 0) {
      if (tid < g.D) kc[(size_t)in_chunk * g.D + tid] = kn_s[tid];
      if (tid < g.V) vc[(size_t)in_chunk * g.V + tid] = vn_s[tid];
      if (g.vmix == VMIX_KEEP && tid < g.V) a.v_kept[(size_t)b * a.ld_vk + kvh * g.V + tid] = v_raw;
    }
    if (r0 + key == in_chunk) {
#pragma unroll
      for (int u = 0; u < NU; u++)
        if (part * 8 + u * 32 < g.D) kr[u] = oct_load(kn_s + part * 8 + u * 32);
    }
#pragma unroll
    for (int u = 0; u < NV; u++)
      if (r0 + vgrp + u * GR == in_chunk && vcol < g.V) vr[u] = oct_load(vn_s + vcol);
  }
  {
    const int behind = in_chunk - (r0 + key);
    const float dist = (float)(g.window && behind < 0 ? behind + g.span : behind);
    float kk[NU][8];
#pragma unroll
    for (int u = 0; u < NU; u++) oct_floats(kr[u], kk[u]);
    for (int h = 0; h < nh; h++) {
      const float* q = q_s + h * g.D + part * 8;
      float s = 0.f;
#pragma unroll
      for (int u = 0; u < NU; u++) {
        if (part * 8 + u * 32 < g.D) {
          const f32x4 q0 = *(const f32x4*)(q + u * 32), q1 = *(const f32x4*)(q + u * 32 + 4);
#pragma unroll
          for (int e = 0; e < 4; e++) s = __builtin_fmaf(q0[e], kk[u][e], __builtin_fmaf(q1[e], kk[u][e + 4], s));
        }
      }
      s += dpp_f<0xB1>(s);
      s += dpp_f<0x4E>(s);
      s -= hp_s[h] * __logf(__builtin_fmaf(hp_s[MIX_HEADS + h], dist > 0.f ? dist : 0.f, 1.0f));
      if (part == 0) p_s[h * MIX_KEYS + key] = key < nk ? s : -INFINITY;
    }
  }
  __syncthreads();
  for (int h = wave; h < nh; h += 4) {  // one wave per head: MIX_KEYS = 64 scores
    const float s = p_s[h * MIX_KEYS + lane];
    const float m = wave_max_f32(s);
    const float e = __expf(s - m);
    p_s[h * MIX_KEYS + lane] = e;
    const float l = wave_sum_f32(e);
    if (lane == 0) {
      ml[2 * h] = m;
      ml[2 * h + 1] = l;
    }
  }
  __syncthreads();
  {  // weighted value rows, added over the wave's row groups by lane exchange, over the waves through LDS
    float vv[NV][8];
#pragma unroll
    for (int u = 0; u < NV; u++) oct_floats(vr[u], vv[u]);
    for (int h = 0; h < nh; h++) {
      float o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int u = 0; u < NV; u++) {
        const float w = p_s[h * MIX_KEYS + vgrp + u * GR];
#pragma unroll
        for (int e = 0; e < 8; e++) o[e] = __builtin_fmaf(w, vv[u][e], o[e]);
      }
#pragma unroll
      for (int x = CP; x < 64; x <<= 1)
#pragma unroll
        for (int e = 0; e < 8; e++) o[e] += __shfl_xor(o[e], x, 64);
      if (lane < CP && vcol < g.V) {
        float* d = o_s + (wave * MIX_HEADS + h) * g.V + vcol;
        *(f32x4*)d = f32x4{o[0], o[1], o[2], o[3]};
        *(f32x4*)(d + 4) = f32x4{o[4], o[5], o[6], o[7]};
      }
    }
  }
  __syncthreads();
  const int slot = (b * g.G + kvh) * a.head_blocks + hb;
  const int wstr = MIX_HEADS * g.V, pf = mix_part_floats(g.V), n_out = nh * g.V;
  float* base = a.part + (size_t)slot * a.splits * pf;
  __shared__ unsigned s_last;
  if (active > 1) {  // partials through write-through stores; whoever arrives last merges them in row order
    float* mine = base + (size_t)split * pf;
    for (int i = tid; i < n_out; i += 256)
      __hip_atomic_store(mine + i, (o_s[i] + o_s[wstr + i]) + (o_s[2 * wstr + i] + o_s[3 * wstr + i]), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    if (tid < 2 * nh) __hip_atomic_store(mine + wstr + tid, ml[tid], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this thread's write-through stores have been acknowledged
    __syncthreads();
    if (tid == 0) s_last = __hip_atomic_fetch_add(a.tick + slot, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (unsigned)(active - 1);
    __syncthreads();
    if (!s_last) return;
    if (tid == 0) __hip_atomic_store(a.tick + slot, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  for (int i = tid; i < n_out; i += 256) {
    const int h = i / g.V;
    float m = hp_s[2 * MIX_HEADS + h], l = m == -INFINITY ? 0.f : 1.f, o = 0.f;  // the sink: a key without a value (or none)
    if (active == 1) {
      const float mx = fmaxf(m, ml[2 * h]), w = __expf(ml[2 * h] - mx);
      l = __builtin_fmaf(l, __expf(m - mx), ml[2 * h + 1] * w);
      o = ((o_s[i] + o_s[wstr + i]) + (o_s[2 * wstr + i] + o_s[3 * wstr + i])) * w;
    } else {
      for (int s0 = 0; s0 < active; s0 += 16) {
        float ps[16], ms[16], ls[16], mx = m;
#pragma unroll
        for (int s = 0; s < 16; s++) {
          const float* p = base + (size_t)(s0 + s < active ? s0 + s : s0) * pf;
          ps[s] = __hip_atomic_load(p + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
          ms[s] = __hip_atomic_load(p + wstr + 2 * h, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
          ls[s] = __hip_atomic_load(p + wstr + 2 * h + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        }
#pragma unroll
        for (int s = 0; s < 16; s++) mx = fmaxf(mx, ms[s]);
        const float w0 = __expf(m - mx);
        m = mx;
        l *= w0;
        o *= w0;
#pragma unroll
        for (int s = 0; s < 16; s++) {
          const float w = s0 + s < active ? __expf(ms[s] - mx) : 0.f;
          l = __builtin_fmaf(ls[s], w, l);
          o = __builtin_fmaf(ps[s], w, o);
        }
      }
    }
    a.cat[(size_t)b * a.ldc + h0 * g.V + i] = o / l * g_s[i];
  }
}

// one head's slice of value columns: 8 threads x 4 columns, 32 groups of key rows
__device__ __forceinline__ void mix_linear(const MixStep& a, int blk, float* lds) {
  const LinGeom& g = a.li;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg();
  const int slice = blk % g.slices, h = (blk / g.slices) % g.H, b = blk / (g.slices * g.H);
  const StepSeq sq = a.seq[b];
  float* S = (float*)(sq.slab + a.rs.s) + (size_t)h * g.D * g.V;
  const float* pr = a.proj + (size_t)b * a.ldp;
  float* k_s = lds;        // [D]
  float* q_s = k_s + g.D;  // [D]
  float* o_s = q_s + g.D;  // [32][32 + 4]
  const int c = slice * LIN_SLICE + (tid & 7) * 4, grp = tid >> 3;
  const bool live = c < g.V;
  const bool fresh = sq.pos == 0;  // a sequence's first token: whatever the slab holds, the state is zero
  f32x4 s[8];  // (at most 256 key rows)
#pragma unroll
  for (int u = 0; u < 8; u++) {
    const int d = grp + u * 32;
    s[u] = live && !fresh && d < g.D ? *(const f32x4*)(S + (size_t)d * g.V + c) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  if (tid < g.D) {
    k_s[tid] = pr[g.ck + h * g.D + tid];
    q_s[tid] = pr[g.cq + h * g.D + tid];
  }
  const f32x4 v = live ? *(const f32x4*)(pr + g.cv + h * g.V + c) : f32x4{0.f, 0.f, 0.f, 0.f};
  const float dec = g.decay[h * LIN_POW + 1];
  // (the output side's factors, for the half-wave that will need them)
  const int oc = slice * LIN_SLICE + lane, occ = h * g.V + (oc < g.V ? oc : 0);
  float factor = 0.f;
  if (wave == 0 && lane < LIN_SLICE && oc < g.V) factor = g.norm[occ] * (g.out_scale * pr[g.cg + occ]);
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 8; u++) {
    const int d = grp + u * 32;
    if (live && d < g.D) {
      const float k = k_s[d], q = q_s[d];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        s[u][e] = __builtin_fmaf(dec, s[u][e], k * v[e]);
        o[e] = __builtin_fmaf(s[u][e], q, o[e]);
      }
      *(f32x4*)(S + (size_t)d * g.V + c) = s[u];
    }
  }
  *(f32x4*)(o_s + grp * 36 + (tid & 7) * 4) = o;
  __syncthreads();
  if (wave == 0) {  // 32 columns; the upper half-wave adds nothing to the square sum
    float r = 0.f;
    if (lane < LIN_SLICE) {
#pragma unroll
      for (int i = 0; i < 32; i++) r += o_s[i * 36 + lane];
    }
    const bool in = lane < LIN_SLICE && oc < g.V;
    const float ss = wave_sum_f32(in ? r * r : 0.f);
    if (lane == 0) a.ss[(size_t)b * g.H * g.slices + h * g.slices + slice] = ss;
    if (in) a.cat[(size_t)b * a.ldc + a.lin_off + occ] = r * factor;
  }
}

template <typename T, int CLS>
__global__ __launch_bounds__(256) void k_mix_step(const MixStep a) {
  extern __shared__ __attribute__((aligned(16))) float mix_lds[];
  const int n_attn = a.at.H ? a.B * a.at.G * a.head_blocks * a.splits : 0;
  if ((int)blockIdx.x < n_attn)
    mix_attention<T, CLS>(a, blockIdx.x, mix_lds);
  else
    mix_linear(a, blockIdx.x - n_attn, mix_lds);
}
template <typename T, int CLS>
inline void launch_mix_step_t(hipStream_t st, crabml_hip_device::ProfRec* rec, const MixStep& a) {
  const size_t at = a.at.H ? 7 * MIX_HEADS + 2 * CLS * sizeof(T) / 4 + (size_t)MIX_HEADS * (a.at.D + MIX_KEYS + 5 * a.at.V) : 0;
  const size_t li = a.li.H ? (size_t)(2 * a.li.D + 32 * 36) : 0;
  const unsigned grid = (unsigned)(a.B * ((a.at.H ? a.at.G * a.head_blocks * a.splits : 0) + a.li.H * a.li.slices));
  launch_k(st, rec, k_mix_step<T, CLS>, dim3(grid), dim3(256), (at > li ? at : li) * sizeof(float), a);  // (at most 57 KiB)
}
template <typename T>
inline void launch_mix_step(hipStream_t st, crabml_hip_device::ProfRec* rec, const MixStep& a) {
  const int w = a.at.D > a.at.V ? a.at.D : a.at.V;
  if (w <= 64)
    launch_mix_step_t<T, 64>(st, rec, a);
  else if (w <= 128)
    launch_mix_step_t<T, 128>(st, rec, a);
  else
    launch_mix_step_t<T, 256>(st, rec, a);
}

// ---- greedy sampler over the rows of a batch (last maximum, as k_argmax_step) ---------------------------------------------------
__global__ __launch_bounds__(64) void k_argmax_rows_step(const float* __restrict__ pv, const int* __restrict__ pi, int nparts,
                                                         StepSeq* __restrict__ seq, const int* __restrict__ step_d, unsigned* __restrict__ out, int out_cap) {
  const int b = blockIdx.x;
  float bv = -INFINITY;
  int bi = -1;
  for (int i = threadIdx.x; i < nparts; i += 64) argmax_combine(bv, bi, pv[b * nparts + i], pi[b * nparts + i]);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    float ov = __shfl_xor(bv, o, 64);
    int oi = __shfl_xor(bi, o, 64);
    argmax_combine(bv, bi, ov, oi);
  }
  if (threadIdx.x == 0) {
    seq[b].token = bi < 0 ? 0 : bi;
    seq[b].pos++;
    const size_t at = (size_t)*step_d * gridDim.x + b;
    if (at < (size_t)out_cap) out[at] = (unsigned)(bi < 0 ? 0 : bi);
  }
}
__global__ void k_step_advance(int* step_d) { *step_d += 1; }

}  // namespace crabml_hip
