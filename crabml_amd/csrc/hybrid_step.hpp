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
                                                    const float* __restrict__ add_vec) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (c >= width) return;
  const StepSeq s = seq[b];
  const float v = __builtin_fmaf(bf2f(table[(size_t)s.token * width + c]), scale, position_entry(s.pos, c, freq));
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
  unsigned* tick = nullptr;     // arrivals per (sequence, kv head, head block); the last one puts it back to zero
  int B = 0, ldp = 0, ldc = 0, lin_off = 0, splits = 0, head_blocks = 0;
};
// floats of one partial: per head its V sums, the running maximum and the denominator
__host__ __device__ inline int mix_part_floats(int V) { return MIX_HEADS * (V + 2); }

template <typename T>
__device__ __forceinline__ void mix_attention(const MixStep& a, int blk, float* lds) {
  const AttnGeom& g = a.at;
  const int tid = threadIdx.x, lane = tid & 63, wave = wave_in_wg();
  const int split = blk % a.splits;
  int rest = blk / a.splits;
  const int hb = rest % a.head_blocks;
  rest /= a.head_blocks;
  const int kvh = rest % g.G, b = rest / g.G;
  const StepSeq sq = a.seq[b];
  const int in_chunk = sq.pos % g.chunk, n_rows = in_chunk + 1;  // this chunk's rows, the new one included
  const int r0 = split * MIX_KEYS;
  if (r0 >= n_rows) return;  // (whole workgroup)
  const int active = (n_rows + MIX_KEYS - 1) / MIX_KEYS;
  const int nk = n_rows - r0 < MIX_KEYS ? n_rows - r0 : MIX_KEYS;
  const int hpg = g.H / g.G, h0 = kvh * hpg + hb * MIX_HEADS;
  const int nh = hpg - hb * MIX_HEADS < MIX_HEADS ? hpg - hb * MIX_HEADS : MIX_HEADS;
  T* kc = (T*)(sq.slab + a.rs.k) + (size_t)kvh * g.rows * g.D;
  T* vc = (T*)(sq.slab + a.rs.v) + (size_t)kvh * g.rows * g.V;
  const float* pr = a.proj + (size_t)b * a.ldp;
  const bool own_new = in_chunk >= r0 && in_chunk < r0 + MIX_KEYS;
  float* ml = lds;                          // [MIX_HEADS][2]: maximum, denominator
  float* q_s = ml + 2 * MIX_HEADS;          // [MIX_HEADS][D]
  float* p_s = q_s + MIX_HEADS * g.D;       // [MIX_HEADS][MIX_KEYS]
  float* o_s = p_s + MIX_HEADS * MIX_KEYS;  // [MIX_HEADS][256]: column sums by row group
  for (int i = tid; i < nh * g.D; i += 256) q_s[i] = pr[g.cq + h0 * g.D + i] * g.scale;
  if (own_new && hb == 0) {  // cache append (read back below by this workgroup only through pr, never through memory)
    for (int i = tid; i < g.D; i += 256) kc[(size_t)in_chunk * g.D + i] = kv_from<T>(pr[g.ck + kvh * g.D + i]);
    for (int i = tid; i < g.V; i += 256) vc[(size_t)in_chunk * g.V + i] = kv_from<T>(pr[g.cv + kvh * g.V + i]);
  }
  __syncthreads();
  {  // scores: four lanes per row, their 8-element pieces interleaved
    const int key = tid >> 2, part = tid & 3, row = r0 + key;
    float s[MIX_HEADS];
#pragma unroll
    for (int h = 0; h < MIX_HEADS; h++) s[h] = 0.f;
    if (key < nk) {
      for (int c = part * 8; c < g.D; c += 32) {
        float kk[8];
        if (row == in_chunk) {
#pragma unroll
          for (int e = 0; e < 8; e++) kk[e] = kv_to(kv_from<T>(pr[g.ck + kvh * g.D + c + e]));
        } else {
          kv_load8(kc + (size_t)row * g.D + c, kk);
        }
#pragma unroll
        for (int h = 0; h < MIX_HEADS; h++) {
          if (h < nh) {
            const f32x4 q0 = *(const f32x4*)(q_s + h * g.D + c), q1 = *(const f32x4*)(q_s + h * g.D + c + 4);
#pragma unroll
            for (int e = 0; e < 4; e++) s[h] = __builtin_fmaf(q0[e], kk[e], __builtin_fmaf(q1[e], kk[e + 4], s[h]));
          }
        }
      }
    }
    const float dist = (float)(in_chunk - row);
#pragma unroll
    for (int h = 0; h < MIX_HEADS; h++) {
      float v = s[h];
      v += dpp_f<0xB1>(v);
      v += dpp_f<0x4E>(v);
      if (part == 0 && h < nh) {
        if (g.amp) v -= g.amp[h0 + h] * __logf(__builtin_fmaf(g.rate[h0 + h], dist, 1.0f));
        p_s[h * MIX_KEYS + key] = key < nk ? v : -INFINITY;
      }
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
  // weighted value rows: a thread owns one column of one of KG row groups
  const int vp = g.V <= 32 ? 32 : g.V <= 64 ? 64 : g.V <= 128 ? 128 : 256, kg = 256 / vp;
  {
    const int col = tid % vp, grp = tid / vp;
    float o[MIX_HEADS];
#pragma unroll
    for (int h = 0; h < MIX_HEADS; h++) o[h] = 0.f;
    if (col < g.V) {
#pragma unroll 4
      for (int key = grp; key < nk; key += kg) {
        const int row = r0 + key;
        const float v = row == in_chunk ? kv_to(kv_from<T>(pr[g.cv + kvh * g.V + col])) : kv_to(vc[(size_t)row * g.V + col]);
#pragma unroll
        for (int h = 0; h < MIX_HEADS; h++) o[h] = __builtin_fmaf(p_s[h * MIX_KEYS + key], v, o[h]);  // (heads past nh: unused)
      }
    }
#pragma unroll
    for (int h = 0; h < MIX_HEADS; h++) o_s[h * 256 + tid] = o[h];
  }
  __syncthreads();
  const int slot = (b * g.G + kvh) * a.head_blocks + hb;
  auto sum_groups = [&](int h, int c) {
    float s = 0.f;
    for (int k = 0; k < kg; k++) s += o_s[h * 256 + k * vp + c];
    return s;
  };
  auto finish = [&](int h, int c, float o, float l) {
    const int col = (h0 + h) * g.V + c;
    a.cat[(size_t)b * a.ldc + col] = o / l * (g.out_scale * pr[g.cg + col]);
  };
  if (active == 1) {
    for (int i = tid; i < nh * g.V; i += 256) {
      const int h = i / g.V, c = i % g.V;
      float m = ml[2 * h], l = ml[2 * h + 1], o = sum_groups(h, c);
      if (g.sink) {
        const float t = fmaxf(m, g.sink[h0 + h]), w = __expf(m - t);
        l = __builtin_fmaf(l, w, __expf(g.sink[h0 + h] - t));
        o *= w;
      }
      finish(h, c, o, l);
    }
    return;
  }
  // partials through write-through stores; whoever arrives last merges them in row order
  const int pf = mix_part_floats(g.V);
  float* mine = a.part + ((size_t)slot * a.splits + split) * pf;
  for (int i = tid; i < nh * g.V; i += 256)
    __hip_atomic_store(mine + i, sum_groups(i / g.V, i % g.V), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  for (int i = tid; i < 2 * nh; i += 256) __hip_atomic_store(mine + MIX_HEADS * g.V + i, ml[i], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this thread's write-through stores have been acknowledged
  __shared__ unsigned s_last;
  __syncthreads();
  if (tid == 0) s_last = __hip_atomic_fetch_add(a.tick + slot, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (unsigned)(active - 1);
  __syncthreads();
  if (!s_last) return;
  if (tid == 0) __hip_atomic_store(a.tick + slot, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  const float* base = a.part + (size_t)slot * a.splits * pf;
  // weights e^(m_s - m) / l per head and split, in LDS over the queries and scores
  float* w_s = q_s;  // [MIX_HEADS][active]
  __syncthreads();
  for (int h = wave; h < nh; h += 4) {
    float m = -INFINITY;
    for (int s = lane; s < active; s += 64)
      m = fmaxf(m, __hip_atomic_load(base + (size_t)s * pf + MIX_HEADS * g.V + 2 * h, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT));
    m = wave_max_f32(m);
    if (g.sink) m = fmaxf(m, g.sink[h0 + h]);
    float l = 0.f;
    for (int s = lane; s < active; s += 64) {
      const float* p = base + (size_t)s * pf + MIX_HEADS * g.V + 2 * h;
      const float w = __expf(__hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) - m);
      w_s[h * active + s] = w;
      l = __builtin_fmaf(__hip_atomic_load(p + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT), w, l);
    }
    l = wave_sum_f32(l);
    if (g.sink) l += __expf(g.sink[h0 + h] - m);
    if (lane == 0) ml[2 * h + 1] = l;
  }
  __syncthreads();
  for (int i = tid; i < nh * g.V; i += 256) {
    const int h = i / g.V, c = i % g.V;
    float o = 0.f;
#pragma unroll 4
    for (int s = 0; s < active; s++)
      o = __builtin_fmaf(__hip_atomic_load(base + (size_t)s * pf + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT), w_s[h * active + s], o);
    finish(h, c, o, ml[2 * h + 1]);
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
  for (int i = tid; i < g.D; i += 256) {
    k_s[i] = pr[g.ck + h * g.D + i];
    q_s[i] = pr[g.cq + h * g.D + i];
  }
  const int c = slice * LIN_SLICE + (tid & 7) * 4, grp = tid >> 3;
  const bool live = c < g.V;
  const f32x4 v = live ? *(const f32x4*)(pr + g.cv + h * g.V + c) : f32x4{0.f, 0.f, 0.f, 0.f};
  const float dec = g.decay[h * LIN_POW + 1];
  const bool fresh = sq.pos == 0;  // a sequence's first token: whatever the slab holds, the state is zero
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  __syncthreads();
  if (live) {
#pragma unroll 4
    for (int d = grp; d < g.D; d += 32) {
      f32x4* p = (f32x4*)(S + (size_t)d * g.V + c);
      f32x4 s = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *p;
      const float k = k_s[d], q = q_s[d];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        s[e] = __builtin_fmaf(dec, s[e], k * v[e]);
        o[e] = __builtin_fmaf(s[e], q, o[e]);
      }
      *p = s;
    }
  }
  *(f32x4*)(o_s + grp * 36 + (tid & 7) * 4) = o;
  __syncthreads();
  if (wave == 0) {  // 32 columns; the upper half-wave adds nothing to the square sum
    const int col = slice * LIN_SLICE + lane;
    float r = 0.f;
    if (lane < LIN_SLICE)
      for (int i = 0; i < 32; i++) r += o_s[i * 36 + lane];
    const bool in = lane < LIN_SLICE && col < g.V;
    const float ss = wave_sum_f32(in ? r * r : 0.f);
    if (lane == 0) a.ss[(size_t)b * g.H * g.slices + h * g.slices + slice] = ss;
    if (in) {
      const int cc = h * g.V + col;
      a.cat[(size_t)b * a.ldc + a.lin_off + cc] = r * (g.norm[cc] * (g.out_scale * pr[g.cg + cc]));
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void k_mix_step(const MixStep a) {
  extern __shared__ __attribute__((aligned(16))) float mix_lds[];
  const int n_attn = a.at.H ? a.B * a.at.G * a.head_blocks * a.splits : 0;
  if ((int)blockIdx.x < n_attn)
    mix_attention<T>(a, blockIdx.x, mix_lds);
  else
    mix_linear(a, blockIdx.x - n_attn, mix_lds);
}
inline size_t mix_step_lds(const MixStep& a) {
  const size_t work = (size_t)(MIX_HEADS * a.at.D + MIX_HEADS * MIX_KEYS + 256 * MIX_HEADS), merge = (size_t)MIX_HEADS * a.splits;
  const size_t at = a.at.H ? 2 * MIX_HEADS + (work > merge ? work : merge) : 0;
  const size_t li = a.li.H ? (size_t)(2 * a.li.D + 32 * 36) : 0;
  return (at > li ? at : li) * sizeof(float);
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
