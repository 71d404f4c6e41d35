// sampler.hpp -- the greedy sampler's first stage, shared by the llama step (fused_ffn.hpp) and the hybrid decoder's
// (hybrid_step.hpp): Iterator::max_by keeps the LAST maximum (sampler.rs:109-116).
// ARGMAX_BLOCKS workgroups per row of logits, each over a contiguous slice; a second launch combines and advances.
#pragma once
#include "devutil.hpp"

namespace crabml_hip {

#define ARGMAX_BLOCKS 128
__device__ __forceinline__ void argmax_combine(float& cv, int& ci, float ov, int oi) {
  // keep the later index among equal maxima; an index of -1 means "empty"
  bool take = oi >= 0 && (ci < 0 || ov > cv || (!(cv > ov) && oi > ci));
  if (take) {
    cv = ov;
    ci = oi;
  }
}
// base: global index of logits[0] (a vocabulary shard of a tensor-parallel classifier; 0 otherwise).  blockIdx.y: row of a batch
// (row_stride floats apart; its partials follow the previous row's)
static __global__ __launch_bounds__(256) void k_argmax_partial(const float* __restrict__ logits, int n, float* __restrict__ pv,
                                                        int* __restrict__ pi, int base, int row_stride) {
  logits += (size_t)blockIdx.y * row_stride;
  pv += blockIdx.y * gridDim.x;
  pi += blockIdx.y * gridDim.x;
  __shared__ float sv[4];
  __shared__ int si[4];
  const int per = (n + gridDim.x - 1) / gridDim.x;
  const int lo = blockIdx.x * per, hi = min(n, lo + per);
  float bv = -INFINITY;
  int bi = -1;
  for (int i = lo + threadIdx.x; i < hi; i += blockDim.x) argmax_combine(bv, bi, logits[i], base + i);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    float ov = __shfl_xor(bv, o, 64);
    int oi = __shfl_xor(bi, o, 64);
    argmax_combine(bv, bi, ov, oi);
  }
  if ((threadIdx.x & 63) == 0) {
    sv[threadIdx.x >> 6] = bv;
    si[threadIdx.x >> 6] = bi;
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 4; w++) argmax_combine(bv, bi, sv[w], si[w]);
    pv[blockIdx.x] = bv;
    pi[blockIdx.x] = bi;
  }
}

}  // namespace crabml_hip
