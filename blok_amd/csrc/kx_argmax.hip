// kx_argmax.hip -- lowest-index argmax over logits (sample_lm_head, src/kimi_exec.cu:718-734; argmax_k, :477-493), in
// two stages: KX_ARGMAX_PARTS workgroups per row each reduce a slice, then one wave per row merges them.
#include "kx_argmax.h"
#include "kx_common.h"

namespace {

__device__ __forceinline__ void argmax_merge(float &best, uint32_t &bi, float ov, uint32_t oi) {
  if (ov > best || (ov == best && oi < bi)) { best = ov; bi = oi; }
}
__device__ __forceinline__ void argmax_wave(float &best, uint32_t &bi) {
  for (int m = 32; m; m >>= 1) {
    float ov = __shfl_xor(best, m);
    uint32_t oi = (uint32_t)__shfl_xor((int)bi, m);
    argmax_merge(best, bi, ov, oi);
  }
}

__global__ void __launch_bounds__(256) argmax_part_k(const float *__restrict__ logits, int n, int stride,
                                                     float *__restrict__ pv, uint32_t *__restrict__ pi) {
  __shared__ float sv[4];
  __shared__ uint32_t si[4];
  const float *p = logits + (size_t)blockIdx.y * stride;
  const int per = (n + KX_ARGMAX_PARTS - 1) / KX_ARGMAX_PARTS;
  const int lo = blockIdx.x * per, hi = min(n, lo + per);
  float best = -__builtin_inff();
  uint32_t bi = 0xffffffffu;
  for (int i = lo + threadIdx.x; i < hi; i += blockDim.x) {
    float v = p[i];
    if (v > best) { best = v; bi = (uint32_t)i; }
  }
  argmax_wave(best, bi);
  if ((threadIdx.x & 63) == 0) { sv[threadIdx.x >> 6] = best; si[threadIdx.x >> 6] = bi; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 4; ++w) argmax_merge(best, bi, sv[w], si[w]);
    pv[blockIdx.y * KX_ARGMAX_PARTS + blockIdx.x] = best;
    pi[blockIdx.y * KX_ARGMAX_PARTS + blockIdx.x] = bi;
  }
}
__global__ void __launch_bounds__(64) argmax_final_k(const float *__restrict__ pv, const uint32_t *__restrict__ pi,
                                                     uint32_t *__restrict__ out) {
  float best = pv[blockIdx.x * KX_ARGMAX_PARTS + threadIdx.x];
  uint32_t bi = pi[blockIdx.x * KX_ARGMAX_PARTS + threadIdx.x];
  argmax_wave(best, bi);
  if (threadIdx.x == 0) out[blockIdx.x] = bi == 0xffffffffu ? 0u : bi;  // every logit -inf or NaN: id 0 as :481
}

}  // namespace

// scratch: tokens * KX_ARGMAX_PARTS floats and as many uint32
int kx_argmax_launch(const float *logits, int tokens, int n, int stride, uint32_t *out, float *scratch, hipStream_t st) {
  float *pv = scratch;
  uint32_t *pi = (uint32_t *)(scratch + (size_t)tokens * KX_ARGMAX_PARTS);
  hipLaunchKernelGGL(argmax_part_k, dim3(KX_ARGMAX_PARTS, tokens), dim3(256), 0, st, logits, n, stride, pv, pi);
  KX_LAUNCH_CHECK();
  hipLaunchKernelGGL(argmax_final_k, dim3(tokens), dim3(64), 0, st, pv, pi, out);
  KX_LAUNCH_CHECK();
  return KX_OK;
}
