// kx_experts.hip -- see kx_experts.h.
//
// The counterpart of the router and of expert_accum_k (src/kimi_exec.cu:372-391, :835-877) for a decoder whose experts are
// bf16 or f32 matrices of any size: the host never sees the expert ids.
#include "kx_common.h"
#include "kx_experts.h"

namespace {

__global__ void __launch_bounds__(256) route_k(KxExpertArgs e, int tokens) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t < tokens) kxe::route_wave(e.logits + (size_t)t * e.logits_ld, e.bias, e.experts, e.top, e.ids + (size_t)t * e.top, e.weights + (size_t)t * e.top);
}

// one workgroup: counts per expert, their running sums, tiles, and a slot for every pair
__global__ void __launch_bounds__(KX_MAX_EXPERTS) bucket_k(KxExpertArgs e, KxExpertSlots s, int pairs) {
  __shared__ int count[KX_MAX_EXPERTS], at[2][KX_MAX_EXPERTS], tile_at[2][KX_MAX_EXPERTS];
  const int tid = threadIdx.x;
  count[tid] = 0;
  __syncthreads();
  for (int p = tid; p < pairs; p += KX_MAX_EXPERTS) atomicAdd(&count[s.ids[p]], 1);
  __syncthreads();
  const int n = count[tid], tiles = (n + e.tile_slots - 1) / e.tile_slots;
  int cur = 0;
  at[0][tid] = n;
  tile_at[0][tid] = tiles;
  __syncthreads();
  for (int d = 1; d < KX_MAX_EXPERTS; d <<= 1, cur ^= 1) {  // inclusive sums
    at[cur ^ 1][tid] = at[cur][tid] + (tid >= d ? at[cur][tid - d] : 0);
    tile_at[cur ^ 1][tid] = tile_at[cur][tid] + (tid >= d ? tile_at[cur][tid - d] : 0);
    __syncthreads();
  }
  const int slot0 = at[cur][tid] - n, tile0 = tile_at[cur][tid] - tiles;
  if (tid == KX_MAX_EXPERTS - 1) *s.n_tiles = tile_at[cur][tid];
  for (int i = 0; i < tiles; ++i) s.tiles[tile0 + i] = make_int4(tid, slot0 + i * e.tile_slots, min(e.tile_slots, n - i * e.tile_slots), 0);
  count[tid] = slot0;
  __syncthreads();
  for (int p = tid; p < pairs; p += KX_MAX_EXPERTS) {
    const int slot = atomicAdd(&count[s.ids[p]], 1);
    s.gather[slot] = p / e.top;
    s.slot_weight[slot] = s.weights[p];
    s.slot_of[p] = slot;
  }
}

__global__ void __launch_bounds__(256) combine_k(KxExpertSlots s, const float *__restrict__ y, float *__restrict__ x, int top, int width) {
  __shared__ int slot[KX_MAX_TOP];
  const size_t t = blockIdx.x;
  if ((int)threadIdx.x < top) slot[threadIdx.x] = s.slot_of[t * top + threadIdx.x];
  __syncthreads();
  for (int c = blockIdx.y * 256 + threadIdx.x; c < width; c += gridDim.y * 256) {
    float v = y[(size_t)slot[0] * width + c];
    for (int j = 1; j < top; ++j) v += y[(size_t)slot[j] * width + c];
    x[t * width + c] += v;
  }
}

}  // namespace

int kx_expert_route_launch(bool f32, KxExpertArgs &e, const KxExpertSlots &s, int tokens, hipStream_t st) {
  KX_REQUIRE(e.experts > 0 && e.experts <= KX_MAX_EXPERTS && e.top > 0 && e.top <= e.experts && e.top <= KX_MAX_TOP && tokens > 0 && e.logits && e.bias,
             "experts: %d of %d for %d tokens", e.top, e.experts, tokens);
  e.ids = s.ids; e.weights = s.weights;
  e.tile_slots = kx_expert_tile(f32, tokens, e.top, e.experts);
  e.max_tiles = kx_expert_tiles(tokens, e.top, e.experts, e.tile_slots);
  e.tiles = s.tiles; e.n_tiles = s.n_tiles; e.slot_weight = s.slot_weight;
  hipLaunchKernelGGL(route_k, dim3(kx_cdiv(tokens, 4)), dim3(256), 0, st, e, tokens);
  KX_LAUNCH_CHECK();
  hipLaunchKernelGGL(bucket_k, dim3(1), dim3(KX_MAX_EXPERTS), 0, st, e, s, tokens * e.top);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

int kx_expert_combine_launch(const KxExpertSlots &s, const float *y, float *x, int tokens, int top, int width, hipStream_t st) {
  hipLaunchKernelGGL(combine_k, dim3(tokens, kx_cdiv(width, 1024)), dim3(256), 0, st, s, y, x, top, width);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

int kx_expert_ff_launch(bool f32, const KxExpertFf &f, int tokens, hipStream_t st) {
  KxLinArgs gu = f.gu;
  gu.epi = KX_LIN_GLU;
  gu.mid = f.mid;
  gu.mid_ld = f.down.ld;
  KxExpertArgs e = f.e, eo = f.e;
  e.ids = eo.ids = f.s.ids;
  e.weights = eo.weights = f.s.weights;
  e.stride = f.gu_stride;
  eo.stride = f.down_stride; eo.w = f.down.w; eo.ld = f.down.ld; eo.mid = f.mid; eo.mid_ld = f.down.ld;
  if (kx_expert_small(f32, gu, f.out, eo, tokens)) {
    KX_DO(kx_expert_in_launch(f32, gu, e, st));
    return kx_expert_out_launch(f32, f.out, eo, st);
  }
  const void *h = f.h;
  if (!h) {
    KX_DO(kx_rows_launch(f32, gu.row, tokens, f.h_buf, gu.m.ld, st));
    h = f.h_buf;
  }
  KX_DO(kx_expert_route_launch(f32, e, f.s, tokens, st));
  e.gather = f.s.gather;
  KX_DO(kx_expert_gemm_launch(f32, gu, e, h, gu.m.ld, st));
  KX_DO(kx_linear_launch(f32, f.out, f.row_buf, st));
  KxLinArgs down;
  down.m = f.down;
  down.tokens = tokens;
  down.row.cols = f.down.cols;
  down.out = f.y;
  down.out_ld = f.down.rows;
  e.gather = nullptr;
  e.stride = f.down_stride;
  KX_DO(kx_expert_gemm_launch(f32, down, e, f.mid, f.down.ld, st));
  return kx_expert_combine_launch(f.s, f.y, f.out.streams, tokens, e.top, f.down.rows, st);
}
