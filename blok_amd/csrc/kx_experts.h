// kx_experts.h -- a mixture of gated feed-forward experts: routing by logits, softmax over the chosen ones
// (kx_experts.hip); the products are kx_linear's.
#pragma once
#include "kx_linear.h"
#include "kx_math.h"
#include "kx_wave.h"

// A step's (token, choice) pairs sorted by expert.
struct KxExpertSlots {
  int *ids = nullptr, *gather = nullptr, *slot_of = nullptr;  // [tokens * top]: expert of a pair; token of a slot; slot of a pair
  float *weights = nullptr, *slot_weight = nullptr;
  int4 *tiles = nullptr;
  int *n_tiles = nullptr;
};
// slots per tile of a step (those of the GEMM that will read them), and the most tiles its pairs make
inline int kx_expert_tile(bool f32, int tokens, int top, int experts) { return !f32 && (long)tokens * top >= 96L * experts ? 128 : 64; }
inline int kx_expert_tiles(int tokens, int top, int experts, int tile) {
  const int pairs = tokens * top;
  return (pairs + tile - 1) / tile + (experts < pairs ? experts : pairs);
}
// Routes `tokens` tokens (e.logits, e.bias) and sorts the pairs into s; fills in e what kx_expert_gemm_launch reads.
int kx_expert_route_launch(bool f32, KxExpertArgs &e, const KxExpertSlots &s, int tokens, hipStream_t st);
// x[t] += sum_j y[slot of choice j of t], f32 rows of `width`
int kx_expert_combine_launch(const KxExpertSlots &s, const float *y, float *x, int tokens, int top, int width, hipStream_t st);

// A feed-forward of experts beside another product that is added to the same residual rows:
//   x_t <- x_t + out.m row_t + sum_j weight_j down[id_j] glu(gu[id_j] h_t)
struct KxExpertFf {
  KxLinArgs gu, out;          // the first expert's (gate, up) with the rows h in front (one norm of x); the other product
  KxMat down;                 // the first expert's
  size_t gu_stride = 0, down_stride = 0;  // elements from one expert's matrix to the next
  KxExpertArgs e;             // experts, top, logits, logits_ld, bias
  KxExpertSlots s;
  const void *h = nullptr;    // the rows h, if they are in memory, rows of gu.m.ld elements; nullptr: built where they are needed
  void *h_buf = nullptr, *row_buf = nullptr;  // room for them and for the other product's rows
  void *mid = nullptr;        // [tokens * top][down.ld] of the model's type
  float *y = nullptr;         // f32 [tokens * top][width]
};
// Up to KX_GEMV_TOKENS tokens two launches where the sizes allow; otherwise sorted by expert.
int kx_expert_ff_launch(bool f32, const KxExpertFf &f, int tokens, hipStream_t st);

namespace kxe {

// The `top` largest of logits + bias, the lower index first where two are equal, and the softmax over them.  One wave.
__device__ __forceinline__ void route_wave(const float *__restrict__ logits, const float *__restrict__ bias, int experts, int top, int *ids, float *weights) {
  constexpr int PER = KX_MAX_EXPERTS / 64;
  const int lane = threadIdx.x & 63;
  float z[PER];
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int e = j * 64 + lane;
    z[j] = e < experts ? logits[e] + bias[e] : -__builtin_inff();
  }
  float first = 0.0f, mine = 0.0f, sum = 0.0f;  // mine: lane k holds the weight of choice k
  int id = 0;
  for (int k = 0; k < top; ++k) {
    float best = -__builtin_inff();
    int at = 0x7fffffff;
#pragma unroll
    for (int j = 0; j < PER; ++j)
      if (j * 64 < experts && z[j] > best) {
        best = z[j];
        at = j * 64 + lane;
      }
    const float m = kxw::wave_max_f32(best);
    int chosen = kxw::wave_min_i32(best == m ? at : 0x7fffffff);
    if (chosen >= experts) chosen = 0;  // only where logits are not numbers
    if (k == 0) first = m;
    const float w = kx_expf(m - first);
    sum += w;
    if (lane == k) {
      mine = w;
      id = chosen;
    }
#pragma unroll
    for (int j = 0; j < PER; ++j)
      if (chosen == j * 64 + lane) z[j] = -__builtin_inff();
  }
  if (lane < top) {
    ids[lane] = id;
    weights[lane] = mine / sum;
  }
}

}  // namespace kxe
