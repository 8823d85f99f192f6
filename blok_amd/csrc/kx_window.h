// kx_window.h -- grouped-query attention over a sliding window and pooled blocks of what lies before it, with its cache
// (kx_window.hip).
//
// Position i attends to the positions j with 0 <= i - j < size and, one key and value each, to the blocks
// [b pool, (b + 1) pool) with b pool + pool - 1 <= i - size: the means of the block's cached keys and values.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

struct KxWindowSpec {
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  float scale = 1;
  int size = 0x3fffffff;  // window; the default is every position
  int pool = 0;           // block length; 0: nothing is seen beyond the window
  int sink = 0;           // 1: the softmax's denominator has exp(0) more, or exp(KxWindowArgs::sinks[head])
};

// The cache of one layer.  Per sequence and key/value head a ring of `cap` positions (position j in slot j % cap) and
// one row per completed block.  Rows are padded to whole multiples of 32 elements with zeros.
struct KxWindowCache {
  void *k = nullptr, *v = nullptr;    // [batch][kv_heads][cap][dp], [..][vp]
  void *pk = nullptr, *pv = nullptr;  // [batch][kv_heads][blocks][dp], [..][vp]
  int cap = 0, blocks = 0, dp = 0, vp = 0;
};
// Shape of the cache for sequences of up to max_context positions and steps of up to max_positions of them; the
// element counts of one of k, v, pk, pv per sequence go to elems[4].
void kx_window_shape(const KxWindowSpec &s, int max_context, int max_positions, KxWindowCache *c, size_t elems[4]);

struct KxWindowArgs {
  KxWindowSpec s;
  KxWindowCache c;
  const float *proj = nullptr;  // f32 [tokens][proj_ld]: q at q_off, k, v, and the output gate
  int proj_ld = 0, q_off = 0, k_off = 0, v_off = 0, g_off = -1;  // g_off < 0: no gate
  const float *q_norm = nullptr, *k_norm = nullptr;  // RMS norm over the whole projection; nullptr: none
  float eps = 0;
  const float *sinks = nullptr;           // [heads]; nullptr: zeros
  int batch = 0, positions = 0, pos = 0;  // token i * batch + b is position pos + i of sequence b
  void *out = nullptr;                    // [tokens][out_ld] of the model's type: heads * vdim, gated
  int out_ld = 0;
  void *q = nullptr;        // scratch [tokens][heads][dp] of the model's type
  float *part = nullptr;    // scratch of part_floats floats (kx_window_part_floats)
  size_t part_floats = 0;
};
// floats of `part` that let `tokens` tokens attend in one launch
size_t kx_window_part_floats(const KxWindowSpec &s, int max_context, int tokens);
int kx_window_launch(bool f32, const KxWindowArgs &a, hipStream_t st);
// The attention alone, with a.q and the cache's rows in place.
int kx_window_attend(bool f32, const KxWindowArgs &a, hipStream_t st);
