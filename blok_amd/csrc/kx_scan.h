// kx_scan.h -- linear recurrences with a diagonal decay over many positions (kx_scan.hip): per head, with key k, query q,
// value v and decay w (one number, or one per key channel),
//   S_t = diag(w_t) S_{t-1} + k_t v_t^T,   o_t = S^T q_t,
// taken in blocks of KX_SCAN_BLOCK tokens.  With S the state before a block,
//   o_j = gamma_j S^T q_j + sum_{i <= j} inner[j][i] v_i,   S <- diag(total) S + sum_i end_i k_i v_i^T.
// The caller makes these numbers, which do not depend on the value's column (kx_ssd.hip, kx_wkv.hip).  With a decay per
// channel, gamma and end are part of q and k.
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>

constexpr int KX_SCAN_BLOCK = 16, KX_SCAN_MAX_DIM = 512;
__host__ __device__ inline int kx_scan_padded(int positions) { return (positions + KX_SCAN_BLOCK - 1) / KX_SCAN_BLOCK * KX_SCAN_BLOCK; }

struct KxScanArgs {
  int heads = 0, groups = 0, dim = 0, vdim = 0;  // groups: heads / groups consecutive heads share q and k
  int batch = 0, positions = 0;                  // token i * batch + b is the i-th position of sequence b
  bool channel = false;                          // a decay per key channel
  const float *q = nullptr, *k = nullptr, *v = nullptr;  // f32 rows per token, a group's (head's) columns one after the other
  int q_ld = 0, k_ld = 0, v_ld = 0;
  const float *inner = nullptr;                        // [batch][heads][padded][KX_SCAN_BLOCK]; zero for i > j and past the last position
  const float *gamma = nullptr, *end = nullptr;        // !channel: [batch][heads][padded]; end is zero past the last position
  const float *total = nullptr;                        // channel: [batch][heads][blocks][dim]
  float *state = nullptr;                              // [batch][heads][dim][vdim]
  float *o = nullptr;                                  // f32 [tokens][heads * vdim]
};
int kx_scan_launch(const KxScanArgs &a, hipStream_t st);
