// kx_wkv.h -- a linear recurrence with a decay per key channel and a bonus for the current token (RWKV time mixing)
// (kx_wkv.hip).
//
// Per head, with receptance r, key k, value v, bonus u and decay w = exp(-exp(W2 tanh(.) + w0)) of the token:
//   o = (S + diag(u) k v^T)^T r;  S <- diag(w) S + k v^T.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include "kx_linear.h"
#include "kx_scan.h"

struct KxWkvSpec {
  int heads = 0, dim = 0;  // of keys and values
  int rank = 0;            // of the decay's projection
};
struct KxWkvArgs {
  KxWkvSpec s;
  const float *proj = nullptr;  // f32 [tokens][proj_ld]: r, k, v, and the decay's low-rank projection before its tanh
  int proj_ld = 0, r_off = 0, k_off = 0, v_off = 0, w_off = 0;
  KxMat w2;                     // [heads * dim][rank], of the model's type
  const float *w0 = nullptr, *u = nullptr;  // [heads * dim]
  float *state = nullptr;       // [batch][heads][dim][dim]
  int batch = 0, positions = 0; // token i * batch + b is the i-th new position of sequence b
  float *o = nullptr;           // f32 [tokens][heads * dim]
  float *work = nullptr;        // kx_wkv_work_floats (not used for one position)
  void *rows = nullptr;         // tokens * w2.ld elements of the model's type (not used for one position)
};
inline size_t kx_wkv_work_floats(const KxWkvSpec &s, int batch, int positions) {
  const size_t padded = kx_scan_padded(positions), hd = (size_t)s.heads * s.dim;
  return (size_t)batch * (3 * positions * hd + padded * s.heads * KX_SCAN_BLOCK + padded / KX_SCAN_BLOCK * hd) + 64;
}
int kx_wkv_launch(bool f32, const KxWkvArgs &a, hipStream_t st);
