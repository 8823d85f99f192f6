// kx_delta.h -- the gated delta rule: a linear-attention layer with a recurrent state per head, behind short causal
// convolutions (kx_delta.hip).
//
// Per head, with unit query and key q, k, value v, step size beta and decay g of the token:
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

struct KxDeltaSpec {
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  int taps = 1;            // of the convolutions on q, k and v (silu behind them)
  float unit_eps = 1e-6f;  // x / sqrt(sum x^2 + unit_eps)
};
__host__ __device__ inline int kx_delta_channels(const KxDeltaSpec &s) { return 2 * s.kv_heads * s.dim + s.heads * s.vdim; }  // q, k, v

struct KxDeltaArgs {
  KxDeltaSpec s;
  const float *proj = nullptr;  // f32 [tokens][proj_ld]: q, k, v (before the convolution), beta's and the decay's projection
  int proj_ld = 0, q_off = 0, k_off = 0, v_off = 0, b_off = 0, a_off = 0;
  const float *conv = nullptr;    // [channels][taps], the last column meets the current token
  const float *a_log = nullptr, *dt_bias = nullptr;  // [heads]
  float *state = nullptr;         // [batch][heads][dim][vdim]
  const float *hist = nullptr;    // [batch][taps - 1][channels]: the convolutions' last inputs, oldest first
  float *hist_out = nullptr;      // the same after this step (another buffer)
  int batch = 0, positions = 0;   // token i * batch + b is the i-th new position of sequence b
  float *o = nullptr;             // f32 [tokens][heads * vdim]
  float *work = nullptr;          // kx_delta_work_floats(s, batch, positions) floats (not used for one position)
};
// Tokens go through the state in blocks of KX_DELTA_BLOCK; per token and head there are KX_DELTA_COEF numbers.
constexpr int KX_DELTA_BLOCK = 4, KX_DELTA_COEF = 12;
// keys and queries lie in the scratch with rows of 32, 64, 128 or 256
__host__ __device__ inline int kx_delta_row(const KxDeltaSpec &s) { return s.dim <= 32 ? 32 : s.dim <= 64 ? 64 : s.dim <= 128 ? 128 : 256; }
inline size_t kx_delta_work_floats(const KxDeltaSpec &s, int batch, int positions) {
  const size_t padded = (size_t)batch * ((positions + KX_DELTA_BLOCK - 1) / KX_DELTA_BLOCK * KX_DELTA_BLOCK);
  return padded * ((size_t)KX_DELTA_COEF * s.heads + kx_delta_channels(s) + 2 * s.kv_heads * kx_delta_row(s));
}
int kx_delta_launch(const KxDeltaArgs &a, hipStream_t st);
