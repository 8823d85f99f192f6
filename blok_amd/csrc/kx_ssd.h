// kx_ssd.h -- state-space duality (Mamba-2): a recurrence with one decay per head and keys shared by groups of heads, behind
// a short causal convolution (kx_ssd.hip).
//
// Per head, with x, B, C behind convolution and silu, dt = softplus(. + dt_bias) and a = exp(-exp(A_log) dt):
//   S <- a S + dt B x^T;  y = S^T C + D x.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include "kx_scan.h"

struct KxSsdSpec {
  int heads = 0, vdim = 0, state = 0, groups = 1;  // state: rows of S; head h has B and C of group h / (heads / groups)
  int taps = 1;
};
__host__ __device__ inline int kx_ssd_inner(const KxSsdSpec &s) { return s.heads * s.vdim; }
__host__ __device__ inline int kx_ssd_channels(const KxSsdSpec &s) { return kx_ssd_inner(s) + 2 * s.groups * s.state; }  // x, B, C

struct KxSsdArgs {
  KxSsdSpec s;
  const float *proj = nullptr;  // f32 [tokens][proj_ld]: x, B, C from x_off on (before the convolution), dt at dt_off
  int proj_ld = 0, x_off = 0, dt_off = 0;
  const float *conv = nullptr, *conv_bias = nullptr;  // [channels][taps], the last column meets the current token; [channels]
  const float *a_log = nullptr, *dt_bias = nullptr, *skip = nullptr;  // [heads]
  float *state = nullptr;                             // [batch][heads][state][vdim]
  const float *hist = nullptr;                        // [batch][taps - 1][channels]
  float *hist_out = nullptr;                          // the same after this step (another buffer)
  int batch = 0, positions = 0;                       // token i * batch + b is the i-th new position of sequence b
  float *y = nullptr;                                 // f32 [tokens][heads * vdim]
  float *work = nullptr;                              // kx_ssd_work_floats (not used for one position)
};
inline size_t kx_ssd_work_floats(const KxSsdSpec &s, int batch, int positions) {
  return (size_t)batch * ((size_t)positions * kx_ssd_channels(s) + (size_t)kx_scan_padded(positions) * s.heads * (KX_SCAN_BLOCK + 2)) + 64;
}
int kx_ssd_launch(const KxSsdArgs &a, hipStream_t st);
