// kx_conv.h -- short causal convolutions with silu, one per channel, in front of a recurrent layer (kx_conv.hip).
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include "kx_math.h"

struct KxConvArgs {
  const float *proj = nullptr;  // f32 [tokens][proj_ld]: the inputs; token i * batch + b is the i-th new position of sequence b
  int proj_ld = 0;
  int segs = 1, end[3] = {}, off[3] = {};  // channels [end[i - 1], end[i]) are the columns from off[i] on
  int channels = 0, taps = 1;
  const float *w = nullptr;     // [channels][taps], the last column meets the current token
  const float *bias = nullptr;  // [channels]; nullptr: none
  const float *hist = nullptr;  // [batch][taps - 1][channels]: the last inputs before this step, oldest first
  float *hist_out = nullptr;    // the same after this step (another buffer)
  int batch = 0, positions = 0;
};
// raw[token][channel] = silu(convolution); leaves hist_out
int kx_conv_launch(const KxConvArgs &a, float *raw, hipStream_t st);

namespace kxc {

__device__ __forceinline__ int column(const KxConvArgs &a, int ch) {
  if (a.segs > 2 && ch >= a.end[1]) return a.off[2] + ch - a.end[1];
  if (a.segs > 1 && ch >= a.end[0]) return a.off[1] + ch - a.end[0];
  return a.off[0] + ch;
}
// input of channel ch at position i of the step (i < 0: before it) of sequence b
__device__ __forceinline__ float input(const KxConvArgs &a, int b, int i, int ch, int col) {
  return i >= 0 ? a.proj[(size_t)(i * a.batch + b) * a.proj_ld + col] : a.hist[((size_t)b * (a.taps - 1) + a.taps - 1 + i) * a.channels + ch];
}
__device__ __forceinline__ float conv_silu(const KxConvArgs &a, int b, int i, int ch) {
  const int col = column(a, ch);
  float v = a.bias ? a.bias[ch] : 0.0f;
  for (int j = 0; j < a.taps; ++j) v = __builtin_fmaf(a.w[(size_t)ch * a.taps + j], input(a, b, i - (a.taps - 1) + j, ch, col), v);
  return kx_siluf(v);
}
// the inputs of channel ch that the next step needs
__device__ __forceinline__ void shift(const KxConvArgs &a, int b, int ch) {
  const int keep = a.taps - 1, col = column(a, ch);
  for (int j = 0; j < keep; ++j) a.hist_out[((size_t)b * keep + j) * a.channels + ch] = input(a, b, a.positions - keep + j, ch, col);
}

}  // namespace kxc
