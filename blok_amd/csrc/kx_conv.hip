// kx_conv.hip -- see kx_conv.h.  Everything here is 32-bit.  No counterpart in the reference.
#include "kx_common.h"
#include "kx_conv.h"

namespace {

constexpr int CONV_TOKENS = 16;  // positions a thread goes through
template <int TAPS>              // 0: any number
__global__ void __launch_bounds__(256) conv_silu_k(KxConvArgs a, float *__restrict__ raw) {
  const int C = a.channels, ch = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z;
  const int i0 = blockIdx.y * CONV_TOKENS, i1 = min(i0 + CONV_TOKENS, a.positions);
  if (ch >= C) return;
  if constexpr (TAPS == 0) {
    for (int i = i0; i < i1; ++i) raw[(size_t)(i * a.batch + b) * C + ch] = kxc::conv_silu(a, b, i, ch);
  } else {
    const int col = kxc::column(a, ch);
    const float bias = a.bias ? a.bias[ch] : 0.0f;
    float w[TAPS], x[CONV_TOKENS + TAPS - 1];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j] = a.w[(size_t)ch * TAPS + j];
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) x[j] = kxc::input(a, b, i0 - (TAPS - 1) + j, ch, col);
#pragma unroll
    for (int j = 0; j < CONV_TOKENS; ++j) x[TAPS - 1 + j] = a.proj[(size_t)(min(i0 + j, a.positions - 1) * a.batch + b) * a.proj_ld + col];
#pragma unroll
    for (int j = 0; j < CONV_TOKENS; ++j) {
      float v = bias;
#pragma unroll
      for (int t = 0; t < TAPS; ++t) v = __builtin_fmaf(w[t], x[j + t], v);
      if (i0 + j < i1) raw[(size_t)((i0 + j) * a.batch + b) * C + ch] = kx_siluf(v);
    }
  }
}

__global__ void __launch_bounds__(256) conv_hist_k(KxConvArgs a) {
  const int ch = blockIdx.x * 256 + threadIdx.x;
  if (ch < a.channels) kxc::shift(a, blockIdx.y, ch);
}

}  // namespace

int kx_conv_launch(const KxConvArgs &a, float *raw, hipStream_t st) {
  KX_REQUIRE(a.channels > 0 && a.taps > 0 && a.batch > 0 && a.positions > 0 && raw && (a.taps == 1 || (a.hist && a.hist_out && a.hist != a.hist_out)),
             "convolution: %d channels, %d taps, %d x %d tokens", a.channels, a.taps, a.batch, a.positions);
  const dim3 grid(kx_cdiv(a.channels, 256), kx_cdiv(a.positions, CONV_TOKENS), a.batch);
  if (a.taps == 2) hipLaunchKernelGGL(conv_silu_k<2>, grid, dim3(256), 0, st, a, raw);
  else if (a.taps == 3) hipLaunchKernelGGL(conv_silu_k<3>, grid, dim3(256), 0, st, a, raw);
  else if (a.taps == 4) hipLaunchKernelGGL(conv_silu_k<4>, grid, dim3(256), 0, st, a, raw);
  else hipLaunchKernelGGL(conv_silu_k<0>, grid, dim3(256), 0, st, a, raw);
  KX_LAUNCH_CHECK();
  if (a.taps > 1) {
    hipLaunchKernelGGL(conv_hist_k, dim3(kx_cdiv(a.channels, 256), a.batch), dim3(256), 0, st, a);
    KX_LAUNCH_CHECK();
  }
  return KX_OK;
}
