// kx_rows.h -- activation rows of the hybrid decoder, built by one workgroup: what a matrix product reads as its
// input.  The same code fills a row in LDS (the prologue of a decode GEMV, kx_linear.hip) and in memory (row_k, for
// steps of many tokens).  No counterpart in the reference, whose decoder has one residual stream.
//
//   NORM   h = w * groupnorm(sum_s in[s] x_s): the input of a sublayer with several residual streams
//   GATED  per head: a recurrence's read-out over its root mean square, times a weight, with silu(gate) behind the norm or in
//          front of it
//   SHIFT  several mixes of a normed row with the one of the position before it, and the row itself
//   TANH   tanh of a 32-bit row
//   PLAIN  a row that is in memory already
// Rows are padded to the matrix's leading dimension; pad columns are zero (or, in memory, finite: the matrix's pad
// columns are zero).
#pragma once
#include "kx_linear.h"
#include "kx_math.h"
#include "kx_wave.h"

namespace kxr {

typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));

template <class T> struct Elem;
template <> struct Elem<uint16_t> {
  static __device__ __forceinline__ float load(const uint16_t *p) { return kx_bf16_f32(*p); }
  static __device__ __forceinline__ uint16_t make(float v) { return kx_bf16_rne(v); }
  // eight elements of a weight stream, as they come
  struct Raw { u32x4 a; };
  static __device__ __forceinline__ Raw stream(const uint16_t *p) { return Raw{__builtin_nontemporal_load((const u32x4 *)p)}; }
  static __device__ __forceinline__ Raw cached(const uint16_t *p) { return Raw{*(const u32x4 *)p}; }
  static __device__ __forceinline__ void unpack(float (&f)[8], const Raw &r) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f[2 * i] = kx_bits_f32(r.a[i] << 16);
      f[2 * i + 1] = kx_bits_f32(r.a[i] & 0xffff0000u);
    }
  }
};
template <> struct Elem<float> {
  static __device__ __forceinline__ float load(const float *p) { return *p; }
  static __device__ __forceinline__ float make(float v) { return v; }
  struct Raw { u32x4 a, b; };
  static __device__ __forceinline__ Raw stream(const float *p) {
    return Raw{__builtin_nontemporal_load((const u32x4 *)p), __builtin_nontemporal_load((const u32x4 *)(p + 4))};
  }
  static __device__ __forceinline__ Raw cached(const float *p) { return Raw{((const u32x4 *)p)[0], ((const u32x4 *)p)[1]}; }
  static __device__ __forceinline__ void unpack(float (&f)[8], const Raw &r) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f[i] = kx_bits_f32(r.a[i]);
      f[4 + i] = kx_bits_f32(r.b[i]);
    }
  }
};

// sigmoid for a value that is rounded to T next: without branches and with the approximate reciprocal for bf16
template <class T>
__device__ __forceinline__ float sigmoid_for(float x) {
  if constexpr (sizeof(T) == 4) return kx_sigmoidf(x);
  else return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.44269504088896341f * x));
}

// log(1 + exp(x))
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.0f) + log1pf(kx_expf(-fabsf(x))); }

// sum over the lanes of a wave, in every lane
__device__ __forceinline__ float wave_sum(float v) {
  float t = v;
  kxw::swap_halves32(v, t);
  v += t;
  t = v;
  kxw::swap_rows16(v, t);
  v += t;
  v += kxw::dpp_f<kxw::DPP_ROW_MIRROR>(v);
  v += kxw::dpp_f<kxw::DPP_ROW_HALF_MIRROR>(v);
  v += kxw::dpp_f<kxw::DPP_QUAD_XOR2>(v);
  v += kxw::dpp_f<kxw::DPP_QUAD_XOR1>(v);
  return v;
}
// sum over a workgroup, in every thread; red: one float per wave
__device__ __forceinline__ float block_sum(float v, float *red) {
  v = wave_sum(v);
  const int nw = blockDim.x >> 6;
  __syncthreads();  // red may still be read from the last call
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = red[0];
  for (int w = 1; w < nw; ++w) s += red[w];
  return s;
}

// sums of squares of `groups` equal parts of u[0 .. cols) -> part[g * spg] = 1 / root mean square; spg slices per group, whose
// sums are in part[] and behind a barrier
__device__ __forceinline__ void group_scales(float *part, int groups, int spg, int gs, float eps) {
  for (int g = threadIdx.x; g < groups; g += blockDim.x) {
    float s = part[g * spg];
    for (int j = 1; j < spg; ++j) s += part[g * spg + j];
    part[g * spg] = kx_rsqrtf(s / (float)gs + eps);
  }
  __syncthreads();
}

// Row `tok` into dst[0 .. ld), variants vstride apart.  u: LDS scratch of kx_row_scratch(a) floats.  Whole workgroup; ends
// with a barrier.  keep: this workgroup writes what the row's kind carries over to the next step.  need: the variants
// to build, a bit each.
// KIND: the row's kind where it is known when the kernel is compiled.
template <class T, int KIND = -1>
__device__ __forceinline__ void build_row(const KxRowArgs &a, int tok, T *dst, int ld, float *u, size_t vstride = 0, bool keep = false,
                                          uint32_t need = ~0u) {
  const int tid = threadIdx.x, n = blockDim.x, lane = tid & 63, wave = tid >> 6, nw = n >> 6, kind = KIND >= 0 ? KIND : a.kind;
  if (a.rows_map) tok = a.rows_map[tok];
  const int xld = a.streams_ld ? a.streams_ld : a.n_streams * a.cols;
  if (kind == KX_ROW_NORM) {
    float *part = u + a.cols;
    const float *x = a.streams + (size_t)tok * xld;
    const int gs = a.cols / a.groups, spg = max(1, nw / a.groups), units = a.groups * spg, per = (gs + spg - 1) / spg;
    for (int k = wave; k < units; k += nw) {  // a wave takes a slice of one group
      const int g = k / spg, s = k - g * spg, hi = min(gs, (s + 1) * per);
      float v = 0.0f;
      for (int j = s * per + lane; j < hi; j += 64) {
        const int c = g * gs + j;
        float y = 0.0f;
        for (int t = 0; t < a.n_streams; ++t) y = __builtin_fmaf(a.in ? a.in[t] : 1.0f, x[(size_t)t * a.cols + c], y);
        u[c] = y;
        v = __builtin_fmaf(y, y, v);
      }
      v = wave_sum(v);
      if (lane == 0) part[k] = v;
    }
    __syncthreads();
    group_scales(part, a.groups, spg, gs, a.eps);
    for (int c = tid; c < ld; c += n) dst[c] = Elem<T>::make(c < a.cols ? u[c] * part[(c / gs) * spg] * a.w[c] : 0.0f);
  } else if (kind == KX_ROW_SHIFT) {
    const bool first = tok < a.batch;
    const float *x = a.streams + (size_t)tok * xld, *x1 = first ? a.prev + (size_t)tok * a.cols : x - (size_t)a.batch * xld;
    float v = 0.0f, v1 = 0.0f;
    for (int c = tid; c < a.cols; c += n) {
      v = __builtin_fmaf(x[c], x[c], v);
      v1 = __builtin_fmaf(x1[c], x1[c], v1);
    }
    const float sc = kx_rsqrtf(block_sum(v, u) / (float)a.cols + a.eps), sc1 = kx_rsqrtf(block_sum(v1, u) / (float)a.cols + a.eps);
    const bool last = keep && tok + a.batch >= a.tokens;
    for (int c = tid; c < ld; c += n) {
      float h = 0.0f, d = 0.0f;
      if (c < a.cols) {
        const float w = a.w[c];
        h = x[c] * sc * w;
        d = (first ? x1[c] : x1[c] * sc1 * w) - h;
        if (last) a.prev_out[(size_t)(tok + a.batch - a.tokens) * a.cols + c] = h;
      }
      for (int m = 0; m < a.n_mix; ++m)
        if (need >> m & 1) dst[m * vstride + c] = Elem<T>::make(c < a.cols ? __builtin_fmaf(d, a.mu[(size_t)m * a.cols + c], h) : 0.0f);
      dst[a.n_mix * vstride + c] = Elem<T>::make(h);
    }
  } else if (kind == KX_ROW_GATED) {
    const int cols = a.heads * a.vdim, hl = a.tail ? a.head_ld : ld;
    const float *o = a.o + (size_t)tok * cols, *gate = a.gate + (size_t)tok * a.gate_ld;
    auto gated = [&](int c) { return a.gate_first ? o[c] * gate[c] * sigmoid_for<T>(gate[c]) : o[c]; };
    auto out = [&](int c, int d, float y) {
      y *= a.w[a.w_per_column ? c : d];
      dst[c] = Elem<T>::make(a.gate_first ? y : y * gate[c] * sigmoid_for<T>(gate[c]));
    };
    if (a.heads < 8) {  // a few long parts: several waves each
      float *part = u + cols;
      const int spg = max(1, nw / a.heads), units = a.heads * spg, per = (a.vdim + spg - 1) / spg;
      for (int k = wave; k < units; k += nw) {
        const int h = k / spg, s = k - h * spg, hi = min(a.vdim, (s + 1) * per);
        float v = 0.0f;
        for (int d = s * per + lane; d < hi; d += 64) {
          const float y = gated(h * a.vdim + d);
          u[h * a.vdim + d] = y;
          v = __builtin_fmaf(y, y, v);
        }
        v = wave_sum(v);
        if (lane == 0) part[k] = v;
      }
      __syncthreads();
      group_scales(part, a.heads, spg, a.vdim, a.eps);
      for (int c = tid; c < cols; c += n) out(c, c % a.vdim, u[c] * part[(c / a.vdim) * spg]);
    } else {
      for (int h = wave; h < a.heads; h += nw) {
        float v = 0.0f;
        for (int d = lane; d < a.vdim; d += 64) {
          const float y = gated(h * a.vdim + d);
          v = __builtin_fmaf(y, y, v);
        }
        const float sc = kx_rsqrtf(wave_sum(v) / (float)a.vdim + a.eps);
        for (int d = lane; d < a.vdim; d += 64) out(h * a.vdim + d, d, gated(h * a.vdim + d) * sc);
      }
    }
    for (int c = cols + tid; c < hl; c += n) dst[c] = Elem<T>::make(0.0f);
    if (a.tail) {
      const T *x = (const T *)a.tail + (size_t)tok * a.tail_ld;
      for (int c = tid * 8; c < ld - hl; c += n * 8) *(typename Elem<T>::Raw *)(dst + hl + c) = Elem<T>::cached(x + c);
    }
  } else if (kind == KX_ROW_TANH) {
    const float *x = a.streams + (size_t)tok * xld;
    for (int c = tid; c < ld; c += n) dst[c] = Elem<T>::make(c < a.cols ? tanhf(x[c]) : 0.0f);
  } else {
    const T *x = (const T *)a.x + (size_t)tok * a.x_ld;
    for (int c = tid * 8; c < ld; c += n * 8) *(typename Elem<T>::Raw *)(dst + c) = Elem<T>::cached(x + c);
  }
  __syncthreads();
}

}  // namespace kxr
