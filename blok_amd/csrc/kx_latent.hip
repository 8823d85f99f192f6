// kx_latent.hip -- see kx_latent.h.
//
// The counterpart of the reference's multi-head latent attention (src/kimi_exec.cu:355-475, :677-716) for any sizes, with
// a sink and an output gate; kx_mla.hip is the same for Kimi-K2's.
//
// Few positions: W_uk is applied to the query (absorb_k, which also writes the cache rows), so that all heads attend to the
// cached rows themselves (kx_window.hip: one set of rows for groups of heads, values the first columns of the keys), and
// latent_out_k merges the parts, applies W_uv and the gate.
// Longer steps: prep_k writes queries and cache rows, two products make the keys and values of every position up to the
// step's last one, and kx_window.hip attends on the matrix cores.
#include <math.h>
#include <algorithm>
#include <vector>
#include "kx_common.h"
#include "kx_latent.h"
#include "kx_rows.h"

namespace {

using kxr::Elem;
constexpr int ABS_COLS = 128, OUT_ROWS = 32, HEAD_GROUP = 8;
constexpr size_t EXPAND_BYTES = (size_t)8 << 30;  // most memory for the keys (and as much for the values) of a step's context

int window_row(const KxLatentSpec &s) { return kx_pad(s.kv_rank + s.rot_dim, 32); }

// element d of a vector whose first `rot` elements are rotated
template <class F>
__device__ __forceinline__ float turned(const KxLatentSpec &s, const float2 *turn, int d, F &&x) {
  const int half = s.rot / 2;
  if (d >= 2 * half) return x(d);
  const float2 t = turn[d < half ? d : d - half];
  return d < half ? x(d) * t.x - x(d + half) * t.y : x(d) * t.x + x(d - half) * t.y;
}

// the cache row of token `tok`; the whole workgroup of 256
template <class T>
__device__ __forceinline__ void cache_row(const KxLatentArgs &a, int tok, float *red) {
  const KxLatentSpec &s = a.s;
  const int i = tok / a.batch, b = tok - i * a.batch, p = a.pos + i, ld = kx_pad(s.kv_rank + s.rot_dim, KX_LD);
  const float *kv = a.proj + (size_t)tok * a.proj_ld + a.kv_off;
  float v = 0.0f;
  for (int c = threadIdx.x; c < s.kv_rank; c += 256) v = __builtin_fmaf(kv[c], kv[c], v);
  const float sc = kx_rsqrtf(kxr::block_sum(v, red) / (float)s.kv_rank + a.eps);
  const float2 *turn = a.turns + (size_t)p * (s.rot / 2);
  T *row = (T *)a.rows + ((size_t)b * a.cap + p) * ld;
  for (int c = threadIdx.x; c < ld; c += 256) {
    const int d = c - s.kv_rank;
    row[c] = Elem<T>::make(d < 0 ? kv[c] * sc * a.kv_norm[c] : d < s.rot_dim ? turned(s, turn, d, [&](int x) { return kv[s.kv_rank + x]; }) : 0.0f);
  }
}

// blockIdx.x: (head, ABS_COLS columns of the latent), and at the end one workgroup for the token's cache row
template <class T>
__global__ void __launch_bounds__(256) absorb_k(KxLatentArgs a, int row) {
  extern __shared__ float ab_q[];  // [dim]
  __shared__ float red[16][ABS_COLS + 4];
  const KxLatentSpec &s = a.s;
  const int tok = blockIdx.y, tid = threadIdx.x, slices = (s.kv_rank + ABS_COLS - 1) / ABS_COLS;
  if ((int)blockIdx.x == s.heads * slices) {
    cache_row<T>(a, tok, &red[0][0]);
    return;
  }
  const int h = blockIdx.x / slices, c0 = (blockIdx.x - h * slices) * ABS_COLS, p = tid & 15, ds = tid >> 4;
  const float *q = a.q + (size_t)tok * a.q_ld + h * (s.dim + s.rot_dim);
  float *out = a.x.q + ((size_t)tok * s.heads + h) * row;
  for (int d = tid; d < s.dim; d += 256) ab_q[d] = q[d];
  if (c0 == 0) {
    const float2 *turn = a.turns + (size_t)(a.pos + tok / a.batch) * (s.rot / 2);
    for (int c = s.kv_rank + tid; c < row; c += 256) {
      const int d = c - s.kv_rank;
      out[c] = d < s.rot_dim ? turned(s, turn, d, [&](int x) { return q[s.dim + x]; }) : 0.0f;
    }
  }
  __syncthreads();
  float acc[8] = {};
  const int col = min(c0 + p * 8, a.uk.ld - 8);
  const T *w = (const T *)a.uk.w + (size_t)h * s.dim * a.uk.ld + col;
#pragma unroll 8
  for (int d = ds; d < s.dim; d += 16) {
    float f[8];
    Elem<T>::unpack(f, Elem<T>::cached(w + (size_t)d * a.uk.ld));
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = __builtin_fmaf(ab_q[d], f[e], acc[e]);
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) red[ds][p * 8 + e] = acc[e];
  __syncthreads();
  for (int c = tid; c < ABS_COLS && c0 + c < s.kv_rank; c += 256) {
    float v = red[0][c];
#pragma unroll
    for (int j = 1; j < 16; ++j) v += red[j][c];
    out[c0 + c] = v;
  }
}

// the parts of one head of one token merged with the sink, OUT_ROWS rows of its W_uv, the gate
template <class T>
__global__ void __launch_bounds__(256) latent_out_k(KxLatentArgs a, KxWindowParts w, int tok0, int vp) {
  using E = Elem<T>;
  extern __shared__ float lo_lds[];
  const KxLatentSpec &s = a.s;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, slices = (s.vdim + OUT_ROWS - 1) / OUT_ROWS;
  const int h = blockIdx.x / slices, v0 = (blockIdx.x - h * slices) * OUT_ROWS, tok = tok0 + blockIdx.y, ld = a.uv.ld;
  float *lat = lo_lds, *weight = lat + ld;  // [ld], [parts]
  const size_t row = (size_t)blockIdx.y * w.parts;
  if (wave == 0) {
    const float sink = a.sinks ? a.sinks[h] : 0.0f;
    float m = s.sink ? sink : -__builtin_inff(), z = 0.0f;
    for (int k = lane; k < w.parts; k += 64) m = fmaxf(m, w.m[(row + k) * s.heads + h]);
    m = kxw::wave_max_f32(m);
    for (int k = lane; k < w.parts; k += 64) {
      const float y = kx_expf(w.m[(row + k) * s.heads + h] - m);
      weight[k] = y;
      z = __builtin_fmaf(w.z[(row + k) * s.heads + h], y, z);
    }
    const float inv = 1.0f / (kxr::wave_sum(z) + (s.sink ? kx_expf(sink - m) : 0.0f));
    for (int k = lane; k < w.parts; k += 64) weight[k] *= inv;
  }
  __syncthreads();
  for (int c = tid; c < ld; c += 256) {
    float v = 0.0f;
    if (c < s.kv_rank) {
#pragma unroll 8
      for (int k = 0; k < w.parts; ++k) {  // a part without keys has not written its sums
        const float x = w.o[((row + k) * s.heads + h) * vp + c];
        v = weight[k] > 0.0f ? __builtin_fmaf(x, weight[k], v) : v;
      }
    }
    lat[c] = v;
  }
  __syncthreads();
  constexpr int RW = OUT_ROWS / 4;  // rows per wave
  float acc[RW] = {};
  for (int x = lane * 8; x < ld; x += 512) {
    float l[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) l[e] = lat[x + e];
#pragma unroll
    for (int r = 0; r < RW; ++r) {
      float f[8];
      E::unpack(f, E::cached((const T *)a.uv.w + (size_t)(h * s.vdim + min(v0 + wave * RW + r, s.vdim - 1)) * ld + x));
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[r] = __builtin_fmaf(f[e], l[e], acc[r]);
    }
  }
  T *out = (T *)a.out + (size_t)tok * a.out_ld + h * s.vdim;
#pragma unroll
  for (int r = 0; r < RW; ++r) {
    const int d = v0 + wave * RW + r;
    const float y = kxr::wave_sum(acc[r]);
    if (lane == 0 && d < s.vdim) out[d] = E::make(y * (a.g_off >= 0 ? kx_sigmoidf(a.proj[(size_t)tok * a.proj_ld + a.g_off + h * s.vdim + d]) : 1.0f));
  }
}

// a token's queries, rotated, and its cache row
template <class T>
__global__ void __launch_bounds__(256) prep_k(KxLatentArgs a, int dp) {
  __shared__ float red[4];
  const KxLatentSpec &s = a.s;
  const int tok = blockIdx.x, w = s.dim + s.rot_dim;
  const float *q = a.q + (size_t)tok * a.q_ld;
  const float2 *turn = a.turns + (size_t)(a.pos + tok / a.batch) * (s.rot / 2);
  T *out = (T *)a.x.qx + (size_t)tok * s.heads * dp;
  for (int x = threadIdx.x; x < s.heads * dp; x += 256) {
    const int h = x / dp, d = x - h * dp;
    const float *qh = q + h * w;
    out[x] = Elem<T>::make(d < s.dim ? qh[d] : d < w ? turned(s, turn, d - s.dim, [&](int y) { return qh[s.dim + y]; }) : 0.0f);
  }
  cache_row<T>(a, tok, red);
}

// the shared key part behind every head's own keys, positions [0, n) of sequence blockIdx.y
template <class T>
__global__ void __launch_bounds__(256) share_k(KxLatentArgs a, int n, int cap, int dp) {
  const KxLatentSpec &s = a.s;
  const int ld = kx_pad(s.kv_rank + s.rot_dim, KX_LD), per = dp - s.dim, b = blockIdx.y;
  const size_t total = (size_t)n * s.heads * per;
  for (size_t x = (size_t)blockIdx.x * 256 + threadIdx.x; x < total; x += (size_t)gridDim.x * 256) {
    const int d = (int)(x % per), h = (int)(x / per % s.heads), p = (int)(x / per / s.heads);
    const T v = d < s.rot_dim ? ((const T *)a.rows)[((size_t)b * a.cap + p) * ld + s.kv_rank + d] : Elem<T>::make(0.0f);
    ((T *)a.x.kx)[(((size_t)b * s.heads + h) * cap + p) * dp + s.dim + d] = v;
  }
}

template <class T>
int few(const KxLatentArgs &a, hipStream_t st) {
  const KxLatentSpec &s = a.s;
  const int tokens = a.batch * a.positions, row = window_row(s);
  KX_REQUIRE(tokens <= a.x.q_tokens, "latent attention: %d tokens, room for %d", tokens, a.x.q_tokens);
  hipLaunchKernelGGL(absorb_k<T>, dim3(s.heads * kx_cdiv(s.kv_rank, ABS_COLS) + 1, tokens), dim3(256), (size_t)s.dim * 4, st, a, row);
  KX_LAUNCH_CHECK();
  KxWindowArgs w;
  w.s.heads = s.heads; w.s.dim = s.kv_rank + s.rot_dim; w.s.vdim = s.kv_rank; w.s.scale = s.scale; w.s.sink = s.sink;
  int group = std::min(HEAD_GROUP, s.heads);
  while (s.heads % group) --group;
  w.s.kv_heads = s.heads / group;
  w.c.k = w.c.v = a.rows; w.c.cap = a.cap; w.c.dp = row; w.c.vp = kx_pad(s.kv_rank, 32);
  w.c.k_ld = w.c.v_ld = kx_latent_row(s);
  w.c.shared = true;
  w.q_f32 = a.x.q;
  w.batch = a.batch; w.positions = a.positions; w.pos = a.pos;
  w.part = a.x.part; w.part_floats = a.x.part_floats;
  KxWindowParts p;
  for (int t0 = 0; t0 < tokens; t0 += p.n) {
    int rc = kx_window_parts_launch(sizeof(T) == 4, w, t0, tokens - t0, &p, st);
    if (rc) return rc;
    const size_t lds = ((size_t)a.uv.ld + p.parts) * 4;
    KX_REQUIRE(lds <= 64 * 1024, "latent attention: %d parts of %d columns", p.parts, s.kv_rank);
    hipLaunchKernelGGL(latent_out_k<T>, dim3(s.heads * kx_cdiv(s.vdim, OUT_ROWS), p.n), dim3(256), lds, st, a, p, t0, w.c.vp);
    KX_LAUNCH_CHECK();
  }
  return KX_OK;
}

template <class T>
int expanded(const KxLatentArgs &a, hipStream_t st) {
  const KxLatentSpec &s = a.s;
  const int tokens = a.batch * a.positions, n = a.pos + a.positions, cap = kx_pad(n, 64), dp = kx_pad(s.dim + s.rot_dim, 32), vp = kx_pad(s.vdim, 32);
  hipLaunchKernelGGL(prep_k<T>, dim3(tokens), dim3(256), 0, st, a, dp);
  KX_LAUNCH_CHECK();
  for (int b = 0; b < a.batch; ++b)
    for (int value = 0; value < 2; ++value) {
      const int ld = value ? vp : dp;
      KxLinArgs g;
      g.m = value ? a.uv : a.uk;
      g.tokens = n;
      g.row.cols = s.kv_rank;
      g.row.x = (const T *)a.rows + (size_t)b * a.cap * kx_latent_row(s);
      g.row.x_ld = kx_latent_row(s);
      g.epi = KX_LIN_HEADS;
      g.mid = (T *)(value ? a.x.vx : a.x.kx) + (size_t)b * s.heads * cap * ld;
      g.mid_ld = ld;
      g.head_dim = value ? s.vdim : s.dim;
      g.head_stride = (size_t)cap * ld;
      int rc = kx_linear_launch(sizeof(T) == 4, g, nullptr, st);
      if (rc) return rc;
    }
  if (dp > s.dim) {
    const size_t total = (size_t)n * s.heads * (dp - s.dim);
    hipLaunchKernelGGL(share_k<T>, dim3((unsigned)std::min<size_t>((total + 255) / 256, 4096), a.batch), dim3(256), 0, st, a, n, cap, dp);
    KX_LAUNCH_CHECK();
  }
  KxWindowArgs w;
  w.s.heads = w.s.kv_heads = s.heads; w.s.dim = s.dim + s.rot_dim; w.s.vdim = s.vdim; w.s.scale = s.scale; w.s.sink = s.sink;
  w.c.k = a.x.kx; w.c.v = a.x.vx; w.c.cap = cap; w.c.dp = dp; w.c.vp = vp;
  w.proj = a.proj; w.proj_ld = a.proj_ld; w.g_off = a.g_off;
  w.sinks = a.sinks;
  w.batch = a.batch; w.positions = a.positions; w.pos = a.pos;
  w.out = a.out; w.out_ld = a.out_ld; w.q = a.x.qx; w.part = a.x.part; w.part_floats = a.x.part_floats;
  return kx_window_attend(sizeof(T) == 4, w, st);
}

template <class T>
int latent(const KxLatentArgs &a, hipStream_t st) {
  const KxLatentSpec &s = a.s;
  const size_t cap = kx_pad(a.pos + a.positions, 64), heads = (size_t)a.batch * s.heads;
  const bool fits = heads * cap * kx_pad(s.dim + s.rot_dim, 32) <= a.x.k_elems && heads * cap * kx_pad(s.vdim, 32) <= a.x.v_elems;
  if (a.positions > KX_LATENT_FEW && fits) return expanded<T>(a, st);
  const int at_once = std::max(1, a.x.q_tokens / a.batch);
  for (int i = 0; i < a.positions; i += at_once) {
    KxLatentArgs p = a;
    const size_t tok = (size_t)i * a.batch;
    p.pos = a.pos + i;
    p.positions = std::min(at_once, a.positions - i);
    p.proj = a.proj + tok * a.proj_ld;
    p.q = a.q + tok * a.q_ld;
    p.out = (T *)a.out + tok * a.out_ld;
    int rc = few<T>(p, st);
    if (rc) return rc;
  }
  return KX_OK;
}

}  // namespace

void kx_latent_scratch(const KxLatentSpec &s, int max_batch, int max_context, int step_tokens, KxLatentScratch *x, size_t *q_floats, size_t *qx_elems) {
  x->q_tokens = KX_LATENT_FEW * max_batch;
  *q_floats = (size_t)x->q_tokens * s.heads * window_row(s);
  *qx_elems = (size_t)step_tokens * s.heads * kx_pad(s.dim + s.rot_dim, 32);
  const size_t rows = (size_t)max_batch * s.heads * kx_pad(max_context, 64);
  x->k_elems = std::min(rows * kx_pad(s.dim + s.rot_dim, 32), EXPAND_BYTES / 2);
  x->v_elems = std::min(rows * kx_pad(s.vdim, 32), EXPAND_BYTES / 2);
  KxWindowSpec few, many;  // partials: of all heads against the latent, and of every head against its own keys
  few.heads = many.heads = many.kv_heads = s.heads; few.kv_heads = 1;
  few.vdim = s.kv_rank; many.vdim = s.vdim;
  x->part_floats = std::max(kx_window_part_floats(few, max_context, std::min(x->q_tokens, 64)),
                            kx_window_part_floats(many, max_context, std::min(std::max(max_batch, step_tokens), 64)));
}

void kx_latent_turns(const KxLatentSpec &s, int positions, float *out) {
  const int half = s.rot / 2;
  std::vector<double> f(half);
  for (int i = 0; i < half; ++i) f[i] = pow(s.base, -2.0 * i / s.rot);
  for (int p = 0; p < positions; ++p)
    for (int i = 0; i < half; ++i) {
      out[((size_t)p * half + i) * 2] = (float)cos(p * f[i]);
      out[((size_t)p * half + i) * 2 + 1] = (float)sin(p * f[i]);
    }
}

int kx_latent_launch(bool f32, const KxLatentArgs &a, hipStream_t st) {
  const KxLatentSpec &s = a.s;
  KX_REQUIRE(s.heads > 0 && s.dim > 0 && s.rot_dim >= 0 && s.vdim > 0 && s.kv_rank > 0 && s.rot >= 0 && s.rot <= s.rot_dim && s.rot % 2 == 0,
             "latent attention: heads=%d dim=%d rot_dim=%d (%d rotated) vdim=%d kv_rank=%d", s.heads, s.dim, s.rot_dim, s.rot, s.vdim, s.kv_rank);
  KX_REQUIRE(a.uk.rows == s.heads * s.dim && a.uv.rows == s.heads * s.vdim && a.uk.cols == s.kv_rank && a.uv.cols == s.kv_rank, "latent attention: matrices of %d and %d rows",
             a.uk.rows, a.uv.rows);
  KX_REQUIRE(a.batch > 0 && a.positions > 0 && a.pos >= 0 && a.pos <= a.cap - a.positions, "latent attention: %d positions at %d of %d", a.positions, a.pos, a.cap);
  return f32 ? latent<float>(a, st) : latent<uint16_t>(a, st);
}
