// kx_latent.hip -- see kx_latent.h.
//
// The counterpart of the reference's multi-head latent attention (src/kimi_exec.cu:355-475, :677-716) for any sizes, with
// a sink and an output gate; kx_mla.hip is the same for Kimi-K2's.
//
// Few positions: W_uk is applied to the query (absorb_k, which also writes the cache rows), so that all heads attend to the
// cached rows themselves: latent_part_k takes tiles of them into LDS once for a group of heads, keys and, in their first
// columns, values; latent_out_k merges the parts, applies W_uv and the gate.
// Longer steps: prep_k writes queries and cache rows, two products make the keys and values of every position up to the
// step's last one, and kx_window.hip attends on the matrix cores.
#include <math.h>
#include <algorithm>
#include <atomic>
#include <vector>
#include "kx_common.h"
#include "kx_latent.h"
#include "kx_lds_copy.h"
#include "kx_rows.h"

namespace {

using kxr::Elem;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int ABS_COLS = 128, OUT_ROWS = 32;
constexpr int GROUP = 8, KEYS = 64;             // heads of a workgroup of latent_part_k, keys of a tile
constexpr int MAX_PARTS = 1024;
constexpr size_t PART_LDS = 78 * 1024;  // two workgroups per CU, where a tile of 16 keys allows
constexpr size_t MOST_LDS = 158 * 1024;
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

struct Parts {
  int n, parts, per, keys;  // tokens of the launch; parts per token, tiles per part, keys per tile
  float *o, *m, *z;         // [n][parts][heads][vp] sums, [n][parts][heads] maxima, denominators
};

// Part blockIdx.x of the keys of token tok0 + blockIdx.z for the heads of group blockIdx.y: p.per tiles of p.keys keys.  A
// tile's rows go from memory to LDS whole, the 16-byte pieces of row r at place piece ^ (r % 8), so that lanes on
// neighbouring rows read different banks.  A lane scores a key (f32) or four keys of a head on the matrix cores (bf16);
// then a thread owns 2 NC columns of all heads' sums.
template <class T, int NC>
__global__ void __launch_bounds__(256) latent_part_k(KxLatentArgs a, Parts p, int tok0, int row, int vp) {
  constexpr int PE = 16 / sizeof(T);  // elements per piece
  constexpr bool MC = sizeof(T) == 2;
  extern __shared__ __attribute__((aligned(16))) uint8_t lp_lds[];
  const KxLatentSpec &s = a.s;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int tok = tok0 + blockIdx.z, i = tok / a.batch, b = tok - i * a.batch, total = a.pos + i + 1;
  const int ld = kx_pad(s.kv_rank + s.rot_dim, KX_LD), pieces = ld / PE, qs_ld = row + 8, h0 = blockIdx.y * GROUP, heads = min(GROUP, s.heads - h0);
  T *tile = (T *)lp_lds;                                       // [keys][ld]
  T *qs = tile + (size_t)p.keys * ld;                          // [GROUP][row + 8]
  float *sc = (float *)(qs + (size_t)GROUP * qs_ld), *st_m = sc + GROUP * KEYS, *st_a = st_m + GROUP;
  const size_t out0 = ((size_t)blockIdx.z * p.parts + blockIdx.x) * s.heads + h0;
  const int first = blockIdx.x * p.per * p.keys;
  if (first >= total) {  // fewer keys than the launch's largest token has
    if (tid < heads) {
      p.m[out0 + tid] = -__builtin_inff();
      p.z[out0 + tid] = 0.0f;
    }
    return;
  }
  const uint32_t lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) uint8_t *)lp_lds;
  const T *rows = (const T *)a.rows + (size_t)b * a.cap * ld;
  const float *q = a.x.q + ((size_t)tok * s.heads + h0) * row;
  float acc[NC * 2][GROUP] = {};
  float m[2] = {-__builtin_inff(), -__builtin_inff()}, z[2] = {0.0f, 0.0f};  // of heads wave, wave + 4
  for (int t = 0; t < p.per; ++t) {
    const int k0 = first + t * p.keys, n = min(p.keys, total - k0);
    if (n <= 0) break;
    if (t) __syncthreads();  // the tile before is done with
    for (int x = wave * 64; x < p.keys * pieces; x += 256) {
      const int at = x + lane, r = at / pieces, c = at - r * pieces;
      kx_copy16_to_lds(rows + (size_t)(k0 + min(r, n - 1)) * ld + (c ^ (r & 7)) * PE, __builtin_amdgcn_readfirstlane(lds0 + x * 16));
    }
    if (t == 0)
#pragma unroll 5
      for (int x = tid; x < GROUP * row / 4; x += 256) {  // heads lie one after the other
        const int r = 4 * x / row, d = 4 * x - r * row;
        const f32x4 y = *(const f32x4 *)(q + 4 * min(x, heads * row / 4 - 1));
#pragma unroll
        for (int e = 0; e < 4; ++e) qs[r * qs_ld + d + e] = Elem<T>::make(r < heads ? y[e] : 0.0f);
      }
    kx_wait_copies<0>();
    __syncthreads();
    if constexpr (MC) {
      const int lk = lane & 15, g = lane >> 4;
      for (int kb = wave * 16; kb < p.keys; kb += 64) {
        f32x4 d[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}};
        const T *kr = tile + (size_t)(kb + lk) * ld;
        int x = 0;
        for (; x + 64 <= row; x += 64)
#pragma unroll
          for (int y = 0; y < 2; ++y) {
            const bf16x8 kf = *(const bf16x8 *)(kr + ((x / 8 + 4 * y + g) ^ (lk & 7)) * 8), qf = *(const bf16x8 *)(qs + (lk & 7) * qs_ld + x + 32 * y + 8 * g);
            d[y] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, d[y], 0, 0, 0);
          }
        if (x < row) {
          const bf16x8 kf = *(const bf16x8 *)(kr + ((x / 8 + g) ^ (lk & 7)) * 8), qf = *(const bf16x8 *)(qs + (lk & 7) * qs_ld + x + 8 * g);
          d[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, d[0], 0, 0, 0);
        }
        if (lk < GROUP) *(f32x4 *)(sc + lk * KEYS + kb + 4 * g) = (d[0] + d[1]) * s.scale;
      }
    } else {
      float d[2] = {};
      const T *kr = tile + (size_t)min(lane, p.keys - 1) * ld;
      for (int x = 0; x < row; x += 4) {
        const f32x4 kf = *(const f32x4 *)(kr + ((x / 4) ^ (lane & 7)) * 4);
#pragma unroll
        for (int y = 0; y < 2; ++y) {
          const f32x4 qf = *(const f32x4 *)(qs + (wave + 4 * y) * qs_ld + x);
#pragma unroll
          for (int e = 0; e < 4; ++e) d[y] = __builtin_fmaf(kf[e], qf[e], d[y]);
        }
      }
      if (lane < p.keys)
#pragma unroll
        for (int y = 0; y < 2; ++y) sc[(wave + 4 * y) * KEYS + lane] = d[y] * s.scale;
    }
    __syncthreads();
#pragma unroll
    for (int y = 0; y < 2; ++y) {
      const int h = wave + 4 * y;
      const float v = lane < n ? sc[h * KEYS + lane] : -__builtin_inff(), m1 = fmaxf(m[y], kxw::wave_max_f32(v)), al = kx_expf(m[y] - m1);
      const float e = lane < n ? kx_expf(v - m1) : 0.0f;
      sc[h * KEYS + lane] = e;
      z[y] = z[y] * al + kxr::wave_sum(e);
      m[y] = m1;
      if (lane == 0) st_a[h] = al;
    }
    __syncthreads();
    float al[GROUP];
#pragma unroll
    for (int h = 0; h < GROUP; ++h) al[h] = t ? st_a[h] : 1.0f;
#pragma unroll
    for (int c = 0; c < NC * 2; ++c)
#pragma unroll
      for (int h = 0; h < GROUP; ++h) acc[c][h] *= al[h];
    for (int k = 0; k < n; k += 4) {
      f32x4 wt[GROUP];
#pragma unroll
      for (int h = 0; h < GROUP; ++h) wt[h] = *(const f32x4 *)(sc + h * KEYS + k);
#pragma unroll
      for (int kk = 0; kk < 4; ++kk) {
        const T *kr = tile + (size_t)min(k + kk, p.keys - 1) * ld;
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          const int col = c * 512 + tid * 2;
          float v0 = 0.0f, v1 = 0.0f;
          if (col < vp) {
            const T *x = kr + ((col / PE) ^ ((k + kk) & 7)) * PE + col % PE;
            if constexpr (MC) {
              const uint32_t two = *(const uint32_t *)x;
              v0 = kx_bits_f32(two << 16);
              v1 = kx_bits_f32(two & 0xffff0000u);
            } else {
              v0 = x[0];
              v1 = x[1];
            }
          }
#pragma unroll
          for (int h = 0; h < GROUP; ++h) {
            acc[2 * c][h] = __builtin_fmaf(wt[h][kk], v0, acc[2 * c][h]);
            acc[2 * c + 1][h] = __builtin_fmaf(wt[h][kk], v1, acc[2 * c + 1][h]);
          }
        }
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int col = c * 512 + tid * 2;
    if (col < vp)
#pragma unroll
      for (int h = 0; h < GROUP; ++h)
        if (h < heads) *(float2 *)(p.o + (out0 + h) * vp + col) = make_float2(acc[2 * c][h], acc[2 * c + 1][h]);
  }
#pragma unroll
  for (int y = 0; y < 2; ++y)
    if (lane == 0 && wave + 4 * y < heads) {
      p.m[out0 + wave + 4 * y] = m[y];
      p.z[out0 + wave + 4 * y] = z[y];
    }
}

// the parts of one head of one token merged with the sink, OUT_ROWS rows of its W_uv, the gate
constexpr int OUT_THREADS = 512, OUT_AHEAD = 20;  // OUT_AHEAD: a thread's parts that are asked for before the weights are known
template <class T>
__global__ void __launch_bounds__(OUT_THREADS) latent_out_k(KxLatentArgs a, Parts w, int tok0, int vp) {
  using E = Elem<T>;
  extern __shared__ __attribute__((aligned(16))) float lo_lds[];
  const KxLatentSpec &s = a.s;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, slices = (s.vdim + OUT_ROWS - 1) / OUT_ROWS;
  const int h = blockIdx.x / slices, v0 = (blockIdx.x - h * slices) * OUT_ROWS, tok = tok0 + blockIdx.y, ld = a.uv.ld;
  float *lat = lo_lds, *sum = lat + ld, *weight = sum + 4 * ld, *den = weight + w.parts;  // [ld], [4][ld], [parts], [parts]
  const size_t row = (size_t)blockIdx.y * w.parts;
  // four columns per thread; where fewer threads hold them all, the others take parts of their own
  const int quads = vp / 4, shares = quads <= OUT_THREADS / 4 ? 4 : quads <= OUT_THREADS / 2 ? 2 : 1, per = OUT_THREADS / shares, share = tid / per, tq = tid - share * per;
  const float *po = w.o + (row * s.heads + h) * vp;
  auto part = [&](int k, int x) { return *(const f32x4 *)(po + (size_t)min(k, w.parts - 1) * s.heads * vp + 4 * min(x, quads - 1)); };
  f32x4 y[OUT_AHEAD];
#pragma unroll
  for (int j = 0; j < OUT_AHEAD; ++j) y[j] = part(share + j * shares, tq);
  constexpr int RW = OUT_ROWS / (OUT_THREADS / 64);  // rows per wave
  typename E::Raw uv[RW];
  float gate[RW];
#pragma unroll
  for (int r = 0; r < RW; ++r) {
    const int d = min(v0 + wave * RW + r, s.vdim - 1);
    uv[r] = E::cached((const T *)a.uv.w + (size_t)(h * s.vdim + d) * ld + min(lane * 8, ld - 8));
    gate[r] = a.g_off >= 0 ? a.proj[(size_t)tok * a.proj_ld + a.g_off + h * s.vdim + d] : 0.0f;
  }
  if (wave == 0) {
    const float sink = a.sinks ? a.sinks[h] : 0.0f;
    float m = s.sink ? sink : -__builtin_inff(), z = 0.0f;
    for (int k = lane; k < w.parts; k += 64) {
      const float mk = w.m[(row + k) * s.heads + h];
      den[k] = w.z[(row + k) * s.heads + h];
      weight[k] = mk;
      m = fmaxf(m, mk);
    }
    m = kxw::wave_max_f32(m);
    for (int k = lane; k < w.parts; k += 64) {
      const float e = kx_expf(weight[k] - m);
      weight[k] = e;
      z = __builtin_fmaf(den[k], e, z);
    }
    const float inv = 1.0f / (kxr::wave_sum(z) + (s.sink ? kx_expf(sink - m) : 0.0f));
    for (int k = lane; k < w.parts; k += 64) weight[k] *= inv;
  }
  __syncthreads();
  for (int x = tq; x < quads; x += per) {
    f32x4 v = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int k0 = share; k0 < w.parts; k0 += OUT_AHEAD * shares) {
      if (x != tq || k0 != share)
#pragma unroll
        for (int j = 0; j < OUT_AHEAD; ++j) y[j] = part(k0 + j * shares, x);
#pragma unroll
      for (int j = 0; j < OUT_AHEAD; ++j) {
        const int k = k0 + j * shares;
        const float wt = k < w.parts ? weight[k] : 0.0f;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = wt > 0.0f ? __builtin_fmaf(y[j][e], wt, v[e]) : v[e];  // a part without keys has not written its sums
      }
    }
    *(f32x4 *)(sum + share * ld + 4 * x) = v;
  }
  __syncthreads();
  for (int c = tid; c < ld; c += OUT_THREADS) {
    float v = 0.0f;
    if (c < s.kv_rank)
      for (int j = 0; j < shares; ++j) v += sum[j * ld + c];
    lat[c] = v;
  }
  __syncthreads();
  float acc[RW] = {};
  for (int x = lane * 8; x < ld; x += 512) {
    float l[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) l[e] = lat[x + e];
#pragma unroll
    for (int r = 0; r < RW; ++r) {
      float f[8];
      if (x >= 512) uv[r] = E::cached((const T *)a.uv.w + (size_t)(h * s.vdim + min(v0 + wave * RW + r, s.vdim - 1)) * ld + x);
      E::unpack(f, uv[r]);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[r] = __builtin_fmaf(f[e], l[e], acc[r]);
    }
  }
  T *out = (T *)a.out + (size_t)tok * a.out_ld + h * s.vdim;
#pragma unroll
  for (int r = 0; r < RW; ++r) {
    const int d = v0 + wave * RW + r;
    const float o = kxr::wave_sum(acc[r]);
    if (lane == 0 && d < s.vdim) out[d] = E::make(a.g_off >= 0 ? o * kx_sigmoidf(gate[r]) : o);
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

// LDS of latent_part_k without its tile, and keys of the tile that fits beside it
template <class T>
size_t part_lds(int row) { return (size_t)GROUP * (row + 8) * sizeof(T) + (GROUP * KEYS + 2 * GROUP) * 4; }
template <class T>
int part_keys(const KxLatentSpec &s) {
  int keys = KEYS;
  while (keys > 16 && (size_t)keys * kx_latent_row(s) * sizeof(T) + part_lds<T>(window_row(s)) > PART_LDS) keys >>= 1;  // 16: as the matrix cores take them
  return keys;
}
// Parts of a step whose last token sees `total` keys: whole tiles, and no more workgroups than run at once as long as a
// part has few tiles.
template <class T>
void plan_parts(const KxLatentSpec &s, int total, int tokens, Parts &p) {
  p.keys = part_keys<T>(s);
  const int tiles = kx_cdiv(total, p.keys), at_once = std::max(1, 2 * kx_device_cus());
  p.per = std::max(1, (int)((long)tiles * kx_cdiv(s.heads, GROUP) * tokens / at_once));
  p.parts = kx_cdiv(tiles, p.per);
  while (p.parts > MAX_PARTS) p.parts = kx_cdiv(tiles, ++p.per);
}
size_t part_room(const KxLatentSpec &s) { return (size_t)s.heads * (kx_pad(s.kv_rank, 32) + 2); }

template <class T, int NC>
int parts_launch(const KxLatentArgs &a, const Parts &p, int tok0, int row, int vp, hipStream_t st) {
  static std::atomic<bool> attr{false};
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)latent_part_k<T, NC>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)MOST_LDS));
    attr = true;
  }
  const size_t lds = (size_t)p.keys * kx_latent_row(a.s) * sizeof(T) + part_lds<T>(row);
  KX_REQUIRE(lds <= MOST_LDS, "latent attention: cached rows of %d columns do not fit a workgroup", kx_latent_row(a.s));
  hipLaunchKernelGGL((latent_part_k<T, NC>), dim3(p.parts, kx_cdiv(a.s.heads, GROUP), p.n), dim3(256), lds, st, a, p, tok0, row, vp);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

template <class T>
int few(const KxLatentArgs &a, hipStream_t st) {
  const KxLatentSpec &s = a.s;
  const int tokens = a.batch * a.positions, row = window_row(s), vp = kx_pad(s.kv_rank, 32);
  KX_REQUIRE(tokens <= a.x.q_tokens, "latent attention: %d tokens, room for %d", tokens, a.x.q_tokens);
  hipLaunchKernelGGL(absorb_k<T>, dim3(s.heads * kx_cdiv(s.kv_rank, ABS_COLS) + 1, tokens), dim3(256), (size_t)s.dim * 4, st, a, row);
  KX_LAUNCH_CHECK();
  Parts p;
  for (int t0 = 0; t0 < tokens; t0 += p.n) {
    plan_parts<T>(s, a.pos + a.positions, tokens - t0, p);
    const size_t per_token = p.parts * part_room(s);
    KX_REQUIRE(per_token <= a.x.part_floats, "latent attention: %zu floats of partials, room for %zu", per_token, a.x.part_floats);
    p.n = (int)std::min<size_t>({(size_t)(tokens - t0), a.x.part_floats / per_token, (size_t)65535});
    p.o = a.x.part;
    p.m = p.o + (size_t)p.n * p.parts * s.heads * vp;
    p.z = p.m + (size_t)p.n * p.parts * s.heads;
    int rc = vp <= 512 ? parts_launch<T, 1>(a, p, t0, row, vp, st) : vp <= 1024 ? parts_launch<T, 2>(a, p, t0, row, vp, st) : parts_launch<T, 4>(a, p, t0, row, vp, st);
    if (rc) return rc;
    const size_t lds = ((size_t)5 * a.uv.ld + 2 * p.parts) * 4;
    KX_REQUIRE(lds <= 64 * 1024, "latent attention: %d parts of %d columns", p.parts, s.kv_rank);
    hipLaunchKernelGGL(latent_out_k<T>, dim3(s.heads * kx_cdiv(s.vdim, OUT_ROWS), p.n), dim3(OUT_THREADS), lds, st, a, p, t0, vp);
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
  KxWindowSpec own;  // partials: of all heads against the latent , and of every head against its own keys
  own.heads = own.kv_heads = s.heads; own.vdim = s.vdim;
  const size_t parts = std::min(kx_cdiv(max_context, 8), MAX_PARTS);
  x->part_floats = std::max(parts * part_room(s) * std::min(x->q_tokens, 4), kx_window_part_floats(own, max_context, std::min(std::max(max_batch, step_tokens), 64)));
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
