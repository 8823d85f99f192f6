// kx_window.hip -- see kx_window.h.
//
// The counterpart of the tiled attention over cached keys and values (attn_tile_* and tiled_attention,
// src/kimi_exec.cu:414-475, :692-716) for a window with pooled blocks; the scores and the softmax are 32-bit.
//
// One token per sequence: win_partial_k<T, true>.  A workgroup takes up to CH keys of one key/value head for one token:
// it norms the query itself, and the workgroup that holds the newest key also norms that key, writes the cache rows
// and, where a block completes, its means.  win_merge_k merges the parts, adds the sink and applies the output gate.
// Steps of several positions: win_prep_k norms the projections and writes queries and cache rows, win_pool_k the
// blocks that complete, and then win_flash_k (bf16; matrix cores) or win_partial_k<T, false> + win_merge_k (f32) attend.
#include <algorithm>
#include <atomic>
#include "kx_common.h"
#include "kx_rows.h"
#include "kx_window.h"

namespace {

using kxr::Elem;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
typedef float f32x2 __attribute__((ext_vector_type(2)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));

constexpr float NEG_INF = -__builtin_inff();
constexpr int RB = 4;            // query heads whose values are summed together in win_partial_k
constexpr int PART_THREADS = 256;

__host__ __device__ __forceinline__ int seen_blocks(int p, int size, int pool) {
  return pool > 0 && p - size + 1 > 0 ? (p - size + 1) / pool : 0;
}
__host__ __device__ __forceinline__ int window_lo(int p, int size) { return p - size + 1 > 0 ? p - size + 1 : 0; }

// mean of block b of one head into the pooled rows; the whole workgroup
template <class T>
__device__ __forceinline__ void pool_block(const KxWindowArgs &a, size_t head, int b, int tid, int n) {
  const KxWindowCache &c = a.c;
  const float inv = 1.0f / (float)a.s.pool;
  for (int x = tid; x < c.dp + c.vp; x += n) {
    const bool key = x < c.dp;
    const int col = key ? x : x - c.dp, w = key ? c.dp : c.vp;
    const T *src = (const T *)(key ? c.k : c.v) + head * c.cap * w + col;
    float sum = 0.0f;
    int slot = (int)((long)b * a.s.pool % c.cap);
    for (int j = 0; j < a.s.pool; ++j) {
      sum += Elem<T>::load(src + (size_t)slot * w);
      if (++slot == c.cap) slot = 0;
    }
    ((T *)(key ? c.pk : c.pv))[(head * c.blocks + b) * w + col] = Elem<T>::make(sum * inv);
  }
}

template <class T>
__global__ void __launch_bounds__(256) win_prep_k(KxWindowArgs a) {
  __shared__ float red[4];
  const KxWindowSpec &s = a.s;
  const KxWindowCache &c = a.c;
  const int tok = blockIdx.x, i = tok / a.batch, b = tok - i * a.batch, p = a.pos + i;
  const float *pr = a.proj + (size_t)tok * a.proj_ld;
  const int nq = s.heads * s.dim, nk = s.kv_heads * s.dim;
  float qs = 1.0f, ks = 1.0f;
  if (a.q_norm) {
    float v = 0.0f, w = 0.0f;
    for (int x = threadIdx.x; x < nq; x += 256) v = __builtin_fmaf(pr[a.q_off + x], pr[a.q_off + x], v);
    for (int x = threadIdx.x; x < nk; x += 256) w = __builtin_fmaf(pr[a.k_off + x], pr[a.k_off + x], w);
    qs = kx_rsqrtf(kxr::block_sum(v, red) / (float)nq + a.eps);
    ks = kx_rsqrtf(kxr::block_sum(w, red) / (float)nk + a.eps);
  }
  T *q = (T *)a.q + (size_t)tok * s.heads * c.dp;
  for (int x = threadIdx.x; x < s.heads * c.dp; x += 256) {
    const int h = x / c.dp, d = x - h * c.dp, y = h * s.dim + d;
    q[x] = Elem<T>::make(d < s.dim ? pr[a.q_off + y] * qs * (a.q_norm ? a.q_norm[y] : 1.0f) : 0.0f);
  }
  const int slot = p % c.cap;
  for (int x = threadIdx.x; x < s.kv_heads * c.dp; x += 256) {
    const int g = x / c.dp, d = x - g * c.dp, y = g * s.dim + d;
    ((T *)c.k)[((size_t)(b * s.kv_heads + g) * c.cap + slot) * c.dp + d] =
        Elem<T>::make(d < s.dim ? pr[a.k_off + y] * ks * (a.k_norm ? a.k_norm[y] : 1.0f) : 0.0f);
  }
  for (int x = threadIdx.x; x < s.kv_heads * c.vp; x += 256) {
    const int g = x / c.vp, d = x - g * c.vp;
    ((T *)c.v)[((size_t)(b * s.kv_heads + g) * c.cap + slot) * c.vp + d] = Elem<T>::make(d < s.vdim ? pr[a.v_off + g * s.vdim + d] : 0.0f);
  }
}

template <class T>
__global__ void __launch_bounds__(256) win_pool_k(KxWindowArgs a, int b0) {
  pool_block<T>(a, (size_t)blockIdx.z * a.s.kv_heads + blockIdx.y, b0 + blockIdx.x, threadIdx.x, 256);
}

// Part `blockIdx.x` of the keys of token tok0 + blockIdx.z for key/value head blockIdx.y: up to ch keys, blocks first.
// part: [tokens][parts][heads * vp] sums, then [tokens][parts][heads] maxima, then as many denominators.
template <class T, bool FUSED>
__global__ void __launch_bounds__(PART_THREADS) win_partial_k(KxWindowArgs a, int tok0, int ch, float *po, float *pm, float *pz) {
  using E = Elem<T>;
  extern __shared__ __attribute__((aligned(16))) float win_lds[];
  __shared__ float red[4];
  const KxWindowSpec &s = a.s;
  const KxWindowCache &c = a.c;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int tok = tok0 + blockIdx.z, i = tok / a.batch, b = tok - i * a.batch, p = a.pos + i;
  const int g = blockIdx.y, R = s.heads / s.kv_heads, parts = gridDim.x;
  const int nb = seen_blocks(p, s.size, s.pool), lo = window_lo(p, s.size), total = nb + p - lo + 1;
  const int e0 = blockIdx.x * ch, n = min(ch, total - e0);
  const size_t out0 = (size_t)blockIdx.z * parts + blockIdx.x;
  if (n <= 0) {  // fewer keys than the launch's largest token has
    for (int r = tid; r < R; r += PART_THREADS) {
      pm[out0 * s.heads + g * R + r] = NEG_INF;
      pz[out0 * s.heads + g * R + r] = 0.0f;
    }
    return;
  }
  float *qv = win_lds;                 // [R][dp]
  float *sc = qv + R * c.dp;           // [R][ch]
  float *sum = sc + R * ch;            // [groups][RB][vp]
  const size_t head = (size_t)b * s.kv_heads + g;
  const T *kc = (const T *)c.k + head * c.cap * c.dp, *vc = (const T *)c.v + head * c.cap * c.vp;
  const T *pkc = (const T *)c.pk + head * c.blocks * c.dp, *pvc = (const T *)c.pv + head * c.blocks * c.vp;
  if (FUSED) {
    const float *pr = a.proj + (size_t)tok * a.proj_ld;
    const int nq = s.heads * s.dim, nk = s.kv_heads * s.dim;
    float qs = 1.0f, ks = 1.0f;
    if (a.q_norm) {
      float v = 0.0f, w = 0.0f;
      for (int x = tid; x < nq; x += PART_THREADS) v = __builtin_fmaf(pr[a.q_off + x], pr[a.q_off + x], v);
      for (int x = tid; x < nk; x += PART_THREADS) w = __builtin_fmaf(pr[a.k_off + x], pr[a.k_off + x], w);
      qs = kx_rsqrtf(kxr::block_sum(v, red) / (float)nq + a.eps);
      ks = kx_rsqrtf(kxr::block_sum(w, red) / (float)nk + a.eps);
    }
    for (int x = tid; x < R * c.dp; x += PART_THREADS) {
      const int r = x / c.dp, d = x - r * c.dp, y = (g * R + r) * s.dim + d;
      float v = d < s.dim ? pr[a.q_off + y] * qs * (a.q_norm ? a.q_norm[y] : 1.0f) : 0.0f;
      if (sizeof(T) == 2) v = kx_bfround(v);  // the query the other kernels read
      qv[x] = v;
    }
    if (e0 + n == total) {  // this workgroup holds the newest key: it writes the cache
      const int slot = p % c.cap;
      for (int d = tid; d < c.dp; d += PART_THREADS) {
        const int y = g * s.dim + d;
        ((T *)c.k)[(head * c.cap + slot) * c.dp + d] = E::make(d < s.dim ? pr[a.k_off + y] * ks * (a.k_norm ? a.k_norm[y] : 1.0f) : 0.0f);
      }
      for (int d = tid; d < c.vp; d += PART_THREADS)
        ((T *)c.v)[(head * c.cap + slot) * c.vp + d] = E::make(d < s.vdim ? pr[a.v_off + g * s.vdim + d] : 0.0f);
      __threadfence_block();
      __syncthreads();
      if (s.pool > 0 && (p + 1) % s.pool == 0 && p / s.pool < c.blocks) pool_block<T>(a, head, p / s.pool, tid, PART_THREADS);
    }
  } else {
    const T *q = (const T *)a.q + ((size_t)tok * s.heads + g * R) * c.dp;
    for (int x = tid; x < R * c.dp; x += PART_THREADS) qv[x] = E::load(q + x);
  }
  __syncthreads();
  const int base = p / c.cap * c.cap;  // position j of the window: slot j - base, one ring length more below it
  auto slot_of = [&](int e) {
    const int j = lo + e - nb - base;
    return j < 0 ? j + c.cap : j;
  };
  // scores: 8 lanes per key
  const int l8 = lane & 7;
  for (int k0 = wave * 8; k0 < n; k0 += 32) {
    const int e = e0 + min(k0 + (lane >> 3), n - 1);
    const T *key = e < nb ? pkc + (size_t)e * c.dp : kc + (size_t)slot_of(e) * c.dp;
    for (int r0 = 0; r0 < R; r0 += RB) {
      float d[RB] = {};
      for (int x = l8 * 8; x < c.dp; x += 64) {
        float kf[8];
        E::unpack(kf, E::cached(key + x));
#pragma unroll
        for (int r = 0; r < RB; ++r) {
          const float *q = qv + min(r0 + r, R - 1) * c.dp + x;
          const float4 qa = *(const float4 *)q, qb = *(const float4 *)(q + 4);
          d[r] = __builtin_fmaf(kf[0], qa.x, d[r]); d[r] = __builtin_fmaf(kf[1], qa.y, d[r]);
          d[r] = __builtin_fmaf(kf[2], qa.z, d[r]); d[r] = __builtin_fmaf(kf[3], qa.w, d[r]);
          d[r] = __builtin_fmaf(kf[4], qb.x, d[r]); d[r] = __builtin_fmaf(kf[5], qb.y, d[r]);
          d[r] = __builtin_fmaf(kf[6], qb.z, d[r]); d[r] = __builtin_fmaf(kf[7], qb.w, d[r]);
        }
      }
#pragma unroll
      for (int r = 0; r < RB; ++r) {
        d[r] += kxw::dpp_f<kxw::DPP_QUAD_XOR1>(d[r]);
        d[r] += kxw::dpp_f<kxw::DPP_QUAD_XOR2>(d[r]);
        d[r] += kxw::dpp_f<kxw::DPP_ROW_HALF_MIRROR>(d[r]);
        if (l8 == 0 && r0 + r < R && k0 + (lane >> 3) < n) sc[(r0 + r) * ch + k0 + (lane >> 3)] = d[r] * s.scale;
      }
    }
  }
  __syncthreads();
  for (int r = wave; r < R; r += 4) {
    float m = NEG_INF, z = 0.0f;
    for (int k = lane; k < n; k += 64) m = fmaxf(m, sc[r * ch + k]);
    m = kxw::wave_max_f32(m);
    for (int k = lane; k < n; k += 64) {
      const float e = kx_expf(sc[r * ch + k] - m);
      sc[r * ch + k] = e;
      z += e;
    }
    z = kxr::wave_sum(z);
    if (lane == 0) {
      pm[out0 * s.heads + g * R + r] = m;
      pz[out0 * s.heads + g * R + r] = z;
    }
  }
  __syncthreads();
  // weighted values: vp / 8 threads per key
  const int tpk = c.vp >> 3, groups = PART_THREADS / tpk, grp = tid / tpk, col = (tid - grp * tpk) * 8;
  for (int r0 = 0; r0 < R; r0 += RB) {
    float acc[RB][8] = {};
    if (grp < groups)
      for (int k = grp; k < n; k += groups) {
        const int e = e0 + k;
        float vf[8];
        E::unpack(vf, E::cached((e < nb ? pvc + (size_t)e * c.vp : vc + (size_t)slot_of(e) * c.vp) + col));
#pragma unroll
        for (int r = 0; r < RB; ++r) {
          const float w = sc[min(r0 + r, R - 1) * ch + k];
#pragma unroll
          for (int x = 0; x < 8; ++x) acc[r][x] = __builtin_fmaf(w, vf[x], acc[r][x]);
        }
      }
    if (grp < groups)
#pragma unroll
      for (int r = 0; r < RB; ++r)
#pragma unroll
        for (int x = 0; x < 8; ++x) sum[(grp * RB + r) * c.vp + col + x] = acc[r][x];
    __syncthreads();
    for (int x = tid; x < RB * c.vp; x += PART_THREADS) {
      const int r = x / c.vp, d = x - r * c.vp;
      if (r0 + r >= R) continue;
      float v = sum[x];
      for (int y = 1; y < groups; ++y) v += sum[y * RB * c.vp + x];
      po[(out0 * s.heads + g * R + r0 + r) * c.vp + d] = v;
    }
    __syncthreads();
  }
}

// the parts of one head of one token merged, with the sink, times sigmoid(gate); one wave finds the parts' weights
constexpr int MERGE_THREADS = 128;
template <class T>
__global__ void __launch_bounds__(MERGE_THREADS) win_merge_k(KxWindowArgs a, int tok0, int parts, const float *po, const float *pm, const float *pz) {
  extern __shared__ float weight[];  // [parts]
  const KxWindowSpec &s = a.s;
  const int h = blockIdx.x, tok = tok0 + blockIdx.y, tid = threadIdx.x;
  const size_t row = (size_t)blockIdx.y * parts;
  if (tid < 64) {
    const float sink = a.sinks ? a.sinks[h] : 0.0f;
    float m = s.sink ? sink : NEG_INF, z = 0.0f;
    for (int k = tid; k < parts; k += 64) m = fmaxf(m, pm[(row + k) * s.heads + h]);
    m = kxw::wave_max_f32(m);
    for (int k = tid; k < parts; k += 64) {
      const float w = kx_expf(pm[(row + k) * s.heads + h] - m);
      weight[k] = w;
      z = __builtin_fmaf(pz[(row + k) * s.heads + h], w, z);
    }
    const float inv = 1.0f / (kxr::wave_sum(z) + (s.sink ? kx_expf(sink - m) : 0.0f));
    for (int k = tid; k < parts; k += 64) weight[k] *= inv;
  }
  __syncthreads();
  T *out = (T *)a.out + (size_t)tok * a.out_ld + h * s.vdim;
  for (int d = tid; d < s.vdim; d += MERGE_THREADS) {
    const float gate = a.g_off >= 0 ? kx_sigmoidf(a.proj[(size_t)tok * a.proj_ld + a.g_off + h * s.vdim + d]) : 1.0f;
    float v = 0.0f;
#pragma unroll 8
    for (int k = 0; k < parts; ++k) {  // a part without keys has not written its sums
      const float x = po[((row + k) * s.heads + h) * a.c.vp + d];
      v = weight[k] > 0.0f ? __builtin_fmaf(x, weight[k], v) : v;
    }
    out[d] = Elem<T>::make(v * gate);
  }
}

// ---- bf16, several positions: one head, 128 consecutive positions of one sequence, 4 waves of 32 queries ----
// S^T = K Q^T and O^T = V^T P^T, so that a lane holds one query (lane % 32) in both products: the running maximum and
// denominator are one value per lane, and the weights go from the first product's result into the second product's
// operand without leaving the registers.  The result layout gives lane (q, h) the keys 8 (v / 4) + 4 h + v % 4 of a tile of
// 32; the operand layout wants 8 keys in a row per lane, so within 16 keys the V^T tile stores keys 0-3, 8-11 for
// h = 0 and 4-7, 12-15 for h = 1.  The 8-key pieces of a V^T row are xor-swizzled by the row, which spreads the
// transposing writes over the banks.  The next tile's rows are on their way to registers while a tile is multiplied;
// scores are in units of log 2, so that a weight is one exp2.
constexpr int FQ = 128, FK = 64;
__device__ __forceinline__ int vt_piece(int d, int piece) { return (piece ^ (d >> 1) ^ (d >> 4)) & 7; }

template <int ND, int NV>  // 32-column blocks of a key and of a value
__global__ void __launch_bounds__(256) win_flash_k(KxWindowArgs a) {
  constexpr int KSTR = ND * 32 + 8, VSTR = FK + 8;
  extern __shared__ __attribute__((aligned(16))) uint16_t fl_lds[];
  uint16_t *ks = fl_lds;                // [FK][KSTR]
  uint16_t *vt = ks + FK * KSTR;        // [NV * 32][VSTR]
  const KxWindowSpec &s = a.s;
  const KxWindowCache &c = a.c;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 31, hh = lane >> 5;
  const int h = blockIdx.y, b = blockIdx.z, g = h / (s.heads / s.kv_heads);
  const int i0 = blockIdx.x * FQ, i = i0 + wave * 32 + lq;  // this lane's position of the step
  const bool live = i < a.positions;
  const int p = a.pos + min(i, a.positions - 1), tok = min(i, a.positions - 1) * a.batch + b;
  const int p_first = a.pos + i0, p_last = a.pos + min(i0 + FQ, a.positions) - 1;
  const int nb = seen_blocks(p, s.size, s.pool), lo = window_lo(p, s.size);
  const size_t head = (size_t)b * s.kv_heads + g;
  const uint16_t *kc = (const uint16_t *)c.k + head * c.cap * c.dp, *vc = (const uint16_t *)c.v + head * c.cap * c.vp;
  const uint16_t *pkc = (const uint16_t *)c.pk + head * c.blocks * c.dp, *pvc = (const uint16_t *)c.pv + head * c.blocks * c.vp;
  bf16x8 q[ND * 2];
  {
    const uint16_t *qr = (const uint16_t *)a.q + ((size_t)tok * s.heads + h) * c.dp;
#pragma unroll
    for (int kk = 0; kk < ND * 2; ++kk) q[kk] = kk * 16 < c.dp ? *(const bf16x8 *)(qr + kk * 16 + hh * 8) : bf16x8{};
  }
  f32x16 o[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j)
#pragma unroll
    for (int v = 0; v < 16; ++v) o[j][v] = 0.0f;
  float m = s.sink ? (a.sinks ? a.sinks[h] * 1.44269504088896341f : 0.0f) : NEG_INF, z = s.sink && hh == 0 ? 1.0f : 0.0f;  // z: this lane's half of the keys
  const float scale2 = s.scale * 1.44269504088896341f;

  // tiles: the blocks the last query sees, then the positions from the first query's window on
  const int tb = (seen_blocks(p_last, s.size, s.pool) + FK - 1) / FK;
  const int j0 = window_lo(p_first, s.size) & ~(FK - 1), tiles = tb + (p_last - j0) / FK + 1;
  // what all and what any of this wave's queries see
  const int q0 = __builtin_amdgcn_readfirstlane(a.pos + min(i0 + wave * 32, a.positions - 1));
  const int q1 = __builtin_amdgcn_readfirstlane(a.pos + min(i0 + wave * 32 + 31, a.positions - 1));
  const int nb0 = seen_blocks(q0, s.size, s.pool), nb1 = seen_blocks(q1, s.size, s.pool), lo0 = window_lo(q0, s.size), lo1 = window_lo(q1, s.size);
  auto first_key = [&](int t) { return t < tb ? t * FK : j0 + (t - tb) * FK; };
  constexpr int VT = (FK / 8) * NV * 16, VN = (VT + 255) / 256;  // V is taken by 8 keys x 2 columns
  u32x4 kreg[ND];
  uint32_t vreg[VN][8];
  // Rows of a tile: a window tile starts at a multiple of FK and the ring's length is one, so it does not wrap inside; past the
  // last block there is nothing to read.  What is read beyond a row's columns or the keys a query sees meets zeros.
  auto fetch = [&](int t) {
    const bool pooled = t < tb;
    const int k0 = first_key(t), last = pooled ? c.blocks - 1 - k0 : FK - 1;
    const uint16_t *kr = pooled ? pkc + (size_t)k0 * c.dp : kc + (size_t)(k0 % c.cap) * c.dp;
    const uint16_t *vr = pooled ? pvc + (size_t)k0 * c.vp : vc + (size_t)(k0 % c.cap) * c.vp;
#pragma unroll
    for (int y = 0; y < ND; ++y) {
      const int x = y * 256 + tid, r = x / (ND * 4), d = (x - r * (ND * 4)) * 8;
      kreg[y] = *(const u32x4 *)(kr + (size_t)min(r, last) * c.dp + min(d, c.dp - 8));
    }
#pragma unroll
    for (int y = 0; y < VN; ++y) {
      const int x = min(y * 256 + tid, VT - 1), oct = x / (NV * 16), d = min((x - oct * (NV * 16)) * 2, c.vp - 2);
#pragma unroll
      for (int r = 0; r < 8; ++r) vreg[y][r] = *(const uint32_t *)(vr + (size_t)min(oct * 8 + r, last) * c.vp + d);
    }
  };
  auto put = [&]() {
#pragma unroll
    for (int y = 0; y < ND; ++y) {
      const int x = y * 256 + tid, r = x / (ND * 4), d = (x - r * (ND * 4)) * 8;
      *(u32x4 *)(ks + r * KSTR + d) = kreg[y];
    }
#pragma unroll
    for (int y = 0; y < VN; ++y) {
      const int x = y * 256 + tid, oct = x / (NV * 16), d = (x - oct * (NV * 16)) * 2;
      if (x >= VT) continue;
      const uint32_t *w = vreg[y];
#pragma unroll
      for (int half = 0; half < 2; ++half) {  // keys 0-3 of the octet, keys 4-7
        const int at = vt_piece(d, (oct >> 1) * 2 + half) * 8 + (oct & 1) * 4;
        const uint32_t *k4 = w + 4 * half;
        *(u32x2 *)(vt + d * VSTR + at) = u32x2{(k4[0] & 0xffffu) | (k4[1] << 16), (k4[2] & 0xffffu) | (k4[3] << 16)};
        *(u32x2 *)(vt + (d + 1) * VSTR + at) = u32x2{(k4[0] >> 16) | (k4[1] & 0xffff0000u), (k4[2] >> 16) | (k4[3] & 0xffff0000u)};
      }
    }
  };
  fetch(0);
  for (int t = 0; t < tiles; ++t) {
    const bool pooled = t < tb;
    const int k0 = first_key(t);
    __syncthreads();  // the tile before has been multiplied
    put();
    __syncthreads();
    fetch(min(t + 1, tiles - 1));
    const bool none = pooled ? k0 >= nb1 : k0 > q1 || k0 + FK - 1 < lo0;
    const bool all = pooled ? k0 + FK <= nb0 : k0 >= lo1 && k0 + FK - 1 <= q0;
    if (none) continue;
    f32x16 sc[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
      for (int v = 0; v < 16; ++v) sc[kt][v] = 0.0f;
#pragma unroll
      for (int kk = 0; kk < ND * 2; ++kk) {
        const bf16x8 kf = *(const bf16x8 *)(ks + (kt * 32 + lq) * KSTR + kk * 16 + hh * 8);
        sc[kt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, q[kk], sc[kt], 0, 0, 0);
      }
    }
    const int from = (pooled ? 0 : lo) - k0 - 4 * hh, to = (pooled ? nb - 1 : p) - k0 - 4 * hh;  // the keys this lane's query sees, from its first one on
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int v = 0; v < 16; ++v) sc[kt][v] *= scale2;
    if (!all) {
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int v = 0; v < 16; ++v) {
          const int e = kt * 32 + 8 * (v >> 2) + (v & 3);
          sc[kt][v] = ((e < from) | (e > to)) ? NEG_INF : sc[kt][v];
        }
    }
    float tm = NEG_INF;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int v = 0; v < 16; ++v) tm = fmaxf(tm, sc[kt][v]);
    tm = fmaxf(tm, __shfl_xor(tm, 32));
    if (__any(tm > m)) {
      const float m1 = fmaxf(m, tm), al = m == NEG_INF ? 0.0f : __builtin_amdgcn_exp2f(m - m1);
      m = m1;
      z *= al;
#pragma unroll
      for (int j = 0; j < NV; ++j)
#pragma unroll
        for (int v = 0; v < 16; ++v) o[j][v] *= al;
    }
    const float mm = m == NEG_INF ? 0.0f : m;  // nothing seen so far
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        sc[kt][v] = __builtin_amdgcn_exp2f(sc[kt][v] - mm);
        z += sc[kt][v];
      }
#pragma unroll
    for (int ss = 0; ss < FK / 16; ++ss) {
      const f32x16 &f = sc[ss >> 1];
      const int v0 = (ss & 1) * 8;
      uint32_t pw[4];
#pragma unroll
      for (int y = 0; y < 4; ++y) {
        const f32x2 two = {f[v0 + 2 * y], f[v0 + 2 * y + 1]};
        pw[y] = __builtin_bit_cast(uint32_t, __builtin_convertvector(two, bf16x2));
      }
      const bf16x8 pf = __builtin_bit_cast(bf16x8, make_uint4(pw[0], pw[1], pw[2], pw[3]));
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int d = j * 32 + lq;
        const bf16x8 vf = *(const bf16x8 *)(vt + d * VSTR + vt_piece(d, ss * 2 + hh) * 8);
        o[j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf, o[j], 0, 0, 0);
      }
    }
  }
  z += __shfl_xor(z, 32);
  if (!live) return;
  const float inv = 1.0f / z;
  uint16_t *out = (uint16_t *)a.out + (size_t)tok * a.out_ld + h * s.vdim;
  const float *gate = a.g_off >= 0 ? a.proj + (size_t)tok * a.proj_ld + a.g_off + h * s.vdim : nullptr;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    float gt[16];
#pragma unroll
    for (int v = 0; v < 16; ++v) gt[v] = gate ? gate[min(j * 32 + 8 * (v >> 2) + 4 * hh + (v & 3), s.vdim - 1)] : 0.0f;
#pragma unroll
    for (int v = 0; v < 16; ++v) asm volatile("" : "+v"(gt[v]));  // all sixteen are asked for before the first is used
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int d = j * 32 + 8 * (v >> 2) + 4 * hh + (v & 3);
      const float y = o[j][v] * inv * (gate ? kxr::sigmoid_for<uint16_t>(gt[v]) : 1.0f);
      if (d < s.vdim) out[d] = kx_bf16_rne(y);
    }
  }
}

// keys per workgroup of win_partial_k: few parts, but enough workgroups
int part_keys(const KxWindowSpec &s, int total, int tokens) {
  const int R = s.heads / s.kv_heads;
  int ch = R <= 16 ? 256 : R <= 32 ? 128 : 64;  // R * ch scores in LDS
  while (ch > 64 && (long)kx_cdiv(total, ch) * s.kv_heads * tokens < 256) ch >>= 1;
  return ch;
}
// most keys a token of a sequence of `context` positions sees
int most_keys(const KxWindowSpec &s, int context) { return std::min(s.size, context) + seen_blocks(context - 1, s.size, s.pool); }
size_t floats_per_part(const KxWindowSpec &s) { return (size_t)s.heads * (kx_pad(s.vdim, 32) + 2); }

template <int ND>
int flash_nv(const KxWindowArgs &a, int nv, hipStream_t st) {
  const dim3 grid(kx_cdiv(a.positions, FQ), a.s.heads, a.batch);
#define KX_FLASH(NV)                                                                                                          \
  {                                                                                                                           \
    const size_t lds = ((size_t)FK * (ND * 32 + 8) + (size_t)NV * 32 * (FK + 8)) * 2;                                         \
    static std::atomic<bool> attr{false};                                                                                     \
    if (!attr) {                                                                                                              \
      KX_HIP(hipFuncSetAttribute((const void *)win_flash_k<ND, NV>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));   \
      attr = true;                                                                                                            \
    }                                                                                                                         \
    hipLaunchKernelGGL((win_flash_k<ND, NV>), grid, dim3(256), lds, st, a);                                                   \
  }
  if (nv == 1) KX_FLASH(1) else if (nv == 2) KX_FLASH(2) else if (nv <= 4) KX_FLASH(4) else KX_FLASH(8)
#undef KX_FLASH
  KX_LAUNCH_CHECK();
  return KX_OK;
}

int check(const KxWindowArgs &a) {
  const KxWindowSpec &s = a.s;
  KX_REQUIRE(s.heads > 0 && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.vdim > 0 && s.size > 0 && s.pool >= 0,
             "window attention: heads=%d kv_heads=%d dim=%d vdim=%d size=%d pool=%d", s.heads, s.kv_heads, s.dim, s.vdim, s.size, s.pool);
  KX_REQUIRE(a.c.vp <= 2048, "window attention: values of %d columns", s.vdim);
  KX_REQUIRE(a.batch > 0 && a.positions > 0 && a.pos >= 0, "window attention: %d x %d tokens at position %d", a.batch, a.positions, a.pos);
  return KX_OK;
}

// parts and merge
template <class T>
int attend_parts(const KxWindowArgs &a, bool fused, hipStream_t st) {
  const KxWindowSpec &s = a.s;
  const int tokens = a.batch * a.positions, R = s.heads / s.kv_heads;
  const int total = most_keys(s, a.pos + a.positions), ch = part_keys(s, total, tokens), parts = kx_cdiv(total, ch);
  const size_t per_token = (size_t)parts * floats_per_part(s);
  KX_REQUIRE(per_token <= a.part_floats, "window attention: %zu floats of partials, room for %zu", per_token, a.part_floats);
  const int at_once = (int)std::min<size_t>({(size_t)tokens, a.part_floats / per_token, (size_t)65535});
  const size_t lds = ((size_t)R * a.c.dp + (size_t)R * ch + (size_t)(PART_THREADS / (a.c.vp / 8)) * RB * a.c.vp) * 4;
  KX_REQUIRE(lds <= 160 * 1024 - 256, "window attention: %d query heads of %d per key head do not fit a workgroup", R, s.dim);
  static std::atomic<bool> attr{false};
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)win_partial_k<T, true>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 256));
    KX_HIP(hipFuncSetAttribute((const void *)win_partial_k<T, false>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 256));
    attr = true;
  }
  for (int t0 = 0; t0 < tokens; t0 += at_once) {
    const int n = std::min(at_once, tokens - t0);
    float *po = a.part, *pm = po + (size_t)n * parts * s.heads * a.c.vp, *pz = pm + (size_t)n * parts * s.heads;
    const dim3 grid(parts, s.kv_heads, n);
    if (fused) hipLaunchKernelGGL((win_partial_k<T, true>), grid, dim3(PART_THREADS), lds, st, a, t0, ch, po, pm, pz);
    else hipLaunchKernelGGL((win_partial_k<T, false>), grid, dim3(PART_THREADS), lds, st, a, t0, ch, po, pm, pz);
    KX_LAUNCH_CHECK();
    hipLaunchKernelGGL((win_merge_k<T>), dim3(s.heads, n), dim3(MERGE_THREADS), (size_t)parts * 4, st, a, t0, parts, po, pm, pz);
    KX_LAUNCH_CHECK();
  }
  return KX_OK;
}

// queries and cache rows in place
template <class T>
int attend(const KxWindowArgs &a, hipStream_t st) {
  if (sizeof(T) == 2 && a.c.dp <= 256 && a.c.vp <= 256) {
    const int nd = a.c.dp / 32, nv = a.c.vp / 32;
    return nd == 1 ? flash_nv<1>(a, nv, st) : nd == 2 ? flash_nv<2>(a, nv, st) : nd <= 4 ? flash_nv<4>(a, nv, st)
         : nd <= 6 ? flash_nv<6>(a, nv, st) : flash_nv<8>(a, nv, st);
  }
  return attend_parts<T>(a, false, st);
}

template <class T>
int attention(const KxWindowArgs &a, hipStream_t st) {
  const KxWindowSpec &s = a.s;
  int rc = check(a);
  if (rc) return rc;
  if (a.positions == 1) return attend_parts<T>(a, true, st);
  hipLaunchKernelGGL((win_prep_k<T>), dim3(a.batch * a.positions), dim3(256), 0, st, a);
  KX_LAUNCH_CHECK();
  if (s.pool > 0) {  // blocks whose last position is in this step
    const int b0 = a.pos / s.pool, b1 = std::min((a.pos + a.positions) / s.pool, a.c.blocks);
    if (b1 > b0) {
      hipLaunchKernelGGL((win_pool_k<T>), dim3(b1 - b0, s.kv_heads, a.batch), dim3(256), 0, st, a, b0);
      KX_LAUNCH_CHECK();
    }
  }
  return attend<T>(a, st);
}

}  // namespace

void kx_window_shape(const KxWindowSpec &s, int max_context, int max_positions, KxWindowCache *c, size_t elems[4]) {
  // a step writes its positions before any of them attends, and a block that completes in it may have begun before it
  const int64_t back = std::max(std::min(s.size, max_context), std::min(s.pool, max_context));
  c->cap = (int)std::min<int64_t>(kx_pad(max_context, FK), (back - 1 + max_positions + FK - 1) / FK * FK);
  c->blocks = s.pool > 0 ? max_context / s.pool : 0;
  c->dp = kx_pad(s.dim, 32);
  c->vp = kx_pad(s.vdim, 32);
  elems[0] = (size_t)s.kv_heads * c->cap * c->dp;
  elems[1] = (size_t)s.kv_heads * c->cap * c->vp;
  elems[2] = (size_t)s.kv_heads * c->blocks * c->dp;
  elems[3] = (size_t)s.kv_heads * c->blocks * c->vp;
}

size_t kx_window_part_floats(const KxWindowSpec &s, int max_context, int tokens) {
  // part_keys never goes below 64
  return (size_t)kx_cdiv(most_keys(s, max_context), 64) * floats_per_part(s) * tokens;
}

int kx_window_launch(bool f32, const KxWindowArgs &a, hipStream_t st) { return f32 ? attention<float>(a, st) : attention<uint16_t>(a, st); }

int kx_window_attend(bool f32, const KxWindowArgs &a, hipStream_t st) {
  const int rc = check(a);
  return rc ? rc : f32 ? attend<float>(a, st) : attend<uint16_t>(a, st);
}
