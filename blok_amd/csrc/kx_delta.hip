// kx_delta.hip -- see kx_delta.h.  Everything here is 32-bit.  No counterpart in the reference, which has no recurrent layer.
//
// One token per sequence: delta_step_k.  A workgroup owns 32 columns of one head's state; it convolves and norms the
// head's q and k itself, reads its columns once, and writes them once.
//
// Several positions: the convolutions (kx_conv.hip), delta_unit_k (unit norms and the numbers below) and delta_scan_k, which
// keeps the state in registers:
// the columns of a head's state do not meet, so a column is spread over dim / 8 lanes with 8 rows each, and a wave goes
// through the tokens.  It takes them in blocks of four, so that the sums over a column's lanes do not wait for each
// other: with S the state before the block, D(i, j) the product of the decays of tokens i + 1 .. j and D(j) that of tokens
// 1 .. j of the block,
//   u_j = beta_j (v_j - D(j) S^T k_j - sum_{i < j} D(i, j) (k_i . k_j) u_i)
//   o_j = D(j) S^T q_j + sum_{i <= j} D(i, j) (k_i . q_j) u_i
//   S  <- D(4) S + sum_i D(i, 4) k_i u_i^T,
// which is the recurrence written out for four tokens.  The numbers that do not depend on the column -- per token D(j),
// beta, D(j, 4), D(j - d, j) (k_{j-d} . k_j) for d = 1..3 and D(j - d, j) (k_{j-d} . q_j) for d = 0..3 -- are made
// once per head by delta_unit_k.
#include <algorithm>
#include <atomic>
#include "kx_common.h"
#include "kx_conv.h"
#include "kx_rows.h"
#include "kx_delta.h"

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int SC = 32;  // columns per workgroup of delta_step_k

__device__ __forceinline__ float decay_of(const KxDeltaArgs &a, const float *pr, int h) {
  return kx_expf(-kx_expf(a.a_log[h]) * kxr::softplus(pr[a.a_off + h] + a.dt_bias[h]));
}

__host__ __device__ __forceinline__ KxConvArgs conv_of(const KxDeltaArgs &a) {
  const int nq = a.s.kv_heads * a.s.dim;
  KxConvArgs c;
  c.proj = a.proj; c.proj_ld = a.proj_ld;
  c.segs = 3;
  c.end[0] = nq; c.end[1] = 2 * nq; c.end[2] = c.channels = kx_delta_channels(a.s);
  c.off[0] = a.q_off; c.off[1] = a.k_off; c.off[2] = a.v_off;
  c.taps = a.s.taps; c.w = a.conv;
  c.hist = a.hist; c.hist_out = a.hist_out; c.batch = a.batch; c.positions = a.positions;
  return c;
}

__global__ void __launch_bounds__(256) delta_step_k(KxDeltaArgs a, KxConvArgs cv) {
  extern __shared__ float dl_lds[];
  __shared__ float red[4];
  __shared__ float part[2][8][SC];
  const KxDeltaSpec &s = a.s;
  const int D = s.dim, V = s.vdim, tid = threadIdx.x, slices = (V + SC - 1) / SC;
  const int h = blockIdx.x / slices, c0 = (blockIdx.x - h * slices) * SC, b = blockIdx.y;
  const int kvh = h / (s.heads / s.kv_heads), nq = s.kv_heads * D;
  float *q = dl_lds, *k = q + D, *v = k + D, *S = v + SC;  // S [D][SC]
  const int c = tid & (SC - 1), rg = tid / SC, col = min(c0 + c, V - 1);
  float *st = a.state + ((size_t)b * s.heads + h) * D * V;
  for (int r = rg; r < D; r += 8) S[r * SC + c] = st[(size_t)r * V + col];
  float qq = 0.0f, kk = 0.0f;
  for (int x = tid; x < 2 * D; x += 256) {
    const bool key = x >= D;
    const int d = key ? x - D : x;
    const float y = kxc::conv_silu(cv, b, 0, (key ? nq : 0) + kvh * D + d);
    (key ? k : q)[d] = y;
    if (key) kk = __builtin_fmaf(y, y, kk);
    else qq = __builtin_fmaf(y, y, qq);
  }
  if (tid < SC) v[tid] = c0 + tid < V ? kxc::conv_silu(cv, b, 0, 2 * nq + h * V + c0 + tid) : 0.0f;
  qq = kxr::block_sum(qq, red);
  kk = kxr::block_sum(kk, red);
  const float qsc = kx_rsqrtf(qq + s.unit_eps) * kx_rsqrtf((float)D), ksc = kx_rsqrtf(kk + s.unit_eps);
  const float *pr = a.proj + (size_t)b * a.proj_ld;
  const float beta = kx_sigmoidf(pr[a.b_off + h]), g = decay_of(a, pr, h);
  // the convolutions' inputs for the next token: this workgroup's value channels, and q and k once per head of theirs
  if (s.taps > 1) {
    if (tid < SC && c0 + tid < V) kxc::shift(cv, b, 2 * nq + h * V + c0 + tid);
    if (c0 == 0 && h % (s.heads / s.kv_heads) == 0)
      for (int x = tid; x < 2 * D; x += 256) kxc::shift(cv, b, x < D ? kvh * D + x : nq + kvh * D + x - D);
  }
  float sk = 0.0f;
  for (int r = rg; r < D; r += 8) sk = __builtin_fmaf(S[r * SC + c], k[r], sk);
  part[0][rg][c] = sk;
  __syncthreads();
  sk = 0.0f;
#pragma unroll
  for (int j = 0; j < 8; ++j) sk += part[0][j][c];
  const float u = beta * (v[c] - g * (sk * ksc)) * ksc;
  float o = 0.0f;
  for (int r = rg; r < D; r += 8) {
    const float n = __builtin_fmaf(k[r], u, g * S[r * SC + c]);
    o = __builtin_fmaf(n, q[r], o);
    if (c0 + c < V) st[(size_t)r * V + c0 + c] = n;
  }
  part[1][rg][c] = o;
  __syncthreads();
  if (rg == 0 && c0 + c < V) {
    o = 0.0f;
#pragma unroll
    for (int j = 0; j < 8; ++j) o += part[1][j][c];
    a.o[(size_t)b * s.heads * V + h * V + c0 + c] = o * qsc;
  }
}

constexpr int NB = KX_DELTA_BLOCK, NCF = KX_DELTA_COEF;
enum { CF_GAMMA = 0, CF_BETA = 1, CF_END = 2, CF_KK = 3, CF_KQ = 6 };  // places of a token's numbers

struct Work {
  float *coef;  // [batch][heads][padded positions][NCF]
  float *qk;    // [tokens][kv_heads][2][kx_delta_row]: unit k, unit q times dim^-1/2, zeros behind them
  float *raw;   // [tokens][channels]: q, k, v behind convolution and silu
  int padded;
};
__host__ __device__ __forceinline__ Work work_of(const KxDeltaArgs &a) {
  Work w;
  w.padded = (a.positions + NB - 1) / NB * NB;
  w.coef = a.work;
  w.qk = w.coef + (size_t)a.batch * a.s.heads * w.padded * NCF;
  w.raw = w.qk + (size_t)a.batch * a.positions * a.s.kv_heads * 2 * kx_delta_row(a.s);
  return w;
}

// one wave per (position, key head)
__global__ void __launch_bounds__(256) delta_unit_k(KxDeltaArgs a) {
  const KxDeltaSpec &s = a.s;
  const int lane = threadIdx.x & 63, D = s.dim, nq = s.kv_heads * D, C = kx_delta_channels(s), ratio = s.heads / s.kv_heads;
  const Work w = work_of(a);
  const int item = blockIdx.x * 4 + (threadIdx.x >> 6), kvh = item % s.kv_heads, i = item / s.kv_heads, b = blockIdx.y;
  if (i >= w.padded) return;
  const int j = i % NB, t0 = i - j;  // place in the block, and the block's first position
  float dot[NB + NB - 1] = {}, inv[NB] = {};  // kk of d = 1.., kq of d = 0..
  if (i < a.positions) {
    const float *row[NB];
#pragma unroll
    for (int d = 0; d < NB; ++d) row[d] = w.raw + (size_t)((i - min(d, j)) * a.batch + b) * C + kvh * D;
    float qq = 0.0f, ss[NB] = {};
    for (int x = lane; x < D; x += 64) {
      const float q = row[0][x];
      float k[NB];
#pragma unroll
      for (int d = 0; d < NB; ++d) k[d] = row[d][nq + x];
      qq = __builtin_fmaf(q, q, qq);
#pragma unroll
      for (int d = 0; d < NB; ++d) {
        ss[d] = __builtin_fmaf(k[d], k[d], ss[d]);
        dot[NB - 1 + d] = __builtin_fmaf(k[d], q, dot[NB - 1 + d]);
        if (d) dot[d - 1] = __builtin_fmaf(k[d], k[0], dot[d - 1]);
      }
    }
    const float qsc = kx_rsqrtf(kxr::wave_sum(qq) + s.unit_eps) * kx_rsqrtf((float)D);
#pragma unroll
    for (int d = 0; d < NB; ++d) inv[d] = kx_rsqrtf(kxr::wave_sum(ss[d]) + s.unit_eps);
#pragma unroll
    for (int d = 0; d < NB; ++d) {
      dot[NB - 1 + d] = kxr::wave_sum(dot[NB - 1 + d]) * inv[d] * qsc;
      if (d) dot[d - 1] = kxr::wave_sum(dot[d - 1]) * inv[d] * inv[0];
    }
    const int DP = kx_delta_row(s);
    float *out = w.qk + ((size_t)(i * a.batch + b) * s.kv_heads + kvh) * 2 * DP;
    for (int x = lane; x < DP; x += 64) {
      out[x] = x < D ? row[0][nq + x] * inv[0] : 0.0f;
      out[DP + x] = x < D ? row[0][x] * qsc : 0.0f;
    }
  }
  for (int r = lane; r < ratio; r += 64) {  // the heads that share the key
    const int h = kvh * ratio + r;
    float g[NB];  // decays of the block; a position past the end leaves the state as it is
#pragma unroll
    for (int d = 0; d < NB; ++d)
      g[d] = t0 + d < a.positions ? decay_of(a, a.proj + (size_t)((t0 + d) * a.batch + b) * a.proj_ld, h) : 1.0f;
    float *cf = w.coef + (((size_t)b * s.heads + h) * w.padded + i) * NCF;
    float gamma = 1.0f, end = 1.0f;
#pragma unroll
    for (int d = 0; d < NB; ++d) {
      if (d <= j) gamma *= g[d];
      else end *= g[d];
    }
    cf[CF_GAMMA] = gamma;
    cf[CF_BETA] = i < a.positions ? kx_sigmoidf(a.proj[(size_t)(i * a.batch + b) * a.proj_ld + a.b_off + h]) : 0.0f;
    cf[CF_END] = end;
    float down = 1.0f;  // D(j - d, j)
#pragma unroll
    for (int d = 0; d < NB; ++d) {
      const bool in = d <= j;  // the other token is in the block
      cf[CF_KQ + d] = in ? down * dot[NB - 1 + d] : 0.0f;
      if (d) cf[CF_KK + d - 1] = in ? down * dot[d - 1] : 0.0f;
#pragma unroll
      for (int x = 0; x < NB; ++x)
        if (x == j - d) down *= g[x];
    }
  }
}

template <int LPC>
__device__ __forceinline__ float column_sum(float v) {  // over the LPC lanes of a column, in every one of them
  v += kxw::dpp_f<kxw::DPP_QUAD_XOR1>(v);
  v += kxw::dpp_f<kxw::DPP_QUAD_XOR2>(v);
  if (LPC >= 8) v += kxw::dpp_f<kxw::DPP_ROW_HALF_MIRROR>(v);
  if (LPC >= 16) v += kxw::dpp_f<kxw::DPP_ROW_MIRROR>(v);
  if (LPC >= 32) {
    float t = v;
    kxw::swap_rows16(v, t);
    v += t;
  }
  return v;
}

// A block's numbers, one per lane as they are loaded, in scalar registers as they are used: they are the same for the whole
// workgroup.  (Scalar loads would come from the memory side of the caches, 1-2 us away, once per block.)
struct Coefs {
  float v[NB][NCF];
  __device__ __forceinline__ void from_lanes(float x) {
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
      for (int y = 0; y < NCF; ++y) v[j][y] = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, x), j * NCF + y));
  }
};
static_assert(NB * NCF <= 64, "a block's numbers are one wave load");

template <int LPC>  // lanes per column, 8 rows of the state each
__global__ void __launch_bounds__(256) delta_scan_k(KxDeltaArgs a) {
  constexpr int DP = LPC * 8, COLS = 256 / LPC, CT = LPC >= 16 ? 16 : 32;  // CT: tokens per staged block
  __shared__ __attribute__((aligned(16))) float kq_s[2][CT][2][DP];
  __shared__ float v_s[2][CT][COLS], o_s[2][CT][COLS];
  const KxDeltaSpec &s = a.s;
  const int D = s.dim, V = s.vdim, tid = threadIdx.x;
  const int h = blockIdx.y, b = blockIdx.z, c0 = blockIdx.x * COLS, kvh = h / (s.heads / s.kv_heads), nq = s.kv_heads * D;
  const int C = kx_delta_channels(s), l4 = (tid % LPC) * 4, cl = tid / LPC, col = c0 + cl, n = a.positions;
  const Work w = work_of(a);
  const float *coef = w.coef + ((size_t)b * s.heads + h) * w.padded * NCF;
  float *st = a.state + ((size_t)b * s.heads + h) * D * V;
  auto row = [&](int r) { return (r < 4 ? 0 : DP / 2 - 4) + l4 + r; };  // two runs of four rows: neighbouring lanes read neighbouring words
  float S[8];
#pragma unroll
  for (int r = 0; r < 8; ++r) S[r] = row(r) < D && col < V ? st[(size_t)row(r) * V + col] : 0.0f;
  // A stage of tokens goes through registers into one of two LDS stages while the other is worked on.  Places past the last
  // token repeat it: their numbers in `coef` make them leave the state alone.
  constexpr int NK = CT * DP * 2 / 4 / 256, NV = (CT * COLS + 255) / 256;
  f32x4 rk[NK];
  float rv[NV], rc[CT / NB], rn[CT / NB];  // rc, rn: the numbers of this stage's blocks and of the next
  auto fetch = [&](int t0) {
#pragma unroll
    for (int x = 0; x < NK; ++x) {
      const int at = (x * 256 + tid) * 4, t = min(t0 + at / (2 * DP), n - 1);
      rk[x] = *(const f32x4 *)(w.qk + ((size_t)(t * a.batch + b) * s.kv_heads + kvh) * 2 * DP + at % (2 * DP));
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int at = min(x * 256 + tid, CT * COLS - 1), t = min(t0 + at / COLS, n - 1), cc = min(c0 + at % COLS, V - 1);
      rv[x] = w.raw[(size_t)(t * a.batch + b) * C + 2 * nq + h * V + cc];
    }
#pragma unroll
    for (int x = 0; x < CT / NB; ++x) rn[x] = coef[(size_t)min(t0 + x * NB, w.padded - NB) * NCF + min(tid & 63, NB * NCF - 1)];
  };
  auto put = [&](int stage) {
#pragma unroll
    for (int x = 0; x < CT / NB; ++x) rc[x] = rn[x];
#pragma unroll
    for (int x = 0; x < NK; ++x) *(f32x4 *)(&kq_s[stage][0][0][0] + (x * 256 + tid) * 4) = rk[x];
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int at = x * 256 + tid;
      if (at < CT * COLS) v_s[stage][at / COLS][at % COLS] = rv[x];
    }
  };
  // keys, queries and values of a block, read from LDS while the block before it is worked on
  float k[2][NB][8], q[2][NB][8], v[2][NB];
  auto read = [&](int x, int stage, int tb) {
#pragma unroll
    for (int j = 0; j < NB; ++j) {
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const f32x4 kk = *(const f32x4 *)&kq_s[stage][tb + j][0][half * (DP / 2) + l4], qq = *(const f32x4 *)&kq_s[stage][tb + j][1][half * (DP / 2) + l4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          k[x][j][half * 4 + e] = kk[e];
          q[x][j][half * 4 + e] = qq[e];
        }
      }
      v[x][j] = v_s[stage][tb + j][cl];
    }
  };
  fetch(0);
  put(0);
  __syncthreads();
  for (int t0 = 0, stage = 0; t0 < n; t0 += CT, stage ^= 1) {
    fetch(t0 + CT);  // past the end: the last token again
    read(0, stage, 0);
#pragma unroll
    for (int tb = 0; tb < CT; tb += NB) {
      if (t0 + tb >= n) break;
      const int x = (tb / NB) & 1;
      float sk[NB], sq[NB];
#pragma unroll
      for (int j = 0; j < NB; ++j) {
        sk[j] = sq[j] = 0.0f;
#pragma unroll
        for (int r = 0; r < 8; ++r) {
          sk[j] = __builtin_fmaf(S[r], k[x][j][r], sk[j]);
          sq[j] = __builtin_fmaf(S[r], q[x][j][r], sq[j]);
        }
      }
      if (tb + NB < CT) read(x ^ 1, stage, tb + NB);
#pragma unroll
      for (int j = 0; j < NB; ++j) {
        sk[j] = column_sum<LPC>(sk[j]);
        sq[j] = column_sum<LPC>(sq[j]);
      }
      Coefs now;
      now.from_lanes(rc[tb / NB]);
      float u[NB];
#pragma unroll
      for (int j = 0; j < NB; ++j) {
        float e = __builtin_fmaf(-now.v[j][CF_GAMMA], sk[j], v[x][j]), o = now.v[j][CF_GAMMA] * sq[j];
#pragma unroll
        for (int d = 1; d <= j; ++d) {
          e = __builtin_fmaf(-now.v[j][CF_KK + d - 1], u[j - d], e);
          o = __builtin_fmaf(now.v[j][CF_KQ + d], u[j - d], o);
        }
        u[j] = now.v[j][CF_BETA] * e;
        o = __builtin_fmaf(now.v[j][CF_KQ], u[j], o);
        if (l4 == 0) o_s[stage][tb + j][cl] = o;
      }
#pragma unroll
      for (int r = 0; r < 8; ++r) S[r] *= now.v[NB - 1][CF_GAMMA];
#pragma unroll
      for (int j = 0; j < NB; ++j) {
        const float y = u[j] * now.v[j][CF_END];
#pragma unroll
        for (int r = 0; r < 8; ++r) S[r] = __builtin_fmaf(k[x][j][r], y, S[r]);
      }
    }
    put(stage ^ 1);
    __syncthreads();
    // the read-outs go to memory here, behind the wait for the next stage's rows, so that no wait is for a store just made
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int at = x * 256 + tid, t = t0 + at / COLS, cc = c0 + at % COLS;
      if (at < CT * COLS && t < n && cc < V) a.o[((size_t)(t * a.batch + b) * s.heads + h) * V + cc] = o_s[stage][at / COLS][at % COLS];
    }
  }
#pragma unroll
  for (int r = 0; r < 8; ++r)
    if (row(r) < D && col < V) st[(size_t)row(r) * V + col] = S[r];
}

}  // namespace

int kx_delta_launch(const KxDeltaArgs &a, hipStream_t st) {
  const KxDeltaSpec &s = a.s;
  KX_REQUIRE(s.heads > 0 && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.vdim > 0 && s.taps > 0,
             "delta rule: heads=%d kv_heads=%d dim=%d vdim=%d taps=%d", s.heads, s.kv_heads, s.dim, s.vdim, s.taps);
  KX_REQUIRE(s.dim <= 256, "delta rule: keys of %d columns, at most 256", s.dim);
  KX_REQUIRE(a.batch > 0 && a.positions > 0 && (s.taps == 1 || (a.hist && a.hist_out && a.hist != a.hist_out)), "delta rule: %d x %d tokens", a.batch, a.positions);
  if (a.positions == 1) {
    const size_t lds = ((size_t)2 * s.dim + SC + (size_t)s.dim * SC) * 4;
    hipLaunchKernelGGL(delta_step_k, dim3(s.heads * kx_cdiv(s.vdim, SC), a.batch), dim3(256), lds, st, a, conv_of(a));
    KX_LAUNCH_CHECK();
    return KX_OK;
  }
  KX_REQUIRE(a.work, "delta rule: no scratch");
  const int rc = kx_conv_launch(conv_of(a), work_of(a).raw, st);
  if (rc) return rc;
  hipLaunchKernelGGL(delta_unit_k, dim3(kx_cdiv(work_of(a).padded * s.kv_heads, 4), a.batch), dim3(256), 0, st, a);
  KX_LAUNCH_CHECK();
#define KX_SCAN(LPC) hipLaunchKernelGGL(delta_scan_k<LPC>, dim3(kx_cdiv(s.vdim, 256 / LPC), s.heads, a.batch), dim3(256), 0, st, a)
  if (s.dim <= 32) KX_SCAN(4);
  else if (s.dim <= 64) KX_SCAN(8);
  else if (s.dim <= 128) KX_SCAN(16);
  else KX_SCAN(32);
#undef KX_SCAN
  KX_LAUNCH_CHECK();
  return KX_OK;
}
