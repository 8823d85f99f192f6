// kx_delta.hip -- see kx_delta.h.  Everything here is 32-bit.  No counterpart in the reference, which has no recurrent layer.
//
// One token per sequence: delta_step_k.  A workgroup owns 32 columns of one head's state; it convolves and norms the
// head's q and k itself, reads its columns once, and writes them once.
// Several positions: delta_prep_k (convolutions, unit norms, beta, decay; tokens in parallel), delta_hist_k (the
// convolutions' inputs that the next step needs) and delta_scan_k, which keeps the state in registers: the columns of
// a head's state do not meet, so a column is spread over dim / 8 lanes with 8 rows each, and a wave goes through the
// tokens with two sums over those lanes per token, S^T k and S^T q; the read-out after the write is
// g S^T q + u (k . q).
#include <algorithm>
#include <atomic>
#include "kx_common.h"
#include "kx_rows.h"
#include "kx_delta.h"

namespace {

constexpr int SC = 32;  // columns per workgroup of delta_step_k

// log(1 + exp(x))
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.0f) + log1pf(kx_expf(-fabsf(x))); }
__device__ __forceinline__ float decay_of(const KxDeltaArgs &a, const float *pr, int h) {
  return kx_expf(-kx_expf(a.a_log[h]) * softplus(pr[a.a_off + h] + a.dt_bias[h]));
}

// offset in a projection row of convolution channel ch (q, k, v in turn)
__device__ __forceinline__ int channel_off(const KxDeltaArgs &a, int ch) {
  const int nq = a.s.kv_heads * a.s.dim;
  return ch < nq ? a.q_off + ch : ch < 2 * nq ? a.k_off + ch - nq : a.v_off + ch - 2 * nq;
}
// input of channel ch at position i of the step (i < 0: before it) of sequence b
__device__ __forceinline__ float conv_input(const KxDeltaArgs &a, int b, int i, int ch, int off) {
  return i >= 0 ? a.proj[(size_t)(i * a.batch + b) * a.proj_ld + off]
                : a.hist[((size_t)b * (a.s.taps - 1) + a.s.taps - 1 + i) * kx_delta_channels(a.s) + ch];
}
__device__ __forceinline__ float conv_silu(const KxDeltaArgs &a, int b, int i, int ch) {
  const int off = channel_off(a, ch);
  float v = 0.0f;
  for (int j = 0; j < a.s.taps; ++j) v = __builtin_fmaf(a.conv[(size_t)ch * a.s.taps + j], conv_input(a, b, i - (a.s.taps - 1) + j, ch, off), v);
  return kx_siluf(v);
}

__global__ void __launch_bounds__(256) delta_step_k(KxDeltaArgs a) {
  extern __shared__ float dl_lds[];
  __shared__ float red[4];
  __shared__ float part[2][8][SC];
  const KxDeltaSpec &s = a.s;
  const int D = s.dim, V = s.vdim, tid = threadIdx.x, slices = (V + SC - 1) / SC;
  const int h = blockIdx.x / slices, c0 = (blockIdx.x - h * slices) * SC, b = blockIdx.y;
  const int kvh = h / (s.heads / s.kv_heads), nq = s.kv_heads * D, C = kx_delta_channels(s);
  float *q = dl_lds, *k = q + D, *v = k + D, *S = v + SC;  // S [D][SC]
  const int c = tid & (SC - 1), rg = tid / SC, col = min(c0 + c, V - 1);
  float *st = a.state + ((size_t)b * s.heads + h) * D * V;
  for (int r = rg; r < D; r += 8) S[r * SC + c] = st[(size_t)r * V + col];
  float qq = 0.0f, kk = 0.0f;
  for (int x = tid; x < 2 * D; x += 256) {
    const bool key = x >= D;
    const int d = key ? x - D : x;
    const float y = conv_silu(a, b, 0, (key ? nq : 0) + kvh * D + d);
    (key ? k : q)[d] = y;
    if (key) kk = __builtin_fmaf(y, y, kk);
    else qq = __builtin_fmaf(y, y, qq);
  }
  if (tid < SC) v[tid] = c0 + tid < V ? conv_silu(a, b, 0, 2 * nq + h * V + c0 + tid) : 0.0f;
  qq = kxr::block_sum(qq, red);
  kk = kxr::block_sum(kk, red);
  const float qsc = kx_rsqrtf(qq + s.unit_eps) * kx_rsqrtf((float)D), ksc = kx_rsqrtf(kk + s.unit_eps);
  const float *pr = a.proj + (size_t)b * a.proj_ld;
  const float beta = kx_sigmoidf(pr[a.b_off + h]), g = decay_of(a, pr, h);
  // the convolutions' inputs for the next token: this workgroup's value channels, and q and k once per head of theirs
  const int keep = s.taps - 1;
  auto shift = [&](int ch) {
    const int off = channel_off(a, ch);
    for (int j = 0; j < keep; ++j) a.hist_out[((size_t)b * keep + j) * C + ch] = conv_input(a, b, j - keep + 1, ch, off);
  };
  if (keep) {
    if (tid < SC && c0 + tid < V) shift(2 * nq + h * V + c0 + tid);
    if (c0 == 0 && h % (s.heads / s.kv_heads) == 0)
      for (int x = tid; x < 2 * D; x += 256) shift(x < D ? kvh * D + x : nq + kvh * D + x - D);
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

// work, per token: q [kv_heads * dim], k, v [heads * vdim], decay and beta [heads], k . q [kv_heads]
struct Work {
  float *qkv, *gb, *kq;
};
__device__ __forceinline__ Work work_of(const KxDeltaArgs &a) {
  const size_t T = (size_t)a.batch * a.positions;
  Work w;
  w.qkv = a.work;
  w.gb = w.qkv + T * kx_delta_channels(a.s);
  w.kq = w.gb + T * 2 * a.s.heads;
  return w;
}

__global__ void __launch_bounds__(256) delta_prep_k(KxDeltaArgs a) {
  const KxDeltaSpec &s = a.s;
  const int tok = blockIdx.x, i = tok / a.batch, b = tok - i * a.batch, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int D = s.dim, nq = s.kv_heads * D, C = kx_delta_channels(s);
  const Work w = work_of(a);
  float *out = w.qkv + (size_t)tok * C;
  const float *pr = a.proj + (size_t)tok * a.proj_ld;
  for (int h = wave; h < s.kv_heads; h += 4) {
    float qq = 0.0f, kk = 0.0f, kq = 0.0f;
    for (int d = lane; d < D; d += 64) {
      const float q = conv_silu(a, b, i, h * D + d), k = conv_silu(a, b, i, nq + h * D + d);
      qq = __builtin_fmaf(q, q, qq);
      kk = __builtin_fmaf(k, k, kk);
      kq = __builtin_fmaf(k, q, kq);
      out[h * D + d] = q;  // this lane's own words, scaled below
      out[nq + h * D + d] = k;
    }
    qq = kx_rsqrtf(kxr::wave_sum(qq) + s.unit_eps) * kx_rsqrtf((float)D);
    kk = kx_rsqrtf(kxr::wave_sum(kk) + s.unit_eps);
    kq = kxr::wave_sum(kq) * qq * kk;
    for (int d = lane; d < D; d += 64) {
      out[h * D + d] *= qq;
      out[nq + h * D + d] *= kk;
    }
    if (lane == 0) w.kq[(size_t)tok * s.kv_heads + h] = kq;
  }
  for (int x = threadIdx.x; x < s.heads * s.vdim; x += 256) out[2 * nq + x] = conv_silu(a, b, i, 2 * nq + x);
  for (int h = threadIdx.x; h < s.heads; h += 256) {
    w.gb[((size_t)tok * s.heads + h) * 2] = decay_of(a, pr, h);
    w.gb[((size_t)tok * s.heads + h) * 2 + 1] = kx_sigmoidf(pr[a.b_off + h]);
  }
}

__global__ void __launch_bounds__(256) delta_hist_k(KxDeltaArgs a) {
  const int C = kx_delta_channels(a.s), keep = a.s.taps - 1, ch = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (ch >= C) return;
  const int off = channel_off(a, ch);
  for (int j = 0; j < keep; ++j)
    a.hist_out[((size_t)b * keep + j) * C + ch] = conv_input(a, b, a.positions - keep + j, ch, off);
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

template <int LPC>  // lanes per column, 8 rows of the state each
__global__ void __launch_bounds__(256) delta_scan_k(KxDeltaArgs a) {
  constexpr int DP = LPC * 8, COLS = 256 / LPC, CT = LPC >= 16 ? 16 : 32;  // CT: tokens per staged block
  __shared__ __attribute__((aligned(16))) float kq_s[2][CT][2][DP];
  __shared__ float v_s[2][CT][COLS];
  __shared__ float sc_s[2][CT][4];  // decay, beta, k . q
  const KxDeltaSpec &s = a.s;
  const int D = s.dim, V = s.vdim, tid = threadIdx.x;
  const int h = blockIdx.y, b = blockIdx.z, c0 = blockIdx.x * COLS, kvh = h / (s.heads / s.kv_heads), nq = s.kv_heads * D;
  const int C = kx_delta_channels(s), r0 = (tid % LPC) * 8, cl = tid / LPC, col = c0 + cl, n = a.positions;
  const Work w = work_of(a);
  float *st = a.state + ((size_t)b * s.heads + h) * D * V;
  float S[8];
#pragma unroll
  for (int r = 0; r < 8; ++r) S[r] = r0 + r < D && col < V ? st[(size_t)(r0 + r) * V + col] : 0.0f;
  // A block of tokens goes through registers into one of two LDS stages while the other is worked on.  Places past the
  // last token hold a token that leaves the state as it is.
  constexpr int NK = CT * DP * 2 / 256, NV = (CT * COLS + 255) / 256;
  float rk[NK], rv[NV], rs = 0.0f;
  auto fetch = [&](int t0) {
#pragma unroll
    for (int x = 0; x < NK; ++x) {
      const int at = x * 256 + tid, d = at % DP, q = at / DP & 1, t = t0 + at / (2 * DP);
      rk[x] = t < n && d < D ? w.qkv[(size_t)(t * a.batch + b) * C + (q ? 0 : nq) + kvh * D + d] : 0.0f;
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int at = x * 256 + tid, t = t0 + at / COLS, cc = c0 + at % COLS;
      rv[x] = t < n && cc < V && at < CT * COLS ? w.qkv[(size_t)(t * a.batch + b) * C + 2 * nq + h * V + cc] : 0.0f;
    }
    if (tid < CT * 3) {
      const int t = t0 + tid / 3, f = tid % 3;
      rs = t >= n ? (f == 0 ? 1.0f : 0.0f) : f < 2 ? w.gb[((size_t)(t * a.batch + b) * s.heads + h) * 2 + f] : w.kq[(size_t)(t * a.batch + b) * s.kv_heads + kvh];
    }
  };
  auto put = [&](int stage) {
#pragma unroll
    for (int x = 0; x < NK; ++x) {
      const int at = x * 256 + tid;
      kq_s[stage][at / (2 * DP)][at / DP & 1][at % DP] = rk[x];
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int at = x * 256 + tid;
      if (at < CT * COLS) v_s[stage][at / COLS][at % COLS] = rv[x];
    }
    if (tid < CT * 3) sc_s[stage][tid / 3][tid % 3] = rs;
  };
  fetch(0);
  put(0);
  __syncthreads();
  for (int t0 = 0, stage = 0; t0 < n; t0 += CT, stage ^= 1) {
    if (t0 + CT < n) fetch(t0 + CT);
#pragma unroll 4
    for (int t = 0; t < CT; ++t) {
      const float *kp = &kq_s[stage][t][0][r0], *qp = &kq_s[stage][t][1][r0];
      const float4 ka = *(const float4 *)kp, kb = *(const float4 *)(kp + 4), qa = *(const float4 *)qp, qb = *(const float4 *)(qp + 4);
      const float k[8] = {ka.x, ka.y, ka.z, ka.w, kb.x, kb.y, kb.z, kb.w}, q[8] = {qa.x, qa.y, qa.z, qa.w, qb.x, qb.y, qb.z, qb.w};
      const float g = sc_s[stage][t][0], beta = sc_s[stage][t][1], kq = sc_s[stage][t][2];
      float sk = 0.0f, sq = 0.0f;
#pragma unroll
      for (int r = 0; r < 8; ++r) {
        sk = __builtin_fmaf(S[r], k[r], sk);
        sq = __builtin_fmaf(S[r], q[r], sq);
      }
      sk = column_sum<LPC>(sk);
      sq = column_sum<LPC>(sq);
      const float u = beta * (v_s[stage][t][cl] - g * sk);
#pragma unroll
      for (int r = 0; r < 8; ++r) S[r] = __builtin_fmaf(k[r], u, g * S[r]);
      if (r0 == 0 && col < V && t0 + t < n) a.o[((size_t)((t0 + t) * a.batch + b) * s.heads + h) * V + col] = __builtin_fmaf(u, kq, g * sq);
    }
    if (t0 + CT < n) put(stage ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int r = 0; r < 8; ++r)
    if (r0 + r < D && col < V) st[(size_t)(r0 + r) * V + col] = S[r];
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
    hipLaunchKernelGGL(delta_step_k, dim3(s.heads * kx_cdiv(s.vdim, SC), a.batch), dim3(256), lds, st, a);
    KX_LAUNCH_CHECK();
    return KX_OK;
  }
  KX_REQUIRE(a.work, "delta rule: no scratch");
  hipLaunchKernelGGL(delta_prep_k, dim3(a.batch * a.positions), dim3(256), 0, st, a);
  KX_LAUNCH_CHECK();
  if (s.taps > 1) {
    hipLaunchKernelGGL(delta_hist_k, dim3(kx_cdiv(kx_delta_channels(s), 256), a.batch), dim3(256), 0, st, a);
    KX_LAUNCH_CHECK();
  }
#define KX_SCAN(LPC) hipLaunchKernelGGL(delta_scan_k<LPC>, dim3(kx_cdiv(s.vdim, 256 / LPC), s.heads, a.batch), dim3(256), 0, st, a)
  if (s.dim <= 32) KX_SCAN(4);
  else if (s.dim <= 64) KX_SCAN(8);
  else if (s.dim <= 128) KX_SCAN(16);
  else KX_SCAN(32);
#undef KX_SCAN
  KX_LAUNCH_CHECK();
  return KX_OK;
}
