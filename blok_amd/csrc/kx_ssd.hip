// kx_ssd.hip -- see kx_ssd.h.  Everything here is 32-bit.  No counterpart in the reference, which has no recurrent layer.
//
// One token per sequence: ssd_step_k.  A workgroup owns 32 columns of one head's state; it convolves its x, B and C itself,
// reads its columns once, and writes them once.
// Several positions: the convolutions (kx_conv.hip), ssd_coef_k (the numbers of kx_scan.h's blocks, with dt and the skip
// weight in them) and kx_scan.hip.
#include "kx_common.h"
#include "kx_conv.h"
#include "kx_rows.h"
#include "kx_ssd.h"

namespace {

constexpr int SC = 32;  // columns per workgroup of ssd_step_k
constexpr int NB = KX_SCAN_BLOCK;

KxConvArgs conv_of(const KxSsdArgs &a) {
  KxConvArgs c;
  c.proj = a.proj; c.proj_ld = a.proj_ld;
  c.end[0] = c.channels = kx_ssd_channels(a.s);
  c.off[0] = a.x_off;
  c.taps = a.s.taps; c.w = a.conv; c.bias = a.conv_bias;
  c.hist = a.hist; c.hist_out = a.hist_out; c.batch = a.batch; c.positions = a.positions;
  return c;
}
__device__ __forceinline__ float step_size(const KxSsdArgs &a, size_t tok, int h) { return kxr::softplus(a.proj[tok * a.proj_ld + a.dt_off + h] + a.dt_bias[h]); }
__device__ __forceinline__ float decay_of(const KxSsdArgs &a, int h, float dt) { return kx_expf(-kx_expf(a.a_log[h]) * dt); }

template <int RPT>  // rows of the state per thread
__global__ void __launch_bounds__(256) ssd_step_k(KxSsdArgs a, KxConvArgs cv) {
  __shared__ float bc[2 * 8 * RPT], xs[SC], part[8][SC];
  const KxSsdSpec &s = a.s;
  const int N = s.state, V = s.vdim, tid = threadIdx.x, slices = (V + SC - 1) / SC;
  const int h = blockIdx.x / slices, c0 = (blockIdx.x - h * slices) * SC, b = blockIdx.y, ratio = s.heads / s.groups, g = h / ratio;
  const int c = tid & (SC - 1), rg = tid / SC, col = min(c0 + c, V - 1), inner = kx_ssd_inner(s);
  float *st = a.state + ((size_t)b * s.heads + h) * N * V;
  float S[RPT];
#pragma unroll
  for (int r = 0; r < RPT; ++r) S[r] = st[(size_t)min(rg + 8 * r, N - 1) * V + col];
  auto channel = [&](int i) { return inner + (i < N ? g * N + i : s.groups * N + g * N + i - N); };
  for (int i = tid; i < 2 * N; i += 256) bc[i] = kxc::conv_silu(cv, b, 0, channel(i));
  if (tid < SC) xs[tid] = c0 + tid < V ? kxc::conv_silu(cv, b, 0, h * V + c0 + tid) : 0.0f;
  const float dt = step_size(a, b, h), decay = decay_of(a, h, dt);
  // the convolutions' inputs for the next token: this workgroup's x channels, and B and C once per group
  if (s.taps > 1) {
    if (tid < SC && c0 + tid < V) kxc::shift(cv, b, h * V + c0 + tid);
    if (c0 == 0 && h % ratio == 0)
      for (int i = tid; i < 2 * N; i += 256) kxc::shift(cv, b, channel(i));
  }
  __syncthreads();
  const float x = xs[c] * dt;
  float y = 0.0f;
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int row = rg + 8 * r;
    if (row < N) {
      const float v = __builtin_fmaf(bc[row], x, decay * S[r]);
      y = __builtin_fmaf(v, bc[N + row], y);
      if (c0 + c < V) st[(size_t)row * V + c0 + c] = v;
    }
  }
  part[rg][c] = y;
  __syncthreads();
  if (rg == 0 && c0 + c < V) {
    y = a.skip[h] * xs[c];
#pragma unroll
    for (int j = 0; j < 8; ++j) y += part[j][c];
    a.y[(size_t)b * inner + h * V + c0 + c] = y;
  }
}

struct Work {
  float *raw, *inner, *gamma, *end;
};
__host__ __device__ __forceinline__ Work work_of(const KxSsdArgs &a) {
  const size_t rows = (size_t)a.batch * a.s.heads * kx_scan_padded(a.positions);
  Work w;
  w.inner = a.work;  // 16-byte pieces are read from here
  w.gamma = w.inner + rows * NB;
  w.end = w.gamma + rows;
  w.raw = w.end + rows;
  return w;
}

// one workgroup per (block, 16 heads of a group): thread (j, i) has the dot product of C_j and B_i, then goes through the heads
constexpr int HEADS = 16, BC_COLS = 64;
__global__ void __launch_bounds__(256) ssd_coef_k(KxSsdArgs a) {
  __shared__ float bs[NB][BC_COLS + 1], cs[NB][BC_COLS + 1], dt_s[HEADS][NB], a_s[HEADS][NB];
  const KxSsdSpec &s = a.s;
  const Work w = work_of(a);
  const int tid = threadIdx.x, i = tid & 15, j = tid >> 4, t0 = blockIdx.x * NB, b = blockIdx.z;
  const int ratio = s.heads / s.groups, per = (ratio + HEADS - 1) / HEADS, g = blockIdx.y / per, h0 = g * ratio + (blockIdx.y - g * per) * HEADS;
  const int heads = min(HEADS, (g + 1) * ratio - h0), C = kx_ssd_channels(s), N = s.state, padded = kx_scan_padded(a.positions);
  const float *rows = w.raw + kx_ssd_inner(s) + g * N;
  float dot = 0.0f;
  for (int n0 = 0; n0 < N; n0 += BC_COLS) {
    __syncthreads();
    for (int x = tid; x < 2 * NB * BC_COLS; x += 256) {
      const int d = n0 + x % BC_COLS, t = x / BC_COLS % NB;
      const bool c = x >= NB * BC_COLS, in = t0 + t < a.positions && d < N;
      const float v = in ? rows[((size_t)(t0 + t) * a.batch + b) * C + (c ? s.groups * N : 0) + d] : 0.0f;
      (c ? cs : bs)[t][x % BC_COLS] = v;
    }
    __syncthreads();
#pragma unroll 16
    for (int d = 0; d < BC_COLS; ++d) dot = __builtin_fmaf(cs[j][d], bs[i][d], dot);
  }
  {
    const int hh = j, h = h0 + min(hh, heads - 1);  // here a thread is (head, position)
    const bool in = t0 + i < a.positions;
    const float dt = in ? step_size(a, (size_t)(t0 + i) * a.batch + b, h) : 0.0f;
    dt_s[hh][i] = dt;
    a_s[hh][i] = in ? decay_of(a, h, dt) : 1.0f;  // a position past the end leaves the state as it is
  }
  __syncthreads();
  if (j < heads) {
    float gamma = 1.0f, end = dt_s[j][i];
    for (int t = 0; t <= i; ++t) gamma *= a_s[j][t];
    for (int t = i + 1; t < NB; ++t) end *= a_s[j][t];
    const size_t at = ((size_t)b * s.heads + h0 + j) * padded + t0 + i;
    w.gamma[at] = gamma;
    w.end[at] = end;
  }
  for (int hh = 0; hh < heads; ++hh) {
    float v = dot * dt_s[hh][i];
    for (int t = i + 1; t <= j; ++t) v *= a_s[hh][t];
    if (i == j) v += a.skip[h0 + hh];
    w.inner[(((size_t)b * s.heads + h0 + hh) * padded + t0 + j) * NB + i] = i <= j ? v : 0.0f;
  }
}

}  // namespace

int kx_ssd_launch(const KxSsdArgs &a, hipStream_t st) {
  const KxSsdSpec &s = a.s;
  KX_REQUIRE(s.heads > 0 && s.groups > 0 && s.heads % s.groups == 0 && s.state > 0 && s.state <= KX_SCAN_MAX_DIM && s.vdim > 0 && s.taps > 0,
             "state space: heads=%d groups=%d state=%d vdim=%d taps=%d", s.heads, s.groups, s.state, s.vdim, s.taps);
  KX_REQUIRE(a.batch > 0 && a.positions > 0 && (s.taps == 1 || (a.hist && a.hist_out && a.hist != a.hist_out)), "state space: %d x %d tokens", a.batch, a.positions);
  if (a.positions == 1) {
    const dim3 grid(s.heads * kx_cdiv(s.vdim, SC), a.batch);
    const KxConvArgs cv = conv_of(a);
    if (s.state <= 32) hipLaunchKernelGGL(ssd_step_k<4>, grid, dim3(256), 0, st, a, cv);
    else if (s.state <= 64) hipLaunchKernelGGL(ssd_step_k<8>, grid, dim3(256), 0, st, a, cv);
    else if (s.state <= 128) hipLaunchKernelGGL(ssd_step_k<16>, grid, dim3(256), 0, st, a, cv);
    else if (s.state <= 256) hipLaunchKernelGGL(ssd_step_k<32>, grid, dim3(256), 0, st, a, cv);
    else hipLaunchKernelGGL(ssd_step_k<64>, grid, dim3(256), 0, st, a, cv);
    KX_LAUNCH_CHECK();
    return KX_OK;
  }
  KX_REQUIRE(a.work && ((uintptr_t)a.work & 15) == 0, "state space: no scratch");
  const Work w = work_of(a);
  int rc = kx_conv_launch(conv_of(a), w.raw, st);
  if (rc) return rc;
  const int padded = kx_scan_padded(a.positions), ratio = s.heads / s.groups;
  hipLaunchKernelGGL(ssd_coef_k, dim3(padded / NB, s.groups * kx_cdiv(ratio, HEADS), a.batch), dim3(256), 0, st, a);
  KX_LAUNCH_CHECK();
  KxScanArgs c;
  const int C = kx_ssd_channels(s), inner = kx_ssd_inner(s);
  c.heads = s.heads; c.groups = s.groups; c.dim = s.state; c.vdim = s.vdim; c.batch = a.batch; c.positions = a.positions;
  c.k = w.raw + inner; c.q = c.k + s.groups * s.state; c.v = w.raw;
  c.q_ld = c.k_ld = c.v_ld = C;
  c.inner = w.inner; c.gamma = w.gamma; c.end = w.end;
  c.state = a.state; c.o = a.y;
  return kx_scan_launch(c, st);
}
