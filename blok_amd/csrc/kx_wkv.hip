// kx_wkv.hip -- see kx_wkv.h.  The recurrence and everything that enters it is 32-bit.  No counterpart in the reference.
//
// One token per sequence: wkv_step_k.  A workgroup owns 32 columns of one head's state and makes the head's decays itself.
// Several positions: the decays' second product (kx_linear.hip), wkv_coef_k and kx_scan.hip.  With W(i, j) the product per
// channel of the decays of tokens i .. j of a block, the block's numbers are
//   q_j = r_j W(1, j - 1),  k_i W(i + 1, 16),  total = W(1, 16),
//   inner[j][i] = sum_c r_jc k_ic W_c(i + 1, j - 1) for i < j,  inner[j][j] = sum_c r_jc u_c k_jc:
// products of decays only, none is divided by another.
#include <atomic>
#include "kx_common.h"
#include "kx_rows.h"
#include "kx_wkv.h"

namespace {

constexpr int SC = 32;  // columns per workgroup of wkv_step_k
constexpr int NB = KX_SCAN_BLOCK;

template <class T, int RPT>  // rows of the state per thread
__global__ void __launch_bounds__(256) wkv_step_k(KxWkvArgs a) {
  using E = kxr::Elem<T>;
  extern __shared__ float th[];  // [w2.ld]: tanh of the low-rank projection, zeros behind it
  __shared__ float rs[8 * RPT], ks[8 * RPT], us[8 * RPT], ws[8 * RPT], part[8][SC];
  const int D = a.s.dim, tid = threadIdx.x, lane = tid & 63, slices = (D + SC - 1) / SC;
  const int h = blockIdx.x / slices, c0 = (blockIdx.x - h * slices) * SC, b = blockIdx.y;
  const int c = tid & (SC - 1), rg = tid / SC, col = min(c0 + c, D - 1);
  const float *pr = a.proj + (size_t)b * a.proj_ld;
  float *st = a.state + ((size_t)b * a.s.heads + h) * D * D;
  float S[RPT];
#pragma unroll
  for (int r = 0; r < RPT; ++r) S[r] = st[(size_t)min(rg + 8 * r, D - 1) * D + col];
  for (int x = tid; x < a.w2.ld; x += 256) th[x] = x < a.s.rank ? tanhf(pr[a.w_off + x]) : 0.0f;
  for (int d = tid; d < D; d += 256) {
    rs[d] = pr[a.r_off + h * D + d];
    ks[d] = pr[a.k_off + h * D + d];
    us[d] = a.u[h * D + d];
  }
  const float v = pr[a.v_off + h * D + col];
  __syncthreads();
  const int l8 = lane & 7;
  for (int d0 = 0; d0 < D; d0 += 32) {  // eight lanes per channel
    const int d = d0 + (tid >> 3);
    const T *w2 = (const T *)a.w2.w + (size_t)(h * D + min(d, D - 1)) * a.w2.ld;
    float y = 0.0f;
    for (int x = l8 * 8; x < a.w2.ld; x += 64) {
      float f[8];
      E::unpack(f, E::cached(w2 + x));
#pragma unroll
      for (int e = 0; e < 8; ++e) y = __builtin_fmaf(f[e], th[x + e], y);
    }
    y += kxw::dpp_f<kxw::DPP_QUAD_XOR1>(y);
    y += kxw::dpp_f<kxw::DPP_QUAD_XOR2>(y);
    y += kxw::dpp_f<kxw::DPP_ROW_HALF_MIRROR>(y);
    if (l8 == 0 && d < D) ws[d] = kx_expf(-kx_expf(y + a.w0[h * D + d]));
  }
  __syncthreads();
  float o = 0.0f;
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int row = rg + 8 * r;
    if (row < D) {
      const float kv = ks[row] * v;
      o = __builtin_fmaf(rs[row], __builtin_fmaf(us[row], kv, S[r]), o);
      if (c0 + c < D) st[(size_t)row * D + c0 + c] = __builtin_fmaf(ws[row], S[r], kv);
    }
  }
  part[rg][c] = o;
  __syncthreads();
  if (rg == 0 && c0 + c < D) {
    o = part[0][c];
#pragma unroll
    for (int j = 1; j < 8; ++j) o += part[j][c];
    a.o[((size_t)b * a.s.heads + h) * D + c0 + c] = o;
  }
}

struct Work {
  float *inner, *total, *wl, *q, *k;
};
__host__ __device__ __forceinline__ Work work_of(const KxWkvArgs &a) {
  const size_t padded = kx_scan_padded(a.positions), hd = (size_t)a.s.heads * a.s.dim, tokens = (size_t)a.batch * a.positions;
  Work w;
  w.inner = a.work;  // 16-byte pieces are read from here
  w.total = w.inner + a.batch * padded * a.s.heads * NB;
  w.wl = w.total + a.batch * padded / NB * hd;  // the decays' logarithms of logarithms, without w0
  w.q = w.wl + tokens * hd;
  w.k = w.q + tokens * hd;
  return w;
}

// One workgroup per (block, head): thread (j, s) goes through token j's channels s, s + 16, ...  Keys and decays have NB - 1 rows
// of zeros in front, which the tokens before the block are.
__host__ __device__ constexpr int coef_stride(int dim) { return dim + (dim < KX_SCAN_MAX_DIM ? 16 : 4); }
constexpr size_t coef_lds(int dim) { return (size_t)(5 * NB - 2) * coef_stride(dim) * 4; }
__global__ void __launch_bounds__(256) wkv_coef_k(KxWkvArgs a) {
  extern __shared__ float cf_lds[];
  const int D = a.s.dim, STR = coef_stride(D), tid = threadIdx.x, sl = tid & 15, j = tid >> 4;
  const int t0 = blockIdx.x * NB, h = blockIdx.y, b = blockIdx.z, padded = kx_scan_padded(a.positions);
  const Work w = work_of(a);
  const int HD = a.s.heads * D;
  float *rs = cf_lds, *ks = rs + (2 * NB - 1) * STR, *ws = ks + (2 * NB - 1) * STR;  // row 0 is the block's first token
  for (int x = tid; x < (NB - 1) * STR; x += 256) {
    rs[NB * STR + x] = 0.0f;
    ks[NB * STR + x] = 0.0f;
  }
#pragma unroll 4
  for (int x = tid; x < NB * D; x += 256) {
    const int t = x / D, d = x - t * D;
    const bool in = t0 + t < a.positions;
    const size_t tok = (size_t)min(t0 + t, a.positions - 1) * a.batch + b;
    const float *pr = a.proj + tok * a.proj_ld;
    const float r = pr[a.r_off + h * D + d], k = pr[a.k_off + h * D + d], y = w.wl[tok * HD + h * D + d];
    rs[t * STR + d] = in ? r : 0.0f;
    ks[t * STR + d] = in ? k : 0.0f;
    ws[t * STR + d] = in ? kx_expf(-kx_expf(y + a.w0[h * D + d])) : 1.0f;  // a position past the end leaves the state as it is
  }
  __syncthreads();
  float acc[NB] = {};  // of token j - d
  for (int c = sl; c < D; c += 16) {
    float p = rs[j * STR + c];
    const float *k = ks + j * STR + c, *wt = ws + j * STR + c;
    acc[0] = __builtin_fmaf(p * a.u[h * D + c], k[0], acc[0]);
#pragma unroll
    for (int d = 1; d < NB; ++d) {
      acc[d] = __builtin_fmaf(p, k[-d * STR], acc[d]);
      p *= wt[-d * STR];
    }
  }
  float mine = 0.0f;  // lane s holds i = s
#pragma unroll
  for (int d = 0; d < NB; ++d) {
    float v = acc[d];
    v += kxw::dpp_f<kxw::DPP_QUAD_XOR1>(v);
    v += kxw::dpp_f<kxw::DPP_QUAD_XOR2>(v);
    v += kxw::dpp_f<kxw::DPP_ROW_HALF_MIRROR>(v);
    v += kxw::dpp_f<kxw::DPP_ROW_MIRROR>(v);
    if (j - d == sl) mine = v;
  }
  w.inner[(((size_t)b * a.s.heads + h) * padded + t0 + j) * NB + sl] = mine;
  constexpr int Q = 4, PER = NB / Q;  // a thread has a quarter of the block's tokens of one channel
  for (int x = tid; x < Q * D; x += 256) {
    const int quarter = x / D, c = x - quarter * D, first = quarter * PER;
    float dec[NB], p = 1.0f, s = 1.0f;
#pragma unroll
    for (int t = 0; t < NB; ++t) dec[t] = ws[t * STR + c];
#pragma unroll
    for (int t = 0; t < NB; ++t) {
      p *= t < first ? dec[t] : 1.0f;
      s *= t >= first + PER ? dec[t] : 1.0f;
    }
#pragma unroll
    for (int y = 0; y < PER; ++y) {
      const int t = first + y, u = first + PER - 1 - y;
      if (t0 + t < a.positions) w.q[((size_t)(t0 + t) * a.batch + b) * HD + h * D + c] = rs[t * STR + c] * p;
      if (t0 + u < a.positions) w.k[((size_t)(t0 + u) * a.batch + b) * HD + h * D + c] = ks[u * STR + c] * s;
      p *= ws[t * STR + c];
      s *= ws[u * STR + c];
    }
    if (quarter == Q - 1) w.total[(((size_t)b * a.s.heads + h) * (padded / NB) + blockIdx.x) * D + c] = p;
  }
}

template <class T>
int step(const KxWkvArgs &a, hipStream_t st) {
  const dim3 grid(a.s.heads * kx_cdiv(a.s.dim, SC), a.batch);
  const size_t lds = (size_t)a.w2.ld * 4;
  KX_REQUIRE(lds <= 32 * 1024, "time mixing: a decay projection of rank %d", a.s.rank);
  if (a.s.dim <= 32) hipLaunchKernelGGL((wkv_step_k<T, 4>), grid, dim3(256), lds, st, a);
  else if (a.s.dim <= 64) hipLaunchKernelGGL((wkv_step_k<T, 8>), grid, dim3(256), lds, st, a);
  else if (a.s.dim <= 128) hipLaunchKernelGGL((wkv_step_k<T, 16>), grid, dim3(256), lds, st, a);
  else if (a.s.dim <= 256) hipLaunchKernelGGL((wkv_step_k<T, 32>), grid, dim3(256), lds, st, a);
  else hipLaunchKernelGGL((wkv_step_k<T, 64>), grid, dim3(256), lds, st, a);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

}  // namespace

int kx_wkv_launch(bool f32, const KxWkvArgs &a, hipStream_t st) {
  const KxWkvSpec &s = a.s;
  KX_REQUIRE(s.heads > 0 && s.dim > 0 && s.dim <= KX_SCAN_MAX_DIM && s.rank > 0 && a.w2.rows == s.heads * s.dim && a.w2.cols == s.rank,
             "time mixing: heads=%d dim=%d rank=%d", s.heads, s.dim, s.rank);
  KX_REQUIRE(a.batch > 0 && a.positions > 0, "time mixing: %d x %d tokens", a.batch, a.positions);
  if (a.positions == 1) return f32 ? step<float>(a, st) : step<uint16_t>(a, st);
  KX_REQUIRE(a.work && ((uintptr_t)a.work & 15) == 0 && a.rows, "time mixing: no scratch");
  const Work w = work_of(a);
  const int hd = s.heads * s.dim, padded = kx_scan_padded(a.positions);
  KxLinArgs g;
  g.m = a.w2;
  g.tokens = a.batch * a.positions;
  g.row.kind = KX_ROW_TANH; g.row.cols = s.rank; g.row.streams = a.proj + a.w_off; g.row.streams_ld = a.proj_ld;
  g.out = w.wl;
  g.out_ld = hd;
  int rc = kx_linear_launch(f32, g, a.rows, st);
  if (rc) return rc;
  const size_t lds = coef_lds(s.dim);
  static std::atomic<bool> attr{false};
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)wkv_coef_k, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
    attr = true;
  }
  hipLaunchKernelGGL(wkv_coef_k, dim3(padded / NB, s.heads, a.batch), dim3(256), lds, st, a);
  KX_LAUNCH_CHECK();
  KxScanArgs c;
  c.heads = c.groups = s.heads; c.dim = c.vdim = s.dim; c.batch = a.batch; c.positions = a.positions; c.channel = true;
  c.q = w.q; c.k = w.k; c.q_ld = c.k_ld = hd;
  c.v = a.proj + a.v_off; c.v_ld = a.proj_ld;
  c.inner = w.inner; c.total = w.total;
  c.state = a.state; c.o = a.o;
  return kx_scan_launch(c, st);
}
