// kx_scan.hip -- see kx_scan.h.  Everything here is 32-bit.  No counterpart in the reference, which has no recurrent layer.
//
// scan_k: a wave owns 16 columns of a head's state, in registers as results of v_mfma_f32_16x16x4_f32, and goes through the
// blocks.  Register v of tile t is row 16 t + 4 (lane / 16) + v of column lane % 16, which is also what the second operand of
// that instruction holds if its four inner indices are taken to be those rows: the read-out S^T q uses the state as it
// lies, and the update's result lands where the state is.  Four waves share a block's queries and keys, which go through
// registers into one of two LDS stages while the other is worked on; values and block numbers go straight to registers.
#include <atomic>
#include "kx_common.h"
#include "kx_scan.h"

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int NB = KX_SCAN_BLOCK, COLS = 64;

template <int KT, bool CHANNEL>
constexpr size_t lds_floats() { return 2 * (2 * NB * (KT * 16 + 4) + (CHANNEL ? KT * 16 : 0)); }

template <int KT, bool CHANNEL>  // 16 KT >= dim
__global__ void __launch_bounds__(256) scan_k(KxScanArgs a) {
  constexpr int K = KT * 16, STR = K + 4, STAGE = 2 * NB * STR + (CHANNEL ? K : 0), NS = 2 * NB * K / 256, NT = (K + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) float sc_lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lj = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, b = blockIdx.z, grp = h / (a.heads / a.groups), D = a.dim, V = a.vdim, n = a.positions;
  const int col = blockIdx.x * COLS + wave * 16 + lj, vcol = h * V + min(col, V - 1);
  const int padded = kx_scan_padded(n), blocks = padded / NB;
  const size_t hb = (size_t)b * a.heads + h;
  float *st = a.state + hb * D * V;
  f32x4 S[KT];
#pragma unroll
  for (int t = 0; t < KT; ++t)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int r = 16 * t + 4 * g + v;
      S[t][v] = r < D && col < V ? st[(size_t)r * V + col] : 0.0f;
    }
  float rs[NS], rt[NT];
  f32x4 xv, in, gam, end, xn, inn, gamn, endn;
  float tot = 1.0f, totn = 1.0f;
  auto fetch = [&](int blk) {
    const int t0 = blk * NB;
#pragma unroll
    for (int x = 0; x < NS; ++x) {
      const int at = x * 256 + tid, d = at % K, t = t0 + at / K % NB;
      const bool key = at >= NB * K;
      const size_t tok = (size_t)min(t, n - 1) * a.batch + b;
      const float y = key ? a.k[tok * a.k_ld + grp * D + min(d, D - 1)] : a.q[tok * a.q_ld + grp * D + min(d, D - 1)];
      rs[x] = t < n && d < D ? y : 0.0f;
    }
    if constexpr (CHANNEL)
#pragma unroll
      for (int x = 0; x < NT; ++x) {
        const int d = x * 256 + tid;
        rt[x] = d < D ? a.total[(hb * blocks + blk) * D + d] : 1.0f;
      }
#pragma unroll
    for (int v = 0; v < 4; ++v) xn[v] = a.v[((size_t)min(t0 + 4 * g + v, n - 1) * a.batch + b) * a.v_ld + vcol];
    inn = *(const f32x4 *)(a.inner + (hb * padded + t0 + lj) * NB + 4 * g);
    if constexpr (!CHANNEL) {
      gamn = *(const f32x4 *)(a.gamma + hb * padded + t0 + 4 * g);
      endn = *(const f32x4 *)(a.end + hb * padded + t0 + 4 * g);
      totn = a.gamma[hb * padded + t0 + NB - 1];
    }
  };
  auto put = [&](int stage) {
    float *s = sc_lds + stage * STAGE;
#pragma unroll
    for (int x = 0; x < NS; ++x) {
      const int at = x * 256 + tid;
      s[at / K * STR + at % K] = rs[x];
    }
    if constexpr (CHANNEL)
#pragma unroll
      for (int x = 0; x < NT; ++x)
        if (x * 256 + tid < K) s[2 * NB * STR + x * 256 + tid] = rt[x];
    xv = xn;
    in = inn;
    gam = gamn;
    end = endn;
    tot = totn;
  };
  fetch(0);
  put(0);
  __syncthreads();
  for (int blk = 0, stage = 0; blk < blocks; ++blk, stage ^= 1) {
    fetch(min(blk + 1, blocks - 1));
    const float *q = sc_lds + stage * STAGE, *k = q + NB * STR, *w = k + NB * STR;
    f32x4 o[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}};
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      const f32x4 qq = *(const f32x4 *)(q + lj * STR + 16 * t + 4 * g);
#pragma unroll
      for (int v = 0; v < 4; ++v) o[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(qq[v], S[t][v], o[t & 1], 0, 0, 0);
    }
    f32x4 y, xe;
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      y[v] = o[0][v] + o[1][v];
      if (!CHANNEL) y[v] *= gam[v];
      xe[v] = CHANNEL ? xv[v] : xv[v] * end[v];
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) y = __builtin_amdgcn_mfma_f32_16x16x4f32(in[v], xv[v], y, 0, 0, 0);
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      if constexpr (CHANNEL) {
        const f32x4 ww = *(const f32x4 *)(w + 16 * t + 4 * g);
#pragma unroll
        for (int v = 0; v < 4; ++v) S[t][v] *= ww[v];
      } else {
#pragma unroll
        for (int v = 0; v < 4; ++v) S[t][v] *= tot;
      }
#pragma unroll
      for (int v = 0; v < 4; ++v) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[(4 * g + v) * STR + 16 * t + lj], xe[v], S[t], 0, 0, 0);
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int t = blk * NB + 4 * g + v;
      if (t < n && col < V) a.o[((size_t)t * a.batch + b) * a.heads * V + vcol] = y[v];
    }
    put(stage ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < KT; ++t)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int r = 16 * t + 4 * g + v;
      if (r < D && col < V) st[(size_t)r * V + col] = S[t][v];
    }
}

template <int KT, bool CHANNEL>
int scan(const KxScanArgs &a, hipStream_t st) {
  constexpr size_t lds = lds_floats<KT, CHANNEL>() * 4;
  static_assert(lds <= 160 * 1024, "a block's keys and queries fit a workgroup");
  static std::atomic<bool> attr{false};
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)scan_k<KT, CHANNEL>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    attr = true;
  }
  hipLaunchKernelGGL((scan_k<KT, CHANNEL>), dim3(kx_cdiv(a.vdim, COLS), a.heads, a.batch), dim3(256), lds, st, a);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

template <bool CHANNEL>
int scan_dim(const KxScanArgs &a, hipStream_t st) {
  const int kt = kx_cdiv(a.dim, 16);
  if (kt <= 1) return scan<1, CHANNEL>(a, st);
  if (kt <= 2) return scan<2, CHANNEL>(a, st);
  if (kt <= 3) return scan<3, CHANNEL>(a, st);
  if (kt <= 4) return scan<4, CHANNEL>(a, st);
  if (kt <= 6) return scan<6, CHANNEL>(a, st);
  if (kt <= 8) return scan<8, CHANNEL>(a, st);
  if (kt <= 16) return scan<16, CHANNEL>(a, st);
  return scan<32, CHANNEL>(a, st);
}

}  // namespace

int kx_scan_launch(const KxScanArgs &a, hipStream_t st) {
  KX_REQUIRE(a.heads > 0 && a.groups > 0 && a.heads % a.groups == 0 && a.dim > 0 && a.dim <= KX_SCAN_MAX_DIM && a.vdim > 0 && a.batch > 0 && a.positions > 0,
             "recurrence: heads=%d groups=%d dim=%d vdim=%d, %d x %d tokens", a.heads, a.groups, a.dim, a.vdim, a.batch, a.positions);
  KX_REQUIRE(a.q && a.k && a.v && a.inner && a.state && a.o && (a.channel ? a.total != nullptr : a.gamma && a.end), "recurrence: null argument");
  return a.channel ? scan_dim<true>(a, st) : scan_dim<false>(a, st);
}
