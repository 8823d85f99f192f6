// kx_scan.hip -- see kx_scan.h.  Everything here is 32-bit.  No counterpart in the reference, which has no recurrent layer.
//
// scan_k: a wave owns 16 columns of a head's state (or, with KS = 2, half of their rows), in registers as results of
// v_mfma_f32_16x16x4_f32, and goes through the blocks.  Register v of tile t is row 16 t + 4 (lane / 16) + v of column
// lane % 16, which is also what the second operand of that instruction holds if its four inner indices are taken to be those
// rows: the read-out S^T q uses the state as it lies, and the update's result lands where the state is.  The waves share a
// block's queries and keys, which are asked for two blocks ahead and go through registers into one of two LDS stages; values
// and block numbers stay in registers.  Barriers wait for LDS only: a block's read-outs are still on their way to memory
// when the next block begins.  With KS = 2 the second half's read-outs go through LDS to the first half's wave, which adds
// and stores them behind the block's barrier.
#include <algorithm>
#include <atomic>
#include "kx_common.h"
#include "kx_lds_copy.h"
#include "kx_scan.h"

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int NB = KX_SCAN_BLOCK;

template <int KT, bool CHANNEL, int KS>
constexpr size_t lds_floats() { return 2 * (2 * NB * (KT * 16 + 4) + (CHANNEL ? KT * 16 : 0) + (KS > 1 ? 4 / KS * 256 : 0)); }

template <int KT, bool CHANNEL, int KS>  // 16 KT >= dim
__global__ void __launch_bounds__(256) scan_k(KxScanArgs a) {
  constexpr int K = KT * 16, KW = KT / KS, COLS = 64 / KS, STR = K + 4, KEYS = 2 * NB * STR, STAGE = KEYS + (CHANNEL ? K : 0), NS = 2 * NB * K / 256, NT = (K + 255) / 256;
  static_assert(KT % KS == 0, "a wave has whole tiles");
  extern __shared__ __attribute__((aligned(16))) float sc_lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lj = lane & 15, g = lane >> 4;
  const int kw = wave % KS, cw = wave / KS, d0 = kw * KW * 16;  // this wave's rows of the state begin at d0
  // consecutive workgroups go to different XCDs: the heads of a group to one, so that its L2 holds their keys and queries
  const int h = a.heads % 8 ? blockIdx.y : blockIdx.y % 8 * (a.heads / 8) + blockIdx.y / 8, b = blockIdx.z, grp = h / (a.heads / a.groups), D = a.dim, V = a.vdim, n = a.positions;
  const int col = blockIdx.x * COLS + cw * 16 + lj, vcol = h * V + min(col, V - 1);
  const int padded = kx_scan_padded(n), blocks = padded / NB, HV = a.heads * V;
  const size_t hb = (size_t)b * a.heads + h;
  float *st = a.state + hb * D * V;
  f32x4 S[KW];
#pragma unroll
  for (int t = 0; t < KW; ++t)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int r = d0 + 16 * t + 4 * g + v;
      S[t][v] = r < D && col < V ? st[(size_t)r * V + col] : 0.0f;
    }
  // offsets from a block's first token; a block that is not whole repeats its last one
  int at_s[NS], at_v[4];
  auto offsets = [&](int last) {
#pragma unroll
    for (int x = 0; x < NS; ++x) {
      const int e = x * 256 + tid, t = min(e / K % NB, last), d = grp * D + min(e % K, D - 1);
      at_s[x] = t * a.batch * (x < NS / 2 ? a.q_ld : a.k_ld) + d;
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) at_v[v] = min(4 * g + v, last) * a.batch * a.v_ld + vcol;
  };
  offsets(min(NB, n) - 1);
  struct Block {  // of what is on its way
    float rs[NS], rt[NT], tot;
    f32x4 x, in, gam, end;
  } ahead[2];
  f32x4 xv, in, gam, end;
  float tot = 1.0f;
  auto fetch = [&](Block &f, int blk) {
    const int t0 = min(blk, blocks - 1) * NB;
    if (t0 + NB > n) offsets(n - 1 - t0);
    const size_t tok = (size_t)t0 * a.batch + b;
    const float *q = a.q + tok * a.q_ld, *k = a.k + tok * a.k_ld, *vv = a.v + tok * a.v_ld;
#pragma unroll
    for (int x = 0; x < NS; ++x) f.rs[x] = (x < NS / 2 ? q : k)[at_s[x]];
    if constexpr (CHANNEL)
#pragma unroll
      for (int x = 0; x < NT; ++x) f.rt[x] = a.total[(hb * blocks + t0 / NB) * D + min(x * 256 + tid, D - 1)];
#pragma unroll
    for (int v = 0; v < 4; ++v) f.x[v] = vv[at_v[v]];
    f.in = *(const f32x4 *)(a.inner + (hb * padded + t0 + lj) * NB + 4 * g);
    if constexpr (!CHANNEL) {
      f.gam = *(const f32x4 *)(a.gamma + hb * padded + t0 + 4 * g);
      f.end = *(const f32x4 *)(a.end + hb * padded + t0 + 4 * g);
      f.tot = a.gamma[hb * padded + t0 + NB - 1];
    }
  };
  auto put = [&](const Block &f, int blk, int stage) {
    float *s = sc_lds + stage * STAGE;
    if (D == K && (blk + 1) * NB <= n) {
#pragma unroll
      for (int x = 0; x < NS; ++x) s[(x * 256 + tid) / K * STR + (x * 256 + tid) % K] = f.rs[x];
    } else {
#pragma unroll
      for (int x = 0; x < NS; ++x) {
        const int e = x * 256 + tid;
        s[e / K * STR + e % K] = blk * NB + e / K % NB < n && e % K < D ? f.rs[x] : 0.0f;
      }
    }
    if constexpr (CHANNEL)
#pragma unroll
      for (int x = 0; x < NT; ++x)
        if (x * 256 + tid < K) s[KEYS + x * 256 + tid] = f.rt[x];
    xv = f.x;
    in = f.in;
    if constexpr (!CHANNEL) {
      gam = f.gam;
      end = f.end;
      tot = f.tot;
    }
  };
  f32x4 *xo = (f32x4 *)(sc_lds + 2 * STAGE);  // [2][column waves][64]: read-outs of the second half
  f32x4 yp = {0.0f, 0.0f, 0.0f, 0.0f};
  auto store = [&](const f32x4 &y, int blk) {
    float *o = a.o + ((size_t)blk * NB * a.batch + b) * HV;
    if ((blk + 1) * NB <= n && (int)blockIdx.x * COLS + COLS <= V) {
#pragma unroll
      for (int v = 0; v < 4; ++v) o[(4 * g + v) * a.batch * HV + vcol] = y[v];
    } else {
#pragma unroll
      for (int v = 0; v < 4; ++v)
        if (blk * NB + 4 * g + v < n && col < V) o[(4 * g + v) * a.batch * HV + vcol] = y[v];
    }
  };
  auto work = [&](int blk, int stage) {
    const float *q = sc_lds + stage * STAGE + d0, *k = q + NB * STR, *w = sc_lds + stage * STAGE + KEYS + d0;
    if (KS > 1 && kw == 0 && blk > 0) store(yp + xo[((stage ^ 1) * (4 / KS) + cw) * 64 + lane], blk - 1);
    f32x4 o[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}}, xe;
#pragma unroll
    for (int v = 0; v < 4; ++v) xe[v] = CHANNEL ? xv[v] : xv[v] * end[v];
#pragma unroll
    for (int t = 0; t < KW; ++t) {
      const f32x4 qq = *(const f32x4 *)(q + lj * STR + 16 * t + 4 * g);
      f32x4 ss = S[t];
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        if constexpr (!CHANNEL) ss[v] *= tot;
      }
      if constexpr (CHANNEL) {
        const f32x4 ww = *(const f32x4 *)(w + 16 * t + 4 * g);
#pragma unroll
        for (int v = 0; v < 4; ++v) ss[v] *= ww[v];
      }
#pragma unroll
      for (int v = 0; v < 4; ++v) {  // two chains in turn
        o[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(qq[v], S[t][v], o[t & 1], 0, 0, 0);
        ss = __builtin_amdgcn_mfma_f32_16x16x4f32(k[(4 * g + v) * STR + 16 * t + lj], xe[v], ss, 0, 0, 0);
      }
      S[t] = ss;
    }
    f32x4 y;
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      y[v] = o[0][v] + o[1][v];
      if (!CHANNEL) y[v] *= gam[v];
    }
    if (KS == 1 || kw == 0)
#pragma unroll
      for (int v = 0; v < 4; ++v) y = __builtin_amdgcn_mfma_f32_16x16x4f32(in[v], xv[v], y, 0, 0, 0);
    if (KS == 1) store(y, blk);
    else if (kw == 0) yp = y;
    else xo[(stage * (4 / KS) + cw) * 64 + lane] = y;
  };
  fetch(ahead[0], 0);
  fetch(ahead[1], 1);
  put(ahead[0], 0, 0);
  kx_lds_barrier();
  for (int blk = 0; blk < blocks; blk += 2) {
    fetch(ahead[0], blk + 2);
    work(blk, 0);
    put(ahead[1], blk + 1, 1);
    kx_lds_barrier();
    if (blk + 1 >= blocks) break;
    fetch(ahead[1], blk + 3);
    work(blk + 1, 1);
    put(ahead[0], blk + 2, 0);
    kx_lds_barrier();
  }
  if (KS > 1 && kw == 0) store(yp + xo[(((blocks - 1) & 1) * (4 / KS) + cw) * 64 + lane], blocks - 1);
#pragma unroll
  for (int t = 0; t < KW; ++t)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int r = d0 + 16 * t + 4 * g + v;
      if (r < D && col < V) st[(size_t)r * V + col] = S[t][v];
    }
}

template <int KT, bool CHANNEL, int KS>
int scan_ks(const KxScanArgs &a, hipStream_t st) {
  constexpr size_t lds = lds_floats<KT, CHANNEL, KS>() * 4;
  static_assert(lds <= 160 * 1024, "a block's keys and queries fit a workgroup");
  static std::atomic<bool> attr{false};
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)scan_k<KT, CHANNEL, KS>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    attr = true;
  }
  hipLaunchKernelGGL((scan_k<KT, CHANNEL, KS>), dim3(kx_cdiv(a.vdim, 64 / KS), a.heads, a.batch), dim3(256), lds, st, a);
  KX_LAUNCH_CHECK();
  return KX_OK;
}
// halves of the state's rows on two waves where whole columns would leave CUs without work
template <int KT, bool CHANNEL>
int scan(const KxScanArgs &a, hipStream_t st) {
  if constexpr (KT % 2 == 0)
    if ((long)kx_cdiv(a.vdim, 64) * a.heads * a.batch < kx_device_cus()) return scan_ks<KT, CHANNEL, 2>(a, st);
  return scan_ks<KT, CHANNEL, 1>(a, st);
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
  KX_REQUIRE((int64_t)a.batch * NB * (std::max(std::max(a.q_ld, a.k_ld), std::max(a.v_ld, a.heads * a.vdim))) < ((int64_t)1 << 31), "recurrence: rows of a block too far apart");
  return a.channel ? scan_dim<true>(a, st) : scan_dim<false>(a, st);
}
