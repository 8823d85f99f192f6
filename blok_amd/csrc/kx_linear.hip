// kx_linear.hip -- matrix products of the hybrid decoder, y[t][r] = sum_k x[t][k] w[r][k].
//
// The counterpart of matvec_bf16_k / matvec_bf16_f32_k and the kernels around them (src/kimi_exec.cu:248-298) for a
// decoder whose shapes come from its config.json: nothing here asks for a multiple of 512 columns.
//
// lin_gemv_k (up to 4 tokens): a workgroup of 8 waves builds the activation rows in LDS (kx_rows.h: residual streams
// and norm, or the gated read-out of the delta rule) while the first weight loads are under way, then every wave
// streams two rows of the matrix at a time, 8 columns per lane and load, the next pieces in flight while the present
// ones are multiplied; the epilogue stores the product, forms the gated activation of a (gate, up) pair, or updates
// all residual streams of the row.
// lin_gemm_k (bf16, more tokens): tiles of BM tokens x 128 rows, v_mfma_f32_32x32x16_bf16, both operands staged through
// LDS by global -> LDS copies in blocks of 64 columns, two stages, 16-byte pieces xor-swizzled by the row.
// lin_gemm_f32_k (f32): tiles of 64 x 64 on the vector ALU; true 32-bit products.
#include <algorithm>
#include <atomic>
#include "kx_common.h"
#include "kx_lds_copy.h"
#include "kx_linear.h"
#include "kx_rows.h"

namespace {

using kxr::Elem;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

// ---- epilogues, one output element (or pair) at a time ----
template <class T>
__device__ __forceinline__ void put_glu(const KxLinArgs &a, int t, int col, float g, float u) {
  g = fminf(g, a.limit);
  u = fminf(fmaxf(u, -a.limit), a.limit);
  ((T *)a.mid)[(size_t)t * a.mid_ld + col] = Elem<T>::make(g * kxr::sigmoid_for<T>(a.alpha * g) * (u + a.bias));
}
// EPI of the kernels: KX_LIN_F32, KX_LIN_GLU, or KX_LIN_STREAMS + number of streams (streams_any: up to KX_MAX_STREAMS)
constexpr int STREAMS_ANY = KX_LIN_STREAMS + KX_MAX_STREAMS;
__host__ __device__ constexpr int most_streams(int epi) { return epi > KX_LIN_STREAMS ? epi - KX_LIN_STREAMS : 1; }
// The streams of one element of the residual row, read early and written late.  The small matrices come through the scalar
// cache: every lane uses the same numbers and nothing writes them.
typedef const __attribute__((address_space(4))) float *ScalarPtr;
template <int EPI>
struct Streams {
  static constexpr int S = most_streams(EPI);
  float old[S];
  static __device__ __forceinline__ bool has(const KxLinArgs &a, int s) { return EPI != STREAMS_ANY || s < a.n_streams; }
  __device__ __forceinline__ void load(const KxLinArgs &a, int t, int r) {
    const float *x = a.streams + (size_t)t * a.n_streams * a.m.rows + r;
#pragma unroll
    for (int s = 0; s < S; ++s) old[s] = x[(size_t)(has(a, s) ? s : 0) * a.m.rows];
  }
  __device__ __forceinline__ void store(const KxLinArgs &a, int t, int r, float y) const {
    float *x = a.streams + (size_t)t * a.n_streams * a.m.rows + r;
    if (!a.mix) {
      *x = old[0] + y;
      return;
    }
    const ScalarPtr mix = (ScalarPtr)a.mix, outw = (ScalarPtr)a.outw;
    const int n = EPI == STREAMS_ANY ? a.n_streams : S;
#pragma unroll
    for (int d = 0; d < S; ++d) {
      if (has(a, d)) {
        float v = outw[d] * y;
#pragma unroll
        for (int s = 0; s < S; ++s)
          if (has(a, s)) v = __builtin_fmaf(mix[s * n + d], old[s], v);
        x[(size_t)d * a.m.rows] = v;
      }
    }
  }
};

// matrix row of half i (0, 1) of unit k: a (gate, up) pair, or two consecutive rows
template <int EPI>
__device__ __forceinline__ int unit_row(int k, int i) {
  return EPI == KX_LIN_GLU ? (k / KX_GLU_BLOCK) * (2 * KX_GLU_BLOCK) + (k % KX_GLU_BLOCK) + i * KX_GLU_BLOCK : 2 * k + i;
}

constexpr int GEMV_WAVES = 8, UP = 4;  // UP: pieces per row in flight
__host__ __device__ __forceinline__ int gemv_row(int ld) { return (ld + 64 * UP * 8 - 1) / (64 * UP * 8) * (64 * UP * 8); }

template <class T, int NT, int EPI>
__global__ void __launch_bounds__(GEMV_WAVES * 64) __attribute__((amdgpu_waves_per_eu(sizeof(T) == 2 ? 4 : 2)))
lin_gemv_k(KxLinArgs a) {
  using E = Elem<T>;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  __shared__ float red[GEMV_WAVES][2 * NT];
  const int xl = gemv_row(a.m.ld);                          // a row in LDS, with zeros up to whole passes of the wave
  T *xs = (T *)lds;                                         // [NT][xl]
  float *u = (float *)(lds + (size_t)NT * xl * sizeof(T));  // row scratch
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int ld = a.m.ld, np = ld >> 3, nc = (np + 64 * UP - 1) / (64 * UP);
  const int units = (a.m.rows + 1) >> 1, nblk = (units + GEMV_WAVES - 1) / GEMV_WAVES;
  const T *w = (const T *)a.m.w;
  typename E::Raw bufA[2][UP], bufB[2][UP];
  // Past the last block the first row is asked for once more, by every wave: the number of loads in flight has to be the
  // same on every path, or the compiler waits for all of them.
  auto load = [&](typename E::Raw (&b)[2][UP], int blk, int c) {
    const int k = blk < nblk ? min(blk * GEMV_WAVES + wave, units - 1) : 0;
    if (blk >= nblk) c = 0;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const T *wr = w + (size_t)min(unit_row<EPI>(k, i), a.m.rows - 1) * ld;
#pragma unroll
      for (int j = 0; j < UP; ++j) {
        const int p = (c * UP + j) * 64 + lane;
        b[i][j] = E::stream(wr + min(p, np - 1) * 8);  // a lane past the row meets zeros
      }
    }
  };
  int blk = blockIdx.x, c = 0;
  load(bufA, blk, 0);
#pragma unroll
  for (int t = 0; t < NT; ++t)
    if (t < a.tokens) {
      for (int x = ld + threadIdx.x; x < xl; x += GEMV_WAVES * 64) xs[(size_t)t * xl + x] = E::make(0.0f);
      kxr::build_row<T>(a.row, t, xs + (size_t)t * xl, ld, u);
    }
  float acc[2 * NT];
#pragma unroll
  for (int v = 0; v < 2 * NT; ++v) acc[v] = 0.0f;
  auto step = [&](typename E::Raw (&cur)[2][UP], typename E::Raw (&nxt)[2][UP]) {  // one chunk of columns of one unit per wave
    const bool last = c + 1 == nc;
    const int nblk_ = last ? blk + gridDim.x : blk, nc_ = last ? 0 : c + 1;
    // lane i * NT + t < 2 NT finishes row i of the unit for token t; what it updates is asked for ahead of the next weights
    const int unit = blk * GEMV_WAVES + wave, row = unit_row<EPI>(unit, lane / NT & 1), tok = NT > 1 ? lane % NT : 0;
    const bool finish = EPI == KX_LIN_GLU ? lane < NT && tok < a.tokens && unit < units : lane < 2 * NT && row < a.m.rows && tok < a.tokens;
    Streams<EPI> res;
    if (EPI >= KX_LIN_STREAMS && last && finish) res.load(a, tok, row);
    load(nxt, nblk_, nc_);
    __builtin_amdgcn_sched_barrier(0);  // these loads are on their way before the last ones are waited for
#pragma unroll
    for (int j = 0; j < UP; ++j) {
      const int p = (c * UP + j) * 64 + lane;
      float wf[2][8];
      E::unpack(wf[0], cur[0][j]);
      E::unpack(wf[1], cur[1][j]);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        float xf[8];
        E::unpack(xf, E::cached(xs + (size_t)(NT > 1 ? min(t, a.tokens - 1) : 0) * xl + p * 8));
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          acc[t] = __builtin_fmaf(wf[0][e], xf[e], acc[t]);
          acc[NT + t] = __builtin_fmaf(wf[1][e], xf[e], acc[NT + t]);
        }
      }
    }
    if (last) {
      kxw::reduce<2 * NT, 64>(acc, lane);
      if (kxw::reduce_writer<2 * NT, 64>(lane))
#pragma unroll
        for (int j = 0; j < kxw::reduce_out<2 * NT, 64>(); ++j) red[wave][kxw::reduce_index<2 * NT, 64>(lane, j)] = acc[j];
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // the wave reads its own sums back
      if (finish) {
        if constexpr (EPI == KX_LIN_GLU) put_glu<T>(a, tok, unit, red[wave][lane], red[wave][NT + lane]);
        else if constexpr (EPI == KX_LIN_F32) a.out[(size_t)tok * a.out_ld + row] = red[wave][lane];
        else res.store(a, tok, row, red[wave][lane]);
      }
      asm volatile("" ::: "memory");
#pragma unroll
      for (int v = 0; v < 2 * NT; ++v) acc[v] = 0.0f;
    }
    blk = nblk_;
    c = nc_;
  };
  for (;;) {
    step(bufA, bufB);
    if (blk >= nblk) break;
    step(bufB, bufA);
    if (blk >= nblk) break;
  }
}

template <class T>
__global__ void __launch_bounds__(256) row_k(KxRowArgs a, T *out, int ld) {
  extern __shared__ float row_lds[];
  kxr::build_row<T>(a, blockIdx.x, out + (size_t)blockIdx.x * ld, ld, row_lds);
}

// ---- bf16 GEMM ----
// 4 waves as 2 x 2: wave (wm, wn) owns MI blocks of 32 tokens and 64 rows (two blocks of 32: with GLU rows, gate and up).
template <int MI, int EPI>
__global__ void __launch_bounds__(256, 2) lin_gemm_k(KxLinArgs a, const uint16_t *__restrict__ x, int x_ld) {
  constexpr int BM = MI * 64, BN = 128, ROWS = BM + BN, STAGE = ROWS * 128, CPW = ROWS / 32;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  const uint32_t lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) uint8_t *)lds;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int wm = wave >> 1, wn = wave & 1, lr = lane & 31, h = lane >> 5;
  const int m0 = blockIdx.y * BM, n0 = blockIdx.x * BN;
  const int nb = a.m.ld >> 6;  // blocks of 64 columns
  // copy instruction i of this wave moves 8 rows of 128 bytes: lane l the piece (l % 8) ^ (row % 8) of row l / 8
  const uint16_t *src[CPW];
  uint32_t dst[CPW];
#pragma unroll
  for (int i = 0; i < CPW; ++i) {
    const int r0 = (i * 4 + wave) * 8, row = r0 + (lane >> 3), piece = (lane & 7) ^ (row & 7);
    src[i] = (row < BM ? x + (size_t)min(m0 + row, a.tokens - 1) * x_ld
                       : (const uint16_t *)a.m.w + (size_t)min(n0 + row - BM, a.m.rows - 1) * a.m.ld) + piece * 8;
    dst[i] = r0 * 128;
  }
  auto copy = [&](int b) {
    const uint32_t st = lds0 + (b & 1) * STAGE;
#pragma unroll
    for (int i = 0; i < CPW; ++i) kx_copy16_to_lds(src[i] + b * 64, __builtin_amdgcn_readfirstlane(st + dst[i]));
  };
  f32x16 acc[MI][2];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[i][j][v] = 0.0f;
  copy(0);
  for (int b = 0; b < nb; ++b) {
    kx_wait_copies<0>();
    kx_lds_barrier();  // block b is in LDS for every wave, and every wave is done with block b - 1
    if (b + 1 < nb) copy(b + 1);
    const uint8_t *st = lds + (b & 1) * STAGE;
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
      const int p = ((2 * kk + h) ^ (lr & 7)) * 16;  // rows of a block of 32 start at a multiple of 8
      bf16x8 xa[MI], wb[2];
#pragma unroll
      for (int i = 0; i < MI; ++i) xa[i] = *(const bf16x8 *)(st + ((wm * MI + i) * 32 + lr) * 128 + p);
#pragma unroll
      for (int j = 0; j < 2; ++j) wb[j] = *(const bf16x8 *)(st + (BM + (wn * 2 + j) * 32 + lr) * 128 + p);
#pragma unroll
      for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xa[i], wb[j], acc[i][j], 0, 0, 0);
    }
  }
  // D[i][j]: j = lane % 32 (row of the matrix), i = 8 (v / 4) + 4 (lane / 32) + v % 4 (token)
  const int rg = n0 + wn * 64 + lr;
  auto token = [&](int i, int v) { return m0 + (wm * MI + i) * 32 + 8 * (v >> 2) + 4 * h + (v & 3); };
#pragma unroll
  for (int i = 0; i < MI; ++i) {
    if constexpr (EPI == KX_LIN_GLU) {
#pragma unroll
      for (int v = 0; v < 16; ++v)
        if (token(i, v) < a.tokens && rg < a.m.rows) put_glu<uint16_t>(a, token(i, v), (n0 + wn * 64) / 2 + lr, acc[i][0][v], acc[i][1][v]);
    } else {
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int r = rg + 32 * j;
        if constexpr (EPI == KX_LIN_F32) {
#pragma unroll
          for (int v = 0; v < 16; ++v)
            if (token(i, v) < a.tokens && r < a.m.rows) a.out[(size_t)token(i, v) * a.out_ld + r] = acc[i][j][v];
        } else {
          constexpr int G = most_streams(EPI) > 2 ? 4 : 16;  // elements read before the first is written
#pragma unroll
          for (int v0 = 0; v0 < 16; v0 += G) {
            Streams<EPI> res[G];
#pragma unroll
            for (int v = 0; v < G; ++v) res[v].load(a, min(token(i, v0 + v), a.tokens - 1), min(r, a.m.rows - 1));
#pragma unroll
            for (int v = 0; v < G; ++v)
              if (token(i, v0 + v) < a.tokens && r < a.m.rows) res[v].store(a, token(i, v0 + v), r, acc[i][j][v0 + v]);
          }
        }
      }
    }
  }
}

// ---- f32 GEMM: 64 tokens x 64 rows, a thread owns 4 x 4; its rows are r, r + 16, ..., so that (gate, up) pairs, 32
// rows apart, meet in one thread ----
template <int EPI>
__global__ void __launch_bounds__(256) lin_gemm_f32_k(KxLinArgs a, const float *__restrict__ x, int x_ld) {
  constexpr int BK = 16, STR = 68;
  __shared__ float xs[BK][STR], ws[BK][STR];
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int m0 = blockIdx.y * 64, n0 = blockIdx.x * 64;
  const int lrow = tid >> 2, lc = (tid & 3) * 4;
  const float *xp = x + (size_t)min(m0 + lrow, a.tokens - 1) * x_ld + lc;
  const float *wp = (const float *)a.m.w + (size_t)min(n0 + lrow, a.m.rows - 1) * a.m.ld + lc;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < a.m.ld; k0 += BK) {
    const float4 xv = *(const float4 *)(xp + k0), wv = *(const float4 *)(wp + k0);
    __syncthreads();
    xs[lc][lrow] = xv.x; xs[lc + 1][lrow] = xv.y; xs[lc + 2][lrow] = xv.z; xs[lc + 3][lrow] = xv.w;
    ws[lc][lrow] = wv.x; ws[lc + 1][lrow] = wv.y; ws[lc + 2][lrow] = wv.z; ws[lc + 3][lrow] = wv.w;
    __syncthreads();
#pragma unroll
    for (int k = 0; k < BK; ++k) {
      float xr[4], wr[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        xr[i] = xs[k][ty + 16 * i];
        wr[i] = ws[k][tx + 16 * i];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_fmaf(xr[i], wr[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = m0 + ty + 16 * i;
    if (t >= a.tokens) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int r = n0 + tx + 16 * j;
      if (r >= a.m.rows) continue;
      if constexpr (EPI == KX_LIN_F32) {
        a.out[(size_t)t * a.out_ld + r] = acc[i][j];
      } else if constexpr (EPI == KX_LIN_GLU) {
        if (j < 2) put_glu<float>(a, t, n0 / 2 + tx + 16 * j, acc[i][j], acc[i][(j + 2) & 3]);
      } else {
        Streams<EPI> res;
        res.load(a, t, r);
        res.store(a, t, r, acc[i][j]);
      }
    }
  }
}

constexpr size_t GEMV_LDS = 150 * 1024;

template <class T, int NT, int EPI>
int gemv_nt(const KxLinArgs &a, size_t lds, hipStream_t st) {
  static std::atomic<bool> attr{false};  // setting it twice from two threads is harmless
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)lin_gemv_k<T, NT, EPI>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)GEMV_LDS));
    attr = true;
  }
  const int nblk = kx_cdiv((a.m.rows + 1) / 2, GEMV_WAVES);
  hipLaunchKernelGGL((lin_gemv_k<T, NT, EPI>), dim3(std::min(nblk, 2 * std::max(1, kx_device_cus()))), dim3(GEMV_WAVES * 64), lds, st, a);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

template <class T, int EPI>
int linear_epi(const KxLinArgs &a, void *row_buf, hipStream_t st) {
  const size_t scratch = (size_t)kx_row_scratch(a.row) * 4;
  if (a.tokens <= KX_GEMV_TOKENS) {
    const int nt = a.tokens > 2 ? 4 : a.tokens;
    const size_t lds = (size_t)nt * gemv_row(a.m.ld) * sizeof(T) + scratch;
    if (lds <= GEMV_LDS) {
      if (nt == 1) return gemv_nt<T, 1, EPI>(a, lds, st);
      if (nt == 2) return gemv_nt<T, 2, EPI>(a, lds, st);
      return gemv_nt<T, 4, EPI>(a, lds, st);
    }
  }
  const T *x = (const T *)a.row.x;
  int x_ld = a.row.x_ld;
  if (a.row.kind != KX_ROW_PLAIN) {
    KX_REQUIRE(row_buf && scratch <= 160 * 1024 - 1024, "kx_linear: rows of %d columns do not fit a workgroup", a.row.cols);
    static std::atomic<bool> attr{false};
    if (!attr) {
      KX_HIP(hipFuncSetAttribute((const void *)row_k<T>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024));
      attr = true;
    }
    hipLaunchKernelGGL((row_k<T>), dim3(a.tokens), dim3(256), scratch, st, a.row, (T *)row_buf, a.m.ld);
    KX_LAUNCH_CHECK();
    x = (const T *)row_buf;
    x_ld = a.m.ld;
  }
  KX_REQUIRE(a.row.kind != KX_ROW_PLAIN || !a.row.rows_map, "kx_linear: mapped rows have to be built");
  KX_REQUIRE(x && x_ld >= a.m.ld, "kx_linear: activation rows of %d, the matrix has %d", x_ld, a.m.ld);
  if constexpr (sizeof(T) == 2 && EPI == STREAMS_ANY) {  // more streams than the matrix-core kernel is built for: a few tokens at a time
    KX_REQUIRE(gemv_row(a.m.ld) * sizeof(T) <= GEMV_LDS, "kx_linear: rows of %d columns with %d streams do not fit a workgroup", a.m.ld, a.n_streams);
    const int most = (size_t)4 * gemv_row(a.m.ld) * sizeof(T) <= GEMV_LDS ? 4 : 1;
    for (int t = 0; t < a.tokens; t += most) {
      KxLinArgs b = a;
      b.row = KxRowArgs();
      b.row.cols = a.row.cols; b.row.x = x + (size_t)t * x_ld; b.row.x_ld = x_ld;
      b.tokens = std::min(most, a.tokens - t);
      b.streams = a.streams + (size_t)t * a.n_streams * a.m.rows;
      const size_t lds = (size_t)most * gemv_row(a.m.ld) * sizeof(T);
      int rc = most == 4 ? gemv_nt<T, 4, EPI>(b, lds, st) : gemv_nt<T, 1, EPI>(b, lds, st);
      if (rc) return rc;
    }
    return KX_OK;
  } else if constexpr (sizeof(T) == 4) {
    hipLaunchKernelGGL((lin_gemm_f32_k<EPI>), dim3(kx_cdiv(a.m.rows, 64), kx_cdiv(a.tokens, 64)), dim3(256), 0, st, a, x, x_ld);
  } else {
    static std::atomic<bool> attr{false};
    if (!attr) {
      KX_HIP(hipFuncSetAttribute((const void *)lin_gemm_k<2, EPI>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024));
      attr = true;
    }
    if (a.tokens > 64) hipLaunchKernelGGL((lin_gemm_k<2, EPI>), dim3(kx_cdiv(a.m.rows, 128), kx_cdiv(a.tokens, 128)), dim3(256), 2 * 256 * 128, st, a, x, x_ld);
    else hipLaunchKernelGGL((lin_gemm_k<1, EPI>), dim3(kx_cdiv(a.m.rows, 128), 1), dim3(256), 2 * 192 * 128, st, a, x, x_ld);
  }
  KX_LAUNCH_CHECK();
  return KX_OK;
}

template <class T>
int linear(const KxLinArgs &a, void *row_buf, hipStream_t st) {
  KX_REQUIRE(a.m.w && a.m.rows > 0 && a.m.cols > 0 && a.m.ld >= a.m.cols && a.m.ld % KX_LD == 0, "kx_linear: matrix of %d x %d (%d)", a.m.rows, a.m.cols, a.m.ld);
  KX_REQUIRE(a.tokens > 0 && a.row.cols == a.m.cols, "kx_linear: tokens=%d, rows of %d for %d columns", a.tokens, a.row.cols, a.m.cols);
  KX_REQUIRE(a.epi != KX_LIN_GLU || a.m.rows % (2 * KX_GLU_BLOCK) == 0, "kx_linear: %d rows are no (gate, up) blocks", a.m.rows);
  KX_REQUIRE(a.n_streams >= 1 && a.n_streams <= KX_MAX_STREAMS && (a.mix || a.n_streams == 1), "kx_linear: %d streams", a.n_streams);
  if (a.epi == KX_LIN_F32) return linear_epi<T, KX_LIN_F32>(a, row_buf, st);
  if (a.epi == KX_LIN_GLU) return linear_epi<T, KX_LIN_GLU>(a, row_buf, st);
  if constexpr (sizeof(T) == 2) {
    if (a.n_streams == 1) return linear_epi<T, KX_LIN_STREAMS + 1>(a, row_buf, st);
    if (a.n_streams == 2) return linear_epi<T, KX_LIN_STREAMS + 2>(a, row_buf, st);
    if (a.n_streams == 3) return linear_epi<T, KX_LIN_STREAMS + 3>(a, row_buf, st);
    if (a.n_streams == 4) return linear_epi<T, KX_LIN_STREAMS + 4>(a, row_buf, st);
  }
  return linear_epi<T, STREAMS_ANY>(a, row_buf, st);
}

}  // namespace

int kx_linear_launch(bool f32, const KxLinArgs &a, void *row_buf, hipStream_t st) {
  return f32 ? linear<float>(a, row_buf, st) : linear<uint16_t>(a, row_buf, st);
}
