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
//
// Products with experts: up to 4 tokens lin_gemv_k with a matrix per (token, choice), the routing in its prologue, and with
// the residual update's own product and the chosen experts' as one sum over consecutive segments of columns; beyond that
// the GEMMs with tiles of slots sorted by expert.
#include <algorithm>
#include <atomic>
#include "kx_common.h"
#include "kx_experts.h"
#include "kx_lds_copy.h"
#include "kx_linear.h"
#include "kx_rows.h"

namespace {

using kxr::Elem;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

// ---- epilogues, one output element (or pair) at a time ----
template <class T>
__device__ __forceinline__ void put_glu(const KxLinArgs &a, int t, int col, float g, float u, float weight = 1.0f) {
  g = fminf(g, a.limit);
  u = fminf(fmaxf(u, -a.limit), a.limit);
  ((T *)a.mid)[(size_t)t * a.mid_ld + col] = Elem<T>::make(g * kxr::sigmoid_for<T>(a.alpha * g) * (u + a.bias) * weight);
}
// 0.5 z (1 + tanh(y)) = z sigmoid(2 y)
template <class T>
__device__ __forceinline__ float gelu(float z) {
  return z * kxr::sigmoid_for<T>(1.5957691216057308f * __builtin_fmaf(0.044715f * z * z, z, z));
}
template <class T>
__device__ __forceinline__ void put_f32(const KxLinArgs &a, int t, int r, float y) {
  if (r < a.act_from) a.out[(size_t)t * a.out_ld + r] = y;
  else ((T *)a.mid)[(size_t)t * a.mid_ld + r - a.act_from] = Elem<T>::make(gelu<T>(y));
}
template <class T>
__device__ __forceinline__ void put_head(const KxLinArgs &a, int t, int r, float y) {
  const int h = r / a.head_dim;
  ((T *)a.mid)[h * a.head_stride + (size_t)t * a.mid_ld + r - h * a.head_dim] = Elem<T>::make(y);
}
// variant of the activation rows that matrix rows from r on meet
__device__ __forceinline__ int variant_of(const KxLinArgs &a, int r) {
  int v = 0;
  for (int i = 1; i < a.n_var; ++i) v += r >= a.var_row[i];
  return v;
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
constexpr int CHUNK = 64 * UP * 8;     // columns per pass of a wave
__host__ __device__ __forceinline__ int gemv_row(int ld) { return (ld + CHUNK - 1) / CHUNK * CHUNK; }
// what a launch of lin_gemv_k goes over: one matrix for all tokens, the same with several variants of the rows, a matrix per
// (token, choice), or per token one matrix and then the chosen experts'
enum { GV_PLAIN = 0, GV_VARIANTS = 1, GV_EXPERT_IN = 2, GV_EXPERT_OUT = 3 };

template <class T, int NT, int EPI, int MODE>
__global__ void __launch_bounds__(GEMV_WAVES * 64) __attribute__((amdgpu_waves_per_eu(sizeof(T) == 2 ? 4 : 2)))
lin_gemv_k(KxLinArgs a, KxExpertArgs x) {
  using E = Elem<T>;
  constexpr bool OWN = MODE >= GV_EXPERT_IN;  // a token of its own per blockIdx.y
  static_assert(!OWN || NT == 1, "one token per workgroup");
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  __shared__ float red[GEMV_WAVES][2 * NT];
  __shared__ int eid[OWN ? KX_MAX_TOP : 1];
  __shared__ float ewt[MODE == GV_EXPERT_IN ? KX_MAX_TOP : 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int ld = a.m.ld, np = ld >> 3, nc0 = (np + 64 * UP - 1) / (64 * UP);
  const int nce = MODE == GV_EXPERT_OUT ? gemv_row(x.ld) / CHUNK : 0, nc = nc0 + (MODE == GV_EXPERT_OUT ? x.top * nce : 0);
  const int xl = nc * CHUNK;  // a row in LDS, with zeros up to whole passes of the wave
  const int nv = MODE == GV_VARIANTS ? a.n_var : 1;
  T *xs = (T *)lds;                                              // [NT][nv][xl]
  float *u = (float *)(lds + (size_t)NT * nv * xl * sizeof(T));  // row scratch
  const int tokens = OWN ? 1 : a.tokens, pair = MODE == GV_EXPERT_IN ? blockIdx.y : 0;
  const int tok0 = MODE == GV_EXPERT_IN ? pair / x.top : MODE == GV_EXPERT_OUT ? blockIdx.y : 0;
  const int units = (a.m.rows + 1) >> 1, nblk = (units + GEMV_WAVES - 1) / GEMV_WAVES;
  const T *w = (const T *)a.m.w;
  float weight = 1.0f;
  if constexpr (MODE == GV_EXPERT_IN) {
    const int choice = pair - tok0 * x.top;
    if (wave == 0) kxe::route_wave(x.logits + (size_t)tok0 * x.logits_ld, x.bias, x.experts, x.top, eid, ewt);
    __syncthreads();
    if (blockIdx.x == 0 && choice == 0 && (int)threadIdx.x < x.top) {
      x.ids[tok0 * x.top + threadIdx.x] = eid[threadIdx.x];
      x.weights[tok0 * x.top + threadIdx.x] = ewt[threadIdx.x];
    }
    w += (size_t)__builtin_amdgcn_readfirstlane(eid[choice]) * x.stride;
    weight = ewt[choice];
  }
  typename E::Raw bufA[2][UP], bufB[2][UP];
  // Past the last block the first row is asked for once more, by every wave: the number of loads in flight has to be the
  // same on every path, or the compiler waits for all of them.
  auto load = [&](typename E::Raw (&b)[2][UP], int blk, int c) {
    const int k = blk < nblk ? min(blk * GEMV_WAVES + wave, units - 1) : 0;
    if (blk >= nblk) c = 0;
    const T *base = w;
    int bld = ld, bnp = np;
    if (MODE == GV_EXPERT_OUT && c >= nc0) {  // the columns go on with the experts' matrices
      const int j = (c - nc0) / nce;
      c -= nc0 + j * nce;
      base = (const T *)x.w + (size_t)__builtin_amdgcn_readfirstlane(eid[j]) * x.stride;
      bld = x.ld;
      bnp = x.ld >> 3;
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const T *wr = base + (size_t)min(unit_row<EPI>(k, i), a.m.rows - 1) * bld;
#pragma unroll
      for (int j = 0; j < UP; ++j) {
        const int p = (c * UP + j) * 64 + lane;
        b[i][j] = E::stream(wr + min(p, bnp - 1) * 8);  // a lane past the row meets zeros
      }
    }
  };
  int blk = blockIdx.x, c = 0;
  load(bufA, blk, 0);
  if (MODE == GV_EXPERT_OUT && (int)threadIdx.x < x.top) eid[threadIdx.x] = x.ids[tok0 * x.top + threadIdx.x];
  uint32_t need = ~0u;  // variants that this workgroup's rows meet
  if constexpr (MODE == GV_VARIANTS) {
    need = 0;
    for (int k = blockIdx.x; k < nblk; k += gridDim.x) need |= 1u << variant_of(a, 2 * k * GEMV_WAVES);
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
    if (t < tokens) {
      T *row = xs + (size_t)t * nv * xl;
      for (int v = 0; v < nv; ++v)
        for (int y = ld + threadIdx.x; y < nc0 * CHUNK; y += GEMV_WAVES * 64) row[(size_t)v * xl + y] = E::make(0.0f);
      if constexpr (MODE == GV_EXPERT_OUT) {
        const int el = nce * CHUNK;
        for (int j = 0; j < x.top; ++j) {
          const T *m = (const T *)x.mid + (size_t)(tok0 * x.top + j) * x.mid_ld;
          for (int y = threadIdx.x; y < el; y += GEMV_WAVES * 64) row[nc0 * CHUNK + j * el + y] = y < x.ld ? m[y] : E::make(0.0f);
        }
      }
      kxr::build_row<T>(a.row, tok0 + t, row, ld, u, xl, blockIdx.x == 0, need);
    }
  float acc[2 * NT];
#pragma unroll
  for (int v = 0; v < 2 * NT; ++v) acc[v] = 0.0f;
  auto step = [&](typename E::Raw (&cur)[2][UP], typename E::Raw (&nxt)[2][UP]) {  // one chunk of columns of one unit per wave
    const bool last = c + 1 == nc;
    const int nblk_ = last ? blk + gridDim.x : blk, nc_ = last ? 0 : c + 1;
    // lane i * NT + t < 2 NT finishes row i of the unit for token t; what it updates is asked for ahead of the next weights
    const int unit = blk * GEMV_WAVES + wave, row = unit_row<EPI>(unit, lane / NT & 1), tok = NT > 1 ? lane % NT : 0;
    const bool finish = EPI == KX_LIN_GLU ? lane < NT && tok < tokens && unit < units : lane < 2 * NT && row < a.m.rows && tok < tokens;
    Streams<EPI> res;
    if (EPI >= KX_LIN_STREAMS && last && finish) res.load(a, tok0 + tok, row);
    load(nxt, nblk_, nc_);
    __builtin_amdgcn_sched_barrier(0);  // these loads are on their way before the last ones are waited for
    const T *xv = xs + (MODE == GV_VARIANTS ? (size_t)variant_of(a, 2 * blk * GEMV_WAVES) * xl : 0);
#pragma unroll
    for (int j = 0; j < UP; ++j) {
      const int p = (c * UP + j) * 64 + lane;
      float wf[2][8];
      E::unpack(wf[0], cur[0][j]);
      E::unpack(wf[1], cur[1][j]);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        float xf[8];
        E::unpack(xf, E::cached(xv + (size_t)(NT > 1 ? min(t, tokens - 1) : 0) * nv * xl + p * 8));
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
        if constexpr (EPI == KX_LIN_GLU) put_glu<T>(a, MODE == GV_EXPERT_IN ? pair : tok, unit, red[wave][lane], red[wave][NT + lane], weight);
        else if constexpr (EPI == KX_LIN_F32) put_f32<T>(a, tok, row, red[wave][lane]);
        else if constexpr (EPI == KX_LIN_HEADS) put_head<T>(a, tok, row, red[wave][lane]);
        else res.store(a, tok0 + tok, row, red[wave][lane]);
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

template <class T, int KIND>
__global__ void __launch_bounds__(256) row_k(KxRowArgs a, T *out, int ld) {
  extern __shared__ float row_lds[];
  kxr::build_row<T, KIND>(a, blockIdx.x, out + (size_t)blockIdx.x * ld, ld, row_lds, (size_t)gridDim.x * ld, true);
}

// ---- bf16 GEMM ----
// 4 waves as 2 x 2: wave (wm, wn) owns MI blocks of 32 tokens and 64 rows (two blocks of 32: with GLU rows, gate and up).
// GROUP: blockIdx.y is a tile of slots of one expert.
struct Tile {
  int m0, end;  // rows of the result
  size_t w;     // offset of the matrix
};
template <bool GROUP>
__device__ __forceinline__ bool tile_of(const KxLinArgs &a, const KxExpertArgs &e, int bm, Tile &t) {
  if constexpr (GROUP) {
    if ((int)blockIdx.y >= *e.n_tiles) return false;
    const int4 r = e.tiles[blockIdx.y];
    t.m0 = r.y;
    t.end = r.y + r.z;
    t.w = (size_t)r.x * e.stride;
  } else {
    t.m0 = blockIdx.y * bm;
    t.end = a.tokens;
    t.w = 0;
  }
  return true;
}
template <bool GROUP>
__device__ __forceinline__ size_t source_row(const KxExpertArgs &e, const Tile &t, int i) {
  const int s = min(t.m0 + i, t.end - 1);
  return GROUP && e.gather ? e.gather[s] : s;
}

template <int MI, int EPI, bool GROUP>
__global__ void __launch_bounds__(256, 2) lin_gemm_k(KxLinArgs a, KxExpertArgs e, const uint16_t *__restrict__ x, int x_ld) {
  constexpr int BM = MI * 64, BN = 128, ROWS = BM + BN, STAGE = ROWS * 128, CPW = ROWS / 32;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  const uint32_t lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) uint8_t *)lds;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int wm = wave >> 1, wn = wave & 1, lr = lane & 31, h = lane >> 5;
  const int n0 = blockIdx.x * BN;
  Tile tl;
  if (!tile_of<GROUP>(a, e, BM, tl)) return;
  const int m0 = tl.m0;
  x += (size_t)variant_of(a, n0) * a.tokens * x_ld;
  const int nb = a.m.ld >> 6;  // blocks of 64 columns
  // copy instruction i of this wave moves 8 rows of 128 bytes: lane l the piece (l % 8) ^ (row % 8) of row l / 8
  const uint16_t *src[CPW];
  uint32_t dst[CPW];
#pragma unroll
  for (int i = 0; i < CPW; ++i) {
    const int r0 = (i * 4 + wave) * 8, row = r0 + (lane >> 3), piece = (lane & 7) ^ (row & 7);
    src[i] = (row < BM ? x + source_row<GROUP>(e, tl, row) * x_ld
                       : (const uint16_t *)a.m.w + tl.w + (size_t)min(n0 + row - BM, a.m.rows - 1) * a.m.ld) + piece * 8;
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
        if (token(i, v) < tl.end && rg < a.m.rows)
          put_glu<uint16_t>(a, token(i, v), (n0 + wn * 64) / 2 + lr, acc[i][0][v], acc[i][1][v], GROUP ? e.slot_weight[token(i, v)] : 1.0f);
    } else {
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int r = rg + 32 * j;
        if constexpr (EPI == KX_LIN_F32) {
#pragma unroll
          for (int v = 0; v < 16; ++v)
            if (token(i, v) < tl.end && r < a.m.rows) put_f32<uint16_t>(a, token(i, v), r, acc[i][j][v]);
        } else if constexpr (EPI == KX_LIN_HEADS) {
#pragma unroll
          for (int v = 0; v < 16; ++v)
            if (token(i, v) < tl.end && r < a.m.rows) put_head<uint16_t>(a, token(i, v), r, acc[i][j][v]);
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
template <int EPI, bool GROUP>
__global__ void __launch_bounds__(256) lin_gemm_f32_k(KxLinArgs a, KxExpertArgs e, const float *__restrict__ x, int x_ld) {
  constexpr int BK = 16, STR = 68;
  __shared__ float xs[BK][STR], ws[BK][STR];
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int n0 = blockIdx.x * 64;
  Tile tl;
  if (!tile_of<GROUP>(a, e, 64, tl)) return;
  const int m0 = tl.m0;
  x += (size_t)variant_of(a, n0) * a.tokens * x_ld;
  const int lrow = tid >> 2, lc = (tid & 3) * 4;
  const float *xp = x + source_row<GROUP>(e, tl, lrow) * x_ld + lc;
  const float *wp = (const float *)a.m.w + tl.w + (size_t)min(n0 + lrow, a.m.rows - 1) * a.m.ld + lc;
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
    if (t >= tl.end) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int r = n0 + tx + 16 * j;
      if (r >= a.m.rows) continue;
      if constexpr (EPI == KX_LIN_F32) {
        put_f32<float>(a, t, r, acc[i][j]);
      } else if constexpr (EPI == KX_LIN_HEADS) {
        put_head<float>(a, t, r, acc[i][j]);
      } else if constexpr (EPI == KX_LIN_GLU) {
        if (j < 2) put_glu<float>(a, t, n0 / 2 + tx + 16 * j, acc[i][j], acc[i][(j + 2) & 3], GROUP ? e.slot_weight[t] : 1.0f);
      } else {
        Streams<EPI> res;
        res.load(a, t, r);
        res.store(a, t, r, acc[i][j]);
      }
    }
  }
}

constexpr size_t GEMV_LDS = 150 * 1024;

// `lds` bytes of the dynamic part; grid_y: 1, or the tokens or (token, choice) pairs
template <class T, int NT, int EPI, int MODE>
int gemv_launch(const KxLinArgs &a, const KxExpertArgs &x, size_t lds, int grid_y, hipStream_t st) {
  static std::atomic<bool> attr{false};  // setting it twice from two threads is harmless
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)lin_gemv_k<T, NT, EPI, MODE>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)GEMV_LDS));
    attr = true;
  }
  const int nblk = kx_cdiv((a.m.rows + 1) / 2, GEMV_WAVES), most = std::max(1, 2 * std::max(1, kx_device_cus()) / grid_y);
  hipLaunchKernelGGL((lin_gemv_k<T, NT, EPI, MODE>), dim3(std::min(nblk, most), grid_y), dim3(GEMV_WAVES * 64), lds, st, a, x);
  KX_LAUNCH_CHECK();
  return KX_OK;
}
template <class T, int NT, int EPI>
int gemv_nt(const KxLinArgs &a, size_t lds, hipStream_t st) {
  if constexpr (EPI == KX_LIN_F32)
    if (a.row.kind == KX_ROW_SHIFT) return gemv_launch<T, NT, EPI, GV_VARIANTS>(a, KxExpertArgs(), lds, 1, st);
  return gemv_launch<T, NT, EPI, GV_PLAIN>(a, KxExpertArgs(), lds, 1, st);
}

template <class T, int KIND>
int rows_kind(const KxRowArgs &r, int tokens, T *out, int ld, hipStream_t st) {
  const size_t scratch = (size_t)kx_row_scratch(r) * 4;
  KX_REQUIRE(out && scratch <= 160 * 1024 - 1024, "kx_linear: rows of %d columns do not fit a workgroup", r.cols);
  static std::atomic<bool> attr{false};
  if (!attr) {
    KX_HIP(hipFuncSetAttribute((const void *)row_k<T, KIND>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024));
    attr = true;
  }
  hipLaunchKernelGGL((row_k<T, KIND>), dim3(tokens), dim3(256), scratch, st, r, out, ld);
  KX_LAUNCH_CHECK();
  return KX_OK;
}
template <class T>
int rows_launch(const KxRowArgs &r, int tokens, T *out, int ld, hipStream_t st) {
  switch (r.kind) {
    case KX_ROW_NORM: return rows_kind<T, KX_ROW_NORM>(r, tokens, out, ld, st);
    case KX_ROW_GATED: return rows_kind<T, KX_ROW_GATED>(r, tokens, out, ld, st);
    case KX_ROW_SHIFT: return rows_kind<T, KX_ROW_SHIFT>(r, tokens, out, ld, st);
    case KX_ROW_TANH: return rows_kind<T, KX_ROW_TANH>(r, tokens, out, ld, st);
  }
  return rows_kind<T, KX_ROW_PLAIN>(r, tokens, out, ld, st);
}

// GEMM over rows in memory; GROUP: e.max_tiles tiles of slots
template <class T, int EPI, bool GROUP>
int gemm_launch(const KxLinArgs &a, const KxExpertArgs &e, const T *x, int x_ld, hipStream_t st) {
  KX_REQUIRE(x && x_ld >= a.m.ld, "kx_linear: activation rows of %d, the matrix has %d", x_ld, a.m.ld);
  if constexpr (sizeof(T) == 4) {
    hipLaunchKernelGGL((lin_gemm_f32_k<EPI, GROUP>), dim3(kx_cdiv(a.m.rows, 64), GROUP ? e.max_tiles : kx_cdiv(a.tokens, 64)), dim3(256), 0, st, a, e, x, x_ld);
  } else {
    static std::atomic<bool> attr{false};
    if (!attr) {
      KX_HIP(hipFuncSetAttribute((const void *)lin_gemm_k<2, EPI, GROUP>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024));
      attr = true;
    }
    const bool wide = GROUP ? e.tile_slots > 64 : a.tokens > 64;
    const int tiles = GROUP ? e.max_tiles : kx_cdiv(a.tokens, wide ? 128 : 64);
    if (wide) hipLaunchKernelGGL((lin_gemm_k<2, EPI, GROUP>), dim3(kx_cdiv(a.m.rows, 128), tiles), dim3(256), 2 * 256 * 128, st, a, e, x, x_ld);
    else hipLaunchKernelGGL((lin_gemm_k<1, EPI, GROUP>), dim3(kx_cdiv(a.m.rows, 128), tiles), dim3(256), 2 * 192 * 128, st, a, e, x, x_ld);
  }
  KX_LAUNCH_CHECK();
  return KX_OK;
}

template <class T, int EPI>
int linear_epi(const KxLinArgs &a, void *row_buf, hipStream_t st) {
  const size_t scratch = (size_t)kx_row_scratch(a.row) * 4;
  if (a.tokens <= KX_GEMV_TOKENS) {
    const int nt = a.tokens > 2 ? 4 : a.tokens;
    const size_t lds = (size_t)nt * kx_row_variants(a.row) * gemv_row(a.m.ld) * sizeof(T) + scratch;
    if (lds <= GEMV_LDS) {
      if (nt == 1) return gemv_nt<T, 1, EPI>(a, lds, st);
      if (nt == 2) return gemv_nt<T, 2, EPI>(a, lds, st);
      return gemv_nt<T, 4, EPI>(a, lds, st);
    }
  }
  const T *x = (const T *)a.row.x;
  int x_ld = a.row.x_ld;
  if (a.row.kind != KX_ROW_PLAIN) {
    int rc = rows_launch<T>(a.row, a.tokens, (T *)row_buf, a.m.ld, st);
    if (rc) return rc;
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
  } else {
    return gemm_launch<T, EPI, false>(a, KxExpertArgs(), x, x_ld, st);
  }
}

int check_matrix(const KxLinArgs &a) {
  KX_REQUIRE(a.m.w && a.m.rows > 0 && a.m.cols > 0 && a.m.ld >= a.m.cols && a.m.ld % KX_LD == 0, "kx_linear: matrix of %d x %d (%d)", a.m.rows, a.m.cols, a.m.ld);
  KX_REQUIRE(a.tokens > 0 && a.row.cols == a.m.cols, "kx_linear: tokens=%d, rows of %d for %d columns", a.tokens, a.row.cols, a.m.cols);
  KX_REQUIRE(a.epi != KX_LIN_GLU || a.m.rows % (2 * KX_GLU_BLOCK) == 0, "kx_linear: %d rows are no (gate, up) blocks", a.m.rows);
  KX_REQUIRE(a.n_streams >= 1 && a.n_streams <= KX_MAX_STREAMS && (a.mix || a.n_streams == 1), "kx_linear: %d streams", a.n_streams);
  KX_REQUIRE(a.epi != KX_LIN_F32 || a.act_from >= a.m.rows || (a.mid && a.mid_ld >= a.m.rows - a.act_from), "kx_linear: no room for %d activations", a.m.rows - a.act_from);
  KX_REQUIRE(a.epi != KX_LIN_HEADS || (a.head_dim > 0 && a.mid), "kx_linear: heads of %d", a.head_dim);
  KX_REQUIRE(a.row.kind != KX_ROW_SHIFT || (a.epi == KX_LIN_F32 && a.row.n_streams == 1 && a.row.batch > 0 && a.row.tokens == a.tokens && a.row.prev && a.row.prev_out &&
                                            a.row.prev != a.row.prev_out && a.n_var == a.row.n_mix + 1 && a.n_var <= KX_MAX_VARIANTS),
             "kx_linear: %d mixes of %d tokens", a.row.n_mix, a.row.tokens);
  for (int v = 1; v < a.n_var; ++v) KX_REQUIRE(a.var_row[v] % KX_VARIANT_ROWS == 0, "kx_linear: variant %d from row %d on", v, a.var_row[v]);
  KX_REQUIRE(!a.row.tail || (a.row.kind == KX_ROW_GATED && a.row.head_ld % KX_LD == 0 && a.row.head_ld >= a.row.heads * a.row.vdim && a.row.tail_ld >= a.m.ld - a.row.head_ld),
             "kx_linear: a row of %d and its tail of %d", a.row.head_ld, a.row.tail_ld);
  return KX_OK;
}

template <class T>
int linear(const KxLinArgs &a, void *row_buf, hipStream_t st) {
  int rc = check_matrix(a);
  if (rc) return rc;
  if (a.epi == KX_LIN_F32) return linear_epi<T, KX_LIN_F32>(a, row_buf, st);
  if (a.epi == KX_LIN_GLU) return linear_epi<T, KX_LIN_GLU>(a, row_buf, st);
  if (a.epi == KX_LIN_HEADS) return linear_epi<T, KX_LIN_HEADS>(a, row_buf, st);
  if constexpr (sizeof(T) == 2) {
    if (a.n_streams == 1) return linear_epi<T, KX_LIN_STREAMS + 1>(a, row_buf, st);
    if (a.n_streams == 2) return linear_epi<T, KX_LIN_STREAMS + 2>(a, row_buf, st);
    if (a.n_streams == 3) return linear_epi<T, KX_LIN_STREAMS + 3>(a, row_buf, st);
    if (a.n_streams == 4) return linear_epi<T, KX_LIN_STREAMS + 4>(a, row_buf, st);
  }
  return linear_epi<T, STREAMS_ANY>(a, row_buf, st);
}

template <class T>
size_t expert_in_lds(const KxLinArgs &a) { return (size_t)gemv_row(a.m.ld) * sizeof(T) + (size_t)kx_row_scratch(a.row) * 4; }
template <class T>
size_t expert_out_lds(const KxLinArgs &a, const KxExpertArgs &e) {
  return ((size_t)gemv_row(a.m.ld) + (size_t)e.top * gemv_row(e.ld)) * sizeof(T) + (size_t)kx_row_scratch(a.row) * 4;
}
int check_experts(const KxExpertArgs &e) {
  KX_REQUIRE(e.experts > 0 && e.experts <= KX_MAX_EXPERTS && e.top > 0 && e.top <= e.experts && e.top <= KX_MAX_TOP, "experts: %d of %d", e.top, e.experts);
  return KX_OK;
}
template <class T>
int expert_in(const KxLinArgs &a, const KxExpertArgs &e, hipStream_t st) {
  KX_REQUIRE(a.epi == KX_LIN_GLU && e.logits && e.ids && e.weights && expert_in_lds<T>(a) <= GEMV_LDS, "experts: rows of %d columns", a.m.cols);
  return gemv_launch<T, 1, KX_LIN_GLU, GV_EXPERT_IN>(a, e, expert_in_lds<T>(a), a.tokens * e.top, st);
}
template <class T>
int expert_out(const KxLinArgs &a, const KxExpertArgs &e, hipStream_t st) {
  KX_REQUIRE(a.epi == KX_LIN_STREAMS && a.n_streams == 1 && !a.mix && e.ids && e.w && e.mid && e.mid_ld >= e.ld && e.ld % KX_LD == 0 && expert_out_lds<T>(a, e) <= GEMV_LDS,
             "experts: rows of %d and %d x %d columns", a.m.cols, e.top, e.ld);
  return gemv_launch<T, 1, KX_LIN_STREAMS + 1, GV_EXPERT_OUT>(a, e, expert_out_lds<T>(a, e), a.tokens, st);
}
template <class T>
int expert_gemm(const KxLinArgs &a, const KxExpertArgs &e, const T *x, int x_ld, hipStream_t st) {
  KX_REQUIRE(e.tiles && e.n_tiles && e.max_tiles > 0 && e.max_tiles <= 65535 && a.n_var == 1, "experts: %d tiles", e.max_tiles);
  KX_REQUIRE(e.tile_slots > 0 && e.tile_slots <= (sizeof(T) == 4 ? 64 : 128), "experts: tiles of %d", e.tile_slots);
  KX_REQUIRE(a.epi != KX_LIN_GLU || e.slot_weight, "experts: no weights");
  if (a.epi == KX_LIN_GLU) return gemm_launch<T, KX_LIN_GLU, true>(a, e, x, x_ld, st);
  KX_REQUIRE(a.epi == KX_LIN_F32, "experts: epilogue %d", a.epi);
  return gemm_launch<T, KX_LIN_F32, true>(a, e, x, x_ld, st);
}

}  // namespace

int kx_linear_launch(bool f32, const KxLinArgs &a, void *row_buf, hipStream_t st) {
  return f32 ? linear<float>(a, row_buf, st) : linear<uint16_t>(a, row_buf, st);
}
int kx_rows_launch(bool f32, const KxRowArgs &r, int tokens, void *out, int ld, hipStream_t st) {
  return f32 ? rows_launch<float>(r, tokens, (float *)out, ld, st) : rows_launch<uint16_t>(r, tokens, (uint16_t *)out, ld, st);
}
bool kx_expert_small(bool f32, const KxLinArgs &in, const KxLinArgs &out, const KxExpertArgs &e, int tokens) {
  return tokens <= KX_GEMV_TOKENS && (f32 ? expert_in_lds<float>(in) <= GEMV_LDS && expert_out_lds<float>(out, e) <= GEMV_LDS
                                          : expert_in_lds<uint16_t>(in) <= GEMV_LDS && expert_out_lds<uint16_t>(out, e) <= GEMV_LDS);
}
int kx_expert_in_launch(bool f32, const KxLinArgs &a, const KxExpertArgs &e, hipStream_t st) {
  int rc = check_matrix(a);
  if (rc || (rc = check_experts(e))) return rc;
  return f32 ? expert_in<float>(a, e, st) : expert_in<uint16_t>(a, e, st);
}
int kx_expert_out_launch(bool f32, const KxLinArgs &a, const KxExpertArgs &e, hipStream_t st) {
  int rc = check_matrix(a);
  if (rc || (rc = check_experts(e))) return rc;
  return f32 ? expert_out<float>(a, e, st) : expert_out<uint16_t>(a, e, st);
}
int kx_expert_gemm_launch(bool f32, const KxLinArgs &a, const KxExpertArgs &e, const void *x, int x_ld, hipStream_t st) {
  int rc = check_matrix(a);
  if (rc) return rc;
  return f32 ? expert_gemm<float>(a, e, (const float *)x, x_ld, st) : expert_gemm<uint16_t>(a, e, (const uint16_t *)x, x_ld, st);
}
