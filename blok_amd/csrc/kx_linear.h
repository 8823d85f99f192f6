// kx_linear.h -- matrix products of the hybrid decoder (kx_linear.hip): any shape, bf16 or f32 weights, activation rows
// built in the product's prologue, residual-stream update or gated activation in its epilogue.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

enum { KX_ROW_PLAIN = 0, KX_ROW_NORM = 1, KX_ROW_GATED = 2, KX_ROW_SHIFT = 3, KX_ROW_TANH = 4 };

struct KxRowArgs {   // see kx_rows.h
  int kind = KX_ROW_PLAIN;
  int cols = 0;                 // row length without padding
  const int *rows_map = nullptr;  // token -> row of the arrays below (nullptr: the token itself)
  const void *x = nullptr;      // PLAIN: rows of x_ld elements of the model's type
  int x_ld = 0;
  const float *streams = nullptr;  // NORM, SHIFT: f32 [tokens][n_streams][cols]; TANH: rows of streams_ld
  int n_streams = 1;
  int streams_ld = 0;              // floats from one token to the next; 0: n_streams * cols
  const float *in = nullptr;    // NORM: weight of each stream; nullptr: ones
  int groups = 1;               // NORM: equal consecutive parts with a root mean square each
  const float *w = nullptr;     // NORM, SHIFT [cols]; GATED [vdim], or [heads * vdim] with w_per_column
  float eps = 0;
  const float *o = nullptr;     // GATED: f32 [tokens][heads * vdim]
  const float *gate = nullptr;  // GATED: f32 rows of gate_ld
  int gate_ld = 0, heads = 0, vdim = 0;
  bool w_per_column = false;
  bool gate_first = false;      // GATED: the gate in front of the norm, not behind it
  // GATED: the row goes on with `cols - head_ld` elements of the model's type from here (the second factor of a
  // concatenated product); nullptr: the read-out alone
  const void *tail = nullptr;
  int tail_ld = 0, head_ld = 0;
  // SHIFT: n_mix rows h + (h' - h) mu[m], h' the row of the position before (prev where the step begins), then h itself
  const float *mu = nullptr;    // [n_mix][cols]
  int n_mix = 0, batch = 1;     // token i * batch + b is the i-th position of sequence b
  const float *prev = nullptr;  // [batch][cols]
  float *prev_out = nullptr;    // the same after this step (another buffer)
  int tokens = 0;
};
inline int kx_row_variants(const KxRowArgs &a) { return a.kind == KX_ROW_SHIFT ? a.n_mix + 1 : 1; }
// LDS floats build_row needs (a workgroup has at most 8 waves)
inline int kx_row_scratch(const KxRowArgs &a) {
  return a.kind == KX_ROW_NORM ? a.cols + (a.groups > 8 ? a.groups : 8) : a.kind == KX_ROW_SHIFT ? 8
       : a.kind == KX_ROW_GATED && a.heads < 8 ? a.heads * a.vdim + 8 : 0;
}

// A matrix as it lies in the arena: rows of ld elements, ld a multiple of KX_LD columns, pad columns zero.
constexpr int KX_LD = 64;
__host__ __device__ inline int kx_pad(int n, int to) { return (n + to - 1) / to * to; }
struct KxMat {
  void *w = nullptr;
  int rows = 0, cols = 0, ld = 0;
};
// Gate and up of a gated feed-forward as one matrix: blocks of 32 gate rows and the 32 up rows that belong to them in
// turn, the row count padded to whole blocks, so that a wave of any of the kernels holds both halves of a pair.
constexpr int KX_GLU_BLOCK = 32;

enum {
  KX_LIN_F32 = 0,     // out[t][row] = y; rows from act_from on: mid[t][row - act_from] = gelu(y) (tanh form)
  KX_LIN_GLU = 1,     // y = g' sigmoid(alpha g') (u' + bias), g' = min(g, limit), u' = clamp(u, -limit, limit), rows as above
  KX_LIN_HEADS = 3,   // matrix rows are heads of head_dim each: y of the model's type into a block per head
  KX_LIN_STREAMS = 4  // x_t[row] <- sum_s mix[s][t] x_s[row] + outw[t] y
};
constexpr int KX_MAX_VARIANTS = 8, KX_VARIANT_ROWS = 128;
struct KxLinArgs {
  KxMat m;
  KxRowArgs row;
  int tokens = 0;
  int epi = KX_LIN_F32;
  float *out = nullptr;  // F32: rows of out_ld
  int out_ld = 0;
  int act_from = 0x7fffffff;
  void *mid = nullptr;   // GLU, F32 with act_from: rows of mid_ld elements of the model's type
  int mid_ld = 0;
  float limit = 0, alpha = 0, bias = 0;
  // HEADS: element (t, h * head_dim + d) goes to mid[h * head_stride + t * mid_ld + d]
  int head_dim = 0;
  size_t head_stride = 0;
  float *streams = nullptr;  // STREAMS: f32 [tokens][n_streams][m.rows]
  int n_streams = 1;
  const float *mix = nullptr, *outw = nullptr;  // nullptr: identity and ones
  // SHIFT rows: the matrix rows [var_row[v], var_row[v + 1]) meet variant v; multiples of KX_VARIANT_ROWS
  int n_var = 1;
  int var_row[KX_MAX_VARIANTS] = {};
};
constexpr int KX_MAX_STREAMS = 8;

// ---- products with experts: every token meets `top` of `experts` matrices (KxExpertArgs), see kx_experts.h ----
struct KxExpertArgs {
  int experts = 0, top = 0;
  const float *logits = nullptr, *bias = nullptr;  // [tokens][logits_ld]; [experts]
  int logits_ld = 0;
  int *ids = nullptr;                // [tokens][top]
  float *weights = nullptr;          // [tokens][top]
  size_t stride = 0;                 // elements from one expert's matrix to the next
  // the matrices the residual update adds behind its own product: [experts][rows][ld], input rows `mid` [tokens * top]
  const void *w = nullptr;
  int ld = 0;
  const void *mid = nullptr;
  int mid_ld = 0;
  // many tokens: (token, choice) pairs sorted by expert; tiles of consecutive ones, each of one expert
  const int4 *tiles = nullptr;       // {expert, first slot, slots, -}
  const int *n_tiles = nullptr;
  int max_tiles = 0, tile_slots = 0;
  const int *gather = nullptr;       // slot -> row of x (nullptr: the slot itself)
  const float *slot_weight = nullptr;  // GLU: the result of a slot is multiplied by it
};
constexpr int KX_MAX_EXPERTS = 1024, KX_MAX_TOP = 64;

// f32: the model's type is float, else bf16.  row_buf: tokens * m.ld elements of scratch, where the rows of a step of
// more than KX_GEMV_TOKENS tokens are built (not used for PLAIN).
constexpr int KX_GEMV_TOKENS = 4;
int kx_linear_launch(bool f32, const KxLinArgs &a, void *row_buf, hipStream_t st);
// The rows alone, [variant][token][ld], into `out`.
int kx_rows_launch(bool f32, const KxRowArgs &r, int tokens, void *out, int ld, hipStream_t st);

// Up to KX_GEMV_TOKENS tokens, each with its own experts.  kx_expert_small says whether the two launches take a
// layer's sizes (their rows have to fit a workgroup).
//   in:  routes every token (kx_experts.h) and leaves ids and weights; mid[t * top + j] = weight_j * GLU of expert ids_j,
//        a.m the first expert's (gate, up) matrix, a.row the tokens' rows
//   out: x_t <- x_t + a.m row_t + sum_j w[ids_j] mid[t * top + j]
bool kx_expert_small(bool f32, const KxLinArgs &in, const KxLinArgs &out, const KxExpertArgs &e, int tokens);
int kx_expert_in_launch(bool f32, const KxLinArgs &a, const KxExpertArgs &e, hipStream_t st);
int kx_expert_out_launch(bool f32, const KxLinArgs &a, const KxExpertArgs &e, hipStream_t st);
// Many tokens: a.m the first expert's matrix, rows x of x_ld elements in memory; epilogue GLU (mid[slot]) or F32 (out[slot]).
int kx_expert_gemm_launch(bool f32, const KxLinArgs &a, const KxExpertArgs &e, const void *x, int x_ld, hipStream_t st);
