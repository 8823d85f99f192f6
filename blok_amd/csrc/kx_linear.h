// kx_linear.h -- matrix products of the hybrid decoder (kx_linear.hip): any shape, bf16 or f32 weights, activation rows
// built in the product's prologue, residual-stream update or gated activation in its epilogue.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

enum { KX_ROW_PLAIN = 0, KX_ROW_NORM = 1, KX_ROW_GATED = 2 };

struct KxRowArgs {   // see kx_rows.h
  int kind = KX_ROW_PLAIN;
  int cols = 0;                 // row length without padding
  const int *rows_map = nullptr;  // token -> row of the arrays below (nullptr: the token itself)
  const void *x = nullptr;      // PLAIN: rows of x_ld elements of the model's type
  int x_ld = 0;
  const float *streams = nullptr;  // NORM: f32 [tokens][n_streams][cols]
  int n_streams = 1;
  const float *in = nullptr;    // NORM: weight of each stream; nullptr: ones
  int groups = 1;               // NORM: equal consecutive parts with a root mean square each
  const float *w = nullptr;     // NORM [cols]; GATED [vdim]
  float eps = 0;
  const float *o = nullptr;     // GATED: f32 [tokens][heads * vdim]
  const float *gate = nullptr;  // GATED: f32 rows of gate_ld
  int gate_ld = 0, heads = 0, vdim = 0;
};
// LDS floats build_row needs (a workgroup has at most 8 waves)
inline int kx_row_scratch(const KxRowArgs &a) { return a.kind == KX_ROW_NORM ? a.cols + (a.groups > 8 ? a.groups : 8) : 0; }

// A matrix as it lies in the arena: rows of ld elements, ld a multiple of KX_LD columns, pad columns zero.
constexpr int KX_LD = 64;
inline int kx_pad(int n, int to) { return (n + to - 1) / to * to; }
struct KxMat {
  void *w = nullptr;
  int rows = 0, cols = 0, ld = 0;
};
// Gate and up of a gated feed-forward as one matrix: blocks of 32 gate rows and the 32 up rows that belong to them in
// turn, the row count padded to whole blocks, so that a wave of any of the kernels holds both halves of a pair.
constexpr int KX_GLU_BLOCK = 32;

enum {
  KX_LIN_F32 = 0,     // out[t][row] = y
  KX_LIN_GLU = 1,     // y = g' sigmoid(alpha g') (u' + bias), g' = min(g, limit), u' = clamp(u, -limit, limit), rows as above
  KX_LIN_STREAMS = 2  // x_t[row] <- sum_s mix[s][t] x_s[row] + outw[t] y
};
struct KxLinArgs {
  KxMat m;
  KxRowArgs row;
  int tokens = 0;
  int epi = KX_LIN_F32;
  float *out = nullptr;  // F32: rows of out_ld
  int out_ld = 0;
  void *mid = nullptr;   // GLU: rows of mid_ld elements of the model's type
  int mid_ld = 0;
  float limit = 0, alpha = 0, bias = 0;
  float *streams = nullptr;  // STREAMS: f32 [tokens][n_streams][m.rows]
  int n_streams = 1;
  const float *mix = nullptr, *outw = nullptr;  // nullptr: identity and ones
};
constexpr int KX_MAX_STREAMS = 8;

// f32: the model's type is float, else bf16.  row_buf: tokens * m.ld elements of scratch, where the rows of a step of
// more than KX_GEMV_TOKENS tokens are built (not used for PLAIN).
constexpr int KX_GEMV_TOKENS = 4;
int kx_linear_launch(bool f32, const KxLinArgs &a, void *row_buf, hipStream_t st);
