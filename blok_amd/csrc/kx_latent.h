// kx_latent.h -- latent attention: keys and values of all heads are products with one cached row per position, a normed
// latent, beside one rotated key part that the heads share (kx_latent.hip).
//
// Head h of position i scores position j <= i with (q_h . W_uk_h c_j + rot_i(q'_h) . rot_j(k'_j)) scale; its values are W_uv_h c_j.
// The softmax may have a learned sink per head, the output a sigmoid gate.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include "kx_linear.h"
#include "kx_window.h"

struct KxLatentSpec {
  int heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0;  // per head: unrotated and rotated query dimensions, values
  int rot = 0;         // rotated dimensions of the rot_dim, in pairs (d, d + rot / 2); the rest passes
  double base = 0;     // the pair d turns by position * base^(-2 d / rot)
  float scale = 1;
  int sink = 0;
};
inline int kx_latent_row(const KxLatentSpec &s) { return kx_pad(s.kv_rank + s.rot_dim, KX_LD); }  // elements of a cached row

struct KxLatentScratch {
  float *q = nullptr;       // [tokens][heads][padded latent row]: queries against the cached rows themselves
  int q_tokens = 0;
  void *qx = nullptr;       // [tokens of a step][heads][pad32(dim + rot_dim)] of the model's type
  void *kx = nullptr, *vx = nullptr;  // keys and values of a step's context, per sequence and head
  size_t k_elems = 0, v_elems = 0;    // room; a step whose context does not fit attends to the cached rows
  float *part = nullptr;
  size_t part_floats = 0;
};
struct KxLatentArgs {
  KxLatentSpec s;
  void *rows = nullptr;         // [batch][cap][kx_latent_row] of the model's type: latent, rotated key part, zeros
  int cap = 0;
  const float *proj = nullptr;  // f32 [tokens][proj_ld]: latent and rotated key part at kv_off, the output gate at g_off
  int proj_ld = 0, kv_off = 0, g_off = -1;  // g_off < 0: no gate
  const float *q = nullptr;     // f32 [tokens][q_ld]: per head dim unrotated, rot_dim to be rotated
  int q_ld = 0;
  const float *kv_norm = nullptr;  // [kv_rank]
  float eps = 0;
  KxMat uk, uv;                 // [heads * dim][kv_rank], [heads * vdim][kv_rank]
  const float *sinks = nullptr; // [heads]
  const float2 *turns = nullptr;  // [cap][rot / 2]: cosine and sine
  int batch = 0, positions = 0, pos = 0;  // token i * batch + b is position pos + i of sequence b
  void *out = nullptr;          // [tokens][out_ld] of the model's type: heads * vdim, gated
  int out_ld = 0;
  KxLatentScratch x;
};
// Steps of up to this many positions attend to the cached rows; longer ones make their context's keys and values first.
constexpr int KX_LATENT_FEW = 8;
// the scratch's sizes for sequences of max_context positions and steps of step_tokens tokens (pointers stay as they are)
void kx_latent_scratch(const KxLatentSpec &s, int max_batch, int max_context, int step_tokens, KxLatentScratch *x, size_t *q_floats, size_t *qx_elems);
// cosines and sines of all positions, [positions][rot / 2], made in double precision
void kx_latent_turns(const KxLatentSpec &s, int positions, float *out);
int kx_latent_launch(bool f32, const KxLatentArgs &a, hipStream_t st);
