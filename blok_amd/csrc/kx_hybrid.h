// kx_hybrid.h -- configuration of the hybrid decoder: layers that each have a mixer (attention over window and pooled blocks,
// latent attention, or one of several recurrences) and a feed-forward (gated, plain, a mixture of experts) or none,
// between residual streams that are read and written through small learned matrices, or one stream and sums.
// The Kagalorn and Rapitar designs' config.json are descriptions of such a decoder (host code only).
#pragma once
#include <vector>
#include "kx_delta.h"
#include "kx_json.h"
#include "kx_latent.h"
#include "kx_ssd.h"
#include "kx_window.h"
#include "kx_wkv.h"

struct KxHybridLayer {
  enum Mixer { ATTENTION, DELTA, SSD, WKV, LATENT } mixer = ATTENTION;
  KxWindowSpec attn;
  bool qk_norm = false, gate = false;  // attention: RMS norm over the whole q and k projections; sigmoid gate on the output
  KxDeltaSpec delta;
  KxSsdSpec ssd;
  int norm_groups = 1;                 // SSD: parts of the read-out's norm
  KxWkvSpec wkv;                       // rank 0: what the weight files say
  KxLatentSpec latent;
  int q_rank = 0;                      // LATENT: of the queries' own latent
  // GLU: gated and clamped (limit, alpha, bias of KX_LIN_GLU); GELU: up, gelu (tanh form), down; EXPERTS: `top` of `experts`
  // gated ones with silu
  enum Ff { NONE, GLU, GELU, EXPERTS } ff_kind = NONE;
  int ff = 0;
  float limit = 0, alpha = 0, bias = 0;
  int experts = 0, top = 0;
};
struct KxHybridConfig {
  int vocab = 0, width = 0, streams = 1, groups = 1;
  bool hyper = false;     // streams are read and written through learned weights; otherwise x <- x + y
  bool parallel = false;  // x <- x + (mixer(h) + ff(h)) with one norm for both; GELU and EXPERTS need it, GLU the opposite
  bool norm_about_one = false;  // the model's norm weights are stored as their difference from one
  float eps = 0;
  std::vector<KxHybridLayer> layers;
};
bool kx_kagalorn_matches(const KxJson &config);
int kx_kagalorn_config(const KxJson &config, KxHybridConfig &out);
bool kx_rapitar_matches(const KxJson &config);
int kx_rapitar_config(const KxJson &config, KxHybridConfig &out);
