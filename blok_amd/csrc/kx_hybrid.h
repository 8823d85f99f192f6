// kx_hybrid.h -- configuration of the hybrid decoder: layers that each have an attention or a delta-rule mixer and a
// gated feed-forward or none, between residual streams that are read and written through small learned matrices.
// The Kagalorn design's config.json is one description of such a decoder (host code only).
#pragma once
#include <vector>
#include "kx_delta.h"
#include "kx_json.h"
#include "kx_window.h"

struct KxHybridLayer {
  enum Mixer { ATTENTION, DELTA } mixer = ATTENTION;
  KxWindowSpec attn;
  bool qk_norm = false, gate = false;  // attention: RMS norm over the whole q and k projections; sigmoid gate on the output
  KxDeltaSpec delta;
  int ff = 0;  // 0: no feed-forward
  float limit = 0, alpha = 0, bias = 0;  // KX_LIN_GLU
};
struct KxHybridConfig {
  int vocab = 0, width = 0, streams = 1, groups = 1;
  bool hyper = false;  // streams are read and written through learned weights; otherwise x <- x + y
  float eps = 0;
  std::vector<KxHybridLayer> layers;
};
bool kx_kagalorn_matches(const KxJson &config);
int kx_kagalorn_config(const KxJson &config, KxHybridConfig &out);
