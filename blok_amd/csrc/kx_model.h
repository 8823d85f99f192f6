// kx_model.h -- what every decoder design of this library shares: one HBM arena, one stream, a batch of sequences that
// step together, greedy sampling, and the registry that maps a config.json to the design that runs it.
//
// Reference: generate() and its run() lambda, src/kimi_exec.cu:780-893, which know one design.  Here a design
// derives from kx_model and supplies step() -- some positions of every sequence through its layers --, and the loops
// around it (kx_stack.hip: prefill, extend, decode step, sample, generate) are the same for all.
#pragma once
#include <string>
#include <vector>
#include "kx_common.h"
#include "kx_json.h"

struct kx_model {
  virtual ~kx_model();
  virtual const char *design() const = 0;
  // Runs C positions of every sequence, from m->pos on; ids on the device, position-major (token i * batch + b is
  // position pos + i of sequence b).  With `sample`, the logits of the last position are left in `logits` and their
  // argmax in `next`.  Advances pos.
  virtual int step(const uint32_t *d_ids, bool sample, int C) = 0;
  // most positions of `batch` sequences one step takes
  virtual int step_positions(int batch_) const = 0;
  // `batch_` new sequences: whatever is not addressed by position (recurrent state) is set to its start
  virtual int restart(int batch_) { return KX_OK; }
  // logits of tokens `rows[0..n)` of the last step into d_out [n][vocab]; n <= logit_rows()
  virtual int row_logits(const int *rows, int n, float *d_out) = 0;
  virtual int logit_rows() const { return max_batch; }
  // called with the stream idle: an error that the kernels reported through device memory
  virtual int device_error() { return KX_OK; }
  virtual int rewind(int positions) = 0;
  virtual int hidden_bf16(uint16_t *h_out) = 0;  // residual stream of the last position, [batch][hidden]
  virtual int set_residual_record(bool on) {
    kx_set_error("kx_model_set_residual_record: not available for %s", design());
    return KX_ERR_ARG;
  }
  virtual int residual(int layer, int pos0, int n, float *h_out) {
    kx_set_error("kx_model_residual: not available for %s", design());
    return KX_ERR_ARG;
  }

  int n_layers = 0, hidden = 0, vocab = 0, max_batch = 0, max_context = 0;
  uint32_t eos_id = 0xffffffffu;
  int dtype = KX_DTYPE_BF16;
  int step_tokens = 1;    // tokens (positions x sequences) a step may carry
  char *arena = nullptr;
  uint64_t weight_bytes = 0, cache_bytes = 0, scratch_bytes = 0;
  float *logits = nullptr, *argmax_scratch = nullptr;                // [logit_rows][vocab], argmax partials
  uint32_t *ids = nullptr, *next = nullptr, *history = nullptr;      // [max_context][B], [B], [max_context][B]
  hipStream_t st = nullptr;
  hipEvent_t ev[3] = {nullptr, nullptr, nullptr};
  int batch = 0, pos = 0;
  int prefill_chunk = 1;  // prompt positions per prefill step (kx_model_set_prefill_chunk)
  int x_row0 = 0;         // first token of the last step that belongs to its last position
  bool sampled = false;
  float ms_prefill = 0, ms_decode = 0;
  int steps_decoded = 0;    // ids sampled per sequence by the last kx_generate (less than asked for when every sequence ended)
  uint64_t load_bytes = 0;  // checkpoint bytes copied in, and the time that took
  double load_seconds = 0;
};

// the stream and the events of a new model
int kx_model_resources(kx_model *m, const char *who);

// ---- the registry ----
struct KxDesign {
  const char *name;
  bool (*matches)(const KxJson &config);                       // is this config.json one of the design's?
  int (*probe)(const std::string &dir, const KxJson &config, kx_model_shape &shape);  // n_layers, hidden, vocab; no GPU
  int (*open)(const std::string &dir, const KxJson &config, const kx_open_options &o, kx_model **out);
};
// A design registers itself from its own file by a static object of this type, so that a program linked from some of
// the library's files knows the designs it holds.
struct KxDesignEntry {
  explicit KxDesignEntry(const KxDesign &d);
};

// byte offsets of everything in an arena
struct KxPlan {
  size_t total = 0;
  size_t take(size_t bytes) {
    size_t at = total;
    total += (bytes + 255) & ~(size_t)255;
    return at;
  }
};
