// kx_stack.hip -- the loops around a design's step: prefill, extend, decode step, greedy sample, generate; and the
// registry that opens a model directory (kx_model.h).
//
// Reference: generate(), src/kimi_exec.cu:780-893 (the loops at :886-890).
#include <string.h>
#include <sys/stat.h>
#include <algorithm>
#include <vector>
#include "kx_argmax.h"
#include "kx_model.h"

namespace {

__global__ void copy_ids_k(const uint32_t *__restrict__ src, uint32_t *__restrict__ dst, int n) {
  int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) dst[i] = src[i];
}

int copy_ids(kx_model *m, const uint32_t *src, uint32_t *dst) {
  hipLaunchKernelGGL(copy_ids_k, dim3(kx_cdiv(m->batch, 64)), dim3(64), 0, m->st, src, dst, m->batch);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

int check_ids(const kx_model *m, const uint32_t *ids, size_t n) {
  for (size_t i = 0; i < n; ++i)
    KX_REQUIRE(ids[i] < (uint32_t)m->vocab, "token id %u outside the vocabulary of %d", ids[i], m->vocab);  // :552, :652
  return KX_OK;
}

// `n` positions of every sequence appended, in steps of at most the prefill chunk; h_ids [batch][n].  Logits are
// wanted at places `want` (ascending or not) of the n, into h_logits [n_want][batch][vocab].
int extend(kx_model *m, const uint32_t *h_ids, int n, const int32_t *want, int n_want, float *h_logits) {
  const int B = m->batch;
  int rc = check_ids(m, h_ids, (size_t)B * n);
  if (rc) return rc;
  std::vector<uint32_t> pm((size_t)n * B);  // position-major
  for (int b = 0; b < B; ++b)
    for (int i = 0; i < n; ++i) pm[(size_t)i * B + b] = h_ids[(size_t)b * n + i];
  uint32_t *d_ids = m->ids + (size_t)m->pos * B;
  KX_HIP(hipMemcpyAsync(d_ids, pm.data(), pm.size() * 4, hipMemcpyHostToDevice, m->st));
  KX_HIP(hipStreamSynchronize(m->st));  // pm goes out of scope
  // :886: one run() per prompt token, sampling on the last; with a prefill chunk set, up to that many positions per step
  const int chunk = std::max(1, std::min(m->prefill_chunk, m->step_positions(B)));
  std::vector<int> rows, at;
  for (int i = 0; i < n; i += chunk) {
    const int c = std::min(chunk, n - i);
    if ((rc = m->step(d_ids + (size_t)i * B, i + c == n, c))) return rc;
    rows.clear();
    at.clear();
    for (int w = 0; w < n_want; ++w)
      if (want[w] >= i && want[w] < i + c)
        for (int b = 0; b < B; ++b) {
          rows.push_back((want[w] - i) * B + b);
          at.push_back(w * B + b);
        }
    if (rows.empty()) continue;
    const size_t V = m->vocab;
    for (size_t r = 0; r < rows.size(); r += m->logit_rows()) {
      const int k = (int)std::min(rows.size() - r, (size_t)m->logit_rows());
      if ((rc = m->row_logits(rows.data() + r, k, m->logits))) return rc;
      for (int j = 0; j < k; ++j)
        KX_HIP(hipMemcpyAsync(h_logits + at[r + j] * V, m->logits + j * V, V * 4, hipMemcpyDeviceToHost, m->st));
      KX_HIP(hipStreamSynchronize(m->st));
    }
    if (i + c == n) {  // the sampled position's logits were overwritten; put them back
      std::vector<int> last(B);
      for (int b = 0; b < B; ++b) last[b] = (c - 1) * B + b;
      if ((rc = m->row_logits(last.data(), B, m->logits))) return rc;
    }
  }
  return KX_OK;
}

// Synchronises the model's stream and reports what its kernels have flagged.
int sync_and_check(kx_model *m) {
  KX_HIP(hipStreamSynchronize(m->st));
  return m->device_error();
}

std::vector<KxDesign> &designs() {
  static std::vector<KxDesign> d;
  return d;
}

// the design that dir/config.json names
int find_design(const std::string &dir, KxJson &config, const KxDesign **out) {
  int rc = kx_json_file(dir + "/config.json", config);
  if (rc) return rc;
  std::string known;
  for (const KxDesign &d : designs()) {
    if (d.matches(config)) {
      *out = &d;
      return KX_OK;
    }
    known += (known.empty() ? "" : ", ") + std::string(d.name);
  }
  kx_set_error("%s/config.json names none of the designs here (%s)", dir.c_str(), known.c_str());
  return KX_ERR_ARG;
}

}  // namespace

KxDesignEntry::KxDesignEntry(const KxDesign &d) { designs().push_back(d); }

kx_model::~kx_model() {
  for (auto &e : ev)
    if (e) (void)hipEventDestroy(e);
  if (st) (void)hipStreamDestroy(st);
  if (arena) (void)hipFree(arena);
}

int kx_model_resources(kx_model *m, const char *who) {
  bool ok = hipStreamCreate(&m->st) == hipSuccess;
  for (auto &e : m->ev) ok = ok && hipEventCreate(&e) == hipSuccess;
  if (!ok) kx_set_error("%s: HIP resource creation failed", who);
  return ok ? KX_OK : KX_ERR_HIP;
}

extern "C" int kx_open_options_default(kx_open_options *o) {
  KX_REQUIRE(o, "kx_open_options_default: null options");
  memset(o, 0, sizeof *o);
  o->dtype = KX_DTYPE_BF16;
  o->max_batch = 1;
  o->max_context = 4096;
  o->step_tokens = 2048;
  o->eos_id = 0xffffffffu;
  o->init_sigma = 0.02f;
  return KX_OK;
}

extern "C" int kx_model_open(const char *dir, const kx_open_options *opt, kx_model **out) {
  KX_REQUIRE(out, "kx_model_open: null out pointer");
  *out = nullptr;
  KX_REQUIRE(dir && dir[0] && opt, "kx_model_open: null argument");
  KX_REQUIRE(opt->dtype == KX_DTYPE_BF16 || opt->dtype == KX_DTYPE_F32, "kx_model_open: dtype=%d", opt->dtype);
  KX_REQUIRE(opt->max_batch > 0 && opt->max_context > 0 && opt->step_tokens > 0 && opt->layers >= 0,
             "kx_model_open: max_batch=%d max_context=%d step_tokens=%d layers=%d", opt->max_batch, opt->max_context, opt->step_tokens, opt->layers);
  return kx_guard("kx_model_open", [&]() -> int {
    KxJson config;
    const KxDesign *d = nullptr;
    int rc = find_design(dir, config, &d);
    return rc ? rc : d->open(dir, config, *opt, out);
  });
}

extern "C" int kx_model_probe(const char *dir, kx_model_shape *out) {
  KX_REQUIRE(dir && dir[0] && out, "kx_model_probe: null argument");
  memset(out, 0, sizeof *out);
  return kx_guard("kx_model_probe", [&]() -> int {
    KxJson config;
    const KxDesign *d = nullptr;
    int rc = find_design(dir, config, &d);
    if (rc) return rc;
    snprintf(out->design, sizeof out->design, "%s", d->name);
    return d->probe(dir, config, *out);
  });
}

extern "C" int kx_model_destroy(kx_model *m) {
  if (!m) return KX_OK;
  if (m->st) (void)hipStreamSynchronize(m->st);
  delete m;
  return KX_OK;
}

extern "C" int kx_model_info(kx_model *m, kx_model_shape *out) {
  KX_REQUIRE(m && out, "kx_model_info: null argument");
  memset(out, 0, sizeof *out);
  snprintf(out->design, sizeof out->design, "%s", m->design());
  out->n_layers = m->n_layers; out->hidden = m->hidden; out->vocab = m->vocab; out->dtype = m->dtype;
  out->max_batch = m->max_batch; out->max_context = m->max_context; out->step_tokens = m->step_tokens;
  out->weight_bytes = m->weight_bytes; out->cache_bytes = m->cache_bytes; out->scratch_bytes = m->scratch_bytes;
  return KX_OK;
}

extern "C" int kx_model_load_info(kx_model *m, uint64_t *bytes, double *seconds) {
  KX_REQUIRE(m, "kx_model_load_info: null model");
  if (bytes) *bytes = m->load_bytes;
  if (seconds) *seconds = m->load_seconds;
  return KX_OK;
}

extern "C" int kx_restart(kx_model *m, int32_t batch) {
  KX_REQUIRE(m, "kx_restart: null model");
  KX_REQUIRE(batch > 0 && batch <= m->max_batch, "kx_restart: batch=%d outside [1, %d]", batch, m->max_batch);
  m->batch = batch;
  m->pos = 0;
  m->sampled = false;
  return m->restart(batch);
}

extern "C" int kx_extend(kx_model *m, const uint32_t *h_ids, int32_t n, const int32_t *h_want, int32_t n_want, float *h_logits) {
  KX_REQUIRE(m && h_ids, "kx_extend: null argument");
  KX_REQUIRE(m->batch > 0, "kx_extend: no sequences (call kx_restart first)");
  KX_REQUIRE(n > 0 && n <= m->max_context - m->pos, "kx_extend: n=%d outside [1, %d]", n, m->max_context - m->pos);
  KX_REQUIRE(n_want >= 0 && (n_want == 0 || (h_want && h_logits)), "kx_extend: n_want=%d without places or output", n_want);
  for (int i = 0; i < n_want; ++i) KX_REQUIRE(h_want[i] >= 0 && h_want[i] < n, "kx_extend: place %d outside [0, %d)", h_want[i], n);
  return kx_guard("kx_extend", [&]() -> int {
    int rc = extend(m, h_ids, n, h_want, n_want, h_logits);
    return rc || !n_want ? rc : sync_and_check(m);
  });
}

extern "C" int kx_prefill(kx_model *m, const uint32_t *h_ids, int32_t batch, int32_t prompt_len) {
  KX_REQUIRE(m && h_ids, "kx_prefill: null argument");
  KX_REQUIRE(batch > 0 && batch <= m->max_batch, "kx_prefill: batch=%d outside [1, %d]", batch, m->max_batch);
  KX_REQUIRE(prompt_len > 0 && prompt_len <= m->max_context, "kx_prefill: prompt_len=%d outside [1, %d]", prompt_len, m->max_context);  // :555, :784
  int rc = check_ids(m, h_ids, (size_t)batch * prompt_len);
  if (rc) return rc;
  if ((rc = kx_restart(m, batch))) return rc;
  return kx_guard("kx_prefill", [&]() -> int { return extend(m, h_ids, prompt_len, nullptr, 0, nullptr); });
}

extern "C" int kx_decode_step(kx_model *m, const uint32_t *h_ids) {
  KX_REQUIRE(m, "kx_decode_step: null model");
  KX_REQUIRE(m->batch > 0, "kx_decode_step: no prefill has run");
  KX_REQUIRE(m->pos < m->max_context, "kx_decode_step: the context of %d positions is full", m->max_context);  // :784
  uint32_t *slot = m->ids + (size_t)m->pos * m->batch;
  int rc;
  if (h_ids) {
    if ((rc = check_ids(m, h_ids, m->batch))) return rc;
    KX_HIP(hipMemcpyAsync(slot, h_ids, (size_t)m->batch * 4, hipMemcpyHostToDevice, m->st));
    KX_HIP(hipStreamSynchronize(m->st));
  } else {
    KX_REQUIRE(m->sampled, "kx_decode_step: no sampled ids to feed (pass h_ids)");
    if ((rc = copy_ids(m, m->next, slot))) return rc;  // the sampler overwrites `next`; feed a copy
  }
  return m->step(slot, true, 1);
}

extern "C" int kx_greedy_sample(kx_model *m, uint32_t *h_out) {
  KX_REQUIRE(m && h_out, "kx_greedy_sample: null argument");
  KX_REQUIRE(m->sampled, "kx_greedy_sample: the last step did not sample");
  KX_HIP(hipMemcpyAsync(h_out, m->next, (size_t)m->batch * 4, hipMemcpyDeviceToHost, m->st));
  return sync_and_check(m);
}

extern "C" int kx_generate(kx_model *m, const uint32_t *h_prompt, int32_t batch, int32_t prompt_len, int32_t n_tokens,
                           int ignore_eos, uint32_t *h_out, int32_t *h_counts) {
  KX_REQUIRE(m && h_prompt && h_out && h_counts, "kx_generate: null argument");
  KX_REQUIRE(n_tokens > 0, "kx_generate: n_tokens=%d must be positive", n_tokens);  // :542
  KX_REQUIRE((int64_t)prompt_len + n_tokens <= m->max_context, "requested sequence exceeds the context of %d positions", m->max_context);  // :784
  int rc;
  KX_HIP(hipEventRecord(m->ev[0], m->st));
  if ((rc = kx_prefill(m, h_prompt, batch, prompt_len))) return rc;
  KX_HIP(hipEventRecord(m->ev[1], m->st));
  // Steps are enqueued without waiting for the host.  When the end-of-sequence id counts, the ids sampled so far are
  // read back every eighth step, and the loop ends once every sequence has sampled it (:887-888 stop there too):
  // at most eight steps are decoded for nothing.
  std::vector<uint32_t> hist((size_t)n_tokens * batch);
  std::vector<char> ended(batch, 0);
  int made = 0, seen = 0;  // history rows written on the device, and of those, rows the host has read
  auto read_back = [&]() -> int {
    if (seen == made) return KX_OK;
    KX_HIP(hipMemcpyAsync(hist.data() + (size_t)seen * batch, m->history + (size_t)seen * batch, (size_t)(made - seen) * batch * 4,
                          hipMemcpyDeviceToHost, m->st));
    KX_HIP(hipStreamSynchronize(m->st));
    for (; seen < made; ++seen)
      for (int b = 0; b < batch; ++b)
        if (hist[(size_t)seen * batch + b] == m->eos_id) ended[b] = 1;
    return KX_OK;
  };
  for (int i = 0; i < n_tokens; ++i) {  // :887-890
    if ((rc = copy_ids(m, m->next, m->history + (size_t)i * batch))) return rc;
    made = i + 1;
    if (!ignore_eos && (i & 7) == 7) {
      if ((rc = read_back())) return rc;
      bool all = true;
      for (int b = 0; b < batch; ++b) all = all && ended[b];
      if (all) break;
    }
    if (i + 1 < n_tokens && (rc = m->step(m->history + (size_t)i * batch, true, 1))) return rc;
  }
  KX_HIP(hipEventRecord(m->ev[2], m->st));
  if ((rc = read_back())) return rc;
  if ((rc = sync_and_check(m))) return rc;
  KX_HIP(hipEventElapsedTime(&m->ms_prefill, m->ev[0], m->ev[1]));
  KX_HIP(hipEventElapsedTime(&m->ms_decode, m->ev[1], m->ev[2]));
  m->steps_decoded = made;
  for (int b = 0; b < batch; ++b) {  // generation stops before the end-of-sequence id is emitted (:887-888)
    int n = 0;
    for (int i = 0; i < made; ++i) {
      const uint32_t id = hist[(size_t)i * batch + b];
      if (!ignore_eos && id == m->eos_id) break;
      h_out[(size_t)b * n_tokens + n++] = id;
    }
    h_counts[b] = n;
  }
  return KX_OK;
}

extern "C" int kx_model_set_prefill_chunk(kx_model *m, int32_t positions) {
  KX_REQUIRE(m, "kx_model_set_prefill_chunk: null model");
  KX_REQUIRE(positions >= 1 && positions <= m->step_tokens, "kx_model_set_prefill_chunk: positions=%d outside [1, %d]", positions, m->step_tokens);
  m->prefill_chunk = positions;
  return KX_OK;
}

extern "C" int kx_model_rewind(kx_model *m, int32_t positions) {
  KX_REQUIRE(m, "kx_model_rewind: null model");
  KX_REQUIRE(m->batch > 0, "kx_model_rewind: no prefill has run");
  KX_REQUIRE(positions >= 0 && positions <= m->pos, "kx_model_rewind: positions=%d outside [0, %d]", positions, m->pos);
  if (!positions) return KX_OK;
  int rc = m->rewind(positions);
  if (rc) return rc;
  m->pos -= positions;
  m->sampled = false;  // the sampled ids belonged to the last position
  return KX_OK;
}

extern "C" int kx_model_set_residual_record(kx_model *m, int on) {
  KX_REQUIRE(m, "kx_model_set_residual_record: null model");
  return m->set_residual_record(on != 0);
}
extern "C" int kx_model_residual(kx_model *m, int32_t layer, int32_t pos0, int32_t n, float *h_out) {
  KX_REQUIRE(m && h_out, "kx_model_residual: null argument");
  KX_REQUIRE(layer >= 0 && layer < m->n_layers && pos0 >= 0 && n >= 0 && pos0 + n <= m->pos, "kx_model_residual: layer %d, positions [%d, %d) of %d", layer,
             pos0, pos0 + n, m->pos);
  return m->residual(layer, pos0, n, h_out);
}

extern "C" int kx_model_steps_decoded(kx_model *m, int32_t *steps) {
  KX_REQUIRE(m && steps, "kx_model_steps_decoded: null argument");
  *steps = m->steps_decoded;
  return KX_OK;
}
extern "C" int kx_model_timing(kx_model *m, float *ms2) {
  KX_REQUIRE(m && ms2, "kx_model_timing: null argument");
  ms2[0] = m->ms_prefill;
  ms2[1] = m->ms_decode;
  return KX_OK;
}
extern "C" int kx_model_hidden(kx_model *m, uint16_t *h_out) {
  KX_REQUIRE(m && h_out && m->batch > 0, "kx_model_hidden: null argument or no step has run");
  return m->hidden_bf16(h_out);
}
extern "C" int kx_model_logits(kx_model *m, float *h_out) {
  KX_REQUIRE(m && h_out && m->sampled, "kx_model_logits: null argument or the last step did not sample");
  KX_HIP(hipMemcpyAsync(h_out, m->logits, (size_t)m->batch * m->vocab * 4, hipMemcpyDeviceToHost, m->st));
  KX_HIP(hipStreamSynchronize(m->st));
  return KX_OK;
}
extern "C" int kx_model_stream(kx_model *m, void **stream) {
  KX_REQUIRE(m && stream, "kx_model_stream: null argument");
  *stream = (void *)m->st;
  return KX_OK;
}
