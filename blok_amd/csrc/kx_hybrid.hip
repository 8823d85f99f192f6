// kx_hybrid.hip -- the hybrid decoder: weights, cache and state, one step of the stack, and its entry in the registry.
// The loops around a step -- prefill, decode, sampling -- are kx_stack.hip's, as for the other design.
//
// A step of T tokens (T = positions x sequences), per layer:
//   all input projections of the mixer as one product, the streams' read-out and the norm in front of it
//   -> attention over window and pooled blocks (kx_window.hip), latent attention (kx_latent.hip), or one of the recurrences
//      (kx_delta.hip, kx_ssd.hip, kx_wkv.hip)
//   -> output projection; its epilogue updates all residual streams
//   -> gate and up as one product with the clamped activation, norm in front -> down, which updates the streams.
// Where mixer and feed-forward read the same norm, the plain feed-forward's up is rows of the first product and its down
// columns of the output projection, and the router is rows of the first product; the chosen experts' gate and up run
// before the streams change, and up to 4 tokens their down rides in the output projection.
// Up to 4 tokens the products are GEMVs that build their activation rows themselves (kx_linear.hip).
// The residual streams, the projections a mixer reads, router logits, scores, recurrent state and convolution inputs are
// 32-bit in both number formats; bf16 are weights, activation rows of the products and the key/value cache.
#include <math.h>
#include <string.h>
#include <algorithm>
#include <map>
#include <vector>
#include "kx_argmax.h"
#include "kx_experts.h"
#include "kx_hybrid.h"
#include "kx_linear.h"
#include "kx_load.h"
#include "kx_math.h"
#include "kx_model.h"
#include "kx_safetensors.h"

namespace {

// one tensor of the files and where it goes
struct Slot {
  std::string name;
  int rows = 0, cols = 0;  // cols 0: one dimension
  void *dst = nullptr;
  int ld = 0;      // matrices: elements per row of the arena; 0: an array of floats
  int half = -1;   // 0, 1: gate, up rows of KX_GLU_BLOCK blocks
  float add = 0;   // arrays: added to every element
  float mean = 0, sigma = 0;  // random init
  size_t count() const { return (size_t)rows * (cols ? cols : 1); }
};

struct HyperW {
  float *in = nullptr, *mix = nullptr, *out = nullptr;
};
struct LayerW {
  float *norm1 = nullptr, *norm2 = nullptr;
  HyperW hc[2];
  KxMat in, o, gu, down;  // mixer projections back to back; output; gate and up; down
  int q_off = 0, k_off = 0, v_off = 0, g_off = 0, b_off = 0, a_off = 0;  // rows of `in`
  float *q_norm = nullptr, *k_norm = nullptr;
  float *conv = nullptr, *conv_b = nullptr, *a_log = nullptr, *dt_bias = nullptr, *skip = nullptr, *o_norm = nullptr;
  KxWindowCache cache;
  float *state = nullptr, *hist[2] = {nullptr, nullptr};  // hist: convolution inputs, or the position before (WKV)
  size_t state_floats = 0, hist_floats = 0;  // per sequence
  // WKV
  int r_off = 0, w_off = 0, var_row[KX_MAX_VARIANTS] = {}, n_var = 1;
  float *mu = nullptr, *w0 = nullptr, *u = nullptr;
  KxMat w2;
  // LATENT
  int kv_off = 0;
  KxMat uq, uk, uv;
  float *dq_norm = nullptr, *kv_norm = nullptr, *sinks = nullptr;
  void *rows = nullptr;
  const float2 *turns = nullptr;
  // a parallel layer's feed-forward: rows of `in` from up_off on, columns of `o` from o_ld on; or rows of `in` with the
  // router, experts' matrices one after the other in gu and down
  int up_off = 0, o_ld = 0, router_off = 0;
  float *router_b = nullptr;
  size_t gu_stride = 0, down_stride = 0;
};

struct HybridModel : kx_model {
  KxHybridConfig c;
  std::string name;
  bool f32 = false;
  std::vector<LayerW> L;
  KxMat embed, head;
  float *final_norm = nullptr;
  std::vector<Slot> slots;
  float *streams = nullptr, *proj = nullptr, *mixed = nullptr, *work = nullptr, *part = nullptr;
  // rows: of the products in front of a sublayer (with EXPERTS read twice); out_rows: of those inside it and behind it
  void *rows = nullptr, *out_rows = nullptr, *att = nullptr, *q = nullptr, *mid = nullptr;
  float *lat_q = nullptr, *expert_y = nullptr;
  KxLatentScratch lat;
  KxExpertSlots slots_of;        // of a step's experts
  std::map<std::pair<int, double>, std::pair<float2 *, KxLatentSpec>> turns;  // by rotated dimensions and base
  int proj_ld = 0, mid_ld = 0, part_tokens = 0;
  size_t part_floats = 0;
  int *want = nullptr;           // token rows of row_logits
  float init_sigma_ = 0;
  int hist_cur = 0;              // which of the two convolution histories the next step reads
  float *record = nullptr;       // [n_layers][max_context][max_batch][width]

  const char *design() const override { return name.c_str(); }
  int step(const uint32_t *d_ids, bool sample, int C) override;
  int step_positions(int batch_) const override { return std::max(1, step_tokens / batch_); }
  int restart(int batch_) override;
  int row_logits(const int *token_rows, int n, float *d_out) override;
  int logit_rows() const override { return std::max(max_batch, 64); }
  int rewind(int positions) override {
    kx_set_error("kx_model_rewind: %s keeps recurrent state, which does not go back", design());
    return KX_ERR_ARG;
  }
  int hidden_bf16(uint16_t *h_out) override;
  int set_residual_record(bool on) override;
  int residual(int layer, int pos0, int n, float *h_out) override;
  ~HybridModel() override {
    if (record) (void)hipFree(record);
  }
  size_t layout(char *base);
  int find(const std::string &dir, const KxTensorMap &files) const;
  void ranks(const KxTensorMap &files);
  int latent(const KxHybridLayer &l, const LayerW &w, int C);
  int fill(const KxTensorMap &files, const kx_open_options &o);
  int pack(const Slot &s, const void *src, bool src_f32);
  int logits_of(const float *x, const int *map, int n, float *d_out);
};

// ---- kernels ----
template <class T>
__global__ void __launch_bounds__(256) pack_k(const void *src, int src_f32, T *dst, int rows, int cols, int ld, int half, float add) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (size_t)rows * cols) return;
  const int r = (int)(i / cols), col = (int)(i - (size_t)r * cols);
  const float v = (src_f32 ? ((const float *)src)[i] : kx_bf16_f32(((const uint16_t *)src)[i])) + add;
  const int to = half < 0 ? r : (r / KX_GLU_BLOCK) * 2 * KX_GLU_BLOCK + r % KX_GLU_BLOCK + half * KX_GLU_BLOCK;
  if constexpr (sizeof(T) == 4) dst[(size_t)to * ld + col] = v;
  else dst[(size_t)to * ld + col] = kx_bf16_rne(v);
}
template <class T>
__global__ void __launch_bounds__(256) embed_streams_k(const T *__restrict__ embed, int ld, const uint32_t *__restrict__ ids, float *__restrict__ x, int width,
                                                       int streams) {
  const T *e = embed + (size_t)ids[blockIdx.x] * ld;
  float *o = x + (size_t)blockIdx.x * streams * width;
  for (int c = threadIdx.x; c < width; c += 256) {
    float v;
    if constexpr (sizeof(T) == 4) v = e[c];
    else v = kx_bf16_f32(e[c]);
    for (int s = 0; s < streams; ++s) o[(size_t)s * width + c] = v;
  }
}
// sum of the streams of token blockIdx.x into row (blockIdx.x / nb) * stride + blockIdx.x % nb of out
__global__ void __launch_bounds__(256) sum_streams_k(const float *__restrict__ x, float *__restrict__ out, int width, int streams, int nb, int stride) {
  const int t = blockIdx.x;
  const float *p = x + (size_t)t * streams * width;
  float *o = out + ((size_t)(t / nb) * stride + t % nb) * width;
  for (int c = threadIdx.x; c < width; c += 256) {
    float v = p[c];
    for (int s = 1; s < streams; ++s) v += p[(size_t)s * width + c];
    o[c] = v;
  }
}

// Lays everything out from `base` on (nullptr: sizes only) and lists the tensors the files have to hold.
size_t HybridModel::layout(char *base) {
  KxPlan p;
  slots.clear();
  L.assign(c.layers.size(), LayerW());
  turns.clear();
  const size_t es = f32 ? 4 : 2;
  const int S = c.streams, W = c.width;
  const size_t T = step_tokens, B = max_batch;
  auto at = [&](size_t bytes) -> char * {
    const size_t off = p.take(bytes);
    return base ? base + off : nullptr;
  };
  auto vec_at = [&](const std::string &n, int rows, int cols, float *dst, float mean, float sigma, float add = 0.0f) {
    Slot s;
    s.name = n; s.rows = rows; s.cols = cols; s.mean = mean; s.sigma = sigma; s.add = add; s.dst = dst;
    slots.push_back(s);
    return dst;
  };
  auto vec = [&](const std::string &n, int rows, int cols, float mean, float sigma) {
    return vec_at(n, rows, cols, (float *)at((size_t)rows * (cols ? cols : 1) * 4), mean, sigma);
  };
  auto model_norm = [&](const std::string &n) {
    return c.norm_about_one ? vec_at(n, W, 0, (float *)at((size_t)W * 4), 0.0f, 0.02f, 1.0f) : vec(n, W, 0, 1.0f, 0.02f);
  };
  auto mat = [&](int rows, int cols, size_t copies = 1) {
    KxMat m;
    m.rows = rows; m.cols = cols; m.ld = kx_pad(cols, KX_LD);
    m.w = at(copies * rows * m.ld * es);
    return m;
  };
  const float sg = init_sigma_;
  // rows x cols of m from (row0, col0) on
  auto part_of = [&](const KxMat &m, size_t row0, int col0, const std::string &n, int rows, int cols, int half, float sigma) {
    Slot s;
    s.name = n; s.rows = rows; s.cols = cols; s.ld = m.ld; s.half = half; s.sigma = sigma;
    s.dst = m.w ? (char *)m.w + (row0 * m.ld + col0) * es : nullptr;
    slots.push_back(s);
  };
  embed = mat(c.vocab, W);
  part_of(embed, 0, 0, "embed", c.vocab, W, -1, 1.0f);
  int row_ld = kx_pad(W, KX_LD), out_ld = 0, variants = 1, att_ld = 0;
  proj_ld = mid_ld = 0;
  size_t q_cols = 0, o_cols = 0, work_floats = 0, expert_slots = 0, expert_mid = 0, tiles = 0, lat_q_floats = 0, lat_qx = 0, lat_cols = 0;
  part_floats = 0;
  lat = KxLatentScratch();
  for (size_t i = 0; i < c.layers.size(); ++i) {
    const KxHybridLayer &l = c.layers[i];
    LayerW &w = L[i];
    const std::string n = "l" + std::to_string(i) + ".", m = n + "mix.", ffn = n + "mlp.";
    auto hyper = [&](int q) {
      HyperW h;
      if (!c.hyper) return h;
      const std::string k = n + "hc" + std::to_string(q) + ".";
      h.in = vec(k + "in", S, 0, 1.0f / S, 0.02f);
      h.out = vec(k + "out", S, 0, 1.0f, 0.02f);
      h.mix = vec(k + "mix", S, S, 1.0f / S, 0.02f);
      return h;
    };
    w.norm1 = model_norm(n + "norm1");
    w.hc[0] = hyper(1);
    // the mixer's projections and what else reads its norm, each from a multiple of 32 rows on (of KX_VARIANT_ROWS where
    // the rows differ)
    struct Piece { std::string name; int rows; int *off; };
    std::vector<Piece> pieces;
    int out_cols = 0;
    if (l.mixer == KxHybridLayer::ATTENTION) {
      out_cols = l.attn.heads * l.attn.vdim;
      pieces = {{m + "q", l.attn.heads * l.attn.dim, &w.q_off}, {m + "k", l.attn.kv_heads * l.attn.dim, &w.k_off}, {m + "v", l.attn.kv_heads * l.attn.vdim, &w.v_off}};
      if (l.gate) pieces.push_back({m + "g", out_cols, &w.g_off});
    } else if (l.mixer == KxHybridLayer::DELTA) {
      out_cols = l.delta.heads * l.delta.vdim;
      pieces = {{m + "q", l.delta.kv_heads * l.delta.dim, &w.q_off}, {m + "k", l.delta.kv_heads * l.delta.dim, &w.k_off}, {m + "v", out_cols, &w.v_off},
                {m + "g", out_cols, &w.g_off}, {m + "b", l.delta.heads, &w.b_off}, {m + "a", l.delta.heads, &w.a_off}};
    } else if (l.mixer == KxHybridLayer::SSD) {
      out_cols = kx_ssd_inner(l.ssd);
      pieces = {{m + "in", out_cols + kx_ssd_channels(l.ssd) + l.ssd.heads, &w.q_off}};  // gate; x, B, C; dt
    } else if (l.mixer == KxHybridLayer::WKV) {
      out_cols = l.wkv.heads * l.wkv.dim;
      pieces = {{m + "r", out_cols, &w.r_off}, {m + "k", out_cols, &w.k_off}, {m + "v", out_cols, &w.v_off}, {m + "g", out_cols, &w.g_off}, {m + "w1", l.wkv.rank, &w.w_off}};
    } else {
      out_cols = l.latent.heads * l.latent.vdim;
      pieces = {{m + "dq", l.q_rank, &w.q_off}, {m + "dkv", l.latent.kv_rank + l.latent.rot_dim, &w.kv_off}};
      if (l.gate) pieces.push_back({m + "g", out_cols, &w.g_off});
    }
    const bool up = c.parallel && l.ff_kind == KxHybridLayer::GELU, experts = l.ff_kind == KxHybridLayer::EXPERTS;
    if (up) pieces.push_back({ffn + "up", l.ff, &w.up_off});
    if (experts) pieces.push_back({ffn + "router", l.experts, &w.router_off});
    const bool shifted = l.mixer == KxHybridLayer::WKV;
    int rows_in = 0;
    for (size_t x = 0; x < pieces.size(); ++x) {
      if (shifted) {
        rows_in = kx_pad(rows_in, KX_VARIANT_ROWS);
        w.var_row[x] = rows_in;
      }
      *pieces[x].off = rows_in;
      rows_in += kx_pad(pieces[x].rows, 32);
    }
    if (shifted) {
      w.n_var = 6;  // five mixes and the row itself
      if (pieces.size() < 6) w.var_row[5] = kx_pad(rows_in, KX_VARIANT_ROWS);
      variants = 6;
      w.mu = (float *)at((size_t)5 * W * 4);
      for (int x = 0; x < 5; ++x) vec_at(m + "mu." + "rkvgw"[x], W, 0, w.mu ? w.mu + (size_t)x * W : nullptr, 0.5f, 0.2f);
    }
    w.in = mat(rows_in, W);
    for (const Piece &x : pieces) part_of(w.in, *x.off, 0, x.name, x.rows, W, -1, sg);
    w.o_ld = kx_pad(out_cols, KX_LD);
    w.o = mat(W, up ? w.o_ld + l.ff : out_cols);
    part_of(w.o, 0, 0, m + "o", W, out_cols, -1, sg);
    if (up) part_of(w.o, 0, w.o_ld, ffn + "down", W, l.ff, -1, sg);
    proj_ld = std::max(proj_ld, up ? w.up_off : rows_in);
    out_ld = std::max(out_ld, w.o.ld);
    const int steps = step_tokens + max_batch * (KX_SCAN_BLOCK - 1);  // a batch's sequences are padded to blocks each
    if (l.mixer == KxHybridLayer::ATTENTION) {
      if (l.qk_norm) {
        w.q_norm = vec(m + "q.norm", l.attn.heads * l.attn.dim, 0, 1.0f, 0.02f);
        w.k_norm = vec(m + "k.norm", l.attn.kv_heads * l.attn.dim, 0, 1.0f, 0.02f);
      }
      att_ld = std::max(att_ld, w.o.ld);
      q_cols = std::max(q_cols, (size_t)l.attn.heads * kx_pad(l.attn.dim, 32));
      part_floats = std::max(part_floats, kx_window_part_floats(l.attn, max_context, part_tokens));
    } else if (l.mixer == KxHybridLayer::DELTA) {
      const KxDeltaSpec &d = l.delta;
      const int C = kx_delta_channels(d), nq = d.kv_heads * d.dim;
      w.conv = (float *)at((size_t)C * d.taps * 4);  // q, k and v channels back to back
      int ch = 0;
      for (const Piece &x : {Piece{"q.conv", nq, nullptr}, Piece{"k.conv", nq, nullptr}, Piece{"v.conv", out_cols, nullptr}}) {
        vec_at(m + x.name, x.rows, d.taps, w.conv ? w.conv + (size_t)ch * d.taps : nullptr, 0.0f, 0.5f);
        ch += x.rows;
      }
      w.a_log = vec(m + "A_log", d.heads, 0, 0.0f, 0.5f);
      w.dt_bias = vec(m + "dt_bias", d.heads, 0, -2.0f, 0.5f);
      w.o_norm = vec(m + "norm", d.vdim, 0, 1.0f, 0.02f);
      work_floats = std::max(work_floats, kx_delta_work_floats(d, 1, step_tokens + max_batch * (KX_DELTA_BLOCK - 1)));
      w.state_floats = (size_t)d.heads * d.dim * d.vdim;
      w.hist_floats = (size_t)(d.taps - 1) * C;
    } else if (l.mixer == KxHybridLayer::SSD) {
      const KxSsdSpec &s = l.ssd;
      const int C = kx_ssd_channels(s);
      w.conv = vec(m + "conv", C, s.taps, 0.0f, 0.5f);
      w.conv_b = vec(m + "conv.b", C, 0, 0.0f, 0.1f);
      w.dt_bias = vec(m + "dt_bias", s.heads, 0, -2.0f, 0.5f);
      w.a_log = vec(m + "A_log", s.heads, 0, 0.0f, 0.5f);
      w.skip = vec(m + "D", s.heads, 0, 1.0f, 0.1f);
      w.o_norm = vec(m + "norm", out_cols, 0, 1.0f, 0.02f);
      work_floats = std::max(work_floats, kx_ssd_work_floats(s, 1, steps));
      w.state_floats = (size_t)s.heads * s.state * s.vdim;
      w.hist_floats = (size_t)(s.taps - 1) * C;
    } else if (l.mixer == KxHybridLayer::WKV) {
      const KxWkvSpec &s = l.wkv;
      w.w2 = mat(out_cols, s.rank);
      part_of(w.w2, 0, 0, m + "w2", out_cols, s.rank, -1, sg);
      w.w0 = vec(m + "w0", out_cols, 0, -2.0f, 0.5f);
      w.u = vec(m + "u", s.heads, s.dim, 0.0f, 0.5f);
      w.o_norm = vec(m + "norm", out_cols, 0, 1.0f, 0.02f);
      out_ld = std::max(out_ld, w.w2.ld);
      work_floats = std::max(work_floats, kx_wkv_work_floats(s, 1, steps));
      w.state_floats = (size_t)s.heads * s.dim * s.dim;
      w.hist_floats = W;
    } else {
      const KxLatentSpec &s = l.latent;
      w.uq = mat(s.heads * (s.dim + s.rot_dim), l.q_rank);
      part_of(w.uq, 0, 0, m + "uq", w.uq.rows, l.q_rank, -1, sg);
      w.uk = mat(s.heads * s.dim, s.kv_rank);
      part_of(w.uk, 0, 0, m + "uk", w.uk.rows, s.kv_rank, -1, sg);
      w.uv = mat(out_cols, s.kv_rank);
      part_of(w.uv, 0, 0, m + "uv", out_cols, s.kv_rank, -1, sg);
      w.dq_norm = vec(m + "dq.norm", l.q_rank, 0, 1.0f, 0.02f);
      w.kv_norm = vec(m + "dkv.norm", s.kv_rank, 0, 1.0f, 0.02f);
      if (s.sink) w.sinks = vec(m + "sink", s.heads, 0, 0.0f, 0.5f);
      att_ld = std::max(att_ld, w.o.ld);
      out_ld = std::max(out_ld, w.uq.ld);
      lat_cols = std::max(lat_cols, (size_t)w.uq.rows);
      KxLatentScratch x;
      size_t qf, qx;
      kx_latent_scratch(s, max_batch, max_context, step_tokens, &x, &qf, &qx);
      lat_q_floats = std::max(lat_q_floats, qf);
      lat_qx = std::max(lat_qx, qx);
      lat.q_tokens = x.q_tokens;
      lat.k_elems = std::max(lat.k_elems, x.k_elems);
      lat.v_elems = std::max(lat.v_elems, x.v_elems);
      part_floats = std::max(part_floats, x.part_floats);
      if (s.rot) turns[{s.rot, s.base}] = {nullptr, s};
    }
    if (l.mixer != KxHybridLayer::ATTENTION && l.mixer != KxHybridLayer::LATENT) o_cols = std::max(o_cols, (size_t)out_cols);
    if (l.ff_kind == KxHybridLayer::GLU) {
      w.norm2 = model_norm(n + "norm2");
      w.hc[1] = hyper(2);
      w.gu = mat(2 * kx_pad(l.ff, KX_GLU_BLOCK), W);
      part_of(w.gu, 0, 0, ffn + "gate", l.ff, W, 0, sg);
      part_of(w.gu, 0, 0, ffn + "up", l.ff, W, 1, sg);
      w.down = mat(W, l.ff);
      part_of(w.down, 0, 0, ffn + "down", W, l.ff, -1, sg);
      mid_ld = std::max(mid_ld, w.down.ld);
    } else if (up) {
      mid_ld = std::max(mid_ld, w.o.ld - w.o_ld);
    } else if (experts) {
      w.router_b = vec(ffn + "router.b", l.experts, 0, 0.0f, 0.1f);
      w.gu = mat(2 * kx_pad(l.ff, KX_GLU_BLOCK), W, l.experts);
      w.down = mat(W, l.ff, l.experts);
      w.gu_stride = (size_t)w.gu.rows * w.gu.ld;
      w.down_stride = (size_t)W * w.down.ld;
      for (int e = 0; e < l.experts; ++e) {
        const std::string k = ffn + "e" + std::to_string(e) + ".";
        part_of(w.gu, (size_t)e * w.gu.rows, 0, k + "gate", l.ff, W, 0, sg);
        part_of(w.gu, (size_t)e * w.gu.rows, 0, k + "up", l.ff, W, 1, sg);
        part_of(w.down, (size_t)e * W, 0, k + "down", W, l.ff, -1, sg);
      }
      const size_t pairs = std::max(T, B) * l.top;
      expert_slots = std::max(expert_slots, pairs);
      expert_mid = std::max(expert_mid, pairs * w.down.ld);
      tiles = std::max(tiles, (size_t)kx_expert_tiles((int)std::max(T, B), l.top, l.experts, 64));
    }
  }
  final_norm = model_norm("final.norm");
  head = mat(c.vocab, W);
  part_of(head, 0, 0, "head", c.vocab, W, -1, sg);
  for (auto &t : turns) t.second.first = (float2 *)at((size_t)max_context * (t.first.first / 2) * sizeof(float2));
  weight_bytes = p.total;

  for (size_t i = 0; i < c.layers.size(); ++i) {
    const KxHybridLayer &l = c.layers[i];
    LayerW &w = L[i];
    if (l.mixer == KxHybridLayer::ATTENTION) {
      size_t e[4];
      kx_window_shape(l.attn, max_context, std::min(step_tokens, max_context), &w.cache, e);
      w.cache.k = at(e[0] * max_batch * es);
      w.cache.v = at(e[1] * max_batch * es);
      w.cache.pk = at(e[2] * max_batch * es);
      w.cache.pv = at(e[3] * max_batch * es);
    } else if (l.mixer == KxHybridLayer::LATENT) {
      w.rows = at(B * max_context * kx_latent_row(l.latent) * es);
      w.turns = l.latent.rot ? turns[{l.latent.rot, l.latent.base}].first : nullptr;
    } else {
      w.state = (float *)at(w.state_floats * max_batch * 4);
      for (auto &h : w.hist) h = (float *)at(w.hist_floats * max_batch * 4);
    }
  }
  cache_bytes = p.total - weight_bytes;

  streams = (float *)at(T * S * W * 4);
  proj = (float *)at(T * proj_ld * 4);
  mixed = (float *)at(T * o_cols * 4);
  work = (float *)at(work_floats * 4);
  part = (float *)at(part_floats * 4);
  rows = at(std::max(T * variants, (size_t)logit_rows()) * row_ld * es);
  out_rows = at(T * out_ld * es);
  att = at(T * att_ld * es);
  q = at(T * q_cols * es);
  mid = at(std::max(T * mid_ld, expert_mid) * es);
  lat_q = (float *)at(T * lat_cols * 4);
  lat.q = (float *)at(lat_q_floats * 4);
  lat.qx = at(lat_qx * es);
  lat.kx = at(lat.k_elems * es);
  lat.vx = at(lat.v_elems * es);
  lat.part = part;
  lat.part_floats = part_floats;
  slots_of.ids = (int *)at(expert_slots * 4);
  slots_of.gather = (int *)at(expert_slots * 4);
  slots_of.slot_of = (int *)at(expert_slots * 4);
  slots_of.weights = (float *)at(expert_slots * 4);
  slots_of.slot_weight = (float *)at(expert_slots * 4);
  slots_of.tiles = (int4 *)at(tiles * sizeof(int4));
  slots_of.n_tiles = (int *)at(4);
  expert_y = (float *)at(expert_slots * W * 4);
  logits = (float *)at((size_t)logit_rows() * c.vocab * 4);
  argmax_scratch = (float *)at(KX_ARGMAX_SCRATCH_FLOATS(B) * 4);
  ids = (uint32_t *)at((size_t)max_context * B * 4);
  next = (uint32_t *)at(B * 4);
  history = (uint32_t *)at((size_t)max_context * B * 4);
  want = (int *)at((size_t)logit_rows() * 4);
  scratch_bytes = p.total - weight_bytes - cache_bytes;
  return p.total;
}

// sizes that a configuration leaves to the shapes of the tensors
void HybridModel::ranks(const KxTensorMap &files) {
  for (size_t i = 0; i < c.layers.size(); ++i) {
    KxHybridLayer &l = c.layers[i];
    if (l.mixer != KxHybridLayer::WKV || l.wkv.rank) continue;
    l.wkv.rank = 64;  // of random weights
    const auto f = files.find("l" + std::to_string(i) + ".mix.w1");
    if (f != files.end()) l.wkv.rank = std::max(1, atoi(f->second.shape.c_str()));
  }
}

int HybridModel::pack(const Slot &s, const void *src, bool src_f32) {
  const int rows_ = s.rows, cols = s.cols ? s.cols : 1, ld = s.ld ? s.ld : cols;
  const dim3 grid((unsigned)((s.count() + 255) / 256));
  if (f32 || !s.ld) hipLaunchKernelGGL(pack_k<float>, grid, dim3(256), 0, st, src, src_f32, (float *)s.dst, rows_, cols, ld, s.half, s.add);
  else hipLaunchKernelGGL(pack_k<uint16_t>, grid, dim3(256), 0, st, src, src_f32, (uint16_t *)s.dst, rows_, cols, ld, s.half, s.add);
  KX_LAUNCH_CHECK();
  return KX_OK;
}

struct Staging {  // device memory that is gone at the end of a scope
  char *p = nullptr;
  ~Staging() { if (p) (void)hipFree(p); }
};

// each of the tensors the model reads with the shape it has to have; needs no GPU
int HybridModel::find(const std::string &dir, const KxTensorMap &files) const {
  for (const Slot &s : slots) {
    const auto f = files.find(s.name);
    KX_REQUIRE(f != files.end(), "missing tensor: %s (%s)", s.name.c_str(), dir.c_str());
    const std::string shape = std::to_string(s.rows) + (s.cols ? "x" + std::to_string(s.cols) : "");
    KX_REQUIRE(f->second.shape == shape && f->second.dtype != "i32", "tensor %s is %s %s, expected bf16 or f32 %s", s.name.c_str(), f->second.dtype.c_str(),
               f->second.shape.c_str(), shape.c_str());
  }
  return KX_OK;
}

// The tensors from the files (or from the generator), through a staging buffer: the files have rows without padding,
// gate and up apart, and bf16 where the arena may have f32.
int HybridModel::fill(const KxTensorMap &files, const kx_open_options &o) {
  constexpr size_t BATCH = (size_t)1 << 30;
  auto bytes_of = [&](const Slot &s) { return ((o.random_init ? s.count() * 2 : files.at(s.name).data_bytes) + 255) & ~(size_t)255; };
  size_t most = 0;
  for (size_t i = 0; i < slots.size();) {  // the largest batch
    size_t sum = bytes_of(slots[i]), j = i + 1;
    while (j < slots.size() && sum + bytes_of(slots[j]) <= BATCH) sum += bytes_of(slots[j++]);
    most = std::max(most, sum);
    i = j;
  }
  Staging stage;
  KX_HIP(hipMalloc((void **)&stage.p, most));
  for (size_t i = 0; i < slots.size();) {
    std::vector<KxLoadItem> items;
    size_t sum = 0, j = i;
    for (; j < slots.size() && (j == i || sum + bytes_of(slots[j]) <= BATCH); ++j) {
      if (o.random_init) KX_DO(kx_fill_affine_bf16(stage.p + sum, slots[j].count(), o.seed, 1 + j, slots[j].mean, slots[j].sigma, st));
      else items.push_back(KxLoadItem{&files.at(slots[j].name), stage.p + sum, false});
      sum += bytes_of(slots[j]);
    }
    uint64_t bytes = 0;
    double seconds = 0;
    if (!o.random_init) KX_DO(kx_load_run(items, &bytes, &seconds));
    load_bytes += bytes;
    load_seconds += seconds;
    sum = 0;
    for (; i < j; ++i) {
      KX_DO(pack(slots[i], stage.p + sum, !o.random_init && files.at(slots[i].name).dtype == "f32"));
      sum += bytes_of(slots[i]);
    }
    KX_HIP(hipStreamSynchronize(st));  // the buffer is used again
  }
  return KX_OK;
}

int HybridModel::restart(int batch_) {
  for (const LayerW &w : L) {
    if (w.state) KX_HIP(hipMemsetAsync(w.state, 0, w.state_floats * batch_ * 4, st));
    if (w.hist_floats) KX_HIP(hipMemsetAsync(w.hist[hist_cur], 0, w.hist_floats * batch_ * 4, st));
  }
  return KX_OK;
}

int HybridModel::logits_of(const float *x, const int *map, int n, float *d_out) {
  KxLinArgs g;
  g.m = head;
  g.tokens = n;
  g.row.kind = KX_ROW_NORM; g.row.cols = c.width; g.row.rows_map = map; g.row.streams = x; g.row.n_streams = c.streams; g.row.groups = c.groups;
  g.row.w = final_norm; g.row.eps = c.eps;
  g.out = d_out;
  g.out_ld = c.vocab;
  return kx_linear_launch(f32, g, rows, st);
}

// latent attention of a layer, from proj into att
int HybridModel::latent(const KxHybridLayer &l, const LayerW &w, int C) {
  KxLinArgs g;  // the queries from their latent
  g.m = w.uq;
  g.tokens = batch * C;
  g.row.kind = KX_ROW_NORM; g.row.cols = l.q_rank; g.row.streams = proj + w.q_off; g.row.streams_ld = proj_ld; g.row.w = w.dq_norm; g.row.eps = c.eps;
  g.out = lat_q;
  g.out_ld = w.uq.rows;
  KX_DO(kx_linear_launch(f32, g, out_rows, st));
  KxLatentArgs a;
  a.s = l.latent;
  a.rows = w.rows; a.cap = max_context;
  a.proj = proj; a.proj_ld = proj_ld; a.kv_off = w.kv_off; a.g_off = l.gate ? w.g_off : -1;
  a.q = lat_q; a.q_ld = w.uq.rows;
  a.kv_norm = w.kv_norm; a.eps = c.eps;
  a.uk = w.uk; a.uv = w.uv;
  a.sinks = w.sinks; a.turns = w.turns;
  a.batch = batch; a.positions = C; a.pos = pos;
  a.out = att; a.out_ld = w.o.ld;
  a.x = lat;
  return kx_latent_launch(f32, a, st);
}

int HybridModel::step(const uint32_t *d_ids, bool sample, int C) {
  const int T = batch * C, S = c.streams, W = c.width;
  KX_REQUIRE(T > 0 && T <= std::max(step_tokens, max_batch), "%s: a step of %d tokens, at most %d", design(), T, step_tokens);
  const size_t es = f32 ? 4 : 2;
  if (f32) hipLaunchKernelGGL(embed_streams_k<float>, dim3(T), dim3(256), 0, st, (const float *)embed.w, embed.ld, d_ids, streams, W, S);
  else hipLaunchKernelGGL(embed_streams_k<uint16_t>, dim3(T), dim3(256), 0, st, (const uint16_t *)embed.w, embed.ld, d_ids, streams, W, S);
  KX_LAUNCH_CHECK();
  for (int i = 0; i < n_layers; ++i) {
    const KxHybridLayer &l = c.layers[i];
    LayerW &w = L[i];
    auto read = [&](KxLinArgs &g, const KxMat &m, const float *norm, const HyperW &h) {  // norm(sum_s in[s] x_s) in front of m
      g.m = m;
      g.tokens = T;
      g.row.kind = KX_ROW_NORM; g.row.cols = W; g.row.streams = streams; g.row.n_streams = S; g.row.in = h.in; g.row.groups = c.groups;
      g.row.w = norm; g.row.eps = c.eps;
    };
    auto write = [&](KxLinArgs &g, const KxMat &m, const HyperW &h) {  // the product into the streams
      g.m = m;
      g.tokens = T;
      g.row.cols = m.cols;
      g.epi = KX_LIN_STREAMS;
      g.streams = streams; g.n_streams = S; g.mix = h.mix; g.outw = h.out;
    };
    const bool up = c.parallel && l.ff_kind == KxHybridLayer::GELU, experts = l.ff_kind == KxHybridLayer::EXPERTS, shifted = l.mixer == KxHybridLayer::WKV;
    const bool in_memory = l.mixer == KxHybridLayer::ATTENTION || l.mixer == KxHybridLayer::LATENT;  // the mixer leaves rows of the output product
    KxLinArgs in, out;
    read(in, w.in, w.norm1, w.hc[0]);
    in.out = proj;
    in.out_ld = proj_ld;
    if (shifted) {
      in.row.kind = KX_ROW_SHIFT; in.row.mu = w.mu; in.row.n_mix = 5; in.row.batch = batch; in.row.tokens = T;
      in.row.prev = w.hist[hist_cur]; in.row.prev_out = w.hist[hist_cur ^ 1];
      in.n_var = w.n_var;
      memcpy(in.var_row, w.var_row, sizeof in.var_row);
    }
    if (up) {  // behind the mixer's rows, or in a buffer that the output product's rows go on with
      in.act_from = w.up_off;
      in.mid = in_memory ? (char *)att + w.o_ld * es : mid;
      in.mid_ld = in_memory ? w.o.ld : w.o.ld - w.o_ld;
    }
    KX_DO(kx_linear_launch(f32, in, rows, st));
    write(out, w.o, w.hc[0]);
    if (in_memory) {
      out.row.x = att;
      out.row.x_ld = w.o.ld;
    } else {
      out.row.kind = KX_ROW_GATED;
      out.row.o = mixed; out.row.gate = proj + w.g_off; out.row.gate_ld = proj_ld; out.row.w = w.o_norm; out.row.eps = c.eps;
      out.row.w_per_column = l.mixer != KxHybridLayer::DELTA;
      if (up) {
        out.row.tail = mid; out.row.tail_ld = in.mid_ld; out.row.head_ld = w.o_ld;
      }
    }
    if (l.mixer == KxHybridLayer::ATTENTION) {
      KxWindowArgs a;
      a.s = l.attn; a.c = w.cache;
      a.proj = proj; a.proj_ld = proj_ld; a.q_off = w.q_off; a.k_off = w.k_off; a.v_off = w.v_off; a.g_off = l.gate ? w.g_off : -1;
      a.q_norm = w.q_norm; a.k_norm = w.k_norm; a.eps = c.eps;
      a.batch = batch; a.positions = C; a.pos = pos;
      a.out = att; a.out_ld = w.o.ld; a.q = q; a.part = part; a.part_floats = part_floats;
      KX_DO(kx_window_launch(f32, a, st));
    } else if (l.mixer == KxHybridLayer::DELTA) {
      KxDeltaArgs d;
      d.s = l.delta;
      d.proj = proj; d.proj_ld = proj_ld; d.q_off = w.q_off; d.k_off = w.k_off; d.v_off = w.v_off; d.b_off = w.b_off; d.a_off = w.a_off;
      d.conv = w.conv; d.a_log = w.a_log; d.dt_bias = w.dt_bias;
      d.state = w.state; d.hist = w.hist[hist_cur]; d.hist_out = w.hist[hist_cur ^ 1];
      d.batch = batch; d.positions = C;
      d.o = mixed; d.work = work;
      KX_DO(kx_delta_launch(d, st));
      out.row.heads = l.delta.heads; out.row.vdim = l.delta.vdim;
    } else if (l.mixer == KxHybridLayer::SSD) {
      KxSsdArgs d;
      const int inner = kx_ssd_inner(l.ssd);
      d.s = l.ssd;
      d.proj = proj; d.proj_ld = proj_ld; d.x_off = inner; d.dt_off = inner + kx_ssd_channels(l.ssd);
      d.conv = w.conv; d.conv_bias = w.conv_b; d.a_log = w.a_log; d.dt_bias = w.dt_bias; d.skip = w.skip;
      d.state = w.state; d.hist = w.hist[hist_cur]; d.hist_out = w.hist[hist_cur ^ 1];
      d.batch = batch; d.positions = C;
      d.y = mixed; d.work = work;
      KX_DO(kx_ssd_launch(d, st));
      out.row.heads = l.norm_groups; out.row.vdim = inner / l.norm_groups; out.row.gate_first = true;
    } else if (l.mixer == KxHybridLayer::WKV) {
      KxWkvArgs d;
      d.s = l.wkv;
      d.proj = proj; d.proj_ld = proj_ld; d.r_off = w.r_off; d.k_off = w.k_off; d.v_off = w.v_off; d.w_off = w.w_off;
      d.w2 = w.w2; d.w0 = w.w0; d.u = w.u;
      d.state = w.state;
      d.batch = batch; d.positions = C;
      d.o = mixed; d.work = work; d.rows = out_rows;
      KX_DO(kx_wkv_launch(f32, d, st));
      out.row.heads = l.wkv.heads; out.row.vdim = l.wkv.dim;
    } else {
      KX_DO(latent(l, w, C));
    }
    if (experts) {
      KxExpertFf f;
      read(f.gu, w.gu, w.norm1, w.hc[0]);
      f.gu.limit = l.limit; f.gu.alpha = l.alpha; f.gu.bias = l.bias;
      f.out = out;
      f.down = w.down; f.gu_stride = w.gu_stride; f.down_stride = w.down_stride;
      f.e.experts = l.experts; f.e.top = l.top; f.e.logits = proj + w.router_off; f.e.logits_ld = proj_ld; f.e.bias = w.router_b;
      f.s = slots_of;
      if (T > KX_GEMV_TOKENS) f.h = (const char *)rows + (shifted ? (size_t)in.row.n_mix * T * w.in.ld * es : 0);  // the first product has built them
      f.h_buf = rows; f.row_buf = out_rows; f.mid = mid; f.y = expert_y;
      KX_DO(kx_expert_ff_launch(f32, f, T, st));
    } else {
      KX_DO(kx_linear_launch(f32, out, out_rows, st));
    }
    if (l.ff_kind == KxHybridLayer::GLU) {
      KxLinArgs gu, down;
      read(gu, w.gu, w.norm2, w.hc[1]);
      gu.epi = KX_LIN_GLU;
      gu.mid = mid; gu.mid_ld = mid_ld; gu.limit = l.limit; gu.alpha = l.alpha; gu.bias = l.bias;
      KX_DO(kx_linear_launch(f32, gu, rows, st));
      write(down, w.down, w.hc[1]);
      down.row.x = mid;
      down.row.x_ld = mid_ld;
      KX_DO(kx_linear_launch(f32, down, out_rows, st));
    }
    if (record) {
      hipLaunchKernelGGL(sum_streams_k, dim3(T), dim3(256), 0, st, streams, record + ((size_t)i * max_context + pos) * max_batch * W, W, S, batch, max_batch);
      KX_LAUNCH_CHECK();
    }
  }
  hist_cur ^= 1;
  x_row0 = (C - 1) * batch;
  if (sample) {
    KX_DO(logits_of(streams + (size_t)x_row0 * S * W, nullptr, batch, logits));
    KX_DO(kx_argmax_launch(logits, batch, c.vocab, c.vocab, next, argmax_scratch, st));
  }
  sampled = sample;
  pos += C;
  return KX_OK;
}

int HybridModel::row_logits(const int *token_rows, int n, float *d_out) {
  KX_HIP(hipMemcpyAsync(want, token_rows, (size_t)n * 4, hipMemcpyHostToDevice, st));
  KX_HIP(hipStreamSynchronize(st));
  return logits_of(streams, want, n, d_out);
}

int HybridModel::hidden_bf16(uint16_t *h_out) {
  std::vector<float> x((size_t)batch * c.streams * c.width);
  KX_HIP(hipMemcpyAsync(x.data(), streams + (size_t)x_row0 * c.streams * c.width, x.size() * 4, hipMemcpyDeviceToHost, st));
  KX_HIP(hipStreamSynchronize(st));
  for (int b = 0; b < batch; ++b)
    for (int k = 0; k < c.width; ++k) {
      float v = 0.0f;
      for (int s = 0; s < c.streams; ++s) v += x[((size_t)b * c.streams + s) * c.width + k];
      h_out[(size_t)b * c.width + k] = kx_bf16_rne(v);
    }
  return KX_OK;
}

int HybridModel::set_residual_record(bool on) {
  KX_HIP(hipStreamSynchronize(st));
  if (!on) {
    if (record) KX_HIP(hipFree(record));
    record = nullptr;
  } else if (!record) {
    const size_t bytes = (size_t)n_layers * max_context * max_batch * c.width * 4;
    KX_HIP(hipMalloc((void **)&record, bytes));
    KX_HIP(hipMemset(record, 0, bytes));
  }
  return KX_OK;
}
int HybridModel::residual(int layer, int pos0, int n, float *h_out) {
  KX_REQUIRE(record, "kx_model_residual: the record is off (kx_model_set_residual_record)");
  const size_t row = (size_t)c.width * 4;
  KX_HIP(hipMemcpy2DAsync(h_out, batch * row, record + ((size_t)layer * max_context + pos0) * max_batch * c.width, max_batch * row, batch * row, n,
                          hipMemcpyDeviceToHost, st));
  KX_HIP(hipStreamSynchronize(st));
  return KX_OK;
}

int hybrid_open(const char *name, const std::string &dir, const KxHybridConfig &config, const kx_open_options &o, kx_model **out) {
  for (const KxHybridLayer &l : config.layers) {
    const bool parallel = l.ff_kind == KxHybridLayer::GELU || l.ff_kind == KxHybridLayer::EXPERTS;
    KX_REQUIRE(l.ff_kind == KxHybridLayer::NONE || parallel == config.parallel, "kx_model_open: a feed-forward that runs %s its mixer only", parallel ? "beside" : "behind");
    KX_REQUIRE(!parallel || (!config.hyper && config.streams == 1 && config.groups == 1), "kx_model_open: mixer and feed-forward beside each other need one stream");
    KX_REQUIRE(l.mixer != KxHybridLayer::WKV || (!config.hyper && config.streams == 1 && config.groups == 1), "kx_model_open: time mixing needs one stream");
  }
  KX_REQUIRE((size_t)o.layers <= config.layers.size(), "kx_model_open: the model has %zu layers, %d asked for", config.layers.size(), o.layers);
  HybridModel *m = new HybridModel();
  m->name = name;
  m->c = config;
  if (o.layers) m->c.layers.resize(o.layers);
  m->n_layers = (int)m->c.layers.size(); m->hidden = config.width; m->vocab = config.vocab;
  m->max_batch = o.max_batch; m->max_context = o.max_context; m->eos_id = o.eos_id;
  m->dtype = o.dtype; m->f32 = o.dtype == KX_DTYPE_F32;
  m->step_tokens = (int)std::min<int64_t>(std::max(o.step_tokens, o.max_batch), (int64_t)o.max_context * o.max_batch);
  m->prefill_chunk = m->step_tokens;
  m->part_tokens = std::max(o.max_batch, std::min(64, m->step_tokens));
  m->init_sigma_ = o.init_sigma;
  auto build = [&]() -> int {
    KxTensorMap files;
    if (!o.random_init) KX_DO(kx_safetensors_scan(dir, files));
    m->ranks(files);
    const size_t total = m->layout(nullptr);
    if (!o.random_init) KX_DO(m->find(dir, files));
    size_t free_b = 0, total_b = 0;
    KX_HIP(hipMemGetInfo(&free_b, &total_b));
    KX_REQUIRE(total + ((size_t)1 << 30) <= free_b, "kx_model_open: the model needs %.1f GB of HBM, %.1f GB are free", total / 1e9, free_b / 1e9);
    KX_HIP(hipMalloc((void **)&m->arena, total));
    KX_DO(kx_model_resources(m, "kx_model_open"));
    KX_HIP(hipMemsetAsync(m->arena, 0, total, m->st));  // padding stays zero, cache rows that were never written are finite
    m->layout(m->arena);
    KX_DO(m->fill(files, o));
    for (const auto &t : m->turns) {
      std::vector<float> table((size_t)o.max_context * t.first.first);
      kx_latent_turns(t.second.second, o.max_context, table.data());
      KX_HIP(hipMemcpy(t.second.first, table.data(), table.size() * 4, hipMemcpyHostToDevice));
    }
    KX_HIP(hipStreamSynchronize(m->st));
    return KX_OK;
  };
  const int rc = build();
  if (rc) {
    delete m;
    return rc;
  }
  *out = m;
  return KX_OK;
}

template <int (*CONFIG)(const KxJson &, KxHybridConfig &)>
int probe(const std::string &dir, const KxJson &json, kx_model_shape &shape) {
  KxHybridConfig c;
  KX_DO(CONFIG(json, c));
  shape.n_layers = (int)c.layers.size(); shape.hidden = c.width; shape.vocab = c.vocab;
  return KX_OK;
}
int kagalorn_open(const std::string &dir, const KxJson &json, const kx_open_options &o, kx_model **out) {
  KxHybridConfig c;
  KX_DO(kx_kagalorn_config(json, c));
  return hybrid_open("Kagalorn", dir, c, o, out);
}
int rapitar_open(const std::string &dir, const KxJson &json, const kx_open_options &o, kx_model **out) {
  KxHybridConfig c;
  KX_DO(kx_rapitar_config(json, c));
  return hybrid_open("Rapitar", dir, c, o, out);
}

const KxDesignEntry kagalorn(KxDesign{"Kagalorn", kx_kagalorn_matches, probe<kx_kagalorn_config>, kagalorn_open});
const KxDesignEntry rapitar(KxDesign{"Rapitar", kx_rapitar_matches, probe<kx_rapitar_config>, rapitar_open});

}  // namespace
