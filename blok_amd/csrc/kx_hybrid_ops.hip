// kx_hybrid_ops.hip -- the hybrid decoder's mechanisms as operators of the C ABI (include/kx.h).
#include <algorithm>
#include <vector>
#include "kx_common.h"
#include "kx_delta.h"
#include "kx_experts.h"
#include "kx_latent.h"
#include "kx_linear.h"
#include "kx_ssd.h"
#include "kx_window.h"
#include "kx_wkv.h"

struct kx_window {
  KxWindowArgs a;
  bool f32 = false;
  int max_batch = 0, max_context = 0, max_positions = 0;
  char *mem = nullptr;
};
struct kx_delta {
  KxDeltaArgs a;
  int max_batch = 0, max_positions = 0, cur = 0;
  size_t state_bytes = 0, hist_bytes = 0;
  char *mem = nullptr;
  float *hist[2] = {nullptr, nullptr};
};

// device memory of an operator: offsets first, then one zeroed allocation
struct OpMem {
  char *p = nullptr;
  size_t total = 0;
  size_t take(size_t bytes) {
    const size_t at = total;
    total += (bytes + 255) & ~(size_t)255;
    return at;
  }
  int alloc(const char *who) {
    if (hipMalloc((void **)&p, total) != hipSuccess || hipMemset(p, 0, total) != hipSuccess) {
      kx_set_error("%s: no device memory for %zu bytes", who, total);
      return KX_ERR_HIP;
    }
    return KX_OK;
  }
  ~OpMem() {
    if (p) (void)hipFree(p);
  }
};
struct kx_ssd {
  KxSsdArgs a;
  int max_batch = 0, max_positions = 0, cur = 0;
  size_t kept = 0;  // bytes of state and inputs at the start of mem
  float *hist[2] = {nullptr, nullptr};
  OpMem mem;
};
struct kx_wkv {
  KxWkvArgs a;
  bool f32 = false;
  int max_batch = 0, max_positions = 0;
  size_t kept = 0;
  OpMem mem;
};
struct kx_latent {
  KxLatentArgs a;
  bool f32 = false, gate = false;
  int max_batch = 0, max_positions = 0;
  OpMem mem;
};
struct kx_experts {
  kx_experts_config c;
  KxExpertFf f;
  bool f32 = false;
  int max_tokens = 0;
  float *logits = nullptr;
  OpMem mem;
};

extern "C" int kx_window_create(const kx_window_config *c, int f32, int32_t max_batch, int32_t max_context, int32_t max_positions, kx_window **out) {
  KX_REQUIRE(c && out, "kx_window_create: null argument");
  *out = nullptr;
  KX_REQUIRE(c->heads > 0 && c->kv_heads > 0 && c->heads % c->kv_heads == 0 && c->dim > 0 && c->vdim > 0 && c->size > 0 && c->pool >= 0,
             "kx_window_create: heads=%d kv_heads=%d dim=%d vdim=%d size=%d pool=%d", c->heads, c->kv_heads, c->dim, c->vdim, c->size, c->pool);
  KX_REQUIRE(max_batch > 0 && max_context > 0 && max_positions > 0, "kx_window_create: max_batch=%d max_context=%d max_positions=%d", max_batch, max_context, max_positions);
  kx_window *w = new kx_window();
  w->f32 = f32 != 0;
  w->max_batch = max_batch; w->max_context = max_context; w->max_positions = std::min(max_positions, max_context);
  KxWindowSpec &s = w->a.s;
  s.heads = c->heads; s.kv_heads = c->kv_heads; s.dim = c->dim; s.vdim = c->vdim; s.scale = c->scale; s.size = c->size; s.pool = c->pool; s.sink = c->sink;
  w->a.eps = c->eps;
  w->a.g_off = c->gate ? 0 : -1;
  size_t e[4], at[6], total = 0;
  kx_window_shape(s, max_context, w->max_positions, &w->a.c, e);
  const size_t es = f32 ? 4 : 2, T = (size_t)max_batch * w->max_positions;
  w->a.part_floats = kx_window_part_floats(s, max_context, std::max(max_batch, 16));
  const size_t sizes[6] = {e[0] * max_batch * es, e[1] * max_batch * es, e[2] * max_batch * es, e[3] * max_batch * es,
                           T * s.heads * w->a.c.dp * es, w->a.part_floats * 4};
  for (int i = 0; i < 6; ++i) {
    at[i] = total;
    total += (sizes[i] + 255) & ~(size_t)255;
  }
  if (hipMalloc((void **)&w->mem, total) != hipSuccess || hipMemset(w->mem, 0, total) != hipSuccess) {
    kx_set_error("kx_window_create: no device memory for %zu bytes", total);
    kx_window_destroy(w);
    return KX_ERR_HIP;
  }
  w->a.c.k = w->mem + at[0]; w->a.c.v = w->mem + at[1]; w->a.c.pk = w->mem + at[2]; w->a.c.pv = w->mem + at[3];
  w->a.q = w->mem + at[4];
  w->a.part = (float *)(w->mem + at[5]);
  *out = w;
  return KX_OK;
}
extern "C" int kx_window_destroy(kx_window *w) {
  if (!w) return KX_OK;
  if (w->mem) (void)hipFree(w->mem);
  delete w;
  return KX_OK;
}
extern "C" int kx_window_run(kx_window *w, const void *d_proj, int32_t proj_ld, int32_t q_off, int32_t k_off, int32_t v_off, int32_t g_off,
                             const void *d_q_norm, const void *d_k_norm, int32_t batch, int32_t positions, int32_t pos, void *d_out, int32_t out_ld,
                             void *stream) {
  KX_REQUIRE(w && d_proj && d_out, "kx_window_run: null argument");
  KX_REQUIRE(!d_q_norm == !d_k_norm, "kx_window_run: a norm for q and k or for neither");
  KX_REQUIRE(batch > 0 && batch <= w->max_batch && positions > 0 && positions <= w->max_positions && pos >= 0 && pos <= w->max_context - positions,
             "kx_window_run: batch=%d, positions [%d, %d + %d)", batch, pos, pos, positions);
  KxWindowArgs a = w->a;
  const KxWindowSpec &s = a.s;
  auto fits = [&](int off, int n) { return off >= 0 && off <= proj_ld - n; };
  KX_REQUIRE(fits(q_off, s.heads * s.dim) && fits(k_off, s.kv_heads * s.dim) && fits(v_off, s.kv_heads * s.vdim) &&
                 (a.g_off < 0 || fits(g_off, s.heads * s.vdim)) && out_ld >= s.heads * s.vdim, "kx_window_run: columns outside the rows");
  a.proj = (const float *)d_proj; a.proj_ld = proj_ld; a.q_off = q_off; a.k_off = k_off; a.v_off = v_off;
  if (a.g_off >= 0) a.g_off = g_off;
  a.q_norm = (const float *)d_q_norm; a.k_norm = (const float *)d_k_norm;
  a.batch = batch; a.positions = positions; a.pos = pos;
  a.out = d_out; a.out_ld = out_ld;
  return kx_window_launch(w->f32, a, kx_stream(stream));
}

extern "C" int kx_delta_create(const kx_delta_config *c, int32_t max_batch, int32_t max_positions, kx_delta **out) {
  KX_REQUIRE(c && out, "kx_delta_create: null argument");
  *out = nullptr;
  KX_REQUIRE(c->heads > 0 && c->kv_heads > 0 && c->heads % c->kv_heads == 0 && c->dim > 0 && c->dim <= 256 && c->vdim > 0 && c->taps > 0,
             "kx_delta_create: heads=%d kv_heads=%d dim=%d vdim=%d taps=%d", c->heads, c->kv_heads, c->dim, c->vdim, c->taps);
  KX_REQUIRE(max_batch > 0 && max_positions > 0, "kx_delta_create: max_batch=%d max_positions=%d", max_batch, max_positions);
  kx_delta *d = new kx_delta();
  KxDeltaSpec &s = d->a.s;
  s.heads = c->heads; s.kv_heads = c->kv_heads; s.dim = c->dim; s.vdim = c->vdim; s.taps = c->taps; s.unit_eps = c->unit_eps;
  d->max_batch = max_batch; d->max_positions = max_positions;
  d->state_bytes = (size_t)max_batch * s.heads * s.dim * s.vdim * 4;
  d->hist_bytes = (size_t)max_batch * (s.taps - 1) * kx_delta_channels(s) * 4;
  const size_t total = d->state_bytes + 2 * d->hist_bytes + kx_delta_work_floats(s, max_batch, max_positions) * 4;
  if (hipMalloc((void **)&d->mem, total) != hipSuccess || hipMemset(d->mem, 0, total) != hipSuccess) {
    kx_set_error("kx_delta_create: no device memory for %zu bytes", total);
    kx_delta_destroy(d);
    return KX_ERR_HIP;
  }
  d->a.state = (float *)d->mem;
  d->hist[0] = (float *)(d->mem + d->state_bytes);
  d->hist[1] = (float *)(d->mem + d->state_bytes + d->hist_bytes);
  d->a.work = (float *)(d->mem + d->state_bytes + 2 * d->hist_bytes);
  *out = d;
  return KX_OK;
}
extern "C" int kx_delta_destroy(kx_delta *d) {
  if (!d) return KX_OK;
  if (d->mem) (void)hipFree(d->mem);
  delete d;
  return KX_OK;
}
extern "C" int kx_delta_restart(kx_delta *d, void *stream) {
  KX_REQUIRE(d, "kx_delta_restart: null argument");
  KX_HIP(hipMemsetAsync(d->mem, 0, d->state_bytes + 2 * d->hist_bytes, kx_stream(stream)));
  return KX_OK;
}
extern "C" int kx_delta_run(kx_delta *d, const void *d_proj, int32_t proj_ld, int32_t q_off, int32_t k_off, int32_t v_off, int32_t b_off, int32_t a_off,
                            const void *d_conv, const void *d_a_log, const void *d_dt_bias, int32_t batch, int32_t positions, void *d_o, void *stream) {
  KX_REQUIRE(d && d_proj && d_conv && d_a_log && d_dt_bias && d_o, "kx_delta_run: null argument");
  KX_REQUIRE(batch > 0 && batch <= d->max_batch && positions > 0 && positions <= d->max_positions, "kx_delta_run: batch=%d positions=%d", batch, positions);
  KxDeltaArgs a = d->a;
  const KxDeltaSpec &s = a.s;
  auto fits = [&](int off, int n) { return off >= 0 && off <= proj_ld - n; };
  KX_REQUIRE(fits(q_off, s.kv_heads * s.dim) && fits(k_off, s.kv_heads * s.dim) && fits(v_off, s.heads * s.vdim) && fits(b_off, s.heads) && fits(a_off, s.heads),
             "kx_delta_run: columns outside the rows");
  a.proj = (const float *)d_proj; a.proj_ld = proj_ld; a.q_off = q_off; a.k_off = k_off; a.v_off = v_off; a.b_off = b_off; a.a_off = a_off;
  a.conv = (const float *)d_conv; a.a_log = (const float *)d_a_log; a.dt_bias = (const float *)d_dt_bias;
  a.batch = batch; a.positions = positions;
  a.o = (float *)d_o;
  a.hist = d->hist[d->cur];
  a.hist_out = d->hist[d->cur ^ 1];
  int rc = kx_delta_launch(a, kx_stream(stream));
  if (!rc) d->cur ^= 1;
  return rc;
}

extern "C" int kx_ssd_create(const kx_ssd_config *c, int32_t max_batch, int32_t max_positions, kx_ssd **out) {
  KX_REQUIRE(c && out, "kx_ssd_create: null argument");
  *out = nullptr;
  KX_REQUIRE(c->heads > 0 && c->vdim > 0 && c->state > 0 && c->state <= KX_SCAN_MAX_DIM && c->groups > 0 && c->heads % c->groups == 0 && c->taps > 0,
             "kx_ssd_create: heads=%d vdim=%d state=%d groups=%d taps=%d", c->heads, c->vdim, c->state, c->groups, c->taps);
  KX_REQUIRE(max_batch > 0 && max_positions > 0, "kx_ssd_create: max_batch=%d max_positions=%d", max_batch, max_positions);
  kx_ssd *d = new kx_ssd();
  KxSsdSpec &s = d->a.s;
  s.heads = c->heads; s.vdim = c->vdim; s.state = c->state; s.groups = c->groups; s.taps = c->taps;
  d->max_batch = max_batch; d->max_positions = max_positions;
  const size_t hist = (size_t)max_batch * (s.taps - 1) * kx_ssd_channels(s) * 4;
  const size_t state = d->mem.take((size_t)max_batch * s.heads * s.state * s.vdim * 4), h0 = d->mem.take(hist), h1 = d->mem.take(hist);
  d->kept = d->mem.total;
  const size_t work = d->mem.take(kx_ssd_work_floats(s, max_batch, max_positions) * 4);
  const int rc = d->mem.alloc("kx_ssd_create");
  if (rc) {
    delete d;
    return rc;
  }
  d->a.state = (float *)(d->mem.p + state); d->hist[0] = (float *)(d->mem.p + h0); d->hist[1] = (float *)(d->mem.p + h1); d->a.work = (float *)(d->mem.p + work);
  *out = d;
  return KX_OK;
}
extern "C" int kx_ssd_destroy(kx_ssd *d) {
  delete d;
  return KX_OK;
}
extern "C" int kx_ssd_restart(kx_ssd *d, void *stream) {
  KX_REQUIRE(d, "kx_ssd_restart: null argument");
  KX_HIP(hipMemsetAsync(d->mem.p, 0, d->kept, kx_stream(stream)));
  return KX_OK;
}
extern "C" int kx_ssd_run(kx_ssd *d, const void *d_proj, int32_t proj_ld, int32_t x_off, int32_t dt_off, const void *d_conv, const void *d_conv_bias,
                          const void *d_a_log, const void *d_dt_bias, const void *d_skip, int32_t batch, int32_t positions, void *d_y, void *stream) {
  KX_REQUIRE(d && d_proj && d_conv && d_a_log && d_dt_bias && d_skip && d_y, "kx_ssd_run: null argument");
  KX_REQUIRE(batch > 0 && batch <= d->max_batch && positions > 0 && positions <= d->max_positions, "kx_ssd_run: batch=%d positions=%d", batch, positions);
  KxSsdArgs a = d->a;
  KX_REQUIRE(x_off >= 0 && x_off <= proj_ld - kx_ssd_channels(a.s) && dt_off >= 0 && dt_off <= proj_ld - a.s.heads, "kx_ssd_run: columns outside the rows");
  a.proj = (const float *)d_proj; a.proj_ld = proj_ld; a.x_off = x_off; a.dt_off = dt_off;
  a.conv = (const float *)d_conv; a.conv_bias = (const float *)d_conv_bias;
  a.a_log = (const float *)d_a_log; a.dt_bias = (const float *)d_dt_bias; a.skip = (const float *)d_skip;
  a.batch = batch; a.positions = positions;
  a.y = (float *)d_y;
  a.hist = d->hist[d->cur];
  a.hist_out = d->hist[d->cur ^ 1];
  const int rc = kx_ssd_launch(a, kx_stream(stream));
  if (!rc) d->cur ^= 1;
  return rc;
}

extern "C" int kx_wkv_create(const kx_wkv_config *c, int f32, int32_t max_batch, int32_t max_positions, kx_wkv **out) {
  KX_REQUIRE(c && out, "kx_wkv_create: null argument");
  *out = nullptr;
  KX_REQUIRE(c->heads > 0 && c->dim > 0 && c->dim <= KX_SCAN_MAX_DIM && c->rank > 0, "kx_wkv_create: heads=%d dim=%d rank=%d", c->heads, c->dim, c->rank);
  KX_REQUIRE(max_batch > 0 && max_positions > 0, "kx_wkv_create: max_batch=%d max_positions=%d", max_batch, max_positions);
  kx_wkv *d = new kx_wkv();
  KxWkvSpec &s = d->a.s;
  s.heads = c->heads; s.dim = c->dim; s.rank = c->rank;
  d->f32 = f32 != 0;
  d->max_batch = max_batch; d->max_positions = max_positions;
  d->a.w2.rows = s.heads * s.dim; d->a.w2.cols = s.rank; d->a.w2.ld = kx_pad(s.rank, KX_LD);
  const size_t state = d->mem.take((size_t)max_batch * s.heads * s.dim * s.dim * 4);
  d->kept = d->mem.total;
  const size_t work = d->mem.take(kx_wkv_work_floats(s, max_batch, max_positions) * 4), rows = d->mem.take((size_t)max_batch * max_positions * d->a.w2.ld * (f32 ? 4 : 2));
  const int rc = d->mem.alloc("kx_wkv_create");
  if (rc) {
    delete d;
    return rc;
  }
  d->a.state = (float *)(d->mem.p + state); d->a.work = (float *)(d->mem.p + work); d->a.rows = d->mem.p + rows;
  *out = d;
  return KX_OK;
}
extern "C" int kx_wkv_destroy(kx_wkv *d) {
  delete d;
  return KX_OK;
}
extern "C" int kx_wkv_restart(kx_wkv *d, void *stream) {
  KX_REQUIRE(d, "kx_wkv_restart: null argument");
  KX_HIP(hipMemsetAsync(d->mem.p, 0, d->kept, kx_stream(stream)));
  return KX_OK;
}
extern "C" int kx_wkv_run(kx_wkv *d, const void *d_proj, int32_t proj_ld, int32_t r_off, int32_t k_off, int32_t v_off, int32_t w_off, const void *d_w2,
                          const void *d_w0, const void *d_u, int32_t batch, int32_t positions, void *d_o, void *stream) {
  KX_REQUIRE(d && d_proj && d_w2 && d_w0 && d_u && d_o, "kx_wkv_run: null argument");
  KX_REQUIRE(batch > 0 && batch <= d->max_batch && positions > 0 && positions <= d->max_positions, "kx_wkv_run: batch=%d positions=%d", batch, positions);
  KxWkvArgs a = d->a;
  const int hd = a.s.heads * a.s.dim;
  auto fits = [&](int off, int n) { return off >= 0 && off <= proj_ld - n; };
  KX_REQUIRE(fits(r_off, hd) && fits(k_off, hd) && fits(v_off, hd) && fits(w_off, a.s.rank), "kx_wkv_run: columns outside the rows");
  a.proj = (const float *)d_proj; a.proj_ld = proj_ld; a.r_off = r_off; a.k_off = k_off; a.v_off = v_off; a.w_off = w_off;
  a.w2.w = (void *)d_w2; a.w0 = (const float *)d_w0; a.u = (const float *)d_u;
  a.batch = batch; a.positions = positions;
  a.o = (float *)d_o;
  return kx_wkv_launch(d->f32, a, kx_stream(stream));
}

extern "C" int kx_latent_create(const kx_latent_config *c, int f32, int32_t max_batch, int32_t max_context, int32_t max_positions, kx_latent **out) {
  KX_REQUIRE(c && out, "kx_latent_create: null argument");
  *out = nullptr;
  KX_REQUIRE(c->heads > 0 && c->dim > 0 && c->rot_dim >= 0 && c->rot >= 0 && c->rot % 2 == 0 && c->rot <= c->rot_dim && c->vdim > 0 && c->kv_rank > 0 && c->kv_rank <= 2048,
             "kx_latent_create: heads=%d dim=%d rot_dim=%d (%d rotated) vdim=%d kv_rank=%d", c->heads, c->dim, c->rot_dim, c->rot, c->vdim, c->kv_rank);
  KX_REQUIRE(max_batch > 0 && max_context > 0 && max_positions > 0, "kx_latent_create: max_batch=%d max_context=%d max_positions=%d", max_batch, max_context, max_positions);
  kx_latent *d = new kx_latent();
  KxLatentArgs &a = d->a;
  KxLatentSpec &s = a.s;
  s.heads = c->heads; s.dim = c->dim; s.rot_dim = c->rot_dim; s.rot = c->rot; s.vdim = c->vdim; s.kv_rank = c->kv_rank; s.sink = c->sink;
  s.scale = c->scale; s.base = c->base;
  a.eps = c->eps;
  a.cap = max_context;
  d->f32 = f32 != 0; d->gate = c->gate != 0;
  d->max_batch = max_batch; d->max_positions = std::min(max_positions, max_context);
  a.uk.rows = s.heads * s.dim; a.uv.rows = s.heads * s.vdim;
  a.uk.cols = a.uv.cols = s.kv_rank;
  a.uk.ld = a.uv.ld = kx_pad(s.kv_rank, KX_LD);
  size_t qf, qx;
  kx_latent_scratch(s, max_batch, max_context, max_batch * d->max_positions, &a.x, &qf, &qx);
  if (c->no_expand) a.x.k_elems = a.x.v_elems = 0;
  const size_t es = f32 ? 4 : 2;
  OpMem &m = d->mem;
  const size_t rows = m.take((size_t)max_batch * max_context * kx_latent_row(s) * es), turns = m.take((size_t)max_context * (s.rot / 2) * 8), q = m.take(qf * 4),
               x = m.take(qx * es), k = m.take(a.x.k_elems * es), v = m.take(a.x.v_elems * es), part = m.take(a.x.part_floats * 4);
  int rc = m.alloc("kx_latent_create");
  if (!rc && s.rot) {
    std::vector<float> table((size_t)max_context * s.rot);
    kx_latent_turns(s, max_context, table.data());
    if (hipMemcpy(m.p + turns, table.data(), table.size() * 4, hipMemcpyHostToDevice) != hipSuccess) {
      kx_set_error("kx_latent_create: copy failed");
      rc = KX_ERR_HIP;
    }
  }
  if (rc) {
    delete d;
    return rc;
  }
  a.rows = m.p + rows; a.turns = (const float2 *)(m.p + turns); a.x.q = (float *)(m.p + q); a.x.qx = m.p + x; a.x.kx = m.p + k; a.x.vx = m.p + v;
  a.x.part = (float *)(m.p + part);
  *out = d;
  return KX_OK;
}
extern "C" int kx_latent_destroy(kx_latent *d) {
  delete d;
  return KX_OK;
}
extern "C" int kx_latent_run(kx_latent *d, const void *d_q, int32_t q_ld, const void *d_proj, int32_t proj_ld, int32_t kv_off, int32_t g_off, const void *d_kv_norm,
                             const void *d_uk, const void *d_uv, const void *d_sinks, int32_t batch, int32_t positions, int32_t pos, void *d_out, int32_t out_ld,
                             void *stream) {
  KX_REQUIRE(d && d_q && d_proj && d_kv_norm && d_uk && d_uv && d_out, "kx_latent_run: null argument");
  KxLatentArgs a = d->a;
  const KxLatentSpec &s = a.s;
  KX_REQUIRE(batch > 0 && batch <= d->max_batch && positions > 0 && positions <= d->max_positions && pos >= 0 && pos <= a.cap - positions,
             "kx_latent_run: batch=%d, positions [%d, %d + %d)", batch, pos, pos, positions);
  KX_REQUIRE(kv_off >= 0 && kv_off <= proj_ld - s.kv_rank - s.rot_dim && (!d->gate || (g_off >= 0 && g_off <= proj_ld - s.heads * s.vdim)) &&
                 q_ld >= s.heads * (s.dim + s.rot_dim) && out_ld >= s.heads * s.vdim, "kx_latent_run: columns outside the rows");
  a.q = (const float *)d_q; a.q_ld = q_ld;
  a.proj = (const float *)d_proj; a.proj_ld = proj_ld; a.kv_off = kv_off; a.g_off = d->gate ? g_off : -1;
  a.kv_norm = (const float *)d_kv_norm;
  a.uk.w = (void *)d_uk; a.uv.w = (void *)d_uv;
  a.sinks = (const float *)d_sinks;
  a.batch = batch; a.positions = positions; a.pos = pos;
  a.out = d_out; a.out_ld = out_ld;
  return kx_latent_launch(d->f32, a, kx_stream(stream));
}

extern "C" int kx_experts_create(const kx_experts_config *c, int f32, int32_t max_tokens, kx_experts **out) {
  KX_REQUIRE(c && out, "kx_experts_create: null argument");
  *out = nullptr;
  KX_REQUIRE(c->width > 0 && c->ff > 0 && c->cols > 0 && c->experts > 0 && c->experts <= KX_MAX_EXPERTS && c->top > 0 && c->top <= c->experts && c->top <= KX_MAX_TOP && max_tokens > 0,
             "kx_experts_create: width=%d ff=%d cols=%d, %d of %d experts, %d tokens", c->width, c->ff, c->cols, c->top, c->experts, max_tokens);
  kx_experts *d = new kx_experts();
  d->c = *c;
  d->f32 = f32 != 0;
  d->max_tokens = max_tokens;
  KxExpertFf &f = d->f;
  const size_t es = f32 ? 4 : 2, T = max_tokens, pairs = T * c->top;
  f.gu.m.rows = 2 * kx_pad(c->ff, KX_GLU_BLOCK); f.gu.m.cols = c->width; f.gu.m.ld = kx_pad(c->width, KX_LD);
  f.down.rows = c->width; f.down.cols = c->ff; f.down.ld = kx_pad(c->ff, KX_LD);
  f.out.m.rows = c->width; f.out.m.cols = c->cols; f.out.m.ld = kx_pad(c->cols, KX_LD);
  f.gu_stride = (size_t)f.gu.m.rows * f.gu.m.ld;
  f.down_stride = (size_t)f.down.rows * f.down.ld;
  f.gu.limit = c->limit; f.gu.alpha = c->alpha; f.gu.bias = c->bias;
  f.e.experts = c->experts; f.e.top = c->top; f.e.logits_ld = c->experts;
  OpMem &m = d->mem;
  const size_t logits = m.take(T * c->experts * 4), ids = m.take(pairs * 4), gather = m.take(pairs * 4), slot_of = m.take(pairs * 4), weights = m.take(pairs * 4),
               slot_weight = m.take(pairs * 4), tiles = m.take((size_t)kx_expert_tiles(max_tokens, c->top, c->experts, 64) * sizeof(int4)), n_tiles = m.take(4),
               h = m.take(T * f.gu.m.ld * es), mid = m.take(pairs * f.down.ld * es), y = m.take(pairs * c->width * 4);
  const int rc = m.alloc("kx_experts_create");
  if (rc) {
    delete d;
    return rc;
  }
  d->logits = (float *)(m.p + logits);
  f.e.logits = d->logits;
  f.s.ids = (int *)(m.p + ids); f.s.gather = (int *)(m.p + gather); f.s.slot_of = (int *)(m.p + slot_of); f.s.weights = (float *)(m.p + weights);
  f.s.slot_weight = (float *)(m.p + slot_weight); f.s.tiles = (int4 *)(m.p + tiles); f.s.n_tiles = (int *)(m.p + n_tiles);
  f.h_buf = m.p + h; f.mid = m.p + mid; f.y = (float *)(m.p + y);
  *out = d;
  return KX_OK;
}
extern "C" int kx_experts_destroy(kx_experts *d) {
  delete d;
  return KX_OK;
}
extern "C" int kx_experts_run(kx_experts *d, void *d_x, const void *d_norm, float eps, const void *d_router, const void *d_router_bias, const void *d_gu, const void *d_down,
                              const void *d_w, const void *d_rows, int32_t tokens, void *d_ids, void *stream) {
  KX_REQUIRE(d && d_x && d_norm && d_router && d_router_bias && d_gu && d_down && d_w && d_rows, "kx_experts_run: null argument");
  KX_REQUIRE(tokens > 0 && tokens <= d->max_tokens, "kx_experts_run: tokens=%d", tokens);
  KxExpertFf f = d->f;
  const kx_experts_config &c = d->c;
  f.gu.m.w = (void *)d_gu; f.down.w = (void *)d_down; f.out.m.w = (void *)d_w;
  f.e.bias = (const float *)d_router_bias;
  f.gu.tokens = f.out.tokens = tokens;
  f.gu.row.kind = KX_ROW_NORM; f.gu.row.cols = c.width; f.gu.row.streams = (const float *)d_x; f.gu.row.w = (const float *)d_norm; f.gu.row.eps = eps;
  f.out.row.cols = c.cols; f.out.row.x = d_rows; f.out.row.x_ld = f.out.m.ld;
  f.out.epi = KX_LIN_STREAMS;
  f.out.streams = (float *)d_x;
  KxLinArgs r;  // the router's logits
  r.m.w = (void *)d_router; r.m.rows = c.experts; r.m.cols = c.width; r.m.ld = f.gu.m.ld;
  r.row = f.gu.row;
  r.tokens = tokens;
  r.out = d->logits;
  r.out_ld = c.experts;
  int rc = kx_linear_launch(d->f32, r, f.h_buf, kx_stream(stream));
  if (rc || (rc = kx_expert_ff_launch(d->f32, f, tokens, kx_stream(stream)))) return rc;
  if (d_ids) KX_HIP(hipMemcpyAsync(d_ids, f.s.ids, (size_t)tokens * c.top * 4, hipMemcpyDeviceToDevice, kx_stream(stream)));
  return KX_OK;
}

extern "C" int kx_linear_run(const kx_linear_args *x, void *d_row_scratch, void *stream) {
  KX_REQUIRE(x && x->d_w && x->d_out, "kx_linear_run: null argument");
  KX_REQUIRE(x->row_kind >= KX_ROW_PLAIN && x->row_kind <= KX_ROW_TANH && x->epilogue >= 0 && x->epilogue <= 3,
             "kx_linear_run: row_kind=%d epilogue=%d", x->row_kind, x->epilogue);
  KX_REQUIRE(x->streams >= 1 && x->streams <= KX_MAX_STREAMS, "kx_linear_run: streams=%d", x->streams);
  KxLinArgs a;
  a.m.w = (void *)x->d_w; a.m.rows = x->rows; a.m.cols = x->cols; a.m.ld = x->ld;
  a.tokens = x->tokens;
  static const int epilogues[4] = {KX_LIN_F32, KX_LIN_GLU, KX_LIN_STREAMS, KX_LIN_HEADS};
  a.epi = epilogues[x->epilogue];
  KxRowArgs &r = a.row;
  r.kind = x->row_kind;
  r.cols = x->cols;
  if (r.kind == KX_ROW_NORM) {
    KX_REQUIRE(x->d_streams_in && x->d_norm && x->groups > 0 && x->cols % x->groups == 0, "kx_linear_run: groups=%d of %d columns", x->groups, x->cols);
    r.streams = (const float *)x->d_streams_in; r.n_streams = x->streams; r.in = (const float *)x->d_in; r.groups = x->groups;
    r.w = (const float *)x->d_norm; r.eps = x->eps;
  } else if (r.kind == KX_ROW_GATED) {
    KX_REQUIRE(x->d_o && x->d_gate && x->d_norm && x->heads > 0 && x->vdim > 0 && x->gate_ld >= x->heads * x->vdim &&
                   (x->d_tail ? x->head_ld >= x->heads * x->vdim && x->head_ld < x->cols && x->tail_ld >= x->ld - x->head_ld : (int64_t)x->heads * x->vdim == x->cols),
               "kx_linear_run: %d heads of %d in %d columns", x->heads, x->vdim, x->cols);
    r.o = (const float *)x->d_o; r.gate = (const float *)x->d_gate; r.gate_ld = x->gate_ld; r.heads = x->heads; r.vdim = x->vdim;
    r.w = (const float *)x->d_norm; r.eps = x->eps;
    r.w_per_column = x->w_per_column != 0; r.gate_first = x->gate_first != 0;
    r.tail = x->d_tail; r.tail_ld = x->tail_ld; r.head_ld = x->head_ld;
  } else if (r.kind == KX_ROW_SHIFT) {
    KX_REQUIRE(x->d_streams_in && x->d_norm && x->d_mu && x->d_prev && x->d_prev_out && x->n_mix > 0 && x->n_mix < KX_MAX_VARIANTS && x->batch > 0 && x->tokens % x->batch == 0,
               "kx_linear_run: %d mixes, %d tokens of %d sequences", x->n_mix, x->tokens, x->batch);
    r.streams = (const float *)x->d_streams_in; r.w = (const float *)x->d_norm; r.eps = x->eps;
    r.mu = (const float *)x->d_mu; r.n_mix = x->n_mix; r.batch = x->batch; r.prev = (const float *)x->d_prev; r.prev_out = (float *)x->d_prev_out; r.tokens = x->tokens;
    a.n_var = x->n_mix + 1;
    for (int v = 0; v < a.n_var; ++v) a.var_row[v] = x->var_row[v];
  } else if (r.kind == KX_ROW_TANH) {
    KX_REQUIRE(x->d_streams_in && x->streams_ld >= x->cols, "kx_linear_run: streams_ld=%d", x->streams_ld);
    r.streams = (const float *)x->d_streams_in; r.streams_ld = x->streams_ld;
  } else {
    KX_REQUIRE(x->d_x && x->x_ld >= x->ld && x->x_ld % KX_LD == 0, "kx_linear_run: x_ld=%d", x->x_ld);
    r.x = x->d_x; r.x_ld = x->x_ld;
  }
  if (a.epi == KX_LIN_F32) {
    KX_REQUIRE(x->act_rows >= 0 && x->act_rows <= x->rows && x->out_ld >= x->rows - x->act_rows && (!x->act_rows || (x->d_mid && x->mid_ld >= x->act_rows)),
               "kx_linear_run: out_ld=%d, %d activations in rows of %d", x->out_ld, x->act_rows, x->mid_ld);
    a.out = (float *)x->d_out; a.out_ld = x->out_ld;
    if (x->act_rows) {
      a.act_from = x->rows - x->act_rows; a.mid = x->d_mid; a.mid_ld = x->mid_ld;
    }
  } else if (a.epi == KX_LIN_HEADS) {
    KX_REQUIRE(x->head_dim > 0 && x->rows % x->head_dim == 0 && x->out_ld >= x->head_dim && x->head_stride >= (int64_t)x->tokens * x->out_ld,
               "kx_linear_run: %d rows in heads of %d", x->rows, x->head_dim);
    a.mid = x->d_out; a.mid_ld = x->out_ld; a.head_dim = x->head_dim; a.head_stride = x->head_stride;
  } else if (a.epi == KX_LIN_GLU) {
    KX_REQUIRE(x->out_ld >= x->rows / 2, "kx_linear_run: out_ld=%d", x->out_ld);
    a.mid = x->d_out; a.mid_ld = x->out_ld; a.limit = x->limit; a.alpha = x->alpha; a.bias = x->bias;
  } else {
    KX_REQUIRE(!x->d_mix == !x->d_outw, "kx_linear_run: mix and outw or neither");
    a.streams = (float *)x->d_out; a.n_streams = x->streams; a.mix = (const float *)x->d_mix; a.outw = (const float *)x->d_outw;
  }
  return kx_linear_launch(x->f32 != 0, a, d_row_scratch, kx_stream(stream));
}
