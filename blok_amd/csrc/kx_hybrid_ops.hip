// kx_hybrid_ops.hip -- the hybrid decoder's mechanisms as operators of the C ABI (include/kx.h).
#include <algorithm>
#include "kx_common.h"
#include "kx_delta.h"
#include "kx_linear.h"
#include "kx_window.h"

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

extern "C" int kx_linear_run(const kx_linear_args *x, void *d_row_scratch, void *stream) {
  KX_REQUIRE(x && x->d_w && x->d_out, "kx_linear_run: null argument");
  KX_REQUIRE(x->row_kind >= KX_ROW_PLAIN && x->row_kind <= KX_ROW_GATED && x->epilogue >= KX_LIN_F32 && x->epilogue <= KX_LIN_STREAMS,
             "kx_linear_run: row_kind=%d epilogue=%d", x->row_kind, x->epilogue);
  KX_REQUIRE(x->streams >= 1 && x->streams <= KX_MAX_STREAMS, "kx_linear_run: streams=%d", x->streams);
  KxLinArgs a;
  a.m.w = (void *)x->d_w; a.m.rows = x->rows; a.m.cols = x->cols; a.m.ld = x->ld;
  a.tokens = x->tokens;
  a.epi = x->epilogue;
  KxRowArgs &r = a.row;
  r.kind = x->row_kind;
  r.cols = x->cols;
  if (r.kind == KX_ROW_NORM) {
    KX_REQUIRE(x->d_streams_in && x->d_norm && x->groups > 0 && x->cols % x->groups == 0, "kx_linear_run: groups=%d of %d columns", x->groups, x->cols);
    r.streams = (const float *)x->d_streams_in; r.n_streams = x->streams; r.in = (const float *)x->d_in; r.groups = x->groups;
    r.w = (const float *)x->d_norm; r.eps = x->eps;
  } else if (r.kind == KX_ROW_GATED) {
    KX_REQUIRE(x->d_o && x->d_gate && x->d_norm && x->heads > 0 && x->vdim > 0 && (int64_t)x->heads * x->vdim == x->cols && x->gate_ld >= x->cols,
               "kx_linear_run: %d heads of %d in %d columns", x->heads, x->vdim, x->cols);
    r.o = (const float *)x->d_o; r.gate = (const float *)x->d_gate; r.gate_ld = x->gate_ld; r.heads = x->heads; r.vdim = x->vdim;
    r.w = (const float *)x->d_norm; r.eps = x->eps;
  } else {
    KX_REQUIRE(x->d_x && x->x_ld >= x->ld && x->x_ld % KX_LD == 0, "kx_linear_run: x_ld=%d", x->x_ld);
    r.x = x->d_x; r.x_ld = x->x_ld;
  }
  if (a.epi == KX_LIN_F32) {
    KX_REQUIRE(x->out_ld >= x->rows, "kx_linear_run: out_ld=%d", x->out_ld);
    a.out = (float *)x->d_out; a.out_ld = x->out_ld;
  } else if (a.epi == KX_LIN_GLU) {
    KX_REQUIRE(x->out_ld >= x->rows / 2, "kx_linear_run: out_ld=%d", x->out_ld);
    a.mid = x->d_out; a.mid_ld = x->out_ld; a.limit = x->limit; a.alpha = x->alpha; a.bias = x->bias;
  } else {
    KX_REQUIRE(!x->d_mix == !x->d_outw, "kx_linear_run: mix and outw or neither");
    a.streams = (float *)x->d_out; a.n_streams = x->streams; a.mix = (const float *)x->d_mix; a.outw = (const float *)x->d_outw;
  }
  return kx_linear_launch(x->f32 != 0, a, d_row_scratch, kx_stream(stream));
}
