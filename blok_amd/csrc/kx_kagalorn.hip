// kx_kagalorn.hip -- config.json of the Kagalorn design -> a hybrid decoder's configuration (host code only).
//
// The file gives vocab, width, streams, norm {eps, groups} and per layer its mixer's type and sizes and its
// feed-forward; what the design fixes for all its models is set here.
#include "kx_config.h"
#include "kx_hybrid.h"
#include "kx_linear.h"

namespace {

constexpr float SIGMOID_SLOPE = 1.702f, UP_BIAS = 1.0f;  // of the clamped gated feed-forward
constexpr float UNIT_EPS = 1e-6f;                        // under the root of the delta rule's unit norms

int layer_config(const KxFields &f, KxHybridLayer &L) {
  std::string type;
  KX_DO(f.text("type", type));
  KxFields m;
  KX_DO(f.object("mixer", m));
  int heads, kv, dim, vdim;
  KX_DO(m.integer("heads", 1, heads));
  KX_DO(m.integer("kv_heads", 1, kv));
  KX_DO(m.integer("dim", 1, dim));
  KX_DO(m.integer("vdim", 1, vdim));
  KX_REQUIRE(heads % kv == 0, "config.json: %s: %d heads on %d kv_heads", m.where.c_str(), heads, kv);
  if (type == "attention") {
    L.mixer = KxHybridLayer::ATTENTION;
    KxWindowSpec &a = L.attn;
    a.heads = heads; a.kv_heads = kv; a.dim = dim; a.vdim = vdim;
    a.sink = 1;
    L.qk_norm = L.gate = true;
    KX_DO(m.real("scale", a.scale));
    KxFields mask;
    KX_DO(m.object("mask", mask));
    KX_DO(mask.integer("size", 1, a.size));
    KX_DO(mask.integer("pool", 1, a.pool));
  } else if (type == "delta") {
    L.mixer = KxHybridLayer::DELTA;
    KxDeltaSpec &d = L.delta;
    d.heads = heads; d.kv_heads = kv; d.dim = dim; d.vdim = vdim;
    d.unit_eps = UNIT_EPS;
    KX_DO(m.integer("conv", 1, d.taps));
    KX_REQUIRE(dim <= 256, "config.json: %s.dim=%d: the delta rule takes keys of up to 256", m.where.c_str(), dim);
  } else {
    kx_set_error("config.json: %s.type is %s (attention and delta are known)", f.where.c_str(), type.c_str());
    return KX_ERR_ARG;
  }
  if (!f.has("mlp")) return KX_OK;
  KxFields p;
  KX_DO(f.object("mlp", p));
  std::string kind;
  KX_DO(p.text("kind", kind));
  KX_REQUIRE(kind == "dense", "config.json: %s.kind has to be dense", p.where.c_str());
  L.ff_kind = KxHybridLayer::GLU;
  KX_DO(p.integer("ff", 1, L.ff));
  KX_DO(p.real("limit", L.limit));
  L.alpha = SIGMOID_SLOPE;
  L.bias = UP_BIAS;
  return KX_OK;
}

}  // namespace

bool kx_kagalorn_matches(const KxJson &config) { return kx_config_names(config, "Kagalorn"); }

int kx_kagalorn_config(const KxJson &config, KxHybridConfig &out) {
  out = KxHybridConfig();
  const KxFields top{&config, "model"};
  KX_DO(top.integer("vocab", 1, out.vocab));
  KX_DO(top.integer("width", 1, out.width));
  KX_DO(top.integer("streams", 1, out.streams));
  KX_REQUIRE(out.streams <= KX_MAX_STREAMS, "config.json: %d streams, at most %d", out.streams, KX_MAX_STREAMS);
  out.hyper = true;
  KxFields norm;
  KX_DO(top.object("norm", norm));
  KX_DO(norm.real("eps", out.eps));
  KX_DO(norm.integer("groups", 1, out.groups));
  KX_REQUIRE(out.width % out.groups == 0 && out.groups <= 1024, "config.json: a width of %d in %d groups", out.width, out.groups);
  return top.each("layers", [&](const KxFields &f) {
    out.layers.emplace_back();
    return layer_config(f, out.layers.back());
  });
}
