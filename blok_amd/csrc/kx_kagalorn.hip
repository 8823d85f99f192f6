// kx_kagalorn.hip -- config.json of the Kagalorn design -> a hybrid decoder's configuration (host code only).
//
// The file gives vocab, width, streams, norm {eps, groups} and per layer its mixer's type and sizes and its
// feed-forward; what the design fixes for all its models is set here.
#include <math.h>
#include "kx_common.h"
#include "kx_hybrid.h"
#include "kx_linear.h"

namespace {

constexpr float SIGMOID_SLOPE = 1.702f, UP_BIAS = 1.0f;  // of the clamped gated feed-forward
constexpr float UNIT_EPS = 1e-6f;                        // under the root of the delta rule's unit norms

struct Fields {  // the members of one object, with the object's name for messages
  const KxJson *o;
  std::string where;
  int integer(const char *key, int lo, int &v) const {
    const KxJson *x = o->get(key);
    KX_REQUIRE(x && x->is(KxJson::NUMBER) && x->num == floor(x->num) && x->num >= lo && x->num <= 1 << 30, "config.json: %s.%s has to be an integer from %d on",
               where.c_str(), key, lo);
    v = (int)x->num;
    return KX_OK;
  }
  int real(const char *key, float &v) const {
    const KxJson *x = o->get(key);
    KX_REQUIRE(x && x->is(KxJson::NUMBER), "config.json: %s.%s has to be a number", where.c_str(), key);
    v = (float)x->num;
    return KX_OK;
  }
  int object(const char *key, Fields &f) const {
    f.o = o->get(key);
    f.where = where + "." + key;
    KX_REQUIRE(f.o && f.o->is(KxJson::OBJECT), "config.json: %s has to be an object", f.where.c_str());
    return KX_OK;
  }
};

#define KX_TRY(call) do { if (int rc_ = (call)) return rc_; } while (0)

int layer_config(const Fields &f, KxHybridLayer &L) {
  const KxJson *type = f.o->get("type");
  KX_REQUIRE(type && type->is(KxJson::STRING), "config.json: %s.type has to be a string", f.where.c_str());
  Fields m;
  KX_TRY(f.object("mixer", m));
  int heads, kv, dim, vdim;
  KX_TRY(m.integer("heads", 1, heads));
  KX_TRY(m.integer("kv_heads", 1, kv));
  KX_TRY(m.integer("dim", 1, dim));
  KX_TRY(m.integer("vdim", 1, vdim));
  KX_REQUIRE(heads % kv == 0, "config.json: %s: %d heads on %d kv_heads", m.where.c_str(), heads, kv);
  if (type->str == "attention") {
    L.mixer = KxHybridLayer::ATTENTION;
    KxWindowSpec &a = L.attn;
    a.heads = heads; a.kv_heads = kv; a.dim = dim; a.vdim = vdim;
    a.sink = 1;
    L.qk_norm = L.gate = true;
    KX_TRY(m.real("scale", a.scale));
    Fields mask;
    KX_TRY(m.object("mask", mask));
    KX_TRY(mask.integer("size", 1, a.size));
    KX_TRY(mask.integer("pool", 1, a.pool));
  } else if (type->str == "delta") {
    L.mixer = KxHybridLayer::DELTA;
    KxDeltaSpec &d = L.delta;
    d.heads = heads; d.kv_heads = kv; d.dim = dim; d.vdim = vdim;
    d.unit_eps = UNIT_EPS;
    KX_TRY(m.integer("conv", 1, d.taps));
    KX_REQUIRE(dim <= 256, "config.json: %s.dim=%d: the delta rule takes keys of up to 256", m.where.c_str(), dim);
  } else {
    kx_set_error("config.json: %s.type is %s (attention and delta are known)", f.where.c_str(), type->str.c_str());
    return KX_ERR_ARG;
  }
  const KxJson *mlp = f.o->get("mlp");
  if (!mlp || mlp->is(KxJson::NUL)) return KX_OK;
  Fields p;
  KX_TRY(f.object("mlp", p));
  const KxJson *kind = p.o->get("kind");
  KX_REQUIRE(kind && kind->is(KxJson::STRING) && kind->str == "dense", "config.json: %s.kind has to be dense", p.where.c_str());
  KX_TRY(p.integer("ff", 1, L.ff));
  KX_TRY(p.real("limit", L.limit));
  L.alpha = SIGMOID_SLOPE;
  L.bias = UP_BIAS;
  return KX_OK;
}

}  // namespace

bool kx_kagalorn_matches(const KxJson &config) {
  const KxJson *a = config.get("architecture");
  return a && a->is(KxJson::STRING) && a->str == "Kagalorn";
}

int kx_kagalorn_config(const KxJson &config, KxHybridConfig &out) {
  out = KxHybridConfig();
  const Fields top{&config, "model"};
  KX_TRY(top.integer("vocab", 1, out.vocab));
  KX_TRY(top.integer("width", 1, out.width));
  KX_TRY(top.integer("streams", 1, out.streams));
  KX_REQUIRE(out.streams <= KX_MAX_STREAMS, "config.json: %d streams, at most %d", out.streams, KX_MAX_STREAMS);
  out.hyper = true;
  Fields norm;
  KX_TRY(top.object("norm", norm));
  KX_TRY(norm.real("eps", out.eps));
  KX_TRY(norm.integer("groups", 1, out.groups));
  KX_REQUIRE(out.width % out.groups == 0 && out.groups <= 1024, "config.json: a width of %d in %d groups", out.width, out.groups);
  const KxJson *layers = config.get("layers");
  KX_REQUIRE(layers && layers->is(KxJson::ARRAY) && !layers->items.empty(), "config.json: layers has to be a list");
  for (size_t i = 0; i < layers->items.size(); ++i) {
    const Fields f{&layers->items[i], "layers[" + std::to_string(i) + "]"};
    KX_REQUIRE(f.o->is(KxJson::OBJECT), "config.json: %s has to be an object", f.where.c_str());
    KxHybridLayer L;
    KX_TRY(layer_config(f, L));
    out.layers.push_back(L);
  }
  return KX_OK;
}
