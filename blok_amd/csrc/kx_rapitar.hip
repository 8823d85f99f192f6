// kx_rapitar.hip -- config.json of the Rapitar design -> a hybrid decoder's configuration (host code only).
//
// The file gives vocab, width, norm.eps and per layer its mixer's type and sizes and its feed-forward; what the design
// fixes for all its models is set here: parallel layers, norm weights about one, a sink and a gate in the attention, and
// the feed-forwards' activations.
#include <math.h>
#include "kx_config.h"
#include "kx_hybrid.h"

namespace {

int mamba2_config(const KxFields &m, KxHybridLayer &L) {
  L.mixer = KxHybridLayer::SSD;
  KxSsdSpec &s = L.ssd;
  KX_DO(m.integer("heads", 1, s.heads));
  KX_DO(m.integer("vdim", 1, s.vdim));
  KX_DO(m.integer("state", 1, s.state));
  KX_DO(m.integer("groups", 1, s.groups));
  KX_DO(m.integer("conv", 1, s.taps));
  KX_DO(m.integer("norm_groups", 1, L.norm_groups));
  KX_REQUIRE(s.heads % s.groups == 0, "config.json: %s: %d heads in %d groups", m.where.c_str(), s.heads, s.groups);
  KX_REQUIRE(kx_ssd_inner(s) % L.norm_groups == 0, "config.json: %s: %d columns in %d norm_groups", m.where.c_str(), kx_ssd_inner(s), L.norm_groups);
  KX_REQUIRE(s.state <= KX_SCAN_MAX_DIM, "config.json: %s.state=%d: at most %d", m.where.c_str(), s.state, KX_SCAN_MAX_DIM);
  return KX_OK;
}

int wkv_config(const KxFields &m, KxHybridLayer &L) {
  L.mixer = KxHybridLayer::WKV;
  KX_DO(m.integer("heads", 1, L.wkv.heads));
  KX_DO(m.integer("dim", 1, L.wkv.dim));
  KX_REQUIRE(L.wkv.dim <= KX_SCAN_MAX_DIM, "config.json: %s.dim=%d: at most %d", m.where.c_str(), L.wkv.dim, KX_SCAN_MAX_DIM);
  return KX_OK;
}

int latent_config(const KxFields &m, KxHybridLayer &L) {
  L.mixer = KxHybridLayer::LATENT;
  KxLatentSpec &s = L.latent;
  KX_DO(m.integer("heads", 1, s.heads));
  KX_DO(m.integer("dim", 1, s.dim));
  KX_DO(m.integer("rot_dim", 1, s.rot_dim));
  KX_DO(m.integer("vdim", 1, s.vdim));
  KX_DO(m.integer("kv_rank", 1, s.kv_rank));
  KX_DO(m.integer("q_rank", 1, L.q_rank));
  KX_DO(m.real("scale", s.scale));
  KxFields rot;
  KX_DO(m.object("rot", rot));
  KX_DO(rot.integer("dims", 0, s.rot));
  KX_DO(rot.real("base", s.base));
  KX_REQUIRE(s.rot % 2 == 0 && s.rot <= s.rot_dim && s.base > 0, "config.json: %s: %d of %d dimensions in pairs, base %g", rot.where.c_str(), s.rot, s.rot_dim, s.base);
  KX_REQUIRE(s.kv_rank <= 2048, "config.json: %s.kv_rank=%d: at most 2048", m.where.c_str(), s.kv_rank);
  s.sink = 1;
  L.gate = true;
  return KX_OK;
}

int mlp_config(const KxFields &p, KxHybridLayer &L) {
  std::string kind;
  KX_DO(p.text("kind", kind));
  if (kind == "dense") {
    L.ff_kind = KxHybridLayer::GELU;
    return p.integer("ff", 1, L.ff);
  }
  KX_REQUIRE(kind == "moe", "config.json: %s.kind is %s (dense and moe are known)", p.where.c_str(), kind.c_str());
  L.ff_kind = KxHybridLayer::EXPERTS;
  L.limit = INFINITY;
  L.alpha = 1.0f;
  KxFields e, r;
  KX_DO(p.object("expert", e));
  KX_DO(e.integer("ff", 1, L.ff));
  KX_DO(p.object("router", r));
  KX_DO(r.integer("experts", 1, L.experts));
  KX_DO(r.integer("top", 1, L.top));
  KX_REQUIRE(L.top <= L.experts && L.top <= KX_MAX_TOP && L.experts <= KX_MAX_EXPERTS, "config.json: %s: %d of %d experts (at most %d of %d)", r.where.c_str(), L.top,
             L.experts, KX_MAX_TOP, KX_MAX_EXPERTS);
  return KX_OK;
}

int layer_config(const KxFields &f, KxHybridLayer &L) {
  std::string type;
  KX_DO(f.text("type", type));
  KxFields m;
  KX_DO(f.object("mixer", m));
  if (type == "mamba2") KX_DO(mamba2_config(m, L));
  else if (type == "wkv") KX_DO(wkv_config(m, L));
  else if (type == "latent_attention") KX_DO(latent_config(m, L));
  else {
    kx_set_error("config.json: %s.type is %s (mamba2, wkv and latent_attention are known)", f.where.c_str(), type.c_str());
    return KX_ERR_ARG;
  }
  if (!f.has("mlp")) return KX_OK;
  KxFields p;
  KX_DO(f.object("mlp", p));
  return mlp_config(p, L);
}

}  // namespace

bool kx_rapitar_matches(const KxJson &config) { return kx_config_names(config, "Rapitar"); }

int kx_rapitar_config(const KxJson &config, KxHybridConfig &out) {
  out = KxHybridConfig();
  const KxFields top{&config, "model"};
  KX_DO(top.integer("vocab", 1, out.vocab));
  KX_DO(top.integer("width", 1, out.width));
  out.parallel = out.norm_about_one = true;
  KxFields norm;
  KX_DO(top.object("norm", norm));
  KX_DO(norm.real("eps", out.eps));
  return top.each("layers", [&](const KxFields &f) {
    out.layers.emplace_back();
    return layer_config(f, out.layers.back());
  });
}
