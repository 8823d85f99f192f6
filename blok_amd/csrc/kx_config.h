// kx_config.h -- reading a design's config.json: members of an object, checked, with messages that name the field
// (host code only).
#pragma once
#include <math.h>
#include <string>
#include "kx_common.h"
#include "kx_json.h"

struct KxFields {  // the members of one object, with the object's name for messages
  const KxJson *o;
  std::string where;
  int integer(const char *key, int lo, int &v) const {
    const KxJson *x = o->get(key);
    KX_REQUIRE(x && x->is(KxJson::NUMBER) && x->num == floor(x->num) && x->num >= lo && x->num <= 1 << 30, "config.json: %s.%s has to be an integer from %d on",
               where.c_str(), key, lo);
    v = (int)x->num;
    return KX_OK;
  }
  int real(const char *key, double &v) const {
    const KxJson *x = o->get(key);
    KX_REQUIRE(x && x->is(KxJson::NUMBER), "config.json: %s.%s has to be a number", where.c_str(), key);
    v = x->num;
    return KX_OK;
  }
  int real(const char *key, float &v) const {
    double d = 0;
    KX_DO(real(key, d));
    v = (float)d;
    return KX_OK;
  }
  int text(const char *key, std::string &v) const {
    const KxJson *x = o->get(key);
    KX_REQUIRE(x && x->is(KxJson::STRING), "config.json: %s.%s has to be a string", where.c_str(), key);
    v = x->str;
    return KX_OK;
  }
  bool has(const char *key) const {
    const KxJson *x = o->get(key);
    return x && !x->is(KxJson::NUL);
  }
  int object(const char *key, KxFields &f) const {
    f.o = o->get(key);
    f.where = where + "." + key;
    KX_REQUIRE(f.o && f.o->is(KxJson::OBJECT), "config.json: %s has to be an object", f.where.c_str());
    return KX_OK;
  }
  // `one` for every element of the list `key`, which has to have some
  template <class F>
  int each(const char *key, F &&one) const {
    const KxJson *list = o->get(key);
    KX_REQUIRE(list && list->is(KxJson::ARRAY) && !list->items.empty(), "config.json: %s has to be a list", key);
    for (size_t i = 0; i < list->items.size(); ++i) {
      const KxFields f{&list->items[i], std::string(key) + "[" + std::to_string(i) + "]"};
      KX_REQUIRE(f.o->is(KxJson::OBJECT), "config.json: %s has to be an object", f.where.c_str());
      KX_DO(one(f));
    }
    return KX_OK;
  }
};
inline bool kx_config_names(const KxJson &config, const char *architecture) {
  const KxJson *a = config.get("architecture");
  return a && a->is(KxJson::STRING) && a->str == architecture;
}
