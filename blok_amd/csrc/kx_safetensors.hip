// kx_safetensors.hip -- see kx_safetensors.h (host code only).
#include <dirent.h>
#include <errno.h>
#include <string.h>
#include <algorithm>
#include <vector>
#include "kx_json.h"
#include "kx_safetensors.h"

namespace {

constexpr uint64_t ALIGN = 4096;             // extents of the loader's reads
constexpr uint64_t HEADER_MAX = 1ull << 28;  // a longer header is not one

int scan_file(const std::string &path, KxTensorMap &out) {
  FILE *f = fopen(path.c_str(), "rb");
  KX_REQUIRE(f, "cannot open %s: %s", path.c_str(), strerror(errno));
  unsigned char len8[8];
  uint64_t n = 0, size = 0;
  bool ok = fread(len8, 1, 8, f) == 8;
  for (int i = 0; i < 8; ++i) n |= (uint64_t)len8[i] << (8 * i);
  std::string text;
  if (ok && fseeko(f, 0, SEEK_END) == 0) size = (uint64_t)ftello(f);
  ok = ok && size >= 8 && n <= HEADER_MAX && n <= size - 8 && fseeko(f, 8, SEEK_SET) == 0;
  if (ok) {
    text.resize(n);
    ok = fread(&text[0], 1, n, f) == n;
  }
  fclose(f);
  KX_REQUIRE(ok, "%s is not a safetensors file", path.c_str());
  KxJson doc;
  std::string err;
  KX_REQUIRE(kx_json_parse(text.data(), text.size(), doc, err) && doc.is(KxJson::OBJECT), "%s: bad header (%s)", path.c_str(), err.c_str());
  const uint64_t data = 8 + n;
  for (const auto &m : doc.members) {
    if (m.first == "__metadata__") continue;
    const KxJson *dt = m.second.get("dtype"), *sh = m.second.get("shape"), *of = m.second.get("data_offsets");
    KX_REQUIRE(dt && sh && of && dt->is(KxJson::STRING) && sh->is(KxJson::ARRAY) && of->is(KxJson::ARRAY) && of->items.size() == 2,
               "%s: tensor %s has no dtype, shape and data_offsets", path.c_str(), m.first.c_str());
    KxTensorRec t;
    t.name = m.first;
    t.file = path;
    t.dtype = dt->str == "BF16" ? "bf16" : dt->str == "F32" ? "f32" : dt->str == "I32" ? "i32" : "";
    KX_REQUIRE(!t.dtype.empty(), "%s: tensor %s has dtype %s (BF16, F32 and I32 are read)", path.c_str(), m.first.c_str(), dt->str.c_str());
    uint64_t bytes = t.dtype == "bf16" ? 2 : 4;
    for (const KxJson &d : sh->items) {
      KX_REQUIRE(d.is(KxJson::NUMBER) && d.num >= 0 && d.num < 4294967296.0 && d.num == (double)(uint64_t)d.num && (d.num == 0 || bytes <= size / (uint64_t)d.num),
                 "%s: tensor %s has a bad shape", path.c_str(), m.first.c_str());
      bytes *= (uint64_t)d.num;
      t.shape += (t.shape.empty() ? "" : "x") + std::to_string((uint64_t)d.num);
    }
    const double lo = of->items[0].num, hi = of->items[1].num;
    KX_REQUIRE(lo >= 0 && hi >= lo && hi <= (double)(size - data) && (uint64_t)(hi - lo) == bytes, "%s: tensor %s: %s %s does not fill its data_offsets",
               path.c_str(), m.first.c_str(), t.dtype.c_str(), t.shape.c_str());
    t.data = data + (uint64_t)lo;
    t.data_bytes = bytes;
    t.off = t.data / ALIGN * ALIGN;
    t.bytes = (t.data + bytes - t.off + ALIGN - 1) / ALIGN * ALIGN;
    KX_REQUIRE(out.emplace(m.first, t).second, "%s: tensor %s is in the directory twice", path.c_str(), m.first.c_str());
  }
  return KX_OK;
}

}  // namespace

int kx_safetensors_scan(const std::string &dir, KxTensorMap &out) {
  std::vector<std::string> files;
  DIR *d = opendir(dir.c_str());
  KX_REQUIRE(d, "cannot open %s: %s", dir.c_str(), strerror(errno));
  const std::string ext = ".safetensors";
  while (const dirent *e = readdir(d)) {
    const std::string name = e->d_name;
    if (name.size() > ext.size() && name.compare(name.size() - ext.size(), ext.size(), ext) == 0) files.push_back(dir + "/" + name);
  }
  closedir(d);
  KX_REQUIRE(!files.empty(), "no safetensors files in %s", dir.c_str());
  std::sort(files.begin(), files.end());
  for (const std::string &f : files) {
    int rc = scan_file(f, out);
    if (rc) return rc;
  }
  return KX_OK;
}
