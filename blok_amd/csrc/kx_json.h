// kx_json.h -- a JSON reader for config.json and safetensors headers (host code only).
#pragma once
#include <stdint.h>
#include <string>
#include <utility>
#include <vector>

struct KxJson {
  enum Kind { NUL, BOOL, NUMBER, STRING, ARRAY, OBJECT } kind = NUL;
  bool b = false;
  double num = 0;
  std::string str;
  std::vector<KxJson> items;                            // ARRAY
  std::vector<std::pair<std::string, KxJson>> members;  // OBJECT, in file order
  const KxJson *get(const char *key) const;             // member of an object, or nullptr
  bool is(Kind k) const { return kind == k; }
};

// Parses a whole document.  Returns false with a message that names the byte offset.
bool kx_json_parse(const char *text, size_t len, KxJson &out, std::string &err);
// Reads and parses a file; sets the error message and returns a status like every entry point.
int kx_json_file(const std::string &path, KxJson &out);
