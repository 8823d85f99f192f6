// kx_trace.cpp -- replays a trace of token ids through a model directory and writes the logits that are asked for.
//
//   kx-trace --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
// Standard input has one step a line, {"step": n, "entries": [{"id": s, "tokens": [..], "want": [..]}], "end": [s, ..]}:
// the next tokens of a request, the places among them whose logits are wanted, and the requests that are finished
// after the step.  A step has one entry and requests come one after the other.  Wanted logits go to
// DIR/<step>.f32, and "done <step>" is printed after every step.  The model is opened through the library's registry
// and driven with kx_restart and kx_extend; nothing is sampled.
#include <errno.h>
#include <stdint.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>
#include <iostream>
#include <string>
#include <vector>
#include "../../include/kx.h"
#include "kx_json.h"

[[noreturn]] static void die(const std::string &m, int code = 1) {
  fprintf(stderr, "trace: %s\n", m.c_str());
  exit(code);
}
static void check(int rc) {
  if (rc) die(kx_last_error());
}

static const KxJson &need(const KxJson &o, const char *key, KxJson::Kind kind) {
  const KxJson *v = o.get(key);
  if (!v || !v->is(kind)) die(std::string("a step without a proper \"") + key + "\"");
  return *v;
}
static long integer(const KxJson &v, double lo, double hi) {
  if (!v.is(KxJson::NUMBER) || v.num < lo || v.num > hi || v.num != (double)(long)v.num) die("a number that is not an integer in range");
  return (long)v.num;
}

int main(int argc, char **argv) {
  std::string model, dtype, out;
  long max_tokens = 0;
  for (int i = 1; i < argc; i += 2) {
    const std::string f = argv[i];
    if (i + 1 >= argc) die("usage: kx-trace --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N");
    const char *v = argv[i + 1];
    if (f == "--model") model = v;
    else if (f == "--dtype") dtype = v;
    else if (f == "--out") out = v;
    else if (f == "--max-tokens") {
      char *end = nullptr;
      errno = 0;
      max_tokens = strtol(v, &end, 10);
      if (errno || end == v || *end || max_tokens < 1 || max_tokens > 1 << 30) die("bad --max-tokens");
    } else die("unknown flag: " + f);
  }
  if (model.empty() || out.empty() || !max_tokens) die("--model, --dtype, --out and --max-tokens are needed");
  if (dtype != "bfloat16" && dtype != "float32") die("bad --dtype");
  kx_open_options o;
  check(kx_open_options_default(&o));
  o.dtype = dtype == "float32" ? KX_DTYPE_F32 : KX_DTYPE_BF16;
  o.max_context = (int32_t)max_tokens;
  kx_model *m = nullptr;
  check(kx_model_open(model.c_str(), &o, &m));
  kx_model_shape shape;
  check(kx_model_info(m, &shape));

  std::string line, live, err;  // live: the request whose tokens the model holds
  while (std::getline(std::cin, line)) {
    if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
    KxJson step;
    if (!kx_json_parse(line.data(), line.size(), step, err)) die("bad step: " + err);
    const long number = integer(need(step, "step", KxJson::NUMBER), 0, 1e15);
    for (const KxJson &e : need(step, "entries", KxJson::ARRAY).items) {
      const std::string &id = need(e, "id", KxJson::STRING).str;
      if (live.empty()) check(kx_restart(m, 1));
      else if (live != id) die("request " + id + " while " + live + " is not finished: one request at a time");
      live = id;
      std::vector<uint32_t> tokens;
      for (const KxJson &t : need(e, "tokens", KxJson::ARRAY).items) tokens.push_back((uint32_t)integer(t, 0, shape.vocab - 1));
      std::vector<int32_t> want;
      for (const KxJson &w : need(e, "want", KxJson::ARRAY).items) want.push_back((int32_t)integer(w, 0, (double)tokens.size() - 1));
      if (tokens.empty()) continue;
      std::vector<float> logits(want.size() * (size_t)shape.vocab);
      check(kx_extend(m, tokens.data(), (int32_t)tokens.size(), want.data(), (int32_t)want.size(), logits.data()));
      if (want.empty()) continue;
      const std::string path = out + "/" + std::to_string(number) + ".f32";
      FILE *f = fopen(path.c_str(), &e == &step.get("entries")->items.front() ? "wb" : "ab");
      if (!f) die("cannot write " + path + ": " + strerror(errno));
      const bool ok = fwrite(logits.data(), 4, logits.size(), f) == logits.size();
      if (fclose(f) || !ok) die("cannot write " + path);
    }
    for (const KxJson &e : need(step, "end", KxJson::ARRAY).items)
      if (e.is(KxJson::STRING) && e.str == live) live.clear();
    printf("done %ld\n", number);
    fflush(stdout);
  }
  check(kx_model_destroy(m));
  return 0;
}
