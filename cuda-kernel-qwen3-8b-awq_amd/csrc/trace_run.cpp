// Replays a trace: given token ids go through a model step by step, the logits asked for are written to files.
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
// Steps come from standard input, one JSON object a line:
//   {"step": 4, "entries": [{"id": "x7", "tokens": [12, 8], "want": [1]}], "end": ["x7"]}
// A step's entry brings the next tokens of a request; a request that was not running starts a new sequence, and
// requests come one after the other.  A step in which something is wanted writes DIR/<step>.f32, [wanted][vocab]
// little-endian binary32; every step prints "done <step>".
#include <stdio.h>
#include <stdlib.h>
#include <string.h>

#include <iostream>
#include <string>
#include <vector>

#include "../../include/awq_infer.h"
#include "checkpoint.hpp"

namespace {

int fail(const std::string& what) {
  fprintf(stderr, "trace_run: %s\n", what.c_str());
  return 1;
}

bool int_list(const Json* v, std::vector<int32_t>* out) {
  out->clear();
  if (!v || !v->is(Json::Array)) return false;
  for (const Json& x : v->items) {
    if (!x.is(Json::Number) || !(x.number >= 0.0 && x.number < 2147483648.0) || x.number != (int32_t)x.number) return false;
    out->push_back((int32_t)x.number);
  }
  return true;
}

std::string id_of(const Json& v) { return v.is(Json::Number) ? std::to_string(v.number) : v.str; }

struct Closer {
  awq_engine* e = nullptr;
  ~Closer() { awq_destroy(e); }
};

}  // namespace

int main(int argc, char** argv) {
  std::string model, out, dtype = "bfloat16";
  awq_open_options opt{};
  for (int i = 1; i < argc; i += 2) {
    const std::string key = argv[i];
    if (i + 1 >= argc) return fail(key + " has no value");
    const char* value = argv[i + 1];
    if (key == "--model") model = value;
    else if (key == "--out") out = value;
    else if (key == "--dtype") dtype = value;
    else if (key == "--max-tokens") opt.max_positions = atoll(value);
    else return fail("unknown option " + key);
  }
  if (model.empty() || out.empty()) return fail("--model and --out are required");
  if (dtype == "bfloat16") opt.dtype = AWQ_DTYPE_BFLOAT16;
  else if (dtype == "float32") opt.dtype = AWQ_DTYPE_FLOAT32;
  else return fail("--dtype is bfloat16 or float32");
  Closer engine;
  if (awq_open(model.c_str(), &opt, &engine.e)) return fail(awq_last_error());
  awq_engine* e = engine.e;
  const int64_t vocab = awq_vocab_size(e);

  std::string line, running;
  bool live = false;
  std::vector<int32_t> ids, want;
  std::vector<float> logits;
  while (std::getline(std::cin, line)) {
    if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
    Json j;
    std::string err;
    if (!json_parse(line.data(), line.size(), &j, &err)) return fail("a step is no JSON: " + err);
    const Json *step = j.find("step"), *entries = j.find("entries"), *end = j.find("end");
    if (!step || !step->is(Json::Number) || !entries || !entries->is(Json::Array)) return fail("a step lacks step or entries");
    const std::string name = std::to_string((long long)step->number);
    FILE* f = nullptr;
    for (const Json& en : entries->items) {
      const Json* id = en.find("id");
      if (!id || !int_list(en.find("tokens"), &ids) || !int_list(en.find("want"), &want))
        return fail("step " + name + ": a bad entry");
      if (!live || id_of(*id) != running) {
        if (awq_reset(e)) return fail(awq_last_error());
        running = id_of(*id);
        live = true;
      }
      logits.resize(want.size() * (size_t)vocab);
      if (awq_forward(e, ids.data(), (int32_t)ids.size(), want.data(), (int32_t)want.size(), logits.data()))
        return fail("step " + name + ": " + awq_last_error());
      if (want.empty()) continue;
      if (!f && !(f = fopen((out + "/" + name + ".f32").c_str(), "wb"))) return fail("could not create the output of step " + name);
      if (fwrite(logits.data(), 4, logits.size(), f) != logits.size()) return fail("short write of step " + name);
    }
    if (f && fclose(f) != 0) return fail("short write of step " + name);
    if (end)
      for (const Json& v : end->items)
        if (id_of(v) == running) live = false;
    printf("done %s\n", name.c_str());
    fflush(stdout);
  }
  return 0;
}
