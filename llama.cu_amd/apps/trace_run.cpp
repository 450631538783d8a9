// trace_run: feeds given token ids through a model step by step and writes logits.
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
// Steps come on standard input, one JSON object a line:
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
// Each entry continues the sequence of its id; the logits at the places of `want` go to DIR/<step>.f32 (fp32,
// in order), and "done <step>" follows on standard output.  A sequence named in `end` gives its context
// back, which the next new id takes over.  At the end of the input the program returns 0.
#include <algorithm>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <iostream>
#include <map>
#include <string>
#include <vector>

#include "json.hpp"
#include "llama_cu.h"

using namespace llama_cu;

namespace {

struct options {
  std::string model, out;
  element_type type = element_type::bf16;
  int max_tokens = 0;
};

bool parse_options(int argc, char const** argv, options& opt) {
  for (int i = 1; i + 1 < argc; i += 2) {
    const std::string key = argv[i], value = argv[i + 1];
    if (key == "--model") {
      opt.model = value;
    } else if (key == "--out") {
      opt.out = value;
    } else if (key == "--max-tokens") {
      opt.max_tokens = atoi(value.c_str());
    } else if (key == "--dtype" && (value == "bfloat16" || value == "float32")) {
      opt.type = value == "float32" ? element_type::f32 : element_type::bf16;
    } else {
      return false;
    }
  }
  return argc % 2 == 1 && !opt.model.empty() && !opt.out.empty();
}

// live sequences, and the contexts that ended ones left behind
struct sequences {
  llama_model& model;
  int context_len;
  std::map<std::string, std::unique_ptr<llama_context>> live;
  std::vector<std::unique_ptr<llama_context>> idle;

  llama_context* get(std::string const& id) {
    auto it = live.find(id);
    if (it != live.end()) return it->second.get();
    std::unique_ptr<llama_context> c;
    if (!idle.empty()) {
      c = std::move(idle.back());
      idle.pop_back();
      c->clear_tokens();
    } else {
      c = llama_context::create(&model, context_len, 1.0f);
    }
    return c ? (live[id] = std::move(c)).get() : nullptr;
  }
  void end(std::string const& id) {
    auto it = live.find(id);
    if (it == live.end()) return;
    idle.push_back(std::move(it->second));
    live.erase(it);
  }
};

bool ids_of(json const& list, std::vector<int32_t>& out) {
  out.clear();
  for (json const& v : list.items) {
    int64_t n;
    if (!v.get_int(0, INT32_MAX, n)) return false;
    out.push_back((int32_t)n);
  }
  return true;
}

int fail(const char* what) {
  fprintf(stderr, "trace_run: %s\n", what);
  return 1;
}

}  // namespace

int main(int argc, char const** argv) {
  options opt;
  if (!parse_options(argc, argv, opt)) {
    fprintf(stderr, "usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N\n");
    return 2;
  }
  auto model = llama_model::open(opt.model, opt.max_tokens > 0 ? opt.max_tokens : 2048, opt.type);
  if (!model) return fail("could not load the model");
  const int most = opt.max_tokens > 0 ? model->max_context() : std::min(model->max_context(), 8192);
  sequences seqs{*model, opt.max_tokens > 0 && opt.max_tokens < most ? opt.max_tokens : most, {}, {}};
  const size_t vocab = model->params.n_vocab;
  std::string line, error;
  std::vector<int32_t> tokens, want;
  while (std::getline(std::cin, line)) {
    if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
    json step;
    int64_t number;
    if (!json::parse(line, step, error) || !step["step"].get_int(0, INT64_C(1) << 53, number)) return fail("a step that cannot be read");
    std::vector<float> logits;
    for (json const& entry : step["entries"].items) {
      llama_context* c = seqs.get(entry["id"].text);
      if (!c || !ids_of(entry["tokens"], tokens) || !ids_of(entry["want"], want)) return fail("an entry that cannot be served");
      if (tokens.empty()) continue;
      const size_t at = logits.size();
      logits.resize(at + want.size() * vocab);
      if (c->forward(tokens.data(), (int)tokens.size(), want.data(), (int)want.size(), logits.data() + at) < 0) {
        return fail("tokens that do not fit the model or its context");
      }
    }
    if (!logits.empty()) {
      const std::string path = opt.out + "/" + std::to_string(number) + ".f32";
      FILE* f = fopen(path.c_str(), "wb");
      const bool ok = f && fwrite(logits.data(), sizeof(float), logits.size(), f) == logits.size();
      if (!f || fclose(f) != 0 || !ok) return fail("an output file that cannot be written");
    }
    for (json const& id : step["end"].items) seqs.end(id.text);
    printf("done %lld\n", (long long)number);
    fflush(stdout);
  }
  return 0;
}
