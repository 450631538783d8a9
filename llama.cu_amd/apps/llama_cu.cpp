// llama_cu: greedy text generation from a model directory.
//
//   llama_cu [matmul_type] [model_name] [prompt] [max_tokens = 200] [context_len = 2048] [sample_seed]
//
// The command line, the printed lines, the stop at token 2, the half-context re-prefill when the
// context is full and the times.txt report follow the reference's main.cpp (9-110); the reference's
// own main.cpp also builds unchanged against include/llama_cu.h.  matmul_type is accepted and
// ignored.  A model name is looked up as models/<name>; a name containing '/' is the directory.
// max_tokens and context_len are additions for testing with small contexts; with sample_seed the
// tokens are drawn from the probabilities (the sampler the reference leaves commented out,
// llama_cu.cu:1202-1203) instead of taking the most probable one.  A directory with a config.json holds a model
// of another family (llama_model::open); without a vocab file its prompt is token ids, and so is the output.
#include <algorithm>
#include <chrono>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <memory>
#include <string>
#include <vector>

#include "llama_cu.h"

using namespace llama_cu;
using steady = std::chrono::steady_clock;

namespace {

struct options {
  std::string model = "7B";
  std::string prompt = "Building a website can be done in 10 easy steps:";
  int max_tokens = 200;
  size_t context_len = 2048;
  bool sample = false;
  uint64_t sample_seed = 0;
};

double seconds_since(steady::time_point t0) { return std::chrono::duration<double>(steady::now() - t0).count(); }

std::string model_dir(std::string const& name) {
  return name.find('/') == std::string::npos ? "models/" + name : name;
}

void print_model_facts(llama_params const& p, size_t context_len) {
  const double mb = 1024.0 * 1024.0;
  printf("Dimension: %d\nSwiGLU multiple: %d\nLayers: %d\nHeads: %d\nVocab: %d\nNorm Epsilon: %f\n"
         "Shared Context Memory: %f MB\nPer-Layer Context Memory: %f MB\n",
         p.dim, p.multiple_of, p.n_layers, p.n_heads, p.n_vocab, p.norm_eps,
         p.shared_context_memory_size(context_len) / mb, p.kv_cache_size(context_len) / mb);
}

// A LLaMA in the reference's format; nullptr after a message.
std::unique_ptr<llama_model> load_llama(std::string const& dir, size_t context_len) {
  mapped_buffer params_buf(dir + "/params");
  if (!params_buf.is_ok()) {
    fprintf(stderr, "Could not load params file\n");
    return nullptr;
  }
  if (!mapped_buffer(dir + "/vocab").is_ok()) {
    fprintf(stderr, "Could not load vocab file\n");
    return nullptr;
  }
  llama_params params;
  if (!params.load(params_buf)) {
    fprintf(stderr, "Invalid model parameters\n");
    return nullptr;
  }
  llama_partition partition;
  partition.autopipe(params, context_len);
  partition.debug_print();
  if (!partition.is_valid()) {
    fprintf(stderr, "Could not partition model\n");
    return nullptr;
  }
  print_model_facts(params, context_len);
  auto model = llama_model::load(params, partition, dir);
  if (!model) {
    fprintf(stderr, "Could not load model\n");
  }
  return model;
}

// A model with a config.json; nullptr after a message.
std::unique_ptr<llama_model> load_configured(std::string const& dir, size_t context_len) {
  auto model = llama_model::open(dir, (int)context_len);
  if (!model) {
    fprintf(stderr, "Could not load model\n");
    return nullptr;
  }
  llama_params const& p = model->params;
  printf("Dimension: %d\nLayers: %d\nHeads: %d\nVocab: %d\nNorm Epsilon: %f\n", p.dim, p.n_layers, p.n_heads, p.n_vocab, p.norm_eps);
  return model;
}

// token ids written as numbers; false on anything else
bool parse_ids(std::string const& text, std::vector<int32_t>& ids) {
  const char* at = text.c_str();
  while (true) {
    at += strspn(at, " ,\t\n");
    if (*at == '\0') return !ids.empty();
    char* end = nullptr;
    const long id = strtol(at, &end, 10);
    if (end == at || id < 0 || id > INT32_MAX) return false;
    ids.push_back((int32_t)id);
    at = end;
  }
}

// Generates up to max_tokens tokens after the prompt; returns the per-token wall times.
std::vector<float> generate(llama_context& context, llama_vocabulary* vocab, std::vector<int32_t> const& prompt,
                            options const& opt, int& generated) {
  std::vector<int32_t> history = prompt;  // everything fed or produced so far
  std::vector<int32_t> feed = prompt;     // what the next call consumes
  std::vector<float> times;
  generated = 0;
  while (generated < opt.max_tokens) {
    const auto t0 = steady::now();
    if (context.tokens_left() == 0) {
      // context full: start over from the most recent half of the history (main.cpp:83-87)
      context.clear_tokens();
      const size_t keep = std::min(history.size(), opt.context_len / 2);
      feed.assign(history.end() - keep, history.end());
    }
    const int token = context.forward(feed.data(), (int)feed.size(), nullptr, 0, nullptr);
    const float dt = (float)seconds_since(t0);
    if (token < 0) {
      fprintf(stderr, "\nnext_token failed: %zu tokens do not fit the context or the vocabulary\n", feed.size());
      break;
    }
    if (vocab && token == 2) {  // end of sequence
      break;
    }
    if (vocab) {
      fputs(vocab->tokens[token].text.c_str(), stdout);
    } else {
      printf("%s%d", generated > 0 ? " " : "", token);
    }
    fflush(stdout);
    feed.assign(1, token);
    history.push_back(token);
    times.push_back(dt);
    ++generated;
  }
  return times;
}

}  // namespace

int main(int argc, char const** argv) {
  options opt;
  if (argc > 1) matmul_type = atoi(argv[1]);
  if (argc > 2) opt.model = argv[2];
  if (argc > 3) opt.prompt = argv[3];
  if (argc > 4) opt.max_tokens = atoi(argv[4]);
  if (argc > 5) opt.context_len = (size_t)atol(argv[5]);
  if (argc > 6) {
    opt.sample = true;
    opt.sample_seed = strtoull(argv[6], nullptr, 10);
  }
  if (opt.context_len < 2) {
    fprintf(stderr, "context_len must be at least 2\n");
    return 1;
  }
  initialize();
  const std::string dir = model_dir(opt.model);
  const bool configured = mapped_buffer(dir + "/config.json").is_ok();
  mapped_buffer vocab_buf(dir + "/vocab");
  auto model = configured ? load_configured(dir, opt.context_len) : load_llama(dir, opt.context_len);
  if (!model) {
    return 1;
  }
  std::unique_ptr<llama_vocabulary> vocab;
  if (vocab_buf.is_ok()) {
    vocab = std::make_unique<llama_vocabulary>(vocab_buf);
    if (vocab->tokens.size() != model->params.n_vocab) {
      fprintf(stderr, "Vocab size mismatch\n");
      return 1;
    }
  }
  opt.context_len = std::min(opt.context_len, (size_t)model->max_context());
  auto context = llama_context::create(model.get(), (int)opt.context_len, 0.8f);
  printf("Context memory: %f MB\n", context->context_memory_usage() / 1024.0 / 1024.0);
  if (opt.sample) {
    context->sample_with_seed(opt.sample_seed);
  }

  std::vector<int32_t> prompt;
  if (vocab) {
    const std::vector<short> ids = vocab->tokenize(opt.prompt, true);
    prompt.assign(ids.begin(), ids.end());
  } else if (!parse_ids(opt.prompt, prompt)) {
    fprintf(stderr, "The model has no vocab file: the prompt must be token ids\n");
    return 1;
  }
  if (prompt.size() > opt.context_len) {
    fprintf(stderr, "Prompt of %zu tokens exceeds the context of %zu\n", prompt.size(), opt.context_len);
    return 1;
  }
  int generated = 0;
  const auto start = steady::now();
  const std::vector<float> times = generate(*context, vocab.get(), prompt, opt, generated);
  printf("\ntokens: %d time: %f\n", generated, seconds_since(start));
  // times.txt: prompt length, then one wall time per generated token (plot_times.py reads it)
  FILE* fp = fopen("times.txt", "w");
  if (!fp) {
    fprintf(stderr, "Could not write times.txt\n");
    return 1;
  }
  fprintf(fp, "%zu\n", prompt.size());
  for (float t : times) fprintf(fp, "%f\n", t);
  fclose(fp);
  return 0;
}
