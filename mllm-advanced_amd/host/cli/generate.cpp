// Greedy generation from a model folder, by token ids: the class is chosen by config.json.
//
//   generate --model DIR --tokens 1,2,3 [--max-new N] [--dtype bfloat16|float32] [--max-tokens N] [--chunk N] [--eos ID]
//
// Prints the generated ids on one line. --tokens may be given more than once: the prompts run one after the other.
#include <cstdio>
#include <string>
#include <vector>

#include "mllm/Backends/HIP/HipBackend.hpp"
#include "mllm/Engine/Context.hpp"
#include "mllm/Models/CausalLM.hpp"
#include "mllm/Utils/Log.hpp"

using namespace mllm;  // NOLINT

int main(int argc, char** argv) {
  std::string model_dir;
  std::vector<std::vector<int64_t>> prompts;
  models::CausalLMOptions options;
  int max_new = 32;
  int64_t eos = -1;
  bool ok = argc > 1;
  for (int i = 1; i < argc; i += 2) {
    const std::string key = argv[i];
    if (i + 1 >= argc) {
      ok = false;
      break;
    }
    const std::string value = argv[i + 1];
    if (key == "--model") model_dir = value;
    else if (key == "--dtype") options.dtype = value;
    else if (key == "--max-tokens") options.max_tokens = std::atoi(value.c_str());
    else if (key == "--chunk") options.max_chunk = std::atoi(value.c_str());
    else if (key == "--max-new") max_new = std::atoi(value.c_str());
    else if (key == "--eos") eos = std::atoll(value.c_str());
    else if (key == "--tokens") {
      prompts.emplace_back();
      for (const char* p = value.c_str(); *p;) {
        char* end = nullptr;
        prompts.back().push_back(std::strtoll(p, &end, 10));
        if (end == p) {
          ok = false;
          break;
        }
        p = *end == ',' ? end + 1 : end;
      }
    } else {
      ok = false;
    }
  }
  if (!ok || model_dir.empty() || prompts.empty() || options.max_tokens <= 0 || options.max_chunk <= 0 ||
      (options.dtype != "bfloat16" && options.dtype != "float32")) {
    std::fprintf(stderr, "usage: generate --model DIR --tokens 1,2,3 [--max-new N] [--dtype bfloat16|float32] "
                         "[--max-tokens N] [--chunk N] [--eos ID]\n");
    return 2;
  }
  auto& ctx = MllmEngineCtx::instance();
  ctx.registerBackend(hip::createHostBackend());
  ctx.registerBackend(hip::createHipBackend());
  auto& registry = models::CausalLMRegistry::instance();
  models::registerSuripel(registry);
  models::registerLesarax(registry);
  models::registerQwen2(registry);
  {
    auto model = registry.load(model_dir, options);
    for (const auto& prompt : prompts) {
      const std::vector<int64_t> out = model->generate(prompt, max_new, eos);
      for (size_t i = 0; i < out.size(); ++i) std::printf("%s%lld", i ? " " : "", static_cast<long long>(out[i]));
      std::printf("\n");
      std::fflush(stdout);
    }
  }
  ctx.shutdown();
  return 0;
}
