// Replays a trace of token ids through a model and writes the logits that are asked for.
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]
//
// Standard input, one JSON object a line:
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}
// Each entry appends tokens to the request of that id (a new id starts a sequence); `want` are the places among these
// tokens whose logits are written to OUT/<step>.f32, in order, [wanted][vocab] little-endian f32. Requests under "end"
// are given back after the step. Every step is answered by a line "done <step>".
#include <cstdio>
#include <iostream>
#include <map>
#include <string>
#include <vector>

#include "mllm/Backends/HIP/HipBackend.hpp"
#include "mllm/Engine/Context.hpp"
#include "mllm/Models/CausalLM.hpp"
#include "mllm/Utils/Log.hpp"

using namespace mllm;  // NOLINT

int main(int argc, char** argv) {
  std::string model_dir, out_dir;
  models::CausalLMOptions options;
  bool ok = argc > 1;
  for (int i = 1; i < argc; i += 2) {
    const std::string key = argv[i];
    if (i + 1 >= argc) {
      ok = false;
      break;
    }
    const std::string value = argv[i + 1];
    if (key == "--model") model_dir = value;
    else if (key == "--out") out_dir = value;
    else if (key == "--dtype") options.dtype = value;
    else if (key == "--max-tokens") options.max_tokens = std::atoi(value.c_str());
    else ok = false;
  }
  if (!ok || model_dir.empty() || out_dir.empty() || options.max_tokens <= 0 ||
      (options.dtype != "bfloat16" && options.dtype != "float32")) {
    std::fprintf(stderr, "usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]\n");
    return 2;
  }
  auto& ctx = MllmEngineCtx::instance();
  ctx.registerBackend(hip::createHostBackend());
  ctx.registerBackend(hip::createHipRuntimeBackend());
  auto& registry = models::CausalLMRegistry::instance();
  // the families that give logits at any place
  models::registerSuripel(registry);
  models::registerLesarax(registry);
  {
    auto model = registry.load(model_dir, options);
    std::map<std::string, int32_t> live;
    std::string line;
    while (std::getline(std::cin, line)) {
      if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
      const Json step = Json::parse(line, "request line");
      const int64_t number = step["step"].integer();
      std::vector<float> logits;
      for (const Json& e : step["entries"].array()) {
        const std::string& id = e["id"].string();
        if (live.count(id) == 0) live[id] = model->begin();
        std::vector<int64_t> tokens;
        std::vector<int32_t> want;
        for (const Json& t : e["tokens"].array()) tokens.push_back(t.integer());
        for (const Json& w : e["want"].array()) want.push_back(static_cast<int32_t>(w.integer()));
        const size_t at = logits.size();
        logits.resize(at + want.size() * static_cast<size_t>(model->vocab()));
        model->forward(live[id], tokens, want, logits.data() + at);
      }
      if (!logits.empty()) {
        const std::string path = out_dir + "/" + std::to_string(number) + ".f32";
        std::FILE* f = std::fopen(path.c_str(), "wb");
        if (!f || std::fwrite(logits.data(), sizeof(float), logits.size(), f) != logits.size() || std::fclose(f) != 0) {
          MLLM_ERROR_EXIT(kError, "cannot write {}", path);
        }
      }
      if (step.has("end")) {
        for (const Json& e : step["end"].array()) {
          auto it = live.find(e.string());
          if (it == live.end()) { MLLM_ERROR_EXIT(kError, "request {} is not live", e.string()); }
          model->end(it->second);
          live.erase(it);
        }
      }
      std::printf("done %lld\n", static_cast<long long>(number));
      std::fflush(stdout);
    }
  }
  ctx.shutdown();
  return 0;
}
