// What a program needs of a language model, whatever its design: sequences, logits at chosen positions, greedy
// generation; and the registry that picks the model class by a folder's config.json. (The reference selects a model at
// compile time, one example program per model: examples/Models/DeepSeekDistillQwen2/demo_ds_qwen2.cpp; its
// generation loop is mllm/Models/AutoLLM.hpp:40-105.)
#pragma once

#include <cstdint>
#include <functional>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "mllm/Utils/Json.hpp"

namespace mllm::models {

struct CausalLMOptions {
  std::string dtype = "bfloat16";  // "bfloat16" or "float32"; a family with one format of its own ignores it
  int32_t max_tokens = 4096;       // most tokens one sequence holds
  int32_t max_chunk = 2048;        // longest slice of a prompt one call runs
};

class CausalLM {
 public:
  virtual ~CausalLM() = default;
  [[nodiscard]] virtual int32_t vocab() const = 0;

  // A sequence starts empty; end() gives back what it holds.
  virtual int32_t begin() = 0;
  virtual void end(int32_t seq) = 0;

  // Appends tokens to a sequence. logits [want.size()][vocab] receives the logits behind the tokens at the places
  // `want` (indices into `tokens`, ascending).
  virtual void forward(int32_t seq, const std::vector<int64_t>& tokens, const std::vector<int32_t>& want,
                       float* logits) = 0;

  // Greedy continuation of a prompt in a sequence of its own: at most max_new tokens, ends behind eos (eos < 0: never).
  virtual std::vector<int64_t> generate(const std::vector<int64_t>& prompt, int32_t max_new, int64_t eos) = 0;
};

class CausalLMRegistry {
 public:
  // `dir` holds config.json (already read) and the parameters
  using Factory =
      std::function<std::unique_ptr<CausalLM>(const std::string& dir, const Json& config, const CausalLMOptions&)>;

  static CausalLMRegistry& instance() {
    static CausalLMRegistry r;
    return r;
  }
  void reg(const std::string& architecture, Factory f) { factories_[architecture] = std::move(f); }
  // Reads dir/config.json; the key is its "architecture", or the first of its "architectures".
  std::unique_ptr<CausalLM> load(const std::string& dir, const CausalLMOptions& options) const;

 private:
  std::map<std::string, Factory> factories_;
};

// Model families register themselves by calling these (explicitly: a program links the families it names).
void registerSuripel(CausalLMRegistry& r);
void registerLesarax(CausalLMRegistry& r);
void registerQwen2(CausalLMRegistry& r);

}  // namespace mllm::models
