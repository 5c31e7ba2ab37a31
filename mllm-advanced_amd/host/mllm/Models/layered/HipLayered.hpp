// A decoder-only model whose layers are described one by one, on the layered decoder runner
// (include/w4a32_layered.h). The class owns the device memory (weights, workspace, one state per sequence) and the
// captured decode step; a design's own file (mllm/Models/suripel, mllm/Models/lesarax) reads its configuration and
// parameter names and fills in the specification and the weights through LayeredWeights.
#pragma once

#include <cstdint>
#include <map>
#include <memory>
#include <string>
#include <utility>
#include <vector>

#include "mllm/Core/Tensor.hpp"
#include "mllm/Engine/ParameterReader.hpp"
#include "mllm/Models/CausalLM.hpp"
#include "w4a32_layered.h"

namespace mllm::models {

struct LayeredSpec {
  int32_t hidden = 0, vocab = 0, canon_taps = 1;
  float norm_eps = 1e-5f;
  int dtype = W4A32_LAYERED_BF16;
  std::vector<w4a32_layer_config> layers;
  int norm = W4A32_NORM_LAYER;
  float residual_mult = 1.0f;
  int32_t loop_start = 0, loop_stop = 0, loop_times = 0;
};

// Host parameters (BF16, Fp16 or Fp32) -> device memory in the runner's layouts. Every tensor's shape is checked
// against what the caller expects; padding is zero.
class LayeredWeights {
 public:
  LayeredWeights(const std::shared_ptr<ParameterLoader>& file, int dtype) : file_(file), dtype_(dtype) {}

  struct Part {
    std::string name;
    int32_t rows;
  };
  // [out, in] matrices one below the other, in the model's element type. pad_rows: rows to a multiple of 64 as well.
  const void* matrix(const std::vector<Part>& parts, int32_t in, bool pad_rows = true);
  // [heads * n, in] as operand blocks (w4a32_layered.h): head_rows rows per head, the true ones first
  const void* operandBlocks(const std::string& name, int32_t heads, int32_t n, int32_t head_rows, int32_t in);
  // experts' gate and up [ff, in], one pair of names per expert, in groups of 32 rows of each
  const void* gateUp(const std::vector<std::pair<std::string, std::string>>& experts, int32_t ff, int32_t in);
  // equal matrices [out, in] one behind the other, each padded by itself
  const void* stack(const std::vector<std::string>& names, int32_t out, int32_t in);
  // [out, 2 in] whose two column halves are padded each
  const void* halves(const std::string& name, int32_t out, int32_t in);
  // a vector, f32
  const float* vector(const std::string& name, int32_t n);
  const float* values(const std::vector<float>& v);
  // [channels, taps] convolutions one below the other, f32, transposed to [taps][channels]
  const float* conv(const std::vector<Part>& parts, int32_t taps);

 private:
  Tensor host(const std::string& name, const std::vector<int32_t>& shape);
  const void* upload(const std::vector<uint8_t>& bytes);
  [[nodiscard]] size_t elem() const { return dtype_ == W4A32_LAYERED_BF16 ? 2 : 4; }
  // n elements from element `src` of t on, in the model's element type
  void copy(uint8_t* dst, const Tensor& t, size_t src, int32_t n) const;

  std::shared_ptr<ParameterLoader> file_;
  int dtype_;
  std::vector<Tensor> keep_;
};

class HipLayeredForCausalLM final : public CausalLM {
 public:
  HipLayeredForCausalLM(const LayeredSpec& spec, const CausalLMOptions& options);
  ~HipLayeredForCausalLM() override;

  // Between construction and first use: the weights (pointers into device memory `keep` holds).
  void setWeights(const w4a32_layered_weights& top, std::vector<w4a32_layered_layer> layers,
                  std::shared_ptr<LayeredWeights> keep);

  [[nodiscard]] int32_t vocab() const override { return cfg_.vocab; }
  int32_t begin() override;
  void end(int32_t seq) override;
  void forward(int32_t seq, const std::vector<int64_t>& tokens, const std::vector<int32_t>& want,
               float* logits) override;
  std::vector<int64_t> generate(const std::vector<int64_t>& prompt, int32_t max_new, int64_t eos) override;

 private:
  struct Sequence;
  Sequence& sequence(int32_t seq);
  void slice(Sequence& s, const int64_t* tokens, int32_t n, const int32_t* want, int32_t n_want, float* logits);

  std::vector<w4a32_layer_config> layer_cfg_;
  w4a32_layered_config cfg_{};
  std::vector<w4a32_layered_layer> layer_weights_;
  w4a32_layered_weights weights_{};
  std::shared_ptr<LayeredWeights> keep_;
  Tensor workspace_, ids_, want_, logits_, token_;
  std::map<int32_t, std::unique_ptr<Sequence>> live_;
  std::vector<std::unique_ptr<Sequence>> idle_;  // states of ended sequences, used again
  int32_t next_id_ = 0;
};

}  // namespace mllm::models
