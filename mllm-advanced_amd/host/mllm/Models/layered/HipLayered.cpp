#include "mllm/Models/layered/HipLayered.hpp"

#include <hip/hip_runtime_api.h>

#include <algorithm>
#include <cstring>

#include "mllm/Backends/HIP/HipBackend.hpp"
#include "mllm/Utils/Log.hpp"

namespace mllm::models {

namespace {

void check(int rc, const char* what) {
  if (rc != W4A32_OK) { MLLM_ERROR_EXIT(hip::kHipRuntimeError, "{} failed: {}", what, w4a32_error_string(rc)); }
}

void checkHip(hipError_t e, const char* what) {
  if (e != hipSuccess) { MLLM_ERROR_EXIT(hip::kHipRuntimeError, "{} failed: {}", what, hipGetErrorString(e)); }
}

hipStream_t stream() { return static_cast<hipStream_t>(hip::currentHipBackend().stream()); }

int32_t pad64(int32_t n) { return (n + W4A32_LAYERED_PAD - 1) / W4A32_LAYERED_PAD * W4A32_LAYERED_PAD; }

float halfToFloat(uint16_t h) {
  const uint32_t sign = (h & 0x8000u) << 16, exp = (h >> 10) & 31u, man = h & 0x3FFu;
  float f;
  if (exp == 0) {
    f = static_cast<float>(man) * 5.9604644775390625e-08f;  // 2^-24
    return sign ? -f : f;
  }
  const uint32_t bits = sign | ((exp == 31 ? 255u : exp + 112u) << 23) | (man << 13);
  std::memcpy(&f, &bits, 4);
  return f;
}

float elementAsFloat(const Tensor& t, size_t i) {
  if (t.dtype() == kFp32) return t.ptr<float>()[i];
  if (t.dtype() == kFp16) return halfToFloat(t.ptr<uint16_t>()[i]);
  const uint32_t bits = static_cast<uint32_t>(t.ptr<uint16_t>()[i]) << 16;
  float f;
  std::memcpy(&f, &bits, 4);
  return f;
}

uint16_t floatToBf16(float f) {  // to nearest even
  uint32_t u;
  std::memcpy(&u, &f, 4);
  if ((u & 0x7FFFFFFFu) > 0x7F800000u) return static_cast<uint16_t>((u >> 16) | 0x40u);
  return static_cast<uint16_t>((u + 0x7FFFu + ((u >> 16) & 1u)) >> 16);
}

// device memory in 8-byte elements (a tensor dimension is an int32)
Tensor deviceBytes(size_t bytes) {
  const size_t words = (std::max<size_t>(bytes, 8) + 7) / 8;
  if (words > 0x7FFFFFFFull) { MLLM_ERROR_EXIT(kMemory, "{} bytes exceed one tensor", bytes); }
  return Tensor::empty({static_cast<int32_t>(words)}, kInt64, kHIP).alloc();
}

}  // namespace

// ---------------------------------------------------------------------------- weights
Tensor LayeredWeights::host(const std::string& name, const std::vector<int32_t>& shape) {
  Tensor t((*file_)[name]);
  if (t.dtype() != kBF16 && t.dtype() != kFp16 && t.dtype() != kFp32) {
    MLLM_ERROR_EXIT(kError, "{}: expected BF16, Fp16 or Fp32 values, got {}", name, dataTypes2Str(t.dtype()));
  }
  if (t.shape() != shape) {
    std::string want, got;
    for (auto d : shape) want += " " + std::to_string(d);
    for (auto d : t.shape()) got += " " + std::to_string(d);
    MLLM_ERROR_EXIT(kError, "{}: the configuration asks for shape [{} ], the file has [{} ]", name, want, got);
  }
  return t;
}

const void* LayeredWeights::upload(const std::vector<uint8_t>& bytes) {
  Tensor d = deviceBytes(bytes.size());
  checkHip(hipMemcpyAsync(d.ptr<void>(), bytes.data(), bytes.size(), hipMemcpyHostToDevice, stream()),
           "hipMemcpyAsync(parameter)");
  hip::currentHipBackend().synchronize();  // `bytes` goes away
  keep_.push_back(d);
  return d.ptr<void>();
}

void LayeredWeights::copy(uint8_t* dst, const Tensor& t, size_t src, int32_t n) const {
  if (dtype_ == W4A32_LAYERED_BF16) {
    auto* d = reinterpret_cast<uint16_t*>(dst);
    if (t.dtype() == kBF16) {
      std::memcpy(d, t.ptr<uint16_t>() + src, static_cast<size_t>(n) * 2);
    } else {
      for (int32_t c = 0; c < n; ++c) d[c] = floatToBf16(elementAsFloat(t, src + c));
    }
  } else {
    for (int32_t c = 0; c < n; ++c) reinterpret_cast<float*>(dst)[c] = elementAsFloat(t, src + c);
  }
}

const void* LayeredWeights::matrix(const std::vector<Part>& parts, int32_t in, bool pad_rows) {
  int32_t rows = 0;
  for (const auto& p : parts) rows += p.rows;
  const size_t row = pad64(in) * elem();
  std::vector<uint8_t> buf((pad_rows ? pad64(rows) : rows) * row, 0);
  size_t at = 0;
  for (const auto& p : parts) {
    Tensor t = host(p.name, {p.rows, in});
    for (int32_t r = 0; r < p.rows; ++r, ++at) copy(buf.data() + at * row, t, static_cast<size_t>(r) * in, in);
  }
  return upload(buf);
}

const void* LayeredWeights::operandBlocks(const std::string& name, int32_t heads, int32_t n, int32_t head_rows, int32_t in) {
  const size_t ld = pad64(in);
  std::vector<uint8_t> buf(static_cast<size_t>(heads) * head_rows * ld * elem(), 0);
  Tensor t = host(name, {heads * n, in});
  for (int32_t h = 0; h < heads; ++h)
    for (int32_t i = 0; i < n; ++i) {
      const size_t r = static_cast<size_t>(h) * head_rows + i;
      for (int32_t c = 0; c < in; c += 8) {
        const size_t at = ((r / 32 * (ld / 8) + c / 8) * 32 + r % 32) * 8;
        copy(buf.data() + at * elem(), t, (static_cast<size_t>(h) * n + i) * in + c, std::min(8, in - c));
      }
    }
  return upload(buf);
}

const void* LayeredWeights::gateUp(const std::vector<std::pair<std::string, std::string>>& experts, int32_t ff, int32_t in) {
  const size_t row = pad64(in) * elem(), rows = 2 * pad64(ff);
  std::vector<uint8_t> buf(experts.size() * rows * row, 0);
  for (size_t e = 0; e < experts.size(); ++e) {
    Tensor gate = host(experts[e].first, {ff, in}), up = host(experts[e].second, {ff, in});
    for (int32_t r = 0; r < ff; ++r) {
      uint8_t* dst = buf.data() + (e * rows + r / 32 * 64 + r % 32) * row;
      copy(dst, gate, static_cast<size_t>(r) * in, in);
      copy(dst + 32 * row, up, static_cast<size_t>(r) * in, in);
    }
  }
  return upload(buf);
}

const void* LayeredWeights::stack(const std::vector<std::string>& names, int32_t out, int32_t in) {
  const size_t row = pad64(in) * elem(), rows = pad64(out);
  std::vector<uint8_t> buf(names.size() * rows * row, 0);
  for (size_t e = 0; e < names.size(); ++e) {
    Tensor t = host(names[e], {out, in});
    for (int32_t r = 0; r < out; ++r) copy(buf.data() + (e * rows + r) * row, t, static_cast<size_t>(r) * in, in);
  }
  return upload(buf);
}

const void* LayeredWeights::halves(const std::string& name, int32_t out, int32_t in) {
  const size_t half = pad64(in) * elem();
  std::vector<uint8_t> buf(pad64(out) * 2 * half, 0);
  Tensor t = host(name, {out, 2 * in});
  for (int32_t r = 0; r < out; ++r)
    for (int32_t i = 0; i < 2; ++i)
      copy(buf.data() + (2 * static_cast<size_t>(r) + i) * half, t, (2 * static_cast<size_t>(r) + i) * in, in);
  return upload(buf);
}

const float* LayeredWeights::vector(const std::string& name, int32_t n) {
  Tensor t = host(name, {n});
  std::vector<float> v(n);
  for (int32_t i = 0; i < n; ++i) v[i] = elementAsFloat(t, i);
  return values(v);
}

const float* LayeredWeights::values(const std::vector<float>& v) {
  std::vector<uint8_t> buf(sizeof(float) * pad64(static_cast<int32_t>(v.size())), 0);
  std::memcpy(buf.data(), v.data(), sizeof(float) * v.size());
  return static_cast<const float*>(upload(buf));
}

const float* LayeredWeights::conv(const std::vector<Part>& parts, int32_t taps) {
  int32_t rows = 0;
  for (const auto& p : parts) rows += p.rows;
  const size_t ld = pad64(rows);
  std::vector<uint8_t> buf(sizeof(float) * ld * taps, 0);
  auto* f = reinterpret_cast<float*>(buf.data());
  size_t at = 0;
  for (const auto& p : parts) {
    Tensor t = host(p.name, {p.rows, taps});
    for (int32_t r = 0; r < p.rows; ++r, ++at)
      for (int32_t j = 0; j < taps; ++j) f[j * ld + at] = elementAsFloat(t, static_cast<size_t>(r) * taps + j);
  }
  return static_cast<const float*>(upload(buf));
}

// ---------------------------------------------------------------------------- sequences
struct HipLayeredForCausalLM::Sequence {
  Tensor state;
  int32_t position = 0;
  // the decode step on this state, recorded at its second use (the first one runs eagerly and brings the kernels'
  // code objects in, which must not happen inside a capture)
  bool warmed = false;
  hipGraph_t graph = nullptr;
  hipGraphExec_t exec = nullptr;
  ~Sequence() {
    if (exec) (void)hipGraphExecDestroy(exec);
    if (graph) (void)hipGraphDestroy(graph);
  }
};

HipLayeredForCausalLM::HipLayeredForCausalLM(const LayeredSpec& spec, const CausalLMOptions& options)
    : layer_cfg_(spec.layers) {
  cfg_.hidden = spec.hidden;
  cfg_.vocab = spec.vocab;
  cfg_.n_layers = static_cast<int>(layer_cfg_.size());
  cfg_.canon_taps = spec.canon_taps;
  cfg_.norm_eps = spec.norm_eps;
  cfg_.dtype = spec.dtype;
  cfg_.norm = spec.norm;
  cfg_.residual_mult = spec.residual_mult;
  cfg_.loop_start = spec.loop_start;
  cfg_.loop_stop = spec.loop_stop;
  cfg_.loop_times = spec.loop_times;
  cfg_.max_seq = std::max(options.max_tokens, 1);
  cfg_.max_batch_tokens = std::max(1, std::min(options.max_chunk, cfg_.max_seq));
  cfg_.layers = layer_cfg_.data();
  const int rc = w4a32_layered_check(&cfg_);
  if (rc != W4A32_OK) {
    MLLM_ERROR_EXIT(kError, "this build cannot run the configuration: {}", w4a32_error_string(rc));
  }
  auto& hb = hip::currentHipBackend();
  workspace_ = deviceBytes(w4a32_layered_workspace_bytes(&cfg_));
  ids_ = Tensor::empty({cfg_.max_batch_tokens}, kInt64, kHIP).alloc();
  want_ = Tensor::empty({cfg_.max_batch_tokens}, kInt32, kHIP).alloc();
  token_ = Tensor::empty({1}, kInt64, kHIP).alloc();
  check(w4a32_layered_init_workspace(&cfg_, workspace_.ptr<void>(), hb.stream()), "w4a32_layered_init_workspace");
  hb.synchronize();
}

HipLayeredForCausalLM::~HipLayeredForCausalLM() = default;

void HipLayeredForCausalLM::setWeights(const w4a32_layered_weights& top, std::vector<w4a32_layered_layer> layers,
                                       std::shared_ptr<LayeredWeights> keep) {
  layer_weights_ = std::move(layers);
  weights_ = top;
  weights_.layers = layer_weights_.data();
  keep_ = std::move(keep);
}

HipLayeredForCausalLM::Sequence& HipLayeredForCausalLM::sequence(int32_t seq) {
  auto it = live_.find(seq);
  if (it == live_.end()) { MLLM_ERROR_EXIT(kError, "no sequence {}", seq); }
  return *it->second;
}

int32_t HipLayeredForCausalLM::begin() {
  std::unique_ptr<Sequence> s;
  if (!idle_.empty()) {
    s = std::move(idle_.back());
    idle_.pop_back();
  } else {
    s = std::make_unique<Sequence>();
    s->state = deviceBytes(w4a32_layered_state_bytes(&cfg_));
    auto& hb = hip::currentHipBackend();
    check(w4a32_layered_init_state(&cfg_, s->state.ptr<void>(), hb.stream()), "w4a32_layered_init_state");
  }
  s->position = 0;
  const int32_t id = next_id_++;
  live_[id] = std::move(s);
  return id;
}

void HipLayeredForCausalLM::end(int32_t seq) {
  sequence(seq);
  idle_.push_back(std::move(live_[seq]));
  live_.erase(seq);
}

void HipLayeredForCausalLM::slice(Sequence& s, const int64_t* tokens, int32_t n, const int32_t* want, int32_t n_want,
                                  float* logits) {
  auto st = stream();
  checkHip(hipMemcpyAsync(ids_.ptr<void>(), tokens, sizeof(int64_t) * n, hipMemcpyHostToDevice, st),
           "hipMemcpyAsync(tokens)");
  const size_t floats = static_cast<size_t>(n_want) * cfg_.vocab;
  if (n_want > 0) {
    checkHip(hipMemcpyAsync(want_.ptr<void>(), want, sizeof(int32_t) * n_want, hipMemcpyHostToDevice, st),
             "hipMemcpyAsync(want)");
    if (logits_.isNil() || hip::tensorBytes(logits_) < floats * sizeof(float)) logits_ = deviceBytes(floats * sizeof(float));
  }
  check(w4a32_layered_forward(&cfg_, &weights_, s.state.ptr<void>(), workspace_.ptr<void>(), ids_.ptr<int64_t>(), n,
                              s.position, n_want > 0 ? want_.ptr<int>() : nullptr, n_want,
                              n_want > 0 ? logits_.ptr<float>() : nullptr, 0, st),
        "w4a32_layered_forward");
  s.position += n;
  if (n_want > 0) {
    checkHip(hipMemcpyAsync(logits, logits_.ptr<void>(), floats * sizeof(float), hipMemcpyDeviceToHost, st),
             "hipMemcpyAsync(logits)");
  }
  hip::currentHipBackend().synchronize();  // the host vectors may go away
}

void HipLayeredForCausalLM::forward(int32_t seq, const std::vector<int64_t>& tokens, const std::vector<int32_t>& want,
                                    float* logits) {
  Sequence& s = sequence(seq);
  const auto total = static_cast<int32_t>(tokens.size());
  if (total == 0) { MLLM_ERROR_EXIT(kError, "forward: no tokens"); }
  if (total > cfg_.max_seq - s.position) {
    MLLM_ERROR_EXIT(kError, "forward: {} tokens at position {} exceed the {} a sequence holds", total, s.position,
                    cfg_.max_seq);
  }
  size_t w = 0;
  for (int32_t done = 0; done < total;) {
    const int32_t n = std::min(cfg_.max_batch_tokens, total - done);
    std::vector<int32_t> here;
    const size_t first = w;
    for (; w < want.size() && want[w] < done + n; ++w) {
      if (want[w] < done) { MLLM_ERROR_EXIT(kError, "forward: wanted places must ascend"); }
      here.push_back(want[w] - done);
    }
    slice(s, tokens.data() + done, n, here.data(), static_cast<int32_t>(here.size()),
          logits ? logits + first * static_cast<size_t>(cfg_.vocab) : nullptr);
    done += n;
  }
  if (w != want.size()) { MLLM_ERROR_EXIT(kError, "forward: a wanted place lies past the tokens"); }
}

std::vector<int64_t> HipLayeredForCausalLM::generate(const std::vector<int64_t>& prompt, int32_t max_new, int64_t eos) {
  std::vector<int64_t> out;
  if (max_new <= 0) return out;
  const int32_t id = begin();
  Sequence& s = sequence(id);
  const auto total = static_cast<int32_t>(prompt.size());
  if (total == 0 || total > cfg_.max_seq) {
    MLLM_ERROR_EXIT(kError, "generate: a prompt of {} tokens (a sequence holds {})", total, cfg_.max_seq);
  }
  auto st = stream();
  auto& hb = hip::currentHipBackend();
  for (int32_t done = 0; done < total;) {
    const int32_t n = std::min(cfg_.max_batch_tokens, total - done);
    checkHip(hipMemcpyAsync(ids_.ptr<void>(), prompt.data() + done, sizeof(int64_t) * n, hipMemcpyHostToDevice, st),
             "hipMemcpyAsync(tokens)");
    check(w4a32_layered_prefill(&cfg_, &weights_, s.state.ptr<void>(), workspace_.ptr<void>(), ids_.ptr<int64_t>(), n,
                                s.position, token_.ptr<int64_t>(), st),
          "w4a32_layered_prefill");
    s.position += n;
    done += n;
  }
  auto step = [&] {
    return w4a32_layered_step(&cfg_, &weights_, s.state.ptr<void>(), workspace_.ptr<void>(), token_.ptr<int64_t>(),
                              token_.ptr<int64_t>(), st);
  };
  for (;;) {
    int64_t next = 0;
    checkHip(hipMemcpyAsync(&next, token_.ptr<void>(), sizeof(next), hipMemcpyDeviceToHost, st), "hipMemcpyAsync(token)");
    hb.synchronize();
    out.push_back(next);
    if (next == eos || static_cast<int32_t>(out.size()) >= max_new || s.position >= cfg_.max_seq) break;
    if (!s.warmed) {
      check(step(), "w4a32_layered_step");
      s.warmed = true;
    } else {
      if (!s.exec) {
        checkHip(hipStreamBeginCapture(st, hipStreamCaptureModeThreadLocal), "hipStreamBeginCapture");
        const int rc = step();
        checkHip(hipStreamEndCapture(st, &s.graph), "hipStreamEndCapture");
        check(rc, "w4a32_layered_step");
        checkHip(hipGraphInstantiate(&s.exec, s.graph, nullptr, nullptr, 0), "hipGraphInstantiate");
      }
      checkHip(hipGraphLaunch(s.exec, st), "hipGraphLaunch");
    }
    ++s.position;
  }
  end(id);
  return out;
}

}  // namespace mllm::models
