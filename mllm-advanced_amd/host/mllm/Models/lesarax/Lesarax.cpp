// Lesarax: configuration and parameter names -> the layered decoder.
//
// config.json: vocab, width, norm.eps, residual_mult, loop {start, stop, times}, and "layers", a list of {type, mixer, mlp}:
//   attention         mixer {heads, kv_heads, dim, vdim, scale, rot {dims, base}}; the values are the keys before rotation
//   latent_attention  mixer {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, mask {size}, rot {dims, base}}
//   mlp               null, or {kind "moe", expert {ff, limit}, router {experts, top}}
// Parameters: embed (the head as well), final.norm, loop.in; l<i>.norm1 / norm2; l<i>.mix.* ; l<i>.mlp.router,
// l<i>.mlp.e<j>.gate / up / down.
#include <string>

#include "mllm/Engine/Safetensors.hpp"
#include "mllm/Models/layered/HipLayered.hpp"
#include "mllm/Utils/Log.hpp"

namespace mllm::models {

namespace {

w4a32_layer_config layerConfig(const Json& j) {
  const std::string& type = j["type"].string();
  const Json& m = j["mixer"];
  auto num = [&](const char* key) { return static_cast<int>(m[key].integer()); };
  w4a32_layer_config l{};
  l.heads = num("heads");
  l.kv_heads = m.has("kv_heads") ? num("kv_heads") : l.heads;
  l.dim = num("dim");
  l.vdim = num("vdim");
  l.scale = static_cast<float>(m["scale"].number());
  l.kv_from = -1;
  if (m.has("mask")) l.window = static_cast<int>(m["mask"]["size"].integer());
  if (m.has("rot")) {
    l.rot_dims = static_cast<int>(m["rot"]["dims"].integer());
    l.rot_base = m["rot"]["base"].number();
  }
  if (type == "attention") {
    l.mixer = W4A32_MIX_ROTARY;
    l.tied_values = 1;
  } else if (type == "latent_attention") {
    l.mixer = W4A32_MIX_LATENT;
    l.q_rank = num("q_rank");
    l.kv_rank = num("kv_rank");
    l.rot_part = num("rot_dim");
    l.head_gate = 1;
  } else {
    MLLM_ERROR_EXIT(kError, "config.json: no mixer of type \"{}\"", type);
  }
  if (j.has("mlp")) {
    const Json& f = j["mlp"];
    const std::string& kind = f["kind"].string();
    if (kind != "moe") { MLLM_ERROR_EXIT(kError, "config.json: no feed-forward of kind \"{}\"", kind); }
    l.ff = static_cast<int>(f["expert"]["ff"].integer());
    l.expert_limit = static_cast<float>(f["expert"]["limit"].number());
    l.experts = static_cast<int>(f["router"]["experts"].integer());
    l.top = static_cast<int>(f["router"]["top"].integer());
    if (l.ff <= 0 || l.experts <= 0) { MLLM_ERROR_EXIT(kError, "config.json: {} experts of width {}", l.experts, l.ff); }
  }
  return l;
}

std::unique_ptr<CausalLM> load(const std::string& dir, const Json& config, const CausalLMOptions& options) {
  LayeredSpec spec;
  spec.hidden = static_cast<int32_t>(config["width"].integer());
  spec.vocab = static_cast<int32_t>(config["vocab"].integer());
  spec.canon_taps = 0;
  spec.norm = W4A32_NORM_RMS;
  spec.norm_eps = static_cast<float>(config["norm"]["eps"].number());
  spec.residual_mult = static_cast<float>(config["residual_mult"].number());
  if (config.has("loop")) {
    spec.loop_start = static_cast<int32_t>(config["loop"]["start"].integer());
    spec.loop_stop = static_cast<int32_t>(config["loop"]["stop"].integer());
    spec.loop_times = static_cast<int32_t>(config["loop"]["times"].integer());
  }
  spec.dtype = options.dtype == "float32" ? W4A32_LAYERED_F32 : W4A32_LAYERED_BF16;
  for (const Json& j : config["layers"].array()) spec.layers.push_back(layerConfig(j));

  auto model = std::make_unique<HipLayeredForCausalLM>(spec, options);
  auto w = std::make_shared<LayeredWeights>(loadSafetensors(dir + "/model.safetensors"), spec.dtype);
  const int W = spec.hidden;
  std::vector<w4a32_layered_layer> layers;
  for (size_t i = 0; i < spec.layers.size(); ++i) {
    const w4a32_layer_config& l = spec.layers[i];
    const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.";
    w4a32_layered_layer lw{};
    lw.norm1 = w->vector(p + "norm1", W);
    lw.sinks = w->vector(m + "sink", l.heads);
    if (l.mixer == W4A32_MIX_ROTARY) {
      lw.in_proj = w->matrix({{m + "q", l.heads * l.dim}, {m + "k", l.kv_heads * l.dim}}, W);
    } else {
      lw.in_proj = w->matrix({{m + "dq", l.q_rank}, {m + "dkv", l.kv_rank + l.rot_part}, {m + "g", l.heads}}, W);
      lw.q_norm = w->vector(m + "dq.norm", l.q_rank);
      lw.kv_norm = w->vector(m + "dkv.norm", l.kv_rank);
      lw.q_up = w->matrix({{m + "uq", l.heads * (l.dim + l.rot_part)}}, l.q_rank);
      const int rows = w4a32_layered_head_rows(l.dim, l.vdim);
      lw.k_up = w->operandBlocks(m + "uk", l.heads, l.dim, rows, l.kv_rank);
      lw.v_up = w->operandBlocks(m + "uv", l.heads, l.vdim, rows, l.kv_rank);
    }
    lw.out_proj = w->matrix({{m + "o", W}}, l.heads * l.vdim);
    if (l.ff > 0) {
      lw.norm2 = w->vector(p + "norm2", W);
      lw.router = w->matrix({{p + "mlp.router", l.experts}}, W);
      std::vector<std::pair<std::string, std::string>> gate_up;
      std::vector<std::string> down;
      for (int e = 0; e < l.experts; ++e) {
        const std::string q = p + "mlp.e" + std::to_string(e) + ".";
        gate_up.emplace_back(q + "gate", q + "up");
        down.push_back(q + "down");
      }
      lw.gate_up = w->gateUp(gate_up, l.ff, W);
      lw.experts_down = w->stack(down, W, l.ff);
    }
    layers.push_back(lw);
  }
  w4a32_layered_weights top{};
  top.embedding = top.head = w->matrix({{"embed", spec.vocab}}, W, false);
  top.final_norm = w->vector("final.norm", W);
  if (spec.loop_times > 0) top.loop_in = w->halves("loop.in", W, W);
  model->setWeights(top, std::move(layers), w);
  return model;
}

}  // namespace

void registerLesarax(CausalLMRegistry& r) { r.reg("Lesarax", load); }

}  // namespace mllm::models
