// extern "C" surface of include/w4a32_layered.h: configuration checks, memory geometry and launch order of the
// layered decoder. Host code only.
//
// A prefill layer:  [add + norm + input convolution] [in_proj] mixer [out_proj] [add + norm + input convolution] [up]
//                   [PolyNorm] [down];  mixer = [convolution or rotation + cache append] [block means] [attention], or
//                   [convolution] [chunks] [scan] [output] (retention: without the first), or
//                   [norms + cache append] [q_up] [expand] [attention];
//                   a mixture of experts instead of the last three: [router] [choose] [plan] [gate, up] [down]
// A decode layer:   [add + norm + input convolution + in_proj] [mixer step] [merge or head norm + gate + out_proj]
//                   [add + norm + input convolution + up] [PolyNorm + down]
//                   latent mixer: [norm + q_up] [cache append, query folded] [attention] [merge + values + gate] [out_proj]
//                   mixture of experts: [add + norm + router] [norm + choice + gate, up] [down]
// In front of a pass through looped layers: [add + loop_in].
#include "w4a32_layered.h"

#include <algorithm>
#include <cstring>
#include <vector>

#include "w4a32_layered_kernels.h"

namespace {

using w4::pad64;

inline int from_hip(hipError_t e) { return e == hipSuccess ? W4A32_OK : W4A32_ELAUNCH; }
inline hipStream_t S(void* stream) { return static_cast<hipStream_t>(stream); }
inline size_t align_up(size_t v, size_t a) { return (v + a - 1) / a * a; }

#define W4_TRY(expr)                 \
  do {                               \
    const int rc_ = (expr);          \
    if (rc_ != W4A32_OK) return rc_; \
  } while (0)
#define W4_LAUNCH(expr) W4_TRY(from_hip(expr))

constexpr int kArgmaxParts = 4096;
constexpr size_t kSplitFloats = (size_t)768 * 128 * 128;  // what a product split over k leaves at most (fewer than
                                                          // 768 tiles of 128 x 128, or 1536 of 64 x 64)

struct LayerGeom {
  int rows;         // rows of in_proj
  int conv_rows;    // ... of which pass the short convolution
  int mix;          // heads * vdim
  int D, dv16;
  int src, pool_owner;  // attention: whose keys and values, whose block means (runs)
  int rot;              // index of the rotation table, -1: none
  int q_rows;           // latent: heads * (dim + rot_part)
  int Dc, Dr;           // latent: kv_rank and rot_part, padded
};

// One run of a layer; looped layers run several times, each time on caches of their own.
struct LayerRun {
  int layer;
  bool pass_starts;  // the looped part's input product comes first
};

std::vector<LayerRun> layer_runs(const w4a32_layered_config* c) {
  std::vector<LayerRun> r;
  const bool loop = c->loop_times > 0;
  for (int i = 0; i < (loop ? c->loop_start : c->n_layers); ++i) r.push_back({i, false});
  if (!loop) return r;
  for (int t = 0; t < c->loop_times; ++t)
    for (int i = c->loop_start; i < c->loop_stop; ++i) r.push_back({i, i == c->loop_start});
  for (int i = c->loop_stop; i < c->n_layers; ++i) r.push_back({i, false});
  return r;
}

struct RotTable {
  int dims;
  double base;
  size_t sin_off, cos_off;
};

struct Geom {
  int Hp, elem;
  std::vector<LayerRun> runs;
  std::vector<LayerGeom> layers;  // per run, as `st`
  std::vector<RotTable> rot;
  // state
  struct LayerState {
    size_t canon1, canon2, conv, k, vt, kp, vpt, rec;
    int cap, capp;
  };
  std::vector<LayerState> st;
  size_t state_bytes;
  // workspace
  size_t x[2], y, raw, cx, q, mix, parts, ff, z, o, ml, amax_v, amax_i, logits, last, rec, ws_bytes;
  size_t cq, ke, ve, qa, head_out, router, moe, sel;  // latent attention, mixture of experts
  std::vector<int> expand_blk;                        // per run: blocks of keys the expansion has room for
};

w4::MoeGeom moe_geom(const w4a32_layered_config* c, const w4a32_layer_config& l) {
  return {c->hidden, pad64(c->hidden), l.ff, pad64(l.ff), l.experts, l.top, l.expert_limit};
}

int check_config(const w4a32_layered_config* c) {
  if (!c || !c->layers) return W4A32_EINVAL;
  if (c->hidden <= 0 || c->vocab <= 0 || c->n_layers <= 0 || c->max_seq <= 0 || c->max_batch_tokens <= 0)
    return W4A32_EINVAL;
  if (c->dtype != W4A32_LAYERED_BF16 && c->dtype != W4A32_LAYERED_F32) return W4A32_EINVAL;
  if (c->norm != W4A32_NORM_LAYER && c->norm != W4A32_NORM_RMS) return W4A32_EINVAL;
  if (c->canon_taps < (c->norm == W4A32_NORM_RMS ? 0 : 1) || !(c->norm_eps >= 0.0f)) return W4A32_EINVAL;
  if (c->loop_times < 0) return W4A32_EINVAL;
  if (c->loop_times > 0) {
    if (c->loop_start < 0 || c->loop_stop <= c->loop_start || c->loop_stop > c->n_layers) return W4A32_ESHAPE;
    if (!w4::row_linear_fits(2 * pad64(c->hidden))) return W4A32_ENOTSUP;
  }
  if (c->canon_taps > W4A32_LAYERED_MAX_TAPS) return W4A32_ENOTSUP;
  const int Hp = pad64(c->hidden);
  if (!w4::norm_conv_fits(Hp, c->canon_taps) || !w4::row_linear_fits(Hp)) return W4A32_ENOTSUP;
  for (int i = 0; i < c->n_layers; ++i) {
    const w4a32_layer_config& l = c->layers[i];
    if (l.heads <= 0 || l.kv_heads <= 0 || l.dim <= 0 || l.vdim <= 0 || l.ff < 0) return W4A32_EINVAL;
    if (l.heads % l.kv_heads != 0) return W4A32_ESHAPE;
    if (std::max(l.dim, l.vdim) > W4A32_LAYERED_MAX_DIM || l.conv_taps > W4A32_LAYERED_MAX_TAPS) return W4A32_ENOTSUP;
    if (!w4::row_linear_fits(pad64(l.heads * l.vdim))) return W4A32_ENOTSUP;
    if (l.ff > 0 && l.experts != 0) {
      if (l.experts < 0 || l.top <= 0 || l.top > l.experts || !(l.expert_limit > 0.0f)) return W4A32_EINVAL;
      if (l.experts > W4A32_LAYERED_MAX_EXPERTS || l.top > W4A32_LAYERED_MAX_TOP || !w4::moe_decode_fits(moe_geom(c, l)))
        return W4A32_ENOTSUP;
    } else if (l.ff > 0 && (!w4::row_linear_fits(pad64(l.ff)) || !w4::polynorm_fits(pad64(l.ff)))) return W4A32_ENOTSUP;
    switch (l.mixer) {
      case W4A32_MIX_ATTENTION: {
        if (l.window <= 0 || l.pool <= 0 || l.conv_taps < 0) return W4A32_EINVAL;
        if (l.heads / l.kv_heads * w4::head_bucket(std::max(l.dim, l.vdim)) > 4096 || l.heads / l.kv_heads > 32)
          return W4A32_ENOTSUP;
        if (l.kv_from >= 0) {
          if (l.kv_from >= i) return W4A32_ESHAPE;
          const w4a32_layer_config& s = c->layers[l.kv_from];
          if (s.mixer != W4A32_MIX_ATTENTION || s.kv_from >= 0 || s.kv_heads != l.kv_heads || s.dim != l.dim ||
              s.vdim != l.vdim)
            return W4A32_ESHAPE;
        }
        break;
      }
      case W4A32_MIX_DELTA:
        if (l.conv_taps < 1) return W4A32_EINVAL;
        break;
      case W4A32_MIX_RETENTION:
        if (l.kv_heads != l.heads || l.rot_dims < 0 || l.rot_dims % 2 != 0 || l.rot_dims > l.dim) return W4A32_ESHAPE;
        if (l.rot_dims > 0 && !(l.rot_base > 0.0)) return W4A32_EINVAL;
        break;
      case W4A32_MIX_ROTARY:
        if (l.window < 0 || l.rot_dims < 0) return W4A32_EINVAL;
        if (l.rot_dims % 2 != 0 || l.rot_dims > l.dim || (l.tied_values && l.vdim != l.dim)) return W4A32_ESHAPE;
        if (l.rot_dims > 0 && !(l.rot_base > 0.0)) return W4A32_EINVAL;
        if (l.conv_taps != 0 || l.heads / l.kv_heads * w4::head_bucket(std::max(l.dim, l.vdim)) > 4096 ||
            l.heads / l.kv_heads > 32)
          return W4A32_ENOTSUP;
        break;
      case W4A32_MIX_LATENT:
        if (l.window < 0 || l.rot_dims < 0 || l.q_rank <= 0 || l.kv_rank <= 0 || l.rot_part < 0) return W4A32_EINVAL;
        if (l.kv_heads != l.heads || l.rot_dims % 2 != 0 || l.rot_dims > l.rot_part) return W4A32_ESHAPE;
        if (l.rot_dims > 0 && !(l.rot_base > 0.0)) return W4A32_EINVAL;
        if (l.conv_taps != 0 || l.kv_rank > W4A32_LAYERED_MAX_LATENT || l.rot_part > W4A32_LAYERED_MAX_ROT_PART ||
            !w4::row_linear_fits(pad64(l.q_rank)))
          return W4A32_ENOTSUP;
        break;
      default: return W4A32_EINVAL;
    }
  }
  return W4A32_OK;
}

Geom geometry(const w4a32_layered_config* c) {
  Geom g;
  g.Hp = pad64(c->hidden);
  g.elem = c->dtype == W4A32_LAYERED_BF16 ? 2 : 4;
  const size_t Mb = c->max_batch_tokens;
  const int cap = (c->max_seq + 31) / 32 * 32;
  size_t o = 256;  // the position counter
  auto take = [&](size_t bytes) {
    const size_t at = o;
    o = align_up(o + bytes, 256);
    return at;
  };
  int raw = 0, cx = 0, q = 0, mix = 0, ff = 0, z = 0, ofl = 0, mlfl = 0, cq = 0, qa = 0, head_out = 0, experts = 0;
  size_t rec = 0, expand = 0, moe = 0, parts = g.Hp * Mb;
  g.runs = layer_runs(c);
  auto rot_table = [&](int dims, double base) {
    if (dims == 0) return -1;
    for (size_t r = 0; r < g.rot.size(); ++r)
      if (g.rot[r].dims == dims && g.rot[r].base == base) return (int)r;
    g.rot.push_back({dims, base, 0, 0});
    return (int)g.rot.size() - 1;
  };
  for (int i = 0; i < (int)g.runs.size(); ++i) {
    const w4a32_layer_config& l = c->layers[g.runs[i].layer];
    LayerGeom lg{};
    Geom::LayerState st{};
    lg.mix = l.heads * l.vdim;
    lg.D = w4::head_bucket(std::max(l.dim, l.vdim));
    lg.dv16 = (l.vdim + 15) / 16 * 16;
    lg.src = lg.pool_owner = i;
    lg.rot = -1;
    if (c->canon_taps > 0) st.canon1 = take(sizeof(float) * c->canon_taps * g.Hp);
    if (l.ff > 0 && c->canon_taps > 0) st.canon2 = take(sizeof(float) * c->canon_taps * g.Hp);
    if (l.mixer == W4A32_MIX_ATTENTION) {
      lg.rows = lg.conv_rows = l.heads * l.dim + (l.kv_from < 0 ? l.kv_heads * (l.dim + l.vdim) : 0);
      if (l.kv_from >= 0)  // the last run of that layer
        for (int e = 0; e < i; ++e)
          if (g.runs[e].layer == l.kv_from) lg.src = e;
      for (int e = 0; e < i; ++e) {
        const w4a32_layer_config& le = c->layers[g.runs[e].layer];
        if (le.mixer == W4A32_MIX_ATTENTION && g.layers[e].src == lg.src && le.pool == l.pool) {
          lg.pool_owner = g.layers[e].pool_owner;
          break;
        }
      }
      st.cap = cap;
      st.capp = (c->max_seq / l.pool + 1 + 31) / 32 * 32;
      if (lg.src == i) {
        st.k = take((size_t)g.elem * l.kv_heads * cap * lg.D);
        st.vt = take((size_t)g.elem * l.kv_heads * cap * lg.D);
      } else {
        st.k = g.st[lg.src].k;
        st.vt = g.st[lg.src].vt;
      }
      if (lg.pool_owner == i) {
        st.kp = take((size_t)g.elem * l.kv_heads * st.capp * lg.D);
        st.vpt = take((size_t)g.elem * l.kv_heads * st.capp * lg.D);
      } else {
        st.kp = g.st[lg.pool_owner].kp;
        st.vpt = g.st[lg.pool_owner].vpt;
      }
      if (l.conv_taps > 0) st.conv = take(sizeof(float) * l.conv_taps * pad64(lg.conv_rows));
      q = std::max(q, l.heads * lg.D);
      ofl = std::max(ofl, w4::kPoolAttnSlices * l.heads * lg.D);
      mlfl = std::max(mlfl, w4::kPoolAttnSlices * l.heads * 2);
    } else if (l.mixer == W4A32_MIX_ROTARY) {
      lg.rows = l.heads * l.dim + l.kv_heads * (l.dim + (l.tied_values ? 0 : l.vdim));
      st.cap = cap;
      st.k = take((size_t)g.elem * l.kv_heads * cap * lg.D);
      st.vt = take((size_t)g.elem * l.kv_heads * cap * lg.D);
      lg.rot = rot_table(l.rot_dims, l.rot_base);
      q = std::max(q, l.heads * lg.D);
      ofl = std::max(ofl, w4::kPoolAttnSlices * l.heads * lg.D);
      mlfl = std::max(mlfl, w4::kPoolAttnSlices * l.heads * 2);
    } else if (l.mixer == W4A32_MIX_LATENT) {
      lg.rows = l.q_rank + l.kv_rank + l.rot_part + (l.head_gate ? l.heads : 0);
      lg.q_rows = l.heads * (l.dim + l.rot_part);
      lg.Dc = pad64(l.kv_rank);
      lg.Dr = w4::latent_rot_pad(l.rot_part);
      st.cap = cap;
      st.k = take((size_t)g.elem * cap * (lg.Dc + lg.Dr));
      st.vt = take((size_t)g.elem * cap * lg.Dc);
      lg.rot = rot_table(l.rot_dims, l.rot_base);
      const int window = l.window > 0 ? l.window : w4::kNoWindow;
      g.expand_blk.resize(g.runs.size(), 0);
      g.expand_blk[i] = w4::latent_expand_blocks(window, c->max_seq, c->max_batch_tokens);
      expand = std::max(expand, w4::latent_expand_elems(l.heads, lg.D, g.expand_blk[i]));
      cq = std::max(cq, pad64(l.q_rank));
      // (a decode step's query row is f32)
      q = std::max(q, pad64(lg.q_rows) * (int)(sizeof(float) / g.elem));
      qa = std::max(qa, l.heads * (lg.Dc + lg.Dr));
      ofl = std::max(ofl, w4::kPoolAttnSlices * l.heads * lg.Dc);
      mlfl = std::max(mlfl, w4::kPoolAttnSlices * l.heads * 2);
      head_out = std::max(head_out, pad64(lg.mix));
    } else {
      const bool delta = l.mixer == W4A32_MIX_DELTA;
      const int nq = (delta ? l.kv_heads : l.heads) * l.dim;
      lg.rows = 2 * nq + 2 * lg.mix + (delta ? 2 * l.heads : 0);
      lg.conv_rows = delta ? 2 * nq + lg.mix : 0;
      if (delta) {
        st.conv = take(sizeof(float) * l.conv_taps * pad64(lg.conv_rows));
        cx = std::max(cx, pad64(lg.conv_rows));
      } else {
        lg.rot = rot_table(l.rot_dims, l.rot_base);
      }
      st.rec = take(sizeof(float) * (size_t)l.heads * lg.dv16 * lg.D);
      ofl = std::max(ofl, lg.mix);
      rec = std::max(rec, w4::rec_scratch_floats(l.heads, l.dim, l.vdim, c->max_batch_tokens));
    }
    raw = std::max(raw, pad64(lg.rows));
    mix = std::max(mix, pad64(lg.mix));
    if (l.ff > 0 && l.experts > 0) {
      experts = std::max(experts, l.experts);
      z = std::max(z, l.top * pad64(l.ff));
      moe = std::max(moe, w4::moe_scratch_bytes(c->dtype, c->max_batch_tokens, l.experts, l.top, pad64(l.ff)));
      parts = std::max(parts, (size_t)l.top * Mb * g.Hp);
    } else {
      ff = std::max(ff, pad64(l.ff));
    }
    g.layers.push_back(lg);
    g.st.push_back(st);
  }
  g.state_bytes = o;

  o = 0;
  for (auto& t : g.rot) {
    t.sin_off = take(sizeof(float) * c->max_seq * (t.dims / 2));
    t.cos_off = take(sizeof(float) * c->max_seq * (t.dims / 2));
  }
  g.x[0] = take(sizeof(float) * Mb * g.Hp);
  g.x[1] = take(sizeof(float) * Mb * g.Hp);
  g.y = take((size_t)g.elem * Mb * g.Hp * (c->loop_times > 0 ? 2 : 1));
  g.raw = take(sizeof(float) * Mb * raw);
  g.cx = take(sizeof(float) * Mb * cx);
  g.q = take((size_t)g.elem * Mb * q);
  g.mix = take((size_t)g.elem * Mb * mix);
  g.parts = take(sizeof(float) * std::max(parts, kSplitFloats));
  g.ff = take((size_t)g.elem * Mb * ff);
  g.z = take(sizeof(float) * std::max(ff, z));
  g.o = take(sizeof(float) * ofl);
  g.ml = take(sizeof(float) * mlfl);
  g.amax_v = take(sizeof(float) * kArgmaxParts);
  g.amax_i = take(sizeof(int) * kArgmaxParts);
  g.logits = take(sizeof(float) * c->vocab);
  g.last = take(sizeof(int));
  g.rec = take(sizeof(float) * rec);
  g.cq = take((size_t)g.elem * Mb * cq);
  g.ke = take(g.elem * expand);
  g.ve = take(g.elem * expand);
  g.qa = take(sizeof(float) * qa);
  g.head_out = take(sizeof(float) * head_out);
  g.router = take(sizeof(float) * w4::kMoeLogitParts * Mb * pad64(experts));
  g.moe = take(moe);
  g.sel = take(sizeof(int) * W4A32_LAYERED_MAX_TOP);
  g.ws_bytes = o;
  return g;
}

// One call's view of everything.
struct Run {
  const w4a32_layered_config* c;
  const w4a32_layered_weights* w;
  const Geom& g;
  uint8_t *st, *ws;
  hipStream_t s;

  float* f32(size_t off) const { return reinterpret_cast<float*>(ws + off); }
  float* stf(size_t off) const { return reinterpret_cast<float*>(st + off); }
  int* pos() const { return reinterpret_cast<int*>(st); }
  bool bf16() const { return c->dtype == W4A32_LAYERED_BF16; }
  // of run i
  const w4a32_layer_config& layer(int i) const { return c->layers[g.runs[i].layer]; }
  const w4a32_layered_layer& weights(int i) const { return w->layers[g.runs[i].layer]; }
  w4::NormSpec norm_spec() const {
    return {c->norm_eps, c->residual_mult != 0.0f ? c->residual_mult : 1.0f, c->norm == W4A32_NORM_RMS};
  }
  const float *sin_t(int i) const { return g.layers[i].rot >= 0 ? f32(g.rot[g.layers[i].rot].sin_off) : nullptr; }
  const float *cos_t(int i) const { return g.layers[i].rot >= 0 ? f32(g.rot[g.layers[i].rot].cos_off) : nullptr; }

  w4::AttnGeom attn_geom(int i) const {
    const w4a32_layer_config& l = layer(i);
    w4::AttnGeom a{};
    if (l.mixer == W4A32_MIX_ROTARY) {
      a.heads = l.heads; a.kv_heads = l.kv_heads; a.dim = l.dim; a.vdim = l.vdim; a.D = g.layers[i].D;
      a.cap = g.st[i].cap; a.capp = 32;
      a.window = l.window > 0 ? l.window : w4::kNoWindow;
      a.scale = l.scale;
      a.own_kv = true;
      a.tied = l.tied_values != 0;
      a.rot_dims = l.rot_dims; a.rot_rows = c->max_seq;
      a.sin_t = sin_t(i); a.cos_t = cos_t(i);
      a.sinks = weights(i).sinks;
      return a;
    }
    a.heads = l.heads; a.kv_heads = l.kv_heads; a.dim = l.dim; a.vdim = l.vdim; a.D = g.layers[i].D;
    a.cap = g.st[i].cap; a.capp = g.st[i].capp;
    a.window = l.window; a.pool = l.pool; a.scale = l.scale;
    a.taps = l.conv_taps; a.ldc = pad64(g.layers[i].conv_rows);
    a.own_kv = l.kv_from < 0;
    a.make_pool = g.layers[i].pool_owner == i;
    return a;
  }
  w4::AttnMem attn_mem(int i) const {
    const auto& t = g.st[i];
    return {st + t.k, st + t.vt, st + t.kp, st + t.vpt, layer(i).conv_taps > 0 ? stf(t.conv) : nullptr};
  }
  w4::LatentGeom latent_geom(int i) const {
    const w4a32_layer_config& l = layer(i);
    const w4a32_layered_layer& lw = weights(i);
    const LayerGeom& lg = g.layers[i];
    w4::LatentGeom a{};
    a.heads = l.heads; a.dim = l.dim; a.vdim = l.vdim; a.D = lg.D;
    a.q_rank = l.q_rank; a.kv_rank = l.kv_rank; a.rot_part = l.rot_part;
    a.Dc = lg.Dc; a.Dr = lg.Dr;
    a.cap = g.st[i].cap;
    a.window = l.window > 0 ? l.window : w4::kNoWindow;
    a.ldr = pad64(lg.rows);
    a.kv_off = l.q_rank; a.rot_off = l.q_rank + l.kv_rank;
    a.gate_off = l.head_gate ? a.rot_off + l.rot_part : -1;
    a.scale = l.scale;
    a.eps = c->norm_eps;
    a.rot_dims = l.rot_dims; a.rot_rows = c->max_seq;
    a.sin_t = sin_t(i); a.cos_t = cos_t(i);
    a.sinks = lw.sinks; a.q_norm = lw.q_norm; a.kv_norm = lw.kv_norm;
    a.k_up = lw.k_up; a.v_up = lw.v_up;
    return a;
  }
  w4::RecGeom rec_geom(int i) const {
    const w4a32_layer_config& l = layer(i);
    const w4a32_layered_layer& lw = weights(i);
    w4::RecGeom r{};
    r.delta = l.mixer == W4A32_MIX_DELTA;
    r.heads = l.heads; r.kv_heads = l.kv_heads; r.dim = l.dim; r.vdim = l.vdim; r.D = g.layers[i].D;
    r.ldr = pad64(g.layers[i].rows);
    const int nq = l.kv_heads * l.dim;
    r.q_off = 0; r.k_off = nq; r.v_off = 2 * nq; r.gate_off = r.v_off + g.layers[i].mix;
    r.a_off = r.gate_off + g.layers[i].mix; r.b_off = r.a_off + l.heads;
    r.taps = l.conv_taps; r.ldc = pad64(g.layers[i].conv_rows);
    r.eps = c->norm_eps;
    r.a_log = lw.a_log; r.dt_bias = lw.dt_bias; r.head_norm = r.delta ? lw.head_norm : nullptr;
    r.decay = lw.decay; r.log_decay = lw.log_decay;
    if (g.layers[i].rot >= 0) {
      r.sin_t = sin_t(i);
      r.cos_t = cos_t(i);
      r.rot_dims = l.rot_dims;
    }
    r.rot_rows = c->max_seq;
    return r;
  }
};

// C f32 or T [M][ldc] = A B^T; *parts: in the partial products the caller can take, out what was written
int product(const Run& r, const void* a, const void* b, void* cc, int M, int N, int K, bool out_t, int* parts) {
  if (r.bf16()) {
    const int p = parts ? w4::matmul_bf16_parts(M, N, K) : 1;
    if (parts) *parts = p;
    return from_hip(w4::launch_matmul_bf16(a, b, cc, M, N, K, N, out_t, p, r.s));
  }
  if (parts) *parts = 1;
  return from_hip(w4::launch_matmul_f32_nt(static_cast<const float*>(a), static_cast<const float*>(b),
                                           static_cast<float*>(cc), M, N, K, r.s));
}

// Rows of a portion. Leaves the residual rows in x[*cur] plus *pending partial rows in `parts`.
int prefill_layers(const Run& r, const int64_t* tokens, int M, int pos0, int n_layers, int* cur_out, int* pending_out) {
  const Geom& g = r.g;
  const w4a32_layered_config* c = r.c;
  const int H = c->hidden, Hp = g.Hp, dt = c->dtype;
  int cur = 0, pending = 0;
  W4_LAUNCH(w4::launch_embed_rows(dt, tokens, r.w->embedding, M, H, Hp, c->vocab, r.f32(g.x[0]), r.s));
  const w4::NormSpec spec = r.norm_spec();
  auto norm = [&](const float* w, const float* conv, size_t ring) {
    const int rc = from_hip(w4::launch_norm_conv(r.f32(g.x[cur]), r.f32(g.parts), pending, r.f32(g.x[cur ^ 1]), w,
                                                 spec, conv, r.stf(ring), c->canon_taps, M, H, Hp, pos0,
                                                 r.ws + g.y, r.bf16(), r.s));
    if (pending) cur ^= 1;
    pending = 0;
    return rc;
  };
  for (int i = 0; i < n_layers; ++i) {
    const w4a32_layer_config& l = r.layer(i);
    const w4a32_layered_layer& lw = r.weights(i);
    const LayerGeom& lg = g.layers[i];
    const int ldr = pad64(lg.rows), ldm = pad64(lg.mix);
    if (g.runs[i].pass_starts) {
      W4_LAUNCH(w4::launch_loop_rows(dt, r.f32(g.x[cur]), r.f32(g.parts), pending, spec.part_scale, tokens, r.w->embedding,
                                     c->vocab, M, Hp, r.ws + g.y, r.s));
      W4_TRY(product(r, r.ws + g.y, r.w->loop_in, r.f32(g.x[cur]), M, Hp, 2 * Hp, false, nullptr));
      pending = 0;
    }
    W4_TRY(norm(lw.norm1, lw.canon1, g.st[i].canon1));
    W4_TRY(product(r, r.ws + g.y, lw.in_proj, r.f32(g.raw), M, ldr, Hp, false, nullptr));
    if (l.mixer == W4A32_MIX_LATENT) {
      const w4::LatentGeom a = r.latent_geom(i);
      uint8_t *k = r.st + g.st[i].k, *vt = r.st + g.st[i].vt;
      const int ldc = pad64(l.q_rank), ldq = pad64(lg.q_rows), nblk = g.expand_blk[i];
      W4_LAUNCH(w4::launch_latent_rows(dt, a, k, vt, r.f32(g.raw), r.ws + g.cq, ldc, M, pos0, r.s));
      W4_TRY(product(r, r.ws + g.cq, lw.q_up, r.ws + g.q, M, ldq, ldc, true, nullptr));
      W4_LAUNCH(w4::launch_latent_expand(dt, a, k, r.ws + g.ke, r.ws + g.ve, nblk, M, pos0, r.s));
      W4_LAUNCH(w4::launch_latent_prefill(dt, a, k, r.ws + g.ke, r.ws + g.ve, nblk, r.ws + g.q, ldq, r.f32(g.raw),
                                          r.ws + g.mix, ldm, M, pos0, r.s));
    } else if (l.mixer == W4A32_MIX_ATTENTION || l.mixer == W4A32_MIX_ROTARY) {
      const w4::AttnGeom a = r.attn_geom(i);
      const w4::AttnMem m = r.attn_mem(i);
      W4_LAUNCH(w4::launch_attn_qkv(dt, a, m, r.f32(g.raw), ldr, l.conv_taps > 0 ? lw.conv : nullptr, r.ws + g.q, M,
                                    pos0, r.s));
      if (a.make_pool) W4_LAUNCH(w4::launch_attn_pool(dt, a, m, M, pos0, r.s));
      W4_LAUNCH(w4::launch_attn_prefill(dt, a, m, r.ws + g.q, r.ws + g.mix, ldm, M, pos0, r.s));
    } else {
      const w4::RecGeom rg = r.rec_geom(i);
      const int ldcx = pad64(lg.conv_rows);
      if (rg.delta) {
        W4_LAUNCH(w4::launch_short_conv(r.f32(g.raw), ldr, r.f32(g.cx), ldcx, lw.conv, r.stf(g.st[i].conv), ldcx,
                                        l.conv_taps, lg.conv_rows, true, M, pos0, r.s));
      }
      W4_LAUNCH(w4::launch_rec_prefill(dt, rg, r.f32(g.raw), r.f32(g.cx), ldcx, r.stf(g.st[i].rec), r.f32(g.rec),
                                       r.ws + g.mix, ldm, M, pos0, r.s));
    }
    W4_TRY(product(r, r.ws + g.mix, lw.out_proj, r.f32(g.parts), M, Hp, ldm, false, &pending));
    if (l.ff > 0 && l.experts > 0) {
      const int Ep = pad64(l.experts);
      W4_TRY(norm(lw.norm2, lw.canon2, g.st[i].canon2));
      int rp = 1;  // few tiles: dealt over k as far as that goes
      if (r.bf16()) {
        rp = std::max(1, std::min(w4::kMoeLogitParts, Hp / 128));
        W4_LAUNCH(w4::launch_matmul_bf16(r.ws + g.y, lw.router, r.f32(g.router), M, Ep, Hp, Ep, false, rp, r.s));
      } else {
        W4_TRY(product(r, r.ws + g.y, lw.router, r.f32(g.router), M, Ep, Hp, false, nullptr));
      }
      W4_LAUNCH(w4::launch_moe_prefill(dt, moe_geom(c, l), r.ws + g.y, r.f32(g.router), rp, Ep, lw.gate_up, lw.experts_down, M,
                                       r.f32(g.parts), r.ws + g.moe, r.s));
      pending = l.top;
    } else if (l.ff > 0) {
      const int Fp = pad64(l.ff);
      W4_TRY(norm(lw.norm2, lw.canon2, g.st[i].canon2));
      W4_TRY(product(r, r.ws + g.y, lw.up, r.ws + g.ff, M, Fp, Hp, true, nullptr));
      W4_LAUNCH(w4::launch_polynorm(r.ws + g.ff, r.bf16(), M, l.ff, Fp, lw.act, c->norm_eps, r.s));
      W4_TRY(product(r, r.ws + g.ff, lw.down, r.f32(g.parts), M, Hp, Fp, false, &pending));
    }
  }
  *cur_out = cur;
  *pending_out = pending;
  return W4A32_OK;
}

// One token at the state's position. Leaves the residual row in x[*cur] plus one partial row.
int decode_layers(const Run& r, const int64_t* token, int n_layers, int* cur_out, int* pending_out) {
  const Geom& g = r.g;
  const w4a32_layered_config* c = r.c;
  const int Hp = g.Hp, dt = c->dtype;
  int cur = 0, pending = 0;
  float* raw = r.f32(g.raw);
  float* part = r.f32(g.parts);
  const w4::NormSpec spec = r.norm_spec();
  for (int i = 0; i < n_layers; ++i) {
    const w4a32_layer_config& l = r.layer(i);
    const w4a32_layered_layer& lw = r.weights(i);
    const LayerGeom& lg = g.layers[i];
    w4::RowPrologue p{};
    p.K = c->hidden;
    p.x = r.f32(g.x[cur]);
    p.table = r.w->embedding;
    p.vocab = c->vocab;
    p.parts = part;
    p.n_parts = pending;
    p.part_stride = Hp;
    p.part_scale = spec.part_scale;
    p.rms = spec.rms;
    if (g.runs[i].pass_starts) {
      w4::RowPrologue q = p;
      q.token = token;
      if (i == 0) q.x = nullptr;
      W4_LAUNCH(w4::launch_row_linear(w4::kRowLoop, dt, q, r.w->loop_in, Hp, 2 * Hp, r.f32(g.x[cur ^ 1]), nullptr, nullptr,
                                      r.s));
      cur ^= 1;
      p.x = r.f32(g.x[cur]);
      p.n_parts = 0;
    } else if (i == 0) {
      p.token = token;
    }
    p.x_out = r.f32(g.x[cur ^ 1]);
    p.norm_w = lw.norm1;
    p.eps = c->norm_eps;
    p.conv = lw.canon1;
    p.ring = r.stf(g.st[i].canon1);
    p.taps = c->canon_taps;
    p.pos = r.pos();
    W4_LAUNCH(w4::launch_row_linear(w4::kRowNorm, dt, p, lw.in_proj, lg.rows, Hp, raw, nullptr, nullptr, r.s));
    cur ^= 1;

    w4::RowPrologue m{};
    m.K = lg.mix;
    m.o = r.f32(g.o);
    m.heads = l.heads;
    m.vdim = l.vdim;
    m.eps = c->norm_eps;
    int kind;
    if (l.mixer == W4A32_MIX_LATENT) {
      const w4::LatentGeom a = r.latent_geom(i);
      void *k = r.st + g.st[i].k, *vt = r.st + g.st[i].vt;
      float *q = r.f32(g.q), *qa = r.f32(g.qa), *o = r.f32(g.o), *ml = r.f32(g.ml);
      w4::RowPrologue n{};
      n.K = l.q_rank;
      n.x = raw;
      n.norm_w = lw.q_norm;
      n.eps = c->norm_eps;
      n.rms = true;
      W4_LAUNCH(w4::launch_row_linear(w4::kRowNorm, dt, n, lw.q_up, lg.q_rows, pad64(l.q_rank), q, nullptr, nullptr, r.s));
      W4_LAUNCH(w4::launch_latent_absorb(dt, a, k, vt, raw, q, r.pos(), qa, r.s));
      W4_LAUNCH(w4::launch_latent_decode(dt, a, k, vt, qa, r.pos(), c->max_seq, o, ml, r.s));
      W4_LAUNCH(w4::launch_latent_out(dt, a, o, ml, w4::latent_slices(a.window, c->max_seq), raw, r.f32(g.head_out), r.s));
      m.x = r.f32(g.head_out);
      kind = w4::kRowPlain;
    } else if (l.mixer == W4A32_MIX_ATTENTION || l.mixer == W4A32_MIX_ROTARY) {
      W4_LAUNCH(w4::launch_attn_decode(dt, r.attn_geom(i), r.attn_mem(i), raw, lw.conv, r.pos(), c->max_seq,
                                       r.f32(g.o), r.f32(g.ml), r.s));
      m.ml = r.f32(g.ml);
      m.slices = w4::attn_slices(r.attn_geom(i), c->max_seq);
      m.dvp = lg.D;
      kind = w4::kRowMerge;
    } else {
      const w4::RecGeom rg = r.rec_geom(i);
      W4_LAUNCH(w4::launch_rec_decode(rg, raw, lw.conv, rg.delta ? r.stf(g.st[i].conv) : nullptr,
                                      r.stf(g.st[i].rec), r.pos(), r.f32(g.o), r.s));
      m.gate = raw + rg.gate_off;
      m.head_w = rg.head_norm;
      kind = w4::kRowGated;
    }
    W4_LAUNCH(w4::launch_row_linear(kind, dt, m, lw.out_proj, Hp, pad64(lg.mix), part, nullptr, nullptr, r.s));
    pending = 1;

    if (l.ff > 0) {
      p.token = nullptr;
      p.x = r.f32(g.x[cur]);
      p.n_parts = 1;
      p.x_out = r.f32(g.x[cur ^ 1]);
      p.norm_w = lw.norm2;
      p.conv = lw.canon2;
      p.ring = r.stf(g.st[i].canon2);
    }
    if (l.ff > 0 && l.experts > 0) {
      W4_LAUNCH(w4::launch_row_linear(w4::kRowNorm, dt, p, lw.router, l.experts, Hp, r.f32(g.router), nullptr, nullptr, r.s));
      cur ^= 1;
      // the completed residual row is there now (an input convolution's ring is written with the same row again)
      p.x = r.f32(g.x[cur]);
      p.n_parts = 0;
      p.x_out = nullptr;
      W4_LAUNCH(w4::launch_moe_decode(dt, moe_geom(c, l), p, r.f32(g.router), lw.gate_up, lw.experts_down, r.f32(g.z),
                                      reinterpret_cast<int*>(r.ws + g.sel), part, r.s));
    } else if (l.ff > 0) {
      W4_LAUNCH(w4::launch_row_linear(w4::kRowNorm, dt, p, lw.up, pad64(l.ff), Hp, r.f32(g.z), nullptr, nullptr, r.s));
      cur ^= 1;
      w4::RowPrologue f{};
      f.K = l.ff;
      f.x = r.f32(g.z);
      f.act = lw.act;
      f.eps = c->norm_eps;
      W4_LAUNCH(w4::launch_row_linear(w4::kRowPoly, dt, f, lw.down, Hp, pad64(l.ff), part, nullptr, nullptr, r.s));
    }
  }
  *cur_out = cur;
  *pending_out = pending;
  return W4A32_OK;
}

// final norm + head of one row (of M) -> logits, with the partial argmax results
int head_row(const Run& r, int cur, int pending, int row, int M, float* logits) {
  const Geom& g = r.g;
  w4::RowPrologue p{};
  p.K = r.c->hidden;
  p.x = r.f32(g.x[cur]) + (size_t)row * g.Hp;
  p.parts = r.f32(g.parts) + (size_t)row * g.Hp;
  p.n_parts = pending;
  p.part_stride = (size_t)M * g.Hp;
  p.part_scale = r.norm_spec().part_scale;
  p.rms = r.norm_spec().rms;
  p.norm_w = r.w->final_norm;
  p.eps = r.c->norm_eps;
  return from_hip(w4::launch_row_linear(w4::kRowNorm, r.c->dtype, p, r.w->head, r.c->vocab, g.Hp, logits,
                                        r.f32(g.amax_v), reinterpret_cast<int*>(r.ws + g.amax_i), r.s));
}

int pick_token(const Run& r, int64_t* token_out, int* pos_to_advance) {
  return from_hip(w4::launch_argmax_parts(r.f32(r.g.amax_v), reinterpret_cast<const int*>(r.ws + r.g.amax_i),
                                          w4::row_linear_partials(w4::kRowNorm, r.c->vocab), token_out, pos_to_advance, r.s));
}

int check_call(const w4a32_layered_config* c, const w4a32_layered_weights* w, const void* st, const void* ws) {
  W4_TRY(check_config(c));
  if (!w || !w->embedding || !w->final_norm || !w->head || !w->layers || !st || !ws) return W4A32_EINVAL;
  if ((reinterpret_cast<uintptr_t>(st) & 255) != 0 || (reinterpret_cast<uintptr_t>(ws) & 255) != 0) return W4A32_EINVAL;
  if (c->loop_times > 0 && !w->loop_in) return W4A32_EINVAL;
  for (int i = 0; i < c->n_layers; ++i) {
    const w4a32_layer_config& l = c->layers[i];
    const w4a32_layered_layer& lw = w->layers[i];
    if (!lw.norm1 || !lw.in_proj || !lw.out_proj) return W4A32_EINVAL;
    if (c->canon_taps > 0 && (!lw.canon1 || (l.ff > 0 && !lw.canon2))) return W4A32_EINVAL;
    if (l.mixer == W4A32_MIX_LATENT && (!lw.q_norm || !lw.kv_norm || !lw.q_up || !lw.k_up || !lw.v_up)) return W4A32_EINVAL;
    if (l.mixer != W4A32_MIX_RETENTION && l.conv_taps > 0 && !lw.conv) return W4A32_EINVAL;
    if (l.mixer == W4A32_MIX_DELTA && (!lw.a_log || !lw.dt_bias || !lw.head_norm)) return W4A32_EINVAL;
    if (l.mixer == W4A32_MIX_RETENTION && (!lw.decay || !lw.log_decay)) return W4A32_EINVAL;
    if (l.ff > 0 && !lw.norm2) return W4A32_EINVAL;
    if (l.ff > 0 && l.experts == 0 && (!lw.up || !lw.down || !lw.act)) return W4A32_EINVAL;
    if (l.ff > 0 && l.experts > 0 && (!lw.router || !lw.gate_up || !lw.experts_down)) return W4A32_EINVAL;
  }
  return W4A32_OK;
}

}  // namespace

extern "C" {

int w4a32_layered_check(const w4a32_layered_config* cfg) { return check_config(cfg); }

int w4a32_layered_head_rows(int dim, int vdim) { return w4::head_bucket(std::max(dim, vdim)); }

int w4a32_layered_runs(const w4a32_layered_config* cfg) {
  return check_config(cfg) == W4A32_OK ? (int)layer_runs(cfg).size() : 0;
}

size_t w4a32_layered_state_bytes(const w4a32_layered_config* cfg) {
  return check_config(cfg) == W4A32_OK ? geometry(cfg).state_bytes : 0;
}

size_t w4a32_layered_workspace_bytes(const w4a32_layered_config* cfg) {
  return check_config(cfg) == W4A32_OK ? geometry(cfg).ws_bytes : 0;
}

size_t w4a32_layered_position_offset(const w4a32_layered_config* cfg) {
  (void)cfg;
  return 0;
}

size_t w4a32_layered_residual_offset(const w4a32_layered_config* cfg) {
  return check_config(cfg) == W4A32_OK ? geometry(cfg).x[0] : 0;
}

int w4a32_layered_init_state(const w4a32_layered_config* cfg, void* d_state, void* stream) {
  W4_TRY(check_config(cfg));
  if (!d_state) return W4A32_EINVAL;
  return from_hip(w4::launch_fill_zero(d_state, geometry(cfg).state_bytes, S(stream)));
}

int w4a32_layered_init_workspace(const w4a32_layered_config* cfg, void* d_ws, void* stream) {
  W4_TRY(check_config(cfg));
  if (!d_ws) return W4A32_EINVAL;
  const Geom g = geometry(cfg);
  W4_LAUNCH(w4::launch_fill_zero(d_ws, g.ws_bytes, S(stream)));
  for (const auto& t : g.rot) {
    W4_LAUNCH(w4::launch_rot_table(reinterpret_cast<float*>(static_cast<uint8_t*>(d_ws) + t.sin_off),
                                   reinterpret_cast<float*>(static_cast<uint8_t*>(d_ws) + t.cos_off), cfg->max_seq,
                                   t.dims, t.base, S(stream)));
  }
  return W4A32_OK;
}

int w4a32_layered_forward(const w4a32_layered_config* cfg, const w4a32_layered_weights* w, void* d_state, void* d_ws,
                          const int64_t* d_tokens, int n_tokens, int pos0, const int* d_want, int n_want,
                          float* d_logits, int stop_after, void* stream) {
  W4_TRY(check_call(cfg, w, d_state, d_ws));
  if (!d_tokens || n_tokens <= 0 || pos0 < 0 || n_want < 0 || stop_after < 0) return W4A32_EINVAL;
  if (n_want > 0 && (!d_want || !d_logits)) return W4A32_EINVAL;
  if (n_tokens > cfg->max_batch_tokens || n_want > n_tokens || pos0 > cfg->max_seq - n_tokens ||
      stop_after > (int)layer_runs(cfg).size())
    return W4A32_ESHAPE;
  const Geom g = geometry(cfg);
  const Run r{cfg, w, g, static_cast<uint8_t*>(d_state), static_cast<uint8_t*>(d_ws), S(stream)};
  const int n_layers = stop_after > 0 ? stop_after : (int)g.runs.size();
  int cur = 0, pending = 0;
  if (n_tokens == 1) {
    W4_LAUNCH(w4::launch_set_int(r.pos(), pos0, r.s));
    W4_TRY(decode_layers(r, d_tokens, n_layers, &cur, &pending));
  } else {
    W4_TRY(prefill_layers(r, d_tokens, n_tokens, pos0, n_layers, &cur, &pending));
  }
  W4_LAUNCH(w4::launch_set_int(r.pos(), pos0 + n_tokens, r.s));
  if (stop_after > 0) {
    return from_hip(w4::launch_add_parts(r.f32(g.x[cur]), r.f32(g.parts), pending, r.norm_spec().part_scale, r.f32(g.x[0]), n_tokens, g.Hp, r.s));
  }
  if (n_want == 0) return W4A32_OK;
  if (n_tokens == 1) return head_row(r, cur, pending, 0, 1, d_logits);
  W4_LAUNCH(w4::launch_norm_want(r.f32(g.x[cur]), r.f32(g.parts), pending, w->final_norm, r.norm_spec(), d_want, n_want,
                                 n_tokens, cfg->hidden, g.Hp, r.ws + g.y, r.bf16(), r.s));
  return product(r, r.ws + g.y, w->head, d_logits, n_want, cfg->vocab, g.Hp, false, nullptr);
}

int w4a32_layered_prefill(const w4a32_layered_config* cfg, const w4a32_layered_weights* w, void* d_state, void* d_ws,
                          const int64_t* d_tokens, int n_tokens, int pos0, int64_t* d_next_token, void* stream) {
  if (!d_next_token) return W4A32_EINVAL;
  W4_TRY(check_call(cfg, w, d_state, d_ws));
  if (!d_tokens || n_tokens <= 0 || pos0 < 0) return W4A32_EINVAL;
  if (n_tokens > cfg->max_batch_tokens || pos0 > cfg->max_seq - n_tokens) return W4A32_ESHAPE;
  const Geom g = geometry(cfg);
  const Run r{cfg, w, g, static_cast<uint8_t*>(d_state), static_cast<uint8_t*>(d_ws), S(stream)};
  int cur = 0, pending = 0;
  if (n_tokens == 1) {
    W4_LAUNCH(w4::launch_set_int(r.pos(), pos0, r.s));
    W4_TRY(decode_layers(r, d_tokens, (int)g.runs.size(), &cur, &pending));
  } else {
    W4_TRY(prefill_layers(r, d_tokens, n_tokens, pos0, (int)g.runs.size(), &cur, &pending));
  }
  W4_LAUNCH(w4::launch_set_int(r.pos(), pos0 + n_tokens, r.s));
  W4_TRY(head_row(r, cur, pending, n_tokens - 1, n_tokens, r.f32(g.logits)));
  return pick_token(r, d_next_token, nullptr);
}

int w4a32_layered_step(const w4a32_layered_config* cfg, const w4a32_layered_weights* w, void* d_state, void* d_ws,
                       const int64_t* d_token_in, int64_t* d_token_out, void* stream) {
  W4_TRY(check_call(cfg, w, d_state, d_ws));
  if (!d_token_in || !d_token_out) return W4A32_EINVAL;
  const Geom g = geometry(cfg);
  const Run r{cfg, w, g, static_cast<uint8_t*>(d_state), static_cast<uint8_t*>(d_ws), S(stream)};
  int cur = 0, pending = 0;
  W4_TRY(decode_layers(r, d_token_in, (int)g.runs.size(), &cur, &pending));
  W4_TRY(head_row(r, cur, pending, 0, 1, r.f32(g.logits)));
  return pick_token(r, d_token_out, r.pos());
}

int w4a32_op_matmul_bf16_nt(const void* d_a, const void* d_b, void* d_c, int M, int N, int K, int ldc, int c_bf16,
                            int parts, void* stream) {
  if (!d_a || !d_b || !d_c || M <= 0 || N <= 0 || K <= 0 || parts < 1) return W4A32_EINVAL;
  if (K % W4A32_LAYERED_PAD != 0 || ldc < N || parts > K / W4A32_LAYERED_PAD || (parts > 1 && c_bf16)) return W4A32_ESHAPE;
  if ((reinterpret_cast<uintptr_t>(d_a) & 15) != 0 || (reinterpret_cast<uintptr_t>(d_b) & 15) != 0) return W4A32_EINVAL;
  return from_hip(w4::launch_matmul_bf16(d_a, d_b, d_c, M, N, K, ldc, c_bf16 != 0, parts, S(stream)));
}

int w4a32_op_layernorm_conv(const float* d_x, const float* d_parts, int n_parts, float* d_x_out, const float* d_norm,
                            float eps, const float* d_conv, float* d_ring, int taps, int M, int H, int pos0, void* d_y,
                            int y_bf16, void* stream) {
  if (!d_x || !d_norm || !d_y || M <= 0 || H <= 0 || pos0 < 0 || n_parts < 0 || taps < 0) return W4A32_EINVAL;
  if (n_parts > 0 && (!d_parts || !d_x_out || d_x_out == d_x)) return W4A32_EINVAL;
  if (taps > 0 && (!d_conv || !d_ring)) return W4A32_EINVAL;
  if (taps > W4A32_LAYERED_MAX_TAPS || !w4::norm_conv_fits(pad64(H), taps)) return W4A32_ENOTSUP;
  w4::NormSpec spec{eps};
  return from_hip(w4::launch_norm_conv(d_x, d_parts, n_parts, d_x_out, d_norm, spec, d_conv, d_ring, taps, M, H, pad64(H),
                                       pos0, d_y, y_bf16 != 0, S(stream)));
}

int w4a32_op_short_conv(const float* d_x, int ldx, float* d_y, int ldy, const float* d_w, float* d_ring, int ldw,
                        int taps, int channels, int apply_silu, int M, int pos0, void* stream) {
  if (!d_x || !d_y || !d_w || !d_ring || channels <= 0 || M <= 0 || pos0 < 0) return W4A32_EINVAL;
  if (taps < 1 || taps > W4A32_LAYERED_MAX_TAPS) return W4A32_ENOTSUP;
  if (ldx < channels || ldy < channels || ldw < channels) return W4A32_ESHAPE;
  return from_hip(w4::launch_short_conv(d_x, ldx, d_y, ldy, d_w, d_ring, ldw, taps, channels, apply_silu != 0, M, pos0,
                                        S(stream)));
}

size_t w4a32_op_experts_scratch_bytes(int dtype, int M, int experts, int top, int ff) {
  if (M <= 0 || experts <= 0 || top <= 0 || ff <= 0) return 0;
  return w4::moe_scratch_bytes(dtype, M, experts, top, pad64(ff));
}

int w4a32_op_experts(int dtype, const void* d_h, const float* d_logits, int ld, const void* d_gate_up, const void* d_down,
                     int M, int hidden, int experts, int top, int ff, float limit, float* d_parts, void* d_scratch,
                     void* stream) {
  if (!d_h || !d_logits || !d_gate_up || !d_down || !d_parts || !d_scratch || M <= 0 || hidden <= 0 || experts <= 0 ||
      top <= 0 || ff <= 0 || !(limit > 0.0f) || (dtype != W4A32_LAYERED_BF16 && dtype != W4A32_LAYERED_F32))
    return W4A32_EINVAL;
  if (top > experts || ld < experts) return W4A32_ESHAPE;
  if (experts > W4A32_LAYERED_MAX_EXPERTS || top > W4A32_LAYERED_MAX_TOP) return W4A32_ENOTSUP;
  const w4::MoeGeom g{hidden, pad64(hidden), ff, pad64(ff), experts, top, limit};
  return from_hip(w4::launch_moe_prefill(dtype, g, d_h, d_logits, 1, ld, d_gate_up, d_down, M, d_parts, d_scratch, S(stream)));
}

int w4a32_op_polynorm(void* d_z, int z_bf16, int M, int F, int ld, const float* d_act, float eps, void* stream) {
  if (!d_z || !d_act || M <= 0 || F <= 0) return W4A32_EINVAL;
  if (ld < F || ld % 4 != 0) return W4A32_ESHAPE;
  if (!w4::polynorm_fits(ld)) return W4A32_ENOTSUP;
  return from_hip(w4::launch_polynorm(d_z, z_bf16 != 0, M, F, ld, d_act, eps, S(stream)));
}

}  // extern "C"
