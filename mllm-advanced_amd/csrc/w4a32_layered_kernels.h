// Launchers of the layered decoder's kernels and the small device pieces they share. Arguments are validated by
// the callers (w4a32_layered.hip).
#pragma once

#include <hip/hip_runtime.h>

#include "w4a32_internal.h"
#include "w4a32_layered.h"
#include "w4a32_quant_math.h"

namespace w4 {

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

constexpr int kPad = 64;
inline int pad64(int n) { return (n + kPad - 1) / kPad * kPad; }

// ---- device pieces ----
// sum over the wavefront, in every lane (all 64 active)
__device__ __forceinline__ float wave_sum64(float v) {
  return __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(wave_sum_to_lane63(v)), 63));
}
__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
// log(1 + e^x) without overflow and without losing small results
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.0f) + log1pf(expf(-fabsf(x))); }

// four consecutive elements as f32, and back
__device__ __forceinline__ float4 load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 load4(const __bf16* p) {
  const uint2 u = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xFFFF0000u), __uint_as_float(u.y << 16),
                     __uint_as_float(u.y & 0xFFFF0000u));
}
__device__ __forceinline__ void store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void store4(__bf16* p, float4 v) {
  bf16x4 b;
  b[0] = (__bf16)v.x; b[1] = (__bf16)v.y; b[2] = (__bf16)v.z; b[3] = (__bf16)v.w;
  *reinterpret_cast<bf16x4*>(p) = b;
}
__device__ __forceinline__ float& at4(float4& v, int i) { return reinterpret_cast<float*>(&v)[i]; }

// one channel of a short convolution for the token at position p; its inputs of earlier positions are in the ring
__device__ __forceinline__ float conv_step(float x, const float* __restrict__ w, const float* __restrict__ ring, int c,
                                           int ldc, int taps, int p) {
  float wv[W4A32_LAYERED_MAX_TAPS], rv[W4A32_LAYERED_MAX_TAPS];
#pragma unroll
  for (int j = 0; j < W4A32_LAYERED_MAX_TAPS; ++j) {  // all requested before the first is used
    if (j >= taps) break;
    const int q = p - taps + 1 + j;
    wv[j] = w[(size_t)j * ldc + c];
    rv[j] = q >= 0 && q < p ? ring[(size_t)(q % taps) * ldc + c] : q == p ? x : 0.0f;
  }
  float y = 0.0f;
#pragma unroll
  for (int j = 0; j < W4A32_LAYERED_MAX_TAPS; ++j) {
    if (j >= taps) break;
    y = __fmaf_rn(wv[j], rv[j], y);
  }
  return y;
}

// ---- what the decode Linear does to its input row before it multiplies ----
enum RowKind {
  kRowNorm = 0,   // residual add of partial rows, layer norm, input convolution
  kRowMerge = 1,  // attention output from its key slices
  kRowGated = 2,  // per head: over its root mean square, times a weight, times silu(gate)
  kRowPoly = 3,   // PolyNorm
  kRowPlain = 4,  // the row as it is
  kRowLoop = 5,   // residual add of partial rows, the token's embedding row behind it (K: twice the padded width)
};
struct RowPrologue {
  int K;                // true length of the row
  // kRowNorm
  const float* x;       // [ld]; not read when `token` is given
  const int64_t* token; // first launch of a step: the row is table[*token] (element type: the weights')
  const void* table;
  int vocab;
  const float* parts;   // n_parts partial rows, part_stride floats apart
  int n_parts;
  size_t part_stride;
  float part_scale;     // factor of the partial rows
  bool rms;             // divided by the root mean square, no mean taken off
  float* x_out;         // [ld], stored by the first workgroup
  const float* norm_w;
  float eps;
  const float* conv;    // [taps][ld], taps may be 0
  float* ring;
  int taps;
  const int* pos;
  // kRowMerge: o [slices][heads][dvp], ml [slices][heads][2] (max, sum)
  const float* o;
  const float* ml;
  int slices, heads, vdim, dvp;
  // kRowGated: o [heads * vdim], gate [heads * vdim], head_w [vdim] or null
  const float* gate;
  const float* head_w;
  // kRowPoly: x is the row
  const float* act;
  // kRowLoop: the residual row is x, or, without it, the embedding row as well
};

// y[n] = sum_k row[k] W[n][k], f32 output; W T [N][Kp]; optionally one (max, first column) pair per wavefront
hipError_t launch_row_linear(int kind, int dtype, const RowPrologue& pro, const void* w, int N, int Kp, float* y,
                             float* amax_val, int* amax_idx, hipStream_t s);
int row_linear_partials(int kind, int N);  // wavefronts of that launch (<= 4096)
bool row_linear_fits(int Kp);

// bf16 product; parts > 1: C [parts][M][ldc] f32 partial products
hipError_t launch_matmul_bf16(const void* a, const void* b, void* c, int M, int N, int K, int ldc, bool c_bf16,
                              int parts, hipStream_t s);
int matmul_bf16_parts(int M, int N, int K);  // parts worth using for few tiles

// ---- rows of a prefill ----
hipError_t launch_embed_rows(int dtype, const int64_t* ids, const void* table, int M, int H, int ld, int vocab,
                             float* x, hipStream_t s);
bool norm_conv_fits(int ld, int taps);
// how a residual row takes in the partial rows behind it, and how it is normed
struct NormSpec {
  float eps, part_scale = 1.0f;
  bool rms = false;
};
hipError_t launch_norm_conv(const float* x, const float* parts, int n_parts, float* x_out, const float* norm_w,
                            const NormSpec& spec, const float* conv, float* ring, int taps, int M, int H, int ld, int pos0,
                            void* y, bool y_bf16, hipStream_t s);
// layer norm of the wanted rows (x + parts), no convolution: y [n_want][ld]
hipError_t launch_norm_want(const float* x, const float* parts, int n_parts, const float* norm_w,
                            const NormSpec& spec, const int* want, int n_want, int M, int H, int ld, void* y, bool y_bf16, hipStream_t s);
// out = x + scale * parts; out may be x
hipError_t launch_add_parts(const float* x, const float* parts, int n_parts, float scale, float* out, int M, int ld,
                            hipStream_t s);
// y [M][2 ld] = [x + scale * parts, embedding row], element type T
hipError_t launch_loop_rows(int dtype, const float* x, const float* parts, int n_parts, float scale, const int64_t* ids,
                            const void* table, int vocab, int M, int ld, void* y, hipStream_t s);
bool polynorm_fits(int ld);
hipError_t launch_polynorm(void* z, bool z_bf16, int M, int F, int ld, const float* act, float eps, hipStream_t s);

// short convolution, plain form
hipError_t launch_short_conv(const float* x, int ldx, float* y, int ldy, const float* w, float* ring, int ldw, int taps,
                             int channels, bool silu, int M, int pos0, hipStream_t s);

// ---- pooled-window attention ----
// Caches of one layer: keys and values T [kv_heads][cap * D] in blocks of 32 entries (layouts in
// w4a32_pooled_attention.hip), their block means likewise with capp entries; D = head_bucket(max(dim, vdim)), padding
// dimensions zero.
struct AttnGeom {
  int heads, kv_heads, dim, vdim, D;
  int cap, capp;        // multiples of 32
  int window, pool;
  float scale;
  int taps;             // of the short convolution; 0: none
  int ldc;              // leading dimension of the convolution's weights and ring
  bool own_kv;          // this layer projects keys and values itself
  bool make_pool;       // ... and / or is the one that keeps the block means it reads
  bool tied;            // the values are the keys before rotation
  int rot_dims, rot_rows;      // rotation of q and k (no convolution with it); rows of the tables
  const float *sin_t, *cos_t;  // [rot_rows][rot_dims / 2]
  const float* sinks;          // [heads], or null
};
constexpr int kNoWindow = 1 << 30;  // window of a layer that sees every token
// pool 0: no block means
struct AttnMem {
  void *k, *vt, *kp, *vpt;
  float* ring;
};
int head_bucket(int d);  // 32, 64, 128, 256
// q, k, v rows of in_proj (f32 [M][ldr]) through the convolution: q -> T [M][heads][D], k and v -> caches
hipError_t launch_attn_qkv(int dtype, const AttnGeom& g, const AttnMem& m, const float* raw, int ldr, const float* conv,
                           void* q, int M, int pos0, hipStream_t s);
hipError_t launch_attn_pool(int dtype, const AttnGeom& g, const AttnMem& m, int M, int pos0, hipStream_t s);
// out T [M][ldo], columns past heads * vdim zero
hipError_t launch_attn_prefill(int dtype, const AttnGeom& g, const AttnMem& m, const void* q, void* out, int ldo, int M,
                               int pos0, hipStream_t s);
constexpr int kPoolAttnSlices = 16;  // most of them
int attn_slices(const AttnGeom& g, int max_seq);
hipError_t launch_attn_decode(int dtype, const AttnGeom& g, const AttnMem& m, const float* raw, const float* conv,
                              const int* pos, int max_seq, float* o, float* ml, hipStream_t s);

// ---- latent attention ----
// Cache of one layer: k [blocks][(Dc + Dr) / 8][32][8] holds a token's latent and rotated key part, vt [blocks][Dc][32] the
// latent once more in the values' order (both as in w4a32_pooled_attention.hip, one kv head).
struct LatentGeom {
  int heads, dim, vdim, D;      // D = head_bucket(max(dim, vdim)): rows per head of the operand blocks
  int q_rank, kv_rank, rot_part;
  int Dc, Dr;                   // kv_rank padded to 64, rot_part to 16
  int cap, window;
  int ldr, kv_off, rot_off, gate_off;  // in_proj row: where the kv latent, the key part and the gates are (gate_off -1: none)
  float scale, eps;
  int rot_dims, rot_rows;
  const float *sin_t, *cos_t, *sinks, *q_norm, *kv_norm;
  const void *k_up, *v_up;
};
int latent_rot_pad(int rot_part);
size_t latent_expand_elems(int heads, int D, int blocks);  // of each, keys and values
int latent_expand_blocks(int window, int max_seq, int max_batch_tokens);
// rows of a portion: the query's latent, normed, -> T cq [M][ldq]; latent and key part -> cache
hipError_t launch_latent_rows(int dtype, const LatentGeom& g, void* k, void* vt, const float* raw, void* cq, int ldq, int M,
                              int pos0, hipStream_t s);
// keys and values of the tokens the portion sees -> ke, ve (nblk blocks allotted per head)
hipError_t launch_latent_expand(int dtype, const LatentGeom& g, const void* k, void* ke, void* ve, int nblk, int M, int pos0,
                                hipStream_t s);
// q T [M][ldq], not yet rotated; out T [M][ldo]
hipError_t launch_latent_prefill(int dtype, const LatentGeom& g, const void* k, const void* ke, const void* ve, int nblk,
                                 const void* q, int ldq, const float* raw, void* out, int ldo, int M, int pos0,
                                 hipStream_t s);
// one token: cache append, q [heads * (dim + rot_part)] folded into the latent space -> qa f32 [heads][Dc + Dr]
hipError_t launch_latent_absorb(int dtype, const LatentGeom& g, void* k, void* vt, const float* raw, const float* q,
                                const int* pos, float* qa, hipStream_t s);
int latent_slices(int window, int max_seq);
// o [slice][heads][Dc] (not divided), ml [slice][heads] (max, sum)
hipError_t launch_latent_decode(int dtype, const LatentGeom& g, const void* k, const void* vt, const float* qa,
                                const int* pos, int max_seq, float* o, float* ml, hipStream_t s);
// slices merged, values read out of the latents, gates: y f32 [heads * vdim]
hipError_t launch_latent_out(int dtype, const LatentGeom& g, const float* o, const float* ml, int slices, const float* raw,
                             float* y, hipStream_t s);

// ---- mixture of experts ----
struct MoeGeom {
  int hidden, Hp, ff, Fp, experts, top;
  float limit;
};
constexpr int kMoeLogitParts = 8;  // most of them
size_t moe_scratch_bytes(int dtype, int M, int experts, int top, int Fp);
// rows: h T [M][Hp], router logits f32 [logit_parts][M][ldl] -> parts f32 [top][M][Hp]
hipError_t launch_moe_prefill(int dtype, const MoeGeom& g, const void* h, const float* logits, int logit_parts, int ldl,
                              const void* gate_up, const void* down, int M, float* parts, void* scratch, hipStream_t s);
// one token: pro is the norm in front (its x_out must be null), z f32 [top * Fp], sel int [top]; out f32 [Hp]
bool moe_decode_fits(const MoeGeom& g);
hipError_t launch_moe_decode(int dtype, const MoeGeom& g, const RowPrologue& pro, const float* logits, const void* gate_up,
                             const void* down, float* z, int* sel, float* out, hipStream_t s);

// ---- recurrences with a matrix state ----
// State of a layer: f32 [heads][dv16][D], transposed (a value row's D key dimensions are contiguous); dv16 = vdim
// rounded up to 16.
struct RecGeom {
  bool delta;                 // gated delta rule, else retention
  int heads, kv_heads, dim, vdim, D;
  int ldr;                    // in_proj rows
  int q_off, k_off, v_off, gate_off, a_off, b_off;  // columns in an in_proj row
  int taps, ldc;              // delta: short convolution
  float eps;
  const float *a_log, *dt_bias, *head_norm;   // delta
  const float *decay, *log_decay;             // retention
  const float *sin_t, *cos_t;                 // retention: [max_seq][rot_dims / 2]
  int rot_dims, rot_rows;                     // rot_rows: positions the tables hold
};
size_t rec_scratch_floats(int heads, int dim, int vdim, int M);
// rows of a prefill. cx: delta only, the convolved q, k, v rows f32 [M][ldcx]. out T [M][ldo]: per-head norm and
// gate applied, columns past heads * vdim zero
hipError_t launch_rec_prefill(int dtype, const RecGeom& g, const float* raw, const float* cx, int ldcx, float* state,
                              float* scratch, void* out, int ldo, int M, int pos0, hipStream_t s);
// one token: o f32 [heads * vdim], before norm and gate
hipError_t launch_rec_decode(const RecGeom& g, const float* raw, const float* conv, float* ring, float* state,
                             const int* pos, float* o, hipStream_t s);
hipError_t launch_rot_table(float* sin_t, float* cos_t, int max_pos, int dims, double base, hipStream_t s);
hipError_t launch_fill_zero(void* p, size_t bytes, hipStream_t s);  // bytes % 16 == 0

}  // namespace w4
