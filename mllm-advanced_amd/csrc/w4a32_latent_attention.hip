// Latent attention: a token leaves one latent (normed) and one rotated key part for all heads, nothing else is cached.
//
//   latent_rows_kernel     a portion's rows: norm of the query's latent, norm of the latent and rotation of the key part, both
//                          into the cache
//   latent_expand_kernel   prefill: keys and values of every head for the tokens the portion sees, from the cached latents;
//                          cache blocks and weights both lie in operand order, so a wavefront loads its operands straight
//                          from memory and stores the results in the order the attention (attn_mfma_kernel) loads them
//   latent_absorb_kernel   decode: cache append, and the key matrix folded into the query (q U_h, one row of kv_rank per head)
//   latent_decode_kernel   one token, bf16: heads stand where the prefill kernel has queries. S^T = C Q^T and O^T += C^T P^T on
//                          v_mfma_f32_32x32x16_bf16, C the latents; a workgroup takes a slice of the blocks of 32 tokens
//   latent_rows_decode_kernel  the same, f32, a thread per key and per latent dimension
//   latent_out_kernel      decode: slices merged, values read out of the merged latent (V_h o_h), gate
//
// Cache layouts are in w4a32_layered_kernels.h; operand blocks of the weights in w4a32_layered.h.
#include <algorithm>
#include <type_traits>

#include "w4a32_attn_blocks.h"
#include "w4a32_layered.h"
#include "w4a32_layered_kernels.h"

namespace w4 {

namespace {

constexpr int kMaxLatent = W4A32_LAYERED_MAX_LATENT, kMaxRot = W4A32_LAYERED_MAX_ROT_PART;

// ---------------------------------------------------------------------------------------------
constexpr int kRowTok = 8;

// What a token leaves in the cache, f32, by one wavefront: s_c [kv_rank] normed latent, then [rot_part] rotated key part.
__device__ __forceinline__ void latent_of_row(const float* __restrict__ raw, int kv_rank, int rot_part, int rot_dims,
                                              int kv_off, int rot_off, const float* __restrict__ norm_w, float eps, int p,
                                              const float* __restrict__ sin_t, const float* __restrict__ cos_t,
                                              float* __restrict__ s_c) {
  const int lane = threadIdx.x & 63;
  constexpr int kRegs = kMaxLatent / 64, kRotRegs = kMaxRot / 64;
  float x[kRegs], w[kRegs], y[kRotRegs], z[kRotRegs], sn[kRotRegs], cs[kRotRegs], ss = 0.0f;
  const int half = rot_dims / 2;
#pragma unroll
  for (int i = 0; i < kRotRegs; ++i) {  // all requested before the first is used
    const int d = min(lane + 64 * i, max(rot_part - 1, 0)), angle = d < half ? d : d - half;
    const bool turn = d < rot_dims;
    y[i] = rot_part > 0 ? raw[rot_off + d] : 0.0f;
    z[i] = turn ? raw[rot_off + rot_partner(d, rot_dims)] : 0.0f;
    cs[i] = turn ? cos_t[(size_t)p * half + angle] : 1.0f;
    sn[i] = turn ? sin_t[(size_t)p * half + angle] : 0.0f;
    if (d < half) sn[i] = -sn[i];
  }
#pragma unroll
  for (int i = 0; i < kRegs; ++i) {
    const int d = min(lane + 64 * i, kv_rank - 1);
    x[i] = 64 * i < kv_rank ? raw[kv_off + d] : 0.0f;
    w[i] = 64 * i < kv_rank ? norm_w[d] : 0.0f;
  }
#pragma unroll
  for (int i = 0; i < kRegs; ++i) {
    if (lane + 64 * i >= kv_rank) x[i] = 0.0f;
    ss += x[i] * x[i];
  }
  const float r = 1.0f / sqrtf(wave_sum64(ss) / (float)kv_rank + eps);
#pragma unroll
  for (int i = 0; i < kRegs; ++i)
    if (lane + 64 * i < kv_rank) s_c[lane + 64 * i] = x[i] * r * w[i];
#pragma unroll
  for (int i = 0; i < kRotRegs; ++i)
    if (lane + 64 * i < rot_part) s_c[kv_rank + lane + 64 * i] = y[i] * cs[i] + z[i] * sn[i];
}

struct RowsArgs {
  int q_rank, kv_rank, rot_part, rot_dims, Dc, Dr, ldr, kv_off, rot_off, ldq;
  float eps;
  const float *q_norm, *kv_norm, *sin_t, *cos_t;
};

// A workgroup takes up to eight tokens, aligned to eight positions (a run of values of one dimension is one store), a
// wavefront each.
template <typename T>
__global__ __launch_bounds__(64 * kRowTok) void latent_rows_kernel(const float* __restrict__ raw, T* __restrict__ cq,
                                                                   T* __restrict__ kc, T* __restrict__ vt, int M, int pos0,
                                                                   const RowsArgs a) {
  extern __shared__ __align__(16) float s_c[];  // [kRowTok][ld], ld odd: the eight tokens' rows start on other banks
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, ld = (a.kv_rank + a.rot_part) | 1;
  const int lead = pos0 & (kRowTok - 1);
  const int t0 = max(0, (int)blockIdx.x * kRowTok - lead), te = min(M, ((int)blockIdx.x + 1) * kRowTok - lead);
  const int t = t0 + wave;
  if (t < te) {
    const float* row = raw + (size_t)t * a.ldr;
    constexpr int kRegs = 32;  // a query latent of up to 2048 stays in registers
    float x[kRegs], w[kRegs], ss = 0.0f;
    if (a.ldq <= 64 * kRegs) {
#pragma unroll
      for (int i = 0; i < kRegs; ++i) {
        const int d = min(lane + 64 * i, a.q_rank - 1);
        x[i] = 64 * i < a.q_rank ? row[d] : 0.0f;
        w[i] = 64 * i < a.q_rank ? a.q_norm[d] : 0.0f;
      }
      latent_of_row(row, a.kv_rank, a.rot_part, a.rot_dims, a.kv_off, a.rot_off, a.kv_norm, a.eps, pos0 + t, a.sin_t,
                    a.cos_t, s_c + (size_t)wave * ld);
#pragma unroll
      for (int i = 0; i < kRegs; ++i) {
        if (lane + 64 * i >= a.q_rank) x[i] = 0.0f;
        ss += x[i] * x[i];
      }
      const float r = 1.0f / sqrtf(wave_sum64(ss) / (float)a.q_rank + a.eps);
#pragma unroll
      for (int i = 0; i < kRegs; ++i) {
        const int d = lane + 64 * i;
        if (d < a.ldq) cq[(size_t)t * a.ldq + d] = (T)(x[i] * r * w[i]);
      }
    } else {
      latent_of_row(row, a.kv_rank, a.rot_part, a.rot_dims, a.kv_off, a.rot_off, a.kv_norm, a.eps, pos0 + t, a.sin_t,
                    a.cos_t, s_c + (size_t)wave * ld);
      for (int d = lane; d < a.q_rank; d += 64) ss += row[d] * row[d];
      const float r = 1.0f / sqrtf(wave_sum64(ss) / (float)a.q_rank + a.eps);
      for (int d = lane; d < a.ldq; d += 64)
        cq[(size_t)t * a.ldq + d] = d < a.q_rank ? (T)(row[d] * r * a.q_norm[d]) : (T)0.0f;
    }
  }
  __syncthreads();
  const int n = te - t0, p0 = pos0 + t0, D = a.Dc + a.Dr;
  T* kb = kc + (size_t)(p0 >> 5) * (32 * D);  // all of them lie in one block
  T* vb = vt + (size_t)(p0 >> 5) * (32 * a.Dc);
  // keys: the tokens of eight dimensions side by side
  for (int it = threadIdx.x; it < (D / 8) * kRowTok; it += 64 * kRowTok) {
    const int s = it / kRowTok, i = it & (kRowTok - 1);
    if (i >= n) continue;
    const float* src = s_c + (size_t)i * ld;
    struct alignas(sizeof(T) * 8) E8 { T e[8]; } v;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int d = 8 * s + e;
      v.e[e] = d < a.kv_rank ? (T)src[d] : d >= a.Dc && d - a.Dc < a.rot_part ? (T)src[a.kv_rank + d - a.Dc] : (T)0.0f;
    }
    *reinterpret_cast<E8*>(kb + (size_t)(s * 32 + ((p0 + i) & 31)) * 8) = v;
  }
  // values: runs of four tokens of a dimension
  for (int it = threadIdx.x; it < a.kv_rank * 2; it += 64 * kRowTok) {
    const int d = it >> 1, first = 4 * (it & 1) - (p0 & (kRowTok - 1));  // this run's first token
    const int q = (p0 & ~(kRowTok - 1)) + 4 * (it & 1);                  // its position
    T* dst = vb + (size_t)d * 32 + v_pos(q & 31);
    if (first >= 0 && first + 4 <= n) {
      struct alignas(sizeof(T) * 4) E4 { T e[4]; } v;
#pragma unroll
      for (int i = 0; i < 4; ++i) v.e[i] = (T)s_c[(size_t)(first + i) * ld + d];
      *reinterpret_cast<E4*>(dst) = v;
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (first + i >= 0 && first + i < n) dst[i] = (T)s_c[(size_t)(first + i) * ld + d];
    }
  }
}

// ---------------------------------------------------------------------------------------------
// Wavefront tile: two blocks of 32 tokens x two blocks of 32 rows of the operand; workgroup: 2 x 2 wavefronts. grid.y: tiles
// of 128 rows of keys, then of values.
__global__ __launch_bounds__(256) void latent_expand_kernel(const __bf16* __restrict__ kc, const __bf16* __restrict__ k_up,
                                                            const __bf16* __restrict__ v_up, __bf16* __restrict__ ke,
                                                            __bf16* __restrict__ ve, int rows, int D, int Dc, int Dr,
                                                            int blk0, int n_blk, int nblk) {
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, j = lane & 31, hh = lane >> 5;
  const int half = (int)gridDim.y / 2;
  const bool is_k = (int)blockIdx.y < half;
  const int rb = 4 * ((int)blockIdx.y - (is_k ? 0 : half)) + 2 * (wave & 1);  // first block of rows
  const int tb = 4 * (int)blockIdx.x + 2 * (wave >> 1);                       // first block of tokens, of those expanded
  const int row_blocks = rows / 32;
  if (rb >= row_blocks || tb >= n_blk) return;
  const int KS = Dc / 16;
  const __bf16* w = (is_k ? k_up : v_up) + 8 * lane;
  const __bf16* wa[2];
  const __bf16* ca[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    wa[i] = w + (size_t)min(rb + i, row_blocks - 1) * 32 * Dc;
    ca[i] = kc + (size_t)(blk0 + min(tb + i, n_blk - 1)) * 32 * (Dc + Dr) + 8 * lane;
  }
  f32x16 acc[2][2];  // [token block][row block]
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int c = 0; c < 2; ++c)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[i][c][v] = 0.0f;
  // four steps of 16 latent dimensions at a time (Dc is a multiple of 64), the next eight on their way
  bf16x8 wf[3][2][4], cf[3][2][4];  // [register set][block][step]
  auto fetch = [&](int s, int set) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        wf[set][i][u] = *reinterpret_cast<const bf16x8*>(wa[i] + 512 * (s + u));
        cf[set][i][u] = *reinterpret_cast<const bf16x8*>(ca[i] + 512 * (s + u));
      }
    __builtin_amdgcn_sched_barrier(0);  // or the loads sink to their uses
  };
  auto products = [&](auto keys, int set) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int c = 0; c < 2; ++c)
          acc[i][c] = decltype(keys)::value ? mfma_bf16(wf[set][c][u], cf[set][i][u], acc[i][c])
                                            : mfma_bf16(cf[set][i][u], wf[set][c][u], acc[i][c]);
  };
  auto all = [&](auto keys) __attribute__((always_inline)) {
    fetch(0, 0);
    fetch(min(4, KS - 4), 1);
    for (int s = 0; s < KS; s += 12) {
      fetch(min(s + 8, KS - 4), 2);
      products(keys, 0);
      if (s + 4 >= KS) break;
      fetch(min(s + 12, KS - 4), 0);
      products(keys, 1);
      if (s + 8 >= KS) break;
      fetch(min(s + 16, KS - 4), 1);
      products(keys, 2);
    }
  };
  const int per_head = D / 32;
  if (is_k) {  // accumulator rows: dimensions, columns: tokens
    all(std::true_type{});
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      if (rb + c >= row_blocks) continue;
      const int h = (rb + c) / per_head, db = (rb + c) % per_head;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        if (tb + i >= n_blk) continue;
        __bf16* dst = ke + ((size_t)h * nblk + tb + i) * 32 * D + (size_t)(4 * db * 32 + j) * 8 + 4 * hh;
#pragma unroll
        for (int g = 0; g < 4; ++g)
          store4(dst + (size_t)g * 32 * 8, make_float4(acc[i][c][4 * g], acc[i][c][4 * g + 1], acc[i][c][4 * g + 2],
                                                       acc[i][c][4 * g + 3]));
      }
    }
  } else {  // accumulator rows: tokens, columns: dimensions
    all(std::false_type{});
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      if (rb + c >= row_blocks) continue;
      const int h = (rb + c) / per_head, db = (rb + c) % per_head;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        if (tb + i >= n_blk) continue;
        __bf16* dst = ve + ((size_t)h * nblk + tb + i) * 32 * D + (size_t)(32 * db + j) * 32 + 8 * hh;
#pragma unroll
        for (int o = 0; o < 2; ++o) {
          bf16x8 v;
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = (__bf16)acc[i][c][8 * o + e];
          *reinterpret_cast<bf16x8*>(dst + 16 * o) = v;
        }
      }
    }
  }
}

// f32: a workgroup per (block of tokens, 32 rows), keys then values; a thread has one token and four rows
__global__ __launch_bounds__(256) void latent_expand_f32_kernel(const float* __restrict__ kc, const float* __restrict__ k_up,
                                                                const float* __restrict__ v_up, float* __restrict__ ke,
                                                                float* __restrict__ ve, int rows, int D, int Dc, int Dr,
                                                                int blk0, int nblk) {
  const int rb = (int)blockIdx.y % (rows / 32);
  const bool is_k = (int)blockIdx.y < rows / 32;
  const int j = threadIdx.x & 31, r0 = 4 * (threadIdx.x >> 5);
  const float* c = kc + (size_t)(blk0 + blockIdx.x) * 32 * (Dc + Dr) + 8 * j;
  const float* w = (is_k ? k_up : v_up) + (size_t)rb * 32 * Dc + 8 * r0;
  float acc[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int s = 0; s < Dc / 8; ++s) {
    const float4 c0 = load4(c + 256 * s), c1 = load4(c + 256 * s + 4);
    const float cs[8] = {c0.x, c0.y, c0.z, c0.w, c1.x, c1.y, c1.z, c1.w};
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[r] = __fmaf_rn(w[256 * s + 8 * r + e], cs[e], acc[r]);
  }
  const int h = rb / (D / 32), d0 = 32 * (rb % (D / 32)) + r0;
  float* dst = (is_k ? ke : ve) + ((size_t)h * nblk + blockIdx.x) * 32 * D;
#pragma unroll
  for (int r = 0; r < 4; ++r) dst[is_k ? k_at(j, d0 + r, D) : v_at(j, d0 + r, D)] = acc[r];
}

// ---------------------------------------------------------------------------------------------
struct AbsorbArgs {
  int heads, dim, D, kv_rank, rot_part, rot_dims, rot_rows, Dc, Dr, kv_off, rot_off;
  float eps;
  const float *kv_norm, *sin_t, *cos_t;
};

// Workgroups 0 .. : a wavefront per (head, 16 latent dimensions), half a wavefront per eight of them, a lane per row of
// the operand block. Then one workgroup for the cache, the rest for the rotated query parts.
template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const float* __restrict__ raw, const float* __restrict__ q,
                                                            const T* __restrict__ k_up, T* __restrict__ kc,
                                                            T* __restrict__ vt, const int* __restrict__ d_pos,
                                                            float* __restrict__ qa, int fold_wgs, const AbsorbArgs a) {
  __shared__ float s_c[kMaxLatent + kMaxRot];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, j = lane & 31, hh = lane >> 5;
  const int D = a.Dc + a.Dr, ldq = a.dim + a.rot_part;
  if ((int)blockIdx.x < fold_wgs) {
    const int pairs = a.Dc / 16, id = 4 * (int)blockIdx.x + wave;
    if (id >= a.heads * pairs) return;
    const int h = id / pairs, s = 2 * (id % pairs) + hh;
    const T* w = k_up + (size_t)h * a.D * a.Dc + (size_t)(s * 32 + j) * 8;
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = 0.0f;
#pragma unroll 4
    for (int d = j; d < a.dim; d += 32) {
      Eight<T> v;
      v.load(w + (size_t)(d >> 5) * 32 * a.Dc);
      const float x = q[(size_t)h * ldq + d];
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = __fmaf_rn(v.get(e), x, acc[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e)
#pragma unroll
      for (int off = 16; off >= 1; off >>= 1) acc[e] += __shfl_xor(acc[e], off, 64);
    if (j == 0) {
      float* dst = qa + (size_t)h * D + 8 * s;
      store4(dst, make_float4(acc[0], acc[1], acc[2], acc[3]));
      store4(dst + 4, make_float4(acc[4], acc[5], acc[6], acc[7]));
    }
    return;
  }
  const int p = min(*d_pos, a.rot_rows - 1);
  if ((int)blockIdx.x == fold_wgs) {
    if (wave == 0)
      latent_of_row(raw, a.kv_rank, a.rot_part, a.rot_dims, a.kv_off, a.rot_off, a.kv_norm, a.eps, p, a.sin_t, a.cos_t, s_c);
    __syncthreads();
    T* kb = kc + (size_t)(p >> 5) * (32 * D) + (size_t)(p & 31) * 8;
    T* vb = vt + (size_t)(p >> 5) * (32 * a.Dc) + v_pos(p & 31);
    for (int d = threadIdx.x; d < a.kv_rank; d += 256) {
      kb[(size_t)(d >> 3) * 256 + (d & 7)] = (T)s_c[d];
      vb[(size_t)d * 32] = (T)s_c[d];
    }
    for (int d = threadIdx.x; d < a.rot_part; d += 256)
      kb[(size_t)((a.Dc + d) >> 3) * 256 + (d & 7)] = (T)s_c[a.kv_rank + d];
    return;
  }
  const int it = ((int)blockIdx.x - fold_wgs - 1) * 256 + threadIdx.x;
  if (it >= a.heads * a.Dr) return;
  const int h = it / a.Dr, d = it - h * a.Dr;
  const float* src = q + (size_t)h * ldq + a.dim;
  float y = d < a.rot_part ? src[d] : 0.0f;
  if (d < a.rot_dims) y = rotated(y, src[rot_partner(d, a.rot_dims)], d, a.rot_dims, (size_t)p, a.sin_t, a.cos_t);
  qa[(size_t)h * D + a.Dc + d] = y;
}

// ---------------------------------------------------------------------------------------------
constexpr int kDecWaves = 4;

// blocks of 32 tokens that a slice of the visible ones takes
__device__ __forceinline__ void slice_blocks(int p, int window, int slices, int slice, int* lo_key, int* b_lo, int* b_hi) {
  const int lo = max(0, p - window + 1), first = lo / 32, blocks = p / 32 - first + 1;
  const int per = (blocks + slices - 1) / slices;
  *lo_key = lo;
  *b_lo = first + min(blocks, slice * per);
  *b_hi = first + min(blocks, (slice + 1) * per);
}

// grid (slices, blocks of 32 heads). Tiles of four blocks of tokens: a wavefront scores one of them (lane: head l % 32), the
// softmax weights go through LDS as operands (sum of two bf16 terms), then a wavefront sums the latent dimensions
// 32 (wave + 4 i) .. of the whole tile. CW: of these at most.
template <int CW>
__global__ __launch_bounds__(64 * kDecWaves) void latent_decode_kernel(
    const __bf16* __restrict__ kc, const __bf16* __restrict__ vt, const float* __restrict__ qa,
    const int* __restrict__ d_pos, int max_seq, int heads, int Dc, int Dr, int window, float scale,
    const float* __restrict__ sinks, float* __restrict__ o, float* __restrict__ ml) {
  extern __shared__ __align__(16) uint8_t smem[];
  const int D = Dc + Dr, KS = D / 16, DB = Dc / 32;
  bf16x8* s_q = reinterpret_cast<bf16x8*>(smem);                   // [8 (CW + 1)][64], zeros past KS
  bf16x8* s_p = s_q + 8 * (CW + 1) * 64;                            // [waves][ks][term][64]
  float* s_max = reinterpret_cast<float*>(s_p + kDecWaves * 4 * 64);  // [2][waves][32]
  float* s_sum = s_max + 2 * kDecWaves * 32;                       // [waves][32]
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, j = lane & 31, hh = lane >> 5;
  const int slice = blockIdx.x, head = 32 * blockIdx.y + j;
  const int p = min(*d_pos, max_seq - 1);
  int lo, b_lo, b_hi;
  slice_blocks(p, window, gridDim.x, slice, &lo, &b_lo, &b_hi);

  // A tile's operands are requested as a whole: this wavefront's block of keys, its latent dimensions of all blocks.
  constexpr int KQ = 8 * (CW + 1);  // most steps of 16 dimensions: Dc up to 128 CW, Dr up to 128
  const __bf16* kb = kc + 8 * lane;
  const __bf16* vb = vt + 32 * j + 8 * hh;
  bf16x8 kop[KQ], vop[kDecWaves][CW][2];
  auto load_k = [&](int bt) __attribute__((always_inline)) {
    const __bf16* src = kb + (size_t)min(bt + wave, b_hi - 1) * 32 * D;
#pragma unroll
    for (int s = 0; s < KQ; ++s) kop[s] = *reinterpret_cast<const bf16x8*>(src + 512 * min(s, KS - 1));
  };
  auto load_v = [&](int bt) __attribute__((always_inline)) {
#pragma unroll
    for (int w = 0; w < kDecWaves; ++w)
#pragma unroll
      for (int i = 0; i < CW; ++i)
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
          vop[w][i][ks] = *reinterpret_cast<const bf16x8*>(
              vb + ((size_t)min(bt + w, b_hi - 1) * Dc + 32 * min(wave + kDecWaves * i, DB - 1)) * 32 + 16 * ks);
  };
  constexpr int NQ = 2 * (CW + 1);  // pieces of the query operands a thread brings
  float4 qx[NQ][2];
#pragma unroll
  for (int i = 0; i < NQ; ++i) {
    const int s = wave + kDecWaves * i, h = min(head, heads - 1);
    const float* src = qa + (size_t)h * D + 16 * min(s, KS - 1) + 8 * hh;
    qx[i][0] = load4(src);
    qx[i][1] = load4(src + 4);
  }
  constexpr bool kAhead = CW <= 2;  // registers for both
  if (b_lo < b_hi) {
    load_k(b_lo);
    if (kAhead) load_v(b_lo);
  }
  __builtin_amdgcn_sched_barrier(0);
#pragma unroll
  for (int i = 0; i < NQ; ++i) {
    const int s = wave + kDecWaves * i;
    const float x[8] = {qx[i][0].x, qx[i][0].y, qx[i][0].z, qx[i][0].w, qx[i][1].x, qx[i][1].y, qx[i][1].z, qx[i][1].w};
    bf16x8 v;
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = s < KS ? (__bf16)x[e] : (__bf16)0.0f;
    s_q[s * 64 + lane] = v;
  }
  f32x16 acc[CW];
#pragma unroll
  for (int i = 0; i < CW; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[i][v] = 0.0f;
  float run_max = -INFINITY, run_sum = 0.0f;  // run_sum: of this wavefront's blocks
  if (sinks && slice == 0) {                  // a term of the denominator without a value
    run_max = sinks[min(head, heads - 1)];
    run_sum = wave == 0 ? 1.0f : 0.0f;
  }
  __syncthreads();

  int turn = 0;
  for (int bt = b_lo; bt < b_hi; bt += kDecWaves, turn ^= 1) {
    const int n = min(kDecWaves, b_hi - bt);
    float blk_max = -INFINITY;
    f32x16 st, st1;
#pragma unroll
    for (int v = 0; v < 16; ++v) st[v] = st1[v] = 0.0f;
    if (wave < n) {
      const int b = bt + wave;
#pragma unroll
      for (int s = 0; s < KQ; s += 2) {
        st = mfma_bf16(kop[s], s_q[s * 64 + lane], st);
        st1 = mfma_bf16(kop[s + 1], s_q[(s + 1) * 64 + lane], st1);
      }
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        const int key = 32 * b + 8 * (v >> 2) + 4 * hh + (v & 3);
        st[v] = key >= lo && key <= p ? (st[v] + st1[v]) * scale : -INFINITY;
        blk_max = fmaxf(blk_max, st[v]);
      }
      blk_max = fmaxf(blk_max, __shfl_xor(blk_max, 32, 64));
    }
    if (!kAhead) load_v(bt);
    float* mx = s_max + turn * kDecWaves * 32;
    if (hh == 0) mx[wave * 32 + j] = blk_max;
    __syncthreads();
    float new_max = run_max;
#pragma unroll
    for (int w = 0; w < kDecWaves; ++w) new_max = fmaxf(new_max, mx[w * 32 + j]);
    const float corr = run_max == -INFINITY ? 0.0f : __expf(run_max - new_max);
    run_max = new_max;
    run_sum *= corr;
    if (wave < n) {
      float psum = 0.0f;
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        st[v] = st[v] == -INFINITY ? 0.0f : __expf(st[v] - new_max);
        psum += st[v];
      }
      run_sum += psum + __shfl_xor(psum, 32, 64);
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        bf16x8 p1, p2;  // the weights as a sum of two bf16 terms
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float x = st[8 * ks + e];
          p1[e] = (__bf16)x;
          p2[e] = (__bf16)(x - (float)p1[e]);
        }
        s_p[((wave * 2 + ks) * 2 + 0) * 64 + lane] = p1;
        s_p[((wave * 2 + ks) * 2 + 1) * 64 + lane] = p2;
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < CW; ++i)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[i][v] *= corr;
#pragma unroll
    for (int w = 0; w < kDecWaves; ++w) {
      if (w >= n) break;
      const int b = bt + w;
      if (32 * b + 31 > p) {  // tokens past the last one may hold anything: a zero weight must not meet them
#pragma unroll
        for (int i = 0; i < CW; ++i)
#pragma unroll
          for (int ks = 0; ks < 2; ++ks)
#pragma unroll
            for (int e = 0; e < 8; ++e)
              if (32 * b + 16 * ks + 8 * (e >> 2) + 4 * hh + (e & 3) > p) vop[w][i][ks][e] = (__bf16)0.0f;
      }
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const bf16x8 p1 = s_p[((w * 2 + ks) * 2 + 0) * 64 + lane], p2 = s_p[((w * 2 + ks) * 2 + 1) * 64 + lane];
#pragma unroll
        for (int i = 0; i < CW; ++i) acc[i] = mfma_bf16(vop[w][i][ks], p2, acc[i]);
#pragma unroll
        for (int i = 0; i < CW; ++i) acc[i] = mfma_bf16(vop[w][i][ks], p1, acc[i]);
      }
    }
    if (bt + kDecWaves < b_hi) {
      load_k(bt + kDecWaves);
      if (kAhead) load_v(bt + kDecWaves);
    }
    // the next tile's weights are written behind its first barrier, which is behind this tile's last read
  }
  if (hh == 0) s_sum[wave * 32 + j] = run_sum;
  __syncthreads();
  if (head >= heads) return;
  if (wave == 0 && hh == 0) {
    float total = 0.0f;
#pragma unroll
    for (int w = 0; w < kDecWaves; ++w) total += s_sum[w * 32 + j];
    float* dst = ml + 2 * ((size_t)slice * heads + head);
    dst[0] = run_max;
    dst[1] = total;
  }
  float* dst = o + ((size_t)slice * heads + head) * Dc + 4 * hh;
#pragma unroll
  for (int i = 0; i < CW; ++i) {
    const int db = wave + kDecWaves * i;
    if (db >= DB) break;
#pragma unroll
    for (int g = 0; g < 4; ++g)
      store4(dst + 32 * db + 8 * g, make_float4(acc[i][4 * g], acc[i][4 * g + 1], acc[i][4 * g + 2], acc[i][4 * g + 3]));
  }
}

// f32: grid (slices, heads); tiles of 256 keys
__global__ __launch_bounds__(256) void latent_rows_decode_kernel(
    const float* __restrict__ kc, const float* __restrict__ vt, const float* __restrict__ qa,
    const int* __restrict__ d_pos, int max_seq, int heads, int Dc, int Dr, int window, float scale,
    const float* __restrict__ sinks, float* __restrict__ o, float* __restrict__ ml) {
  __shared__ float s_q[kMaxLatent + kMaxRot], s_p[256], s_red[8];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, slice = blockIdx.x, h = blockIdx.y, D = Dc + Dr;
  const int p = min(*d_pos, max_seq - 1);
  int lo, b_lo, b_hi;
  slice_blocks(p, window, gridDim.x, slice, &lo, &b_lo, &b_hi);
  for (int d = tid; d < D; d += 256) s_q[d] = qa[(size_t)h * D + d];
  float run_max = -INFINITY, run_sum = 0.0f, acc[kMaxLatent / 256] = {0.0f};
  if (sinks && slice == 0) {
    run_max = sinks[h];
    run_sum = 1.0f;
  }
  __syncthreads();
  for (int bt = b_lo; bt < b_hi; bt += 8) {
    const int key = 32 * bt + tid;
    float s = -INFINITY;
    if (key >= lo && key <= p && key < 32 * b_hi) {
      const float* src = kc + (size_t)(key >> 5) * 32 * D + (size_t)(key & 31) * 8;
      s = 0.0f;
      for (int i = 0; i < D / 8; ++i) {
        const float4 x0 = load4(src + 256 * i), x1 = load4(src + 256 * i + 4);
        const float xs[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
        for (int e = 0; e < 8; ++e) s = __fmaf_rn(s_q[8 * i + e], xs[e], s);
      }
      s *= scale;
    }
    float mx = s;
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
    if (lane == 0) s_red[wave] = mx;
    __syncthreads();
    const float new_max = fmaxf(run_max, fmaxf(fmaxf(s_red[0], s_red[1]), fmaxf(s_red[2], s_red[3])));
    const float corr = run_max == -INFINITY ? 0.0f : expf(run_max - new_max);
    const float w = s == -INFINITY ? 0.0f : expf(s - new_max);
    const float sum = wave_sum64(w);
    if (lane == 0) s_red[4 + wave] = sum;
    s_p[tid] = w;
    __syncthreads();
    run_max = new_max;
    run_sum = run_sum * corr + ((s_red[4] + s_red[5]) + (s_red[6] + s_red[7]));
    const int n = min(256, min(p + 1, 32 * b_hi) - 32 * bt);
#pragma unroll
    for (int i = 0; i < kMaxLatent / 256; ++i) {
      const int d = tid + 256 * i;
      if (d >= Dc) break;
      float a = acc[i] * corr;
      for (int k = 0; k < n; ++k) a = __fmaf_rn(s_p[k], vt[(size_t)((32 * bt + k) >> 5) * 32 * Dc + (size_t)d * 32 + v_pos(k & 31)], a);
      acc[i] = a;
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < kMaxLatent / 256; ++i) {
    const int d = tid + 256 * i;
    if (d < Dc) o[((size_t)slice * heads + h) * Dc + d] = acc[i];
  }
  if (tid == 0) {
    float* dst = ml + 2 * ((size_t)slice * heads + h);
    dst[0] = run_max;
    dst[1] = run_sum;
  }
}

// ---------------------------------------------------------------------------------------------
constexpr int kOutWaves = 8;

// grid (heads, blocks of 32 value dimensions): a lane has one row of the operand block and every other piece of eight latent
// dimensions; the pieces are dealt to the wavefronts.
template <typename T>
__global__ __launch_bounds__(64 * kOutWaves) void latent_out_kernel(const float* __restrict__ o, const float* __restrict__ ml,
                                                                    int slices, int heads, const T* __restrict__ v_up, int D,
                                                                    int Dc, int vdim, const float* __restrict__ gate,
                                                                    float* __restrict__ y) {
  __shared__ __align__(16) float s_o[kMaxLatent];
  __shared__ float s_part[kOutWaves][32];
  const int h = blockIdx.x, vb = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, j = lane & 31, hh = lane >> 5;
  constexpr int kAhead = kMaxLatent / 16 / kOutWaves;
  const T* w = v_up + ((size_t)h * D + 32 * vb) * Dc + 8 * lane;
  Eight<T> f[kAhead];
#pragma unroll
  for (int i = 0; i < kAhead; ++i) f[i].load(w + (size_t)512 * min(wave + kOutWaves * i, Dc / 16 - 1));
  float wt[kPoolAttnSlices], mx = -INFINITY, den = 0.0f;
#pragma unroll
  for (int i = 0; i < kPoolAttnSlices; ++i) {
    const float2 v = *reinterpret_cast<const float2*>(ml + 2 * ((size_t)min(i, slices - 1) * heads + h));
    wt[i] = i < slices ? v.x : -INFINITY;
    mx = fmaxf(mx, wt[i]);
  }
#pragma unroll
  for (int i = 0; i < kPoolAttnSlices; ++i) {
    const float l = ml[2 * ((size_t)min(i, slices - 1) * heads + h) + 1];
    wt[i] = wt[i] == -INFINITY ? 0.0f : expf(wt[i] - mx);  // an empty slice holds no keys
    den = __fmaf_rn(wt[i], l, den);
  }
  const float inv = 1.0f / den;
  for (int d = threadIdx.x; d < Dc; d += 64 * kOutWaves) {
    float part[kPoolAttnSlices], a = 0.0f;
#pragma unroll
    for (int i = 0; i < kPoolAttnSlices; ++i) part[i] = o[((size_t)min(i, slices - 1) * heads + h) * Dc + d];
#pragma unroll
    for (int i = 0; i < kPoolAttnSlices; ++i) a = __fmaf_rn(wt[i], part[i], a);
    s_o[d] = a * inv;
  }
  __syncthreads();
  float acc = 0.0f;
#pragma unroll
  for (int i = 0; i < kAhead; ++i) {
    const int s = wave + kOutWaves * i;
    if (s >= Dc / 16) break;
    const float* x = s_o + 16 * s + 8 * hh;
    const float4 x0 = load4(x), x1 = load4(x + 4);
    const float xs[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
    for (int e = 0; e < 8; ++e) acc = __fmaf_rn(f[i].get(e), xs[e], acc);
  }
  acc += __shfl_xor(acc, 32, 64);
  if (hh == 0) s_part[wave][j] = acc;
  __syncthreads();
  if (threadIdx.x >= 32) return;
  float t = 0.0f;
#pragma unroll
  for (int i = 0; i < kOutWaves; ++i) t += s_part[i][j];
  const int d = 32 * vb + j;
  if (d < vdim) y[(size_t)h * vdim + d] = gate ? t * sigmoid_f(gate[h]) : t;
}

template <typename T>
hipError_t rows_t(const LatentGeom& g, void* k, void* vt, const float* raw, void* cq, int ldq, int M, int pos0,
                  hipStream_t s) {
  const RowsArgs a{g.q_rank, g.kv_rank, g.rot_part, g.rot_dims, g.Dc, g.Dr, g.ldr, g.kv_off, g.rot_off, ldq,
                   g.eps, g.q_norm, g.kv_norm, g.sin_t, g.cos_t};
  const int lead = pos0 & (kRowTok - 1);
  const size_t lds = sizeof(float) * kRowTok * ((g.kv_rank + g.rot_part) | 1);
  hipLaunchKernelGGL(latent_rows_kernel<T>, dim3((M + lead + kRowTok - 1) / kRowTok), dim3(64 * kRowTok), lds, s, raw,
                     static_cast<T*>(cq), static_cast<T*>(k), static_cast<T*>(vt), M, pos0, a);
  return hipGetLastError();
}

template <typename T>
hipError_t absorb_t(const LatentGeom& g, void* k, void* vt, const float* raw, const float* q, const int* pos, float* qa,
                    hipStream_t s) {
  const AbsorbArgs a{g.heads, g.dim, g.D, g.kv_rank, g.rot_part, g.rot_dims, g.rot_rows, g.Dc, g.Dr, g.kv_off, g.rot_off,
                     g.eps, g.kv_norm, g.sin_t, g.cos_t};
  const int fold = (g.heads * (g.Dc / 16) + 3) / 4, rot = (g.heads * g.Dr + 255) / 256;
  hipLaunchKernelGGL(latent_absorb_kernel<T>, dim3(fold + 1 + rot), dim3(256), 0, s, raw, q, static_cast<const T*>(g.k_up),
                     static_cast<T*>(k), static_cast<T*>(vt), pos, qa, fold, a);
  return hipGetLastError();
}

template <int CW>
hipError_t decode_cw(const LatentGeom& g, const void* k, const void* vt, const float* qa, const int* pos, int max_seq,
                     float* o, float* ml, hipStream_t s) {
  constexpr size_t lds = (size_t)8 * (CW + 1) * 1024 + kDecWaves * 4 * 1024 + sizeof(float) * 3 * kDecWaves * 32;
  auto kern = latent_decode_kernel<CW>;
  static LdsLimitOnce raised;
  if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), 80 * 1024); e != hipSuccess) return e;
  hipLaunchKernelGGL(kern, dim3(latent_slices(g.window, max_seq), (g.heads + 31) / 32), dim3(64 * kDecWaves), lds, s,
                     static_cast<const __bf16*>(k), static_cast<const __bf16*>(vt), qa, pos, max_seq, g.heads, g.Dc, g.Dr,
                     g.window, g.scale, g.sinks, o, ml);
  return hipGetLastError();
}

}  // namespace

size_t latent_expand_elems(int heads, int D, int blocks) { return (size_t)heads * D * 32 * blocks; }

int latent_expand_blocks(int window, int max_seq, int max_batch_tokens) {
  // a portion and what its first token sees, at any offset into a block; never more than the cache
  const int tokens = std::min(window, max_seq) + max_batch_tokens;
  return std::min((max_seq + 31) / 32, tokens / 32 + 2);
}

hipError_t launch_latent_rows(int dtype, const LatentGeom& g, void* k, void* vt, const float* raw, void* cq, int ldq, int M,
                              int pos0, hipStream_t s) {
  if (dtype == W4A32_LAYERED_BF16) return rows_t<__bf16>(g, k, vt, raw, cq, ldq, M, pos0, s);
  return rows_t<float>(g, k, vt, raw, cq, ldq, M, pos0, s);
}

hipError_t launch_latent_expand(int dtype, const LatentGeom& g, const void* k, void* ke, void* ve, int nblk, int M, int pos0,
                                hipStream_t s) {
  const int blk0 = std::max(0, pos0 - g.window + 1) / 32, n_blk = (pos0 + M - 1) / 32 - blk0 + 1, rows = g.heads * g.D;
  if (n_blk > nblk) return hipErrorInvalidValue;
  if (dtype == W4A32_LAYERED_BF16) {
    hipLaunchKernelGGL(latent_expand_kernel, dim3((n_blk + 3) / 4, 2 * ((rows + 127) / 128)), dim3(256), 0, s,
                       static_cast<const __bf16*>(k), static_cast<const __bf16*>(g.k_up),
                       static_cast<const __bf16*>(g.v_up), static_cast<__bf16*>(ke), static_cast<__bf16*>(ve), rows, g.D,
                       g.Dc, g.Dr, blk0, n_blk, nblk);
  } else {
    hipLaunchKernelGGL(latent_expand_f32_kernel, dim3(n_blk, 2 * (rows / 32)), dim3(256), 0, s,
                       static_cast<const float*>(k), static_cast<const float*>(g.k_up), static_cast<const float*>(g.v_up),
                       static_cast<float*>(ke), static_cast<float*>(ve), rows, g.D, g.Dc, g.Dr, blk0, nblk);
  }
  return hipGetLastError();
}

hipError_t launch_latent_absorb(int dtype, const LatentGeom& g, void* k, void* vt, const float* raw, const float* q,
                                const int* pos, float* qa, hipStream_t s) {
  if (dtype == W4A32_LAYERED_BF16) return absorb_t<__bf16>(g, k, vt, raw, q, pos, qa, s);
  return absorb_t<float>(g, k, vt, raw, q, pos, qa, s);
}

int latent_slices(int window, int max_seq) {
  const int blocks = (std::min(window, max_seq) + 31) / 32 + 1;  // a window may straddle one more
  return std::min((blocks + 1) / 2, kPoolAttnSlices);
}

hipError_t launch_latent_decode(int dtype, const LatentGeom& g, const void* k, const void* vt, const float* qa,
                                const int* pos, int max_seq, float* o, float* ml, hipStream_t s) {
  if (dtype == W4A32_LAYERED_BF16) {
    switch ((g.Dc / 32 + kDecWaves - 1) / kDecWaves) {
      case 1: return decode_cw<1>(g, k, vt, qa, pos, max_seq, o, ml, s);
      case 2: return decode_cw<2>(g, k, vt, qa, pos, max_seq, o, ml, s);
      case 3: return decode_cw<3>(g, k, vt, qa, pos, max_seq, o, ml, s);
      case 4: return decode_cw<4>(g, k, vt, qa, pos, max_seq, o, ml, s);
      default: return hipErrorInvalidValue;
    }
  }
  hipLaunchKernelGGL(latent_rows_decode_kernel, dim3(latent_slices(g.window, max_seq), g.heads), dim3(256), 0, s,
                     static_cast<const float*>(k), static_cast<const float*>(vt), qa, pos, max_seq, g.heads, g.Dc, g.Dr,
                     g.window, g.scale, g.sinks, o, ml);
  return hipGetLastError();
}

hipError_t launch_latent_out(int dtype, const LatentGeom& g, const float* o, const float* ml, int slices, const float* raw,
                             float* y, hipStream_t s) {
  const dim3 grid(g.heads, (g.vdim + 31) / 32);
  const float* gate = g.gate_off >= 0 ? raw + g.gate_off : nullptr;
  if (dtype == W4A32_LAYERED_BF16) {
    hipLaunchKernelGGL(latent_out_kernel<__bf16>, grid, dim3(64 * kOutWaves), 0, s, o, ml, slices, g.heads,
                       static_cast<const __bf16*>(g.v_up), g.D, g.Dc, g.vdim, gate, y);
  } else {
    hipLaunchKernelGGL(latent_out_kernel<float>, grid, dim3(64 * kOutWaves), 0, s, o, ml, slices, g.heads,
                       static_cast<const float*>(g.v_up), g.D, g.Dc, g.vdim, gate, y);
  }
  return hipGetLastError();
}

}  // namespace w4
