// Attention over a sliding window of tokens and the mean keys / values of the blocks the window has left behind, under
// a common softmax: the query at p attends to tokens (p - window, p] and to a block once its last token is at p - window
// or earlier. No rotation; q, k and v pass a short causal convolution first.
//
// Caches of a layer (element type T, bf16 or f32), per kv head, in blocks of 32 entries laid out as the matrix
// instruction's operands, so that an operand load of a wavefront is one contiguous kilobyte (bf16):
//   keys     [block][dim / 8][entry % 32][dim % 8]
//   values   [block][dim][position], 16 entries of a block at positions 8 (o / 4 % 2) + 4 (o / 8) + o % 4: the order in
//            which the first product leaves the scores in its registers
// The block means have the same two layouts with pooled blocks as entries. D, the dimensions of a row, is 32, 64, 128
// or 256, padding dimensions zero.
//
//   attn_qkv_kernel       a portion's q, k, v rows through the convolution; q to a buffer, k and v to the caches
//   attn_pool_kernel      means of the blocks that the portion completed, from the caches
//   attn_mfma_kernel      prefill, bf16: both products on v_mfma_f32_32x32x16_bf16, transposed (a lane stands for one
//                         query, the online softmax is per lane, scores go from accumulator to operand without a
//                         cross-lane move). The softmax weights stay f32: they enter the second product as a sum of
//                         two bf16 terms.
//   attn_rows_kernel      prefill, f32: one wavefront per (head, query)
//   attn_decode_kernel    one token: convolution, cache append, block mean and attention over one slice of the visible
//                         keys per workgroup; the slices are merged by the Linear that follows
#include <algorithm>

#include "w4a32_attn_blocks.h"
#include "w4a32_layered.h"
#include "w4a32_layered_kernels.h"

namespace w4 {

namespace {

// ---------------------------------------------------------------------------------------------
constexpr int kQkvTok = 8;

// One thread per channel and block of tokens. Blocks are aligned to eight absolute positions so that a value
// channel's eight tokens are one store; the first block also takes the partial one in front of it (so no other
// block's convolution reaches the ring, which this one rewrites at its end).
// ROT: no convolution, q and k are rotated; with `tied` the values are the keys before that.
template <typename T, int TAPS, bool ROT>
__global__ __launch_bounds__(256) void attn_qkv_kernel(const float* __restrict__ raw, int ldr,
                                                       const float* __restrict__ conv, float* __restrict__ ring,
                                                       int ldc, T* __restrict__ q, T* __restrict__ kc,
                                                       T* __restrict__ vt, int heads, int kv_heads, int dim, int vdim,
                                                       int D, int cap, int channels, int M, int pos0, int tied,
                                                       int rot, const float* __restrict__ sin_t,
                                                       const float* __restrict__ cos_t) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= channels) return;
  const int first = 2 * kQkvTok - (pos0 & (kQkvTok - 1));  // end of block 0
  const int t0 = blockIdx.y == 0 ? 0 : first + ((int)blockIdx.y - 1) * kQkvTok;
  const int te = min(M, first + (int)blockIdx.y * kQkvTok);
  float wt[TAPS], win[TAPS];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) wt[j] = conv ? conv[(size_t)j * ldc + c] : 1.0f;
#pragma unroll
  for (int j = 1; j < TAPS; ++j) {
    const int t = t0 - j, p = pos0 + t;
    win[j] = t >= 0 ? raw[(size_t)t * ldr + c] : p >= 0 ? ring[(size_t)(p % TAPS) * ldc + c] : 0.0f;
  }
  const int nq = heads * dim, nk = kv_heads * dim;
  const int kind = c < nq ? 0 : c < nq + nk ? 1 : 2;  // q, k, v
  const int cc = kind == 0 ? c : kind == 1 ? c - nq : c - nq - nk, hd = kind == 2 ? vdim : dim;
  const int head = cc / hd, d = cc - head * hd;
  T* dst = kind == 0 ? q + (size_t)head * D + d : (kind == 1 ? kc : vt) + (size_t)head * cap * D;
  const bool turn = ROT && kind < 2 && d < rot, store_v = kind == 2 || (ROT && tied && kind == 1);
  const int partner = turn ? c + rot_partner(d, rot) - d : c, angle = turn ? (d < rot / 2 ? d : d - rot / 2) : 0;
  T* dst_v = vt + (size_t)head * cap * D;
  for (int tb = t0; tb < te;) {
    // up to the next multiple of eight positions
    const int n = min(te - tb, kQkvTok - ((pos0 + tb) & (kQkvTok - 1)));
    T out[kQkvTok], turned[kQkvTok];  // as projected (and convolved), and rotated
    if constexpr (ROT) {
      float x[kQkvTok], y[kQkvTok], sn[kQkvTok], cs[kQkvTok];
#pragma unroll
      for (int i = 0; i < kQkvTok; ++i) {  // all requested before the first is used
        const int t = tb + min(i, n - 1);
        x[i] = raw[(size_t)t * ldr + c];
        y[i] = raw[(size_t)t * ldr + partner];
        sn[i] = turn ? sin_t[(size_t)(pos0 + t) * (rot / 2) + angle] : 0.0f;
        cs[i] = turn ? cos_t[(size_t)(pos0 + t) * (rot / 2) + angle] : 1.0f;
      }
#pragma unroll
      for (int i = 0; i < kQkvTok; ++i) {
        out[i] = (T)x[i];
        turned[i] = (T)(partner > c ? x[i] * cs[i] - y[i] * sn[i] : x[i] * cs[i] + y[i] * sn[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < kQkvTok; ++i) {
      if (ROT || i >= n) break;
      win[0] = raw[(size_t)(tb + i) * ldr + c];
      float acc = 0.0f;
#pragma unroll
      for (int j = TAPS - 1; j >= 0; --j) acc = __fmaf_rn(wt[TAPS - 1 - j], win[j], acc);
#pragma unroll
      for (int j = TAPS - 1; j >= 1; --j) win[j] = win[j - 1];
      out[i] = (T)acc;
    }
    const int p = pos0 + tb;
    if (store_v && n == kQkvTok) {  // eight values of a dimension: two runs of four
      struct alignas(sizeof(T) * 4) Four { T e[4]; } lo, hi;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        lo.e[i] = out[i];
        hi.e[i] = out[4 + i];
      }
      *reinterpret_cast<Four*>(dst_v + v_at(p, d, D)) = lo;
      *reinterpret_cast<Four*>(dst_v + v_at(p + 4, d, D)) = hi;
    } else if (store_v) {
#pragma unroll
      for (int i = 0; i < kQkvTok; ++i)
        if (i < n) dst_v[v_at(p + i, d, D)] = out[i];
    }
    if (kind < 2) {
#pragma unroll
      for (int i = 0; i < kQkvTok; ++i) {
        if (i >= n) break;
        const T y = ROT ? turned[i] : out[i];
        if (kind == 0) dst[(size_t)(tb + i) * heads * D] = y;
        else dst[k_at(p + i, d, D)] = y;
      }
    }
    tb += n;
  }
  if (conv && blockIdx.y == 0) {
    for (int t = max(0, M - TAPS + 1); t < M; ++t) ring[(size_t)((pos0 + t) % TAPS) * ldc + c] = raw[(size_t)t * ldr + c];
  }
}

// grid (blocks completed, kv heads)
template <typename T>
__global__ __launch_bounds__(256) void attn_pool_kernel(const T* __restrict__ kc, const T* __restrict__ vt,
                                                        T* __restrict__ kp, T* __restrict__ vpt, int dim, int vdim,
                                                        int D, int cap, int capp, int pool, int b0) {
  const int b = b0 + blockIdx.x, g = blockIdx.y;
  for (int it = threadIdx.x; it < dim + vdim; it += 256) {
    const bool is_k = it < dim;
    const int d = is_k ? it : it - dim;
    const T* src = (is_k ? kc : vt) + (size_t)g * cap * D;
    float sum = 0.0f;
#pragma unroll 8
    for (int i = 0; i < pool; ++i) sum += (float)src[is_k ? k_at(b * pool + i, d, D) : v_at(b * pool + i, d, D)];
    T* dst = (is_k ? kp : vpt) + (size_t)g * capp * D;
    dst[is_k ? k_at(b, d, D) : v_at(b, d, D)] = (T)(sum / (float)pool);
  }
}

// ---------------------------------------------------------------------------------------------
constexpr int kMfmaWaves = 4;

// what not every design's attention has
struct PrefillExtra {
  const float* sinks;      // [heads], or null
  const float* gate;       // [M][ldg], a column per head, or null
  int ldg;
  int qld, qstride;        // elements between rows and between heads of q
  int blk0;                // first block that the key and value buffers hold
  // second part of the keys (KR > 0)
  const void* kr;
  size_t kr_block;         // elements between blocks
  int rot_part, rot_dims;
  const float *sin_t, *cos_t;
};

// Workgroup = (head, 32 queries); its wavefronts take the blocks of 32 pooled entries and of 32 tokens round-robin and
// merge through LDS. S^T = K Q^T: A = keys (lane: key l % 32, dims 16 s + 8 (l / 32) ..), B = queries from LDS.
// O^T += V^T P^T: A = values (lane: dim 32 c + l % 32, keys in the order the first product's registers have:
// k-step ks, element e holds key 16 ks + 8 (e / 4) + 4 (l / 32) + e % 4), B = the softmaxed registers.
//
// KR > 0: keys have a second part of 16 KR dimensions, rotated and shared by all heads (latent attention; its first parts
// and values come expanded, blocks from `blk0` on); q is then as projected, [M][qld] with qstride per head, and its second
// part is rotated here.
template <int D, int KR>
__global__ __launch_bounds__(64 * kMfmaWaves) void attn_mfma_kernel(
    const __bf16* __restrict__ q, const __bf16* __restrict__ kc, const __bf16* __restrict__ vt,
    const __bf16* __restrict__ kp, const __bf16* __restrict__ vpt, __bf16* __restrict__ out, int ldo, int M, int heads,
    int kv_heads, int dim, int vdim, int cap, int capp, int window, int pool, int pos0, float scale, const PrefillExtra x) {
  constexpr int KS = D / 16, C = D / 32, R = 16 * C + 2;  // R: floats a lane hands over in the merge
  extern __shared__ __align__(16) uint8_t smem[];
  bf16x8* s_q = reinterpret_cast<bf16x8*>(smem);                              // [KS + KR][64 lanes]
  float* s_merge = reinterpret_cast<float*>(smem + (KS + KR) * 64 * 16);       // [waves - 1][R][64]
  const int h = blockIdx.x, g = h / (heads / kv_heads);
  // the later query blocks see more keys (until the window is full): they start first
  const int qb = (int)gridDim.y - 1 - (int)blockIdx.y;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int j = lane & 31, hh = lane >> 5;

  const int m_q = min(32 * qb + j, M - 1);
  const int p = pos0 + m_q;                              // this lane's query position
  const int p_first = pos0 + 32 * qb, p_last = pos0 + min(32 * qb + 31, M - 1);
  const int nb = pooled_visible(p, window, pool);        // pooled blocks this query sees
  const int nb_last = pooled_visible(p_last, window, pool);
  const int pool_blocks = (nb_last + 31) / 32;
  const int tok_first = max(0, p_first - window + 1) / 32, tok_blocks = p_last / 32 - tok_first + 1;
  const int blocks = pool_blocks + tok_blocks;

  for (int it = threadIdx.x; it < KS * 64; it += 64 * kMfmaWaves) {
    const int s = it >> 6, l = it & 63, d0 = 16 * s + 8 * (l >> 5);
    const __bf16* src = q + (size_t)min(32 * qb + (l & 31), M - 1) * x.qld + (size_t)h * x.qstride + d0;
    bf16x8 v;
    if (KR == 0 || ((x.qstride & 7) == 0 && d0 + 8 <= dim)) {
      v = *reinterpret_cast<const bf16x8*>(src);
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (d0 + e >= dim) v[e] = (__bf16)0.0f;
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = d0 + e < dim ? src[e] : (__bf16)0.0f;
    }
    s_q[it] = v;
  }
  if constexpr (KR > 0) {
    for (int it = threadIdx.x; it < KR * 64; it += 64 * kMfmaWaves) {
      const int s = it >> 6, l = it & 63, d0 = 16 * s + 8 * (l >> 5), m = min(32 * qb + (l & 31), M - 1);
      const __bf16* src = q + (size_t)m * x.qld + (size_t)h * x.qstride + dim;
      bf16x8 v;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int d = d0 + e;
        float y = d < x.rot_part ? (float)src[d] : 0.0f;
        if (d < x.rot_dims)
          y = rotated(y, (float)src[rot_partner(d, x.rot_dims)], d, x.rot_dims, (size_t)(pos0 + m), x.sin_t, x.cos_t);
        v[e] = (__bf16)y;
      }
      s_q[KS * 64 + it] = v;
    }
  }
  __syncthreads();

  constexpr int kBlk = 32 * D;  // elements of a block
  const __bf16* kt = kc + (size_t)g * cap * D + (size_t)(tok_first - x.blk0) * kBlk + 8 * lane;
  const __bf16* kpt = kp + (size_t)g * capp * D + 8 * lane;
  const __bf16* vtt = vt + (size_t)g * cap * D + (size_t)(tok_first - x.blk0) * kBlk + 32 * j + 8 * hh;
  const __bf16* vptt = vpt + (size_t)g * capp * D + 32 * j + 8 * hh;

  f32x16 o[C];
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int v = 0; v < 16; ++v) o[c][v] = 0.0f;
  float run_max = -INFINITY, run_sum = 0.0f;
  if (x.sinks && wave == 0) {  // a term of the denominator without a value
    run_max = x.sinks[h];
    run_sum = 1.0f;
  }

  bf16x8 kop[KS], krop[KR > 0 ? KR : 1];
  auto load_k = [&](int b) {
    const __bf16* src = b < pool_blocks ? kpt + (size_t)b * kBlk : kt + (size_t)(b - pool_blocks) * kBlk;
#pragma unroll
    for (int s = 0; s < KS; ++s) kop[s] = *reinterpret_cast<const bf16x8*>(src + 512 * s);
    if constexpr (KR > 0) {
      const __bf16* rsrc = static_cast<const __bf16*>(x.kr) + (size_t)(tok_first + b - pool_blocks) * x.kr_block + 8 * lane;
#pragma unroll
      for (int s = 0; s < KR; ++s) krop[s] = *reinterpret_cast<const bf16x8*>(rsrc + 512 * s);
    }
  };
  if (wave < blocks) load_k(wave);
  for (int b = wave; b < blocks; b += kMfmaWaves) {
    const bool pooled = b < pool_blocks;
    const int key0 = 32 * (pooled ? b : tok_first + b - pool_blocks);
    bf16x8 vop[C][2];
    {
      const __bf16* src = pooled ? vptt + (size_t)b * kBlk : vtt + (size_t)(b - pool_blocks) * kBlk;
#pragma unroll
      for (int c = 0; c < C; ++c)
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) vop[c][ks] = *reinterpret_cast<const bf16x8*>(src + 1024 * c + 16 * ks);
    }
    f32x16 st, st1;
#pragma unroll
    for (int v = 0; v < 16; ++v) st[v] = st1[v] = 0.0f;
#pragma unroll
    for (int s = 0; s < KS; s += 2) {  // two accumulators take turns
      st = mfma_bf16(kop[s], s_q[s * 64 + lane], st);
      st1 = mfma_bf16(kop[s + 1], s_q[(s + 1) * 64 + lane], st1);
    }
    if constexpr (KR > 0) {
#pragma unroll
      for (int s = 0; s < KR; ++s) {
        if (s & 1) st1 = mfma_bf16(krop[s], s_q[(KS + s) * 64 + lane], st1);
        else st = mfma_bf16(krop[s], s_q[(KS + s) * 64 + lane], st);
      }
    }
    if (b + kMfmaWaves < blocks) load_k(b + kMfmaWaves);
    // the range of this block's keys that the lane's query sees
    const int lo = pooled ? 0 : p - window + 1, hi = pooled ? nb - 1 : p;
    float blk_max = -INFINITY;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int key = key0 + 8 * (v >> 2) + 4 * hh + (v & 3);
      st[v] = key >= lo && key <= hi ? (st[v] + st1[v]) * scale : -INFINITY;
      blk_max = fmaxf(blk_max, st[v]);
    }
    blk_max = fmaxf(blk_max, __shfl_xor(blk_max, 32, 64));
    const float new_max = fmaxf(run_max, blk_max);
    const float corr = run_max == -INFINITY ? 0.0f : __expf(run_max - new_max);
    float psum = 0.0f;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      st[v] = st[v] == -INFINITY ? 0.0f : __expf(st[v] - new_max);
      psum += st[v];
    }
    psum += __shfl_xor(psum, 32, 64);
    run_sum = run_sum * corr + psum;
    run_max = new_max;
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
      for (int v = 0; v < 16; ++v) o[c][v] *= corr;
    // entries past the last one any query sees may hold anything: a zero weight must not meet them
    const int hi_last = pooled ? nb_last - 1 : p_last;
    if (key0 + 31 > hi_last) {
#pragma unroll
      for (int c = 0; c < C; ++c)
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if (key0 + 16 * ks + 8 * (e >> 2) + 4 * hh + (e & 3) > hi_last) vop[c][ks][e] = (__bf16)0.0f;
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 p1, p2;  // the weights as a sum of two bf16 terms
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float x = st[8 * ks + e];
        p1[e] = (__bf16)x;
        p2[e] = (__bf16)(x - (float)p1[e]);
      }
#pragma unroll
      for (int c = 0; c < C; ++c) o[c] = mfma_bf16(vop[c][ks], p2, o[c]);
#pragma unroll
      for (int c = 0; c < C; ++c) o[c] = mfma_bf16(vop[c][ks], p1, o[c]);
    }
  }

  if (wave > 0) {
    float* dst = s_merge + (size_t)(wave - 1) * R * 64 + lane;
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
      for (int v = 0; v < 16; ++v) dst[(16 * c + v) * 64] = o[c][v];
    dst[(R - 2) * 64] = run_max;
    dst[(R - 1) * 64] = run_sum;
  }
  __syncthreads();
  if (wave > 0) return;
  float wmax[kMfmaWaves - 1], total_max = run_max;
#pragma unroll
  for (int w = 0; w < kMfmaWaves - 1; ++w) {
    wmax[w] = s_merge[((size_t)w * R + R - 2) * 64 + lane];
    total_max = fmaxf(total_max, wmax[w]);
  }
  const float own = run_max == -INFINITY ? 0.0f : __expf(run_max - total_max);
  float total = run_sum * own;
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int v = 0; v < 16; ++v) o[c][v] *= own;
#pragma unroll
  for (int w = 0; w < kMfmaWaves - 1; ++w) {
    const float wt = wmax[w] == -INFINITY ? 0.0f : __expf(wmax[w] - total_max);
    const float* src = s_merge + (size_t)w * R * 64 + lane;
    total += src[(R - 1) * 64] * wt;
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
      for (int v = 0; v < 16; ++v) o[c][v] += src[(16 * c + v) * 64] * wt;
  }
  if (32 * qb + j >= M) return;
  float inv = 1.0f / total;  // every query sees its own key
  if (x.gate) inv *= sigmoid_f(x.gate[(size_t)(32 * qb + j) * x.ldg + h]);
  __bf16* row = out + (size_t)(32 * qb + j) * ldo;
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int g4 = 0; g4 < 4; ++g4) {
      const int d = 32 * c + 8 * g4 + 4 * hh;
      const float4 v = make_float4(o[c][4 * g4] * inv, o[c][4 * g4 + 1] * inv, o[c][4 * g4 + 2] * inv,
                                   o[c][4 * g4 + 3] * inv);
      if ((vdim & 3) == 0) {
        if (d < vdim) store4(row + h * vdim + d, v);
      } else {
        const float f[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < vdim) row[h * vdim + d + e] = (__bf16)f[e];
      }
    }
  if (h == heads - 1) {
    for (int c = heads * vdim + hh; c < ldo; c += 2) row[c] = (__bf16)0.0f;
  }
}

// ---------------------------------------------------------------------------------------------
// One wavefront per (head, query), everything f32: a lane per key for the scores, a lane per value dimension for
// the sums.
template <typename T>
__global__ __launch_bounds__(64) void attn_rows_kernel(const T* __restrict__ q, const T* __restrict__ kc,
                                                       const T* __restrict__ vt, const T* __restrict__ kp,
                                                       const T* __restrict__ vpt, T* __restrict__ out, int ldo,
                                                       int heads, int kv_heads, int dim, int vdim, int D, int cap,
                                                       int capp, int window, int pool, int pos0, float scale,
                                                       const PrefillExtra x) {
  __shared__ float s_q[W4A32_LAYERED_MAX_DIM + W4A32_LAYERED_MAX_ROT_PART], s_p[64];
  const int h = blockIdx.x, m = blockIdx.y, lane = threadIdx.x, g = h / (heads / kv_heads);
  const int p = pos0 + m;
  const T* qrow = q + (size_t)m * x.qld + (size_t)h * x.qstride;
  for (int d = lane; d < dim; d += 64) s_q[d] = (float)qrow[d];
  for (int d = lane; d < x.rot_part; d += 64) {
    const T* src = qrow + dim;
    float y = (float)src[d];
    if (d < x.rot_dims) y = rotated(y, (float)src[rot_partner(d, x.rot_dims)], d, x.rot_dims, (size_t)p, x.sin_t, x.cos_t);
    s_q[dim + d] = y;
  }
  constexpr int kPer = W4A32_LAYERED_MAX_DIM / 64;
  float acc[kPer] = {0};
  float run_max = -INFINITY, run_sum = 0.0f;
  if (x.sinks) {
    run_max = x.sinks[h];
    run_sum = 1.0f;
  }
  __syncthreads();
  // entries lo .. hi - 1; the buffers start at block blk0
  auto segment = [&](const T* keys, const T* vals, int lo, int hi, int blk0) {
    const int off = 32 * blk0;
    for (int b = lo; b < hi; b += 64) {
      const int n = min(64, hi - b);
      float s = -INFINITY;
      if (lane < n) {
        s = 0.0f;
        for (int d = 0; d < dim; ++d) s = __fmaf_rn(s_q[d], (float)keys[k_at(b + lane - off, d, D)], s);
        const T* kr = static_cast<const T*>(x.kr) + (size_t)((b + lane) >> 5) * x.kr_block;
        for (int d = 0; d < x.rot_part; ++d) s = __fmaf_rn(s_q[dim + d], (float)kr[k_at((b + lane) & 31, d, 0)], s);
        s *= scale;
      }
      float mx = s;
#pragma unroll
      for (int off = 32; off >= 1; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
      const float new_max = fmaxf(run_max, mx);
      const float corr = run_max == -INFINITY ? 0.0f : expf(run_max - new_max);
      const float w = s == -INFINITY ? 0.0f : expf(s - new_max);
      run_sum = run_sum * corr + wave_sum64(w);
      run_max = new_max;
      __syncthreads();
      s_p[lane] = w;
      __syncthreads();
#pragma unroll
      for (int i = 0; i < kPer; ++i) {
        const int d = lane + 64 * i;
        if (d >= vdim) break;
        float a = acc[i] * corr;
        for (int k = 0; k < n; ++k) a = __fmaf_rn(s_p[k], (float)vals[v_at(b + k - off, d, D)], a);
        acc[i] = a;
      }
    }
  };
  segment(kp + (size_t)g * capp * D, vpt + (size_t)g * capp * D, 0, pooled_visible(p, window, pool), 0);
  segment(kc + (size_t)g * cap * D, vt + (size_t)g * cap * D, max(0, p - window + 1), p + 1, x.blk0);
  const float gate = x.gate ? sigmoid_f(x.gate[(size_t)m * x.ldg + h]) : 1.0f;
  T* row = out + (size_t)m * ldo;
#pragma unroll
  for (int i = 0; i < kPer; ++i) {
    const int d = lane + 64 * i;
    if (d < vdim) row[h * vdim + d] = (T)(acc[i] / run_sum * gate);
  }
  if (h == heads - 1)
    for (int c = heads * vdim + lane; c < ldo; c += 64) row[c] = (T)0.0f;
}

// ---------------------------------------------------------------------------------------------
constexpr int kDecThreads = 512, kDecWaves = kDecThreads / 64;
constexpr int kDecTile = 32 * kDecWaves;  // entries a workgroup scores at a time: a block per wavefront

// grid (slices, kv heads). The blocks of 32 entries that hold visible ones (pooled first, then the window) are dealt to
// the slices in equal runs; a wavefront scores a block, lane (hh, j) half of the dimensions of entry j. Leaves
// o [slice][head][D] (not divided) and ml [slice][head] (max, sum). The token's own key and value are not in the
// cache when the launch starts: the workgroups take them from LDS.
template <typename T, int D>
__global__ __launch_bounds__(kDecThreads) void attn_decode_kernel(
    const float* __restrict__ raw, const float* __restrict__ conv, float* __restrict__ ring, int ldc,
    T* __restrict__ kc, T* __restrict__ vt, T* __restrict__ kp, T* __restrict__ vpt, float* __restrict__ o,
    float* __restrict__ ml, const int* __restrict__ d_pos, int max_seq, int heads, int kv_heads, int dim, int vdim,
    int cap, int capp, int window, int pool, float scale, int taps, int own_kv, int make_pool, int tied, int rot,
    const float* __restrict__ sin_t, const float* __restrict__ cos_t, const float* __restrict__ sinks) {
  constexpr int NC = D / 16;              // 8-dimension pieces of a lane
  constexpr int kGroups = kDecThreads / D;  // groups of threads that sum values, a thread per dimension
  extern __shared__ __align__(16) float sm[];
  const int rep = heads / kv_heads;
  float* s_q = sm;                         // [rep][D]
  float* s_k = s_q + rep * D;              // [D]
  float* s_v = s_k + D;                    // [D]
  float* s_o = s_v + D;                    // [rep][D] running sums
  float* s_s = s_o + rep * D;              // [rep][kDecTile]
  float* s_part = s_s + rep * kDecTile;    // [kGroups][rep][D]
  float* s_m = s_part + kDecThreads * rep;  // [rep][3]: running max, sum, correction
  const int slice = blockIdx.x, g = blockIdx.y, tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, j = lane & 31, hh = lane >> 5;
  const int p = min(*d_pos, max_seq - 1);

  const int nb = pooled_visible(p, window, pool), lo = max(0, p - window + 1);
  const int pool_blocks = (nb + 31) / 32, tok_b0 = lo / 32, blocks = pool_blocks + p / 32 - tok_b0 + 1;
  const int per = (blocks + (int)gridDim.x - 1) / (int)gridDim.x;
  const int b_lo = min(blocks, slice * per), b_hi = min(blocks, b_lo + per);
  T* kb = kc + (size_t)g * cap * D;
  T* vb = vt + (size_t)g * cap * D;
  T* kpb = kp + (size_t)g * capp * D;
  T* vpb = vpt + (size_t)g * capp * D;
  auto block_of = [&](int b, const T* tok, const T* pooled) {
    return b < pool_blocks ? pooled + (size_t)b * 32 * D : tok + (size_t)(tok_b0 + b - pool_blocks) * 32 * D;
  };
  Eight<T> kf[NC];  // this lane's half of its entry's key
  auto load_k = [&](int b) __attribute__((always_inline)) {
    const T* src = block_of(b, kb, kpb) + 8 * lane;
#pragma unroll
    for (int i = 0; i < NC; ++i) kf[i].load(src + 512 * i);
  };
  // convolution of this token's channels: the group's query heads, then the key and the value head (item / D), padding
  // dimensions zero. The first two items of a thread are requested ahead of everything else (loads return in order).
  const int nq = heads * dim, nk = kv_heads * dim;
  const int items = rep * D + (own_kv ? 2 * D : 0);
  auto channel = [&](int it) {
    const int r = it / D, d = it - r * D;
    if (it >= items || d >= (r <= rep ? dim : vdim)) return -1;
    return r < rep ? (g * rep + r) * dim + d : r == rep || tied ? nq + g * dim + d : nq + nk + g * vdim + d;
  };
  constexpr int kAhead = 2, kFastTaps = 4;
  const bool ahead = taps > 0 && taps <= kFastTaps;
  float cx[kAhead], cw[kAhead][kFastTaps], cr[kAhead][kFastTaps];
  if (taps == 0) {  // a rotated channel's partner and angle instead
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int it = tid + kDecThreads * i, r = it / D, d = it - r * D, c = max(channel(it), 0);
      const bool turn = d < rot && r <= rep && it < items;
      const int a = turn ? (d < rot / 2 ? d : d - rot / 2) : 0;
      cx[i] = raw[c];
      cr[i][0] = turn ? raw[c + rot_partner(d, rot) - d] : 0.0f;
      cw[i][0] = turn ? cos_t[(size_t)p * (rot / 2) + a] : 1.0f;
      cw[i][1] = turn ? sin_t[(size_t)p * (rot / 2) + a] : 0.0f;
      if (d < rot / 2) cw[i][1] = -cw[i][1];
    }
  }
  if (ahead) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int c = max(channel(tid + kDecThreads * i), 0);
      cx[i] = raw[c];
#pragma unroll
      for (int j = 0; j < kFastTaps; ++j) {  // tap j back from the token's own
        const int q = p - j;
        cw[i][j] = j < taps ? conv[(size_t)(taps - 1 - j) * ldc + c] : 0.0f;
        cr[i][j] = j > 0 && j < taps && q >= 0 ? ring[(size_t)(q % taps) * ldc + c] : 0.0f;
      }
    }
  }
  __builtin_amdgcn_sched_barrier(0);
  // few blocks: two wavefronts share one, each takes every other head
  const bool pairs = per <= kDecWaves / 2;
  const int wb = pairs ? wave & (kDecWaves / 2 - 1) : wave, r_first = pairs ? wave / (kDecWaves / 2) : 0;
  const int r_step = pairs ? 2 : 1;
  if (b_lo + wb < b_hi) load_k(b_lo + wb);
  // ... and the values this thread sums first: group vg of D threads takes a tile's blocks vg, vg + kGroups, ..; a
  // thread has one dimension
  const int vg = tid / D, vd = tid - vg * D;
  Eight<T> vraw[4];
  auto load_v = [&](int b) __attribute__((always_inline)) {
    const T* src = block_of(b, vb, vpb) + (size_t)vd * 32;
#pragma unroll
    for (int i = 0; i < 4; ++i) vraw[i].load(src + 8 * i);
  };
  if (b_lo + vg < b_hi) load_v(b_lo + vg);

  auto finish = [&](int it, int c, float x, float y) {
    if (c >= 0) {
      const int r = it / D, d = it - r * D;
      if (taps > 0 && slice == 0) ring[(size_t)(p % taps) * ldc + c] = x;
      y = (float)(T)y;
      if (slice == 0) {
        if (r == rep) kb[k_at(p, d, D)] = (T)y;
        if (r == rep + 1) vb[v_at(p, d, D)] = (T)y;
      }
    } else {
      y = 0.0f;
    }
    sm[it] = y;
  };
  if (ahead) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int it = tid + kDecThreads * i;
      float y = 0.0f;
#pragma unroll
      for (int j = kFastTaps - 1; j >= 1; --j) y = __fmaf_rn(cw[i][j], cr[i][j], y);
      if (it < items) finish(it, channel(it), cx[i], __fmaf_rn(cw[i][0], cx[i], y));
    }
  }
  if (taps == 0) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int it = tid + kDecThreads * i;
      if (it < items) finish(it, channel(it), cx[i], cx[i] * cw[i][0] + cr[i][0] * cw[i][1]);
    }
  }
  for (int it = tid + (ahead || taps == 0 ? kAhead * kDecThreads : 0); it < items; it += kDecThreads) {
    const int c = channel(it), r = it / D, d = it - r * D;
    const float x = raw[max(c, 0)];
    const bool turn = c >= 0 && d < rot && r <= rep;
    finish(it, c, x,
           turn ? rotated(x, raw[c + rot_partner(d, rot) - d], d, rot, (size_t)p, sin_t, cos_t)
                : taps > 0 ? conv_step(x, conv, ring, max(c, 0), ldc, taps, p) : x);
  }
  for (int it = tid; it < rep * D; it += kDecThreads) s_o[it] = 0.0f;
  for (int r = tid; r < rep; r += kDecThreads) {
    const bool sink = sinks && slice == 0;  // a term of the denominator without a value
    s_m[3 * r] = sink ? sinks[g * rep + r] : -INFINITY;
    s_m[3 * r + 1] = sink ? 1.0f : 0.0f;
  }
  __syncthreads();

  // the block this token completes; nobody sees it before a later token
  if (make_pool && slice == (int)gridDim.x - 1 && (p + 1) % pool == 0) {
    const int b = p / pool, cached = own_kv ? pool - 1 : pool;
    for (int it = tid; it < dim + vdim; it += kDecThreads) {
      const bool is_k = it < dim;
      const int d = is_k ? it : it - dim;
      float sum = 0.0f;
#pragma unroll 8
      for (int i = 0; i < cached; ++i)
        sum += (float)(is_k ? kb[k_at(b * pool + i, d, D)] : vb[v_at(b * pool + i, d, D)]);
      if (own_kv) sum += is_k ? s_k[d] : s_v[d];
      const T mean = (T)(sum / (float)pool);
      if (is_k) kpb[k_at(b, d, D)] = mean;
      else vpb[v_at(b, d, D)] = mean;
    }
  }

  for (int bt = b_lo; bt < b_hi; bt += kDecWaves) {
    const int n_blocks = min(kDecWaves, b_hi - bt), n_keys = 32 * n_blocks;
    if (wb < n_blocks) {
      const int b = bt + wb;
      const bool pooled = b < pool_blocks;
      const int key = 32 * (pooled ? b : tok_b0 + b - pool_blocks) + j;
      const bool seen = pooled ? key < nb : key >= lo && key <= p;
      if (own_kv && !pooled && key == p) {  // this token's key
#pragma unroll
        for (int i = 0; i < NC; ++i) kf[i].set(load4(s_k + 16 * i + 8 * hh), load4(s_k + 16 * i + 8 * hh + 4));
      }
#pragma unroll 1
      for (int r = r_first; r < rep; r += r_step) {
        const float* qr = s_q + r * D + 8 * hh;
        float s0 = 0.0f, s1 = 0.0f;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
          const float4 q0 = load4(qr + 16 * i), q1 = load4(qr + 16 * i + 4);
          s0 = __fmaf_rn(q0.x, kf[i].get(0), s0);
          s1 = __fmaf_rn(q1.x, kf[i].get(4), s1);
          s0 = __fmaf_rn(q0.y, kf[i].get(1), s0);
          s1 = __fmaf_rn(q1.y, kf[i].get(5), s1);
          s0 = __fmaf_rn(q0.z, kf[i].get(2), s0);
          s1 = __fmaf_rn(q1.z, kf[i].get(6), s1);
          s0 = __fmaf_rn(q0.w, kf[i].get(3), s0);
          s1 = __fmaf_rn(q1.w, kf[i].get(7), s1);
        }
        s0 += s1;
        s0 += __shfl_xor(s0, 32, 64);
        if (hh == 0) s_s[r * kDecTile + 32 * wb + j] = seen ? s0 * scale : -INFINITY;
      }
    }
    if (bt + kDecWaves + wb < b_hi) load_k(bt + kDecWaves + wb);
    __syncthreads();
    // softmax weights of the tile: a wavefront per head
    for (int r = wave; r < rep; r += kDecWaves) {
      float s[kDecTile / 64], mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < kDecTile / 64; ++i) {
        s[i] = lane + 64 * i < n_keys ? s_s[r * kDecTile + lane + 64 * i] : -INFINITY;
        mx = fmaxf(mx, s[i]);
      }
#pragma unroll
      for (int off = 32; off >= 1; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
      const float old = s_m[3 * r], new_max = fmaxf(old, mx);
      float sum = 0.0f;
#pragma unroll
      for (int i = 0; i < kDecTile / 64; ++i) {
        const float w = s[i] == -INFINITY ? 0.0f : expf(s[i] - new_max);
        // weights in the order the values have in memory
        const int k = lane + 64 * i;
        if (k < n_keys) s_s[r * kDecTile + (k & ~31) + v_pos(k & 31)] = w;
        sum += w;
      }
      sum = wave_sum64(sum);
      const float corr = old == -INFINITY ? 0.0f : expf(old - new_max);
      if (lane == 0) {
        s_m[3 * r] = new_max;
        s_m[3 * r + 1] = s_m[3 * r + 1] * corr + sum;
        s_m[3 * r + 2] = corr;
      }
    }
    __syncthreads();
    // values
    {
      for (int r0 = 0; r0 < rep; r0 += 8) {
        float acc[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[i] = 0.0f;
        if (vd < vdim) {
          for (int bi = vg; bi < n_blocks; bi += kGroups) {
            const int b = bt + bi;
            const bool pooled = b < pool_blocks;
            if (bt > b_lo || bi > vg || r0 > 0) load_v(b);
            // entries nobody sees may hold anything: their zero weights must not meet it
            const int e0 = 32 * (pooled ? b : tok_b0 + b - pool_blocks), hi = pooled ? nb - 1 : p;
            const bool edge = e0 + 31 >= hi;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              float v[8];
#pragma unroll
              for (int e = 0; e < 8; ++e) v[e] = vraw[i].get(e);
              if (edge) {
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                  const int key = e0 + 16 * (i >> 1) + 4 * (i & 1) + 8 * (e >> 2) + (e & 3);
                  if (key > hi) v[e] = 0.0f;
                  if (own_kv && !pooled && key == p) v[e] = s_v[vd];
                }
              }
#pragma unroll
              for (int r = 0; r < 8; ++r) {
                if (r0 + r >= rep) break;
                const float* w = s_s + (r0 + r) * kDecTile + 32 * bi + 8 * i;
                const float4 w0 = load4(w), w1 = load4(w + 4);
                acc[r] = __fmaf_rn(w0.x, v[0], acc[r]);
                acc[r] = __fmaf_rn(w0.y, v[1], acc[r]);
                acc[r] = __fmaf_rn(w0.z, v[2], acc[r]);
                acc[r] = __fmaf_rn(w0.w, v[3], acc[r]);
                acc[r] = __fmaf_rn(w1.x, v[4], acc[r]);
                acc[r] = __fmaf_rn(w1.y, v[5], acc[r]);
                acc[r] = __fmaf_rn(w1.z, v[6], acc[r]);
                acc[r] = __fmaf_rn(w1.w, v[7], acc[r]);
              }
            }
          }
        }
#pragma unroll
        for (int r = 0; r < 8; ++r)
          if (r0 + r < rep) s_part[(vg * rep + r0 + r) * D + vd] = acc[r];
      }
    }
    __syncthreads();
    for (int it = tid; it < rep * D; it += kDecThreads) {
      float a = s_o[it] * s_m[3 * (it / D) + 2];
      for (int gi = 0; gi < kGroups; ++gi) a += s_part[gi * rep * D + it];
      s_o[it] = a;
    }
    // the next tile's scores are written behind this tile's weights' last reader, which was before the last barrier
  }
  for (int it = tid; it < rep * D; it += kDecThreads) o[((size_t)slice * heads + g * rep) * D + it] = s_o[it];
  for (int r = tid; r < rep; r += kDecThreads) {
    float* dst = ml + 2 * ((size_t)slice * heads + g * rep + r);
    dst[0] = s_m[3 * r];
    dst[1] = s_m[3 * r + 1];
  }
}

template <typename T>
hipError_t qkv_t(const AttnGeom& g, const AttnMem& m, const float* raw, int ldr, const float* conv, void* q, int M,
                 int pos0, hipStream_t s) {
  const int channels = g.heads * g.dim + (g.own_kv ? g.kv_heads * (g.dim + (g.tied ? 0 : g.vdim)) : 0);
  const int first = 2 * kQkvTok - (pos0 & (kQkvTok - 1));
  const int blocks = M <= first ? 1 : 1 + (M - first + kQkvTok - 1) / kQkvTok;
  const dim3 grid((channels + 255) / 256, blocks);
  if (g.rot_dims > 0 || g.tied) {
    if (g.taps > 0) return hipErrorInvalidValue;
    hipLaunchKernelGGL((attn_qkv_kernel<T, 1, true>), grid, dim3(256), 0, s, raw, ldr, nullptr, nullptr, 0,
                       static_cast<T*>(q), static_cast<T*>(m.k), static_cast<T*>(m.vt), g.heads, g.kv_heads, g.dim, g.vdim,
                       g.D, g.cap, channels, M, pos0, (int)g.tied, g.rot_dims, g.sin_t, g.cos_t);
    return hipGetLastError();
  }
#define W4_QKV(TP)                                                                                                \
  case TP:                                                                                                        \
    hipLaunchKernelGGL((attn_qkv_kernel<T, TP, false>), grid, dim3(256), 0, s, raw, ldr, conv, m.ring, g.ldc,            \
                       static_cast<T*>(q), static_cast<T*>(m.k), static_cast<T*>(m.vt), g.heads, g.kv_heads, g.dim, \
                       g.vdim, g.D, g.cap, channels, M, pos0, 0, 0, nullptr, nullptr);                             \
    break
  switch (g.taps > 0 ? g.taps : 1) {
    W4_QKV(1); W4_QKV(2); W4_QKV(3); W4_QKV(4); W4_QKV(5); W4_QKV(6); W4_QKV(7); W4_QKV(8);
    default: return hipErrorInvalidValue;
  }
#undef W4_QKV
  return hipGetLastError();
}

template <int D, int KR>
hipError_t mfma_d(const AttnGeom& g, const AttnMem& m, const PrefillExtra& x, const void* q, void* out, int ldo, int M,
                  int pos0, hipStream_t s) {
  auto kern = attn_mfma_kernel<D, KR>;
  constexpr size_t lds = (D / 16 + KR) * 64 * 16 + sizeof(float) * (kMfmaWaves - 1) * (D / 2 + 2) * 64;
  static LdsLimitOnce raised;
  if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), lds); e != hipSuccess) return e;
  hipLaunchKernelGGL(kern, dim3(g.heads, (M + 31) / 32), dim3(64 * kMfmaWaves), lds, s, static_cast<const __bf16*>(q),
                     static_cast<const __bf16*>(m.k), static_cast<const __bf16*>(m.vt),
                     static_cast<const __bf16*>(m.kp), static_cast<const __bf16*>(m.vpt), static_cast<__bf16*>(out), ldo,
                     M, g.heads, g.kv_heads, g.dim, g.vdim, g.cap, g.capp, g.window, g.pool, pos0, g.scale, x);
  return hipGetLastError();
}

template <typename T, int D>
hipError_t decode_d(const AttnGeom& g, const AttnMem& m, const float* raw, const float* conv, const int* pos,
                    int max_seq, float* o, float* ml, hipStream_t s) {
  const int rep = g.heads / g.kv_heads;
  const size_t lds = sizeof(float) * ((size_t)2 * rep * D + 2 * D + (size_t)rep * (kDecTile + kDecThreads) + 3 * rep);
  auto kern = attn_decode_kernel<T, D>;
  static LdsLimitOnce raised;
  if (lds > 160 * 1024) return hipErrorInvalidValue;
  if (lds > 64 * 1024)
    if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), 160 * 1024); e != hipSuccess) return e;
  hipLaunchKernelGGL(kern, dim3(attn_slices(g, max_seq), g.kv_heads), dim3(kDecThreads), lds, s, raw, conv,
                     m.ring, g.ldc, static_cast<T*>(m.k), static_cast<T*>(m.vt), static_cast<T*>(m.kp),
                     static_cast<T*>(m.vpt), o, ml, pos, max_seq, g.heads, g.kv_heads, g.dim, g.vdim, g.cap, g.capp,
                     g.window, g.pool, g.scale, g.taps, (int)g.own_kv, (int)g.make_pool, (int)g.tied, g.rot_dims, g.sin_t, g.cos_t,
                     g.sinks);
  return hipGetLastError();
}

template <typename T>
hipError_t decode_t(const AttnGeom& g, const AttnMem& m, const float* raw, const float* conv, const int* pos,
                    int max_seq, float* o, float* ml, hipStream_t s) {
  switch (g.D) {
    case 32: return decode_d<T, 32>(g, m, raw, conv, pos, max_seq, o, ml, s);
    case 64: return decode_d<T, 64>(g, m, raw, conv, pos, max_seq, o, ml, s);
    case 128: return decode_d<T, 128>(g, m, raw, conv, pos, max_seq, o, ml, s);
    case 256: return decode_d<T, 256>(g, m, raw, conv, pos, max_seq, o, ml, s);
    default: return hipErrorInvalidValue;
  }
}

}  // namespace

int attn_slices(const AttnGeom& g, int max_seq) {
  // four blocks of 32 entries a slice, what one pass of the kernel's value threads takes at D = 128; more slices would
  // cost the merge more than they save
  const int blocks = std::min(g.window, max_seq) / 32 + 2 + (g.pool > 0 ? max_seq / g.pool / 32 + 1 : 0);
  return std::min(std::max((blocks + 3) / 4, 4), kPoolAttnSlices);
}

int head_bucket(int d) { return d <= 32 ? 32 : d <= 64 ? 64 : d <= 128 ? 128 : 256; }

hipError_t launch_attn_qkv(int dtype, const AttnGeom& g, const AttnMem& m, const float* raw, int ldr, const float* conv,
                           void* q, int M, int pos0, hipStream_t s) {
  if (dtype == W4A32_LAYERED_BF16) return qkv_t<__bf16>(g, m, raw, ldr, conv, q, M, pos0, s);
  return qkv_t<float>(g, m, raw, ldr, conv, q, M, pos0, s);
}

hipError_t launch_attn_pool(int dtype, const AttnGeom& g, const AttnMem& m, int M, int pos0, hipStream_t s) {
  const int b0 = pos0 / g.pool, b1 = (pos0 + M) / g.pool;  // blocks whose last token lies in the portion
  if (b1 <= b0) return hipSuccess;
  const dim3 grid(b1 - b0, g.kv_heads);
  if (dtype == W4A32_LAYERED_BF16) {
    hipLaunchKernelGGL(attn_pool_kernel<__bf16>, grid, dim3(256), 0, s, static_cast<const __bf16*>(m.k),
                       static_cast<const __bf16*>(m.vt), static_cast<__bf16*>(m.kp), static_cast<__bf16*>(m.vpt), g.dim,
                       g.vdim, g.D, g.cap, g.capp, g.pool, b0);
  } else {
    hipLaunchKernelGGL(attn_pool_kernel<float>, grid, dim3(256), 0, s, static_cast<const float*>(m.k),
                       static_cast<const float*>(m.vt), static_cast<float*>(m.kp), static_cast<float*>(m.vpt), g.dim,
                       g.vdim, g.D, g.cap, g.capp, g.pool, b0);
  }
  return hipGetLastError();
}

template <int KR>
static hipError_t prefill_bf16(const AttnGeom& g, const AttnMem& m, const PrefillExtra& x, const void* q, void* out, int ldo,
                               int M, int pos0, hipStream_t s) {
  switch (g.D) {
    case 32: return mfma_d<32, KR>(g, m, x, q, out, ldo, M, pos0, s);
    case 64: return mfma_d<64, KR>(g, m, x, q, out, ldo, M, pos0, s);
    case 128: return mfma_d<128, KR>(g, m, x, q, out, ldo, M, pos0, s);
    case 256: return mfma_d<256, KR>(g, m, x, q, out, ldo, M, pos0, s);
    default: return hipErrorInvalidValue;
  }
}

static hipError_t prefill_f32(const AttnGeom& g, const AttnMem& m, const PrefillExtra& x, const void* q, void* out, int ldo,
                              int M, int pos0, hipStream_t s) {
  hipLaunchKernelGGL(attn_rows_kernel<float>, dim3(g.heads, M), dim3(64), 0, s, static_cast<const float*>(q),
                     static_cast<const float*>(m.k), static_cast<const float*>(m.vt), static_cast<const float*>(m.kp),
                     static_cast<const float*>(m.vpt), static_cast<float*>(out), ldo, g.heads, g.kv_heads, g.dim, g.vdim,
                     g.D, g.cap, g.capp, g.window, g.pool, pos0, g.scale, x);
  return hipGetLastError();
}

hipError_t launch_attn_prefill(int dtype, const AttnGeom& g, const AttnMem& m, const void* q, void* out, int ldo, int M,
                               int pos0, hipStream_t s) {
  PrefillExtra x{};
  x.sinks = g.sinks;
  x.qld = g.heads * g.D;
  x.qstride = g.D;
  if (dtype == W4A32_LAYERED_BF16) return prefill_bf16<0>(g, m, x, q, out, ldo, M, pos0, s);
  return prefill_f32(g, m, x, q, out, ldo, M, pos0, s);
}

int latent_rot_pad(int rot_part) { return rot_part <= 16 ? 16 : rot_part <= 32 ? 32 : rot_part <= 64 ? 64 : 128; }

hipError_t launch_latent_prefill(int dtype, const LatentGeom& g, const void* k, const void* ke, const void* ve, int nblk,
                                 const void* q, int ldq, const float* raw, void* out, int ldo, int M, int pos0,
                                 hipStream_t s) {
  const size_t elem = dtype == W4A32_LAYERED_BF16 ? 2 : 4;
  AttnGeom a{};  // every head has expanded keys and values of its own
  a.heads = a.kv_heads = g.heads;
  a.dim = g.dim; a.vdim = g.vdim; a.D = g.D;
  a.cap = 32 * nblk; a.capp = 32;
  a.window = g.window;
  a.scale = g.scale;
  const AttnMem m{const_cast<void*>(ke), const_cast<void*>(ve), nullptr, nullptr, nullptr};
  PrefillExtra x{};
  x.sinks = g.sinks;
  x.gate = g.gate_off >= 0 ? raw + g.gate_off : nullptr;
  x.ldg = g.ldr;
  x.qld = ldq;
  x.qstride = g.dim + g.rot_part;
  x.blk0 = std::max(0, pos0 - g.window + 1) / 32;
  x.kr = static_cast<const uint8_t*>(k) + elem * 32 * g.Dc;  // behind a block's latents
  x.kr_block = (size_t)32 * (g.Dc + g.Dr);
  x.rot_part = g.rot_part;
  x.rot_dims = g.rot_dims;
  x.sin_t = g.sin_t;
  x.cos_t = g.cos_t;
  if (dtype != W4A32_LAYERED_BF16) return prefill_f32(a, m, x, q, out, ldo, M, pos0, s);
  switch (g.Dr) {
    case 16: return prefill_bf16<1>(a, m, x, q, out, ldo, M, pos0, s);
    case 32: return prefill_bf16<2>(a, m, x, q, out, ldo, M, pos0, s);
    case 64: return prefill_bf16<4>(a, m, x, q, out, ldo, M, pos0, s);
    case 128: return prefill_bf16<8>(a, m, x, q, out, ldo, M, pos0, s);
    default: return hipErrorInvalidValue;
  }
}

hipError_t launch_attn_decode(int dtype, const AttnGeom& g, const AttnMem& m, const float* raw, const float* conv,
                              const int* pos, int max_seq, float* o, float* ml, hipStream_t s) {
  if (dtype == W4A32_LAYERED_BF16) return decode_t<__bf16>(g, m, raw, conv, pos, max_seq, o, ml, s);
  return decode_t<float>(g, m, raw, conv, pos, max_seq, o, ml, s);
}

}  // namespace w4
