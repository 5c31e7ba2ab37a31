// What a decode Linear does to its input row before it multiplies, and the weights it streams; device code of
// row_linear_kernel (w4a32_lin16.hip) and of the experts' decode kernels (w4a32_moe.hip).
#pragma once

#include "w4a32_layered.h"
#include "w4a32_layered_kernels.h"

namespace w4 {

constexpr int kRowThreads = 512, kRowWaves = kRowThreads / 64;

// Sums over the workgroup of N values per thread, in every thread; s_red holds N * kRowWaves floats.
template <int N>
__device__ __forceinline__ void block_totals(float (&v)[N], float* s_red) {
#pragma unroll
  for (int i = 0; i < N; ++i) {
    v[i] = wave_sum64(v[i]);
    if ((threadIdx.x & 63) == 0) s_red[i * kRowWaves + (threadIdx.x >> 6)] = v[i];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < N; ++i) {
    v[i] = 0.0f;
#pragma unroll
    for (int w = 0; w < kRowWaves; ++w) v[i] += s_red[i * kRowWaves + w];
  }
}

// Mean and 1 / sqrt(variance + eps) of K values, of which each wavefront holds `n` with sum `sum` (this lane's share);
// `spread(mean)` returns the lane's share of the squared deviations from a mean. One barrier: the wavefronts'
// means and squared deviations are combined, which loses no digits to the mean's size.
template <typename Spread>
__device__ __forceinline__ void block_norm_stats(float sum, float n, float K, float eps, Spread spread, float* s_red,
                                                 float* mean_out, float* rstd_out) {
  const float m = n > 0.0f ? wave_sum64(sum) / n : 0.0f;
  const float d = wave_sum64(spread(m));
  if ((threadIdx.x & 63) == 0) {
    const int w = threadIdx.x >> 6;
    s_red[w] = n;
    s_red[kRowWaves + w] = m;
    s_red[2 * kRowWaves + w] = d;
  }
  __syncthreads();
  float mean = 0.0f, dev = 0.0f;
#pragma unroll
  for (int w = 0; w < kRowWaves; ++w) mean = __fmaf_rn(s_red[w], s_red[kRowWaves + w], mean);
  mean /= K;
#pragma unroll
  for (int w = 0; w < kRowWaves; ++w) {
    const float e = s_red[kRowWaves + w] - mean;
    dev += s_red[2 * kRowWaves + w] + s_red[w] * e * e;
  }
  *mean_out = mean;
  *rstd_out = 1.0f / sqrtf(dev / K + eps);
}

// The same outputs for a norm that takes no mean off; `ss`: this lane's share of the squares.
__device__ __forceinline__ void block_rms_stats(float ss, float K, float eps, float* s_red, float* mean_out,
                                                float* rstd_out) {
  float t[1] = {ss};
  block_totals(t, s_red);
  *mean_out = 0.0f;
  *rstd_out = 1.0f / sqrtf(t[0] / K + eps);
}

// The row a decode Linear multiplies, into s_x [Kp] (zeros past K), by 512 threads. Each kind comes in two steps, what it
// requests from memory and what it makes of that: a CU's loads return in the order they were issued, so the
// row's inputs are requested in front of the first weights and the arithmetic runs while those arrive. Rows that
// do not fit one step's registers are read in the second one.
constexpr int kFastTaps = 4;  // input convolutions up to this length are requested ahead

struct NormRegs {
  bool fast;
  int pos;
  f32x4 x, w, cw[kFastTaps], rg[kFastTaps];
};

__device__ __forceinline__ f32x4 load_row4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 load_row4(const __bf16* p) {
  const float4 v = load4(p);
  return f32x4{v.x, v.y, v.z, v.w};
}
__device__ __forceinline__ void store_row4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }

template <typename WT>
__device__ __forceinline__ const WT* token_row(const RowPrologue& p, int Kp) {
  if (!p.token) return nullptr;
  const int64_t id = *p.token;
  return static_cast<const WT*>(p.table) + (size_t)(id < 0 ? 0 : id >= p.vocab ? p.vocab - 1 : id) * Kp;
}

template <typename WT>
__device__ __forceinline__ f32x4 norm_input(const RowPrologue& p, const WT* trow, int c) {
  f32x4 v = trow ? load_row4(trow + c) : load_row4(p.x + c);
  for (int i = 0; i < p.n_parts; ++i) v += load_row4(p.parts + i * p.part_stride + c) * p.part_scale;
  return v;
}

template <typename WT>
__device__ __forceinline__ void row_norm_request(const RowPrologue& p, int Kp, NormRegs& r) {
  r.fast = Kp <= 4 * kRowThreads && p.taps <= kFastTaps;
  r.pos = p.taps > 0 ? *p.pos : 0;
  if (!r.fast) return;
  const int c = min(4 * (int)threadIdx.x, Kp - 4);
  r.x = norm_input(p, token_row<WT>(p, Kp), c);
  r.w = load_row4(p.norm_w + c);
#pragma unroll
  for (int j = 0; j < kFastTaps; ++j) {
    r.cw[j] = r.rg[j] = f32x4{0, 0, 0, 0};
    if (j < p.taps) {
      r.cw[j] = load_row4(p.conv + (size_t)j * Kp + c);
      const int q = r.pos - p.taps + 1 + j;
      if (q >= 0 && q < r.pos) r.rg[j] = load_row4(p.ring + (size_t)(q % p.taps) * Kp + c);
    }
  }
}

template <typename WT>
__device__ __forceinline__ void row_norm(const RowPrologue& p, int Kp, const NormRegs& r, float* s_x, float* s_red) {
  const bool first_wg = blockIdx.x == 0;
  const int c0 = 4 * threadIdx.x;
  float mean, rstd;
  if (r.fast) {
    // one vector per thread
    f32x4 x = r.x;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (c0 + e >= p.K) x[e] = 0.0f;
    const int w0 = 4 * ((int)threadIdx.x & ~63);  // the wavefront's columns
    if (p.rms) {
      block_rms_stats((x[0] * x[0] + x[1] * x[1]) + (x[2] * x[2] + x[3] * x[3]), (float)p.K, p.eps, s_red, &mean, &rstd);
    } else block_norm_stats((x[0] + x[1]) + (x[2] + x[3]), (float)min(max(p.K - w0, 0), 256), (float)p.K, p.eps,
                     [&](float m) {
                       float ss = 0.0f;
#pragma unroll
                       for (int e = 0; e < 4; ++e) {
                         const float d = c0 + e < p.K ? x[e] - m : 0.0f;
                         ss += d * d;
                       }
                       return ss;
                     },
                     s_red, &mean, &rstd);
    if (c0 < Kp) {
      if (p.x_out && first_wg) store_row4(p.x_out + c0, x);
      const f32x4 h = (x - mean) * rstd * r.w;
      if (p.taps > 0 && first_wg) store_row4(p.ring + (size_t)(r.pos % p.taps) * Kp + c0, h);
      f32x4 y = h;
#pragma unroll
      for (int j = 0; j < kFastTaps; ++j) y += r.cw[j] * (j == p.taps - 1 ? h : r.rg[j]);
      store_row4(s_x + c0, y);
    }
    return;
  }
  const WT* trow = token_row<WT>(p, Kp);
  float sum = 0.0f, count = 0.0f;
  for (int c = c0; c < Kp; c += 4 * kRowThreads) {
    f32x4 v = norm_input(p, trow, c);
    count += (float)min(max(p.K - (c & ~255), 0), 256);
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (c + e >= p.K) v[e] = 0.0f;
    store_row4(s_x + c, v);
    sum += p.rms ? (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]) : (v[0] + v[1]) + (v[2] + v[3]);
  }
  if (p.rms) block_rms_stats(sum, (float)p.K, p.eps, s_red, &mean, &rstd);
  // (a wavefront whose last columns lie past Kp counts in its first lane's terms: they cover the whole wavefront)
  else block_norm_stats(sum, __shfl(count, 0, 64), (float)p.K, p.eps,
                   [&](float m) {
                     float ss = 0.0f;
                     for (int c = c0; c < Kp; c += 4 * kRowThreads) {
                       const f32x4 v = load_row4(s_x + c);
#pragma unroll
                       for (int e = 0; e < 4; ++e) {
                         const float d = c + e < p.K ? v[e] - m : 0.0f;
                         ss += d * d;
                       }
                     }
                     return ss;
                   },
                   s_red, &mean, &rstd);
  for (int c = c0; c < Kp; c += 4 * kRowThreads) {
    const f32x4 v = load_row4(s_x + c);
    if (p.x_out && first_wg) store_row4(p.x_out + c, v);
    const f32x4 h = (v - mean) * rstd * load_row4(p.norm_w + c);
    if (p.taps > 0 && first_wg) store_row4(p.ring + (size_t)(r.pos % p.taps) * Kp + c, h);
    f32x4 y = h;
    for (int j = 0; j < p.taps; ++j) {
      const int q = r.pos - p.taps + 1 + j;
      if (q < 0) continue;
      y += load_row4(p.conv + (size_t)j * Kp + c) * (q == r.pos ? h : load_row4(p.ring + (size_t)(q % p.taps) * Kp + c));
    }
    store_row4(s_x + c, y);
  }
}

struct MergeRegs {
  bool fast;
  int head;
  f32x4 part[kPoolAttnSlices];
};

__device__ __forceinline__ void row_merge_request(const RowPrologue& p, int Kp, MergeRegs& r) {
  r.fast = (p.vdim & 3) == 0 && Kp <= 4 * kRowThreads;
  if (!r.fast) return;
  const int c = min(4 * (int)threadIdx.x, p.K - 4);
  r.head = c / p.vdim;
  const float* src = p.o + (size_t)r.head * p.dvp + (c - r.head * p.vdim);
#pragma unroll
  for (int i = 0; i < kPoolAttnSlices; ++i)
    r.part[i] = load_row4(src + (size_t)min(i, p.slices - 1) * p.heads * p.dvp);
}

// s_w: [kPoolAttnSlices][heads], the slices' weights (behind the row)
__device__ __forceinline__ void row_merge(const RowPrologue& p, int Kp, const MergeRegs& r, float* s_x, float* s_w) {
  for (int h = threadIdx.x; h < p.heads; h += kRowThreads) {
    float m[kPoolAttnSlices], l[kPoolAttnSlices], mx = -INFINITY, den = 0.0f;
#pragma unroll
    for (int i = 0; i < kPoolAttnSlices; ++i) {
      const float2 ml = *reinterpret_cast<const float2*>(p.ml + 2 * ((size_t)min(i, p.slices - 1) * p.heads + h));
      m[i] = i < p.slices ? ml.x : -INFINITY;
      l[i] = ml.y;
      mx = fmaxf(mx, m[i]);
    }
#pragma unroll
    for (int i = 0; i < kPoolAttnSlices; ++i) {
      m[i] = m[i] == -INFINITY ? 0.0f : expf(m[i] - mx);  // an empty slice holds no keys
      den = __fmaf_rn(m[i], l[i], den);
    }
    const float inv = 1.0f / den;  // the token's own key is always seen
#pragma unroll
    for (int i = 0; i < kPoolAttnSlices; ++i) s_w[i * p.heads + h] = m[i] * inv;
  }
  __syncthreads();
  if (r.fast) {
    const int c = 4 * threadIdx.x;
    f32x4 y = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < kPoolAttnSlices; ++i) y += r.part[i] * s_w[i * p.heads + r.head];
    if (c < Kp) store_row4(s_x + c, c < p.K ? y : f32x4{0, 0, 0, 0});
    return;
  }
  const size_t stride = (size_t)p.heads * p.dvp;
  for (int c = threadIdx.x; c < Kp; c += kRowThreads) {
    float y = 0.0f;
    if (c < p.K) {
      const int h = c / p.vdim, d = c - h * p.vdim;
      for (int i = 0; i < p.slices; ++i)
        y = __fmaf_rn(s_w[i * p.heads + h], p.o[i * stride + (size_t)h * p.dvp + d], y);
    }
    s_x[c] = y;
  }
}

// a wavefront takes whole heads
__device__ __forceinline__ void row_gated(const RowPrologue& p, int Kp, float* s_x) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  for (int h = wave; h < p.heads; h += kRowWaves) {
    constexpr int kPer = W4A32_LAYERED_MAX_DIM / 64;
    float v[kPer], g[kPer], w[kPer], ss = 0.0f;
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
      const int d = lane + 64 * i;
      v[i] = g[i] = w[i] = 0.0f;
      if (d < p.vdim) {
        v[i] = p.o[h * p.vdim + d];
        g[i] = p.gate[h * p.vdim + d];
        w[i] = p.head_w ? p.head_w[d] : 1.0f;
      }
      ss += v[i] * v[i];
    }
    const float r = 1.0f / sqrtf(wave_sum64(ss) / (float)p.vdim + p.eps);
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
      const int d = lane + 64 * i;
      if (d < p.vdim) s_x[h * p.vdim + d] = v[i] * r * w[i] * silu_f(g[i]);
    }
  }
  for (int c = p.K + threadIdx.x; c < Kp; c += kRowThreads) s_x[c] = 0.0f;
}

constexpr int kPolyRegs = 5;
struct PolyRegs {
  f32x4 z[kPolyRegs];
};

__device__ __forceinline__ void row_poly_request(const RowPrologue& p, int Kp, PolyRegs& r) {
#pragma unroll
  for (int i = 0; i < kPolyRegs; ++i) r.z[i] = load_row4(p.x + min(4 * ((int)threadIdx.x + kRowThreads * i), Kp - 4));
}

__device__ __forceinline__ void row_poly(const RowPrologue& p, int Kp, const PolyRegs& r, float* s_x, float* s_red) {
  float t[3] = {0.0f, 0.0f, 0.0f};
  auto take = [&](int c, f32x4 z) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (c + e >= p.K) z[e] = 0.0f;
      const float q = z[e] * z[e];
      t[0] += q;
      t[1] = __fmaf_rn(q, q, t[1]);
      t[2] = __fmaf_rn(q * q, q, t[2]);
    }
    if (c < Kp) store_row4(s_x + c, z);
  };
#pragma unroll
  for (int i = 0; i < kPolyRegs; ++i) take(4 * ((int)threadIdx.x + kRowThreads * i), r.z[i]);
  for (int c = 4 * ((int)threadIdx.x + kRowThreads * kPolyRegs); c < Kp; c += 4 * kRowThreads) take(c, load_row4(p.x + c));
  block_totals(t, s_red);
  const float inv = 1.0f / (float)p.K, e0 = p.act[3];
  const float r1 = p.act[0] / sqrtf(t[0] * inv + p.eps);
  const float r2 = p.act[1] / sqrtf(t[1] * inv + p.eps);
  const float r3 = p.act[2] / sqrtf(t[2] * inv + p.eps);
  for (int c = 4 * threadIdx.x; c < Kp; c += 4 * kRowThreads) {  // the elements this thread wrote
    f32x4 z = load_row4(s_x + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) z[e] = c + e < p.K ? z[e] * (r1 + z[e] * (r2 + z[e] * r3)) + e0 : 0.0f;
    store_row4(s_x + c, z);
  }
}

constexpr int kPlainRegs = 4;
struct PlainRegs {
  f32x4 x[kPlainRegs];
};

__device__ __forceinline__ void row_plain_request(const RowPrologue& p, int Kp, PlainRegs& r) {
#pragma unroll
  for (int i = 0; i < kPlainRegs; ++i) r.x[i] = load_row4(p.x + min(4 * ((int)threadIdx.x + kRowThreads * i), Kp - 4));
}

__device__ __forceinline__ void row_plain(const RowPrologue& p, int Kp, const PlainRegs& r, float* s_x) {
#pragma unroll
  for (int i = 0; i < kPlainRegs; ++i) {
    const int c = 4 * ((int)threadIdx.x + kRowThreads * i);
    if (c < Kp) store_row4(s_x + c, r.x[i]);
  }
  for (int c = 4 * ((int)threadIdx.x + kRowThreads * kPlainRegs); c < Kp; c += 4 * kRowThreads)
    store_row4(s_x + c, load_row4(p.x + c));
}

// [residual row, embedding row], Kp / 2 columns each
template <typename WT>
__device__ __forceinline__ void row_loop(const RowPrologue& p, int Kp, float* s_x) {
  const int Hp = Kp / 2;
  const WT* trow = token_row<WT>(p, Hp);
  for (int c = 4 * threadIdx.x; c < Hp; c += 4 * kRowThreads) {
    store_row4(s_x + c, norm_input(p, p.x ? static_cast<const WT*>(nullptr) : trow, c));
    store_row4(s_x + Hp + c, load_row4(trow + c));
  }
}

// The row of kind kKind into s_x; `first_weights` issues the caller's first loads of weights. The caller's barrier ends it.
template <typename WT, int kKind, typename FirstWeights>
__device__ __forceinline__ void row_prologue(const RowPrologue& p, int Kp, float* s_x, float* s_red,
                                             FirstWeights first_weights) {
  if constexpr (kKind == kRowNorm) {
    NormRegs regs;
    row_norm_request<WT>(p, Kp, regs);
    first_weights();
    row_norm<WT>(p, Kp, regs, s_x, s_red);
  }
  if constexpr (kKind == kRowMerge) {
    MergeRegs regs;
    row_merge_request(p, Kp, regs);
    first_weights();
    row_merge(p, Kp, regs, s_x, s_x + Kp);
  }
  if constexpr (kKind == kRowGated) {
    first_weights();
    row_gated(p, Kp, s_x);
  }
  if constexpr (kKind == kRowPoly) {
    PolyRegs regs;
    row_poly_request(p, Kp, regs);
    first_weights();
    row_poly(p, Kp, regs, s_x, s_red);
  }
  if constexpr (kKind == kRowPlain) {
    PlainRegs regs;
    row_plain_request(p, Kp, regs);
    first_weights();
    row_plain(p, Kp, regs, s_x);
  }
  if constexpr (kKind == kRowLoop) {
    first_weights();
    row_loop<WT>(p, Kp, s_x);
  }
}

// eight consecutive weights as they come from memory
template <typename WT>
struct Raw;
template <>
struct Raw<__bf16> {
  uint4 v;
  __device__ __forceinline__ void load(const __bf16* p) { v = *reinterpret_cast<const uint4*>(p); }
  __device__ __forceinline__ float get(int e) const {
    const uint32_t w = e < 2 ? v.x : e < 4 ? v.y : e < 6 ? v.z : v.w;
    return __uint_as_float(e & 1 ? w & 0xFFFF0000u : w << 16);
  }
};
template <>
struct Raw<float> {
  float4 a, b;
  __device__ __forceinline__ void load(const float* p) {
    a = load4(p);
    b = load4(p + 4);
  }
  __device__ __forceinline__ float get(int e) const {
    const float f[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
    return f[e];
  }
};

// R rows of weights at a time per wavefront, lane l multiplies k = 512 i + 8 l .. + 7; U steps of i are in flight while the
// previous U are multiplied. ptr(g, r, k): where row r of group g has its elements k .. k + 7 (k a multiple of 8 below Kp).
template <typename WT, int R, int U, typename Ptr>
__device__ __forceinline__ void fetch_rows(Raw<WT> (&raw)[R][U], int g, int bt, int Kp, Ptr ptr) {
  const int lane = threadIdx.x & 63;
#pragma unroll
  for (int r = 0; r < R; ++r)
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = 512 * (bt * U + u) + 8 * lane;
      raw[r][u].load(ptr(g, r, k < Kp ? k : 0));
    }
}

// Groups gw, gw + nw, .. of `groups`; `cur` holds the first batch of group gw. emit(g, sums) with every lane's copy of the
// R products with the row s_x.
template <typename WT, int R, int U, typename Ptr, typename Emit>
__device__ __forceinline__ void stream_rows(Raw<WT> (&cur)[R][U], int gw, int nw, int groups, int Kp, const float* s_x,
                                            Ptr ptr, Emit emit) {
  const int lane = threadIdx.x & 63;
  const int steps = (Kp + 511) / 512, batches = (steps + U - 1) / U;
  for (int g = gw; g < groups; g += nw) {
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.0f;
    for (int bt = 0; bt < batches; ++bt) {
      Raw<WT> nxt[R][U];
      const bool last = bt + 1 == batches;
      const int gn = last ? g + nw : g;
      if (gn < groups) {
        fetch_rows<WT, R, U>(nxt, gn, last ? 0 : bt + 1, Kp, ptr);
      } else {
#pragma unroll
        for (int r = 0; r < R; ++r)
#pragma unroll
          for (int u = 0; u < U; ++u) nxt[r][u] = cur[r][u];
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = 512 * (bt * U + u) + 8 * lane;
        if (k < Kp) {
          const float4 x0 = load4(s_x + k), x1 = load4(s_x + k + 4);
          const float xs[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
          for (int r = 0; r < R; ++r)
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[r] = __fmaf_rn(cur[r][u].get(e), xs[e], acc[r]);
        }
      }
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int u = 0; u < U; ++u) cur[r][u] = nxt[r][u];
    }
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = wave_sum64(acc[r]);
    emit(g, acc);
  }
}

}  // namespace w4
