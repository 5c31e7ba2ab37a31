// Row operators of the layered decoder's prefill: embedding, layer norm with the input convolution, short
// convolutions with a tail per sequence, PolyNorm, and the rotation table. All bound by HBM.
//
// Convolution tails: a sequence keeps the last inputs of every convolution in a ring of `taps` rows, the row of
// position p in slot p % taps; positions before 0 count as zeros, so a new sequence needs no clearing. In a launch of
// many workgroups only the one that reads the ring (the portion's first tokens) writes it, after its reads.
#include <algorithm>

#include "w4a32_layered.h"
#include "w4a32_layered_kernels.h"

namespace w4 {

namespace {

__global__ __launch_bounds__(256) void fill_zero_kernel(uint4* p, size_t n) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256)
    p[i] = make_uint4(0, 0, 0, 0);
}

template <typename WT>
__global__ __launch_bounds__(256) void embed_rows_kernel(const int64_t* __restrict__ ids, const WT* __restrict__ table,
                                                         float* __restrict__ x, int ld, int vocab) {
  const int64_t id = ids[blockIdx.x];
  const WT* src = table + (size_t)(id < 0 ? 0 : id >= vocab ? vocab - 1 : id) * ld;
  float* dst = x + (size_t)blockIdx.x * ld;
  for (int c = 4 * threadIdx.x; c < ld; c += 1024) store4(dst + c, load4(src + c));
}

// Layer norm (or the norm that takes no mean off) of one row by one wavefront: x + scale * parts -> LDS row s_h (h, zeros past H). The completed residual row goes to
// x_out when that is given. Rows of up to 2048 channels stay in registers on the way.
__device__ __forceinline__ void wave_layer_norm(const float* __restrict__ x, const float* __restrict__ parts,
                                                int n_parts, size_t part_stride, float* __restrict__ x_out,
                                                const float* __restrict__ w, const NormSpec& spec, int H, int ld,
                                                float* __restrict__ s_h) {
  const int lane = threadIdx.x & 63;
  const float inv = 1.0f / (float)H, eps = spec.eps, ps = spec.part_scale;
  auto add = [ps](float4& v, const float4& d) { v.x += ps * d.x; v.y += ps * d.y; v.z += ps * d.z; v.w += ps * d.w; };
  auto clip = [&](float4& v, int c) {
    if (c + 3 >= H) {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e >= H) at4(v, e) = 0.0f;
    }
  };
  auto square = [&](float4 v, int c, float mean) {
    float ss = 0.0f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float d = c + e < H ? at4(v, e) - mean : 0.0f;
      ss = __fmaf_rn(d, d, ss);
    }
    return ss;
  };
  constexpr int kRegs = 8;
  if (ld <= 256 * kRegs) {
    // columns past the row are read from its end and count as zeros
    float4 v[kRegs];
#pragma unroll
    for (int i = 0; i < kRegs; ++i) v[i] = load4(x + min(4 * lane + 256 * i, ld - 4));
    float4 ww[kRegs];
#pragma unroll
    for (int i = 0; i < kRegs; ++i) ww[i] = load4(w + min(4 * lane + 256 * i, ld - 4));
#pragma unroll 2
    for (int p = 0; p < n_parts; ++p) {
      float4 d[kRegs];
#pragma unroll
      for (int i = 0; i < kRegs; ++i) d[i] = load4(parts + p * part_stride + min(4 * lane + 256 * i, ld - 4));
#pragma unroll
      for (int i = 0; i < kRegs; ++i) add(v[i], d[i]);
    }
    float sum = 0.0f;
#pragma unroll
    for (int i = 0; i < kRegs; ++i) {
      const int c = 4 * lane + 256 * i;
      clip(v[i], c);
      if (x_out && c < ld) store4(x_out + c, v[i]);
      sum += (v[i].x + v[i].y) + (v[i].z + v[i].w);
    }
    const float mean = spec.rms ? 0.0f : wave_sum64(sum) * inv;
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < kRegs; ++i) ss += square(v[i], 4 * lane + 256 * i, mean);
    const float rstd = 1.0f / sqrtf(wave_sum64(ss) * inv + eps);
#pragma unroll
    for (int i = 0; i < kRegs; ++i) {
      const int c = 4 * lane + 256 * i;
      if (c >= ld) continue;
      store4(s_h + c, make_float4((v[i].x - mean) * rstd * ww[i].x, (v[i].y - mean) * rstd * ww[i].y,
                                  (v[i].z - mean) * rstd * ww[i].z, (v[i].w - mean) * rstd * ww[i].w));
    }
    return;
  }
  float sum = 0.0f;
  for (int c = 4 * lane; c < ld; c += 256) {
    float4 v = load4(x + c);
    for (int i = 0; i < n_parts; ++i) add(v, load4(parts + i * part_stride + c));
    clip(v, c);
    if (x_out) store4(x_out + c, v);
    store4(s_h + c, v);
    sum += (v.x + v.y) + (v.z + v.w);
  }
  const float mean = spec.rms ? 0.0f : wave_sum64(sum) * inv;
  float ss = 0.0f;
  for (int c = 4 * lane; c < ld; c += 256) ss += square(load4(s_h + c), c, mean);  // the elements this lane wrote
  const float rstd = 1.0f / sqrtf(wave_sum64(ss) * inv + eps);
  for (int c = 4 * lane; c < ld; c += 256) {
    const float4 v = load4(s_h + c), ww = load4(w + c);
    store4(s_h + c, make_float4((v.x - mean) * rstd * ww.x, (v.y - mean) * rstd * ww.y, (v.z - mean) * rstd * ww.z,
                                (v.w - mean) * rstd * ww.w));
  }
}

constexpr int kNcWaves = 8;

// A workgroup normalises the rows t0 - (TAPS - 1) .. t0 + TR - 1 into LDS, a wavefront per row (rows before the portion
// come from the ring), and convolves its TR rows from there.
template <int TAPS, typename YT>
__global__ __launch_bounds__(64 * kNcWaves) void norm_conv_kernel(
    const float* __restrict__ x, const float* __restrict__ parts, int n_parts, float* __restrict__ x_out,
    const float* __restrict__ norm_w, NormSpec spec, const float* __restrict__ conv, float* __restrict__ ring, int M, int H,
    int ld, int pos0, int TR, YT* __restrict__ y) {
  extern __shared__ __align__(16) float s_h[];  // [halo + TR][ld]
  constexpr int halo = TAPS > 0 ? TAPS - 1 : 0, kRing = TAPS > 0 ? TAPS : 1;
  const int t0 = blockIdx.x * TR, rows = min(TR, M - t0);
  const int wave = threadIdx.x >> 6;
  float4 w[kRing];  // this thread's first columns of the convolution, requested early
#pragma unroll
  for (int j = 0; j < TAPS; ++j) w[j] = load4(conv + (size_t)j * ld + min(4 * (int)threadIdx.x, ld - 4));
  for (int r = wave; r < halo + rows; r += kNcWaves) {
    const int t = t0 - halo + r;
    float* dst = s_h + (size_t)r * ld;
    if (t >= 0) {
      wave_layer_norm(x + (size_t)t * ld, parts + (size_t)t * ld, n_parts, (size_t)M * ld,
                      x_out && r >= halo ? x_out + (size_t)t * ld : nullptr, norm_w, spec, H, ld, dst);
    } else {
      const int q = pos0 + t;
      for (int c = 4 * (threadIdx.x & 63); c < ld; c += 256)
        store4(dst + c, q >= 0 ? load4(ring + (size_t)(q % kRing) * ld + c) : make_float4(0, 0, 0, 0));
    }
  }
  __syncthreads();
  for (int c = 4 * threadIdx.x; c < ld; c += 256 * kNcWaves) {
    float4 win[kRing];  // win[j]: h of the position j before the current one
    if (c >= 256 * kNcWaves) {
#pragma unroll
      for (int j = 0; j < TAPS; ++j) w[j] = load4(conv + (size_t)j * ld + c);
    }
#pragma unroll
    for (int j = 1; j < TAPS; ++j) win[j] = load4(s_h + (size_t)(halo - j) * ld + c);
    for (int r = 0; r < rows; ++r) {
      win[0] = load4(s_h + (size_t)(halo + r) * ld + c);
      float4 v = win[0];
#pragma unroll
      for (int j = TAPS - 1; j >= 0; --j) {
        v.x = __fmaf_rn(w[TAPS - 1 - j].x, win[j].x, v.x);
        v.y = __fmaf_rn(w[TAPS - 1 - j].y, win[j].y, v.y);
        v.z = __fmaf_rn(w[TAPS - 1 - j].z, win[j].z, v.z);
        v.w = __fmaf_rn(w[TAPS - 1 - j].w, win[j].w, v.w);
      }
#pragma unroll
      for (int j = TAPS - 1; j >= 1; --j) win[j] = win[j - 1];
      store4(y + (size_t)(t0 + r) * ld + c, v);
    }
  }
  if (blockIdx.x != 0 || TAPS < 2) return;
  // the tail for the next portion: this workgroup has read the ring, nobody else does
  __syncthreads();
  for (int t = max(0, M - halo) + wave; t < M; t += kNcWaves) {
    // rows past this workgroup's own are normalised once more, into an LDS row in front of its own ones (a wavefront
    // that has one is below `halo`)
    float* row = s_h + (size_t)(halo + t) * ld;
    if (t >= rows) {
      row = s_h + (size_t)wave * ld;
      wave_layer_norm(x + (size_t)t * ld, parts + (size_t)t * ld, n_parts, (size_t)M * ld, nullptr, norm_w, spec, H, ld,
                      row);
    }
    float* dst = ring + (size_t)((pos0 + t) % kRing) * ld;
    for (int c = 4 * (threadIdx.x & 63); c < ld; c += 256) store4(dst + c, load4(row + c));
  }
}
static_assert(kNcWaves >= W4A32_LAYERED_MAX_TAPS - 1, "a wavefront per row of the tail");

template <typename YT>
__global__ __launch_bounds__(64) void norm_want_kernel(const float* __restrict__ x, const float* __restrict__ parts,
                                                       int n_parts, const float* __restrict__ norm_w,
                                                       NormSpec spec, const int* __restrict__ want, int M, int H, int ld,
                                                       YT* __restrict__ y) {
  extern __shared__ __align__(16) float s_h[];
  const int t = min(max(want[blockIdx.x], 0), M - 1);
  wave_layer_norm(x + (size_t)t * ld, parts + (size_t)t * ld, n_parts, (size_t)M * ld, nullptr, norm_w, spec, H, ld,
                  s_h);
  for (int c = 4 * threadIdx.x; c < ld; c += 256) store4(y + (size_t)blockIdx.x * ld + c, load4(s_h + c));
}

__global__ __launch_bounds__(256) void add_parts_kernel(const float* x, const float* __restrict__ parts,
                                                        int n_parts, float scale, float* out, size_t n) {
  const size_t i = 4 * ((size_t)blockIdx.x * 256 + threadIdx.x);
  if (i >= n) return;
  float4 v = load4(x + i);
  for (int p = 0; p < n_parts; ++p) {
    const float4 d = load4(parts + p * n + i);
    v.x += scale * d.x; v.y += scale * d.y; v.z += scale * d.z; v.w += scale * d.w;
  }
  store4(out + i, v);
}

template <typename T>
__global__ __launch_bounds__(256) void loop_rows_kernel(const float* __restrict__ x, const float* __restrict__ parts,
                                                        int n_parts, float scale, const int64_t* __restrict__ ids,
                                                        const T* __restrict__ table, int vocab, size_t part_stride,
                                                        int ld, T* __restrict__ y) {
  const size_t row = (size_t)blockIdx.x * ld;
  const int64_t id = ids[blockIdx.x];
  const T* src = table + (size_t)(id < 0 ? 0 : id >= vocab ? vocab - 1 : id) * ld;
  for (int c = 4 * threadIdx.x; c < ld; c += 1024) {
    float4 v = load4(x + row + c);
    for (int p = 0; p < n_parts; ++p) {
      const float4 d = load4(parts + p * part_stride + row + c);
      v.x += scale * d.x; v.y += scale * d.y; v.z += scale * d.z; v.w += scale * d.w;
    }
    store4(y + 2 * row + c, v);
    store4(y + 2 * row + ld + c, load4(src + c));
  }
}

template <typename ZT>
__global__ __launch_bounds__(256) void polynorm_kernel(ZT* __restrict__ z, int F, int ld, const float* __restrict__ act,
                                                       float eps) {
  extern __shared__ __align__(16) float s_z[];  // [ld]
  __shared__ float s_part[4][3];
  ZT* row = z + (size_t)blockIdx.x * ld;
  float s2 = 0.0f, s4 = 0.0f, s6 = 0.0f;
  for (int c = 4 * threadIdx.x; c < ld; c += 1024) {
    float4 v = load4(row + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (c + e >= F) at4(v, e) = 0.0f;
      const float q = at4(v, e) * at4(v, e);
      s2 += q;
      s4 = __fmaf_rn(q, q, s4);
      s6 = __fmaf_rn(q * q, q, s6);
    }
    store4(s_z + c, v);
  }
  s2 = wave_sum64(s2);
  s4 = wave_sum64(s4);
  s6 = wave_sum64(s6);
  if ((threadIdx.x & 63) == 0) {
    float* d = s_part[threadIdx.x >> 6];
    d[0] = s2;
    d[1] = s4;
    d[2] = s6;
  }
  __syncthreads();
  float t[3];
#pragma unroll
  for (int i = 0; i < 3; ++i) t[i] = (s_part[0][i] + s_part[1][i]) + (s_part[2][i] + s_part[3][i]);
  const float inv = 1.0f / (float)F;
  const float r1 = act[0] / sqrtf(t[0] * inv + eps), r2 = act[1] / sqrtf(t[1] * inv + eps);
  const float r3 = act[2] / sqrtf(t[2] * inv + eps), e0 = act[3];
  for (int c = 4 * threadIdx.x; c < ld; c += 1024) {  // the elements this thread wrote
    float4 v = load4(s_z + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float q = at4(v, e);
      at4(v, e) = c + e < F ? q * (r1 + q * (r2 + q * r3)) + e0 : 0.0f;
    }
    store4(row + c, v);
  }
}

// One thread per channel and block of kScTok tokens, the last taps - 1 inputs in registers.
constexpr int kScTok = 8;
template <int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(const float* __restrict__ x, int ldx, float* __restrict__ y,
                                                         int ldy, const float* __restrict__ w, float* __restrict__ ring,
                                                         int ldw, int channels, int silu, int M, int pos0) {
  const int c = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * kScTok;
  if (c >= channels) return;
  float wt[TAPS], win[TAPS];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) wt[j] = w[(size_t)j * ldw + c];
#pragma unroll
  for (int j = 1; j < TAPS; ++j) {  // win[j]: the input j positions before the current one
    const int t = t0 - j, q = pos0 + t;
    win[j] = t >= 0 ? x[(size_t)t * ldx + c] : q >= 0 ? ring[(size_t)(q % TAPS) * ldw + c] : 0.0f;
  }
  const int te = min(t0 + kScTok, M);
  for (int t = t0; t < te; ++t) {
    win[0] = x[(size_t)t * ldx + c];
    float acc = 0.0f;
#pragma unroll
    for (int j = TAPS - 1; j >= 0; --j) acc = __fmaf_rn(wt[TAPS - 1 - j], win[j], acc);
    y[(size_t)t * ldy + c] = silu ? silu_f(acc) : acc;
#pragma unroll
    for (int j = TAPS - 1; j >= 1; --j) win[j] = win[j - 1];
  }
  if (blockIdx.y == 0) {  // the only block that reads the ring (kScTok >= TAPS - 1)
    for (int t = max(0, M - TAPS + 1); t < M; ++t) ring[(size_t)((pos0 + t) % TAPS) * ldw + c] = x[(size_t)t * ldx + c];
  }
}
static_assert(kScTok >= W4A32_LAYERED_MAX_TAPS - 1, "the second block of tokens must not reach before the portion");

// angle = position * base^(-2 i / dims), in double: a position of many thousands leaves f32 few correct digits
__global__ __launch_bounds__(256) void rot_table_kernel(float* __restrict__ sin_t, float* __restrict__ cos_t,
                                                        int max_pos, int dims, double base) {
  const int half = dims / 2;
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (size_t)max_pos * half) return;
  const int p = (int)(i / half), f = (int)(i % half);
  const double a = (double)p * pow(base, -2.0 * f / dims);
  sin_t[i] = (float)sin(a);
  cos_t[i] = (float)cos(a);
}

constexpr size_t kNcLds = 80 * 1024;  // two workgroups per CU

}  // namespace

hipError_t launch_fill_zero(void* p, size_t bytes, hipStream_t s) {
  const size_t n = bytes / 16;
  hipLaunchKernelGGL(fill_zero_kernel, dim3((unsigned)std::min<size_t>((n + 255) / 256, 8192)), dim3(256), 0, s,
                     static_cast<uint4*>(p), n);
  return hipGetLastError();
}

hipError_t launch_rot_table(float* sin_t, float* cos_t, int max_pos, int dims, double base, hipStream_t s) {
  const size_t n = (size_t)max_pos * (dims / 2);
  hipLaunchKernelGGL(rot_table_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, sin_t, cos_t, max_pos, dims,
                     base);
  return hipGetLastError();
}

hipError_t launch_embed_rows(int dtype, const int64_t* ids, const void* table, int M, int H, int ld, int vocab,
                             float* x, hipStream_t s) {
  (void)H;
  if (dtype == W4A32_LAYERED_BF16) {
    hipLaunchKernelGGL(embed_rows_kernel<__bf16>, dim3(M), dim3(256), 0, s, ids, static_cast<const __bf16*>(table), x,
                       ld, vocab);
  } else {
    hipLaunchKernelGGL(embed_rows_kernel<float>, dim3(M), dim3(256), 0, s, ids, static_cast<const float*>(table), x, ld,
                       vocab);
  }
  return hipGetLastError();
}

static int norm_conv_rows(int M, int ld, int taps) {
  const int halo = taps > 0 ? taps - 1 : 0;
  const int fit = (int)(kNcLds / (sizeof(float) * ld)) - halo;
  const int round = std::max(kNcWaves - halo, 4);  // with its halo, a row per wavefront
  return std::max(1, std::min(std::min(round, (M + 127) / 128), fit));
}

// LDS for the rows and their halo; the tail pass gives every wavefront that has one a row of its own
static size_t norm_conv_lds(int ld, int taps, int rows) {
  const int halo = taps > 0 ? taps - 1 : 0;
  return sizeof(float) * (size_t)ld * (halo + rows);
}

bool norm_conv_fits(int ld, int taps) { return norm_conv_lds(ld, taps, 1) <= 160 * 1024; }

template <int TAPS, typename YT>
static hipError_t norm_conv_t(const float* x, const float* parts, int n_parts, float* x_out, const float* norm_w,
                              const NormSpec& spec, const float* conv, float* ring, int M, int H, int ld, int pos0, YT* y,
                              hipStream_t s) {
  const int TR = norm_conv_rows(M, ld, TAPS);
  const size_t lds = norm_conv_lds(ld, TAPS, TR);
  auto kern = norm_conv_kernel<TAPS, YT>;
  static LdsLimitOnce raised;
  if (lds > 64 * 1024)
    if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), 160 * 1024); e != hipSuccess) return e;
  hipLaunchKernelGGL(kern, dim3((M + TR - 1) / TR), dim3(64 * kNcWaves), lds, s, x, parts, n_parts, x_out, norm_w, spec,
                     conv, ring, M, H, ld, pos0, TR, y);
  return hipGetLastError();
}

hipError_t launch_norm_conv(const float* x, const float* parts, int n_parts, float* x_out, const float* norm_w,
                            const NormSpec& spec, const float* conv, float* ring, int taps, int M, int H, int ld, int pos0,
                            void* y, bool y_bf16, hipStream_t s) {
  if (!norm_conv_fits(ld, taps)) return hipErrorInvalidValue;
  if (n_parts == 0) x_out = nullptr;  // the residual rows stay where they are
#define W4_NORM_CONV(T)                                                                                            \
  case T:                                                                                                          \
    return y_bf16 ? norm_conv_t<T>(x, parts, n_parts, x_out, norm_w, spec, conv, ring, M, H, ld, pos0,              \
                                   static_cast<__bf16*>(y), s)                                                     \
                  : norm_conv_t<T>(x, parts, n_parts, x_out, norm_w, spec, conv, ring, M, H, ld, pos0,              \
                                   static_cast<float*>(y), s)
  switch (taps) {
    W4_NORM_CONV(0); W4_NORM_CONV(1); W4_NORM_CONV(2); W4_NORM_CONV(3); W4_NORM_CONV(4);
    W4_NORM_CONV(5); W4_NORM_CONV(6); W4_NORM_CONV(7); W4_NORM_CONV(8);
    default: return hipErrorInvalidValue;
  }
#undef W4_NORM_CONV
}

hipError_t launch_norm_want(const float* x, const float* parts, int n_parts, const float* norm_w,
                            const NormSpec& spec, const int* want, int n_want, int M, int H, int ld, void* y, bool y_bf16, hipStream_t s) {
  const size_t lds = sizeof(float) * ld;
  if (lds > 160 * 1024) return hipErrorInvalidValue;
  if (y_bf16) {
    static LdsLimitOnce raised;
    if (lds > 64 * 1024)
      if (hipError_t e = raised.raise(reinterpret_cast<const void*>(norm_want_kernel<__bf16>), 160 * 1024);
          e != hipSuccess)
        return e;
    hipLaunchKernelGGL(norm_want_kernel<__bf16>, dim3(n_want), dim3(64), lds, s, x, parts, n_parts, norm_w, spec, want,
                       M, H, ld, static_cast<__bf16*>(y));
  } else {
    static LdsLimitOnce raised;
    if (lds > 64 * 1024)
      if (hipError_t e = raised.raise(reinterpret_cast<const void*>(norm_want_kernel<float>), 160 * 1024);
          e != hipSuccess)
        return e;
    hipLaunchKernelGGL(norm_want_kernel<float>, dim3(n_want), dim3(64), lds, s, x, parts, n_parts, norm_w, spec, want, M,
                       H, ld, static_cast<float*>(y));
  }
  return hipGetLastError();
}

hipError_t launch_loop_rows(int dtype, const float* x, const float* parts, int n_parts, float scale, const int64_t* ids,
                            const void* table, int vocab, int M, int ld, void* y, hipStream_t s) {
  const size_t stride = (size_t)M * ld;
  if (dtype == W4A32_LAYERED_BF16) {
    hipLaunchKernelGGL(loop_rows_kernel<__bf16>, dim3(M), dim3(256), 0, s, x, parts, n_parts, scale, ids,
                       static_cast<const __bf16*>(table), vocab, stride, ld, static_cast<__bf16*>(y));
  } else {
    hipLaunchKernelGGL(loop_rows_kernel<float>, dim3(M), dim3(256), 0, s, x, parts, n_parts, scale, ids,
                       static_cast<const float*>(table), vocab, stride, ld, static_cast<float*>(y));
  }
  return hipGetLastError();
}

hipError_t launch_add_parts(const float* x, const float* parts, int n_parts, float scale, float* out, int M, int ld,
                            hipStream_t s) {
  const size_t n = (size_t)M * ld;
  hipLaunchKernelGGL(add_parts_kernel, dim3((unsigned)((n / 4 + 255) / 256)), dim3(256), 0, s, x, parts, n_parts,
                     scale, out, n);
  return hipGetLastError();
}

bool polynorm_fits(int ld) { return sizeof(float) * (size_t)ld <= 156 * 1024; }

hipError_t launch_polynorm(void* z, bool z_bf16, int M, int F, int ld, const float* act, float eps, hipStream_t s) {
  if (!polynorm_fits(ld)) return hipErrorInvalidValue;
  const size_t lds = sizeof(float) * ld;
  if (z_bf16) {
    static LdsLimitOnce raised;
    if (lds > 60 * 1024)
      if (hipError_t e = raised.raise(reinterpret_cast<const void*>(polynorm_kernel<__bf16>), 156 * 1024);
          e != hipSuccess)
        return e;
    hipLaunchKernelGGL(polynorm_kernel<__bf16>, dim3(M), dim3(256), lds, s, static_cast<__bf16*>(z), F, ld, act, eps);
  } else {
    static LdsLimitOnce raised;
    if (lds > 60 * 1024)
      if (hipError_t e = raised.raise(reinterpret_cast<const void*>(polynorm_kernel<float>), 156 * 1024);
          e != hipSuccess)
        return e;
    hipLaunchKernelGGL(polynorm_kernel<float>, dim3(M), dim3(256), lds, s, static_cast<float*>(z), F, ld, act, eps);
  }
  return hipGetLastError();
}

hipError_t launch_short_conv(const float* x, int ldx, float* y, int ldy, const float* w, float* ring, int ldw, int taps,
                             int channels, bool silu, int M, int pos0, hipStream_t s) {
  const dim3 grid((channels + 255) / 256, (M + kScTok - 1) / kScTok), block(256);
#define W4_SHORT_CONV(T)                                                                                         \
  case T:                                                                                                        \
    hipLaunchKernelGGL(short_conv_kernel<T>, grid, block, 0, s, x, ldx, y, ldy, w, ring, ldw, channels, (int)silu, M, \
                       pos0);                                                                                    \
    break
  switch (taps) {
    W4_SHORT_CONV(1); W4_SHORT_CONV(2); W4_SHORT_CONV(3); W4_SHORT_CONV(4);
    W4_SHORT_CONV(5); W4_SHORT_CONV(6); W4_SHORT_CONV(7); W4_SHORT_CONV(8);
    default: return hipErrorInvalidValue;
  }
#undef W4_SHORT_CONV
  return hipGetLastError();
}

}  // namespace w4
