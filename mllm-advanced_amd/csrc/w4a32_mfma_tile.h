// The tile of C = A B^T that one workgroup computes: WM x WN wavefronts, each with FM x FN accumulators of 32 x 32. bf16
// operands on v_mfma_f32_32x32x16_bf16, f32 operands on v_mfma_f32_32x32x2_f32. The caller says where the rows lie (a row per
// pointer, so they may be gathered) and what becomes of the accumulators: lane l of a 32 x 32 block holds column l % 32 and,
// in register v, row 8 (v / 4) + 4 (l / 32) + v % 4.
//
// bf16: tiles of 64 k are brought in through registers (requested one or two tiles ahead) and double-buffered in LDS as rows of
// 64 + 8 elements: the 144-byte stride puts 16 consecutive rows' 16-byte operands on all 64 banks once. f32 (the
// exact format, not tuned): tiles of 16 k, rows of 16 + 1 floats.
#pragma once

#include "w4a32_layered_kernels.h"

namespace w4 {

// Workgroups are numbered so that one XCD (number mod 8) gets consecutive tiles: XCD x holds tiles / 8 (+ 1 for the first
// tiles % 8 of them). With rows of C fastest a band of B stays in that XCD's L2 while all of A passes.
__device__ __forceinline__ int xcd_tile(int block, int tiles) {
  const int per = tiles / 8, rem = tiles % 8, x = block & 7, i = block >> 3;
  return x * per + min(x, rem) + i;
}

template <typename T, int BM, int BN, int WM, int WN>
struct MfmaTile;

template <int BM, int BN, int WM, int WN>
struct MfmaTile<__bf16, BM, BN, WM, WN> {
  static constexpr int kThreads = 64 * WM * WN;
  static constexpr int FM = BM / WM / 32, FN = BN / WN / 32;           // 32 x 32 blocks of a wavefront
  static constexpr int LA = BM * 8 / kThreads, LB = BN * 8 / kThreads;  // 16-byte pieces a thread brings per tile
  static constexpr int kBK = 64, kLd = kBK + 8;                         // k per LDS tile; LDS row, elements
  static constexpr size_t kLds = 2 * (BM + BN) * kLd * sizeof(__bf16);
  // the row of A (B) that this thread's piece i is from, and the piece's first k
  static __device__ __forceinline__ int row(int i) { return ((int)threadIdx.x + kThreads * i) >> 3; }
  static __device__ __forceinline__ int k() { return 8 * (threadIdx.x & 7); }

  // acc = rows of A times rows of B over k in [kb, ke), a range of whole tiles that is not empty
  static __device__ __forceinline__ void run(uint8_t* smem, const __bf16* const (&ga)[LA], const __bf16* const (&gb)[LB],
                                             int kb, int ke, f32x16 (&acc)[FM][FN]) {
    __bf16* s_a = reinterpret_cast<__bf16*>(smem);                 // [2][BM][kLd]
    __bf16* s_b = s_a + 2 * BM * kLd;                              // [2][BN][kLd]
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int wm = (wave / WN) * (BM / WM), wn = (wave % WN) * (BN / WN);
    // two register sets: two tiles in flight
    u32x4 ra0[LA], rb0[LB], ra1[LA], rb1[LB];
    auto fetch = [&](int k, u32x4 (&ra)[LA], u32x4 (&rb)[LB]) __attribute__((always_inline)) {
#pragma unroll
      for (int i = 0; i < LA; ++i) ra[i] = *reinterpret_cast<const u32x4*>(ga[i] + k);
#pragma unroll
      for (int i = 0; i < LB; ++i) rb[i] = *reinterpret_cast<const u32x4*>(gb[i] + k);
    };
    __bf16* const sa_w = s_a + (tid >> 3) * kLd + 8 * (tid & 7);
    __bf16* const sb_w = s_b + (tid >> 3) * kLd + 8 * (tid & 7);
    auto stash = [&](int buf, const u32x4 (&ra)[LA], const u32x4 (&rb)[LB]) __attribute__((always_inline)) {
#pragma unroll
      for (int i = 0; i < LA; ++i) *reinterpret_cast<u32x4*>(sa_w + (buf * BM + kThreads / 8 * i) * kLd) = ra[i];
#pragma unroll
      for (int i = 0; i < LB; ++i) *reinterpret_cast<u32x4*>(sb_w + (buf * BN + kThreads / 8 * i) * kLd) = rb[i];
    };
#pragma unroll
    for (int i = 0; i < FM; ++i)
#pragma unroll
      for (int j = 0; j < FN; ++j)
#pragma unroll
        for (int v = 0; v < 16; ++v) acc[i][j][v] = 0.0f;

    auto products = [&](int buf) __attribute__((always_inline)) {
      const __bf16* pa = s_a + (size_t)buf * BM * kLd + (wm + (lane & 31)) * kLd + 8 * (lane >> 5);
      const __bf16* pb = s_b + (size_t)buf * BN * kLd + (wn + (lane & 31)) * kLd + 8 * (lane >> 5);
#pragma unroll
      for (int ks = 0; ks < kBK / 16; ++ks) {
        bf16x8 fa[FM], fb[FN];
#pragma unroll
        for (int i = 0; i < FM; ++i) fa[i] = *reinterpret_cast<const bf16x8*>(pa + 32 * i * kLd + 16 * ks);
#pragma unroll
        for (int j = 0; j < FN; ++j) fb[j] = *reinterpret_cast<const bf16x8*>(pb + 32 * j * kLd + 16 * ks);
#pragma unroll
        for (int i = 0; i < FM; ++i)
#pragma unroll
          for (int j = 0; j < FN; ++j)
            acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
      }
    };

    // Tile i is stashed from register set i & 1 into LDS buffer i & 1; while it is multiplied, tiles i + 1 and i + 2
    // are on their way.
    const int last = ke - kBK;  // a tile past the end is fetched as the last one again and not used
    fetch(kb, ra0, rb0);
    fetch(min(kb + kBK, last), ra1, rb1);
    stash(0, ra0, rb0);
    fetch(min(kb + 2 * kBK, last), ra0, rb0);
    __syncthreads();
    for (int k = kb; k < ke; k += 2 * kBK) {
      // even tile: LDS buffer 0; the next one sits in register set 1
      stash(1, ra1, rb1);
      fetch(min(k + 3 * kBK, last), ra1, rb1);
      products(0);
      __syncthreads();
      if (k + kBK >= ke) break;
      stash(0, ra0, rb0);
      fetch(min(k + 4 * kBK, last), ra0, rb0);
      products(1);
      __syncthreads();
    }
  }
};

template <int BM, int BN, int WM, int WN>
struct MfmaTile<float, BM, BN, WM, WN> {
  static constexpr int kThreads = 64 * WM * WN;
  static constexpr int FM = BM / WM / 32, FN = BN / WN / 32;
  static constexpr int LA = BM * 4 / kThreads, LB = BN * 4 / kThreads;
  static constexpr int kBK = 16, kLd = kBK + 1;
  static constexpr size_t kLds = (BM + BN) * kLd * sizeof(float);
  static __device__ __forceinline__ int row(int i) { return ((int)threadIdx.x + kThreads * i) >> 2; }
  static __device__ __forceinline__ int k() { return 4 * (threadIdx.x & 3); }

  static __device__ __forceinline__ void run(uint8_t* smem, const float* const (&ga)[LA], const float* const (&gb)[LB],
                                             int kb, int ke, f32x16 (&acc)[FM][FN]) {
    float* s_a = reinterpret_cast<float*>(smem);
    float* s_b = s_a + BM * kLd;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int wm = (wave / WN) * (BM / WM), wn = (wave % WN) * (BN / WN);
#pragma unroll
    for (int i = 0; i < FM; ++i)
#pragma unroll
      for (int j = 0; j < FN; ++j)
#pragma unroll
        for (int v = 0; v < 16; ++v) acc[i][j][v] = 0.0f;
    for (int k0 = kb; k0 < ke; k0 += kBK) {
      f32x4 ra[LA], rb[LB];
#pragma unroll
      for (int i = 0; i < LA; ++i) ra[i] = *reinterpret_cast<const f32x4*>(ga[i] + k0);
#pragma unroll
      for (int i = 0; i < LB; ++i) rb[i] = *reinterpret_cast<const f32x4*>(gb[i] + k0);
      __syncthreads();  // the previous tile's reads are done
#pragma unroll
      for (int i = 0; i < LA; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) s_a[row(i) * kLd + k() + e] = ra[i][e];
#pragma unroll
      for (int i = 0; i < LB; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) s_b[row(i) * kLd + k() + e] = rb[i][e];
      __syncthreads();
#pragma unroll
      for (int kk = 0; kk < kBK; kk += 2) {
        float fa[FM], fb[FN];
#pragma unroll
        for (int i = 0; i < FM; ++i) fa[i] = s_a[(wm + 32 * i + (lane & 31)) * kLd + kk + (lane >> 5)];
#pragma unroll
        for (int j = 0; j < FN; ++j) fb[j] = s_b[(wn + 32 * j + (lane & 31)) * kLd + kk + (lane >> 5)];
#pragma unroll
        for (int i = 0; i < FM; ++i)
#pragma unroll
          for (int j = 0; j < FN; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x2f32(fa[i], fb[j], acc[i][j], 0, 0, 0);
      }
    }
  }
};

}  // namespace w4
