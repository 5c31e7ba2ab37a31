// Linears with bf16 (or f32) weights for the layered decoder.
//
//   matmul_bf16_kernel   C = A B^T, bf16 operands, f32 accumulation (v_mfma_f32_32x32x16_bf16), for prefill rows.
//   row_linear_kernel    one decode row through [N][K] weights, read once, with the operator that produces the row
//                        in front (residual add + norm + input convolution, merge of the attention's key slices,
//                        per-head norm and gate, PolyNorm, none): HBM-bound, N * K * sizeof(weight) bytes.
//
// The tile of C a workgroup owns and the rows a decode Linear multiplies are in w4a32_mfma_tile.h and w4a32_row_prologue.h.
#include <algorithm>

#include "w4a32_layered.h"
#include "w4a32_layered_kernels.h"
#include "w4a32_mfma_tile.h"
#include "w4a32_row_prologue.h"

namespace w4 {

namespace {

template <int BM, int BN, int WM, int WN, typename CT>
__global__ __launch_bounds__(64 * WM * WN) void matmul_bf16_kernel(const __bf16* __restrict__ a,
                                                                   const __bf16* __restrict__ b, CT* __restrict__ c,
                                                                   int M, int N, int K, int ldc, int mt, int nt) {
  using Tile = MfmaTile<__bf16, BM, BN, WM, WN>;
  constexpr int FM = Tile::FM, FN = Tile::FN, kBK = Tile::kBK;
  extern __shared__ __align__(16) uint8_t smem[];

  // tile number: consecutive ones on one XCD
  const int t = xcd_tile(blockIdx.x, mt * nt);
  const int m0 = (t % mt) * BM, n0 = (t / mt) * BN;
  // this workgroup's share of the k range, in whole LDS tiles
  const int k_steps = K / kBK;
  const int kb = (int)((long)k_steps * blockIdx.y / gridDim.y) * kBK;
  const int ke = (int)((long)k_steps * (blockIdx.y + 1) / gridDim.y) * kBK;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int wm = (wave / WN) * (BM / WM), wn = (wave % WN) * (BN / WN);

  const __bf16* ga[Tile::LA];
  const __bf16* gb[Tile::LB];
#pragma unroll
  for (int i = 0; i < Tile::LA; ++i) ga[i] = a + (size_t)min(m0 + Tile::row(i), M - 1) * K + Tile::k();
#pragma unroll
  for (int i = 0; i < Tile::LB; ++i) gb[i] = b + (size_t)min(n0 + Tile::row(i), N - 1) * K + Tile::k();
  f32x16 acc[FM][FN];
  Tile::run(smem, ga, gb, kb, ke, acc);

  c += (size_t)blockIdx.y * M * ldc;
#pragma unroll
  for (int i = 0; i < FM; ++i)
#pragma unroll
    for (int j = 0; j < FN; ++j) {
      const int col = n0 + wn + 32 * j + (lane & 31);
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        const int row = m0 + wm + 32 * i + 8 * (v >> 2) + 4 * (lane >> 5) + (v & 3);
        if (row < M && col < N) c[(size_t)row * ldc + col] = (CT)acc[i][j][v];
      }
    }
}

template <int BM, int BN, int WM, int WN>
hipError_t launch_tile(const __bf16* a, const __bf16* b, void* c, int M, int N, int K, int ldc, bool c_bf16, int parts,
                       hipStream_t s) {
  const int mt = (M + BM - 1) / BM, nt = (N + BN - 1) / BN;
  const dim3 grid(mt * nt, parts), block(64 * WM * WN);  // parts <= K / kBK: no share is empty
  constexpr size_t lds = MfmaTile<__bf16, BM, BN, WM, WN>::kLds;
  if (c_bf16) {
    auto kern = matmul_bf16_kernel<BM, BN, WM, WN, __bf16>;
    static LdsLimitOnce raised;
    if (lds > 64 * 1024)
      if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), lds); e != hipSuccess) return e;
    hipLaunchKernelGGL(kern, grid, block, lds, s, a, b, static_cast<__bf16*>(c), M, N, K, ldc, mt, nt);
  } else {
    auto kern = matmul_bf16_kernel<BM, BN, WM, WN, float>;
    static LdsLimitOnce raised;
    if (lds > 64 * 1024)
      if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), lds); e != hipSuccess) return e;
    hipLaunchKernelGGL(kern, grid, block, lds, s, a, b, static_cast<float*>(c), M, N, K, ldc, mt, nt);
  }
  return hipGetLastError();
}

// 128 x 128 tiles where they fill the CUs (dealt over k when the caller takes partial products), else 64 x 64
long tiles_of(int M, int N, int t) { return (long)((M + t - 1) / t) * ((N + t - 1) / t); }
bool small_tiles(int M, int N, int parts) { return tiles_of(M, N, 128) < (parts > 1 ? 96 : 192); }

// ---------------------------------------------------------------------------------------------
template <typename WT, int kKind, int R, int U>
__global__ __launch_bounds__(kRowThreads) void row_linear_kernel(const RowPrologue p, const WT* __restrict__ w, int N,
                                                                 int Kp, float* __restrict__ y,
                                                                 float* __restrict__ amax_val,
                                                                 int* __restrict__ amax_idx) {
  extern __shared__ __align__(16) float s_x[];  // [Kp]
  __shared__ float s_red[3 * kRowWaves];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int gw = (int)blockIdx.x * kRowWaves + wave, nw = (int)gridDim.x * kRowWaves;
  const int groups = (N + R - 1) / R;
  auto ptr = [&](int g, int r, int k) { return w + (size_t)min(g * R + r, N - 1) * Kp + k; };
  Raw<WT> cur[R][U];
  row_prologue<WT, kKind>(p, Kp, s_x, s_red, [&] {
    __builtin_amdgcn_sched_barrier(0);
    if (gw < groups) fetch_rows<WT, R, U>(cur, gw, 0, Kp, ptr);
    __builtin_amdgcn_sched_barrier(0);
  });
  __syncthreads();

  float best_v = -INFINITY;
  int best_n = 0x7fffffff;
  stream_rows<WT, R, U>(cur, gw, nw, groups, Kp, s_x, ptr, [&](int g, const float (&t)[R]) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int n = g * R + r;
      if (n < N) {
        if (lane == 0) y[n] = t[r];
        if (t[r] > best_v || (t[r] == best_v && n < best_n)) {
          best_v = t[r];
          best_n = n;
        }
      }
    }
  });
  if (amax_val && lane == 0) {
    amax_val[gw] = best_v;
    amax_idx[gw] = best_n;
  }
}

// rows of W a wavefront takes at a time. A merged attention row is expensive to produce: fewer workgroups.
int rows_per_group(int kind, int N) { return N >= 4096 ? 4 : N >= 2048 || kind == kRowMerge ? 2 : 1; }
int row_grid(int kind, int N) {
  const int R = rows_per_group(kind, N), groups = (N + R - 1) / R;
  return std::min((groups + kRowWaves - 1) / kRowWaves, 512);
}

template <typename WT, int kKind, int R, int U>
hipError_t launch_row_r(const RowPrologue& p, const void* w, int N, int Kp, float* y, float* av, int* ai,
                        hipStream_t s) {
  auto kern = row_linear_kernel<WT, kKind, R, U>;
  const size_t lds = sizeof(float) * (Kp + (kKind == kRowMerge ? (size_t)kPoolAttnSlices * p.heads : 0));
  static LdsLimitOnce raised;
  if (lds > 159 * 1024) return hipErrorInvalidValue;
  if (lds > 60 * 1024)
    if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), 159 * 1024); e != hipSuccess) return e;
  hipLaunchKernelGGL(kern, dim3(row_grid(kKind, N)), dim3(kRowThreads), lds, s, p, static_cast<const WT*>(w), N, Kp, y, av,
                     ai);
  return hipGetLastError();
}

template <typename WT, int kKind>
hipError_t launch_row_k(const RowPrologue& p, const void* w, int N, int Kp, float* y, float* av, int* ai,
                        hipStream_t s) {
  switch (rows_per_group(kKind, N)) {
    case 4: return launch_row_r<WT, kKind, 4, 3>(p, w, N, Kp, y, av, ai, s);
    case 2: return launch_row_r<WT, kKind, 2, 3>(p, w, N, Kp, y, av, ai, s);
    default:
      if (Kp > 6 * 512) return launch_row_r<WT, kKind, 1, 9>(p, w, N, Kp, y, av, ai, s);
      return launch_row_r<WT, kKind, 1, 3>(p, w, N, Kp, y, av, ai, s);
  }
}

template <typename WT>
hipError_t launch_row_t(int kind, const RowPrologue& p, const void* w, int N, int Kp, float* y, float* av, int* ai,
                        hipStream_t s) {
  switch (kind) {
    case kRowNorm: return launch_row_k<WT, kRowNorm>(p, w, N, Kp, y, av, ai, s);
    case kRowMerge: return launch_row_k<WT, kRowMerge>(p, w, N, Kp, y, av, ai, s);
    case kRowGated: return launch_row_k<WT, kRowGated>(p, w, N, Kp, y, av, ai, s);
    case kRowPoly: return launch_row_k<WT, kRowPoly>(p, w, N, Kp, y, av, ai, s);
    case kRowPlain: return launch_row_k<WT, kRowPlain>(p, w, N, Kp, y, av, ai, s);
    case kRowLoop: return launch_row_k<WT, kRowLoop>(p, w, N, Kp, y, av, ai, s);
    default: return hipErrorInvalidValue;
  }
}

}  // namespace

int matmul_bf16_parts(int M, int N, int K) {
  const bool small = small_tiles(M, N, 2);
  const long tiles = tiles_of(M, N, small ? 64 : 128), enough = small ? 768 : 384;
  int parts = 1;
  while (parts < 8 && tiles * parts < enough && K / (2 * parts) >= 512) parts *= 2;
  return parts;
}

hipError_t launch_matmul_bf16(const void* a, const void* b, void* c, int M, int N, int K, int ldc, bool c_bf16,
                              int parts, hipStream_t s) {
  if (K % kPad != 0 || parts < 1 || parts > K / kPad || (parts > 1 && c_bf16)) return hipErrorInvalidValue;
  const __bf16* pa = static_cast<const __bf16*>(a);
  const __bf16* pb = static_cast<const __bf16*>(b);
  if (small_tiles(M, N, parts)) return launch_tile<64, 64, 2, 2>(pa, pb, c, M, N, K, ldc, c_bf16, parts, s);
  return launch_tile<128, 128, 2, 2>(pa, pb, c, M, N, K, ldc, c_bf16, parts, s);
}

int row_linear_partials(int kind, int N) { return row_grid(kind, N) * kRowWaves; }
// (the slices' weights of a merged attention row lie behind the row)
bool row_linear_fits(int Kp) { return sizeof(float) * (size_t)Kp <= 140 * 1024; }

hipError_t launch_row_linear(int kind, int dtype, const RowPrologue& pro, const void* w, int N, int Kp, float* y,
                             float* amax_val, int* amax_idx, hipStream_t s) {
  if (!row_linear_fits(Kp)) return hipErrorInvalidValue;
  if (dtype == W4A32_LAYERED_BF16) return launch_row_t<__bf16>(kind, pro, w, N, Kp, y, amax_val, amax_idx, s);
  return launch_row_t<float>(kind, pro, w, N, Kp, y, amax_val, amax_idx, s);
}

}  // namespace w4
