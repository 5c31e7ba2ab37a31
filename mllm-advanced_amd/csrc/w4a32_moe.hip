// Mixture of experts of the layered decoder: a token's `top` experts are those with the largest router logits, weighted by the
// softmax over these logits; an expert is down(g sigmoid(1.702 g) (u + 1)) with g = min(gate(h), limit), u = clamp(up(h)).
//
// Prefill: [choose] a wavefront per token; [plan] the (token, slot) pairs sorted by expert, and the tiles of the grouped
// products; [gate, up + activation] rows gathered, a wavefront's two column blocks are gate and up of the same 32
// columns; [down] weighted rows to [slot][token], which the norm that follows adds to the residual stream. Nothing depends on the
// order in which workgroups run.
// Decode: [norm + choice + gate, up + activation] [down of all chosen experts as one product over their joined columns].
#include <algorithm>

#include "w4a32_layered.h"
#include "w4a32_layered_kernels.h"
#include "w4a32_mfma_tile.h"
#include "w4a32_row_prologue.h"

namespace w4 {

namespace {

constexpr float kGluAlpha = 1.702f;
constexpr int kMaxParts = kMoeLogitParts;
constexpr int kLogitRegs = W4A32_LAYERED_MAX_EXPERTS / 64;
static_assert(W4A32_LAYERED_MAX_TOP <= 64, "a lane per chosen expert");

__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f(kGluAlpha * g) * (u + 1.0f);
}

// The `top` largest of a wavefront's values (value i of lane l belongs to expert 64 i + l; equal ones: the lower expert
// first). Lane t < top returns the t-th expert and its softmax weight.
__device__ __forceinline__ void top_experts(float (&v)[kLogitRegs], int experts, int top, int* expert, float* weight) {
  const int lane = threadIdx.x & 63;
  int pick = 0;
  float mine = 0.0f, first = 0.0f, sum = 0.0f;
  for (int t = 0; t < top; ++t) {
    float best = -INFINITY;
    int at = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < kLogitRegs; ++i)
      if (64 * i < experts && v[i] > best) {
        best = v[i];
        at = 64 * i + lane;
      }
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) {
      const float ov = __shfl_xor(best, off, 64);
      const int oa = __shfl_xor(at, off, 64);
      if (ov > best || (ov == best && oa < at)) {
        best = ov;
        at = oa;
      }
    }
    at = min(at, experts - 1);  // (values that do not compare choose the last expert)
#pragma unroll
    for (int i = 0; i < kLogitRegs; ++i)
      if (64 * i + lane == at) v[i] = -INFINITY;
    if (t == 0) first = best;
    const float w = expf(best - first);
    sum += w;
    if (lane == t) {
      pick = at;
      mine = w;
    }
  }
  *expert = pick;
  *weight = mine / sum;
}

// ---------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void moe_choose_kernel(const float* __restrict__ logits, int parts, size_t part_stride,
                                                         int ldl, int M, int experts, int top, int* __restrict__ ids,
                                                         float* __restrict__ wts) {
  const int m = 4 * (int)blockIdx.x + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (m >= M) return;
  float v[kLogitRegs];
#pragma unroll
  for (int i = 0; i < kLogitRegs; ++i) {
    const int e = 64 * i + lane;
    v[i] = -INFINITY;
    if (e < experts) {
      const float* src = logits + (size_t)m * ldl + e;
      float x[kMaxParts], s = 0.0f;
#pragma unroll
      for (int p = 0; p < kMaxParts; ++p) x[p] = src[min(p, parts - 1) * part_stride];  // all requested before the first is used
#pragma unroll
      for (int p = 0; p < kMaxParts; ++p) s += p < parts ? x[p] : 0.0f;
      v[i] = s;
    }
  }
  int e;
  float w;
  top_experts(v, experts, top, &e, &w);
  if (lane < top) {
    ids[(size_t)m * top + lane] = e;
    wts[(size_t)m * top + lane] = w;
  }
}

struct MoeTile {
  int expert, row0, rows;  // rows of the sorted list
  int first, tiles;        // the expert's first tile and how many it has
  int pad[3];
};

constexpr int kPlanThreads = 1024, kPlanWaves = kPlanThreads / 64;

// Sum over the workgroup of one int per thread, and of those of lower threads.
__device__ __forceinline__ int block_scan(int x, int* s_w, int* total) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int inc = x;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const int y = __shfl_up(inc, off, 64);
    if (lane >= off) inc += y;
  }
  __syncthreads();  // s_w of an earlier call
  if (lane == 63) s_w[wave] = inc;
  __syncthreads();
  int before = 0, all = 0;
#pragma unroll
  for (int w = 0; w < kPlanWaves; ++w) {
    before += w < wave ? s_w[w] : 0;
    all += s_w[w];
  }
  *total = all;
  return before + inc - x;
}

// A workgroup per expert: where its run of the sorted list starts (all of them count everything), its pairs in ascending order,
// its tiles.
__global__ __launch_bounds__(kPlanThreads) void moe_plan_kernel(const int* __restrict__ ids, int n, int experts, int bm,
                                                                int* __restrict__ order, MoeTile* __restrict__ tiles,
                                                                int* __restrict__ n_tiles) {
  __shared__ int s_count[W4A32_LAYERED_MAX_EXPERTS];
  __shared__ int s_w[kPlanWaves];
  const int e = blockIdx.x, tid = threadIdx.x;
  for (int i = tid; i < experts; i += kPlanThreads) s_count[i] = 0;
  __syncthreads();
  // a thread takes a run of pairs, up to eight of them in registers
  constexpr int kRegs = 8;
  const int per = (n + kPlanThreads - 1) / kPlanThreads, lo = min(n, tid * per), hi = min(n, lo + per);
  int mine = 0, id[kRegs];
#pragma unroll
  for (int i = 0; i < kRegs; ++i) id[i] = ids[min(lo + i, n - 1)];
#pragma unroll
  for (int i = 0; i < kRegs; ++i)
    if (lo + i < hi) {
      atomicAdd(&s_count[id[i]], 1);
      mine += id[i] == e;
    }
  for (int i = lo + kRegs; i < hi; ++i) {
    atomicAdd(&s_count[ids[i]], 1);
    mine += ids[i] == e;
  }
  __syncthreads();
  int total;
  const bool before = tid < experts && tid < e;
  block_scan(before ? s_count[tid] : 0, s_w, &total);
  const int offset = total;
  block_scan(before ? (s_count[tid] + bm - 1) / bm : 0, s_w, &total);
  const int first = total;
  int at = offset + block_scan(mine, s_w, &total);
#pragma unroll
  for (int i = 0; i < kRegs; ++i)
    if (lo + i < hi && id[i] == e) order[at++] = lo + i;
  for (int i = lo + kRegs; i < hi; ++i)
    if (ids[i] == e) order[at++] = i;
  const int count = total, mt = (count + bm - 1) / bm;
  for (int t = tid; t < mt; t += kPlanThreads)
    tiles[first + t] = MoeTile{e, offset + t * bm, min(bm, count - t * bm), first, mt, {0, 0, 0}};
  if (e == experts - 1 && tid == 0) *n_tiles = first + mt;
}
static_assert(kPlanThreads >= W4A32_LAYERED_MAX_EXPERTS, "a thread per expert");

// The tile of a workgroup: an expert's tiles are numbered rows fastest, experts one after the other; consecutive numbers on one
// XCD. Returns false past the last one.
__device__ __forceinline__ bool moe_tile(const MoeTile* __restrict__ tiles, const int* __restrict__ n_tiles, int nt,
                                         MoeTile* tile, int* n) {
  const int total = *n_tiles * nt;
  if ((int)blockIdx.x >= total) return false;
  const int t = xcd_tile(blockIdx.x, total);
  const MoeTile any = tiles[t / nt];  // a tile of the expert
  if (any.tiles <= 0) return false;
  const int local = t - any.first * nt;
  *tile = tiles[any.first + local % any.tiles];
  *n = local / any.tiles;
  return true;
}

// act [sorted pair][Fp] = glu(h gate^T, h up^T)
template <typename T, int BM>
__global__ __launch_bounds__(256) void moe_gate_up_kernel(const T* __restrict__ h, const T* __restrict__ w,
                                                          T* __restrict__ act, const int* __restrict__ order,
                                                          const MoeTile* __restrict__ tiles, const int* __restrict__ n_tiles,
                                                          int top, int Hp, int Fp, float limit) {
  using Tile = MfmaTile<T, BM, 128, 2, 2>;
  extern __shared__ __align__(16) uint8_t smem[];
  MoeTile tile;
  int n;
  const int N = 2 * Fp;
  if (!moe_tile(tiles, n_tiles, (N + 127) / 128, &tile, &n)) return;
  const int n0 = 128 * n, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const T* we = w + (size_t)tile.expert * N * Hp;
  const T* ga[Tile::LA];
  const T* gb[Tile::LB];
#pragma unroll
  for (int i = 0; i < Tile::LA; ++i)
    ga[i] = h + (size_t)(order[tile.row0 + min(Tile::row(i), tile.rows - 1)] / top) * Hp + Tile::k();
#pragma unroll
  for (int i = 0; i < Tile::LB; ++i) gb[i] = we + (size_t)min(n0 + Tile::row(i), N - 1) * Hp + Tile::k();
  f32x16 acc[Tile::FM][2];
  Tile::run(smem, ga, gb, 0, Hp, acc);
  const int col = (n0 + 64 * (wave & 1)) / 2 + (lane & 31);
  if (col >= Fp) return;
#pragma unroll
  for (int i = 0; i < Tile::FM; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int r = (wave >> 1) * (BM / 2) + 32 * i + 8 * (v >> 2) + 4 * (lane >> 5) + (v & 3);
      if (r < tile.rows) act[(size_t)(tile.row0 + r) * Fp + col] = (T)clamped_glu(acc[i][0][v], acc[i][1][v], limit);
    }
}

// parts [slot][token][Hp] = weight * act down^T
template <typename T, int BM>
__global__ __launch_bounds__(256) void moe_down_kernel(const T* __restrict__ act, const T* __restrict__ w,
                                                       float* __restrict__ parts, const int* __restrict__ order,
                                                       const float* __restrict__ wts, const MoeTile* __restrict__ tiles,
                                                       const int* __restrict__ n_tiles, int top, int M, int Hp, int Fp) {
  using Tile = MfmaTile<T, BM, 128, 2, 2>;
  extern __shared__ __align__(16) uint8_t smem[];
  MoeTile tile;
  int n;
  if (!moe_tile(tiles, n_tiles, (Hp + 127) / 128, &tile, &n)) return;
  const int n0 = 128 * n, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const T* we = w + (size_t)tile.expert * Hp * Fp;
  const T* ga[Tile::LA];
  const T* gb[Tile::LB];
#pragma unroll
  for (int i = 0; i < Tile::LA; ++i)
    ga[i] = act + (size_t)(tile.row0 + min(Tile::row(i), tile.rows - 1)) * Fp + Tile::k();
#pragma unroll
  for (int i = 0; i < Tile::LB; ++i) gb[i] = we + (size_t)min(n0 + Tile::row(i), Hp - 1) * Fp + Tile::k();
  f32x16 acc[Tile::FM][Tile::FN];
  Tile::run(smem, ga, gb, 0, Fp, acc);
#pragma unroll
  for (int i = 0; i < Tile::FM; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int r = (wave >> 1) * (BM / 2) + 32 * i + 8 * (v >> 2) + 4 * (lane >> 5) + (v & 3);
      if (r >= tile.rows) continue;
      const int pair = order[tile.row0 + r], m = pair / top;
      const float a = wts[pair];
      float* dst = parts + ((size_t)(pair - m * top) * M + m) * Hp;
#pragma unroll
      for (int c = 0; c < Tile::FN; ++c) {
        const int col = n0 + 64 * (wave & 1) + 32 * c + (lane & 31);
        if (col < Hp) dst[col] = a * acc[i][c][v];
      }
    }
}

// ---------------------------------------------------------------------------------------------
// z [slot][Fp] = weight * glu of the chosen experts; a group is P columns of one expert, gate and up row of each. The first
// workgroup leaves the choice for the launch behind.
template <typename WT, int P, int U>
__global__ __launch_bounds__(kRowThreads) void moe_row_gate_up_kernel(const RowPrologue p, const float* __restrict__ logits,
                                                                      const WT* __restrict__ w, int experts, int top,
                                                                      int Hp, int Fp, float limit, float* __restrict__ z,
                                                                      int* __restrict__ sel) {
  extern __shared__ __align__(16) float s_x[];  // [Hp]
  __shared__ float s_red[3 * kRowWaves];
  constexpr int R = 2 * P;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int gw = (int)blockIdx.x * kRowWaves + wave, nw = (int)gridDim.x * kRowWaves;
  const int per = Fp / P, groups = top * per;
  int expert = 0;
  float weight = 0.0f;
  auto ptr = [&](int g, int r, int k) {
    const int slot = g / per, c = (g - slot * per) * P + (r >> 1);
    const int row = (c >> 5) * 64 + (r & 1) * 32 + (c & 31);
    return w + ((size_t)__builtin_amdgcn_readlane(expert, slot) * 2 * Fp + row) * Hp + k;
  };
  float v[kLogitRegs];
#pragma unroll
  for (int i = 0; i < kLogitRegs; ++i) v[i] = 64 * i + lane < experts ? logits[64 * i + lane] : -INFINITY;
  Raw<WT> cur[R][U];
  row_prologue<WT, kRowNorm>(p, Hp, s_x, s_red, [&] {
    top_experts(v, experts, top, &expert, &weight);
    __builtin_amdgcn_sched_barrier(0);
    if (gw < groups) fetch_rows<WT, R, U>(cur, gw, 0, Hp, ptr);
    __builtin_amdgcn_sched_barrier(0);
  });
  if (blockIdx.x == 0 && wave == 0 && lane < top) sel[lane] = expert;
  __syncthreads();
  stream_rows<WT, R, U>(cur, gw, nw, groups, Hp, s_x, ptr, [&](int g, const float (&t)[R]) {
    const int slot = g / per;
    const float a = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(weight), slot));
#pragma unroll
    for (int i = 0; i < P; ++i)
      if (lane == 0) z[(size_t)g * P + i] = a * clamped_glu(t[2 * i], t[2 * i + 1], limit);
  });
}

// out [Hp] = sum over the chosen experts of z_slot down^T: one product over the joined columns
template <typename WT, int R, int U>
__global__ __launch_bounds__(kRowThreads) void moe_row_down_kernel(const RowPrologue p, const int* __restrict__ sel,
                                                                   const WT* __restrict__ w, int top, int Hp, int Fp,
                                                                   unsigned magic, float* __restrict__ out) {
  extern __shared__ __align__(16) float s_x[];  // [top * Fp]
  __shared__ float s_red[3 * kRowWaves];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int gw = (int)blockIdx.x * kRowWaves + wave, nw = (int)gridDim.x * kRowWaves;
  const int groups = (Hp + R - 1) / R, K = top * Fp;
  const int expert = sel[min(lane, top - 1)];
  auto ptr = [&](int g, int r, int k) {
    const int slot = (int)__umulhi((unsigned)k, magic);  // k / Fp
    const int e = __shfl(expert, slot, 64);
    return w + ((size_t)e * Hp + min(g * R + r, Hp - 1)) * Fp + (k - slot * Fp);
  };
  Raw<WT> cur[R][U];
  row_prologue<WT, kRowPlain>(p, K, s_x, s_red, [&] {
    __builtin_amdgcn_sched_barrier(0);
    if (gw < groups) fetch_rows<WT, R, U>(cur, gw, 0, K, ptr);
    __builtin_amdgcn_sched_barrier(0);
  });
  __syncthreads();
  stream_rows<WT, R, U>(cur, gw, nw, groups, K, s_x, ptr, [&](int g, const float (&t)[R]) {
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (lane == 0 && g * R + r < Hp) out[g * R + r] = t[r];
  });
}

// ---------------------------------------------------------------------------------------------
inline size_t up256(size_t v) { return (v + 255) / 256 * 256; }

// what a portion's experts work in
struct Scratch {
  size_t ids, wts, order, tiles, n_tiles, act, bytes;
  int max_tiles;
};
int tile_rows(int M, int experts, int top) { return (long)M * top >= 96L * experts ? 128 : 64; }
Scratch scratch_of(int dtype, int M, int experts, int top, int Fp) {
  const size_t n = (size_t)M * top, elem = dtype == W4A32_LAYERED_BF16 ? 2 : 4;
  Scratch c;
  c.max_tiles = (int)((n + 63) / 64) + experts;
  size_t o = 0;
  auto take = [&](size_t bytes) {
    const size_t at = o;
    o += up256(bytes);
    return at;
  };
  c.ids = take(4 * n);
  c.wts = take(4 * n);
  c.order = take(4 * n);
  c.tiles = take(sizeof(MoeTile) * c.max_tiles);
  c.n_tiles = take(4);
  c.act = take(elem * n * Fp);
  c.bytes = o;
  return c;
}

template <typename T, int BM>
hipError_t grouped(const MoeGeom& g, const T* h, const T* gate_up, const T* down, int M, float* parts, uint8_t* ws,
                   const Scratch& c, hipStream_t s) {
  int* order = reinterpret_cast<int*>(ws + c.order);
  MoeTile* tiles = reinterpret_cast<MoeTile*>(ws + c.tiles);
  int* n_tiles = reinterpret_cast<int*>(ws + c.n_tiles);
  T* act = reinterpret_cast<T*>(ws + c.act);
  const int most = (int)(((size_t)M * g.top + BM - 1) / BM) + g.experts;  // workgroups past the last tile return
  constexpr size_t lds = MfmaTile<T, BM, 128, 2, 2>::kLds;
  auto up = moe_gate_up_kernel<T, BM>;
  auto dn = moe_down_kernel<T, BM>;
  static LdsLimitOnce raised_up, raised_dn;
  if (lds > 64 * 1024) {
    if (hipError_t e = raised_up.raise(reinterpret_cast<const void*>(up), lds); e != hipSuccess) return e;
    if (hipError_t e = raised_dn.raise(reinterpret_cast<const void*>(dn), lds); e != hipSuccess) return e;
  }
  hipLaunchKernelGGL(up, dim3((unsigned)most * ((2 * g.Fp + 127) / 128)), dim3(256), lds, s, h, gate_up, act, order, tiles,
                     n_tiles, g.top, g.Hp, g.Fp, g.limit);
  if (hipError_t e = hipGetLastError(); e != hipSuccess) return e;
  hipLaunchKernelGGL(dn, dim3((unsigned)most * ((g.Hp + 127) / 128)), dim3(256), lds, s, act, down, parts, order,
                     reinterpret_cast<const float*>(ws + c.wts), tiles, n_tiles, g.top, M, g.Hp, g.Fp);
  return hipGetLastError();
}

template <typename T>
hipError_t prefill_t(int dtype, const MoeGeom& g, const T* h, const float* logits, int logit_parts, int ldl, const T* gate_up,
                     const T* down, int M, float* parts, uint8_t* ws, hipStream_t s) {
  if (logit_parts < 1 || logit_parts > kMaxParts) return hipErrorInvalidValue;
  const Scratch c = scratch_of(dtype, M, g.experts, g.top, g.Fp);
  const int bm = tile_rows(M, g.experts, g.top);
  int* ids = reinterpret_cast<int*>(ws + c.ids);
  hipLaunchKernelGGL(moe_choose_kernel, dim3((M + 3) / 4), dim3(256), 0, s, logits, logit_parts, (size_t)M * ldl, ldl, M,
                     g.experts, g.top, ids, reinterpret_cast<float*>(ws + c.wts));
  if (hipError_t e = hipGetLastError(); e != hipSuccess) return e;
  hipLaunchKernelGGL(moe_plan_kernel, dim3(g.experts), dim3(kPlanThreads), 0, s, ids, M * g.top, g.experts, bm,
                     reinterpret_cast<int*>(ws + c.order), reinterpret_cast<MoeTile*>(ws + c.tiles),
                     reinterpret_cast<int*>(ws + c.n_tiles));
  if (hipError_t e = hipGetLastError(); e != hipSuccess) return e;
  return bm == 128 ? grouped<T, 128>(g, h, gate_up, down, M, parts, ws, c, s)
                   : grouped<T, 64>(g, h, gate_up, down, M, parts, ws, c, s);
}

template <typename WT>
hipError_t decode_t(const MoeGeom& g, const RowPrologue& pro, const float* logits, const WT* gate_up, const WT* down, float* z,
                    int* sel, float* out, hipStream_t s) {
  {
    constexpr int P = sizeof(WT) == 2 ? 2 : 1, U = 3;
    auto kern = moe_row_gate_up_kernel<WT, P, U>;
    const size_t lds = sizeof(float) * g.Hp;
    static LdsLimitOnce raised;
    if (lds > 60 * 1024)
      if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), 159 * 1024); e != hipSuccess) return e;
    const int groups = g.top * g.Fp / P;
    hipLaunchKernelGGL(kern, dim3(std::min((groups + kRowWaves - 1) / kRowWaves, 512)), dim3(kRowThreads), lds, s, pro, logits,
                       gate_up, g.experts, g.top, g.Hp, g.Fp, g.limit, z, sel);
    if (hipError_t e = hipGetLastError(); e != hipSuccess) return e;
  }
  RowPrologue p{};
  p.K = g.top * g.Fp;
  p.x = z;
  constexpr int U = 6;
  auto kern = moe_row_down_kernel<WT, 1, U>;
  const size_t lds = sizeof(float) * g.top * g.Fp;
  static LdsLimitOnce raised;
  if (lds > 60 * 1024)
    if (hipError_t e = raised.raise(reinterpret_cast<const void*>(kern), 159 * 1024); e != hipSuccess) return e;
  const unsigned magic = (unsigned)(((1ull << 32) + g.Fp - 1) / g.Fp);  // exact quotients below 2^32 / Fp
  hipLaunchKernelGGL(kern, dim3(std::min((g.Hp + kRowWaves - 1) / kRowWaves, 512)), dim3(kRowThreads), lds, s, p, sel, down,
                     g.top, g.Hp, g.Fp, magic, out);
  return hipGetLastError();
}

}  // namespace

size_t moe_scratch_bytes(int dtype, int M, int experts, int top, int Fp) { return scratch_of(dtype, M, experts, top, Fp).bytes; }

hipError_t launch_moe_prefill(int dtype, const MoeGeom& g, const void* h, const float* logits, int logit_parts, int ldl,
                              const void* gate_up, const void* down, int M, float* parts, void* scratch, hipStream_t s) {
  uint8_t* ws = static_cast<uint8_t*>(scratch);
  if (dtype == W4A32_LAYERED_BF16)
    return prefill_t(dtype, g, static_cast<const __bf16*>(h), logits, logit_parts, ldl, static_cast<const __bf16*>(gate_up),
                     static_cast<const __bf16*>(down), M, parts, ws, s);
  return prefill_t(dtype, g, static_cast<const float*>(h), logits, logit_parts, ldl, static_cast<const float*>(gate_up),
                   static_cast<const float*>(down), M, parts, ws, s);
}

bool moe_decode_fits(const MoeGeom& g) { return row_linear_fits(g.Hp) && (long)g.top * g.Fp <= 35840; }

hipError_t launch_moe_decode(int dtype, const MoeGeom& g, const RowPrologue& pro, const float* logits, const void* gate_up,
                             const void* down, float* z, int* sel, float* out, hipStream_t s) {
  if (!moe_decode_fits(g)) return hipErrorInvalidValue;
  if (dtype == W4A32_LAYERED_BF16)
    return decode_t(g, pro, logits, static_cast<const __bf16*>(gate_up), static_cast<const __bf16*>(down), z, sel, out, s);
  return decode_t(g, pro, logits, static_cast<const float*>(gate_up), static_cast<const float*>(down), z, sel, out, s);
}

}  // namespace w4
