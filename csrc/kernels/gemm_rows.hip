// Narrow projections of few rows with what follows them in the same launch: a
// router's logits and the choice of experts, or a gated row times the token's own
// row.  The weights are read once from memory, so they are spread over many CUs:
// in splits of K whose last arriver adds up the partial logits and routes, or in
// column tiles of 16.  Operands go from global memory straight into the MFMA
// fragments; a block's waves share its K, and their partial sums meet in LDS.
#include "common.h"
#include "moe_params.h"
#include "route.h"

namespace lsd {
namespace {

constexpr int STEP = 64;  // of K: whole lines of 16 rows

// Partial products of 16 rows and NT x 16 columns over the 64-wide steps first,
// first + stride, .. < end of K, UP of them in flight.
template <int NT, int UP>
__device__ __forceinline__ void steps_of(const RowsParams& p, int row0, int n0, int first, int stride, int end, f32x4 (&acc)[NT]) {
  const int lane = lane_id(), r = lane & 15, g = lane >> 4;
  const bf16* ap = static_cast<const bf16*>(p.a) + (long)min(row0 + r, p.T - 1) * p.lda + g * 8;
  const bf16* wp[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) {
    wp[j] = static_cast<const bf16*>(p.w) + (long)min(n0 + j * 16 + r, p.N - 1) * p.ldw + g * 8;
    acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  for (int s0 = first; s0 < end; s0 += UP * stride) {
    bf16x8 a[UP][2], b[UP][NT][2];
#pragma unroll
    for (int u = 0; u < UP; ++u) {
      const int k = min(s0 + u * stride, end - 1) * STEP;
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        a[u][q] = ld8(ap + k + q * 32);
#pragma unroll
        for (int j = 0; j < NT; ++j) b[u][j][q] = ld8(wp[j] + k + q * 32);
      }
    }
#pragma unroll
    for (int u = 0; u < UP; ++u)
      if (s0 + u * stride < end) {
#pragma unroll
        for (int q = 0; q < 2; ++q)
#pragma unroll
          for (int j = 0; j < NT; ++j) acc[j] = mfma16(a[u][q], b[u][j][q], acc[j]);
      }
  }
}

// Block (row tile, K split): four waves multiply, all sixteen route a row each.
// part: [row tiles][splits][16][NT 16] fp32.
template <int NT>
__global__ __launch_bounds__(1024) void router_kernel(RowsParams p) {
  constexpr int LDC = NT * 16 + 4, Q = NT * 4;  // groups of four columns
  __shared__ __attribute__((aligned(16))) float sums[4][16 * LDC];
  __shared__ int last;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4, row0 = blockIdx.x * 16, split = blockIdx.y, S = p.splits;
  const int all = p.K / STEP, per = (all + S - 1) / S;
  if (w < 4) {
    f32x4 acc[NT];
    steps_of<NT, 2>(p, row0, 0, split * per + w, 4, min(all, (split + 1) * per), acc);
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) sums[w][(4 * g + i) * LDC + j * 16 + r] = acc[j][i];
  }
  __syncthreads();
  const int id = threadIdx.x, at = id / Q * LDC + id % Q * 4;  // the first 16 Q threads hold four columns
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if (id < 16 * Q) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v += *reinterpret_cast<const f32x4*>(&sums[i][at]);
  }
  if (S > 1) {
    // write-through stores, a ticket, and the last arriver sums all splits in their
    // order (its own too), read past the caches
    constexpr int TILE = 16 * Q * 16;  // bytes
    const __amdgpu_buffer_rsrc_t rs =
        __builtin_amdgcn_make_buffer_rsrc(p.part + (long)blockIdx.x * S * (TILE / 4), (short)0, S * TILE, 0x00020000);
    if (id < 16 * Q)
      __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, v), rs, split * TILE + id * 16, 0, 16);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (id == 0) {
      const int t = __hip_atomic_fetch_add(p.counters + blockIdx.x, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      last = t == S - 1;
      if (t == S - 1) __hip_atomic_store(p.counters + blockIdx.x, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    __syncthreads();
    if (last == 0) return;
    v = f32x4{0.f, 0.f, 0.f, 0.f};
    constexpr int FLY = 8;
    for (int s0 = 0; s0 < S && id < 16 * Q; s0 += FLY) {
      f32x4 u[FLY];
#pragma unroll
      for (int i = 0; i < FLY; ++i)
        u[i] = __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(
                                             rs, min(s0 + i, S - 1) * TILE + id * 16, 0, 16));
#pragma unroll
      for (int i = 0; i < FLY; ++i)
        if (s0 + i < S) v += u[i];
    }
  }
  if (id < 16 * Q) *reinterpret_cast<f32x4*>(&sums[0][at]) = v;  // (read last by this thread itself)
  __syncthreads();
  if (row0 + w < p.T) route_few(p.r, &sums[0][w * LDC], row0 + w);
}

// Block (row tile, 16 columns), eight waves.
__global__ __launch_bounds__(512) void side_gate_kernel(RowsParams p) {
  constexpr int LDC = 20;
  __shared__ __attribute__((aligned(16))) float sums[8][16 * LDC];
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4, row0 = blockIdx.x * 16, n0 = blockIdx.y * 16;
  f32x4 acc[1];
  steps_of<1, 4>(p, row0, n0, w, 8, p.K / STEP, acc);
#pragma unroll
  for (int i = 0; i < 4; ++i) sums[w][(4 * g + i) * LDC + r] = acc[0][i];
  __syncthreads();
  const int t = row0 + threadIdx.x / 16, col = threadIdx.x % 16;
  if (threadIdx.x >= 256 || t >= p.T) return;
  float v = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) v += sums[i][threadIdx.x / 16 * LDC + col];
  int id = p.ids[t];
  id = id < 0 ? 0 : (id >= p.vocab ? p.vocab - 1 : id);
  const float e = bf2f(static_cast<const bf16*>(p.table)[(long)id * p.N + n0 + col]);
  static_cast<bf16*>(p.out)[(long)t * p.ldo + n0 + col] = f2bf(gelu_new(v) * e);
}

}  // namespace
}  // namespace lsd

using namespace lsd;

extern "C" hipError_t lsd_router(const RowsParams* p, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  if (p->K % STEP || p->N % 16 || p->N > 64 || p->r.experts > 64 || p->r.top > p->r.experts || p->splits < 1 ||
      p->splits > p->K / STEP || (p->splits > 1 && (!p->part || !p->counters)))
    return hipErrorInvalidValue;
  const dim3 grid((p->T + 15) / 16, p->splits);
  if (p->N <= 16) hipLaunchKernelGGL((router_kernel<1>), grid, dim3(1024), 0, st, *p);
  else if (p->N <= 32) hipLaunchKernelGGL((router_kernel<2>), grid, dim3(1024), 0, st, *p);
  else hipLaunchKernelGGL((router_kernel<4>), grid, dim3(1024), 0, st, *p);
  return hipGetLastError();
}

extern "C" hipError_t lsd_side_gate(const RowsParams* p, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  if (p->K % STEP || p->N % 16) return hipErrorInvalidValue;
  hipLaunchKernelGGL(side_gate_kernel, dim3((p->T + 15) / 16, p->N / 16), dim3(512), 0, st, *p);
  return hipGetLastError();
}
