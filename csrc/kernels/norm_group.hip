// RMS norms of a row's equal consecutive parts, and the step between two
// sublayers that are normed on both sides: the sublayer's output (split-K slabs
// and bias) is normed and added to the fp32 residual, and the residual normed for
// the next sublayer, in one pass.  Both norms work on the same parts, so a part
// of a row is all that a wave (or 16 lanes, or a block) ever needs.
#include "common.h"
#include "mixer_params.h"

namespace lsd {
namespace {

typedef float f32x1 __attribute__((ext_vector_type(1)));
template <int N> struct Vec;
template <> struct Vec<4> { typedef f32x4 type; };
template <> struct Vec<1> { typedef f32x1 type; };

// N elements as stored, and widened
template <typename T, int N> struct Raw { typedef typename Vec<N>::type type; };
template <int N> struct Raw<bf16, N> { typedef bf16 type __attribute__((ext_vector_type(N))); };
template <int N, typename T>
__device__ __forceinline__ typename Raw<T, N>::type load(const T* p) {
  if constexpr (N == 4 && sizeof(T) == 2) return ld4(p);
  else return *reinterpret_cast<const typename Raw<T, N>::type*>(p);
}
template <int N, typename R>
__device__ __forceinline__ typename Vec<N>::type wide(R v) {
  return __builtin_convertvector(v, typename Vec<N>::type);
}
template <int N>
__device__ __forceinline__ void store(float* p, typename Vec<N>::type v) {
  *reinterpret_cast<typename Vec<N>::type*>(p) = v;
}
template <int N>
__device__ __forceinline__ void store(bf16* p, typename Vec<N>::type v) {
  if constexpr (N == 4) st4(p, pack4(v));
  else *p = f2bf(v[0]);
}

// LPI lanes per (row, part), MAXC chunks of N columns each; FLY slabs (of S) in flight.
template <typename T, typename S, int N, int LPI, int MAXC, int FLY>
__global__ __launch_bounds__(256) void part_norm_kernel(GroupNormParams p) {
  typedef typename Vec<N>::type V;
  __shared__ float red[16];
  const int n_rows = p.rows ? p.n_rows : p.T, lane = threadIdx.x % LPI;
  const long at = (long)blockIdx.x * (256 / LPI) + threadIdx.x / LPI;
  const bool live = at < (long)n_rows * p.groups;
  const long item = live ? at : 0;
  const long row = item / p.groups;
  const int g = (int)(item % p.groups), size = p.size, c0 = g * size;
  const long src = p.rows ? p.rows[row] : row;
  float* x = p.x + src * p.H + c0;
  auto total = [&](float v) {
    if constexpr (LPI == 256) return block_sum(v, red);
    v += wave_xchg<1>(v);
    v += wave_xchg<2>(v);
    v += wave_xchg<4>(v);
    v += wave_xchg<8>(v);
    if constexpr (LPI > 16) {
      v += wave_xchg<16>(v);
      v += wave_xchg<32>(v);
    }
    return v;
  };
  int col[MAXC];
  bool on[MAXC];
  V v[MAXC];
  typename Raw<T, N>::type wp[MAXC];
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (lane + i * LPI) * N;
    on[i] = c < size;
    col[i] = min(c, size - N);
    v[i] = load<N>(x + col[i]);
    if (p.out) wp[i] = load<N>(static_cast<const T*>(p.w_pre) + c0 + col[i]);
  }
  if (p.slab) {
    V y[MAXC];
    typename Raw<T, N>::type w[MAXC];
#pragma unroll
    for (int i = 0; i < MAXC; ++i) {
      w[i] = load<N>(static_cast<const T*>(p.w_post) + c0 + col[i]);
      y[i] = V(0.f);
      if (p.bias) y[i] = wide<N>(load<N>(static_cast<const T*>(p.bias) + c0 + col[i]));
    }
    const long step = (long)p.T * p.H, first = src * p.H + c0;
    for (int s = 0; s < p.splits; s += FLY) {  // added in order
      typename Raw<S, N>::type u[MAXC][FLY];
#pragma unroll
      for (int j = 0; j < FLY; ++j) {
        const long sl = min(s + j, p.splits - 1) * step + first;
#pragma unroll
        for (int i = 0; i < MAXC; ++i) u[i][j] = load<N>(static_cast<const S*>(p.slab) + sl + col[i]);
      }
#pragma unroll
      for (int j = 0; j < FLY; ++j)
        if (s + j < p.splits) {
#pragma unroll
          for (int i = 0; i < MAXC; ++i) y[i] += wide<N>(u[i][j]);
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < MAXC; ++i)
#pragma unroll
      for (int e = 0; e < N; ++e) ss += on[i] ? y[i][e] * y[i][e] : 0.f;
    const float rs = 1.f / sqrtf(total(ss) / size + p.eps);
#pragma unroll
    for (int i = 0; i < MAXC; ++i) {
      v[i] += y[i] * rs * wide<N>(w[i]);
      if (live && on[i]) store<N>(x + col[i], v[i]);
    }
  }
  if (!p.out) return;  // uniform
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < MAXC; ++i)
#pragma unroll
    for (int e = 0; e < N; ++e) ss += on[i] ? v[i][e] * v[i][e] : 0.f;
  const float rs = 1.f / sqrtf(total(ss) / size + p.eps);
  T* out = static_cast<T*>(p.out) + row * p.H;
#pragma unroll
  for (int i = 0; i < MAXC; ++i)
    if (live && on[i]) store<N>(out + c0 + col[i], v[i] * rs * wide<N>(wp[i]));
  if (live && g == p.groups - 1)
    for (int c = p.groups * size + lane; c < p.H; c += LPI) out[c] = (T)0.f;
}

}  // namespace
}  // namespace lsd

using namespace lsd;

template <typename T, typename S>
static hipError_t group_norm(const GroupNormParams& p, hipStream_t st) {
  const int vec = p.size % 4 == 0 ? 4 : 1;
  const long items = (long)(p.rows ? p.n_rows : p.T) * p.groups;
  const int chunks = (p.size + vec - 1) / vec;
  if (items == 0) return hipSuccess;
#define LSD_GN_F(N, LPI, MAXC, FLY) \
  hipLaunchKernelGGL((part_norm_kernel<T, S, N, LPI, MAXC, FLY>), dim3((unsigned)((items * LPI + 255) / 256)), dim3(256), 0, st, p)
#define LSD_GN(N, LPI, MAXC)                                 \
  do {                                                       \
    if (p.splits <= 1) LSD_GN_F(N, LPI, MAXC, 1);            \
    else LSD_GN_F(N, LPI, MAXC, (MAXC > 4 ? 2 : 4));         \
  } while (0)
#define LSD_GN_N(N)                                         \
  if (chunks <= 16) LSD_GN(N, 16, 1);                       \
  else if (chunks <= 64) LSD_GN(N, 64, 1);                  \
  else if (chunks <= 128) LSD_GN(N, 64, 2);                 \
  else if (chunks <= 256) LSD_GN(N, 64, 4);                 \
  else if (chunks <= 512 && items >= 2048) LSD_GN(N, 64, 8);\
  else if (chunks <= 512) LSD_GN(N, 256, 2);                \
  else if (chunks <= 1024) LSD_GN(N, 256, 4);               \
  else if (chunks <= 2048) LSD_GN(N, 256, 8);               \
  else if (chunks <= 4096) LSD_GN(N, 256, 16);              \
  else return hipErrorInvalidValue;
  if (vec == 4) {
    LSD_GN_N(4)
  } else {
    LSD_GN_N(1)
  }
#undef LSD_GN_N
#undef LSD_GN
#undef LSD_GN_F
  return hipGetLastError();
}

extern "C" hipError_t lsd_group_rows_norm(const GroupNormParams* p, int f32, hipStream_t st) {
  if (f32) return p->slab && p->slab_bf16 ? hipErrorInvalidValue : group_norm<float, float>(*p, st);
  return p->slab_bf16 ? group_norm<bf16, bf16>(*p, st) : group_norm<bf16, float>(*p, st);
}
