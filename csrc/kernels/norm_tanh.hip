// Elementwise norms (dynamic tanh) fused with what stands around them.
//
//  * tanh_step: between two sublayers that are normed on both sides.  The
//    sublayer's output (split-K slabs) is summed, normed and added to the fp32
//    residual, and the residual normed (or narrowed) for what follows, in one
//    pass; nothing needs the rest of the row.
//  * shift_norm: in front of a mixer.  Folds the previous layer's token-side rows
//    (RMS norm of the summed slabs), norms the residual and moves every row
//    towards the previous token's.  A block walks a run of rows, the previous
//    row in registers; the residual goes to new rows, so that the row in front of
//    a run can be formed again.
//  * shift_tail: keeps a portion's last row for the next one.
#include "common.h"
#include "mixer_params.h"

namespace lsd {
namespace {

template <typename T> struct Quad { typedef f32x4 type; };
template <> struct Quad<bf16> { typedef bf16x4 type; };
__device__ __forceinline__ f32x4 get4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ bf16x4 get4(const bf16* p) { return ld4(p); }
__device__ __forceinline__ f32x4 wide4(f32x4 v) { return v; }
__device__ __forceinline__ f32x4 wide4(bf16x4 v) { return __builtin_convertvector(v, f32x4); }
__device__ __forceinline__ void put4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
__device__ __forceinline__ void put4(bf16* p, f32x4 v) { st4(p, pack4(v)); }

// tanh: an odd series near zero (no cancellation), else 1 - 2 / (1 + e^{2 |z|})
__device__ __forceinline__ float tanh_fast(float z) {
  const float a = fabsf(z), s = z * z;
  const float big = 1.f - 2.f * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(2.885390081777927f * a));
  float t = fmaf(s, 62.f / 2835.f, -17.f / 315.f);
  t = fmaf(s, t, 2.f / 15.f);
  t = fmaf(s, t, -1.f / 3.f);
  const float small = fmaf(s * t, a, a);
  return copysignf(a < 0.25f ? small : big, z);
}
template <typename T>
__device__ __forceinline__ f32x4 norm4(float alpha, f32x4 x, f32x4 w, f32x4 b) {
  f32x4 o;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float t = sizeof(T) == 2 ? tanh_fast(alpha * x[e]) : tanhf(alpha * x[e]);
    o[e] = fmaf(t, w[e], b[e]);
  }
  return o;
}
template <typename T>
__device__ __forceinline__ typename Quad<T>::type vec4(const void* p, int c) { return get4(static_cast<const T*>(p) + c); }

// Sum of the slabs at `at`, added in order, FLY of them in flight
template <typename S, int FLY>
__device__ __forceinline__ f32x4 slab_sum(const void* slab, int splits, long step, long at) {
  const S* s = static_cast<const S*>(slab) + at;
  f32x4 y = {0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < splits; k += FLY) {
    typename Quad<S>::type u[FLY];
#pragma unroll
    for (int j = 0; j < FLY; ++j) u[j] = get4(s + min(k + j, splits - 1) * step);
#pragma unroll
    for (int j = 0; j < FLY; ++j)
      if (k + j < splits) y += wide4(u[j]);
  }
  return y;
}

// Thread: four columns of RPT rows.
template <typename T, typename S, int RPT, int FLY>
__global__ __launch_bounds__(256) void tanh_step_kernel(TanhStepParams p) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (c >= p.H) return;
  const int n = p.rows ? p.n_rows : p.T, r0 = blockIdx.y * RPT;
  typedef typename Quad<T>::type Q;
  Q wp{}, bp{}, wq{}, bq{};
  if (p.slab) {
    wp = vec4<T>(p.post.w, c);
    bp = vec4<T>(p.post.b, c);
  }
  const bool norm = p.out && p.pre.w;
  if (norm) {
    wq = vec4<T>(p.pre.w, c);
    bq = vec4<T>(p.pre.b, c);
  }
  f32x4 x[RPT], y[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = min(r0 + i, n - 1);
    const long at = (long)(p.rows ? p.rows[r] : r) * p.H + c;
    x[i] = get4(p.x + at);
    if (p.slab) y[i] = slab_sum<S, FLY>(p.slab, p.splits, (long)p.T * p.H, at);
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = r0 + i;
    if (r >= n) return;
    if (p.slab) {
      x[i] += norm4<T>(p.post.alpha, y[i], wide4(wp), wide4(bp));
      put4(p.x + (long)r * p.H + c, x[i]);
    }
    if (p.out) put4(static_cast<T*>(p.out) + (long)r * p.H + c, norm ? norm4<T>(p.pre.alpha, x[i], wide4(wq), wide4(bq)) : x[i]);
  }
}

// One block per `run` rows; MAXC groups of four columns per thread.
template <typename T, typename S, int NT, int MAXC, int FLY>
__global__ __launch_bounds__(NT) void shift_norm_kernel(ShiftNormParams p, int run) {
  constexpr int NW = NT / 64;
  __shared__ float red[2][NW];
  const int row0 = blockIdx.x * run, row1 = min(p.T, row0 + run);
  const int tid = threadIdx.x, w = tid >> 6;
  typedef typename Quad<T>::type Q;
  int col[MAXC];
  bool on[MAXC];
  Q ws[MAXC], wn[MAXC], bn[MAXC], mx[MAXC];
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (tid + i * NT) * 4;
    on[i] = c < p.H;
    col[i] = min(c, p.H - 4);
    if (p.slab) ws[i] = vec4<T>(p.w_side, col[i]);
    wn[i] = vec4<T>(p.pre.w, col[i]);
    bn[i] = vec4<T>(p.pre.b, col[i]);
    mx[i] = vec4<T>(p.mix, col[i]);
  }
  // bit i: row row0 - 1 + i continues the row before it
  const int lane = lane_id(), at_row = row0 - 1 + lane;
  const bool cont = lane <= run + 1 && at_row > 0 && at_row < p.T && p.tslot[at_row] == p.tslot[at_row - 1] &&
                    p.tpos[at_row] == p.tpos[at_row - 1] + 1;
  const unsigned long long conts = __ballot(cont);
  auto follows = [&](int row) { return (conts >> (row - row0 + 1)) & 1; };
  f32x4 x[MAXC], y[MAXC], prev[MAXC], kept[MAXC];
  int slot = 0;
  auto load = [&](int row) {
    const long at = (long)row * p.H;
    if (row >= row0 && !follows(row)) {  // a portion begins: the row in front of it is kept, or zero
      slot = p.tslot[row];
      const bool zero = p.tpos[row] == 0;
#pragma unroll
      for (int i = 0; i < MAXC; ++i) kept[i] = zero ? f32x4{0.f, 0.f, 0.f, 0.f} : get4(p.last + (long)slot * p.H + col[i]);
    }
#pragma unroll
    for (int i = 0; i < MAXC; ++i) {
      x[i] = get4(p.x + at + col[i]);
      if (p.slab) y[i] = slab_sum<S, FLY>(p.slab, p.splits, (long)p.T * p.H, at + col[i]);
    }
  };
  const bool inside = follows(row0);
  const int first = inside ? row0 - 1 : row0;
  load(first);
  bool own = false;  // the current portion began in this run
  for (int row = first; row < row1; ++row) {
    f32x4 v[MAXC], z[MAXC];
    const bool begins = row >= row0 && !follows(row);
    const int mine = slot;
#pragma unroll
    for (int i = 0; i < MAXC; ++i) {
      v[i] = x[i];
      z[i] = y[i];
      if (begins) prev[i] = kept[i];
    }
    if (row + 1 < row1) load(row + 1);  // in flight under the sum
    if (p.slab) {
      float ss = 0.f;  // padding columns are zero
#pragma unroll
      for (int i = 0; i < MAXC; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += on[i] ? z[i][e] * z[i][e] : 0.f;
      ss = wave_sum(ss);
      float* rd = red[(row - first) & 1];  // alternating: one barrier a row
      if (lane_id() == 0) rd[w] = ss;
      __syncthreads();
      float all = 0.f;
#pragma unroll
      for (int i = 0; i < NW; ++i) all += rd[i];
      const float rs = 1.f / sqrtf(all / p.size + p.eps);
#pragma unroll
      for (int i = 0; i < MAXC; ++i) v[i] += z[i] * rs * wide4(ws[i]);
    }
    f32x4 h[MAXC];
#pragma unroll
    for (int i = 0; i < MAXC; ++i) h[i] = norm4<T>(p.pre.alpha, v[i], wide4(wn[i]), wide4(bn[i]));
    if (row >= row0) {
      own |= begins;
      const bool ends = own && !follows(row + 1);
#pragma unroll
      for (int i = 0; i < MAXC; ++i) {
        if (!on[i]) continue;
        if (p.slab) put4(p.x_new + (long)row * p.H + col[i], v[i]);
        put4(static_cast<T*>(p.out) + (long)row * p.H + col[i], h[i] + (prev[i] - h[i]) * wide4(mx[i]));
        // read by this thread alone, above
        if (ends) put4(p.last + (long)mine * p.H + col[i], h[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < MAXC; ++i) prev[i] = h[i];
  }
}

template <typename T>
__global__ __launch_bounds__(256) void shift_tail_kernel(ShiftNormParams p) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (c >= p.H) return;
  const int row = p.tail[blockIdx.y];
  const f32x4 h = norm4<T>(p.pre.alpha, get4(p.x + (long)row * p.H + c), wide4(vec4<T>(p.pre.w, c)), wide4(vec4<T>(p.pre.b, c)));
  put4(p.last + (long)p.tslot[row] * p.H + c, h);
}

template <typename T, typename S>
hipError_t tanh_step(const TanhStepParams& p, hipStream_t st) {
  const int n = p.rows ? p.n_rows : p.T, cols = (p.H + 1023) / 1024;
  if (n == 0) return hipSuccess;
#define LSD_TS(RPT, FLY) \
  hipLaunchKernelGGL((tanh_step_kernel<T, S, RPT, FLY>), dim3(cols, (n + RPT - 1) / RPT), dim3(256), 0, st, p)
  if (n <= 1024) {
    if (p.splits <= 1) LSD_TS(1, 1);
    else LSD_TS(1, 4);
  } else {
    if (p.splits <= 1) LSD_TS(4, 1);
    else if (p.splits <= 2) LSD_TS(4, 2);
    else LSD_TS(2, 4);
  }
#undef LSD_TS
  return hipGetLastError();
}

template <typename T, typename S>
hipError_t shift_norm(const ShiftNormParams& p, hipStream_t st) {
  if (p.T == 0) return hipSuccess;
  const int run = p.T <= 1024 ? 1 : p.T <= 16384 ? 8 : 16;
#define LSD_SN_F(NT, MAXC, FLY) \
  hipLaunchKernelGGL((shift_norm_kernel<T, S, NT, MAXC, FLY>), dim3((p.T + run - 1) / run), dim3(NT), 0, st, p, run)
#define LSD_SN(NT, MAXC)                      \
  do {                                        \
    if (p.splits <= 1) LSD_SN_F(NT, MAXC, 1); \
    else LSD_SN_F(NT, MAXC, 2);               \
  } while (0)
  const int chunks = (p.H + 2047) / 2048;  // of 512 threads
  if (p.H <= 1024) LSD_SN(256, 1);
  else if (chunks <= 1) LSD_SN(512, 1);
  else if (chunks <= 2) LSD_SN(512, 2);
  else if (chunks <= 4) LSD_SN(512, 4);
  else if (chunks <= 8) LSD_SN(512, 8);
  else return hipErrorInvalidValue;
#undef LSD_SN_F
#undef LSD_SN
  return hipGetLastError();
}

}  // namespace
}  // namespace lsd

using namespace lsd;

extern "C" hipError_t lsd_tanh_step(const TanhStepParams* p, int f32, hipStream_t st) {
  if (f32) return p->slab && p->slab_bf16 ? hipErrorInvalidValue : tanh_step<float, float>(*p, st);
  return p->slab_bf16 ? tanh_step<bf16, bf16>(*p, st) : tanh_step<bf16, float>(*p, st);
}

extern "C" hipError_t lsd_shift_norm(const ShiftNormParams* p, int f32, hipStream_t st) {
  if (f32) return p->slab && p->slab_bf16 ? hipErrorInvalidValue : shift_norm<float, float>(*p, st);
  return p->slab_bf16 ? shift_norm<bf16, bf16>(*p, st) : shift_norm<bf16, float>(*p, st);
}

extern "C" hipError_t lsd_shift_tail(const ShiftNormParams* p, int f32, hipStream_t st) {
  if (p->n_tail == 0) return hipSuccess;
  const dim3 grid((p->H + 1023) / 1024, p->n_tail);
  if (f32) hipLaunchKernelGGL((shift_tail_kernel<float>), grid, dim3(256), 0, st, *p);
  else hipLaunchKernelGGL((shift_tail_kernel<bf16>), grid, dim3(256), 0, st, *p);
  return hipGetLastError();
}
