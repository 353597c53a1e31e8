// What the recurrent kernels share (recurrence.hip, recurrence_forget.hip): gate
// functions, sums over state rows, and matrix products of fp32 operands that are
// split in two bf16 terms.
#pragma once
#include "common.h"

namespace lsd {
namespace {

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void from_f(float* o, float v) { *o = v; }
__device__ __forceinline__ void from_f(bf16* o, float v) { *o = f2bf(v); }

__device__ __forceinline__ float sigmoid_x(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float silu_x(float z) { return z / (1.f + expf(-z)); }
// log(1 + e) = 2 atanh(s), s = e / (2 + e) <= 1/3 for e <= 1: the series is exact to fp32
__device__ __forceinline__ float log1p_series(float s) {
  const float q = s * s;
  float t = fmaf(q, 2.f / 15.f, 2.f / 13.f);
  t = fmaf(q, t, 2.f / 11.f);
  t = fmaf(q, t, 2.f / 9.f);
  t = fmaf(q, t, 2.f / 7.f);
  t = fmaf(q, t, 2.f / 5.f);
  t = fmaf(q, t, 2.f / 3.f);
  return fmaf(q * t, s, 2.f * s);
}
// log(1 + exp(z)) = max(z, 0) + log(1 + exp(-|z|)), small values to full relative precision
__device__ __forceinline__ float softplus_x(float z) {
  const float e = expf(-fabsf(z));
  return fmaxf(z, 0.f) + log1p_series(e / (2.f + e));
}
constexpr float LOG2E = 1.4426950408889634f;
// hardware exp2 / reciprocal (about an ulp each) for the chunked forms
__device__ __forceinline__ float exp_f(float z) { return __builtin_amdgcn_exp2f(z * LOG2E); }
__device__ __forceinline__ float softplus_f(float z) {
  const float e = exp_f(-fabsf(z));
  return fmaxf(z, 0.f) + log1p_series(e * __builtin_amdgcn_rcpf(2.f + e));
}
// Sum over the threads of equal (tid % LV): every thread gets its column group's total.
template <int LV>
__device__ __forceinline__ f32x4 column_sum(f32x4 v, float (*red)[LV * 4]) {
#pragma unroll
  for (int off = LV; off < 64; off <<= 1)
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] += shfl_xor(v[i], off);
  const int lane = lane_id(), w = threadIdx.x >> 6;
  __syncthreads();
  if (lane < LV) *reinterpret_cast<f32x4*>(&red[w][lane * 4]) = v;
  __syncthreads();
  const int lv = threadIdx.x % LV;
  f32x4 t = *reinterpret_cast<f32x4*>(&red[0][lv * 4]);
#pragma unroll
  for (int i = 1; i < 4; ++i) t += *reinterpret_cast<f32x4*>(&red[i][lv * 4]);
  return t;
}

typedef short s16x4 __attribute__((ext_vector_type(4)));

// A[row r][k = 4 g + j] . B[k = 4 g + j][col r]
__device__ __forceinline__ f32x4 mfma16k16(bf16x4 a, bf16x4 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_bit_cast(s16x4, a), __builtin_bit_cast(s16x4, b), c, 0, 0, 0);
}

__device__ __forceinline__ bf16x4 ds_read_tr(const bf16* lds_ptr) {
  typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)(lds_ptr));
}

__device__ __forceinline__ void lds_fence() {
  __builtin_amdgcn_s_waitcnt(0xC07F);  // lgkmcnt(0)
  __builtin_amdgcn_wave_barrier();
}

__device__ __forceinline__ bf16x4 hi4(f32x4 v) { return pack4(v); }
__device__ __forceinline__ bf16x4 lo4(f32x4 v, bf16x4 h) {
  return pack4(f32x4{v[0] - bf2f(h[0]), v[1] - bf2f(h[1]), v[2] - bf2f(h[2]), v[3] - bf2f(h[3])});
}
__device__ __forceinline__ bf16x8 cat(bf16x4 a, bf16x4 b) { return bf16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]}; }
// two bf16 terms of eight values (two accumulator tiles: k-slots 4 g + j and 16 + 4 g + j)
__device__ __forceinline__ void split8(f32x4 a, f32x4 b, bf16x8& hi, bf16x8& lo) {
  const bf16x4 ha = hi4(a), hb = hi4(b);
  hi = cat(ha, hb);
  lo = cat(lo4(a, ha), lo4(b, hb));
}
// a (two terms) . b (two terms)
__device__ __forceinline__ f32x4 mfma3(bf16x8 ah, bf16x8 al, bf16x8 bh, bf16x8 bl, f32x4 c) {
  c = mfma16(ah, bh, c);
  c = mfma16(ah, bl, c);
  return mfma16(al, bh, c);
}
__device__ __forceinline__ f32x4 mfma3s(bf16x4 ah, bf16x4 al, bf16x4 bh, bf16x4 bl, f32x4 c) {
  c = mfma16k16(ah, bh, c);
  c = mfma16k16(ah, bl, c);
  return mfma16k16(al, bh, c);
}

}  // namespace
}  // namespace lsd
