// Helpers of the attention kernels over a paged cache (attention_talk.hip,
// attention_paged.hip).
#pragma once
#include "common.h"
#include "mixer_params.h"

namespace lsd {
namespace {

constexpr int PAGE = 64;
constexpr float NEG = -1e30f;
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void from_f(float* o, float v) { *o = v; }
__device__ __forceinline__ void from_f(bf16* o, float v) { *o = f2bf(v); }

__device__ __forceinline__ int first_key(int pos, int window) { return window > pos ? 0 : pos - window + 1; }

// Tiles of TK keys that a range of queries reaches: [0, ns) for the kept first
// tokens, and [t0, t1) for the window.
struct KeyTiles {
  int ns, t0, t1;
  __device__ __forceinline__ int count() const { return ns + t1 - t0; }
  __device__ __forceinline__ int at(int i) const { return i < ns ? i : i - ns + t0; }
};
// queries at positions first .. last
template <int TK>
__device__ __forceinline__ KeyTiles key_tiles(int first, int last, int window, int keep) {
  KeyTiles t;
  t.t0 = first_key(first, window) / TK;
  t.ns = min((keep + TK - 1) / TK, t.t0);
  t.t1 = last / TK + 1;
  return t;
}
__device__ __forceinline__ bool seen(int key, int pos, int lo, int keep) { return key <= pos && (key >= lo || key < keep); }

__device__ __forceinline__ float sigmoid_x(float z) { return 1.f / (1.f + expf(-z)); }
template <typename T>
__device__ __forceinline__ float head_gate(const TalkParams& p, long row, int h) {
  return p.gate ? sigmoid_x(to_f(static_cast<const T*>(p.gate)[row * p.ldg + h])) : 1.f;
}

typedef _Float16 half8 __attribute__((ext_vector_type(8)));
typedef _Float16 half4 __attribute__((ext_vector_type(4)));
typedef _Float16 half2 __attribute__((ext_vector_type(2)));
__device__ __forceinline__ half2 pack_half(float a, float b) {  // rounds towards zero
  const auto h = __builtin_amdgcn_cvt_pkrtz(a, b);
  return __builtin_bit_cast(half2, h);
}

__device__ __forceinline__ f32x4 mfma_f16(half8 a, half8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_f16(a, b, c, 0, 0, 0);
}

// Transposed read of 4 x 16 LDS blocks: k runs over rows, the result's lanes over columns.
__device__ __forceinline__ bf16x4 ds_read_tr(const bf16* lds_ptr) {
  typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)(lds_ptr));
}

// This wave's LDS accesses are done
__device__ __forceinline__ void lds_fence() {
  __builtin_amdgcn_s_waitcnt(0xC07F);  // lgkmcnt(0)
  __builtin_amdgcn_wave_barrier();
}

// Two bf16 terms of eight weights
__device__ __forceinline__ void split_p(const float* a, const float* b, u32x4& hi, u32x4& lo) {
  const bf16x4 ha = pack4(f32x4{a[0], a[1], a[2], a[3]}), hb = pack4(f32x4{b[0], b[1], b[2], b[3]});
  const bf16x4 la = pack4(f32x4{a[0] - bf2f(ha[0]), a[1] - bf2f(ha[1]), a[2] - bf2f(ha[2]), a[3] - bf2f(ha[3])});
  const bf16x4 lb = pack4(f32x4{b[0] - bf2f(hb[0]), b[1] - bf2f(hb[1]), b[2] - bf2f(hb[2]), b[3] - bf2f(hb[3])});
  hi = __builtin_bit_cast(u32x4, (bf16x8{ha[0], ha[1], ha[2], ha[3], hb[0], hb[1], hb[2], hb[3]}));
  lo = __builtin_bit_cast(u32x4, (bf16x8{la[0], la[1], la[2], la[3], lb[0], lb[1], lb[2], lb[3]}));
}

constexpr int VLD = 64 + 8;  // row pitch of 64 staged V columns

}  // namespace
}  // namespace lsd
