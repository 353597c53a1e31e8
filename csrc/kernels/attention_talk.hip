// Attention over a paged K / V cache whose scores are capped and then mixed over
// the heads by a learned [H][H] matrix before the softmax, with grouped K / V
// heads, a sliding window, and rotation of part of a head's dimensions.
//
//  * rope_append: behind the in-projection, rotates q and k, appends k and v to
//    their page.
//  * talk_plain: one token per block, any sizes, bf16 or fp32.
//
// Every head's score of a (query, key) pair is needed before any head's weight
// of it is known, so a block works on all heads of its queries.
#include "common.h"
#include "mixer_params.h"

namespace lsd {
namespace {

constexpr int PAGE = 64;
constexpr float NEG = -1e30f;

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void from_f(float* o, float v) { *o = v; }
__device__ __forceinline__ void from_f(bf16* o, float v) { *o = f2bf(v); }

__device__ __forceinline__ int first_key(int pos, int window) { return window > pos ? 0 : pos - window + 1; }

// One block per token.
template <typename T>
__global__ __launch_bounds__(256) void rope_append_kernel(RopeAppendParams p) {
  const long row = blockIdx.x;
  const int pos = p.tpos[row], half = p.half;
  const long page = p.table[(long)p.tslot[row] * p.tw + pos / PAGE];
  const int nq = p.H * p.dim, nk = p.G * p.dim, nv = p.G * p.vdim;
  const T* y = static_cast<const T*>(p.y) + row * p.ldy;
  const float* cs = p.rope + (long)pos * half * 2;
  for (int i = threadIdx.x; i < nq + nk + nv; i += 256) {
    float v = to_f(y[i]) * p.gain;
    if (i < nq + nk) {
      const int d = i % p.dim;  // the k columns start at a multiple of dim
      if (d < half) v = v * cs[2 * d] - to_f(y[i + half]) * p.gain * cs[2 * d + 1];
      else if (d < 2 * half) v = v * cs[2 * (d - half)] + to_f(y[i - half]) * p.gain * cs[2 * (d - half) + 1];
    }
    if (i < nq) {
      from_f(static_cast<T*>(p.q) + row * nq + i, v);
    } else if (i < nq + nk) {
      const int g = (i - nq) / p.dim, d = (i - nq) % p.dim;
      from_f(static_cast<T*>(p.k) + ((page * p.G + g) * PAGE + pos % PAGE) * p.dim + d, v);
    } else {
      const int g = (i - nq - nk) / p.vdim, d = (i - nq - nk) % p.vdim;
      from_f(static_cast<T*>(p.v) + ((page * p.G + g) * PAGE + pos % PAGE) * p.vdim + d, v);
    }
  }
}

// One token per block, KT keys at a time.  Dynamic LDS: queries [H][dim], scores
// before and after mixing [H][KT + 1], outputs [H][vdim], and per head the
// running maximum, sum and rescaling factor.
constexpr int PLAIN_KT = 32;
template <typename T>
__global__ __launch_bounds__(256) void talk_plain_kernel(TalkParams p) {
  constexpr int KT = PLAIN_KT, LD = KT + 1;
  extern __shared__ float sh[];
  const int H = p.H, tid = threadIdx.x, rep = H / p.G;
  float* qs = sh;
  float* s0 = qs + H * p.dim;
  float* s1 = s0 + H * LD;
  float* acc = s1 + H * LD;
  float* m = acc + H * p.vdim;
  float* l = m + H;
  float* al = l + H;
  const long row = blockIdx.x;
  const int pos = p.pos[row], lo = first_key(pos, p.window);
  const int* table = p.table + (long)p.slots[row] * p.tw;
  const T* K = static_cast<const T*>(p.k);
  const T* V = static_cast<const T*>(p.v);
  const T* q = static_cast<const T*>(p.q) + row * H * p.dim;
  for (int i = tid; i < H * p.dim; i += 256) qs[i] = to_f(q[i]);
  for (int i = tid; i < H * p.vdim; i += 256) acc[i] = 0.f;
  for (int h = tid; h < H; h += 256) {
    m[h] = NEG;
    l[h] = 0.f;
  }
  __syncthreads();
  for (int k0 = lo; k0 <= pos; k0 += KT) {
    const int nk = min(KT, pos - k0 + 1);
    for (int i = tid; i < H * KT; i += 256) {
      const int h = i / KT, kk = i % KT, key = k0 + kk;
      float s = 0.f;
      if (kk < nk) {
        const T* kp = K + (((long)table[key / PAGE] * p.G + h / rep) * PAGE + key % PAGE) * p.dim;
        for (int d = 0; d < p.dim; ++d) s = fmaf(qs[h * p.dim + d], to_f(kp[d]), s);
        s *= p.scale;
        if (p.cap > 0.f) s = p.cap * tanhf(s / p.cap);
      }
      s0[h * LD + kk] = s;
    }
    __syncthreads();
    for (int i = tid; i < H * KT; i += 256) {
      const int h = i / KT, kk = i % KT;
      float s = 0.f;
      if (p.talk) {
        for (int g = 0; g < H; ++g) s = fmaf(p.talk[h * H + g], s0[g * LD + kk], s);
      } else {
        s = s0[h * LD + kk];
      }
      s1[h * LD + kk] = kk < nk ? s : NEG;
    }
    __syncthreads();
    for (int h = tid >> 6; h < H; h += 4) {  // a wave per head; lanes past the tile are neutral
      const int kk = lane_id();
      const float s = kk < KT ? s1[h * LD + kk] : NEG;
      const float mo = m[h], mn = fmaxf(mo, wave_max(s));
      const float e = kk < nk ? expf(s - mn) : 0.f;
      const float sum = wave_sum(e);
      if (kk < KT) s1[h * LD + kk] = e;
      if (kk == 0) {
        const float alpha = expf(mo - mn);
        m[h] = mn;
        l[h] = l[h] * alpha + sum;
        al[h] = alpha;
      }
    }
    __syncthreads();
    for (int i = tid; i < H * p.vdim; i += 256) {
      const int h = i / p.vdim, d = i % p.vdim;
      float a = acc[i] * al[h];
      for (int kk = 0; kk < nk; ++kk) {
        const int key = k0 + kk;
        a = fmaf(s1[h * LD + kk],
                 to_f(V[(((long)table[key / PAGE] * p.G + h / rep) * PAGE + key % PAGE) * p.vdim + d]), a);
      }
      acc[i] = a;
    }
    __syncthreads();
  }
  T* out = static_cast<T*>(p.out) + row * p.ldo;
  for (int i = tid; i < p.out_cols; i += 256) from_f(out + i, i < H * p.vdim ? acc[i] / l[i / p.vdim] : 0.f);
}

}  // namespace
}  // namespace lsd

using namespace lsd;

extern "C" hipError_t lsd_rope_append(const RopeAppendParams* p, int f32, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  if (f32) hipLaunchKernelGGL((rope_append_kernel<float>), dim3(p->T), dim3(256), 0, st, *p);
  else hipLaunchKernelGGL((rope_append_kernel<bf16>), dim3(p->T), dim3(256), 0, st, *p);
  return hipGetLastError();
}

extern "C" long lsd_talk_plain_lds(const TalkParams* p) {
  return 4L * (p->H * (p->dim + p->vdim + 2 * (PLAIN_KT + 1) + 3));
}

extern "C" hipError_t lsd_talk_plain(const TalkParams* p, int f32, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  const size_t lds = lsd_talk_plain_lds(p);
  const void* fn = f32 ? (const void*)talk_plain_kernel<float> : (const void*)talk_plain_kernel<bf16>;
  if (lds > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  if (f32) hipLaunchKernelGGL((talk_plain_kernel<float>), dim3(p->T), dim3(256), lds, st, *p);
  else hipLaunchKernelGGL((talk_plain_kernel<bf16>), dim3(p->T), dim3(256), lds, st, *p);
  return hipGetLastError();
}
