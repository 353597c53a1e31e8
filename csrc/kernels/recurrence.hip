// Recurrent mixers: the gated delta rule with a decay per key channel, and
// Mamba-2 (state-space duality), each behind a short causal convolution.
//
//  * recur_seq: token by token, state in registers.  One launch does the
//    convolution, SiLU, unit norms, decay, state update and read-out, and for
//    the delta rule the output norm and gate.  Decode steps, and prompts of
//    models served in fp32.
//  * conv_tail: keeps the convolution's last inputs after a prompt portion.
//  * head_norm_gate / gated_group_norm: output norms of the unfused forms.
//
// State, decays, step sizes, gates of the recurrence and unit norms are fp32.
#include "common.h"
#include "mixer_params.h"

namespace lsd {
namespace {

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void from_f(float* o, float v) { *o = v; }
__device__ __forceinline__ void from_f(bf16* o, float v) { *o = f2bf(v); }

__device__ __forceinline__ float sigmoid_x(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float silu_x(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float softplus_x(float z) { return z > 20.f ? z : log1pf(expf(z)); }
constexpr float UNIT_EPS = 1e-6f;  // inside the root of a unit vector's length

// Convolution of channel `ch` at packed row `row`, token t of its portion,
// position pos, before bias and SiLU.
template <typename T>
__device__ __forceinline__ float conv_at(const ConvParams& c, int ch, long row, int t, int pos, int slot) {
  const T* y = static_cast<const T*>(c.y) + c.c0 + ch;
  const T* ring = static_cast<const T*>(c.ring) + (long)slot * c.taps * c.channels + ch;
  const float* w = c.w + (long)ch * c.taps;
  float a = 0.f;
  for (int j = 0; j < c.taps; ++j) {
    const int back = c.taps - 1 - j;
    if (back > pos) continue;
    const float x = back <= t ? to_f(y[(row - back) * c.ldy]) : to_f(ring[(long)((pos - back) % c.taps) * c.channels]);
    a = fmaf(w[j], x, a);
  }
  a *= c.gain;
  return c.bias ? a + c.bias[ch] : a;
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

// One (sequence, head, LV * 4 columns of the state) per block; thread (dg, lv)
// holds rows dg + i * 256 / LV of four columns.  Dynamic LDS: q, k, decays [D].
template <typename T, bool DELTA, int LV, int NR>
__global__ __launch_bounds__(256) void recur_seq_kernel(RecurParams p) {
  constexpr int VB = LV * 4, DG = 256 / LV;
  extern __shared__ float dyn[];
  __shared__ __attribute__((aligned(16))) float red[4][LV * 4];
  __shared__ float vs[VB];
  __shared__ float red1[16];
  const int D = p.D, tid = threadIdx.x;
  float *qs = dyn, *ks = dyn + D, *gs = dyn + 2 * D;
  const int nvb = (p.Vp + VB - 1) / VB;
  const int h = blockIdx.x / nvb, v0 = (blockIdx.x % nvb) * VB, b = blockIdx.y;
  const int rep = p.heads / p.groups, kh = h / rep;
  const int slot = p.s.slots[b], start = p.s.start[b], r0 = p.s.cu[b], n = p.s.cu[b + 1] - r0;
  if (n <= 0) return;
  const int lv = tid % LV, dg = tid / LV, col = v0 + lv * 4;
  const bool live = col < p.Vp;
  float* Sg = p.S + ((long)slot * p.heads + h) * D * p.Vp + col;
  f32x4 s[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) s[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  const float A = p.A[h];
  const float inv_sqrt_d = rsqrtf((float)D);

  for (int t = 0; t < n; ++t) {
    const long row = r0 + t;
    const int pos = start + t;
    for (int c = tid; c < 2 * D + VB; c += 256) {
      const int part = c < D ? 0 : c < 2 * D ? 1 : 2;
      const int i = part == 0 ? c : part == 1 ? c - D : c - 2 * D;
      const int ch = part == 0 ? p.q_ch + kh * D + i : part == 1 ? p.k_ch + kh * D + i : p.v_ch + h * p.V + v0 + i;
      const bool real = part < 2 || v0 + i < p.V;
      const float a = real ? silu_x(conv_at<T>(p.c, ch, row, t, pos, slot)) : 0.f;
      (part == 0 ? qs : part == 1 ? ks : vs)[i] = a;
      if (p.write_ring && real && (part == 2 || (h % rep == 0 && v0 == 0)))
        static_cast<T*>(p.c.ring)[((long)slot * p.c.taps + pos % p.c.taps) * p.c.channels + ch] =
            static_cast<const T*>(p.c.y)[row * p.c.ldy + p.c.c0 + ch];
    }
    const float gl = p.c.gain * to_f(static_cast<const T*>(p.c.y)[row * p.c.ldy + p.gate_col + h]);
    float beta = 0.f, a = 0.f, dt = 0.f;
    if constexpr (DELTA) {
      beta = sigmoid_x(gl);
      const T* low = static_cast<const T*>(p.low) + row * p.ldl + (long)h * D;
      for (int d = tid; d < D; d += 256)
        gs[d] = expf(A * softplus_x(p.c.gain * to_f(low[d]) + p.dt_bias[(long)h * D + d]));
    } else {
      dt = softplus_x(gl + p.dt_bias[h]);
      a = expf(A * dt);
    }
    if (t == 0 && start > 0 && live) {
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (dg + i * DG < D) s[i] = *reinterpret_cast<const f32x4*>(Sg + (long)(dg + i * DG) * p.Vp);
    }
    __syncthreads();
    f32x4 v = f32x4{vs[lv * 4], vs[lv * 4 + 1], vs[lv * 4 + 2], vs[lv * 4 + 3]};
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    if constexpr (DELTA) {
      float nq = 0.f, nk = 0.f;
      for (int d = lane_id(); d < D; d += 64) {
        nq += qs[d] * qs[d];
        nk += ks[d] * ks[d];
      }
      const float iq = inv_sqrt_d / sqrtf(wave_sum(nq) + UNIT_EPS), ik = 1.f / sqrtf(wave_sum(nk) + UNIT_EPS);
      f32x4 pr = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int d = dg + i * DG;
        if (d < D) {
          s[i] *= gs[d];
          pr += s[i] * (ks[d] * ik);
        }
      }
      pr = column_sum<LV>(pr, red);
      const f32x4 u = beta * (v - pr);
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int d = dg + i * DG;
        if (d < D) {
          s[i] += u * (ks[d] * ik);
          o += s[i] * (qs[d] * iq);
        }
      }
    } else {
      const f32x4 u = v * dt;
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int d = dg + i * DG;
        if (d < D) {
          s[i] = s[i] * a + u * ks[d];
          o += s[i] * qs[d];
        }
      }
    }
    o = column_sum<LV>(o, red);
    if constexpr (!DELTA) o += v * p.skip[h];
    if (p.raw) {
      if (dg == 0 && live) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < p.V) p.raw[row * p.ldr + (long)h * p.V + col + i] = o[i];
      }
    } else {  // DELTA, one block holds all of V: norm and gate here
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) ss += dg == 0 && col + i < p.V ? o[i] * o[i] : 0.f;
      const float rs = 1.f / sqrtf(block_sum(ss, red1) / p.V + p.eps);
      if (dg == 0) {
        const T* gate = static_cast<const T*>(p.low) + row * p.ldl + p.gate_off + (long)h * p.V;
        T* out = static_cast<T*>(p.out) + row * p.ldo;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < p.V)
            from_f(out + (long)h * p.V + col + i,
                   o[i] * rs * p.norm[col + i] * sigmoid_x(p.c.gain * to_f(gate[col + i])));
      }
      if (h == p.heads - 1)
        for (int c = p.heads * p.V + tid; c < p.out_cols; c += 256) from_f(static_cast<T*>(p.out) + row * p.ldo + c, 0.f);
    }
    __syncthreads();  // the next token overwrites q, k, v and the decays
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < NR; ++i)
      if (dg + i * DG < D) *reinterpret_cast<f32x4*>(Sg + (long)(dg + i * DG) * p.Vp) = s[i];
  }
}

// After a portion: the inputs of its last `taps` positions enter the ring.
template <typename T>
__global__ __launch_bounds__(256) void conv_tail_kernel(ConvParams c, SeqParams s) {
  const int b = blockIdx.y, n = s.cu[b + 1] - s.cu[b], k = blockIdx.z;
  const int ch = blockIdx.x * 256 + threadIdx.x;
  if (k >= n || ch >= c.channels) return;
  const long row = s.cu[b] + n - 1 - k;
  const int pos = s.start[b] + n - 1 - k;
  static_cast<T*>(c.ring)[((long)s.slots[b] * c.taps + pos % c.taps) * c.channels + ch] =
      static_cast<const T*>(c.y)[row * c.ldy + c.c0 + ch];
}

// One wave per (row, head): rms over vdim, times weight, times the sigmoid gate.
template <typename T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(MixOutParams p) {
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long)p.T * p.heads) return;
  const long row = item / p.heads;
  const int h = item % p.heads, lane = lane_id();
  const float* o = p.raw + row * p.ldr + (long)h * p.V;
  float ss = 0.f;
  for (int v = lane; v < p.V; v += 64) ss += o[v] * o[v];
  const float rs = 1.f / sqrtf(wave_sum(ss) / p.V + p.eps);
  const T* gate = static_cast<const T*>(p.low) + row * p.ldl + p.gate_off + (long)h * p.V;
  T* out = static_cast<T*>(p.out) + row * p.ldo;
  for (int v = lane; v < p.V; v += 64)
    from_f(out + (long)h * p.V + v, o[v] * rs * p.norm[v] * sigmoid_x(p.gain * to_f(gate[v])));
  if (h == p.heads - 1)
    for (int c = p.heads * p.V + lane; c < p.out_cols; c += 64) from_f(out + c, 0.f);
}

// One block per (row, norm group): y silu(z), rms over the group, times weight.
template <typename T>
__global__ __launch_bounds__(256) void gated_group_norm_kernel(MixOutParams p) {
  __shared__ float red[16];
  const long row = blockIdx.x;
  const int g = blockIdx.y, W = p.inner / p.groups;
  const float* y = p.raw + row * p.ldr + (long)g * W;
  const T* z = static_cast<const T*>(p.z) + row * p.ldz + (long)g * W;
  constexpr int KEEP = 16;
  float keep[KEEP];
  float ss = 0.f;
  for (int i = 0, c = threadIdx.x; c < W; ++i, c += 256) {
    const float v = y[c] * silu_x(p.gain * to_f(z[c]));
    if (i < KEEP) {
#pragma unroll
      for (int j = 0; j < KEEP; ++j)
        if (j == i) keep[j] = v;
    }
    ss += v * v;
  }
  const float rs = 1.f / sqrtf(block_sum(ss, red) / W + p.eps);
  T* out = static_cast<T*>(p.out) + row * p.ldo;
  for (int i = 0, c = threadIdx.x; c < W; ++i, c += 256) {
    float v = 0.f;
    if (i < KEEP) {
#pragma unroll
      for (int j = 0; j < KEEP; ++j)
        if (j == i) v = keep[j];
    } else {
      v = y[c] * silu_x(p.gain * to_f(z[c]));
    }
    from_f(out + (long)g * W + c, v * rs * p.norm[(long)g * W + c]);
  }
  if (g == p.groups - 1)
    for (int c = p.inner + threadIdx.x; c < p.out_cols; c += 256) from_f(out + c, 0.f);
}

// A loop's pass begins: rows [x | x0] for the projection, and x <- step.
template <typename T>
__global__ __launch_bounds__(256) void loop_pack_kernel(float* __restrict__ x, const float* __restrict__ x0,
                                                        const float* __restrict__ step, T* __restrict__ out, int H) {
  const long row = blockIdx.x;
  for (int c = threadIdx.x; c < H; c += 256) {
    from_f(out + row * 2 * H + c, x[row * H + c]);
    from_f(out + row * 2 * H + H + c, x0[row * H + c]);
    x[row * H + c] = step[c];
  }
}

// fp32 gated activation over [gate | up] rows in 16-row blocks: gelu(s g) (s u), exact
__global__ __launch_bounds__(256) void gelu_mul_f32_kernel(const float* __restrict__ y, float* __restrict__ out, long n,
                                                           int F, long ldo, float s) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const long row = i / F;
  const int f = i % F;
  const float* yr = y + row * 2 * F + (f >> 4) * 32 + (f & 15);
  const float g = yr[0] * s, u = yr[16] * s;
  out[row * ldo + f] = 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
}

}  // namespace
}  // namespace lsd

using namespace lsd;

// Columns of the state one recur_seq block holds (a power of two, 4 .. 128),
// 0: no kernel.  All of V in one block where that fits.
extern "C" int lsd_recur_block(int D, int V) {
  int vb = 4;
  while (vb < V && vb < 128) vb *= 2;
  while (vb > 4 && (long)((D + 1024 / vb - 1) / (1024 / vb)) > 16) vb /= 2;
  return (D + 1024 / vb - 1) / (1024 / vb) <= 16 ? vb : 0;
}

extern "C" hipError_t lsd_recur_seq(const RecurParams* p, int delta, int f32, hipStream_t st) {
  if (p->s.B == 0) return hipSuccess;
  const int vb = lsd_recur_block(p->D, p->V);
  if (vb == 0) return hipErrorInvalidValue;
  const int nvb = (p->Vp + vb - 1) / vb, dgs = 1024 / vb, nr = (p->D + dgs - 1) / dgs;
  if (!p->raw && (nvb != 1 || !delta)) return hipErrorInvalidValue;
  const dim3 grid(p->heads * nvb, p->s.B);
  const size_t lds = 3 * p->D * sizeof(float);
#define LSD_RS(T, DELTA, LV, NR) \
  hipLaunchKernelGGL((recur_seq_kernel<T, DELTA, LV, NR>), grid, dim3(256), lds, st, *p)
#define LSD_RS_N(T, DELTA, LV)                  \
  if (nr <= 1) LSD_RS(T, DELTA, LV, 1);         \
  else if (nr <= 2) LSD_RS(T, DELTA, LV, 2);    \
  else if (nr <= 4) LSD_RS(T, DELTA, LV, 4);    \
  else if (nr <= 8) LSD_RS(T, DELTA, LV, 8);    \
  else LSD_RS(T, DELTA, LV, 16);
#define LSD_RS_V(T, DELTA)                      \
  switch (vb) {                                 \
    case 4: LSD_RS_N(T, DELTA, 1) break;        \
    case 8: LSD_RS_N(T, DELTA, 2) break;        \
    case 16: LSD_RS_N(T, DELTA, 4) break;       \
    case 32: LSD_RS_N(T, DELTA, 8) break;       \
    case 64: LSD_RS_N(T, DELTA, 16) break;      \
    default: LSD_RS_N(T, DELTA, 32) break;      \
  }
  if (f32) {
    if (delta) {
      LSD_RS_V(float, true)
    } else {
      LSD_RS_V(float, false)
    }
  } else {
    if (delta) {
      LSD_RS_V(bf16, true)
    } else {
      LSD_RS_V(bf16, false)
    }
  }
#undef LSD_RS_V
#undef LSD_RS_N
#undef LSD_RS
  return hipGetLastError();
}

extern "C" hipError_t lsd_conv_tail(const ConvParams* c, const SeqParams* s, int f32, hipStream_t st) {
  if (s->B == 0) return hipSuccess;
  const dim3 grid((c->channels + 255) / 256, s->B, c->taps);
  if (f32) hipLaunchKernelGGL((conv_tail_kernel<float>), grid, dim3(256), 0, st, *c, *s);
  else hipLaunchKernelGGL((conv_tail_kernel<bf16>), grid, dim3(256), 0, st, *c, *s);
  return hipGetLastError();
}

extern "C" hipError_t lsd_head_norm_gate(const MixOutParams* p, int f32, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  const dim3 grid((unsigned)(((long)p->T * p->heads + 3) / 4));
  if (f32) hipLaunchKernelGGL((head_norm_gate_kernel<float>), grid, dim3(256), 0, st, *p);
  else hipLaunchKernelGGL((head_norm_gate_kernel<bf16>), grid, dim3(256), 0, st, *p);
  return hipGetLastError();
}

extern "C" hipError_t lsd_gated_group_norm(const MixOutParams* p, int f32, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  const dim3 grid(p->T, p->groups);
  if (f32) hipLaunchKernelGGL((gated_group_norm_kernel<float>), grid, dim3(256), 0, st, *p);
  else hipLaunchKernelGGL((gated_group_norm_kernel<bf16>), grid, dim3(256), 0, st, *p);
  return hipGetLastError();
}

extern "C" hipError_t lsd_loop_pack(float* x, const float* x0, const float* step, void* out, int T, int H, int f32,
                                    hipStream_t st) {
  if (T == 0) return hipSuccess;
  if (f32) hipLaunchKernelGGL((loop_pack_kernel<float>), dim3(T), dim3(256), 0, st, x, x0, step, static_cast<float*>(out), H);
  else hipLaunchKernelGGL((loop_pack_kernel<bf16>), dim3(T), dim3(256), 0, st, x, x0, step, static_cast<bf16*>(out), H);
  return hipGetLastError();
}

extern "C" hipError_t lsd_gelu_mul_f32(const float* y, float* out, int T, int F, long ldo, float s, hipStream_t st) {
  const long n = (long)T * F;
  if (n == 0) return hipSuccess;
  hipLaunchKernelGGL(gelu_mul_f32_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st, y, out, n, F, ldo, s);
  return hipGetLastError();
}
