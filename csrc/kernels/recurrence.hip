// Recurrent mixers: the gated delta rule with a decay per key channel, and
// Mamba-2 (state-space duality), each behind a short causal convolution.
//
//  * recur_seq: token by token, state in registers.  One launch does the
//    convolution, SiLU, unit norms, decay, state update and read-out, and for
//    the delta rule the output norm and gate.  Decode steps, and prompts of
//    models served in fp32.
//  * conv_silu, delta_chunk, ssd_chunk: prompts of bf16 models.  Chunks of 16
//    (delta rule) or 32 tokens (Mamba-2) become matrix products around a state
//    that stays in the accumulators of four waves, each owning columns of it; the
//    accumulator layout of one product is the operand layout of the next, so
//    state, pseudo-values and outputs never leave their wave.  fp32 operands
//    enter the matrix cores as two bf16 terms (three products, 16 bits each).
//  * conv_tail: keeps the convolution's last inputs after a prompt portion.
//  * head_norm_gate: the delta rule's output norm and gate where a head's values
//    take several blocks; group_norm: Mamba-2's output norm.
//
// State, decays, step sizes, gates of the recurrence and unit norms are fp32.
#include "common.h"
#include "mixer_params.h"
#include "recurrence.h"

namespace lsd {
namespace {

constexpr float UNIT_EPS = 1e-6f;  // inside the root of a unit vector's length

// Convolution of channel `ch` at packed row `row`, token t of its portion,
// position pos, before bias and SiLU.
template <typename T>
__device__ __forceinline__ float conv_at(const ConvParams& c, int ch, long row, int t, int pos, int slot) {
  const T* y = static_cast<const T*>(c.y) + c.c0 + ch;
  const T* ring = static_cast<const T*>(c.ring) + (long)slot * c.taps * c.channels + ch;
  const float* w = c.w + (long)ch * c.taps;
  float a = 0.f;
  if (c.taps <= 4) {  // every load in flight at once
    const int now = pos % c.taps;
    float x[4], wv[4];
#pragma unroll
    for (int back = 0; back < 4; ++back) {
      const bool live = back < c.taps && back <= pos;
      const int at = now >= back ? now - back : now - back + c.taps;
      const T* src = !live ? y + row * c.ldy : back <= t ? y + (row - back) * c.ldy : ring + (long)at * c.channels;
      const float v = to_f(*src);
      x[back] = live ? v : 0.f;
      wv[back] = w[max(0, c.taps - 1 - back)];
    }
#pragma unroll
    for (int back = 3; back >= 0; --back) a = fmaf(wv[back], x[back], a);
  } else {
    for (int j = 0; j < c.taps; ++j) {
      const int back = c.taps - 1 - j;
      if (back > pos) continue;
      const float x = back <= t ? to_f(y[(row - back) * c.ldy]) : to_f(ring[(long)((pos - back) % c.taps) * c.channels]);
      a = fmaf(w[j], x, a);
    }
  }
  a *= c.gain;
  return c.bias ? a + c.bias[ch] : a;
}

// One (sequence, head, LV * 4 columns of the state) per block; thread (dg, lv)
// holds rows dg + i * 256 / LV of four columns.  Dynamic LDS: q, k, decays [D].
template <typename T, bool DELTA, int LV, int NR>
__global__ __launch_bounds__(256, NR <= 8 ? 3 : 2) void recur_seq_kernel(RecurParams p) {
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
  for (int i = 0; i < NR; ++i) {
    s[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (start > 0 && live && dg + i * DG < D) s[i] = *reinterpret_cast<const f32x4*>(Sg + (long)(dg + i * DG) * p.Vp);
  }
  const float A = p.A[h];
  const float inv_sqrt_d = rsqrtf((float)D);

  for (int t = 0; t < n; ++t) {
    const long row = r0 + t;
    const int pos = start + t;
    // convolutions: q | k | v channels, a thread's first two together
    auto channel = [&](int c, int& ch, float*& dst) -> bool {
      const int part = c < D ? 0 : c < 2 * D ? 1 : 2;
      const int i = part == 0 ? c : part == 1 ? c - D : c - 2 * D;
      ch = part == 0 ? p.q_ch + kh * D + i : part == 1 ? p.k_ch + kh * D + i : p.v_ch + h * p.V + v0 + i;
      dst = (part == 0 ? qs : part == 1 ? ks : vs) + i;
      return part < 2 || v0 + i < p.V;
    };
    auto keep = [&](int c, int ch, bool real) {
      if (p.write_ring && real && (c >= 2 * D || (h % rep == 0 && v0 == 0)))
        static_cast<T*>(p.c.ring)[((long)slot * p.c.taps + pos % p.c.taps) * p.c.channels + ch] =
            static_cast<const T*>(p.c.y)[row * p.c.ldy + p.c.c0 + ch];
    };
    {
      int ch[2];
      float* dst[2];
      bool real[2];
      float a[2];
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        const int c = min(tid + 256 * q, 2 * D + VB - 1);
        real[q] = channel(c, ch[q], dst[q]);
        a[q] = conv_at<T>(p.c, real[q] ? ch[q] : 0, row, t, pos, slot);
      }
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        if (tid + 256 * q >= 2 * D + VB) continue;
        *dst[q] = real[q] ? silu_x(a[q]) : 0.f;
        keep(tid + 256 * q, ch[q], real[q]);
      }
    }
    for (int c = tid + 512; c < 2 * D + VB; c += 256) {
      int ch;
      float* dst;
      const bool real = channel(c, ch, dst);
      *dst = real ? silu_x(conv_at<T>(p.c, ch, row, t, pos, slot)) : 0.f;
      keep(c, ch, real);
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
    if constexpr (!DELTA) {  // y silu(z): the group norm follows
      if (dg == 0) {
        const T* z = static_cast<const T*>(p.c.y) + row * p.c.ldy + (long)h * p.V;
        T* out = static_cast<T*>(p.out) + row * p.ldo + (long)h * p.V;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < p.V) from_f(out + col + i, o[i] * silu_x(p.c.gain * to_f(z[col + i])));
      }
    } else if (p.raw) {
      if (dg == 0 && live) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < p.V) p.raw[row * p.ldr + (long)h * p.V + col + i] = o[i];
      }
    } else {  // one block holds all of V: norm and gate here
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

// Rows of SiLU(convolution), bf16, any tap count: one block per row and 256 channels.
__global__ __launch_bounds__(256) void conv_silu_any_kernel(ConvParams c, SeqParams s, bf16* __restrict__ out, long ldo) {
  const int row = blockIdx.x;
  int a = 0, b = s.B;  // sequence: last one with cu <= row
  while (b - a > 1) {
    const int m = (a + b) >> 1;
    if (s.cu[m] <= row) a = m;
    else b = m;
  }
  const int t = row - s.cu[a];
  const int ch = blockIdx.y * 256 + threadIdx.x;
  if (ch < c.channels) out[row * ldo + ch] = f2bf(silu_x(conv_at<bf16>(c, ch, row, t, s.start[a] + t, s.slots[a])));
}

// At most four taps, 8 channels per thread, CONV_RUN rows in turn: the taps and
// the last three inputs stay in registers.
constexpr int CONV_RUN = 32;
__global__ __launch_bounds__(256) void conv_silu_kernel(ConvParams c, SeqParams s, int T, bf16* __restrict__ out, long ldo) {
  const int row0 = blockIdx.x * CONV_RUN, row1 = min(T, row0 + CONV_RUN);
  int seq = 0, hi = s.B;  // sequence of row0: last one with cu <= row0
  while (hi - seq > 1) {
    const int m = (seq + hi) >> 1;
    if (s.cu[m] <= row0) seq = m;
    else hi = m;
  }
  const int ch = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (ch >= c.channels) return;
  const bf16* y = static_cast<const bf16*>(c.y) + c.c0 + ch;
  float w[4][8], bias[8];  // w[back]
#pragma unroll
  for (int e = 0; e < 8; ++e) {
#pragma unroll
    for (int back = 0; back < 4; ++back)
      w[back][e] = back < c.taps ? c.w[(long)(ch + e) * c.taps + c.taps - 1 - back] * c.gain : 0.f;
    bias[e] = c.bias ? c.bias[ch + e] : 0.f;
  }
  float past[3][8];
  bool fresh = true;
  int end = s.cu[seq + 1];
  auto emit = [&](const bf16x8& x, int row) {
    bf16x8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float now = bf2f(x[e]);
      float v = fmaf(w[0][e], now, bias[e]);
      v = fmaf(w[1][e], past[0][e], v);
      v = fmaf(w[2][e], past[1][e], v);
      v = fmaf(w[3][e], past[2][e], v);
      past[2][e] = past[1][e];
      past[1][e] = past[0][e];
      past[0][e] = now;
      o[e] = f2bf(silu(v));
    }
    st8(out + (long)row * ldo + ch, o);
  };
  for (int row = row0; row < row1;) {
    while (row >= end) {
      ++seq;
      end = s.cu[seq + 1];
      fresh = true;
    }
    if (fresh) {  // inputs before this row: of this portion, or of earlier ones
      const int t = row - s.cu[seq], pos = s.start[seq] + t;
      const bf16* ring = static_cast<const bf16*>(c.ring) + (long)s.slots[seq] * c.taps * c.channels + ch;
#pragma unroll
      for (int back = 1; back < 4; ++back) {
        bf16x8 v = {};
        if (back < c.taps && back <= pos)
          v = ld8(back <= t ? y + (long)(row - back) * c.ldy : ring + (long)((pos - back) % c.taps) * c.channels);
#pragma unroll
        for (int e = 0; e < 8; ++e) past[back - 1][e] = bf2f(v[e]);
      }
      fresh = false;
    }
    if (row + 8 <= min(row1, end)) {  // eight rows of one sequence: their loads together
      bf16x8 x[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) x[i] = ld8(y + (long)(row + i) * c.ldy);
#pragma unroll
      for (int i = 0; i < 8; ++i) emit(x[i], row + i);
      row += 8;
    } else {
      emit(ld8(y + (long)row * c.ldy), row);
      ++row;
    }
  }
}

// Chunked delta rule.  With G_t the summed log decays of the chunk up to token t
// (per key channel), S0 = diag(e^{G_0}) S and everything relative to G_0:
//   X = V - K~ S0          K~_t = k_t e^{G_t - G_0}
//   U = (I + A)^-1 diag(beta) X,   A_ts = beta_t sum_d K~_td k_sd e^{G_0 - G_s}  (s < t)
//   O = Q~ S0 + P U        P_ts = sum_d Q~_td k_sd e^{G_0 - G_s}                 (s <= t)
//   S = diag(e^{G_15 - G_0}) S0 + K^T U,   K^_s = k_s e^{G_15 - G_s}
// Every factor is at most e^80 in size; channels that decay by more than that
// within a chunk are left out of the two products over d and added term by term
// (e^{G_t - G_s} <= 1 always).  One block per (sequence, head).
template <int DKS, int VTW>
__global__ __launch_bounds__(256, 2) void delta_chunk_kernel(RecurParams p, const bf16* __restrict__ x, long ldx) {
  constexpr int CT = 16, DP = DKS * 32, DT = DKS * 2, LDD = DP + 8, LDT = CT + 4;
  constexpr float RANGE = 80.f;
  __shared__ __attribute__((aligned(16))) bf16 kt_h[CT * LDD], kt_l[CT * LDD], qt_h[CT * LDD], qt_l[CT * LDD];
  __shared__ __attribute__((aligned(16))) bf16 kc_h[CT * LDD], kc_l[CT * LDD];     // columns k_s e^{G_0 - G_s}
  __shared__ __attribute__((aligned(16))) bf16 kh_h[CT * LDD], kh_l[CT * LDD];     // K^
  __shared__ __attribute__((aligned(16))) float Gs[CT][DP], Ks[CT][DP], Qs[CT][DP];
  __shared__ __attribute__((aligned(16))) float e0[DP], s0[DP], er[DP], tot[4][DP], dtb[DP];
  __shared__ __attribute__((aligned(16))) bf16 tm_h[CT * LDT], tm_l[CT * LDT], pm_h[CT * LDT], pm_l[CT * LDT];
  __shared__ float betas[CT], red[4][CT];
  __shared__ int bad[DP], nbad;
  const int h = blockIdx.x, b = blockIdx.y, D = p.D, V = p.V;
  const int tid = threadIdx.x, lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int kh = h / (p.heads / p.groups);
  const int slot = p.s.slots[b], start = p.s.start[b], r0 = p.s.cu[b], n = p.s.cu[b + 1] - r0;
  if (n <= 0) return;
  float* Sg = p.S + ((long)slot * p.heads + h) * D * p.Vp;
  const float A = p.A[h], gain = p.c.gain;
  // uniform bases of the sequence's rows; offsets within a chunk are 32-bit
  const int ldxi = (int)ldx, ldl = (int)p.ldl, ldo = (int)p.ldo, ldy = (int)p.c.ldy;
  const bf16* yb = static_cast<const bf16*>(p.c.y) + r0 * p.c.ldy + p.gate_col + h;
  const bf16* xqb = x + r0 * ldx + p.q_ch + kh * D;
  const bf16* xkb = x + r0 * ldx + p.k_ch + kh * D;
  const bf16* xvb = x + r0 * ldx + p.v_ch + (long)h * V;
  const bf16* lowb = static_cast<const bf16*>(p.low) + r0 * p.ldl + (long)h * D;
  const bf16* gateb = static_cast<const bf16*>(p.low) + r0 * p.ldl + p.gate_off + (long)h * V;
  bf16* outb = static_cast<bf16*>(p.out) + r0 * p.ldo;

  // state: rows d = 16 dt + 4 g + i, columns v = 16 (w VTW + j) + r
  f32x4 S[DT][VTW];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int j = 0; j < VTW; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = dt * 16 + 4 * g + i, v = (w * VTW + j) * 16 + r;
        S[dt][j][i] = start > 0 && d < D && v < V ? Sg[d * p.Vp + v] : 0.f;
      }
  const float inv_sqrt_d = rsqrtf((float)D);
  float nrm[VTW];
#pragma unroll
  for (int j = 0; j < VTW; ++j) nrm[j] = p.norm[min((w * VTW + j) * 16 + r, V - 1)];
  // element work: token tid / 16, channels 8 (tid % 16) ..
  const int et = tid >> 4, ed = (tid & 15) * 8;
  const bool elive = ed < D;  // D % 8 == 0
  for (int d = tid; d < DP; d += 256) dtb[d] = d < D ? p.dt_bias[(long)h * D + d] : 0.f;
  __syncthreads();

  // rows of the next chunk, in flight under this one
  bf16x8 xq, xk, xl;
  float rb = 0.f;
  auto fetch = [&](int t0) {
    // clamped to valid rows and channels; what is not live counts as zero where it is used
    const int tr = min(et, n - 1 - t0), dc = elive ? ed : 0;
    const int ox = tr * ldxi + dc, ol = tr * ldl + dc;
    xq = ld8(xqb + (long)t0 * ldx + ox);
    xk = ld8(xkb + (long)t0 * ldx + ox);
    xl = ld8(lowb + (long)t0 * p.ldl + ol);
    rb = bf2f((yb + (long)t0 * p.c.ldy)[min(tid & 15, n - 1 - t0) * ldy]);
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += CT) {
    const int nt = min(CT, n - t0);
    const bool tlive = et < nt && elive;
    float q8[8], k8[8], lg[8];
    {
      float nq = 0.f, nk = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        q8[e] = elive ? bf2f(xq[e]) : 0.f;
        k8[e] = elive ? bf2f(xk[e]) : 0.f;
        nq = fmaf(q8[e], q8[e], nq);
        nk = fmaf(k8[e], k8[e], nk);
        lg[e] = tlive ? A * softplus_f(gain * bf2f(xl[e]) + dtb[ed + e]) : 0.f;
      }
#pragma unroll
      for (int off = 1; off < 16; off <<= 1) {
        nq += wave_xchg_n(nq, off);
        nk += wave_xchg_n(nk, off);
      }
      const float iq = tlive ? inv_sqrt_d * rsqrtf(nq + UNIT_EPS) : 0.f, ik = tlive ? rsqrtf(nk + UNIT_EPS) : 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        q8[e] *= iq;
        k8[e] *= ik;
      }
    }
    // log decays summed over the tokens: within the wave's four by lanes, across waves by LDS
    float pre[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      pre[e] = lg[e];
#pragma unroll
      for (int off = 16; off < 64; off <<= 1) {
        const float u = __shfl_up(pre[e], off, 64);
        if (lane >= off) pre[e] += u;
      }
    }
    if (ed < DP) {
      if (lane >= 48) {
        *reinterpret_cast<f32x4*>(&tot[w][ed]) = f32x4{pre[0], pre[1], pre[2], pre[3]};
        *reinterpret_cast<f32x4*>(&tot[w][ed + 4]) = f32x4{pre[4], pre[5], pre[6], pre[7]};
      }
      if (et == 0) {
        *reinterpret_cast<f32x4*>(&e0[ed]) = f32x4{lg[0], lg[1], lg[2], lg[3]};
        *reinterpret_cast<f32x4*>(&e0[ed + 4]) = f32x4{lg[4], lg[5], lg[6], lg[7]};
      }
    }
    if (tid < CT) betas[tid] = tid < nt ? sigmoid_x(gain * rb) : 0.f;
    if (t0 + CT < n) fetch(t0 + CT);
    if (tid == 0) nbad = 0;
    __syncthreads();
    if (ed < DP) {
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        asm volatile("" ::: "memory");  // four channels at a time
        const int d0 = ed + 4 * hf;
        const f32x4 g0 = *reinterpret_cast<const f32x4*>(&e0[d0]);
        f32x4 gt = {0.f, 0.f, 0.f, 0.f}, all = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const f32x4 v = *reinterpret_cast<const f32x4*>(&tot[q][d0]);
          if (q < w) gt += v;  // wave-uniform
          all += v;
        }
        f32x4 kt, qt, kc, kf;
        bool wides = false;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int e = 4 * hf + i;
          gt[i] += pre[e];
          const float G0 = g0[i], Gt = gt[i], Gc = all[i];
          const float E = exp_f(Gt - G0);
          const bool wide = G0 - Gc > RANGE;
          kt[i] = k8[e] * E;
          qt[i] = q8[e] * E;
          kc[i] = wide ? 0.f : k8[e] * exp_f(G0 - Gt);
          kf[i] = k8[e] * exp_f(Gc - Gt);
          wides |= wide;
          if (et == 15) {
            s0[ed + e] = exp_f(G0);
            er[ed + e] = exp_f(Gc - G0);
            if (wide) bad[atomicAdd(&nbad, 1)] = ed + e;
          }
        }
        if (wides) {  // the same channels for every token
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            Gs[et][d0 + i] = gt[i];
            Ks[et][d0 + i] = k8[4 * hf + i];
            Qs[et][d0 + i] = q8[4 * hf + i];
          }
        }
        auto put = [&](bf16* hp, bf16* lp, f32x4 v) {
          const bf16x4 a = hi4(v);
          st4(hp + et * LDD + d0, a);
          st4(lp + et * LDD + d0, lo4(v, a));
        };
        put(kt_h, kt_l, kt);
        put(qt_h, qt_l, qt);
        put(kc_h, kc_l, kc);
        put(kh_h, kh_l, kf);
      }
    }
    __syncthreads();
    // values and gates of the chunk in the accumulator layout (tokens 4 g + i, columns r)
    f32x4 vals[VTW], gates[VTW];
#pragma unroll
    for (int j = 0; j < VTW; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 4 * g + i, v = (w * VTW + j) * 16 + r;
        const bool live = t < nt && v < V;
        const int tc = min(t, nt - 1), vc = min(v, V - 1);
        const float xv = bf2f((xvb + (long)t0 * ldx)[tc * ldxi + vc]);
        vals[j][i] = live ? xv : 0.f;
        gates[j][i] = bf2f((gateb + (long)t0 * p.ldl)[tc * ldl + vc]);
      }
    // operand of row r: k-slots (g, j) <-> d = 32 ks + 4 g + j, 32 ks + 16 + 4 g + (j - 4)
    auto opnd = [&](const bf16* a, int ks) {
      return cat(ld4(a + r * LDD + ks * 32 + 4 * g), ld4(a + r * LDD + ks * 32 + 16 + 4 * g));
    };
    if (w < 2) {  // wave 0: A and (I + A)^-1, wave 1: P
      const bf16 *ah = w == 0 ? kt_h : qt_h, *al = w == 0 ? kt_l : qt_l;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) {
        asm volatile("" ::: "memory");  // operands of one step at a time
        acc = mfma3(opnd(ah, ks), opnd(al, ks), opnd(kc_h, ks), opnd(kc_l, ks), acc);
      }
      const int nb = nbad;
      for (int q = 0; q < nb; ++q) {
        const int d = bad[q];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 4 * g + i;
          if (r <= t) acc[i] += (w == 0 ? Ks[t][d] : Qs[t][d]) * Ks[r][d] * exp_f(Gs[t][d] - Gs[r][d]);
        }
      }
      if (w == 1) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 4 * g + i;
          const float v = r <= t ? acc[i] : 0.f;
          const bf16 a = f2bf(v);
          pm_h[t * LDT + r] = a;
          pm_l[t * LDT + r] = f2bf(v - bf2f(a));
        }
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[i] = r < 4 * g + i ? acc[i] * betas[4 * g + i] : 0.f;
        // column r of the inverse by forward substitution (each lane group alike);
        // A_ts is register t % 4 of lane 16 (t / 4) + s
        float inv[CT];
#pragma unroll
        for (int t = 0; t < CT; ++t) {
          float v = t == r ? 1.f : 0.f;
#pragma unroll
          for (int s = 0; s < t; ++s) {
            // (a bit cast of a vector's element would take element 0)
            const int a = __builtin_amdgcn_readlane(__float_as_int(acc[t & 3]), 16 * (t >> 2) + s);
            v = fmaf(-__int_as_float(a), inv[s], v);
          }
          inv[t] = v;
        }
        const float bt = betas[r];
        if (g == 0) {
#pragma unroll
          for (int t = 0; t < CT; ++t) {
            const float v = inv[t] * bt;
            const bf16 a = f2bf(v);
            tm_h[t * LDT + r] = a;
            tm_l[t * LDT + r] = f2bf(v - bf2f(a));
          }
        }
      }
    }
    f32x4 ks_acc[VTW], o[VTW];
#pragma unroll
    for (int j = 0; j < VTW; ++j) ks_acc[j] = o[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < DKS; ++ks) {
      if constexpr (VTW > 1) asm volatile("" ::: "memory");  // operands of one step at a time
      const f32x4 da = *reinterpret_cast<const f32x4*>(&s0[ks * 32 + 4 * g]);
      const f32x4 db = *reinterpret_cast<const f32x4*>(&s0[ks * 32 + 16 + 4 * g]);
      const bf16x8 kah = opnd(kt_h, ks), kal = opnd(kt_l, ks), qah = opnd(qt_h, ks), qal = opnd(qt_l, ks);
#pragma unroll
      for (int j = 0; j < VTW; ++j) {
        S[2 * ks][j] *= da;
        S[2 * ks + 1][j] *= db;
        bf16x8 sh, sl;
        split8(S[2 * ks][j], S[2 * ks + 1][j], sh, sl);
        ks_acc[j] = mfma3(kah, kal, sh, sl, ks_acc[j]);
        o[j] = mfma3(qah, qal, sh, sl, o[j]);
      }
    }
    __syncthreads();
    const bf16x4 th = ld4(tm_h + r * LDT + 4 * g), tl = ld4(tm_l + r * LDT + 4 * g);
    const bf16x4 ph = ld4(pm_h + r * LDT + 4 * g), pl = ld4(pm_l + r * LDT + 4 * g);
    bf16x4 uh[VTW], ul[VTW];
    f32x4 ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < VTW; ++j) {
      const f32x4 xv = vals[j] - ks_acc[j];
      const bf16x4 xh = hi4(xv), xl = lo4(xv, xh);
      f32x4 u = {0.f, 0.f, 0.f, 0.f};
      u = mfma3s(th, tl, xh, xl, u);
      uh[j] = hi4(u);
      ul[j] = lo4(u, uh[j]);
      o[j] = mfma3s(ph, pl, uh[j], ul[j], o[j]);
      ss += o[j] * o[j];  // columns beyond V are zero
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float v = ss[i];
#pragma unroll
      for (int off = 1; off < 16; off <<= 1) v += wave_xchg_n(v, off);
      if (r == 0) red[w][4 * g + i] = v;
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const f32x4 dec = *reinterpret_cast<const f32x4*>(&er[dt * 16 + 4 * g]);
      const int at = (4 * g + (r >> 2)) * LDD + dt * 16 + 4 * (r & 3);
      const bf16x4 ah = ds_read_tr(kh_h + at), al = ds_read_tr(kh_l + at);
#pragma unroll
      for (int j = 0; j < VTW; ++j) S[dt][j] = mfma3s(ah, al, uh[j], ul[j], S[dt][j] * dec);
    }
    __syncthreads();
    bf16* out = outb + (long)t0 * p.ldo;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 4 * g + i;
      if (t >= nt) continue;
      const float rs = rsqrtf((red[0][t] + red[1][t] + red[2][t] + red[3][t]) / V + p.eps);
#pragma unroll
      for (int j = 0; j < VTW; ++j) {
        const int v = (w * VTW + j) * 16 + r;
        if (v >= V) continue;
        out[t * ldo + h * V + v] =
            f2bf(o[j][i] * rs * nrm[j] * __builtin_amdgcn_rcpf(1.f + exp_f(-gain * gates[j][i])));
      }
    }
    if (h == p.heads - 1)
      for (int c = p.heads * V + (tid & 15); c < p.out_cols; c += 16)
        if (et < nt) out[et * ldo + c] = f2bf(0.f);
  }
  int g4 = 4 * g;
  asm volatile("" : "+v"(g4));  // addresses are formed anew: none stays in a register through the loop
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int j = 0; j < VTW; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = dt * 16 + g4 + i, v = (w * VTW + j) * 16 + r;
        if (d < D && v < p.Vp) Sg[d * p.Vp + v] = S[dt][j][i];
      }
}

// Chunked Mamba-2 over x [rows][x | B | C] behind convolution and SiLU (bf16).
// With a_t the summed log decays of the chunk up to token t:
//   y = diag(e^{a}) C S + P x + D x,   P_ts = (C_t . B_s) e^{a_t - a_s} dt_s  (s <= t)
//   S = e^{a_31} S + B^T diag(dt_s e^{a_31 - a_s}) x
// Rows y silu(z) leave in bf16 (z: the first columns of the in-projection).  One block per (sequence, head), wave w owns columns of the state.
template <int NKS, int VTW>
__global__ __launch_bounds__(256, 2) void ssd_chunk_kernel(RecurParams p, const bf16* __restrict__ x, long ldx) {
  constexpr int CT = 32, NP = NKS * 32, NT = NKS * 2, LDB = NP + 8, VP = VTW * 64, LDX = VP + 8;
  constexpr int NB = CT * NP / 1024, NX = CT * VP / 1024;  // groups of four elements per thread
  __shared__ __attribute__((aligned(16))) bf16 bs[2][CT * LDB], cs[2][CT * LDB], xs[2][CT * LDX];
  const int h = blockIdx.x, b = blockIdx.y, N = p.D, V = p.V;
  const int tid = threadIdx.x, lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int kg = h / (p.heads / p.groups);
  const int slot = p.s.slots[b], start = p.s.start[b], r0 = p.s.cu[b], n = p.s.cu[b + 1] - r0;
  if (n <= 0) return;
  float* Sg = p.S + ((long)slot * p.heads + h) * N * p.Vp;
  const float A = p.A[h], gain = p.c.gain, skip = p.skip[h], dtb = p.dt_bias[h];
  const bf16* y = static_cast<const bf16*>(p.c.y) + (long)r0 * p.c.ldy;
  const int ldxi = (int)ldx, ldy = (int)p.c.ldy, ldo = (int)p.ldo;  // offsets within a chunk are 32-bit
  const bf16* xb = x + r0 * ldx + p.k_ch + kg * N;
  const bf16* xc = x + r0 * ldx + p.q_ch + kg * N;
  const bf16* xv = x + r0 * ldx + p.v_ch + (long)h * V;

  f32x4 S[NT][VTW];
#pragma unroll
  for (int dt = 0; dt < NT; ++dt)
#pragma unroll
    for (int j = 0; j < VTW; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = dt * 16 + 4 * g + i, v = (w * VTW + j) * 16 + r;
        S[dt][j][i] = start > 0 && d < N && v < V ? Sg[d * p.Vp + v] : 0.f;
      }
  // rows of the next chunk, in flight under this one's products
  bf16x4 rb[NB], rc[NB], rx[NX];
  float rdt = 0.f;
  const int tl = lane & 31;
  auto fetch = [&](int t0) {
    const bf16x4 z = {};
#pragma unroll
    for (int q = 0; q < NB; ++q) {
      // clamped to valid rows (their dt is zero) and columns (zeros)
      const int c = tid + q * 256, t = min(c / (NP / 4), n - 1 - t0), d = (c % (NP / 4)) * 4;
      const int at = t * ldxi + min(d, N - 4);
      const bf16x4 vb = ld4(xb + (long)t0 * ldx + at), vc = ld4(xc + (long)t0 * ldx + at);
      rb[q] = d < N ? vb : z;
      rc[q] = d < N ? vc : z;
    }
#pragma unroll
    for (int q = 0; q < NX; ++q) {
      const int c = tid + q * 256, t = min(c / (VP / 4), n - 1 - t0), v = (c % (VP / 4)) * 4;
      const bf16x4 vx = ld4(xv + (long)t0 * ldx + t * ldxi + min(v, V - 4));
      rx[q] = v < V ? vx : z;
    }
    rdt = bf2f((y + (long)t0 * p.c.ldy + p.gate_col + h)[min(tl, n - 1 - t0) * ldy]);
  };
  fetch(0);
  for (int t0 = 0, buf = 0; t0 < n; t0 += CT, buf ^= 1) {
    const int nt = min(CT, n - t0);
    const bf16 *B = bs[buf], *C = cs[buf], *X = xs[buf];
#pragma unroll
    for (int q = 0; q < NB; ++q) {
      const int c = tid + q * 256, at = c / (NP / 4) * LDB + (c % (NP / 4)) * 4;
      st4(bs[buf] + at, rb[q]);
      st4(cs[buf] + at, rc[q]);
    }
#pragma unroll
    for (int q = 0; q < NX; ++q) {
      const int c = tid + q * 256;
      st4(xs[buf] + c / (VP / 4) * LDX + (c % (VP / 4)) * 4, rx[q]);
    }
    // lane t (and t + 32): step size and summed log decay
    const float dt = tl < nt ? softplus_f(gain * rdt + dtb) : 0.f;
    float a = A * dt;
#pragma unroll
    for (int off = 1; off < 32; off <<= 1) {
      const float u = __shfl_up(a, off, 32);
      if (tl >= off) a += u;
    }
    const float a_end = __shfl(a, 31, 64);
    const float wend = dt * exp_f(a_end - a);
    __syncthreads();  // the rows are there; the buffers written next were last read before this
    if (t0 + CT < n) fetch(t0 + CT);
    float zg[2][VTW][4];  // the gate of the rows and columns this lane ends with
#pragma unroll
    for (int mt = 0; mt < 2; ++mt)
#pragma unroll
      for (int j = 0; j < VTW; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = min(mt * 16 + 4 * g + i, nt - 1), v = min((w * VTW + j) * 16 + r, V - 1);
          zg[mt][j][i] = bf2f((y + (long)t0 * p.c.ldy + (long)h * V)[t * ldy + v]);
        }
    f32x4 as[2], ds[2], wv[2];  // a, dt and the state weights of rows 16 st + 4 g + i
#pragma unroll
    for (int st = 0; st < 2; ++st)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        as[st][i] = __shfl(a, st * 16 + 4 * g + i, 64);
        ds[st][i] = __shfl(dt, st * 16 + 4 * g + i, 64);
        wv[st][i] = __shfl(wend, st * 16 + 4 * g + i, 64);
      }
    // scores transposed (rows s, column t = r: the operand layout of P), and C S
    f32x4 sc[2][2], o[2][VTW];  // sc[s tile][t tile]
#pragma unroll
    for (int mt = 0; mt < 2; ++mt) {
#pragma unroll
      for (int st = 0; st < 2; ++st) sc[st][mt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < VTW; ++j) o[mt][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks) {
      const int at = r * LDB + ks * 32 + 4 * g;
      bf16x8 cf[2], bf[2];
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        cf[q] = cat(ld4(C + at + q * 16 * LDB), ld4(C + at + q * 16 * LDB + 16));
        bf[q] = cat(ld4(B + at + q * 16 * LDB), ld4(B + at + q * 16 * LDB + 16));
      }
      sc[0][0] = mfma16(bf[0], cf[0], sc[0][0]);
      sc[0][1] = mfma16(bf[0], cf[1], sc[0][1]);
      sc[1][1] = mfma16(bf[1], cf[1], sc[1][1]);
#pragma unroll
      for (int j = 0; j < VTW; ++j) {
        bf16x8 sh, sl;
        split8(S[2 * ks][j], S[2 * ks + 1][j], sh, sl);
#pragma unroll
        for (int mt = 0; mt < 2; ++mt) {
          o[mt][j] = mfma16(cf[mt], sh, o[mt][j]);
          o[mt][j] = mfma16(cf[mt], sl, o[mt][j]);
        }
      }
    }
    bf16x8 xf[VTW], uh[VTW], ul[VTW];
#pragma unroll
    for (int j = 0; j < VTW; ++j) {
      const bf16* xp = X + (4 * g + (r >> 2)) * LDX + (w * VTW + j) * 16 + 4 * (r & 3);
      xf[j] = cat(ds_read_tr(xp), ds_read_tr(xp + 16 * LDX));
      f32x4 u[2];
#pragma unroll
      for (int st = 0; st < 2; ++st)
#pragma unroll
        for (int i = 0; i < 4; ++i) u[st][i] = bf2f(xf[j][st * 4 + i]) * wv[st][i];
      split8(u[0], u[1], uh[j], ul[j]);
    }
#pragma unroll
    for (int mt = 0; mt < 2; ++mt) {
      const float at = __shfl(a, mt * 16 + r, 64);
      f32x4 pm[2];
#pragma unroll
      for (int st = 0; st < 2; ++st)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          pm[st][i] = st * 16 + 4 * g + i <= mt * 16 + r ? sc[st][mt][i] * ds[st][i] * exp_f(at - as[st][i]) : 0.f;
      bf16x8 ph, pl;
      split8(pm[0], pm[1], ph, pl);
      // rows t = 16 mt + 4 g + i: the decays of rows s with the same index
#pragma unroll
      for (int j = 0; j < VTW; ++j) {
#pragma unroll
        for (int i = 0; i < 4; ++i) o[mt][j][i] *= exp_f(as[mt][i]);
        o[mt][j] = mfma16(ph, xf[j], o[mt][j]);
        o[mt][j] = mfma16(pl, xf[j], o[mt][j]);
      }
    }
    const float dec = exp_f(a_end);
#pragma unroll
    for (int dt2 = 0; dt2 < NT; ++dt2) {
      const bf16* bp = B + (4 * g + (r >> 2)) * LDB + dt2 * 16 + 4 * (r & 3);
      const bf16x8 bf = cat(ds_read_tr(bp), ds_read_tr(bp + 16 * LDB));
#pragma unroll
      for (int j = 0; j < VTW; ++j) {
        S[dt2][j] *= dec;
        S[dt2][j] = mfma16(bf, uh[j], S[dt2][j]);
        S[dt2][j] = mfma16(bf, ul[j], S[dt2][j]);
      }
    }
    bf16* out = static_cast<bf16*>(p.out) + (long)(r0 + t0) * p.ldo + (long)h * V;
#pragma unroll
    for (int mt = 0; mt < 2; ++mt)
#pragma unroll
      for (int j = 0; j < VTW; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = mt * 16 + 4 * g + i, v = (w * VTW + j) * 16 + r;
          if (t < nt && v < V)
            out[t * ldo + v] = f2bf((o[mt][j][i] + skip * bf2f(xf[j][mt * 4 + i])) * silu(gain * zg[mt][j][i]));
        }
  }
  int g4 = 4 * g;
  asm volatile("" : "+v"(g4));  // addresses are formed anew: none stays in a register through the loop
#pragma unroll
  for (int dt = 0; dt < NT; ++dt)
#pragma unroll
    for (int j = 0; j < VTW; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = dt * 16 + g4 + i, v = (w * VTW + j) * 16 + r;
        if (d < N && v < p.Vp) Sg[d * p.Vp + v] = S[dt][j][i];
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

// One wave per (row, head): rms over vdim, times weight, times the sigmoid gate if there is one.
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
  const T* gate = p.low ? static_cast<const T*>(p.low) + row * p.ldl + p.gate_off + (long)h * p.V : nullptr;
  T* out = static_cast<T*>(p.out) + row * p.ldo;
  for (int v = lane; v < p.V; v += 64)
    from_f(out + (long)h * p.V + v, o[v] * rs * p.norm[v] * (gate ? sigmoid_x(p.gain * to_f(gate[v])) : 1.f));
  if (h == p.heads - 1)
    for (int c = p.heads * p.V + lane; c < p.out_cols; c += 64) from_f(out + c, 0.f);
}

// One wave per (row, norm group) of at most 1024 columns (a multiple of 4) of
// rows y silu(z), in place: rms over the group, times weight.
__global__ __launch_bounds__(256) void group_norm_wave_kernel(MixOutParams p) {
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long)p.T * p.groups) return;
  const int lane = lane_id(), g = (int)(item % p.groups), W = p.inner / p.groups;
  bf16* row = static_cast<bf16*>(p.out) + item / p.groups * p.ldo;
  bf16* out = row + (long)g * W;
  const float* wt = p.norm + (long)g * W;
  constexpr int KEEP = 4;  // groups of four columns per lane
  f32x4 v[KEEP], w[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = (lane + i * 64) * 4, at = min(c, W - 4);
    const bf16x4 x = ld4(out + at);
    w[i] = f32x4{wt[at], wt[at + 1], wt[at + 2], wt[at + 3]};
    v[i] = f32x4{bf2f(x[0]), bf2f(x[1]), bf2f(x[2]), bf2f(x[3])} * (c < W ? 1.f : 0.f);
    ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
  }
  const float rs = rsqrtf(wave_sum(ss) / W + p.eps);
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = (lane + i * 64) * 4;
    if (c < W) st4(out + c, pack4(v[i] * w[i] * rs));
  }
  if (g == p.groups - 1)
    for (int c = p.inner + lane; c < p.out_cols; c += 64) row[c] = f2bf(0.f);
}

// The same for any sizes, one block per (row, norm group).
template <typename T>
__global__ __launch_bounds__(256) void group_norm_kernel(MixOutParams p) {
  __shared__ float red[16];
  const long row = blockIdx.x;
  const int g = blockIdx.y, W = p.inner / p.groups;
  T* out = static_cast<T*>(p.out) + row * p.ldo + (long)g * W;
  const float* wt = p.norm + (long)g * W;
  constexpr int KEEP = 4;  // groups of four columns per thread
  bool vec = false;
  if constexpr (sizeof(T) == 2) vec = W % 4 == 0 && W <= KEEP * 1024;  // rows are 16-byte aligned
  if (vec) {
    bf16* ob = reinterpret_cast<bf16*>(out);
    f32x4 v[KEEP], w[KEEP];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      const int c = min((int)(threadIdx.x + i * 256) * 4, W - 4);
      const bf16x4 x = ld4(ob + c);
      w[i] = f32x4{wt[c], wt[c + 1], wt[c + 2], wt[c + 3]};
      const float live = (threadIdx.x + i * 256) * 4 < W ? 1.f : 0.f;
      v[i] = f32x4{bf2f(x[0]), bf2f(x[1]), bf2f(x[2]), bf2f(x[3])} * live;
      ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
    }
    const float rs = rsqrtf(block_sum(ss, red) / W + p.eps);
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      const int c = (threadIdx.x + i * 256) * 4;
      const f32x4 o = v[i] * w[i] * rs;
      if (c < W) st4(ob + c, bf16x4{f2bf(o[0]), f2bf(o[1]), f2bf(o[2]), f2bf(o[3])});
    }
  } else {
    float ss = 0.f;
    for (int c = threadIdx.x; c < W; c += 256) ss += to_f(out[c]) * to_f(out[c]);
    const float rs = 1.f / sqrtf(block_sum(ss, red) / W + p.eps);
    for (int c = threadIdx.x; c < W; c += 256) from_f(out + c, to_f(out[c]) * rs * wt[c]);
  }
  if (g == p.groups - 1)
    for (int c = p.inner + threadIdx.x; c < p.out_cols; c += 256) from_f(static_cast<T*>(p.out) + row * p.ldo + c, 0.f);
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

// fp32 gated activation over [gate | up] rows in 16-row blocks (common.h gated), exact: tanh-GELU or clamped
__global__ __launch_bounds__(256) void glu_f32_kernel(const float* __restrict__ y, float* __restrict__ out, long n, int F,
                                                      long ldo, int glu, float s) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const long row = i / F;
  const int f = i % F;
  const float* yr = y + row * 2 * F + (f >> 4) * 32 + (f & 15);
  if (glu == GLU_CLAMPED) {
    const float g = fminf(yr[0], s), u = fminf(fmaxf(yr[16], -s), s);
    out[row * ldo + f] = g / (1.f + expf(-GLU_ALPHA * g)) * (u + 1.f);
    return;
  }
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
  if (delta && !p->raw && nvb != 1) return hipErrorInvalidValue;
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

// Can the chunked kernels take these sizes?
extern "C" int lsd_chunk_ok(int delta, int D, int V, int groups, int heads) {
  if (D > 128 || V > 128) return 0;
  return delta ? D % 8 == 0 && V >= 1 : D % 4 == 0 && V % 4 == 0;
}

extern "C" hipError_t lsd_conv_silu(const ConvParams* c, const SeqParams* s, int T, bf16* out, long ldo, hipStream_t st) {
  if (T == 0) return hipSuccess;
  if (c->taps <= 4 && c->c0 % 8 == 0 && c->channels % 8 == 0)
    hipLaunchKernelGGL(conv_silu_kernel, dim3((T + CONV_RUN - 1) / CONV_RUN, (c->channels + 2047) / 2048), dim3(256), 0,
                       st, *c, *s, T, out, ldo);
  else
    hipLaunchKernelGGL(conv_silu_any_kernel, dim3(T, (c->channels + 255) / 256), dim3(256), 0, st, *c, *s, out, ldo);
  return hipGetLastError();
}

extern "C" hipError_t lsd_recur_chunk(const RecurParams* p, int delta, const bf16* x, long ldx, hipStream_t st) {
  if (p->s.B == 0) return hipSuccess;
  const dim3 grid(p->heads, p->s.B);
#define LSD_CK(KERNEL, KS)                                                                               \
  if (p->V <= 64) hipLaunchKernelGGL((KERNEL<KS, 1>), grid, dim3(256), 0, st, *p, x, ldx);                \
  else hipLaunchKernelGGL((KERNEL<KS, 2>), grid, dim3(256), 0, st, *p, x, ldx);
#define LSD_CK_D(KERNEL)                       \
  if (p->D <= 32) { LSD_CK(KERNEL, 1) }        \
  else if (p->D <= 64) { LSD_CK(KERNEL, 2) }   \
  else if (p->D <= 128) { LSD_CK(KERNEL, 4) }  \
  else return hipErrorInvalidValue;
  if (delta) {
    LSD_CK_D(delta_chunk_kernel)
  } else {
    LSD_CK_D(ssd_chunk_kernel)
  }
#undef LSD_CK_D
#undef LSD_CK
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

extern "C" hipError_t lsd_group_norm(const MixOutParams* p, int f32, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  const dim3 grid(p->T, p->groups);
  const int W = p->inner / p->groups;
  if (!f32 && W % 4 == 0 && W <= 1024)
    hipLaunchKernelGGL(group_norm_wave_kernel, dim3((unsigned)(((long)p->T * p->groups + 3) / 4)), dim3(256), 0, st, *p);
  else if (f32) hipLaunchKernelGGL((group_norm_kernel<float>), grid, dim3(256), 0, st, *p);
  else hipLaunchKernelGGL((group_norm_kernel<bf16>), grid, dim3(256), 0, st, *p);
  return hipGetLastError();
}

extern "C" hipError_t lsd_loop_pack(float* x, const float* x0, const float* step, void* out, int T, int H, int f32,
                                    hipStream_t st) {
  if (T == 0) return hipSuccess;
  if (f32) hipLaunchKernelGGL((loop_pack_kernel<float>), dim3(T), dim3(256), 0, st, x, x0, step, static_cast<float*>(out), H);
  else hipLaunchKernelGGL((loop_pack_kernel<bf16>), dim3(T), dim3(256), 0, st, x, x0, step, static_cast<bf16*>(out), H);
  return hipGetLastError();
}

extern "C" hipError_t lsd_glu_f32(const float* y, float* out, int T, int F, long ldo, int glu, float s, hipStream_t st) {
  const long n = (long)T * F;
  if (n == 0) return hipSuccess;
  hipLaunchKernelGGL(glu_f32_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st, y, out, n, F, ldo, glu, s);
  return hipGetLastError();
}
