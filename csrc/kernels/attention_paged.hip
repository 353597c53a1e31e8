// Attention over a paged K / V cache without mixing of scores, what stands in
// front of it, and decode attention with mixed weights.
//
//  * rope_append_vec, conv_append, append_plain: behind the in-projection.
//  * paged_prefill: MFMA flash attention, 128 (64) queries of a head per block; or
//    only log2 of the softmax sums, for weights that are mixed over the heads.
//  * mix_prefill: MFMA, 16 queries of 4 heads per wave, all heads in a block, with
//    weights mixed over the heads.
//  * paged_decode: MFMA, a token's queries of one K / V head per wave.
//  * mix_decode, mix_combine: MFMA, one token of all heads per block.  With
//    W_g the unnormalised weights of head g over a block's keys,
//      out_h = sum_g T_hg / L_g  W_g V_kv(h),
//    so every head's weights meet the values of every K / V head (the columns of
//    a 16-wide product, which a group's own queries would leave empty), and the
//    mixing follows the merge of the key splits, with the sums L_g known.
//
// Softmax weights enter the matrix cores as two bf16 terms (value, remainder).
#include "attention_paged.h"

namespace lsd {
namespace {

// -- in front of the scores ----------------------------------------------------

// v[8] at columns c .. of a row's values: this layer's own are handed on, earlier ones mixed in
__device__ __forceinline__ void mix_value(const RopeAppendParams& p, long row, int c, float* v) {
  const long at = row * p.G * p.vdim + c;
  if (p.v_out) {
    bf16x8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = f2bf(v[e]);
    st8(static_cast<bf16*>(p.v_out) + at, o);
  }
  if (p.v_first) {
    const bf16x8 f = ld8(static_cast<const bf16*>(p.v_first) + at);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = (1.f - p.lam) * v[e] + p.lam * bf2f(f[e]);
  }
}

// 8 columns per thread; dims and the rotation's half are multiples of 8.  One
// block per four tokens, a wave each (several where tokens are few: blockIdx.y).
__global__ __launch_bounds__(256) void rope_append_vec_kernel(RopeAppendParams p) {
  const long row = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= p.T) return;
  const int pos = p.tpos[row], half = p.half;
  const long page = p.table[(long)p.tslot[row] * p.tw + pos / PAGE];
  const int nq = p.H * p.dim, nk = p.G * p.dim, nv = p.G * p.vdim;
  const bf16* y = static_cast<const bf16*>(p.y) + row * p.ldy;
  const float* cs = p.rope + (long)pos * half * 2;
  for (int i = blockIdx.y * 512 + lane_id() * 8; i < nq + nk + nv; i += 512 * gridDim.y) {
    const bf16x8 x = ld8(y + i);
    float v[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = bf2f(x[e]) * p.gain;
    const int d = i % p.dim;
    if (i < nq + nk && d < 2 * half) {
      const bool first = d < half;
      const bf16x8 o = ld8(first ? y + i + half : y + i - half);
      const float* c = cs + 2 * (first ? d : d - half);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float s = bf2f(o[e]) * p.gain * c[2 * e + 1];
        v[e] = fmaf(v[e], c[2 * e], first ? -s : s);
      }
    }
    if (i >= nq + nk) mix_value(p, row, i - nq - nk, v);
    bf16* dst;
    if (i < nq) dst = static_cast<bf16*>(p.q) + row * nq + i;
    else if (i < nq + nk) dst = static_cast<bf16*>(p.k) + ((page * p.G + (i - nq) / p.dim) * PAGE + pos % PAGE) * p.dim + d;
    else dst = static_cast<bf16*>(p.v) + ((page * p.G + (i - nq - nk) / p.vdim) * PAGE + pos % PAGE) * p.vdim +
               (i - nq - nk) % p.vdim;
    bf16x8 r;
#pragma unroll
    for (int e = 0; e < 8; ++e) r[e] = f2bf(v[e]);
    st8(dst, r);
  }
}

// Input `back` rows before packed row `row` of the sequence in `slot` at position
// pos: a row of the same portion, an earlier portion's (ring), or zero before the start.
template <typename T>
__device__ __forceinline__ const T* conv_input(const RopeAppendParams& p, long row, int slot, int pos, int back, int ch,
                                               int channels) {
  if (back > pos) return nullptr;
  if (row >= back && p.tslot[row - back] == slot && p.tpos[row - back] == pos - back)
    return static_cast<const T*>(p.y) + (row - back) * p.ldy + ch;
  return static_cast<const T*>(p.ring) + ((long)slot * p.n_taps + (pos - back) % p.n_taps) * channels + ch;
}

// Any sizes, every mechanism: one block per token, the row in (dynamic) LDS.
template <typename T>
__global__ __launch_bounds__(256) void append_plain_kernel(RopeAppendParams p) {
  extern __shared__ float xs[];
  const long row = blockIdx.x;
  const int pos = p.tpos[row], slot = p.tslot[row], half = p.half, tid = threadIdx.x;
  const long page = p.table[(long)slot * p.tw + pos / PAGE];
  const int nq = p.H * p.dim, nk = p.G * p.dim, nv = p.G * p.vdim, n = nq + nk + nv;
  float* rs = xs + n;  // [H + G]
  const T* y = static_cast<const T*>(p.y) + row * p.ldy;
  for (int i = tid; i < n; i += 256) {
    float v = to_f(y[i]) * p.gain;
    if (p.taps) {
      v = 0.f;
      for (int j = 0; j < p.n_taps; ++j) {
        const T* src = conv_input<T>(p, row, slot, pos, p.n_taps - 1 - j, i, n);
        if (src) v = fmaf(p.taps[(long)j * n + i], to_f(*src) * p.gain, v);
      }
      if (p.write_ring) static_cast<T*>(p.ring)[((long)slot * p.n_taps + pos % p.n_taps) * n + i] = y[i];
    }
    xs[i] = v;
  }
  __syncthreads();
  for (int h = tid >> 6; h < p.H + p.G; h += 4) {
    float ss = 0.f;
    if (p.eps >= 0.f)
      for (int d = lane_id(); d < p.dim; d += 64) ss += xs[h * p.dim + d] * xs[h * p.dim + d];
    ss = wave_sum(ss);
    if (lane_id() == 0) rs[h] = p.eps >= 0.f ? 1.f / sqrtf(ss / p.dim_own + p.eps) : 1.f;
  }
  __syncthreads();
  const float* cs = p.rope + (long)pos * half * 2;
  for (int i = tid; i < n; i += 256) {
    if (i < nq + nk) {
      const int h = i / p.dim, d = i % p.dim;  // the k columns start at a multiple of dim
      float v = xs[i];
      if (d < half) v = v * cs[2 * d] - xs[i + half] * cs[2 * d + 1];
      else if (d < 2 * half) v = v * cs[2 * (d - half)] + xs[i - half] * cs[2 * (d - half) + 1];
      v *= rs[h];
      if (i < nq) from_f(static_cast<T*>(p.q) + row * nq + i, v);
      else from_f(static_cast<T*>(p.k) + ((page * p.G + h - p.H) * PAGE + pos % PAGE) * p.dim + d, v);
    } else {
      const int c = i - nq - nk, g = c / p.vdim, d = c % p.vdim;
      float v = xs[i];
      if (p.v_out) from_f(static_cast<T*>(p.v_out) + row * nv + c, v);
      if (p.v_first) v = (1.f - p.lam) * v + p.lam * to_f(static_cast<const T*>(p.v_first)[row * nv + c]);
      from_f(static_cast<T*>(p.v) + ((page * p.G + g) * PAGE + pos % PAGE) * p.vdim + d, v);
    }
  }
}

// Convolution (at most four taps), unit norms, value mixing, append: LPH lanes of
// 8 columns hold one head, `run` rows in turn, FLY of one portion together; the taps
// and the last three inputs stay in registers.
template <int LPH, int FLY>
__global__ __launch_bounds__(256) void conv_append_kernel(RopeAppendParams p, int run) {
  const int units = p.H + 2 * p.G, lane = threadIdx.x % LPH;
  const long item = (long)blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  const long runs = (p.T + run - 1) / run;
  const bool live = item < runs * units;
  const int u = (int)((live ? item : 0) % units);
  const long row0 = (live ? item : 0) / units * run;
  const int n_rows = live ? (int)min((long)run, p.T - row0) : 0;
  const int nq = p.H * p.dim, nk = p.G * p.dim, channels = nq + nk + p.G * p.vdim;
  const bool is_v = u >= p.H + p.G, is_q = u < p.H;
  const int width = is_v ? p.vdim : p.dim, d = lane * 8;
  const int ch = (is_v ? nq + nk + (u - p.H - p.G) * p.vdim : u * p.dim) + min(d, width - 8);
  const bool mine = d < width;  // lanes behind the head's columns repeat its last ones
  float w[4][8];                // w[back]
#pragma unroll
  for (int back = 0; back < 4; ++back) {
    const f32x4* t = reinterpret_cast<const f32x4*>(p.taps + (long)max(0, p.n_taps - 1 - back) * channels + ch);
    const f32x4 a = t[0], b = t[1];
    const float f = back < p.n_taps ? p.gain : 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      w[back][e] = a[e] * f;
      w[back][4 + e] = b[e] * f;
    }
  }
  // convolution, norm and stores of one row; x[0] its input, x[1 ..] the ones before
  auto emit = [&](const bf16x8& x0, const bf16x8& x1, const bf16x8& x2, const bf16x8& x3, bool on, long row, int slot, int pos,
                  long page) {
    float v[8], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      v[e] = fmaf(w[3][e], bf2f(x3[e]), fmaf(w[2][e], bf2f(x2[e]), fmaf(w[1][e], bf2f(x1[e]), w[0][e] * bf2f(x0[e]))));
      ss = fmaf(v[e], mine ? v[e] : 0.f, ss);
    }
    if (p.eps >= 0.f) {
      ss += wave_xchg<1>(ss);
      ss += wave_xchg<2>(ss);
      if constexpr (LPH > 4) ss += wave_xchg<4>(ss);
      if constexpr (LPH > 8) ss += wave_xchg<8>(ss);
      if constexpr (LPH > 16) ss += wave_xchg<16>(ss);
      const float rs = is_v ? 1.f : 1.f / sqrtf(ss / p.dim_own + p.eps);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= rs;
    }
    if (!on || !mine) return;
    if (p.write_ring) st8(static_cast<bf16*>(p.ring) + ((long)slot * p.n_taps + pos % p.n_taps) * channels + ch, x0);
    if (is_v) mix_value(p, row, ch - nq - nk, v);
    const bf16x4 lo = pack4(f32x4{v[0], v[1], v[2], v[3]}), hi = pack4(f32x4{v[4], v[5], v[6], v[7]});
    bf16* dst = is_q ? static_cast<bf16*>(p.q) + row * nq + ch
                : is_v ? static_cast<bf16*>(p.v) + ((page * p.G + u - p.H - p.G) * PAGE + pos % PAGE) * p.vdim + d
                       : static_cast<bf16*>(p.k) + ((page * p.G + u - p.H) * PAGE + pos % PAGE) * p.dim + d;
    st8(dst, bf16x8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]});
  };
  auto before = [&](long row, int slot, int pos, int back) {
    const bf16x8 z = {};
    if (back >= p.n_taps) return z;
    const bf16* src = conv_input<bf16>(p, row, slot, pos, back, ch, channels);
    return src ? ld8(src) : z;
  };
  const bf16* y = static_cast<const bf16*>(p.y) + ch;
  bf16x8 x1, x2, x3;  // the inputs before the next row
  int slot = -1, pos = -2;
  for (int i = 0; i < run; i += FLY) {
    const long row = row0 + i;
    if (i + FLY <= n_rows && p.tslot[row + FLY - 1] == p.tslot[row] && p.tpos[row + FLY - 1] == p.tpos[row] + FLY - 1) {
      // rows of one portion (equal for all lanes of a head)
      bf16x8 x[FLY];
#pragma unroll
      for (int j = 0; j < FLY; ++j) x[j] = ld8(y + (row + j) * p.ldy);
      const int sl = p.tslot[row], ps = p.tpos[row];
      const int* table = p.table + (long)sl * p.tw;
      const long page0 = table[ps / PAGE], page1 = table[(ps + FLY - 1) / PAGE];
      if (sl != slot || ps != pos + 1) {
        x1 = before(row, sl, ps, 1);
        x2 = before(row, sl, ps, 2);
        x3 = before(row, sl, ps, 3);
      }
#pragma unroll
      for (int j = 0; j < FLY; ++j) {
        emit(x[j], x1, x2, x3, true, row + j, sl, ps + j, (ps + j) / PAGE == ps / PAGE ? page0 : page1);
        x3 = x2;
        x2 = x1;
        x1 = x[j];
      }
      slot = sl;
      pos = ps + FLY - 1;
    } else {
#pragma unroll 1
      for (int j = 0; j < FLY; ++j) {
        const bool on = i + j < n_rows;
        const long rw = on ? row + j : row0;
        const int sl = p.tslot[rw], ps = p.tpos[rw];
        emit(ld8(y + rw * p.ldy), before(rw, sl, ps, 1), before(rw, sl, ps, 2), before(rw, sl, ps, 3), on, rw, sl, ps,
             p.table[(long)sl * p.tw + ps / PAGE]);
      }
      slot = -1;
      pos = -2;
    }
  }
}

// -- prompts ---------------------------------------------------------------------

__device__ __forceinline__ bool grew(float tmax, float m) { return __any(tmax > m + 6.f); }

__device__ __forceinline__ void split4(const f32x4& a, const f32x4& b, bf16x8& hi, bf16x8& lo) {
  const float x[4] = {a[0], a[1], a[2], a[3]}, y[4] = {b[0], b[1], b[2], b[3]};
  u32x4 h, l;
  split_p(x, y, h, l);
  hi = __builtin_bit_cast(bf16x8, h);
  lo = __builtin_bit_cast(bf16x8, l);
}

// DP / VP: columns of K / V rows in LDS; QT 16-query tiles per wave.  LSE: only
// log2 of the softmax sums.  Scores are S^T = K Q^T, a query per lane, so their
// registers are the second product's operand.
template <int DP, int VP, int QT, bool LSE>
__global__ __launch_bounds__(256, 2) void paged_prefill_kernel(TalkParams p) {
  constexpr int KT = PAGE, LDK = DP + 8, LDV = VP + 8;
  constexpr int CK = KT * (DP / 8) / 256, CV = LSE ? 0 : KT * (VP / 8) / 256;
  __shared__ __attribute__((aligned(16))) bf16 ks[KT * LDK];
  __shared__ __attribute__((aligned(16))) bf16 vs[LSE ? 8 : KT * LDV];
  const int L = xcd_remap(blockIdx.x, gridDim.x);  // tiles of a head side by side on one XCD
  const int h = L / p.n_tiles, x = L % p.n_tiles, kvh = h / (p.H / p.G);
  const int seq = p.tiles[2 * x], off = p.tiles[2 * x + 1];
  const int cu = p.s.cu[seq], qlen = p.s.cu[seq + 1] - cu, st = p.s.start[seq];
  const int* table = p.table + (long)p.s.slots[seq] * p.tw;
  const int lane = lane_id(), w = threadIdx.x >> 6;
  const int r = lane & 15, g = lane >> 4;
  const bf16* K = static_cast<const bf16*>(p.k);
  const bf16* V = static_cast<const bf16*>(p.v);
  const float scale2 = p.scale * LOG2E, slope2 = p.slopes ? p.slopes[h] * LOG2E : 0.f;

  int qi[QT], my_pos[QT], my_lo[QT];
  bf16x8 qf[QT][DP / 32];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    qi[t] = off + (w * QT + t) * 16 + r;
    const int qc = min(qi[t], qlen - 1);
    my_pos[t] = st + qc;
    my_lo[t] = first_key(my_pos[t], p.window);
    const bf16* q = static_cast<const bf16*>(p.q) + ((long)(cu + qc) * p.H + h) * p.dim;
#pragma unroll
    for (int kk = 0; kk < DP / 32; ++kk) {
      const bf16x8 z = {};
      qf[t][kk] = kk * 32 < p.dim ? ld8(q + kk * 32 + g * 8) : z;
    }
  }
  const KeyTiles kts = key_tiles<KT>(st + off, st + min(off + 64 * QT, qlen) - 1, p.window, p.keep);
  const int n_kt = kts.count();

  f32x4 o[QT][LSE ? 1 : VP / 16];
  float m[QT], lsum[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    m[t] = NEG;
    lsum[t] = 0.f;
#pragma unroll
    for (int di = 0; di < (LSE ? 1 : VP / 16); ++di) o[t][di] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  bf16x8 kreg[CK], vreg[CV > 0 ? CV : 1];
  auto load_tile = [&](int it) {
    const long page = table[kts.at(it)];
    const bf16* kp = K + (page * p.G + kvh) * PAGE * p.dim;
    const bf16* vp = V + (page * p.G + kvh) * PAGE * p.vdim;
    const bf16x8 z = {};
#pragma unroll
    for (int c = 0; c < CK; ++c) {
      const int idx = threadIdx.x + c * 256, col = (idx % (DP / 8)) * 8;
      kreg[c] = col < p.dim ? ld8(kp + idx / (DP / 8) * p.dim + col) : z;
    }
#pragma unroll
    for (int c = 0; c < CV; ++c) {
      const int idx = threadIdx.x + c * 256, col = (idx % (VP / 8)) * 8;
      vreg[c] = col < p.vdim ? ld8(vp + idx / (VP / 8) * p.vdim + col) : z;
    }
  };
  load_tile(0);
  for (int it = 0; it < n_kt; ++it) {
    const int kt = kts.at(it);
    __syncthreads();
#pragma unroll
    for (int c = 0; c < CK; ++c) {
      const int idx = threadIdx.x + c * 256;
      st8(ks + (idx / (DP / 8)) * LDK + (idx % (DP / 8)) * 8, kreg[c]);
    }
#pragma unroll
    for (int c = 0; c < CV; ++c) {
      const int idx = threadIdx.x + c * 256;
      st8(vs + (idx / (VP / 8)) * LDV + (idx % (VP / 8)) * 8, vreg[c]);
    }
    __syncthreads();
    if (it + 1 < n_kt) load_tile(it + 1);

    f32x4 s[QT][KT / 16];
#pragma unroll
    for (int ni = 0; ni < KT / 16; ++ni) {
#pragma unroll
      for (int t = 0; t < QT; ++t) s[t][ni] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < DP / 32; ++kk) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(ks + (ni * 16 + r) * LDK + kk * 32 + g * 8);
#pragma unroll
        for (int t = 0; t < QT; ++t) s[t][ni] = mfma16(kf, qf[t][kk], s[t][ni]);
      }
    }
    // tiles every query of the wave sees whole need no mask
    const bool whole = (kt * KT >= my_lo[QT - 1] || (kt + 1) * KT <= p.keep) && (kt + 1) * KT - 1 <= my_pos[0];
    const bool all_whole = __all(whole);
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float tmax = NEG;
      const float bias0 = slope2 * (float)(kt * KT + 4 * g - my_pos[t]);
#pragma unroll
      for (int ni = 0; ni < KT / 16; ++ni)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = kt * KT + ni * 16 + 4 * g + i;
          float sv = fmaf(s[t][ni][i], scale2, fmaf(slope2, (float)(ni * 16 + i), bias0));
          if (!all_whole) sv = seen(key, my_pos[t], my_lo[t], p.keep) ? sv : NEG;
          s[t][ni][i] = sv;
          tmax = fmaxf(tmax, sv);
        }
      tmax = fmaxf(tmax, wave_xchg<16>(tmax));
      tmax = fmaxf(tmax, wave_xchg<32>(tmax));
      // weights are taken relative to m, which follows the running maximum only
      // when that is more than 2^6 ahead
      if (grew(tmax, m[t])) {
        const float mn = fmaxf(m[t], tmax);
        const float alpha = __builtin_amdgcn_exp2f(m[t] - mn);
        m[t] = mn;
        lsum[t] *= alpha;
        if constexpr (!LSE) {
#pragma unroll
          for (int di = 0; di < VP / 16; ++di) o[t][di] *= alpha;
        }
      }
      const float off2 = m[t] > 0.5f * NEG ? m[t] : 0.f;  // no key seen yet: weights of zero
      float ps = 0.f;
#pragma unroll
      for (int ni = 0; ni < KT / 16; ++ni)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = __builtin_amdgcn_exp2f(s[t][ni][i] - off2);
          s[t][ni][i] = e;
          ps += e;
        }
      lsum[t] += ps;
    }
    if constexpr (!LSE) {
#pragma unroll
      for (int kk = 0; kk < KT / 32; ++kk) {
        bf16x8 ph[QT], pl[QT];
#pragma unroll
        for (int t = 0; t < QT; ++t) split4(s[t][2 * kk], s[t][2 * kk + 1], ph[t], pl[t]);
        const int r0 = kk * 32 + 4 * g + (r >> 2);
#pragma unroll
        for (int di = 0; di < VP / 16; ++di) {
          const int col = di * 16 + 4 * (r & 3);
          const bf16x4 a = ds_read_tr(vs + r0 * LDV + col);
          const bf16x4 b = ds_read_tr(vs + (r0 + 16) * LDV + col);
          const bf16x8 vf = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
#pragma unroll
          for (int t = 0; t < QT; ++t) {
            o[t][di] = mfma16(vf, ph[t], o[t][di]);
            o[t][di] = mfma16(vf, pl[t], o[t][di]);
          }
        }
      }
    }
  }
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    float l = lsum[t];
    l += wave_xchg<16>(l);
    l += wave_xchg<32>(l);
    if (qi[t] >= qlen) continue;
    const long row = cu + qi[t];
    if constexpr (LSE) {
      if (g == 0) p.lse[row * p.H + h] = m[t] + log2f(l);
    } else {
      const float inv = head_gate<bf16>(p, row, h) / l;
      bf16* op = static_cast<bf16*>(p.out) + row * p.ldo;
#pragma unroll
      for (int di = 0; di < VP / 16; ++di)
        if (di * 16 < p.vdim) st4(op + h * p.vdim + di * 16 + 4 * g, pack4(o[t][di] * inv));
      if (h == p.H - 1)
        for (int c = p.H * p.vdim + g; c < p.out_cols; c += 4) op[c] = f2bf(0.f);
    }
  }
}

// Weights mixed over the heads, the softmax sums known (lse).  HP / 4 waves share 16
// queries, each scores its 4 heads and writes their weights (times 2^WSHIFT, which
// keeps small ones within fp16; two fp16 terms) to LDS.  Barrier.  Each wave then
// mixes the weights of all heads for some of the tile's 32 keys -- a product
// T [16 heads][heads] . weights [heads][16 queries] per key -- and writes the result
// (two bf16 terms) as the operand fragments of the second product.  Barrier.  Each
// wave multiplies its own heads' values.  Tile buffers:
//   S  [key][(term, 8 heads) HP / 4][query 16]   16-byte chunks of 8 heads; the two
//      4-head halves change places with bit 2 of the key, which spreads the banks
//   P  [term][head][k-slot group 4][query 16]    16-byte chunks of 8 keys: slot j of
//      group k <-> key 4 k + j (j < 4), 16 + 4 k + j - 4
// Wave w of a group mixes the keys of k-slot group w % 4 (and w + 2 with two waves).
constexpr float WSHIFT = 12.f, WUNIT = 1.f / 4096.f;
template <int DKS, int VT, int HP>
__global__ __launch_bounds__(HP == 32 ? 512 : 256, HP == 32 ? 1 : 2) void mix_prefill_kernel(TalkParams p) {
  constexpr int TK = 32, HW = HP / 4, NW = HW > 4 ? HW : 4, QG = NW / HW;
  constexpr int KCH = HP / 4 * 16;          // chunks of one key
  constexpr int SETS = HW == 2 ? 2 : 1;     // k-slot groups a wave mixes
  constexpr int VROW = 64;                  // staged V columns, 16-byte chunks swizzled by the row
  __shared__ __attribute__((aligned(16))) _Float16 ss[QG][TK * KCH * 8];
  __shared__ __attribute__((aligned(16))) bf16 pp[QG][2][HP * 64 * 8];
  __shared__ __attribute__((aligned(16))) bf16 vst[NW][TK * VROW];
  const int tile = xcd_remap(blockIdx.x, gridDim.x);
  const int seq = p.tiles[2 * tile], off = p.tiles[2 * tile + 1];
  const int cu = p.s.cu[seq], qlen = p.s.cu[seq + 1] - cu, st = p.s.start[seq];
  const int* table = p.table + (long)p.s.slots[seq] * p.tw;
  const bf16* K = static_cast<const bf16*>(p.k);
  const bf16* V = static_cast<const bf16*>(p.v);
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int hw = w % HW, qg = w / HW, H = p.H, G = p.G, rep = H / G, dim = p.dim, vdim = p.vdim;
  _Float16* sb = ss[qg];
  bf16* p_hi = pp[qg][0];
  bf16* p_lo = pp[qg][1];
  bf16* vs = vst[w];

  const int qi = off + qg * 16 + r, qc = min(qi, qlen - 1);
  const int my_pos = st + qc, my_lo = first_key(my_pos, p.window);
  const float scale2 = LOG2E * p.scale;
  int kv[4];
  float lse[4], slope[4];
#pragma unroll
  for (int hh = 0; hh < 4; ++hh) {
    const int h = min(hw * 4 + hh, H - 1);
    kv[hh] = h / rep;
    lse[hh] = p.lse[(long)(cu + qc) * H + h] - WSHIFT;
    slope[hh] = p.slopes ? p.slopes[h] * LOG2E : 0.f;
  }
  const int q_at = (cu + qc) * H * dim + g * 8;
  // rows of T for this wave's product: k-slots hold 8 heads of the chunk lane group g reads
  const int set0 = hw % 4, mt = HP == 32 ? hw / 4 : 0;
  half8 tf = {};
  {
    const int trow = mt * 16 + r, tcol = HP == 32 ? g * 8 : HP == 16 ? (g & 1) * 8 : 0;
    if (trow < HP && (HP > 8 || g < 2))
      tf = *reinterpret_cast<const half8*>(static_cast<const _Float16*>(p.talk_frag) + trow * HP + tcol);
    if (set0 & 1) tf = half8{tf[4], tf[5], tf[6], tf[7], tf[0], tf[1], tf[2], tf[3]};
  }

  f32x4 o[4][VT];
#pragma unroll
  for (int hh = 0; hh < 4; ++hh)
#pragma unroll
    for (int di = 0; di < VT; ++di) o[hh][di] = f32x4{0.f, 0.f, 0.f, 0.f};
  const KeyTiles kts = key_tiles<TK>(st + off, st + min(off + QG * 16, qlen) - 1, p.window, p.keep);
  int it0 = 0, it1 = kts.count();
  if (p.splits > 1) {
    const int per = (it1 + p.splits - 1) / p.splits;
    it0 = blockIdx.y * per;
    it1 = min(it1, it0 + per);
  }
  bf16x8 kf[2][DKS], vr[4];
  auto load_k = [&](int kt, int kvh) {
    const bf16* kp = K + (((long)table[kt * TK / PAGE] * G + kvh) * PAGE + kt * TK % PAGE + r) * dim + g * 8;
    const bf16x8 z = {};
#pragma unroll
    for (int ni = 0; ni < 2; ++ni)
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) kf[ni][ks] = ks * 32 < dim ? ld8(kp + ni * 16 * dim + ks * 32) : z;
  };
  auto load_v = [&](int kt, int kvh, int vh) {  // 64 columns of the tile's rows, 16 bytes per lane and 8 rows
    const bf16* vp = V + (((long)table[kt * TK / PAGE] * G + kvh) * PAGE + kt * TK % PAGE) * vdim + vh * 64;
    const int col = (lane & 7) * 8;
    const bf16x8 z = {};
#pragma unroll
    for (int c = 0; c < 4; ++c) vr[c] = vh * 64 + col < vdim ? ld8(vp + (c * 8 + (lane >> 3)) * vdim + col) : z;
  };
  const int s_wr = (hw >> 1) * 128 + r * 8;        // + key, term, half
  const int r0 = 4 * g + (r >> 2), sw = (r0 >> 1) & 7;
  if (it0 < it1) load_k(kts.at(it0), kv[0]);
  for (int it = it0; it < it1; ++it) {
    const int kt = kts.at(it), next = kts.at(min(it + 1, it1 - 1));
    // scores of the own heads; the queries are read again for every tile (from
    // L1 / L2): the outputs take the registers
    f32x4 s[4][2];
    const bf16* qb = static_cast<const bf16*>(p.q);
    asm volatile("" : "+s"(qb));  // not hoisted out of the loop
#pragma unroll
    for (int hh = 0; hh < 4; ++hh) {
      if (hh > 0 && kv[hh] != kv[hh - 1]) load_k(kt, kv[hh]);  // wave-uniform
      const bf16x8 z = {};
      bf16x8 qf[DKS];
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) qf[ks] = ks * 32 < dim ? ld8(qb + q_at + min(hw * 4 + hh, H - 1) * dim + ks * 32) : z;
#pragma unroll
      for (int ni = 0; ni < 2; ++ni) {
        s[hh][ni] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < DKS; ++ks) s[hh][ni] = mfma16(kf[ni][ks], qf[ks], s[hh][ni]);
      }
    }
    const bool whole = (kt * TK >= my_lo || kt * TK + TK <= p.keep) && kt * TK + TK - 1 <= my_pos;
    const bool all_whole = __all(whole);
#pragma unroll
    for (int ni = 0; ni < 2; ++ni)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int in = ni * 16 + 4 * g + i, key = kt * TK + in;
        const float dist = (float)(key - my_pos);
        float e[4];
#pragma unroll
        for (int hh = 0; hh < 4; ++hh)
          e[hh] = __builtin_amdgcn_exp2f(fmaf(s[hh][ni][i], scale2, fmaf(slope[hh], dist, -lse[hh])));
        if (!all_whole && !seen(key, my_pos, my_lo, p.keep)) e[0] = e[1] = e[2] = e[3] = 0.f;
        // the remainder makes up for the truncated first term
        const half2 a = pack_half(e[0], e[1]), b = pack_half(e[2], e[3]);
        const half2 c = pack_half(e[0] - (float)a[0], e[1] - (float)a[1]), d = pack_half(e[2] - (float)b[0], e[3] - (float)b[1]);
        const int at = in * KCH * 8 + s_wr + ((hw ^ g) & 1) * 4;  // bit 2 of the key is g & 1
        *reinterpret_cast<half4*>(sb + at) = half4{a[0], a[1], b[0], b[1]};
        *reinterpret_cast<half4*>(sb + at + HP / 8 * 128) = half4{c[0], c[1], d[0], d[1]};
      }
    __syncthreads();
#pragma unroll
    for (int q = 0; q < SETS; ++q) {
      const int set = set0 + 2 * q;
      f32x4 acc[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int in = (j < 4 ? 0 : 16) + 4 * set + (j & 3);
        const _Float16* src = sb + (in * KCH + g * 16 + r) * 8;
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        half8 a = {};
        if (HP > 8 || g < 2) a = *reinterpret_cast<const half8*>(src);
        acc[j] = mfma_f16(tf, a, zero);
        if constexpr (HP == 32) acc[j] = mfma_f16(tf, *reinterpret_cast<const half8*>(src + 4 * 128), acc[j]);
      }
      if (q == SETS - 1) load_v(kt, kv[0], 0);  // in flight until the barrier
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int h = mt * 16 + 4 * g + i;
        const float x[4] = {acc[0][i], acc[1][i], acc[2][i], acc[3][i]}, y[4] = {acc[4][i], acc[5][i], acc[6][i], acc[7][i]};
        u32x4 hi, lo;
        split_p(x, y, hi, lo);
        if (HP > 8 || g < 2) {
          *reinterpret_cast<u32x4*>(p_hi + ((h * 4 + set) * 16 + r) * 8) = hi;
          *reinterpret_cast<u32x4*>(p_lo + ((h * 4 + set) * 16 + r) * 8) = lo;
        }
      }
    }
    __syncthreads();
    load_k(next, kv[0]);  // in flight under the product
#pragma unroll
    for (int hh = 0; hh < 4; ++hh) {
      if (hh > 0 && kv[hh] == kv[hh - 1]) continue;  // done with the head before
      if (hh > 0) load_v(kt, kv[hh], 0);
#pragma unroll
      for (int vh = 0; vh < VT / 4; ++vh) {
        if (vh * 64 >= vdim) continue;
        lds_fence();  // reads of what is staged now are done
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          const int row = c * 8 + (lane >> 3);
          st8(vs + row * VROW + (((lane & 7) ^ ((row >> 1) & 7)) * 8), vr[c]);
        }
        if ((vh + 1) * 64 < vdim) load_v(kt, kv[hh], vh + 1);
        lds_fence();
        bf16x8 vf[4];
#pragma unroll
        for (int dj = 0; dj < 4; ++dj) {
          const bf16* vp = vs + r0 * VROW + (((dj * 2 + ((r & 3) >> 1)) ^ sw) * 8) + (r & 1) * 4;
          const bf16x4 a = ds_read_tr(vp);
          const bf16x4 b = ds_read_tr(vp + 16 * VROW);
          vf[dj] = bf16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
        }
#pragma unroll
        for (int h2 = 0; h2 < 4; ++h2)
          if (h2 >= hh && kv[h2] == kv[hh]) {  // wave-uniform
            const int at = (((hw * 4 + h2) * 4 + g) * 16 + r) * 8;
            const bf16x8 ph = ld8(p_hi + at), pl = ld8(p_lo + at);
#pragma unroll
            for (int dj = 0; dj < 4; ++dj) {
              o[h2][vh * 4 + dj] = mfma16(vf[dj], ph, o[h2][vh * 4 + dj]);
              o[h2][vh * 4 + dj] = mfma16(vf[dj], pl, o[h2][vh * 4 + dj]);
            }
          }
      }
    }
  }
#pragma unroll
  for (int hh = 0; hh < 4; ++hh) {
    const int h = hw * 4 + hh;
    if (h >= H || qi >= qlen) continue;
    if (p.splits > 1) {  // the partial sums of key splits simply add up: equal maxima, sums of 1 in all
      const long pi = ((long)(cu + qi) * H + h) * p.splits + blockIdx.y;
#pragma unroll
      for (int di = 0; di < VT; ++di)
        if (di * 16 < vdim) *reinterpret_cast<f32x4*>(p.part_o + pi * vdim + di * 16 + 4 * g) = o[hh][di] * WUNIT;
      if (g == 0) {
        p.part_ml[2 * pi] = 0.f;
        p.part_ml[2 * pi + 1] = 1.f / p.splits;
      }
      continue;
    }
    const float f = WUNIT * head_gate<bf16>(p, cu + qi, h);
    bf16* out = static_cast<bf16*>(p.out) + (long)(cu + qi) * p.ldo + h * vdim;
#pragma unroll
    for (int di = 0; di < VT; ++di)
      if (di * 16 < vdim) st4(out + di * 16 + 4 * g, pack4(o[hh][di] * f));
  }
  if (p.splits == 1 && hw == HW - 1 && qi < qlen)
    for (int c = H * vdim + g; c < p.out_cols; c += 4) static_cast<bf16*>(p.out)[(long)(cu + qi) * p.ldo + c] = f2bf(0.f);
}

// -- decode ----------------------------------------------------------------------

// One wave per (token, K / V head, key split): its rep <= 16 queries are the
// columns of the score product.  32-key tiles of K and V, streamed through the
// wave's own LDS, the next one's loads in flight; waves are independent.
template <int DP, int VP>
__global__ __launch_bounds__(256) void paged_decode_kernel(TalkParams p) {
  constexpr int KT = 32, LDK = DP + 8, LDV = VP + 8;
  constexpr int CK = KT * (DP / 8) / 64, CV = KT * (VP / 8) / 64;
  __shared__ __attribute__((aligned(16))) bf16 kst[4][KT * LDK];
  __shared__ __attribute__((aligned(16))) bf16 vst[4][KT * LDV];
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const long item = (long)blockIdx.x * 4 + w;
  if (item >= (long)p.T * p.G) return;  // no barriers below
  bf16* ks = kst[w];
  bf16* vs = vst[w];
  const int b = (int)(item / p.G), kvh = (int)(item % p.G), rep = p.H / p.G;
  const int r = lane & 15, g = lane >> 4, h = kvh * rep + min(r, rep - 1);
  const int pos = p.pos[b], lo = first_key(pos, p.window);
  const int* table = p.table + (long)p.slots[b] * p.tw;
  const float scale2 = p.scale * LOG2E, slope2 = p.slopes ? p.slopes[h] * LOG2E : 0.f;
  const KeyTiles kts = key_tiles<KT>(pos, pos, p.window, p.keep);
  const int n = kts.count(), per = (n + p.splits - 1) / p.splits;
  const int it0 = blockIdx.y * per, it1 = min(it0 + per, n);

  bf16x8 qf[DP / 32];
#pragma unroll
  for (int kk = 0; kk < DP / 32; ++kk) {
    const bf16x8 z = {};
    qf[kk] = kk * 32 < p.dim ? ld8(static_cast<const bf16*>(p.q) + ((long)b * p.H + h) * p.dim + kk * 32 + g * 8) : z;
  }
  f32x4 o[VP / 16];
#pragma unroll
  for (int di = 0; di < VP / 16; ++di) o[di] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = NEG, lsum = 0.f;
  bf16x8 kreg[CK], vreg[CV];
  auto load_tile = [&](int it) {
    const int kt = kts.at(it);
    const long base = ((long)table[kt * KT / PAGE] * p.G + kvh) * PAGE + kt * KT % PAGE;
    const bf16* kp = static_cast<const bf16*>(p.k) + base * p.dim;
    const bf16* vp = static_cast<const bf16*>(p.v) + base * p.vdim;
    const bf16x8 z = {};
#pragma unroll
    for (int c = 0; c < CK; ++c) {
      const int idx = lane + c * 64, col = (idx % (DP / 8)) * 8;
      kreg[c] = col < p.dim ? ld8_nt(kp + idx / (DP / 8) * p.dim + col) : z;
    }
#pragma unroll
    for (int c = 0; c < CV; ++c) {
      const int idx = lane + c * 64, col = (idx % (VP / 8)) * 8;
      vreg[c] = col < p.vdim ? ld8_nt(vp + idx / (VP / 8) * p.vdim + col) : z;
    }
  };
  if (it0 < it1) load_tile(it0);
  for (int it = it0; it < it1; ++it) {
    const int kt = kts.at(it);
    lds_fence();  // the tile before has been read
#pragma unroll
    for (int c = 0; c < CK; ++c) {
      const int idx = lane + c * 64;
      st8(ks + (idx / (DP / 8)) * LDK + (idx % (DP / 8)) * 8, kreg[c]);
    }
#pragma unroll
    for (int c = 0; c < CV; ++c) {
      const int idx = lane + c * 64;
      st8(vs + (idx / (VP / 8)) * LDV + (idx % (VP / 8)) * 8, vreg[c]);
    }
    lds_fence();
    if (it + 1 < it1) load_tile(it + 1);
    f32x4 s[2];
    float tmax = NEG;
#pragma unroll
    for (int ni = 0; ni < 2; ++ni) {
      s[ni] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < DP / 32; ++kk) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(ks + (ni * 16 + r) * LDK + kk * 32 + g * 8);
        s[ni] = mfma16(kf, qf[kk], s[ni]);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = kt * KT + ni * 16 + 4 * g + i;
        const float sv = fmaf(s[ni][i], scale2, slope2 * (float)(key - pos));
        s[ni][i] = seen(key, pos, lo, p.keep) ? sv : NEG;
        tmax = fmaxf(tmax, s[ni][i]);
      }
    }
    tmax = fmaxf(tmax, wave_xchg<16>(tmax));
    tmax = fmaxf(tmax, wave_xchg<32>(tmax));
    const float mn = fmaxf(m, tmax);  // every tile holds a visible key
    const float alpha = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    float ps = 0.f;
#pragma unroll
    for (int ni = 0; ni < 2; ++ni)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[ni][i] = __builtin_amdgcn_exp2f(s[ni][i] - mn);
        ps += s[ni][i];
      }
    lsum = lsum * alpha + ps;
    if (__any(alpha != 1.f)) {
#pragma unroll
      for (int di = 0; di < VP / 16; ++di) o[di] *= alpha;
    }
    bf16x8 ph, pl;
    split4(s[0], s[1], ph, pl);
    const int r0 = 4 * g + (r >> 2);
#pragma unroll
    for (int di = 0; di < VP / 16; ++di) {
      const int col = di * 16 + 4 * (r & 3);
      const bf16x4 a = ds_read_tr(vs + r0 * LDV + col);
      const bf16x4 c = ds_read_tr(vs + (r0 + 16) * LDV + col);
      const bf16x8 vf = {a[0], a[1], a[2], a[3], c[0], c[1], c[2], c[3]};
      o[di] = mfma16(vf, ph, o[di]);
      o[di] = mfma16(vf, pl, o[di]);
    }
  }
  lsum += wave_xchg<16>(lsum);
  lsum += wave_xchg<32>(lsum);
  if (p.splits > 1) {  // unnormalised partial for the combine
    if (r >= rep) return;
    const long pi = ((long)b * p.H + h) * p.splits + blockIdx.y;
#pragma unroll
    for (int di = 0; di < VP / 16; ++di)
      if (di * 16 < p.vdim) *reinterpret_cast<f32x4*>(p.part_o + pi * p.vdim + di * 16 + 4 * g) = o[di];
    if (g == 0) {
      p.part_ml[2 * pi] = m;
      p.part_ml[2 * pi + 1] = lsum;
    }
    return;
  }
  bf16* out = static_cast<bf16*>(p.out) + (long)b * p.ldo;
  if (r < rep) {
    const float inv = head_gate<bf16>(p, b, h) / lsum;
#pragma unroll
    for (int di = 0; di < VP / 16; ++di)
      if (di * 16 < p.vdim) st4(out + h * p.vdim + di * 16 + 4 * g, pack4(o[di] * inv));
  }
  if (kvh == p.G - 1)
    for (int c = p.H * p.vdim + lane; c < p.out_cols; c += 64) out[c] = f2bf(0.f);
}

// One token of all heads per block and key split, 64-key tiles (pages).  Wave w of
// NW owns K / V heads w, w + NW, ..: it scores their queries and writes the weights
// (two bf16 terms) to LDS; behind the barrier it multiplies its heads' values by
// the weights of all MT x 16 query heads.  LDS weights are double-buffered, so a
// tile has one barrier.  In flight: the next K rows under the weights and their
// product, the next V rows under a product with the ones before.
template <int DKS, int VT, int MT, int GC, int NW>
__global__ __launch_bounds__(NW * 64, 2) void mix_decode_kernel(TalkParams p) {
  constexpr int HP = MT * 16, PLD = PAGE + 8, STEPS = VT / 4 * 2;
  __shared__ __attribute__((aligned(16))) bf16 p_hi[2][HP * PLD], p_lo[2][HP * PLD];
  __shared__ __attribute__((aligned(16))) bf16 vst[NW][32 * VLD];
  __shared__ float alphas[2][HP];
  const int b = blockIdx.x, H = p.H, G = p.G, rep = H / G, dim = p.dim, vdim = p.vdim;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int pos = p.pos[b], lo = first_key(pos, p.window);
  const int* table = p.table + (long)p.slots[b] * p.tw;
  const bf16* K = static_cast<const bf16*>(p.k);
  const bf16* V = static_cast<const bf16*>(p.v);
  const KeyTiles kts = key_tiles<PAGE>(pos, pos, p.window, p.keep);
  const int n = kts.count(), per = (n + p.splits - 1) / p.splits;
  const int it0 = blockIdx.y * per, it1 = min(it0 + per, n);
  const float scale2 = p.scale * LOG2E;
  bf16* vs = vst[w];

  f32x4 o[GC][MT][VT];
  float m[GC], lsum[GC], slope2[GC];
#pragma unroll
  for (int c = 0; c < GC; ++c) {
    m[c] = NEG;
    lsum[c] = 0.f;
    slope2[c] = p.slopes ? p.slopes[min((w + NW * c) * rep + min(r, rep - 1), H - 1)] * LOG2E : 0.f;
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
      for (int di = 0; di < VT; ++di) o[c][mt][di] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  bf16x8 vr[4], kf[4][DKS];
  auto load_v = [&](long page, int kvh, int step) {
    const int vh = step >> 1, kk = step & 1;
    const bf16* vp = V + ((page * G + kvh) * PAGE + kk * 32) * vdim + vh * 64;
    const bf16x8 z = {};
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int row = q4 * 8 + (lane >> 3), col = (lane & 7) * 8;
      vr[q4] = vh * 64 + col < vdim ? ld8_nt(vp + (long)row * vdim + col) : z;
    }
  };
  auto load_k = [&](long page, int kvh) {
    const bf16* kp = K + ((page * G + kvh) * PAGE + r) * dim + g * 8;
    const bf16x8 z = {};
#pragma unroll
    for (int ni = 0; ni < 4; ++ni)
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) kf[ni][ks] = ks * 32 < dim ? ld8_nt(kp + (long)ni * 16 * dim + ks * 32) : z;
  };
  if (it0 < it1 && w < G) load_k(table[kts.at(it0)], w);
  for (int it = it0; it < it1; ++it) {
    const int kt = kts.at(it), buf = it & 1;
    const long page = table[kt], next = table[kts.at(min(it + 1, it1 - 1))];
#pragma unroll
    for (int c = 0; c < GC; ++c) {
      const int kvh = w + NW * c;
      if (kvh >= G) continue;  // wave-uniform
      const int h = kvh * rep + min(r, rep - 1);
      const bf16* q = static_cast<const bf16*>(p.q) + ((long)b * H + h) * dim + g * 8;
      const bf16x8 z = {};
      bf16x8 qf[DKS];
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) qf[ks] = ks * 32 < dim ? ld8(q + ks * 32) : z;
      f32x4 s[4];
      float tmax = NEG;
#pragma unroll
      for (int ni = 0; ni < 4; ++ni) {
        s[ni] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < DKS; ++ks) s[ni] = mfma16(kf[ni][ks], qf[ks], s[ni]);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = kt * PAGE + ni * 16 + 4 * g + i;
          const float sv = fmaf(s[ni][i], scale2, slope2[c] * (float)(key - pos));
          s[ni][i] = seen(key, pos, lo, p.keep) ? sv : NEG;
          tmax = fmaxf(tmax, s[ni][i]);
        }
      }
      if (c == 0) load_v(page, kvh, 0);
      if (c + 1 < GC && kvh + NW < G) load_k(page, kvh + NW);
      else load_k(next, w);
      tmax = fmaxf(tmax, wave_xchg<16>(tmax));
      tmax = fmaxf(tmax, wave_xchg<32>(tmax));
      const float mn = tmax > m[c] + 6.f ? tmax : m[c];  // every tile holds a visible key
      const float al = __builtin_amdgcn_exp2f(m[c] - mn);
      m[c] = mn;
      float ps = 0.f;
#pragma unroll
      for (int ni = 0; ni < 4; ++ni) {
        f32x4 e, rest;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          e[i] = __builtin_amdgcn_exp2f(s[ni][i] - mn);
          ps += e[i];
        }
        const bf16x4 hi = pack4(e);
#pragma unroll
        for (int i = 0; i < 4; ++i) rest[i] = e[i] - bf2f(hi[i]);
        if (r < rep) {
          st4(&p_hi[buf][h * PLD + ni * 16 + 4 * g], hi);
          st4(&p_lo[buf][h * PLD + ni * 16 + 4 * g], pack4(rest));
        }
      }
      lsum[c] = lsum[c] * al + ps;
      if (g == 0 && r < rep) alphas[buf][h] = al;
    }
    __syncthreads();
    float al[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) al[mt] = mt * 16 + r < H ? alphas[buf][mt * 16 + r] : 1.f;
#pragma unroll
    for (int c = 0; c < GC; ++c) {
      const int kvh = w + NW * c;
      if (kvh >= G) continue;
#pragma unroll
      for (int mt = 0; mt < MT; ++mt)
        if (__any(al[mt] != 1.f)) {
#pragma unroll
          for (int di = 0; di < VT; ++di) o[c][mt][di] *= al[mt];
        }
#pragma unroll
      for (int step = 0; step < STEPS; ++step) {
        const int vh = step >> 1, kk = step & 1;
        if (vh * 64 >= vdim) continue;
        lds_fence();  // reads of what is staged now are done
#pragma unroll
        for (int q4 = 0; q4 < 4; ++q4) st8(vs + (q4 * 8 + (lane >> 3)) * VLD + (lane & 7) * 8, vr[q4]);
        if (step + 1 < STEPS && ((step + 1) >> 1) * 64 < vdim) load_v(page, kvh, step + 1);
        else if (c + 1 < GC && kvh + NW < G) load_v(page, kvh + NW, 0);
        bf16x8 hf[MT], lf[MT];
#pragma unroll
        for (int mt = 0; mt < MT; ++mt) {  // heads behind H read stale columns, which nobody stores
          const int at = (mt * 16 + r) * PLD + kk * 32 + 4 * g;
          const bf16x4 h0 = ld4(&p_hi[buf][at]), h1 = ld4(&p_hi[buf][at + 16]);
          const bf16x4 l0 = ld4(&p_lo[buf][at]), l1 = ld4(&p_lo[buf][at + 16]);
          hf[mt] = bf16x8{h0[0], h0[1], h0[2], h0[3], h1[0], h1[1], h1[2], h1[3]};
          lf[mt] = bf16x8{l0[0], l0[1], l0[2], l0[3], l1[0], l1[1], l1[2], l1[3]};
        }
        lds_fence();
        const int r0 = 4 * g + (r >> 2);
#pragma unroll
        for (int dj = 0; dj < 4; ++dj) {
          const int col = dj * 16 + 4 * (r & 3);
          const bf16x4 a = ds_read_tr(vs + r0 * VLD + col);
          const bf16x4 d = ds_read_tr(vs + (r0 + 16) * VLD + col);
          const bf16x8 vf = {a[0], a[1], a[2], a[3], d[0], d[1], d[2], d[3]};
#pragma unroll
          for (int mt = 0; mt < MT; ++mt) {
            o[c][mt][vh * 4 + dj] = mfma16(vf, hf[mt], o[c][mt][vh * 4 + dj]);
            o[c][mt][vh * 4 + dj] = mfma16(vf, lf[mt], o[c][mt][vh * 4 + dj]);
          }
        }
      }
    }
  }
  const long part = (long)b * p.splits + blockIdx.y;
#pragma unroll
  for (int c = 0; c < GC; ++c) {
    const int kvh = w + NW * c;
    if (kvh >= G) continue;
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      if (mt * 16 + r >= H) continue;
      float* po = p.part_o + ((part * G + kvh) * H + mt * 16 + r) * vdim;
#pragma unroll
      for (int di = 0; di < VT; ++di)
        if (di * 16 < vdim) *reinterpret_cast<f32x4*>(po + di * 16 + 4 * g) = o[c][mt][di];
    }
    float l = lsum[c];
    l += wave_xchg<16>(l);
    l += wave_xchg<32>(l);
    if (g == 0 && r < rep) {
      p.part_ml[2 * (part * H + kvh * rep + r)] = m[c];
      p.part_ml[2 * (part * H + kvh * rep + r) + 1] = l;
    }
  }
}

// out_h = gate_h sum_g T_hg sum_s e^{m_gs - M_g} / L_g  part_s[kv(h)][g], one block
// per (token, K / V head) and MIX_COLS columns.  Dynamic LDS: factors [H][splits],
// merged rows [H][MIX_COLS].
constexpr int MIX_COLS = 32;
__global__ __launch_bounds__(256) void mix_combine_kernel(TalkParams p) {
  extern __shared__ float sh[];
  constexpr int N4 = MIX_COLS / 4, FLY = 8;
  const int H = p.H, G = p.G, S = p.splits, vdim = p.vdim, rep = H / G, tid = threadIdx.x;
  const int b = blockIdx.x / G, kvh = blockIdx.x % G, col0 = blockIdx.y * MIX_COLS;
  float* rows = sh;              // [H][MIX_COLS]
  float* cf = sh + H * MIX_COLS; // [H][S]
  for (int g0 = 0; g0 < H; g0 += 32) {  // eight lanes per head, all lanes stay
    const int gq = min(g0 + (tid >> 3), H - 1), l8 = tid & 7;
    const float* ml = p.part_ml + 2 * ((long)b * S * H + gq);
    float M = NEG, L = 0.f;
    for (int s = l8; s < S; s += 8) M = fmaxf(M, ml[2L * s * H]);
    M = fmaxf(M, wave_xchg<1>(M));
    M = fmaxf(M, wave_xchg<2>(M));
    M = fmaxf(M, wave_xchg<4>(M));
    for (int s = l8; s < S; s += 8) L += ml[2L * s * H + 1] * exp2f(ml[2L * s * H] - M);
    L += wave_xchg<1>(L);
    L += wave_xchg<2>(L);
    L += wave_xchg<4>(L);
    if (g0 + (tid >> 3) < H)
      for (int s = l8; s < S; s += 8) cf[gq * S + s] = exp2f(ml[2L * s * H] - M) / L;
  }
  __syncthreads();
  for (int i = tid; i < H * N4; i += 256) {
    const int gq = i / N4, d = col0 + i % N4 * 4;
    const float* po = p.part_o + (((long)b * S * G + kvh) * H + gq) * vdim + min(d, vdim - 4);
    f32x4 a = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < S; s += FLY) {
      f32x4 x[FLY];
#pragma unroll
      for (int j = 0; j < FLY; ++j) x[j] = *reinterpret_cast<const f32x4*>(po + (long)min(s + j, S - 1) * G * H * vdim);
#pragma unroll
      for (int j = 0; j < FLY; ++j)
        if (s + j < S) a += x[j] * cf[gq * S + s + j];
    }
    *reinterpret_cast<f32x4*>(rows + 4 * i) = a;
  }
  __syncthreads();
  bf16* out = static_cast<bf16*>(p.out) + (long)b * p.ldo;
  for (int i = tid; i < rep * N4; i += 256) {
    const int h = kvh * rep + i / N4, c = i % N4 * 4, d = col0 + c;
    if (d >= vdim) continue;
    const float* t = p.talk + (long)h * H;
    f32x4 a = {0.f, 0.f, 0.f, 0.f};
    for (int gq = 0; gq < H; ++gq) a += *reinterpret_cast<const f32x4*>(rows + gq * MIX_COLS + c) * t[gq];
    st4(out + h * vdim + d, pack4(a * head_gate<bf16>(p, b, h)));
  }
  if (kvh == G - 1 && blockIdx.y == 0)
    for (int c = H * vdim + tid; c < p.out_cols; c += 256) out[c] = f2bf(0.f);
}

}  // namespace
}  // namespace lsd

using namespace lsd;

extern "C" hipError_t lsd_attention_combine(const TalkParams* p, hipStream_t st);

extern "C" long lsd_append_lds(const RopeAppendParams* p) { return 4L * ((p->H + p->G) * (p->dim + 1) + p->G * p->vdim); }

extern "C" hipError_t lsd_rope_append(const RopeAppendParams* p, int f32, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  const bool vec = !f32 && p->dim % 8 == 0 && p->vdim % 8 == 0;
  if (vec && !p->taps && p->eps < 0.f && p->half % 8 == 0) {
    const int cols = (p->H + p->G) * p->dim + p->G * p->vdim;
    hipLaunchKernelGGL(rope_append_vec_kernel, dim3((p->T + 3) / 4, p->T <= 512 ? (cols + 511) / 512 : 1), dim3(256), 0, st, *p);
    return hipGetLastError();
  }
  const int wide = p->dim > p->vdim ? p->dim : p->vdim;
  if (vec && p->taps && p->n_taps <= 4 && p->half == 0 && wide <= 256) {
    const int run = p->T >= 4096 ? 32 : p->T >= 512 ? 4 : 1, lph = wide <= 32 ? 4 : wide <= 64 ? 8 : wide <= 128 ? 16 : 32;
    const long items = (long)((p->T + run - 1) / run) * (p->H + 2 * p->G);
    const dim3 grid((unsigned)((items * lph + 255) / 256));
#define LSD_CA(L)                                                                             \
  if (run >= 32) hipLaunchKernelGGL((conv_append_kernel<L, 8>), grid, dim3(256), 0, st, *p, run); \
  else if (run == 4) hipLaunchKernelGGL((conv_append_kernel<L, 4>), grid, dim3(256), 0, st, *p, run); \
  else hipLaunchKernelGGL((conv_append_kernel<L, 1>), grid, dim3(256), 0, st, *p, run);
    switch (lph) {
      case 4: LSD_CA(4) break;
      case 8: LSD_CA(8) break;
      case 16: LSD_CA(16) break;
      default: LSD_CA(32)
    }
#undef LSD_CA
    return hipGetLastError();
  }
  const size_t lds = lsd_append_lds(p);
  const void* fn = f32 ? (const void*)append_plain_kernel<float> : (const void*)append_plain_kernel<bf16>;
  if (lds > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  if (f32) hipLaunchKernelGGL((append_plain_kernel<float>), dim3(p->T), dim3(256), lds, st, *p);
  else hipLaunchKernelGGL((append_plain_kernel<bf16>), dim3(p->T), dim3(256), lds, st, *p);
  return hipGetLastError();
}

// Can the MFMA kernels take these heads?
extern "C" int lsd_paged_ok(int dim, int vdim) { return dim % 32 == 0 && dim <= 128 && vdim % 16 == 0 && vdim <= 128; }

// Prompt tiles of 64 qt queries (qt 1 or 2); p->lse: softmax sums only
extern "C" hipError_t lsd_paged_prefill(const TalkParams* p, int qt, int lse, hipStream_t st) {
  if (p->n_tiles == 0) return hipSuccess;
  const dim3 grid((unsigned)(p->n_tiles * p->H));
#define LSD_PP(D, V, Q, L) hipLaunchKernelGGL((paged_prefill_kernel<D, V, Q, L>), grid, dim3(256), 0, st, *p)
#define LSD_PP_Q(Q)                                   \
  if (lse) {                                          \
    if (p->dim <= 64) LSD_PP(64, 64, Q, true);        \
    else LSD_PP(128, 64, Q, true);                    \
  } else if (p->dim <= 64) {                          \
    if (p->vdim <= 64) LSD_PP(64, 64, Q, false);      \
    else LSD_PP(64, 128, Q, false);                   \
  } else {                                            \
    if (p->vdim <= 64) LSD_PP(128, 64, Q, false);     \
    else LSD_PP(128, 128, Q, false);                  \
  }
  if (qt == 1) {
    LSD_PP_Q(1)
  } else if (qt == 2) {
    LSD_PP_Q(2)
  } else {
    return hipErrorInvalidValue;
  }
#undef LSD_PP_Q
#undef LSD_PP
  return hipGetLastError();
}

// hp: 8, 16 or 32 (talk_frag padded to it)
extern "C" hipError_t lsd_mix_prefill(const TalkParams* p, int hp, hipStream_t st) {
  if (p->n_tiles == 0) return hipSuccess;
  const dim3 grid(p->n_tiles, p->splits);
#define LSD_MP(HP, NT)                                                                                                 \
  if (p->dim <= 64 && p->vdim <= 64) hipLaunchKernelGGL((mix_prefill_kernel<2, 4, HP>), grid, dim3(NT), 0, st, *p); \
  else if (p->dim <= 64) hipLaunchKernelGGL((mix_prefill_kernel<2, 8, HP>), grid, dim3(NT), 0, st, *p);             \
  else if (p->vdim <= 64) hipLaunchKernelGGL((mix_prefill_kernel<4, 4, HP>), grid, dim3(NT), 0, st, *p);            \
  else hipLaunchKernelGGL((mix_prefill_kernel<4, 8, HP>), grid, dim3(NT), 0, st, *p);
  switch (hp) {
    case 8: LSD_MP(8, 256) break;
    case 16: LSD_MP(16, 256) break;
    case 32: LSD_MP(32, 512) break;
    default: return hipErrorInvalidValue;
  }
#undef LSD_MP
  if (p->splits > 1) return lsd_attention_combine(p, st);
  return hipGetLastError();
}

extern "C" hipError_t lsd_paged_decode(const TalkParams* p, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  const dim3 grid((unsigned)(((long)p->T * p->G + 3) / 4), p->splits);
#define LSD_PD(D, V) hipLaunchKernelGGL((paged_decode_kernel<D, V>), grid, dim3(256), 0, st, *p)
  if (p->dim <= 64) {
    if (p->vdim <= 64) LSD_PD(64, 64);
    else LSD_PD(64, 128);
  } else {
    if (p->vdim <= 64) LSD_PD(128, 64);
    else LSD_PD(128, 128);
  }
#undef LSD_PD
  if (p->splits > 1) return lsd_attention_combine(p, st);
  return hipGetLastError();
}

// Waves per block times K / V heads per wave of mix_decode cover G; 0: no kernel
static int mix_waves(int G) { return G > 4 ? 8 : 4; }
extern "C" int lsd_mix_decode_gc(int H, int G) {
  if (H > 32 || H / G > 16) return 0;
  const int gc = (G + mix_waves(G) - 1) / mix_waves(G);
  return gc * (H <= 16 ? 1 : 2) > 4 ? 0 : gc <= 2 ? gc : 4;
}

extern "C" long lsd_mix_combine_lds(const TalkParams* p) { return 4L * p->H * (MIX_COLS + p->splits); }

extern "C" hipError_t lsd_mix_decode(const TalkParams* p, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  const dim3 grid(p->T, p->splits);
  const int gc = lsd_mix_decode_gc(p->H, p->G), mt = p->H <= 16 ? 1 : 2, nw = mix_waves(p->G);
#define LSD_MD(MT, GC, NW)                                                                                                 \
  if (p->dim <= 64 && p->vdim <= 64) hipLaunchKernelGGL((mix_decode_kernel<2, 4, MT, GC, NW>), grid, dim3(NW * 64), 0, st, *p); \
  else if (p->dim <= 64) hipLaunchKernelGGL((mix_decode_kernel<2, 8, MT, GC, NW>), grid, dim3(NW * 64), 0, st, *p);         \
  else if (p->vdim <= 64) hipLaunchKernelGGL((mix_decode_kernel<4, 4, MT, GC, NW>), grid, dim3(NW * 64), 0, st, *p);        \
  else hipLaunchKernelGGL((mix_decode_kernel<4, 8, MT, GC, NW>), grid, dim3(NW * 64), 0, st, *p);
  switch (nw * 16 + gc * 4 + mt) {
    case 64 + 5: LSD_MD(1, 1, 4) break;
    case 64 + 6: LSD_MD(2, 1, 4) break;
    case 128 + 5: LSD_MD(1, 1, 8) break;
    case 128 + 6: LSD_MD(2, 1, 8) break;
    case 128 + 9: LSD_MD(1, 2, 8) break;
    case 128 + 10: LSD_MD(2, 2, 8) break;
    default: return hipErrorInvalidValue;
  }
#undef LSD_MD
  hipLaunchKernelGGL(mix_combine_kernel, dim3(p->T * p->G, (p->vdim + MIX_COLS - 1) / MIX_COLS), dim3(256),
                     lsd_mix_combine_lds(p), st, *p);
  return hipGetLastError();
}
