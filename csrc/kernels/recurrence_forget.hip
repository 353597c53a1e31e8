// Linear attention whose forget gate also decides what is written (HGRN2):
//   S <- diag(f) S + (1 - f) v^T;  o = S^T q;  out = rms(o) norm
//
//  * forget_seq: token by token, state in registers, gates, read-out and output norm
//    in one launch.  Decode steps, and prompts of models served in fp32.
//  * forget_chunk: prompts of bf16 models, up to 32 tokens at a time as matrix
//    products around a state that stays in the accumulators of four waves, each
//    owning columns of it.  Few sequences are cut in segments that run together:
//    one launch leaves each segment's own state and decay, forget_join sums up what
//    every segment starts from, and the segments run from there.
//
// Gates, their logarithms, decays and the state are fp32; fp32 operands enter the
// matrix cores as two bf16 terms (16 bits).
#include "common.h"
#include "mixer_params.h"
#include "recurrence.h"

namespace lsd {
namespace {

// 1 - f = (1 - l) sigmoid(-z), without cancellation where f is close to one
__device__ __forceinline__ float write_gate(float z, float lower) { return (1.f - lower) / (1.f + expf(z)); }

// One (sequence, head, LV * 4 columns of the state) per block; thread (dg, lv)
// holds rows dg + i * 256 / LV of four columns.  Dynamic LDS: q, 1 - f [D].
template <typename T, int LV, int NR>
__global__ __launch_bounds__(256, NR <= 8 ? 3 : 2) void forget_seq_kernel(ForgetParams p) {
  constexpr int VB = LV * 4, DG = 256 / LV;
  extern __shared__ float dyn[];
  __shared__ __attribute__((aligned(16))) float red[4][LV * 4];
  __shared__ __attribute__((aligned(16))) float vs[VB];
  const int D = p.D, tid = threadIdx.x;
  float *qs = dyn, *ks = dyn + D;
  const int nvb = (p.Vp + VB - 1) / VB;
  const int h = blockIdx.x / nvb, v0 = (blockIdx.x % nvb) * VB, b = blockIdx.y;
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
  for (int t = 0; t < n; ++t) {
    const long row = r0 + t;
    const T* y = static_cast<const T*>(p.y) + row * p.ldy;
    for (int c = tid; c < 2 * D + VB; c += 256) {
      if (c < D) {
        qs[c] = silu_x(to_f(y[h * D + c]));
      } else if (c < 2 * D) {
        const int at = h * D + c - D;
        ks[c - D] = write_gate(to_f(y[p.heads * D + at]) + p.bias[at], p.lower[at]);
      } else {
        const int v = v0 + c - 2 * D;
        vs[c - 2 * D] = v < p.V ? to_f(y[2 * p.heads * D + h * p.V + v]) : 0.f;
      }
    }
    __syncthreads();
    const f32x4 v = *reinterpret_cast<const f32x4*>(&vs[lv * 4]);
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = dg + i * DG;
      if (d < D) {
        s[i] += (v - s[i]) * ks[d];
        o += s[i] * qs[d];
      }
    }
    o = column_sum<LV>(o, red);  // its barriers also free q, 1 - f and v
    if (p.raw) {
      if (dg == 0 && live) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < p.V) p.raw[row * p.ldr + (long)h * p.V + col + i] = o[i];
      }
    } else {  // one block holds all of V; columns beyond it are zero
      float ss = o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
#pragma unroll
      for (int off = 1; off < LV; off <<= 1) ss += wave_xor_n(ss, off);
      const float rs = 1.f / sqrtf(ss / p.V + p.eps);
      T* out = static_cast<T*>(p.out) + row * p.ldo;
      if (dg == 0) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < p.V) from_f(out + (long)h * p.V + col + i, o[i] * rs * p.norm[col + i]);
      }
      if (h == p.heads - 1)
        for (int c = p.heads * p.V + tid; c < p.out_cols; c += 256) from_f(out + c, 0.f);
    }
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < NR; ++i)
      if (dg + i * DG < D) *reinterpret_cast<f32x4*>(Sg + (long)(dg + i * DG) * p.Vp) = s[i];
  }
}

// log2 of a gate below this stands for zero
constexpr float LOG_MIN = -80.f;
// how far (log2) the decays of one chunk may lie from their reference
constexpr float RANGE = 80.f;

// Chunked form.  With G_t the summed log gates of the chunk up to token t (per
// channel) and a reference m near its middle, S' = diag(e^{G_m}) S:
//   O = Q' S' + P V,   Q'_t = q_t e^{G_t - G_m},  K'_s = (1 - f_s) e^{G_m - G_s}
//   P_ts = Q'_t . K'_s (s <= t),   S <- diag(e^{G_end - G_m}) (S' + K'^T V)
// The factors stay in range because a chunk is cut shorter (32, 16, 8, 4, 2
// tokens) where a channel's gates fall too fast.
// STATES: a segment's own state and decay only.  BLOCK: grid (heads x segments, sequences).
enum ForgetMode : int { FORGET_WHOLE = 0, FORGET_STATES = 1, FORGET_SEGMENT = 2 };

template <int DKS, int VTW, int MODE>
__global__ __launch_bounds__(256, 2) void forget_chunk_kernel(ForgetParams p) {
  constexpr int CT = 32, DP = DKS * 32, DT = DKS * 2, LDD = DP + 8, VP = VTW * 64, LDV = VP + 8, VW = VTW * 16;
  constexpr int NV = CT * VP / 1024;  // groups of four values per thread
  constexpr int LDO = VW + 4;
  __shared__ __attribute__((aligned(16))) bf16 qd_h[CT * LDD], qd_l[CT * LDD], kd_h[CT * LDD], kd_l[CT * LDD];
  __shared__ __attribute__((aligned(16))) bf16 vs[CT * LDV];
  __shared__ __attribute__((aligned(16))) float tot[4][DP], pre[3][DP], s0[DP], er[DP];
  __shared__ __attribute__((aligned(16))) bf16x4 pf[3][2][64];
  __shared__ float red[4][CT];
  __shared__ __attribute__((aligned(16))) bf16 ob[4][CT * LDO];
  constexpr bool OUT = MODE != FORGET_STATES;
  const int D = p.D, V = p.V, H = p.heads;
  const int nseg = MODE == FORGET_WHOLE ? 1 : MODE == FORGET_STATES ? p.segs - 1 : p.segs;
  const int h = blockIdx.x / nseg, seg = blockIdx.x % nseg, b = blockIdx.y;
  const int tid = threadIdx.x, lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int slot = p.s.slots[b], start = p.s.start[b], r0 = p.s.cu[b], n = p.s.cu[b + 1] - r0;
  const int len = MODE == FORGET_WHOLE ? n : ((n + p.segs - 1) / p.segs + CT - 1) / CT * CT;
  const int ta = seg * len, te = min(n, ta + len);
  if (ta >= te) return;
  float* Sg = p.S + ((long)slot * H + h) * D * p.Vp;
  const long part0 = ((long)b * H + h) * p.segs;
  auto part = [&](int k) { return p.part + (part0 + k) * D * p.Vp; };

  // state: rows d = 16 dt + 4 g + i, columns v = 16 (w VTW + j) + r
  f32x4 S[DT][VTW];
  auto save = [&](float* dst) {
    int g4 = 4 * g;
    asm volatile("" : "+v"(g4));  // addresses are formed anew: none stays in a register through the loop
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int j = 0; j < VTW; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = dt * 16 + g4 + i, v = (w * VTW + j) * 16 + r;
          if (d < D && v < V) dst[d * p.Vp + v] = S[dt][j][i];
        }
  };
  auto each = [&](auto&& f) {
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int j = 0; j < VTW; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = dt * 16 + 4 * g + i, v = (w * VTW + j) * 16 + r;
          S[dt][j][i] = f(S[dt][j][i], d, v, d < D && v < V);
        }
  };
  if constexpr (MODE == FORGET_SEGMENT) {
    const float* src = part(seg);
    each([&](float, int d, int v, bool in) { return in ? src[d * p.Vp + v] : 0.f; });
  } else {
    const bool old = start > 0 && seg == 0;
    each([&](float, int d, int v, bool in) { return old && in ? Sg[d * p.Vp + v] : 0.f; });
    if (MODE == FORGET_STATES && seg == 0) {
      save(part(0));
      if (te == n) return;  // nothing follows this segment
    }
  }
  // gates and queries: wave w has tokens 8 w .., a lane two channels
  const int d0 = 2 * lane;
  const bool mine = d0 < DP, chan = d0 < D;  // D is even
  const int dc = chan ? d0 : 0;
  float bias[2], lower[2];
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    bias[e] = p.bias[h * D + dc + e];
    lower[e] = p.lower[h * D + dc + e];
  }
  const bf16* yq = static_cast<const bf16*>(p.y) + (long)r0 * p.ldy + h * D + dc;
  const bf16* yv = static_cast<const bf16*>(p.y) + (long)r0 * p.ldy + 2 * H * D + (long)h * V;
  const int zoff = H * D, ldy = (int)p.ldy;
  // rows of the next chunk, in flight under this one; clamped to the segment, what lies behind it counts as zero
  unsigned xq[8], xz[8];
  bf16x4 rv[NV];
  auto fetch = [&](int t0) {
    const bf16* base = yq + (long)t0 * p.ldy;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int off = min(w * 8 + i, te - 1 - t0) * ldy;
      if (OUT) xq[i] = *reinterpret_cast<const unsigned*>(base + off);
      xz[i] = *reinterpret_cast<const unsigned*>(base + off + zoff);
    }
    const bf16* vb = yv + (long)t0 * p.ldy;
#pragma unroll
    for (int q = 0; q < NV; ++q) {
      const int c = tid + q * 256, t = min(c / (VP / 4), te - 1 - t0), v = (c % (VP / 4)) * 4;
      const bf16x4 x = ld4(vb + t * ldy + min(v, V - 4)), z = {};
      rv[q] = v < V ? x : z;
    }
  };
  auto lo16 = [](unsigned u) { return __builtin_bit_cast(float, u << 16); };
  auto hi16 = [](unsigned u) { return __builtin_bit_cast(float, u & 0xffff0000u); };
  float nrm[VTW];
#pragma unroll
  for (int j = 0; j < VTW; ++j) nrm[j] = OUT ? p.norm[min((w * VTW + j) * 16 + r, V - 1)] : 0.f;
  float decay[2] = {0.f, 0.f};
  fetch(ta);
  for (int t0 = ta; t0 < te;) {
    const int left = te - t0;
    float q[8][2], k[8][2], run[8][2];
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const float x = e ? hi16(xq[i]) : lo16(xq[i]);
        const float z = (e ? hi16(xz[i]) : lo16(xz[i])) + bias[e];
        const bool in = chan && w * 8 + i < left;
        const float u = exp_f(-fabsf(z)), rc = __builtin_amdgcn_rcpf(1.f + u);
        const float kk = (1.f - lower[e]) * (z >= 0.f ? u * rc : rc);  // 1 - f
        const float f = lower[e] + (1.f - lower[e]) * (z >= 0.f ? rc : u * rc);
        const float lg = kk <= 0.5f ? LOG2E * log1p_series(-kk * __builtin_amdgcn_rcpf(2.f - kk))
                                    : fmaxf(__builtin_amdgcn_logf(f), LOG_MIN);
        if (OUT) q[i][e] = silu(x);
        k[i][e] = in ? kk : 0.f;
        run[i][e] = (in ? lg : 0.f) + (i ? run[i - 1][e] : 0.f);
      }
    if (mine) {
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        tot[w][d0 + e] = run[7][e];
        if (w == 0) {
          pre[0][d0 + e] = run[0][e];
          pre[1][d0 + e] = run[1][e];
          pre[2][d0 + e] = run[3][e];
        }
      }
    }
#pragma unroll
    for (int c = 0; c < NV; ++c) {
      const int at = tid + c * 256;
      st4(vs + at / (VP / 4) * LDV + (at % (VP / 4)) * 4, rv[c]);
    }
    __syncthreads();
    // how many tokens this chunk takes (every wave alike), its reference and end
    float T[4][2], P[3][2], base[2], Gm[2], Ge[2];
    bool ok32 = true, ok16 = true, ok8 = true, ok4 = true;
#pragma unroll
    for (int e = 0; e < 2; ++e) {
#pragma unroll
      for (int c = 0; c < 4; ++c) T[c][e] = mine ? tot[c][d0 + e] : 0.f;
#pragma unroll
      for (int c = 0; c < 3; ++c) P[c][e] = mine ? pre[c][d0 + e] : 0.f;
      base[e] = (w > 0 ? T[0][e] : 0.f) + (w > 1 ? T[1][e] : 0.f) + (w > 2 ? T[2][e] : 0.f);
      ok32 &= T[0][e] + T[1][e] >= -RANGE && T[2][e] + T[3][e] >= -RANGE;
      ok16 &= T[0][e] >= -RANGE && T[1][e] >= -RANGE;
      ok8 &= P[2][e] >= -RANGE && T[0][e] - P[2][e] >= -RANGE;
      ok4 &= P[1][e] >= -RANGE && P[2][e] - P[1][e] >= -RANGE;
    }
    const int nt = __all(ok32) ? 32 : __all(ok16) ? 16 : __all(ok8) ? 8 : __all(ok4) ? 4 : 2;
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      Gm[e] = nt == 32 ? T[0][e] + T[1][e] : nt == 16 ? T[0][e] : nt == 8 ? P[2][e] : nt == 4 ? P[1][e] : P[0][e];
      Ge[e] = nt == 32 ? (T[0][e] + T[1][e]) + (T[2][e] + T[3][e]) : nt == 16 ? T[0][e] + T[1][e] : nt == 8 ? T[0][e]
              : nt == 4 ? P[2][e] : P[1][e];
      decay[e] += Ge[e];
    }
    if (mine) {
      if (w == 0) {
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          s0[d0 + e] = __builtin_amdgcn_exp2f(Gm[e]);
          er[d0 + e] = __builtin_amdgcn_exp2f(Ge[e] - Gm[e]);
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int t = w * 8 + i;
        const bool in = t < nt;
        bf16x2 ah, al, kh, kl;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float G = base[e] + run[i][e] - Gm[e];
          const float kv = in && chan ? k[i][e] * __builtin_amdgcn_exp2f(-G) : 0.f;
          kh[e] = f2bf(kv);
          kl[e] = f2bf(kv - bf2f(kh[e]));
          if (OUT) {
            const float qv = in && chan ? q[i][e] * __builtin_amdgcn_exp2f(G) : 0.f;
            ah[e] = f2bf(qv);
            al[e] = f2bf(qv - bf2f(ah[e]));
          }
        }
        if (OUT) {
          *reinterpret_cast<bf16x2*>(qd_h + t * LDD + d0) = ah;
          *reinterpret_cast<bf16x2*>(qd_l + t * LDD + d0) = al;
        }
        *reinterpret_cast<bf16x2*>(kd_h + t * LDD + d0) = kh;
        *reinterpret_cast<bf16x2*>(kd_l + t * LDD + d0) = kl;
      }
    }
    if (t0 + nt < te) fetch(t0 + nt);
    __syncthreads();
    // operand of row r: k-slots (g, j) <-> d = 32 ks + 4 g + j, 32 ks + 16 + 4 g + (j - 4)
    auto opnd = [&](const bf16* a, int row, int ks) {
      const bf16* at = a + (row + r) * LDD + ks * 32 + 4 * g;
      return cat(ld4(at), ld4(at + 16));
    };
    f32x4 o[2][VTW];
    if constexpr (OUT) {
      if (w < 3) {  // scores transposed: rows s of tile w > 1, column t = r of tile w > 0
        const int sr = w > 1 ? 16 : 0, tr = w > 0 ? 16 : 0;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < DKS; ++ks)
          acc = mfma3(opnd(kd_h, sr, ks), opnd(kd_l, sr, ks), opnd(qd_h, tr, ks), opnd(qd_l, tr, ks), acc);
        if (w != 1) {
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[i] = 4 * g + i <= r ? acc[i] : 0.f;
        }
        const bf16x4 hi = hi4(acc);
        pf[w][0][lane] = hi;
        pf[w][1][lane] = lo4(acc, hi);
      }
#pragma unroll
      for (int mt = 0; mt < 2; ++mt)
#pragma unroll
        for (int j = 0; j < VTW; ++j) o[mt][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int ks = 0; ks < DKS; ++ks) {
      const f32x4 da = *reinterpret_cast<const f32x4*>(&s0[ks * 32 + 4 * g]);
      const f32x4 db = *reinterpret_cast<const f32x4*>(&s0[ks * 32 + 16 + 4 * g]);
      bf16x8 qh[2], ql[2];
      if constexpr (OUT) {
#pragma unroll
        for (int mt = 0; mt < 2; ++mt) {
          qh[mt] = opnd(qd_h, 16 * mt, ks);
          ql[mt] = opnd(qd_l, 16 * mt, ks);
        }
      }
#pragma unroll
      for (int j = 0; j < VTW; ++j) {
        S[2 * ks][j] *= da;
        S[2 * ks + 1][j] *= db;
        if constexpr (OUT) {
          bf16x8 sh, sl;
          split8(S[2 * ks][j], S[2 * ks + 1][j], sh, sl);
#pragma unroll
          for (int mt = 0; mt < 2; ++mt) o[mt][j] = mfma3(qh[mt], ql[mt], sh, sl, o[mt][j]);
        }
      }
    }
    bf16x8 vf[VTW];
#pragma unroll
    for (int j = 0; j < VTW; ++j) {
      const bf16* vp = vs + (4 * g + (r >> 2)) * LDV + (w * VTW + j) * 16 + 4 * (r & 3);
      vf[j] = cat(ds_read_tr(vp), ds_read_tr(vp + 16 * LDV));
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const int at = (4 * g + (r >> 2)) * LDD + dt * 16 + 4 * (r & 3);
      const bf16x8 kh = cat(ds_read_tr(kd_h + at), ds_read_tr(kd_h + at + 16 * LDD));
      const bf16x8 kl = cat(ds_read_tr(kd_l + at), ds_read_tr(kd_l + at + 16 * LDD));
      const f32x4 dec = *reinterpret_cast<const f32x4*>(&er[dt * 16 + 4 * g]);
#pragma unroll
      for (int j = 0; j < VTW; ++j) {
        S[dt][j] = mfma16(kh, vf[j], S[dt][j]);
        S[dt][j] = mfma16(kl, vf[j], S[dt][j]) * dec;
      }
    }
    if constexpr (OUT) {
      __syncthreads();  // the scores are there
      const bf16x4 z = {};
      const bf16x8 ph[2] = {cat(pf[0][0][lane], z), cat(pf[1][0][lane], pf[2][0][lane])};
      const bf16x8 pl[2] = {cat(pf[0][1][lane], z), cat(pf[1][1][lane], pf[2][1][lane])};
#pragma unroll
      for (int mt = 0; mt < 2; ++mt) {
        f32x4 ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < VTW; ++j) {
          o[mt][j] = mfma16(ph[mt], vf[j], o[mt][j]);
          o[mt][j] = mfma16(pl[mt], vf[j], o[mt][j]);
          ss += o[mt][j] * o[mt][j];  // columns beyond V are zero
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float u = ss[i];
#pragma unroll
          for (int off = 1; off < 16; off <<= 1) u += wave_xchg_n(u, off);
          if (r == 0) red[w][mt * 16 + 4 * g + i] = u;
        }
      }
    }
    __syncthreads();
    if constexpr (OUT) {
      bf16* mo = ob[w];  // this wave's columns, turned into rows
#pragma unroll
      for (int mt = 0; mt < 2; ++mt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = mt * 16 + 4 * g + i;
          const float rs = rsqrtf((red[0][t] + red[1][t] + red[2][t] + red[3][t]) / V + p.eps);
#pragma unroll
          for (int j = 0; j < VTW; ++j) mo[t * LDO + j * 16 + r] = f2bf(o[mt][j][i] * rs * nrm[j]);
        }
      lds_fence();
      const int rows = min(nt, left);
      bf16* out = static_cast<bf16*>(p.out) + (long)(r0 + t0) * p.ldo;
#pragma unroll
      for (int c = 0; c < CT * VW / 256; ++c) {
        const int at = lane + c * 64, t = at / (VW / 4), v = (at % (VW / 4)) * 4;
        if (t < rows && w * VW + v < V) st4(out + (long)t * p.ldo + (long)h * V + w * VW + v, ld4(mo + t * LDO + v));
      }
      if (h == H - 1)
        for (int c = H * V + lane; c < p.out_cols; c += 64)
          for (int t = w; t < rows; t += 4) out[(long)t * p.ldo + c] = f2bf(0.f);
    }
    t0 += nt;
  }
  if constexpr (MODE == FORGET_STATES) {
    save(part(seg + 1));
    if (w == 0 && chan) {
      p.decay[(part0 + seg + 1) * D + d0] = decay[0];
      p.decay[(part0 + seg + 1) * D + d0 + 1] = decay[1];
    }
  } else if (te == n) {
    save(Sg);
  }
}

// What segments 2 .. start from: the state of the segment before, less its decay,
// and that one's own.  A thread takes four columns of one row.
__global__ __launch_bounds__(256) void forget_join_kernel(ForgetParams p) {
  constexpr int FLY = 4;
  const int q = p.Vp / 4, at = blockIdx.x * 256 + threadIdx.x;
  if (at >= p.D * q) return;
  const long part0 = ((long)blockIdx.z * p.heads + blockIdx.y) * p.segs;
  const int n = p.s.cu[blockIdx.z + 1] - p.s.cu[blockIdx.z];
  const int len = ((n + p.segs - 1) / p.segs + 31) / 32 * 32;  // as in forget_chunk
  const int segs = n > 0 ? (n + len - 1) / len : 0;            // those that hold tokens
  const long size = (long)p.D * p.Vp;
  float* s = p.part + part0 * size + (at / q) * p.Vp + (at % q) * 4;
  const float* dec = p.decay + part0 * p.D + at / q;
  if (segs <= 2) return;
  f32x4 acc = *reinterpret_cast<const f32x4*>(s + size);
  for (int k = 2; k < segs; k += FLY) {
    f32x4 own[FLY];
    float d[FLY];
#pragma unroll
    for (int i = 0; i < FLY; ++i) {
      const int c = min(k + i, segs - 1);
      own[i] = *reinterpret_cast<const f32x4*>(s + c * size);
      d[i] = dec[(long)c * p.D];
    }
#pragma unroll
    for (int i = 0; i < FLY; ++i)
      if (k + i < segs) {
        acc = acc * __builtin_amdgcn_exp2f(d[i]) + own[i];
        *reinterpret_cast<f32x4*>(s + (k + i) * size) = acc;
      }
  }
}

}  // namespace
}  // namespace lsd

using namespace lsd;

// Token by token; raw is needed where lsd_recur_block(D, V) < V
extern "C" hipError_t lsd_forget_seq(const ForgetParams* p, int vb, int f32, hipStream_t st) {
  if (p->s.B == 0) return hipSuccess;
  if (vb == 0) return hipErrorInvalidValue;
  const int nvb = (p->Vp + vb - 1) / vb, dgs = 1024 / vb, nr = (p->D + dgs - 1) / dgs;
  if (!p->raw && nvb != 1) return hipErrorInvalidValue;
  const dim3 grid(p->heads * nvb, p->s.B);
  const size_t lds = 2 * p->D * sizeof(float);
#define LSD_FS(T, LV, NR) hipLaunchKernelGGL((forget_seq_kernel<T, LV, NR>), grid, dim3(256), lds, st, *p)
#define LSD_FS_N(T, LV)                \
  if (nr <= 1) LSD_FS(T, LV, 1);       \
  else if (nr <= 2) LSD_FS(T, LV, 2);  \
  else if (nr <= 4) LSD_FS(T, LV, 4);  \
  else if (nr <= 8) LSD_FS(T, LV, 8);  \
  else LSD_FS(T, LV, 16);
#define LSD_FS_V(T)                    \
  switch (vb) {                        \
    case 4: LSD_FS_N(T, 1) break;      \
    case 8: LSD_FS_N(T, 2) break;      \
    case 16: LSD_FS_N(T, 4) break;     \
    case 32: LSD_FS_N(T, 8) break;     \
    case 64: LSD_FS_N(T, 16) break;    \
    default: LSD_FS_N(T, 32) break;    \
  }
  if (f32) {
    LSD_FS_V(float)
  } else {
    LSD_FS_V(bf16)
  }
#undef LSD_FS_V
#undef LSD_FS_N
#undef LSD_FS
  return hipGetLastError();
}

// Can the chunked kernel take these sizes?
extern "C" int lsd_forget_ok(int D, int V) { return D <= 128 && V <= 128 && D % 2 == 0 && V % 4 == 0; }

extern "C" hipError_t lsd_forget_chunk(const ForgetParams* p, hipStream_t st) {
  if (p->s.B == 0) return hipSuccess;
  if (!lsd_forget_ok(p->D, p->V) || p->segs < 1) return hipErrorInvalidValue;
#define LSD_FC(DKS, VTW, MODE, N) \
  hipLaunchKernelGGL((forget_chunk_kernel<DKS, VTW, MODE>), dim3(p->heads * (N), p->s.B), dim3(256), 0, st, *p)
#define LSD_FC_M(DKS, VTW)                                   \
  if (p->segs == 1) LSD_FC(DKS, VTW, FORGET_WHOLE, 1);       \
  else {                                                     \
    LSD_FC(DKS, VTW, FORGET_STATES, p->segs - 1);            \
    if (p->segs > 2)                                         \
      hipLaunchKernelGGL(forget_join_kernel, dim3((p->D * p->Vp / 4 + 255) / 256, p->heads, p->s.B), dim3(256), 0, st, *p); \
    LSD_FC(DKS, VTW, FORGET_SEGMENT, p->segs);               \
  }
#define LSD_FC_V(DKS)                       \
  if (p->V <= 64) { LSD_FC_M(DKS, 1) }      \
  else { LSD_FC_M(DKS, 2) }
  if (p->D <= 32) { LSD_FC_V(1) }
  else if (p->D <= 64) { LSD_FC_V(2) }
  else { LSD_FC_V(4) }
#undef LSD_FC_V
#undef LSD_FC_M
#undef LSD_FC
  return hipGetLastError();
}
