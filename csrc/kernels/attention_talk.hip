// Attention over a paged K / V cache whose capped scores are mixed over the heads by
// a learned [H][H] matrix before the softmax, with grouped K / V heads and a sliding
// window (mixed weights and no mixing: attention_paged.hip).
//
//  * talk_prefill: MFMA, 16 queries of 4 heads per wave, all heads in a block.
//  * talk_decode: MFMA, one token of all heads per block, keys split over blocks.
//  * talk_plain: one token per block, any sizes, bf16 or fp32, mixed scores, mixed
//    weights or neither.
//
// Every head's score of a (query, key) pair is needed before any head's weight
// of it is known, so a block works on all heads of its queries.  Scores cross
// the waves through LDS as two fp16 terms (value and remainder, 22 bits: the cap
// bounds them) and are mixed by the matrix cores in fp32; softmax weights enter
// the second product as two bf16 terms.
#include "attention_paged.h"

namespace lsd {
namespace {

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
  const int kept = min(p.keep, lo), n_keys = kept + pos - lo + 1;
  auto key_at = [&](int i) { return i < kept ? i : i - kept + lo; };
  // mixed weights: a first pass for the softmax sums, a second with the weights
  for (int pass = p.mix_weights ? 0 : 1; pass < 2; ++pass) {
    for (int k0 = 0; k0 < n_keys; k0 += KT) {
      const int nk = min(KT, n_keys - k0);
      for (int i = tid; i < H * KT; i += 256) {
        const int h = i / KT, kk = i % KT, key = key_at(k0 + kk);
        float s = 0.f;
        if (kk < nk) {
          const T* kp = K + (((long)table[key / PAGE] * p.G + h / rep) * PAGE + key % PAGE) * p.dim;
          for (int d = 0; d < p.dim; ++d) s = fmaf(qs[h * p.dim + d], to_f(kp[d]), s);
          s *= p.scale;
          if (p.cap > 0.f) s = p.cap * tanhf(s / p.cap);
          if (p.slopes) s -= p.slopes[h] * (float)(pos - key);
          if (p.mix_weights && pass == 1) s = expf(s - m[h]) / l[h];
        }
        s0[h * LD + kk] = s;
      }
      __syncthreads();
      const bool mix = p.talk && pass == 1;
      for (int i = tid; i < H * KT; i += 256) {
        const int h = i / KT, kk = i % KT;
        float s = 0.f;
        if (mix) {
          for (int g = 0; g < H; ++g) s = fmaf(p.talk[h * H + g], s0[g * LD + kk], s);
        } else {
          s = s0[h * LD + kk];
        }
        s1[h * LD + kk] = kk < nk ? s : NEG;
      }
      __syncthreads();
      if (!p.mix_weights || pass == 0) {
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
      }
      if (pass == 1) {
        for (int i = tid; i < H * p.vdim; i += 256) {
          const int h = i / p.vdim, d = i % p.vdim;
          float a = p.mix_weights ? acc[i] : acc[i] * al[h];
          for (int kk = 0; kk < nk; ++kk) {
            const int key = key_at(k0 + kk);
            a = fmaf(s1[h * LD + kk],
                     to_f(V[(((long)table[key / PAGE] * p.G + h / rep) * PAGE + key % PAGE) * p.vdim + d]), a);
          }
          acc[i] = a;
        }
        __syncthreads();
      }
    }
  }
  T* out = static_cast<T*>(p.out) + row * p.ldo;
  for (int i = tid; i < p.out_cols; i += 256) {
    const int h = i / p.vdim;
    from_f(out + i, h < H ? acc[i] / (p.mix_weights ? 1.f : l[h]) * head_gate<T>(p, row, h) : 0.f);
  }
}

// cap tanh(x): `two_over` is 2 log2(e) scale / cap, the factor of the raw product
__device__ __forceinline__ float capped(float raw, float two_over, float cap) {
  const float t = __builtin_amdgcn_exp2f(raw * two_over);
  return cap - 2.f * cap * __builtin_amdgcn_rcpf(1.f + t);
}

// x[k] of lane group g  ->  x[g] of lane group k (groups of 16 lanes)
__device__ __forceinline__ void transpose_groups(u32x4 (&x)[4]) {
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const auto a = __builtin_amdgcn_permlane32_swap(x[0][e], x[2][e], false, false);
    const auto b = __builtin_amdgcn_permlane32_swap(x[1][e], x[3][e], false, false);
    const auto c = __builtin_amdgcn_permlane16_swap(a[0], b[0], false, false);
    const auto d = __builtin_amdgcn_permlane16_swap(a[1], b[1], false, false);
    x[0][e] = c[0];
    x[1][e] = c[1];
    x[2][e] = d[0];
    x[3][e] = d[1];
  }
}

// Prompt attention.  HP / 4 waves share 16 queries, each owning 4 consecutive
// heads; a block has at least 4 waves (one or more such groups of queries).  Per
// 32-key tile: scores of
// the own heads -> LDS -> barrier -> every wave mixes the scores of all heads
// into its own four (row 4 g of the product is head g, so lane (r, g) ends with
// all keys of query r, head g) -> barrier -> softmax in the lane, weights
// transposed between lane groups and registers, second product per head.  Few
// queries: the keys are split over blockIdx.y, partial outputs combined after.
template <int DKS, int VT, int HP>
__global__ __launch_bounds__(HP == 32 ? 512 : 256, HP == 32 ? 1 : 2) void talk_prefill_kernel(TalkParams p) {
  constexpr int TK = 32, HW = HP / 4, NW = HW > 4 ? HW : 4, QG = NW / HW;
  constexpr int PITCH = HP == 8 ? 8 : HP + 8;  // fp16 scores of one pair
  constexpr int PLANE = TK * 16 * PITCH;
  __shared__ __attribute__((aligned(16))) _Float16 ss[QG * 2 * PLANE];
  __shared__ __attribute__((aligned(16))) bf16 vst[NW][TK * VLD];
  const int tile = xcd_remap(blockIdx.x, gridDim.x);
  const int seq = p.tiles[2 * tile], off = p.tiles[2 * tile + 1];
  const int cu = p.s.cu[seq], qlen = p.s.cu[seq + 1] - cu, st = p.s.start[seq];
  const int* table = p.table + (long)p.s.slots[seq] * p.tw;
  const bf16* K = static_cast<const bf16*>(p.k);
  const bf16* V = static_cast<const bf16*>(p.v);
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int hw = w % HW, qg = w / HW, H = p.H, G = p.G, rep = H / G, dim = p.dim, vdim = p.vdim;
  _Float16* s_hi = ss + qg * 2 * PLANE;
  _Float16* s_lo = s_hi + PLANE;
  bf16* vs = vst[w];

  const int qi = off + qg * 16 + r, qc = min(qi, qlen - 1);
  const int my_pos = st + qc, my_lo = first_key(my_pos, p.window);
  int kv[4];
#pragma unroll
  for (int hh = 0; hh < 4; ++hh) kv[hh] = min(hw * 4 + hh, H - 1) / rep;
  const int q_at = (cu + qc) * H * dim + g * 8;
  half8 tf = {};
  if ((r & 3) == 0 && g * 8 < HP)
    tf = *reinterpret_cast<const half8*>(static_cast<const _Float16*>(p.talk_frag) + (hw * 4 + (r >> 2)) * HP + g * 8);

  f32x4 o[4][VT];
#pragma unroll
  for (int hh = 0; hh < 4; ++hh)
#pragma unroll
    for (int di = 0; di < VT; ++di) o[hh][di] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = NEG, lsum = 0.f;
  const float two_over = 2.f * LOG2E * p.scale / p.cap;
  const int lo = first_key(st + off, p.window), hi = st + min(off + QG * 16, qlen);
  int kt0 = lo / TK, kt1 = (hi + TK - 1) / TK;
  if (p.splits > 1) {
    const int per = (kt1 - kt0 + p.splits - 1) / p.splits;
    kt0 += blockIdx.y * per;
    kt1 = min(kt1, kt0 + per);
  }
  // 64 columns of the tile's V rows, 16 bytes per lane and 8 rows
  bf16x8 vr[4];
  auto load_v = [&](long page, int koff, int kvh, int vh) {
    const bf16* vp = V + ((page * G + kvh) * PAGE + koff) * vdim + vh * 64;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      const int row = c * 8 + (lane >> 3), col = (lane & 7) * 8;
      const bf16x8 z = {};
      vr[c] = vh * 64 + col < vdim ? ld8(vp + (long)row * vdim + col) : z;
    }
  };

  for (int kt = kt0; kt < kt1; ++kt) {
    const long page = table[kt * TK / PAGE];
    const int koff = (kt * TK) % PAGE;
    // scores of the own heads; the queries are read again for every tile (from
    // L1 / L2): the outputs take the registers
    f32x4 s[4][2];
    bf16x8 kf[2][DKS];
    const bf16* qb = static_cast<const bf16*>(p.q);
    asm volatile("" : "+s"(qb));  // not hoisted out of the loop
#pragma unroll
    for (int hh = 0; hh < 4; ++hh) {
      const bf16x8 z = {};
      if (hh == 0 || kv[hh] != kv[hh - 1]) {  // wave-uniform
        const bf16* kp = K + ((page * G + kv[hh]) * PAGE + koff + r) * dim + g * 8;
#pragma unroll
        for (int ni = 0; ni < 2; ++ni)
#pragma unroll
          for (int ks = 0; ks < DKS; ++ks) kf[ni][ks] = ks * 32 < dim ? ld8(kp + ni * 16 * dim + ks * 32) : z;
      }
      bf16x8 qf[DKS];
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks)
        qf[ks] = ks * 32 < dim ? ld8(qb + q_at + min(hw * 4 + hh, H - 1) * dim + ks * 32) : z;
#pragma unroll
      for (int ni = 0; ni < 2; ++ni) {
        s[hh][ni] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < DKS; ++ks) s[hh][ni] = mfma16(kf[ni][ks], qf[ks], s[hh][ni]);
      }
    }
#pragma unroll
    for (int ni = 0; ni < 2; ++ni)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        half4 a, b;
#pragma unroll
        for (int hh = 0; hh < 4; hh += 2) {  // the remainder makes up for the truncated first term
          const float c = capped(s[hh][ni][i], two_over, p.cap), d = capped(s[hh + 1][ni][i], two_over, p.cap);
          const half2 u = pack_half(c, d), v = pack_half(c - (float)u[0], d - (float)u[1]);
          a[hh] = u[0];
          a[hh + 1] = u[1];
          b[hh] = v[0];
          b[hh + 1] = v[1];
        }
        const int at = ((ni * 16 + 4 * g + i) * 16 + r) * PITCH + hw * 4;
        *reinterpret_cast<half4*>(s_hi + at) = a;
        *reinterpret_cast<half4*>(s_lo + at) = b;
      }
    load_v(page, koff, kv[0], 0);  // in flight under the mixing and the softmax
    __syncthreads();
    float e[TK];
#pragma unroll
    for (int key = 0; key < TK; ++key) {
      half8 a = {}, b = {};
      if (g * 8 < HP) {
        a = *reinterpret_cast<const half8*>(s_hi + (key * 16 + r) * PITCH + g * 8);
        b = *reinterpret_cast<const half8*>(s_lo + (key * 16 + r) * PITCH + g * 8);
      }
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      acc = mfma_f16(tf, a, acc);
      acc = mfma_f16(tf, b, acc);
      e[key] = acc[0] * LOG2E;
    }
    __syncthreads();  // the next tile's scores may be written
    const bool whole = kt * TK >= my_lo && kt * TK + TK - 1 <= my_pos;
    if (!__all(whole)) {
#pragma unroll
      for (int key = 0; key < TK; ++key) {
        const int k = kt * TK + key;
        e[key] = k >= my_lo && k <= my_pos ? e[key] : NEG;
      }
    }
    float tmax = e[0];
#pragma unroll
    for (int key = 1; key < TK; ++key) tmax = fmaxf(tmax, e[key]);
    // weights are taken relative to m, which follows the running maximum only
    // when that is more than 2^6 ahead
    if (__any(tmax > m + 6.f)) {
      const float mn = fmaxf(m, tmax);
      const float alpha = __builtin_amdgcn_exp2f(m - mn);
      m = mn;
      lsum *= alpha;
#pragma unroll
      for (int hh = 0; hh < 4; ++hh) {
        const float ah = __shfl(alpha, hh * 16 + r, 64);
#pragma unroll
        for (int di = 0; di < VT; ++di) o[hh][di] *= ah;
      }
    }
    const float off2 = m > 0.5f * NEG ? m : 0.f;  // no key seen yet: weights of zero
    float ps = 0.f;
#pragma unroll
    for (int key = 0; key < TK; ++key) {
      e[key] = __builtin_amdgcn_exp2f(e[key] - off2);
      ps += e[key];
    }
    lsum += ps;
    // k-slot j of group g <-> key 4 g + j (j < 4), 16 + 4 g + (j - 4) (j >= 4)
    u32x4 ph[4], pl[4];
#pragma unroll
    for (int kg = 0; kg < 4; ++kg) split_p(e + 4 * kg, e + 16 + 4 * kg, ph[kg], pl[kg]);
    transpose_groups(ph);
    transpose_groups(pl);
#pragma unroll
    for (int hh = 0; hh < 4; ++hh) {
      if (hh > 0 && kv[hh] == kv[hh - 1]) continue;  // done with the head before
#pragma unroll
      for (int vh = 0; vh < VT / 4; ++vh) {
        if (vh * 64 >= vdim) continue;
        if (hh > 0 && vh == 0) load_v(page, koff, kv[hh], 0);
        lds_fence();  // reads of what is staged now are done
#pragma unroll
        for (int c = 0; c < 4; ++c) st8(vs + (c * 8 + (lane >> 3)) * VLD + (lane & 7) * 8, vr[c]);
        if ((vh + 1) * 64 < vdim) load_v(page, koff, kv[hh], vh + 1);
        lds_fence();
        const int r0 = 4 * g + (r >> 2);
#pragma unroll
        for (int dj = 0; dj < 4; ++dj) {
          const int col = dj * 16 + 4 * (r & 3);
          const bf16x4 a = ds_read_tr(vs + r0 * VLD + col);
          const bf16x4 b = ds_read_tr(vs + (r0 + 16) * VLD + col);
          const bf16x8 vf = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
#pragma unroll
          for (int h2 = 0; h2 < 4; ++h2)
            if (h2 >= hh && kv[h2] == kv[hh]) {  // wave-uniform
              o[h2][vh * 4 + dj] = mfma16(vf, __builtin_bit_cast(bf16x8, ph[h2]), o[h2][vh * 4 + dj]);
              o[h2][vh * 4 + dj] = mfma16(vf, __builtin_bit_cast(bf16x8, pl[h2]), o[h2][vh * 4 + dj]);
            }
        }
      }
    }
  }
  if (p.splits > 1) {
#pragma unroll
    for (int hh = 0; hh < 4; ++hh) {
      const int h = hw * 4 + hh;
      if (h >= H || qi >= qlen) continue;
      const long pi = ((long)(cu + qi) * H + h) * p.splits + blockIdx.y;
#pragma unroll
      for (int di = 0; di < VT; ++di)
        if (di * 16 < vdim) *reinterpret_cast<f32x4*>(p.part_o + pi * vdim + di * 16 + 4 * g) = o[hh][di];
    }
    const int h = hw * 4 + g;
    if (h < H && qi < qlen) {
      const long pi = ((long)(cu + qi) * H + h) * p.splits + blockIdx.y;
      p.part_ml[2 * pi] = m;
      p.part_ml[2 * pi + 1] = lsum;
    }
    return;
  }
  const float inv = 1.f / lsum;
  bf16* out = static_cast<bf16*>(p.out) + (long)(cu + qc) * p.ldo;
#pragma unroll
  for (int hh = 0; hh < 4; ++hh) {
    const float ih = __shfl(inv, hh * 16 + r, 64);
    const int h = hw * 4 + hh;
    if (h >= H || qi >= qlen) continue;
#pragma unroll
    for (int di = 0; di < VT; ++di) {
      if (di * 16 >= vdim) continue;
      st4(out + h * vdim + di * 16 + 4 * g, bf16x4{f2bf(o[hh][di][0] * ih), f2bf(o[hh][di][1] * ih),
                                                   f2bf(o[hh][di][2] * ih), f2bf(o[hh][di][3] * ih)});
    }
  }
  if (hw == HW - 1 && qi < qlen)
    for (int c = H * vdim + g; c < p.out_cols; c += 4) out[c] = f2bf(0.f);
}

// Decode attention: one token of all heads, keys in 64-key tiles (pages).  Four
// waves share the K / V heads; the columns of a score product are the query heads
// of one K head.  Mixing: wave w takes keys 16 w .. of the tile, all heads.
template <int DKS, int VT, int HP>
__global__ __launch_bounds__(256, 2) void talk_decode_kernel(TalkParams p) {
  constexpr int PITCH = HP + 8, MT = HP / 16, PLD = PAGE + 8;
  constexpr int GW = HP / 4;  // K / V heads per wave at most
  __shared__ __attribute__((aligned(16))) _Float16 s_hi[PAGE * PITCH], s_lo[PAGE * PITCH];
  __shared__ __attribute__((aligned(16))) bf16 p_hi[HP * PLD], p_lo[HP * PLD];
  __shared__ __attribute__((aligned(16))) bf16 vst[4][32 * VLD];
  __shared__ float tmaxs[4][HP], alphas[HP], ms[HP], ls[4][HP];
  const int b = blockIdx.x, H = p.H, G = p.G, rep = H / G, dim = p.dim, vdim = p.vdim;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int pos = p.pos[b], lo = first_key(pos, p.window);
  const int* table = p.table + (long)p.slots[b] * p.tw;
  const bf16* K = static_cast<const bf16*>(p.k);
  const bf16* V = static_cast<const bf16*>(p.v);
  const int t0 = lo / PAGE, nt = pos / PAGE + 1 - t0;
  const int per = (nt + p.splits - 1) / p.splits;
  const int ta = t0 + blockIdx.y * per, tb = min(ta + per, t0 + nt);
  bf16* vs = vst[w];
  const float two_over = 2.f * LOG2E * p.scale / p.cap;

  half8 tf[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const half8 z = {};
    tf[mt] = g * 8 < HP ? *reinterpret_cast<const half8*>(static_cast<const _Float16*>(p.talk_frag) +
                                                           (mt * 16 + r) * HP + g * 8) : z;
  }
  // scores of heads that do not exist stay zero
  for (int i = threadIdx.x; i < PAGE * PITCH; i += 256) s_hi[i] = s_lo[i] = (_Float16)0.f;
  if (threadIdx.x < HP) ms[threadIdx.x] = NEG;
  f32x4 o[GW / 4 > 0 ? GW / 4 : 1][VT];
  constexpr int GMAX = GW / 4 > 0 ? GW / 4 : 1;  // heads per wave the accumulators hold: 4 GMAX >= G
#pragma unroll
  for (int c = 0; c < GMAX; ++c)
#pragma unroll
    for (int di = 0; di < VT; ++di) o[c][di] = f32x4{0.f, 0.f, 0.f, 0.f};
  f32x4 lsum[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) lsum[mt] = f32x4{0.f, 0.f, 0.f, 0.f};
  __syncthreads();

  for (int kt = ta; kt < tb; ++kt) {
    const long page = table[kt];
#pragma unroll
    for (int c = 0; c < GMAX; ++c) {
      const int kvh = w + 4 * c;
      if (kvh >= G) continue;
      bf16x8 qf[DKS], kf[4][DKS];
      const bf16* q = static_cast<const bf16*>(p.q) + ((long)b * H + kvh * rep + min(r, rep - 1)) * dim + g * 8;
      const bf16* kp = K + ((page * G + kvh) * PAGE + r) * dim + g * 8;
      const bf16x8 z = {};
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) qf[ks] = ks * 32 < dim ? ld8(q + ks * 32) : z;
#pragma unroll
      for (int ni = 0; ni < 4; ++ni)
#pragma unroll
        for (int ks = 0; ks < DKS; ++ks) kf[ni][ks] = ks * 32 < dim ? ld8(kp + (long)ni * 16 * dim + ks * 32) : z;
#pragma unroll
      for (int ni = 0; ni < 4; ++ni) {
        f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < DKS; ++ks) s = mfma16(kf[ni][ks], qf[ks], s);
        if (r < rep) {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float cv = capped(s[i], two_over, p.cap);
            const _Float16 a = (_Float16)cv;
            const int at = (ni * 16 + 4 * g + i) * PITCH + kvh * rep + r;
            s_hi[at] = a;
            s_lo[at] = (_Float16)(cv - (float)a);
          }
        }
      }
    }
    __syncthreads();
    // column r: key 16 w + r, rows: heads
    f32x4 e[MT];
    const int key = kt * PAGE + w * 16 + r;
    const bool seen = key >= lo && key <= pos;
    {
      half8 a = {}, bq = {};
      if (g * 8 < HP) {
        a = *reinterpret_cast<const half8*>(s_hi + (w * 16 + r) * PITCH + g * 8);
        bq = *reinterpret_cast<const half8*>(s_lo + (w * 16 + r) * PITCH + g * 8);
      }
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        acc = mfma_f16(tf[mt], a, acc);
        acc = mfma_f16(tf[mt], bq, acc);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          e[mt][i] = seen ? acc[i] * LOG2E : NEG;
          float t = e[mt][i];
          t = fmaxf(t, wave_xchg<1>(t));
          t = fmaxf(t, wave_xchg<2>(t));
          t = fmaxf(t, wave_xchg<4>(t));
          t = fmaxf(t, wave_xchg<8>(t));
          if (r == 0) tmaxs[w][mt * 16 + 4 * g + i] = t;
        }
      }
    }
    __syncthreads();
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int h = mt * 16 + 4 * g + i;
        const float mo = ms[h];
        const float t = fmaxf(fmaxf(tmaxs[0][h], tmaxs[1][h]), fmaxf(tmaxs[2][h], tmaxs[3][h]));
        const float mn = t > mo + 6.f ? t : mo;  // every tile of the range holds a visible key
        const float pw = __builtin_amdgcn_exp2f(e[mt][i] - mn);
        const float al = __builtin_amdgcn_exp2f(mo - mn);
        lsum[mt][i] = lsum[mt][i] * al + pw;
        const bf16 ph = f2bf(pw);
        p_hi[h * PLD + w * 16 + r] = ph;
        p_lo[h * PLD + w * 16 + r] = f2bf(pw - bf2f(ph));
        if (w == 0 && r == 0) alphas[h] = al;
        e[mt][i] = mn;
      }
    }
    __syncthreads();
    if (w == 0 && r == 0) {
#pragma unroll
      for (int mt = 0; mt < MT; ++mt)
#pragma unroll
        for (int i = 0; i < 4; ++i) ms[mt * 16 + 4 * g + i] = e[mt][i];
    }
#pragma unroll
    for (int c = 0; c < GMAX; ++c) {
      const int kvh = w + 4 * c;
      if (kvh >= G) continue;
      const int h = kvh * rep + min(r, rep - 1);
      const float al = alphas[h];
      if (__any(al != 1.f)) {
#pragma unroll
        for (int di = 0; di < VT; ++di) o[c][di] *= al;
      }
#pragma unroll
      for (int vh = 0; vh < VT / 4; ++vh) {
        if (vh * 64 >= vdim) continue;
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
          const bf16* vp = V + ((page * G + kvh) * PAGE + kk * 32) * vdim + vh * 64;
          bf16x8 vr[4];
#pragma unroll
          for (int q4 = 0; q4 < 4; ++q4) {
            const int row = q4 * 8 + (lane >> 3), col = (lane & 7) * 8;
            const bf16x8 z = {};
            vr[q4] = vh * 64 + col < vdim ? ld8(vp + (long)row * vdim + col) : z;
          }
          const bf16* ph = p_hi + h * PLD + kk * 32 + 4 * g;
          const bf16* pl = p_lo + h * PLD + kk * 32 + 4 * g;
          const bf16x4 h0 = ld4(ph), h1 = ld4(ph + 16), l0 = ld4(pl), l1 = ld4(pl + 16);
          const bf16x8 hf = {h0[0], h0[1], h0[2], h0[3], h1[0], h1[1], h1[2], h1[3]};
          const bf16x8 lf = {l0[0], l0[1], l0[2], l0[3], l1[0], l1[1], l1[2], l1[3]};
          lds_fence();
#pragma unroll
          for (int q4 = 0; q4 < 4; ++q4) st8(vs + (q4 * 8 + (lane >> 3)) * VLD + (lane & 7) * 8, vr[q4]);
          lds_fence();
          const int r0 = 4 * g + (r >> 2);
#pragma unroll
          for (int dj = 0; dj < 4; ++dj) {
            const int col = dj * 16 + 4 * (r & 3);
            const bf16x4 a = ds_read_tr(vs + r0 * VLD + col);
            const bf16x4 d = ds_read_tr(vs + (r0 + 16) * VLD + col);
            const bf16x8 vf = {a[0], a[1], a[2], a[3], d[0], d[1], d[2], d[3]};
            o[c][vh * 4 + dj] = mfma16(vf, hf, o[c][vh * 4 + dj]);
            o[c][vh * 4 + dj] = mfma16(vf, lf, o[c][vh * 4 + dj]);
          }
        }
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float t = lsum[mt][i];
      t += wave_xchg<1>(t);
      t += wave_xchg<2>(t);
      t += wave_xchg<4>(t);
      t += wave_xchg<8>(t);
      if (r == 0) ls[w][mt * 16 + 4 * g + i] = t;
    }
  __syncthreads();
#pragma unroll
  for (int c = 0; c < GMAX; ++c) {
    const int kvh = w + 4 * c;
    if (kvh >= G || r >= rep) continue;
    const int h = kvh * rep + r;
    const float l = ls[0][h] + ls[1][h] + ls[2][h] + ls[3][h];
    if (p.splits > 1) {
      const long pi = ((long)b * H + h) * p.splits + blockIdx.y;
#pragma unroll
      for (int di = 0; di < VT; ++di)
        if (di * 16 < vdim) *reinterpret_cast<f32x4*>(p.part_o + pi * vdim + di * 16 + 4 * g) = o[c][di];
      if (g == 0) {
        p.part_ml[2 * pi] = ms[h];
        p.part_ml[2 * pi + 1] = l;
      }
    } else {
      const float inv = 1.f / l;
      bf16* out = static_cast<bf16*>(p.out) + (long)b * p.ldo + h * vdim;
#pragma unroll
      for (int di = 0; di < VT; ++di)
        if (di * 16 < vdim)
          st4(out + di * 16 + 4 * g, bf16x4{f2bf(o[c][di][0] * inv), f2bf(o[c][di][1] * inv), f2bf(o[c][di][2] * inv),
                                            f2bf(o[c][di][3] * inv)});
    }
  }
  if (p.splits == 1)
    for (int c = H * vdim + threadIdx.x; c < p.out_cols; c += 256) static_cast<bf16*>(p.out)[(long)b * p.ldo + c] = f2bf(0.f);
}

// One wave per (query, head); the last head's also clears the pad columns.
__global__ __launch_bounds__(64) void talk_combine_kernel(TalkParams p) {
  constexpr int RUN = 8;  // splits whose rows are loaded together
  __shared__ float ws[256];
  const int b = blockIdx.x / p.H, h = blockIdx.x % p.H, lane = threadIdx.x;
  const long pi = (long)blockIdx.x * p.splits;
  float m[4], l[4], M = NEG, L = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int s = lane + 64 * i;
    m[i] = s < p.splits ? p.part_ml[2 * (pi + s)] : NEG;
    l[i] = s < p.splits ? p.part_ml[2 * (pi + s) + 1] : 0.f;
    M = fmaxf(M, m[i]);
  }
  M = wave_max(M);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float w = lane + 64 * i < p.splits ? exp2f(m[i] - M) : 0.f;
    ws[lane + 64 * i] = w;
    L += l[i] * w;
  }
  const float inv = 1.f / wave_sum(L), gate = head_gate<bf16>(p, b, h);
  __syncthreads();
  bf16* out = static_cast<bf16*>(p.out) + (long)b * p.ldo;
  for (int d = lane; d < p.vdim; d += 64) {
    float v = 0.f;
    for (int s = 0; s < p.splits; s += RUN) {
      float x[RUN];
#pragma unroll
      for (int i = 0; i < RUN; ++i) x[i] = p.part_o[(pi + min(s + i, p.splits - 1)) * p.vdim + d];
#pragma unroll
      for (int i = 0; i < RUN; ++i) v += x[i] * ws[s + i];
    }
    out[h * p.vdim + d] = f2bf(v * inv * gate);
  }
  if (h == p.H - 1)
    for (int c = p.H * p.vdim + lane; c < p.out_cols; c += 64) out[c] = f2bf(0.f);
}

}  // namespace
}  // namespace lsd

using namespace lsd;

// Head padding of the MFMA kernels, 0: sizes they do not take.  cap: of the mixed
// scores, < 0 where weights are mixed.
extern "C" int lsd_talk_heads(int H, int G, int dim, int vdim, float cap) {
  if (H > 32 || H / G > 16 || dim % 32 || dim > 128 || vdim % 16 || vdim > 128 || cap == 0.f || cap > 3e4f) return 0;
  return H <= 8 ? 8 : H <= 16 ? 16 : 32;
}

extern "C" int lsd_talk_tile(int hp) { return hp == 8 ? 32 : 16; }  // queries of a prefill tile

#define LSD_TK_V(KERNEL, GRID, NT, ...)                                                                           \
  if (p->dim <= 64 && p->vdim <= 64) hipLaunchKernelGGL((KERNEL<2, 4, __VA_ARGS__>), GRID, dim3(NT), 0, st, *p); \
  else if (p->dim <= 64) hipLaunchKernelGGL((KERNEL<2, 8, __VA_ARGS__>), GRID, dim3(NT), 0, st, *p);              \
  else if (p->vdim <= 64) hipLaunchKernelGGL((KERNEL<4, 4, __VA_ARGS__>), GRID, dim3(NT), 0, st, *p);             \
  else hipLaunchKernelGGL((KERNEL<4, 8, __VA_ARGS__>), GRID, dim3(NT), 0, st, *p);

extern "C" hipError_t lsd_attention_combine(const TalkParams* p, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  hipLaunchKernelGGL(talk_combine_kernel, dim3(p->T * p->H), dim3(64), 0, st, *p);
  return hipGetLastError();
}

extern "C" hipError_t lsd_talk_prefill(const TalkParams* p, int hp, hipStream_t st) {
  if (p->n_tiles == 0) return hipSuccess;
  const dim3 grid(p->n_tiles, p->splits);
  if (p->mix_weights) return hipErrorInvalidValue;
  switch (hp) {
    case 8: LSD_TK_V(talk_prefill_kernel, grid, 256, 8) break;
    case 16: LSD_TK_V(talk_prefill_kernel, grid, 256, 16) break;
    case 32: LSD_TK_V(talk_prefill_kernel, grid, 512, 32) break;
    default: return hipErrorInvalidValue;
  }
  if (p->splits > 1) return lsd_attention_combine(p, st);
  return hipGetLastError();
}

// hp: 16 or 32 (talk_frag padded to it); needs G <= hp
extern "C" hipError_t lsd_talk_decode(const TalkParams* p, int hp, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  if (p->mix_weights) return hipErrorInvalidValue;
  const dim3 grid(p->T, p->splits);
  switch (hp) {
    case 16: LSD_TK_V(talk_decode_kernel, grid, 256, 16) break;
    case 32: LSD_TK_V(talk_decode_kernel, grid, 256, 32) break;
    default: return hipErrorInvalidValue;
  }
  if (p->splits > 1) return lsd_attention_combine(p, st);
  return hipGetLastError();
}
#undef LSD_TK_V

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
