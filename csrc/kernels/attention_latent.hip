// Attention over a paged cache of latents (multi-query in the latent space).
//
// Keys and values of every head are linear images of one cached latent row per
// token, k_h = U_h c and v_h = V_h c, so the scores are (U_h^T q_h) . c and the
// output is V_h (sum_j p_j c_j): with the queries taken into the latent space
// once per token (group_gemm.hip), all heads attend over the SAME rows, which
// serve as keys and as values.  One cached row per token, no per-head cache.
// A window (`window` keys ending with the query itself) bounds the key range.
//
// A turned key part that all heads share is cached behind the latent: the way into
// the latent space passes the queries' turned part on, and only the first columns
// of a row are values.  A sink is one more score of the softmax, without a value.
//
// Cache: [page][64 tokens][rank], pages found through table[slot][pos / 64].
// A 32- or 64-key tile never crosses a page.
//
//  * prefill: a block takes a tile of consecutive (token, head) query rows of
//    one sequence; key tiles go through LDS once and are read as the K operand
//    (rows) and, through ds_read_b64_tr_b16, as the V^T operand.
//  * expanded prefill: where a prompt scores many keys per latent row, the keys
//    and values of the rows in reach are made once (latent_gather + two plain
//    GEMMs) and a per-head flash kernel runs over them: (dim + vdim) / (2 rank)
//    of the multiply-adds per score.
//  * decode: a block takes 16 heads of one token; its 4 waves take key tiles
//    in turn, each with a private LDS tile, merged at the end, or (wide rows)
//    share a tile and divide the value columns; long ranges are split over
//    blocks (latent_combine).
//  * plain: one (token, head) per block on the VALU -- fp32 models, and ranks
//    without an MFMA instantiation.
//
// The MFMA kernels swap the operands (S^T = K Q^T) as attention.hip does, so a
// lane holds one query's scores and P^T needs no LDS trip.  The softmax weights
// are multiplied as a pair of bf16 terms (value + remainder): 16 bits of
// mantissa against bf16 values, with fp32 accumulation.
#include "common.h"
#include "moe_params.h"

namespace lsd {
namespace {

constexpr float NEG = -1e30f;
constexpr int PAGE = 64;
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ bf16x4 ds_read_tr(const bf16* lds_ptr) {
  typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)(lds_ptr));
}

// first key a query at `pos` sees
__device__ __forceinline__ int first_key(int pos, int window) { return window > pos ? 0 : pos - window + 1; }

// Does any query of the wave need a new reference maximum?  Weights are taken
// relative to m, which follows the running maximum only when that is more than
// 2^6 ahead: the sums stay far from overflow, and most tiles rescale nothing.
__device__ __forceinline__ bool grew(float tmax, float m) { return __any(tmax > m + 6.f); }

// Two bf16 terms of each weight
__device__ __forceinline__ void split_p(const f32x4& a, const f32x4& b, bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    hi[j] = f2bf(a[j]);
    lo[j] = f2bf(a[j] - bf2f(hi[j]));
    hi[4 + j] = f2bf(b[j]);
    lo[4 + j] = f2bf(b[j] - bf2f(hi[4 + j]));
  }
}

template <int RANK, int VR, int QT, int NW, int KT>
__global__ __launch_bounds__(NW * 64) void latent_prefill_kernel(LatentAttnParams p) {
  constexpr int LDR = RANK + 8;
  constexpr int CPR = RANK / 8;
  constexpr int NT = NW * 64;
  constexpr int CH = (KT * CPR + NT - 1) / NT;
  constexpr int ROWS = NW * QT * 16;
  __shared__ __attribute__((aligned(16))) bf16 cs[KT * LDR];
  const int seq = p.tiles[2 * blockIdx.x], off = p.tiles[2 * blockIdx.x + 1];
  const int cu = p.cu_q[seq], H = p.H;
  const int nrows = (p.cu_q[seq + 1] - cu) * H;
  const int st = p.pos[seq];
  const int* table = p.table + (long)p.seq_slots[seq] * p.tw;
  const bf16* cache = static_cast<const bf16*>(p.cache);
  const int lane = lane_id(), w = threadIdx.x >> 6;
  const int r = lane & 15, g = lane >> 4;

  int row[QT], my_pos[QT], my_lo[QT];
  bf16x8 qf[QT][RANK / 32];
  const bf16* qbase = static_cast<const bf16*>(p.q) + (long)cu * H * RANK;
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    row[t] = off + (w * QT + t) * 16 + r;
    const int rc = min(row[t], nrows - 1);
    my_pos[t] = st + rc / H;
    my_lo[t] = first_key(my_pos[t], p.window);
#pragma unroll
    for (int kk = 0; kk < RANK / 32; ++kk) qf[t][kk] = ld8(qbase + (long)rc * RANK + kk * 32 + g * 8);
  }
  const int lo = first_key(st + off / H, p.window);
  const int hi = st + min(off + ROWS - 1, nrows - 1) / H + 1;  // keys [lo, hi)
  const int kt0 = lo / KT, kt1 = (hi + KT - 1) / KT;

  f32x4 o[QT][VR / 16];
  float m[QT], lsum[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    // a sink is a key that was seen first, without a value
    m[t] = p.sink ? p.sink[min(row[t], nrows - 1) % H] * LOG2E : NEG;
    lsum[t] = p.sink && g == 0 ? 1.f : 0.f;
#pragma unroll
    for (int di = 0; di < VR / 16; ++di) o[t][di] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  bf16x8 creg[CH];
  auto load_tile = [&](int kt) {
    const bf16* src = cache + ((long)table[kt * KT / PAGE] * PAGE + (kt * KT) % PAGE) * RANK;
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int idx = threadIdx.x + c * NT;
      if (KT * CPR % NT == 0 || idx < KT * CPR) creg[c] = ld8(src + idx * 8);
    }
  };
  load_tile(kt0);
  for (int kt = kt0; kt < kt1; ++kt) {
    __syncthreads();  // the previous tile's readers are done
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int idx = threadIdx.x + c * NT;
      if (KT * CPR % NT == 0 || idx < KT * CPR) st8(cs + (idx / CPR) * LDR + (idx % CPR) * 8, creg[c]);
    }
    __syncthreads();
    if (kt + 1 < kt1) load_tile(kt + 1);  // in flight under this tile's math

    f32x4 s[QT][KT / 16];
#pragma unroll
    for (int ni = 0; ni < KT / 16; ++ni) {
#pragma unroll
      for (int t = 0; t < QT; ++t) s[t][ni] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < RANK / 32; ++kk) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(cs + (ni * 16 + r) * LDR + kk * 32 + g * 8);
#pragma unroll
        for (int t = 0; t < QT; ++t) s[t][ni] = mfma16(kf, qf[t][kk], s[t][ni]);
      }
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float tmax = NEG;
#pragma unroll
      for (int ni = 0; ni < KT / 16; ++ni)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = kt * KT + ni * 16 + 4 * g + i;
          const float sv = (key <= my_pos[t] && key >= my_lo[t]) ? s[t][ni][i] * p.scale_log2 : NEG;
          s[t][ni][i] = sv;
          tmax = fmaxf(tmax, sv);
        }
      tmax = fmaxf(tmax, wave_xchg<16>(tmax));
      tmax = fmaxf(tmax, wave_xchg<32>(tmax));
      if (grew(tmax, m[t])) {
        const float mn = fmaxf(m[t], tmax);
        const float alpha = exp2f(m[t] - mn);
        m[t] = mn;
        lsum[t] *= alpha;
#pragma unroll
        for (int di = 0; di < VR / 16; ++di) o[t][di] *= alpha;
      }
      // a query whose window has not begun yet: nothing to weigh
      const float off2 = m[t] > 0.5f * NEG ? m[t] : 0.f;
      float ps = 0.f;
#pragma unroll
      for (int ni = 0; ni < KT / 16; ++ni)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = exp2f(s[t][ni][i] - off2);
          s[t][ni][i] = e;
          ps += e;
        }
      lsum[t] += ps;
    }
    // O^T[d][q] += C^T[d][key] . P^T[key][q]; k-slot j of group g <-> key
    // 32 kk + 4 g + j (j < 4), 32 kk + 16 + 4 g + (j - 4) (j >= 4)
#pragma unroll
    for (int kk = 0; kk < KT / 32; ++kk) {
      bf16x8 ph[QT], pl[QT];
#pragma unroll
      for (int t = 0; t < QT; ++t) split_p(s[t][2 * kk], s[t][2 * kk + 1], ph[t], pl[t]);
      const int r0 = kk * 32 + 4 * g + (r >> 2);
#pragma unroll
      for (int di = 0; di < VR / 16; ++di) {
        const int col = di * 16 + 4 * (r & 3);
        const bf16x4 a = ds_read_tr(cs + r0 * LDR + col);
        const bf16x4 b = ds_read_tr(cs + (r0 + 16) * LDR + col);
        const bf16x8 vf = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
#pragma unroll
        for (int t = 0; t < QT; ++t) {
          o[t][di] = mfma16(vf, ph[t], o[t][di]);
          o[t][di] = mfma16(vf, pl[t], o[t][di]);
        }
      }
    }
  }
  bf16* obase = static_cast<bf16*>(p.out) + (long)cu * H * VR;
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    float l = lsum[t];
    l += wave_xchg<16>(l);
    l += wave_xchg<32>(l);
    if (row[t] >= nrows) continue;
    const float inv = 1.f / l;
#pragma unroll
    for (int di = 0; di < VR / 16; ++di) {
      bf16x4 rr;
#pragma unroll
      for (int i = 0; i < 4; ++i) rr[i] = f2bf(o[t][di][i] * inv);
      st4(obase + (long)row[t] * VR + di * 16 + 4 * g, rr);
    }
  }
}

// 16 heads of one token per block; waves take the 32-key tiles in turn.
// Two blocks per CU where the tiles leave the LDS for it.
template <int RANK, int VR>
__global__ __launch_bounds__(256, RANK <= 256 ? 2 : 1) void latent_decode_kernel(LatentAttnParams p) {
  constexpr int KT = 32;
  constexpr int LDR = RANK + 8;
  constexpr int CPR = RANK / 8;
  constexpr int CH = KT * CPR / 64;
  __shared__ __attribute__((aligned(16))) bf16 lds[4][KT * LDR];  // a wave's tile, then its O^T
  __shared__ float ml[4][16][2];
  static_assert(KT * LDR * 2 >= VR * 16 * 4, "the partial output fits the key tile");
  const int H = p.H, HG = (H + 15) / 16;
  const int item = xcd_remap(blockIdx.x, gridDim.x);  // a token's head groups on one XCD
  const int b = item / HG, h0 = (item % HG) * 16;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  bf16* cs = lds[w];
  const int pos = p.pos[b], lo = first_key(pos, p.window);
  const int* table = p.table + (long)p.seq_slots[b] * p.tw;
  const bf16* cache = static_cast<const bf16*>(p.cache);
  const int t0 = lo / KT, nt = pos / KT + 1 - t0;
  const int per = (nt + p.splits - 1) / p.splits;
  const int ta = t0 + blockIdx.y * per, tb = min(ta + per, t0 + nt);

  bf16x8 qf[RANK / 32];
  const bf16* q = static_cast<const bf16*>(p.q) + ((long)b * H + min(h0 + r, H - 1)) * RANK;
#pragma unroll
  for (int kk = 0; kk < RANK / 32; ++kk) qf[kk] = ld8(q + kk * 32 + g * 8);
  f32x4 o[VR / 16];
#pragma unroll
  for (int di = 0; di < VR / 16; ++di) o[di] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = NEG, lsum = 0.f;
  if (p.sink && w == 0 && blockIdx.y == 0) {  // a key that was seen first, without a value
    m = p.sink[min(h0 + r, H - 1)] * LOG2E;
    lsum = g == 0 ? 1.f : 0.f;
  }

  bf16x8 creg[CH];
  auto page_of = [&](int kt) { return table[min(kt, tb - 1) * KT / PAGE]; };
  auto load_tile = [&](int kt, int page) {
    const bf16* src = cache + ((long)page * PAGE + (kt * KT) % PAGE) * RANK;
#pragma unroll
    for (int c = 0; c < CH; ++c) creg[c] = ld8(src + (lane + c * 64) * 8);
  };
  int page = 0;  // of the tile after the one being loaded
  if (ta + w < tb) {
    load_tile(ta + w, page_of(ta + w));
    page = page_of(ta + w + 4);
  }
  for (int kt = ta + w; kt < tb; kt += 4) {
    __builtin_amdgcn_s_waitcnt(0xC07F);  // lgkmcnt(0): this wave's reads of the previous tile
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int idx = lane + c * 64;
      st8(cs + (idx / CPR) * LDR + (idx % CPR) * 8, creg[c]);
    }
    __builtin_amdgcn_s_waitcnt(0xC07F);
    __builtin_amdgcn_wave_barrier();
    if (kt + 4 < tb) {  // in flight under this tile's math
      load_tile(kt + 4, page);
      page = page_of(kt + 8);
    }

    f32x4 s[2], s2[2];  // two chains per 16 keys
#pragma unroll
    for (int ni = 0; ni < 2; ++ni) s[ni] = s2[ni] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < RANK / 32; kk += 2)
#pragma unroll
      for (int ni = 0; ni < 2; ++ni) {
        const bf16* row = cs + (ni * 16 + r) * LDR + kk * 32 + g * 8;
        s[ni] = mfma16(*reinterpret_cast<const bf16x8*>(row), qf[kk], s[ni]);
        s2[ni] = mfma16(*reinterpret_cast<const bf16x8*>(row + 32), qf[kk + 1], s2[ni]);
      }
#pragma unroll
    for (int ni = 0; ni < 2; ++ni) s[ni] += s2[ni];
    float tmax = NEG;
#pragma unroll
    for (int ni = 0; ni < 2; ++ni)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = kt * KT + ni * 16 + 4 * g + i;
        const float sv = (key <= pos && key >= lo) ? s[ni][i] * p.scale_log2 : NEG;
        s[ni][i] = sv;
        tmax = fmaxf(tmax, sv);
      }
    tmax = fmaxf(tmax, wave_xchg<16>(tmax));
    tmax = fmaxf(tmax, wave_xchg<32>(tmax));
    if (grew(tmax, m)) {
      const float mn = fmaxf(m, tmax);
      const float alpha = exp2f(m - mn);
      m = mn;
      lsum *= alpha;
#pragma unroll
      for (int di = 0; di < VR / 16; ++di) o[di] *= alpha;
    }
    float ps = 0.f;
#pragma unroll
    for (int ni = 0; ni < 2; ++ni)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        // every tile of the range holds a visible key, so m is a real score
        const float e = exp2f(s[ni][i] - m);
        s[ni][i] = e;
        ps += e;
      }
    lsum += ps;
    bf16x8 ph, pl;
    split_p(s[0], s[1], ph, pl);
    const int r0 = 4 * g + (r >> 2);
#pragma unroll
    for (int di = 0; di < VR / 16; ++di) {
      const int col = di * 16 + 4 * (r & 3);
      const bf16x4 a = ds_read_tr(cs + r0 * LDR + col);
      const bf16x4 c = ds_read_tr(cs + (r0 + 16) * LDR + col);
      const bf16x8 vf = {a[0], a[1], a[2], a[3], c[0], c[1], c[2], c[3]};
      o[di] = mfma16(vf, ph, o[di]);
      o[di] = mfma16(vf, pl, o[di]);
    }
  }
  lsum += wave_xchg<16>(lsum);
  lsum += wave_xchg<32>(lsum);
  if (g == 0) {
    ml[w][r][0] = m;
    ml[w][r][1] = lsum;
  }
  __syncthreads();
  float M = NEG, L = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) M = fmaxf(M, ml[i][r][0]);
#pragma unroll
  for (int i = 0; i < 4; ++i) L += ml[i][r][1] * exp2f(ml[i][r][0] - M);
  const float f = exp2f(m - M);
  float* ow = reinterpret_cast<float*>(cs);  // [di][g][r][4]
#pragma unroll
  for (int di = 0; di < VR / 16; ++di)
    *reinterpret_cast<f32x4*>(ow + ((di * 4 + g) * 16 + r) * 4) = o[di] * f;
  __syncthreads();
  // thread -> (dimension group, head): its head is r again (256 % 16 == 0)
  const int h = h0 + r;
  for (int u = threadIdx.x; u < VR * 4; u += 256) {
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) v += *reinterpret_cast<const f32x4*>(reinterpret_cast<const float*>(lds[i]) + u * 4);
    if (h >= H) continue;
    const int d = (u >> 4) * 4;
    if (p.splits > 1) {
      const long pi = ((long)b * H + h) * p.splits + blockIdx.y;
      *reinterpret_cast<f32x4*>(p.part_o + pi * VR + d) = v;
      if (d == 0) {
        p.part_ml[2 * pi] = M;
        p.part_ml[2 * pi + 1] = L;
      }
    } else {
      const float inv = 1.f / L;
      st4(static_cast<bf16*>(p.out) + ((long)b * H + h) * VR + d,
          bf16x4{f2bf(v[0] * inv), f2bf(v[1] * inv), f2bf(v[2] * inv), f2bf(v[3] * inv)});
    }
  }
}

// The same for wide rows: the four waves share a 64-key tile.  Each scores 16 of its
// keys, the scores cross LDS, and each weighs a quarter of the value columns, so
// that no wave holds a whole output row and two blocks fit a CU.
template <int RANK, int VR>
__global__ __launch_bounds__(256, 2) void latent_decode_wide_kernel(LatentAttnParams p) {
  constexpr int KT = 64;
  constexpr int LDR = RANK + 8;
  constexpr int CPR = RANK / 8;
  constexpr int CH = KT * CPR / 256;
  constexpr int DW = VR / 64;  // 16-column tiles per wave
  constexpr int LDSC = KT + 4;
  __shared__ __attribute__((aligned(16))) bf16 cs[KT * LDR];
  __shared__ __attribute__((aligned(16))) float sc[16 * LDSC];  // [head][key]
  const int H = p.H, HG = (H + 15) / 16;
  const int item = xcd_remap(blockIdx.x, gridDim.x);  // a token's head groups on one XCD
  const int b = item / HG, h0 = (item % HG) * 16;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int pos = p.pos[b], lo = first_key(pos, p.window);
  const int* table = p.table + (long)p.seq_slots[b] * p.tw;
  const bf16* cache = static_cast<const bf16*>(p.cache);
  const int t0 = lo / KT, nt = pos / KT + 1 - t0;
  const int per = (nt + p.splits - 1) / p.splits;
  const int ta = t0 + blockIdx.y * per, tb = min(ta + per, t0 + nt);

  bf16x8 qf[RANK / 32];
  const bf16* q = static_cast<const bf16*>(p.q) + ((long)b * H + min(h0 + r, H - 1)) * RANK;
#pragma unroll
  for (int kk = 0; kk < RANK / 32; ++kk) qf[kk] = ld8(q + kk * 32 + g * 8);
  f32x4 o[DW];
#pragma unroll
  for (int di = 0; di < DW; ++di) o[di] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = NEG, lsum = 0.f;
  if (p.sink && blockIdx.y == 0) {  // a key that was seen first, without a value
    m = p.sink[min(h0 + r, H - 1)] * LOG2E;
    lsum = g == 0 ? 1.f : 0.f;
  }
  bf16x8 creg[CH];
  auto load_tile = [&](int kt) {  // a tile is a page
    const bf16* src = cache + (long)table[kt] * PAGE * RANK;
#pragma unroll
    for (int c = 0; c < CH; ++c) creg[c] = ld8(src + (threadIdx.x + c * 256) * 8);
  };
  if (ta < tb) load_tile(ta);
  for (int kt = ta; kt < tb; ++kt) {
    __syncthreads();  // the previous tile's readers are done
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int idx = threadIdx.x + c * 256;
      st8(cs + (idx / CPR) * LDR + (idx % CPR) * 8, creg[c]);
    }
    __syncthreads();
    if (kt + 1 < tb) load_tile(kt + 1);  // in flight under this tile's math

    f32x4 s = {0.f, 0.f, 0.f, 0.f}, s2 = s;  // two chains
    const bf16* row = cs + (w * 16 + r) * LDR + g * 8;
#pragma unroll
    for (int kk = 0; kk < RANK / 32; kk += 2) {
      s = mfma16(*reinterpret_cast<const bf16x8*>(row + kk * 32), qf[kk], s);
      s2 = mfma16(*reinterpret_cast<const bf16x8*>(row + kk * 32 + 32), qf[kk + 1], s2);
    }
    s += s2;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int key = kt * KT + w * 16 + 4 * g + i;
      s[i] = key <= pos && key >= lo ? s[i] * p.scale_log2 : NEG;
    }
    *reinterpret_cast<f32x4*>(sc + r * LDSC + w * 16 + 4 * g) = s;
    __syncthreads();
    // k-slot j of group g <-> key 32 kk + 4 g + j (j < 4), 32 kk + 16 + 4 g + (j - 4)
    f32x4 e[4];
    float tmax = NEG;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      e[c] = *reinterpret_cast<const f32x4*>(sc + r * LDSC + c * 16 + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; ++i) tmax = fmaxf(tmax, e[c][i]);
    }
    tmax = fmaxf(tmax, wave_xchg<16>(tmax));
    tmax = fmaxf(tmax, wave_xchg<32>(tmax));
    if (grew(tmax, m)) {
      const float mn = fmaxf(m, tmax);
      const float alpha = exp2f(m - mn);
      m = mn;
      lsum *= alpha;
#pragma unroll
      for (int di = 0; di < DW; ++di) o[di] *= alpha;
    }
#pragma unroll
    for (int c = 0; c < 4; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        // every tile of the range holds a visible key, so m is a real score
        e[c][i] = exp2f(e[c][i] - m);
        lsum += e[c][i];
      }
    bf16x8 ph[2], pl[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) split_p(e[2 * kk], e[2 * kk + 1], ph[kk], pl[kk]);
    const int r0 = 4 * g + (r >> 2);
#pragma unroll
    for (int di = 0; di < DW; ++di) {
      const int col = (w * DW + di) * 16 + 4 * (r & 3);
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const bf16x4 a = ds_read_tr(cs + (kk * 32 + r0) * LDR + col);
        const bf16x4 c = ds_read_tr(cs + (kk * 32 + r0 + 16) * LDR + col);
        const bf16x8 vf = {a[0], a[1], a[2], a[3], c[0], c[1], c[2], c[3]};
        o[di] = mfma16(vf, ph[kk], o[di]);
        o[di] = mfma16(vf, pl[kk], o[di]);
      }
    }
  }
  lsum += wave_xchg<16>(lsum);
  lsum += wave_xchg<32>(lsum);
  const int h = h0 + r;
  if (h >= H) return;
  // column tile 16 (w DW + di): rows 4 g + i of O^T are its columns, lane r the head
  const float inv = 1.f / lsum;
  const long pi = ((long)b * H + h) * p.splits + blockIdx.y;
#pragma unroll
  for (int di = 0; di < DW; ++di) {
    const int d = (w * DW + di) * 16 + 4 * g;
    if (p.splits > 1) *reinterpret_cast<f32x4*>(p.part_o + pi * VR + d) = o[di];
    else st4(static_cast<bf16*>(p.out) + ((long)b * H + h) * VR + d, pack4(o[di] * inv));
  }
  if (p.splits > 1 && w == 0 && g == 0) {
    p.part_ml[2 * pi] = m;
    p.part_ml[2 * pi + 1] = lsum;
  }
}

// Latent rows of every sequence's reach, packed: row cu_k[i] + j of the output is
// position k_lo[i] + j of sequence i (zeros before position 0).  One wave a row.
__global__ __launch_bounds__(256) void latent_gather_kernel(const bf16* __restrict__ cache,
                                                            const int* __restrict__ table, int tw,
                                                            const int* __restrict__ seq_slots,
                                                            const int* __restrict__ k_lo,
                                                            const int* __restrict__ cu_k, int B, int rows, int rank,
                                                            bf16* __restrict__ out) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= rows) return;
  int a = 0, b = B;  // sequence: last i with cu_k[i] <= row
  while (b - a > 1) {
    const int m = (a + b) >> 1;
    if (cu_k[m] <= row) a = m;
    else b = m;
  }
  const int pos = k_lo[a] + row - cu_k[a];
  const bf16* src = nullptr;
  if (pos >= 0) src = cache + ((long)table[(long)seq_slots[a] * tw + pos / PAGE] * PAGE + pos % PAGE) * rank;
  for (int c = lane_id() * 8; c < rank; c += 512) {
    bf16x8 v = {};
    if (src) v = ld8(src + c);
    st8(out + (long)row * rank + c, v);
  }
}

// Flash attention over expanded keys and values: 128 queries of one head per
// block (4 waves x 2 x 16), 64-key tiles of K [rows][H dim] and V [rows][H vdim]
// through LDS.  DP: dim (padded); vdim <= VP at run time.
template <int DP, int VP>
__global__ __launch_bounds__(256, 2) void latent_expanded_kernel(LatentExpandedParams p) {
  constexpr int KT = 64, QT = 2;
  constexpr int LDK = DP + 8, LDV = VP + 8;
  constexpr int CK = KT * (DP / 8) / 256, CV = KT * (VP / 8) / 256;
  __shared__ __attribute__((aligned(16))) bf16 ks[KT * LDK];
  __shared__ __attribute__((aligned(16))) bf16 vs[KT * LDV];
  const int L = xcd_remap(blockIdx.x, gridDim.x);  // tiles of a (sequence, head) side by side on one XCD
  const int h = L / p.n_tiles, x = L % p.n_tiles;
  const int seq = p.tiles[2 * x], off = p.tiles[2 * x + 1];
  const int cu = p.cu_q[seq], qlen = p.cu_q[seq + 1] - cu;
  const int base = p.k_lo[seq], cuk = p.cu_k[seq];
  const int st = p.q_start[seq] - base;  // positions relative to the first expanded row from here on
  const int neg = base < 0 ? -base : 0;  // rows before position 0
  const int lane = lane_id(), w = threadIdx.x >> 6;
  const int r = lane & 15, g = lane >> 4;
  const bf16* K = static_cast<const bf16*>(p.k) + (long)cuk * p.H * DP + (long)h * DP;
  const bf16* V = static_cast<const bf16*>(p.v) + (long)cuk * p.H * p.vdim + (long)h * p.vdim;

  int qi[QT], my_pos[QT], my_lo[QT];
  bf16x8 qf[QT][DP / 32];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    qi[t] = off + (w * QT + t) * 16 + r;
    const int qc = min(qi[t], qlen - 1);
    my_pos[t] = st + qc;
    my_lo[t] = max(neg, first_key(my_pos[t], p.window));
    const bf16* q = static_cast<const bf16*>(p.q) + (long)(cu + qc) * p.H * DP + (long)h * DP;
#pragma unroll
    for (int kk = 0; kk < DP / 32; ++kk) qf[t][kk] = ld8(q + kk * 32 + g * 8);
  }
  const int lo = max(neg, first_key(st + off, p.window));
  const int hi = st + min(off + 64 * QT, qlen);  // keys [lo, hi)
  const int kt0 = lo / KT, kt1 = (hi + KT - 1) / KT;

  f32x4 o[QT][VP / 16];
  float m[QT], lsum[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    m[t] = p.sink ? p.sink[h] * LOG2E : NEG;  // a key that was seen first, without a value
    lsum[t] = p.sink && g == 0 ? 1.f : 0.f;
#pragma unroll
    for (int di = 0; di < VP / 16; ++di) o[t][di] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  bf16x8 kreg[CK], vreg[CV];
  auto load_tile = [&](int kt) {
#pragma unroll
    for (int c = 0; c < CK; ++c) {
      const int idx = threadIdx.x + c * 256;
      kreg[c] = ld8(K + (long)min(kt * KT + idx / (DP / 8), hi - 1) * p.H * DP + (idx % (DP / 8)) * 8);
    }
#pragma unroll
    for (int c = 0; c < CV; ++c) {
      const int idx = threadIdx.x + c * 256, col = (idx % (VP / 8)) * 8;
      const bf16x8 z = {};
      const bf16x8 v =
          ld8(V + (long)min(kt * KT + idx / (VP / 8), hi - 1) * p.H * p.vdim + min(col, p.vdim - 8));
      vreg[c] = col < p.vdim ? v : z;
    }
  };
  load_tile(kt0);
  for (int kt = kt0; kt < kt1; ++kt) {
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
    if (kt + 1 < kt1) load_tile(kt + 1);

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
    // tiles every query of the block sees whole need no mask
    const bool whole = kt * KT >= my_lo[QT - 1] && (kt + 1) * KT - 1 <= my_pos[0];
    const bool all_whole = __all(whole);
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float tmax = NEG;
#pragma unroll
      for (int ni = 0; ni < KT / 16; ++ni)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = kt * KT + ni * 16 + 4 * g + i;
          float sv = s[t][ni][i] * p.scale_log2;
          if (!all_whole) sv = (key <= my_pos[t] && key >= my_lo[t]) ? sv : NEG;
          s[t][ni][i] = sv;
          tmax = fmaxf(tmax, sv);
        }
      tmax = fmaxf(tmax, wave_xchg<16>(tmax));
      tmax = fmaxf(tmax, wave_xchg<32>(tmax));
      if (grew(tmax, m[t])) {
        const float mn = fmaxf(m[t], tmax);
        const float alpha = exp2f(m[t] - mn);
        m[t] = mn;
        lsum[t] *= alpha;
#pragma unroll
        for (int di = 0; di < VP / 16; ++di) o[t][di] *= alpha;
      }
      // a query that has seen no key yet keeps weights of zero
      const float off2 = m[t] > 0.5f * NEG ? m[t] : 0.f;
      float ps = 0.f;
#pragma unroll
      for (int ni = 0; ni < KT / 16; ++ni)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = exp2f(s[t][ni][i] - off2);
          s[t][ni][i] = e;
          ps += e;
        }
      lsum[t] += ps;
    }
#pragma unroll
    for (int kk = 0; kk < KT / 32; ++kk) {
      bf16x8 ph[QT], pl[QT];
#pragma unroll
      for (int t = 0; t < QT; ++t) split_p(s[t][2 * kk], s[t][2 * kk + 1], ph[t], pl[t]);
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
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    float l = lsum[t];
    l += wave_xchg<16>(l);
    l += wave_xchg<32>(l);
    if (qi[t] >= qlen) continue;
    const float inv = 1.f / l;
    bf16* op = static_cast<bf16*>(p.out) + (long)(cu + qi[t]) * p.H * p.vdim + (long)h * p.vdim;
#pragma unroll
    for (int di = 0; di < VP / 16; ++di) {
      if (di * 16 >= p.vdim) continue;
      f32x4 v = o[t][di] * inv;
      if (p.gate) {
        const f32x4 z = *reinterpret_cast<const f32x4*>(p.gate + (cu + qi[t]) * p.ldg + (long)h * p.vdim + di * 16 + 4 * g);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] *= __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-LOG2E * z[i]));
      }
      st4(op + di * 16 + 4 * g, pack4(v));
    }
  }
}

__global__ __launch_bounds__(256) void latent_combine_kernel(const float* __restrict__ part_o,
                                                             const float* __restrict__ part_ml, bf16* out, int rank,
                                                             int splits) {
  const long pi = (long)blockIdx.x * splits;
  float M = NEG, L = 0.f;
  for (int s = 0; s < splits; ++s) M = fmaxf(M, part_ml[2 * (pi + s)]);
  for (int s = 0; s < splits; ++s) L += part_ml[2 * (pi + s) + 1] * exp2f(part_ml[2 * (pi + s)] - M);
  const float inv = 1.f / L;
  for (int d = threadIdx.x; d < rank; d += 256) {
    float v = 0.f;
    for (int s = 0; s < splits; ++s) v += part_o[(pi + s) * rank + d] * exp2f(part_ml[2 * (pi + s)] - M);
    out[(long)blockIdx.x * rank + d] = f2bf(v * inv);
  }
}

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void from_f(float* o, float v) { *o = v; }
__device__ __forceinline__ void from_f(bf16* o, float v) { *o = f2bf(v); }

// One (token, head) per block: 256 keys at a time, online softmax.  Dynamic
// LDS: the query row and one weight per key of the chunk.  seq_slots / pos are
// per token here.  OPT: output columns per thread.
template <typename T, int OPT>
__global__ __launch_bounds__(256) void latent_plain_kernel(LatentAttnParams p) {
  extern __shared__ float sh[];
  __shared__ float red[16];
  float* qs = sh;                 // [rank_pad]
  float* ps = sh + p.rank_pad;    // [256]
  const int t = blockIdx.x, h = blockIdx.y, R = p.rank_pad, tid = threadIdx.x;
  const int pos = p.pos[t], lo = first_key(pos, p.window);
  const int* table = p.table + (long)p.seq_slots[t] * p.tw;
  const T* cache = static_cast<const T*>(p.cache);
  const T* q = static_cast<const T*>(p.q) + ((long)t * p.H + h) * R;
  for (int i = tid; i < R; i += 256) qs[i] = to_f(q[i]) * p.scale_log2;
  float o[OPT] = {};
  float m = p.sink ? p.sink[h] * LOG2E : NEG, l = p.sink ? 1.f : 0.f;
  const int V = p.v_pad;
  __syncthreads();
  for (int k0 = lo; k0 <= pos; k0 += 256) {
    const int key = k0 + tid;
    float s = NEG;
    if (key <= pos) {
      const T* c = cache + ((long)table[key / PAGE] * PAGE + key % PAGE) * R;
      float a = 0.f;
      for (int i = 0; i < R; ++i) a = fmaf(qs[i], to_f(c[i]), a);
      s = a;
    }
    const float wm = wave_max(s);
    __syncthreads();
    if (lane_id() == 0) red[tid >> 6] = wm;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float e = key <= pos ? exp2f(s - mn) : 0.f;
    ps[tid] = e;
    const float alpha = exp2f(m - mn);
    m = mn;
    l = l * alpha + block_sum(e, red);  // its barriers also publish ps
    const int n = min(256, pos - k0 + 1);
#pragma unroll
    for (int j = 0; j < OPT; ++j) o[j] *= alpha;
    for (int i = 0; i < n; ++i) {
      const int kk = k0 + i;
      const T* c = cache + ((long)table[kk / PAGE] * PAGE + kk % PAGE) * R;
      const float pv = ps[i];
#pragma unroll
      for (int j = 0; j < OPT; ++j)
        if (tid + 256 * j < V) o[j] = fmaf(pv, to_f(c[tid + 256 * j]), o[j]);
    }
    __syncthreads();
  }
  T* out = static_cast<T*>(p.out) + ((long)t * p.H + h) * V;
  const float inv = 1.f / l;
#pragma unroll
  for (int j = 0; j < OPT; ++j)
    if (tid + 256 * j < V) from_f(out + tid + 256 * j, o[j] * inv);
}

}  // namespace
}  // namespace lsd

using namespace lsd;

// Query rows of one prefill tile for this rank, 0: no MFMA kernel.
extern "C" int lsd_latent_tile_rows(int rank) {
  if (rank % 64 || rank > 576 || rank == 0) return 0;
  return 128;
}

// Value columns the kernels weigh for cached rows of `rank_pad` columns, the first
// `rank` of which are values: as many, or 64 fewer.
extern "C" int lsd_latent_value_cols(int rank_pad, int rank) {
  return rank <= rank_pad - 64 ? rank_pad - 64 : rank_pad;
}

extern "C" hipError_t lsd_latent_prefill(const LatentAttnParams* p, hipStream_t st) {
  const dim3 grid(p->n_tiles);
  if (p->n_tiles == 0) return hipSuccess;
#define LSD_LP_V(R, V, QT, NW, KT) \
  hipLaunchKernelGGL((latent_prefill_kernel<R, V, QT, NW, KT>), grid, dim3(NW * 64), 0, st, *p)
#define LSD_LP(R, QT, NW, KT)                                                \
  case R:                                                                    \
    if (p->v_pad == R) LSD_LP_V(R, R, QT, NW, KT);                           \
    else LSD_LP_V(R, (R > 64 ? R - 64 : R), QT, NW, KT);                     \
    break;
  if (p->v_pad != p->rank_pad && (p->rank_pad == 64 || p->v_pad != p->rank_pad - 64)) return hipErrorInvalidValue;
  switch (p->rank_pad) {
    LSD_LP(64, 2, 4, 64)
    LSD_LP(128, 2, 4, 64)
    LSD_LP(192, 2, 4, 32)
    LSD_LP(256, 2, 4, 32)
    LSD_LP(320, 1, 8, 32)
    LSD_LP(384, 1, 8, 32)
    LSD_LP(448, 1, 8, 32)
    LSD_LP(512, 1, 8, 32)
    LSD_LP(576, 1, 8, 32)
    default: return hipErrorInvalidValue;
  }
#undef LSD_LP_V
#undef LSD_LP
  return hipGetLastError();
}

// rows from this width on are shared by the four waves of a block
constexpr int WIDE_DECODE = 320;
extern "C" hipError_t lsd_latent_decode(const LatentAttnParams* p, hipStream_t st) {
  if (p->B == 0) return hipSuccess;
  const dim3 grid(p->B * ((p->H + 15) / 16), p->splits);
#define LSD_LD_V(R, V)                                                                                    \
  do {                                                                                                     \
    if constexpr (R >= WIDE_DECODE) hipLaunchKernelGGL((latent_decode_wide_kernel<R, V>), grid, dim3(256), 0, st, *p); \
    else hipLaunchKernelGGL((latent_decode_kernel<R, V>), grid, dim3(256), 0, st, *p);                     \
  } while (0)
#define LSD_LD(R)                                         \
  case R:                                                 \
    if (p->v_pad == R) LSD_LD_V(R, R);                    \
    else LSD_LD_V(R, (R > 64 ? R - 64 : R));              \
    break;
  if (p->v_pad != p->rank_pad && (p->rank_pad == 64 || p->v_pad != p->rank_pad - 64)) return hipErrorInvalidValue;
  switch (p->rank_pad) {
    LSD_LD(64)
    LSD_LD(128)
    LSD_LD(192)
    LSD_LD(256)
    LSD_LD(320)
    LSD_LD(384)
    LSD_LD(448)
    LSD_LD(512)
    LSD_LD(576)
    default: return hipErrorInvalidValue;
  }
#undef LSD_LD_V
#undef LSD_LD
  if (p->splits > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3(p->B * p->H), dim3(256), 0, st, p->part_o, p->part_ml,
                       static_cast<bf16*>(p->out), p->v_pad, p->splits);
  return hipGetLastError();
}

// B query tokens with their own slot and position each
extern "C" hipError_t lsd_latent_plain(const LatentAttnParams* p, int f32, hipStream_t st) {
  if (p->B == 0) return hipSuccess;
  if (p->rank_pad > 4096) return hipErrorInvalidValue;
  const dim3 grid(p->B, p->H);
  const size_t lds = (p->rank_pad + 256) * sizeof(float);
#define LSD_PL(T, OPT) hipLaunchKernelGGL((latent_plain_kernel<T, OPT>), grid, dim3(256), lds, st, *p)
  const int opt = (p->v_pad + 255) / 256;
  if (f32) {
    if (opt <= 1) LSD_PL(float, 1);
    else if (opt <= 4) LSD_PL(float, 4);
    else LSD_PL(float, 16);
  } else {
    if (opt <= 4) LSD_PL(bf16, 4);
    else LSD_PL(bf16, 16);
  }
#undef LSD_PL
  return hipGetLastError();
}

extern "C" hipError_t lsd_latent_gather(const bf16* cache, const int* table, int tw, const int* seq_slots,
                                        const int* k_lo, const int* cu_k, int B, int rows, int rank, bf16* out,
                                        hipStream_t st) {
  if (rows == 0) return hipSuccess;
  hipLaunchKernelGGL(latent_gather_kernel, dim3((rows + 3) / 4), dim3(256), 0, st, cache, table, tw, seq_slots, k_lo,
                     cu_k, B, rows, rank, out);
  return hipGetLastError();
}

extern "C" hipError_t lsd_latent_expanded(const LatentExpandedParams* p, hipStream_t st) {
  if (p->n_tiles == 0) return hipSuccess;
  const dim3 grid(p->n_tiles * p->H);
#define LSD_LE(D, V) hipLaunchKernelGGL((latent_expanded_kernel<D, V>), grid, dim3(256), 0, st, *p)
  if (p->dim == 64 && p->vdim <= 64) LSD_LE(64, 64);
  else if (p->dim == 64 && p->vdim <= 128) LSD_LE(64, 128);
  else if (p->dim == 128 && p->vdim <= 64) LSD_LE(128, 64);
  else if (p->dim == 128 && p->vdim <= 128) LSD_LE(128, 128);
  else if (p->dim == 192 && p->vdim <= 64) LSD_LE(192, 64);
  else if (p->dim == 192 && p->vdim <= 128) LSD_LE(192, 128);
  else return hipErrorInvalidValue;
#undef LSD_LE
  return hipGetLastError();
}
