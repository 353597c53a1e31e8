// Grouped GEMMs: one launch over many [N][K] weight blocks.
//
//  * experts (GG_UP / GG_DOWN): a row tile belongs to one expert (table built
//    on the device by moe_group, moe.hip, so a captured graph follows the
//    routing); the token rows are gathered while they are staged to LDS, the
//    up projection's epilogue applies the clamped gated activation, the down
//    projection's epilogue the routing weight, writing choice k of token t to
//    slab[k][t] -- the same slabs the next norm folds into the residual for
//    split-K projections (norm.hip), so combining costs no launch.  A shared
//    expert of other sizes is one more group of the same launch.
//  * heads (GG_BATCH): per-head projections into and out of the latent space
//    of latent attention (attention_latent.hip).
//
// bf16: MFMA 16x16x32, tiles staged HBM -> LDS by 16-byte LDS-DMA into a ring
// of k-steps (the scheme of gemm_ring in gemm.hip), 4 waves as 2 x 2.
// fp32: plain VALU tiles with fused multiply-adds, for models served in fp32.
//
// A few tokens (single-stream decode): weight streaming instead of tiles, one
// wave per output column and (token, choice), no sorting by expert; the down
// projection sums a token's experts in the wave and adds into the residual.
#include "common.h"
#include "moe_params.h"

namespace lsd {

namespace gg {
constexpr int BK = 64;
typedef __attribute__((address_space(3))) void lds_void;
typedef __attribute__((address_space(1))) const void gbl_cvoid;
constexpr int vmcnt(int n) { return (n & 0xF) | ((n >> 4) << 14) | (0x7 << 4) | (0xF << 8); }

// Where one row tile's operands are.
struct Tile {
  const void* A; const void* W; void* out;
  long lda, ldw, ldo;
  int N, K, rows, row0;   // rows of the tile (<= TM) and its first row
  int n0;
  int group;              // expert / head whose weight block this is (shared expert: 0)
  float limit;
  bool routed, live;
};

// Logical workgroup -> (row tile, column tile): groups of `gr` row tiles walk the
// columns together, so a weight panel is re-read from L2 by its neighbours.  With
// few rows the group is the whole table: an XCD then takes a range of columns of
// every expert, and the unused end of the table costs all XCDs the same.
template <int MODE, int TM, int TN>
__device__ __forceinline__ Tile locate(const GgParams& p) {
  Tile t{};
  t.live = true;
  if constexpr (MODE == GG_UP || MODE == GG_DOWN) {
    // the shared expert's tiles first; shared and routed tiles are each spread over
    // all XCDs on their own (their K loops differ in length)
    const int tiles_s = (p.T + TM - 1) / TM, ntn_s = p.Ns > 0 ? (p.Ns + TN - 1) / TN : 0;
    const int grs = p.gr_s, shared = (tiles_s + grs - 1) / grs * grs * ntn_s;
    int bid = blockIdx.x;
    if (bid < shared) {
      bid = xcd_remap(bid, shared);
      const int gi = bid / (grs * ntn_s), rem = bid % (grs * ntn_s);
      const int tile = gi * grs + rem % grs;
      if (tile >= tiles_s) { t.live = false; return t; }
      t.A = p.As; t.lda = p.ldas; t.W = p.Ws; t.ldw = p.ldws; t.out = p.outs; t.ldo = p.ldos;
      t.N = p.Ns; t.K = p.Ks; t.row0 = tile * TM; t.rows = min(TM, p.T - tile * TM);
      t.n0 = (rem / grs) * TN;
      t.limit = p.limit_s;
      t.routed = false;
      return t;
    }
    const int gr = p.gr, ntn = (p.N + TN - 1) / TN;
    bid = xcd_remap(bid - shared, gridDim.x - shared);
    const int gi = bid / (gr * ntn), rem = bid % (gr * ntn);
    const int tile = gi * gr + rem % gr;
    if (tile >= p.n_tiles) { t.live = false; return t; }
    const int e = p.tiles[4 * tile], s0 = p.tiles[4 * tile + 1], n = p.tiles[4 * tile + 2];
    if (n == 0) { t.live = false; return t; }
    t.A = p.A; t.lda = p.lda; t.W = p.W; t.ldw = p.ldw; t.out = p.out; t.ldo = p.ldo;
    t.N = p.N; t.K = p.K; t.rows = n; t.row0 = s0;
    t.n0 = (rem / gr) * TN;
    t.group = e;
    t.limit = p.limit;
    t.routed = true;
    return t;
  } else {
    const int ntm = (p.M + TM - 1) / TM, ntn = (p.N + TN - 1) / TN;
    const int bid = xcd_remap(blockIdx.x, gridDim.x);
    const int g = bid / (ntm * ntn), rem = bid % (ntm * ntn);
    const int tm = rem % ntm;
    t.A = p.A; t.lda = p.lda; t.W = p.W; t.ldw = p.ldw; t.out = p.out; t.ldo = p.ldo;
    t.N = p.N; t.K = p.K; t.row0 = tm * TM; t.rows = min(TM, p.M - tm * TM);
    t.n0 = (rem / ntm) * TN;
    t.group = g;
    t.routed = true;
    return t;
  }
}

// Advance the operands to the tile's group (the element type is known here).
template <int MODE, typename T>
__device__ __forceinline__ void resolve(const GgParams& p, Tile& t) {
  const long g = t.group;
  if (t.routed) t.W = static_cast<const T*>(t.W) + g * p.w_gs;
  if constexpr (MODE == GG_BATCH) t.out = static_cast<T*>(t.out) + g * p.o_gs;
  if constexpr (MODE == GG_F32 || MODE == GG_ADD) t.out = static_cast<float*>(t.out) + g * p.o_gs;
  if constexpr (MODE != GG_UP && MODE != GG_DOWN) t.A = static_cast<const T*>(t.A) + g * p.a_gs;
}

// Source row of tile row i (clamped to a valid one).
template <int MODE>
__device__ __forceinline__ long a_row(const GgParams& p, const Tile& t, int i) {
  const int r = t.row0 + min(i, t.rows - 1);
  if constexpr (MODE == GG_UP) return t.routed ? p.perm[r] / p.top : r;
  return r;
}

// g = min(gate, limit), u = clamp(up, +-limit): g sigmoid(alpha g) (u + one).  SiLU
// gates have limit = infinity, alpha = 1 and one = 0.
__device__ __forceinline__ float glu_fast(float g, float u, float limit, float alpha, float one) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * alpha * g)) * (u + one);
}
__device__ __forceinline__ float glu_exact(float g, float u, float limit, float alpha, float one) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-alpha * g)) * (u + one);
}
__device__ __forceinline__ float sigmoid_fast(float z) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}
}  // namespace gg

template <int MODE, int TM, int TN, int SLOTS>
__global__ __launch_bounds__(256) void group_gemm_kernel(GgParams p) {
  using namespace gg;
  constexpr int MI = TM / 32, JT = TN / 32;  // 16 x 16 tiles per wave (2 x 2 waves)
  constexpr int A_BYTES = TM * BK * 2, SLOT_BYTES = (TM + TN) * BK * 2;
  constexpr int LPS = TM / 32 + TN / 32;     // LDS-DMA instructions per thread per k-step
  constexpr int D = SLOTS - 1;
  constexpr int CLD = TN + 4;
  constexpr int SMEM = SLOTS * SLOT_BYTES > TM * CLD * 4 ? SLOTS * SLOT_BYTES : TM * CLD * 4;
  __shared__ __attribute__((aligned(16))) char smem[SMEM];
  __shared__ int s_row[MODE == GG_DOWN ? TM : 1];   // GG_DOWN: slab row and weight of the tile's rows
  __shared__ float s_wt[MODE == GG_DOWN ? TM : 1];

  Tile t = locate<MODE, TM, TN>(p);
  if (!t.live) return;
  resolve<MODE, bf16>(p, t);
  const int lane = lane_id(), w = threadIdx.x >> 6;
  const int wm = w >> 1, wn = w & 1, r = lane & 15, g = lane >> 4;

  // per-lane source addresses of this wave's LDS-DMA rows (16-byte chunks
  // XOR-swizzled on the source side, as in gemm.hip stage_tile)
  const bf16* ap[TM / 32];
  const bf16* wp[TN / 32];
#pragma unroll
  for (int q = 0; q < TM / 32; ++q) {
    const int row = (w * (TM / 32) + q) * 8 + (lane >> 3);
    ap[q] = static_cast<const bf16*>(t.A) + a_row<MODE>(p, t, row) * t.lda + (((lane & 7) ^ ((row >> 1) & 7)) << 3);
  }
#pragma unroll
  for (int q = 0; q < TN / 32; ++q) {
    const int row = (w * (TN / 32) + q) * 8 + (lane >> 3);
    wp[q] = static_cast<const bf16*>(t.W) + (long)min(t.n0 + row, t.N - 1) * t.ldw +
            (((lane & 7) ^ ((row >> 1) & 7)) << 3);
  }
  auto issue = [&](int kt, int slot) {
    char* b = smem + slot * SLOT_BYTES;
#pragma unroll
    for (int q = 0; q < TM / 32; ++q)
      __builtin_amdgcn_global_load_lds((gbl_cvoid*)(ap[q] + kt * BK), (lds_void*)(b + (w * (TM / 32) + q) * 1024), 16,
                                       0, 0);
#pragma unroll
    for (int q = 0; q < TN / 32; ++q)
      __builtin_amdgcn_global_load_lds((gbl_cvoid*)(wp[q] + kt * BK),
                                       (lds_void*)(b + A_BYTES + (w * (TN / 32) + q) * 1024), 16, 0, 0);
  };
  auto frag = [&](const char* tile, int row, int chunk) {
    return *reinterpret_cast<const bf16x8*>(tile + row * 128 + ((chunk ^ ((row >> 1) & 7)) << 4));
  };

  if constexpr (MODE == GG_DOWN) {
    if (threadIdx.x < TM) {
      const int m = t.row0 + min((int)threadIdx.x, t.rows - 1);
      int row = m;
      float wt = 1.f;
      if (t.routed) {
        const int ent = p.perm[m];
        wt = p.wts[ent];
        row = (ent % p.top) * p.T + ent / p.top;  // < top * T, checked on the host to fit
      } else if (p.wts_s) {
        wt = p.wts_s[m];
      }
      s_row[threadIdx.x] = row;
      s_wt[threadIdx.x] = wt;
    }
  }
  f32x4 acc[MI][JT];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < JT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  // the routing loads above are done before the counted waits start
  __builtin_amdgcn_s_waitcnt(vmcnt(0));
  const int KT = t.K / BK;
#pragma unroll
  for (int d = 0; d < D; ++d)
    if (d < KT) issue(d, d);
  int slot = 0;
  for (int kt = 0; kt < KT; ++kt) {
    const int later = min(D - 1, KT - 1 - kt);  // k-steps after kt already issued
    if (later >= 2) __builtin_amdgcn_s_waitcnt(vmcnt(2 * LPS));
    else if (later == 1) __builtin_amdgcn_s_waitcnt(vmcnt(LPS));
    else __builtin_amdgcn_s_waitcnt(vmcnt(0));
    __builtin_amdgcn_s_barrier();
    if (kt + D < KT) issue(kt + D, slot == 0 ? SLOTS - 1 : slot - 1);
    const char* ta = smem + slot * SLOT_BYTES;
    const char* tw = ta + A_BYTES;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8 af[MI], wf[JT];
#pragma unroll
      for (int i = 0; i < MI; ++i) af[i] = frag(ta, wm * 16 * MI + i * 16 + r, kk * 4 + g);
#pragma unroll
      for (int j = 0; j < JT; ++j) wf[j] = frag(tw, wn * (TN / 2) + j * 16 + r, kk * 4 + g);
#pragma unroll
      for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < JT; ++j) acc[i][j] = mfma16(af[i], wf[j], acc[i][j]);
    }
    slot = slot == SLOTS - 1 ? 0 : slot + 1;
  }
  __syncthreads();

  // epilogue through LDS: row-contiguous 16-byte stores
  float* ct = reinterpret_cast<float*>(smem);
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < JT; ++j)
#pragma unroll
      for (int q = 0; q < 4; ++q)
        ct[(wm * 16 * MI + i * 16 + 4 * g + q) * CLD + wn * (TN / 2) + j * 16 + r] = acc[i][j][q];
  __syncthreads();
  constexpr int CPR = TN / 8;
  for (int c = threadIdx.x; c < TM * CPR; c += 256) {
    const int row = c / CPR, ch = c % CPR, n = t.n0 + ch * 8;
    if (row >= t.rows || n >= t.N) continue;
    const float* src = ct + row * CLD + ch * 8;
    const int m = t.row0 + row;
    if constexpr (MODE == GG_UP) {
      // gate and up rows interleaved in 16-row blocks: [gate16 | up16]
      if ((ch & 3) >= 2) continue;
      bf16x8 o;
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] = f2bf(glu_fast(src[e], src[16 + e], t.limit, p.alpha, p.up_one));
      st8(static_cast<bf16*>(t.out) + (long)m * t.ldo + (n >> 5) * 16 + (n & 15), o);
    } else if constexpr (MODE == GG_DOWN) {
      const long orow = s_row[row];
      const float wt = s_wt[row];
      if (p.slab_bf16) {
        bf16x8 o;
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = f2bf(src[e] * wt);
        st8(static_cast<bf16*>(t.out) + orow * t.ldo + n, o);
      } else {
        f32x4* o = reinterpret_cast<f32x4*>(static_cast<float*>(t.out) + orow * t.ldo + n);
        o[0] = f32x4{src[0] * wt, src[1] * wt, src[2] * wt, src[3] * wt};
        o[1] = f32x4{src[4] * wt, src[5] * wt, src[6] * wt, src[7] * wt};
      }
    } else {
      bf16x8 o;
      if (p.gate) {
        const float* gt = p.gate + m * p.ldg + t.group * p.o_gs + n;
        const f32x4 ga = *reinterpret_cast<const f32x4*>(gt), gb = *reinterpret_cast<const f32x4*>(gt + 4);
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = f2bf(src[e] * sigmoid_fast(e < 4 ? ga[e & 3] : gb[e & 3]));
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = f2bf(src[e]);
      }
      st8(static_cast<bf16*>(t.out) + (long)m * t.ldo + n, o);
    }
  }
}

// fp32: 64 x 64 tiles, 4 x 4 outputs per thread, 16-deep k-steps.
template <int MODE>
__global__ __launch_bounds__(256) void group_gemm_f32_kernel(GgParams p) {
  using namespace gg;
  constexpr int TM = 64, TN = 64, KS = 16;
  __shared__ float as[KS][TM + 4];
  __shared__ float ws[KS][TN + 4];
  Tile t = locate<MODE, TM, TN>(p);
  if (!t.live) return;
  resolve<MODE, float>(p, t);
  const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
  // loads: thread -> row tid / 4, four k at (tid % 4) * 4
  const int lr = threadIdx.x >> 2, lk = (threadIdx.x & 3) * 4;
  const float* ap = static_cast<const float*>(t.A) + a_row<MODE>(p, t, lr) * t.lda + lk;
  const float* wp = static_cast<const float*>(t.W) + (long)min(t.n0 + lr, t.N - 1) * t.ldw + lk;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < t.K; k0 += KS) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(ap + k0);
    const f32x4 w = *reinterpret_cast<const f32x4*>(wp + k0);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      as[lk + j][lr] = a[j];
      ws[lk + j][lr] = w[j];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      float av[4], wv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        av[i] = as[k][ty * 4 + i];
        // columns tx + 16 j: a gate column's up column (16 to the right in an
        // interleaved 32-row block) belongs to the same thread
        wv[i] = ws[k][tx + 16 * i];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(av[i], wv[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = ty * 4 + i;
    if (row >= t.rows) continue;
    const int m = t.row0 + row;
    if constexpr (MODE == GG_UP) {
#pragma unroll
      for (int j = 0; j < 4; j += 2) {
        const int n = t.n0 + tx + 16 * j;
        if (n < t.N)
          static_cast<float*>(t.out)[(long)m * t.ldo + (n >> 5) * 16 + (n & 15)] =
              glu_exact(acc[i][j], acc[i][j + 1], t.limit, p.alpha, p.up_one);
      }
      continue;
    }
    long orow = m;
    float wt = 1.f;
    if constexpr (MODE == GG_DOWN) {
      if (t.routed) {
        const int ent = p.perm[m];
        wt = p.wts[ent];
        orow = (long)(ent % p.top) * p.T + ent / p.top;
      } else if (p.wts_s) {
        wt = p.wts_s[m];
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = t.n0 + tx + 16 * j;
      if (n >= t.N) continue;
      float* o = static_cast<float*>(t.out) + orow * t.ldo + n;
      if constexpr (MODE == GG_DOWN) *o = acc[i][j] * wt;
      else if constexpr (MODE == GG_ADD) *o += acc[i][j];
      else if constexpr (MODE == GG_F32) {
        const float gt = p.gate ? 1.f / (1.f + expf(-p.gate[m * p.ldg + t.group * p.o_gs + n])) : 1.f;
        *o = (acc[i][j] + (p.bias ? p.bias[n] : 0.f)) * gt;
      }
      else *o = acc[i][j];
    }
  }
}

// ---------------------------------------------------------------------------
// A few tokens: every (token, choice) streams its expert's weight rows
// ---------------------------------------------------------------------------
// One wave computes C gated columns of one (token, expert): 2 C weight rows,
// all lanes on consecutive 16-byte chunks.  Blocks of the shared expert first.
template <int C>
__global__ __launch_bounds__(256) void moe_gemv_up_kernel(MoeGemvParams p) {
  const int lane = lane_id(), w = threadIdx.x >> 6;
  const int nb_s = (p.Fs + 4 * C - 1) / (4 * C), nb = (p.F + 4 * C - 1) / (4 * C);
  int bid = blockIdx.x;
  const bf16 *W, *A;
  bf16* out;
  float limit;
  int F, c0;
  if (bid < nb_s * p.T) {
    const int t = bid / nb_s;
    c0 = (bid % nb_s) * 4 * C;
    A = static_cast<const bf16*>(p.h) + (long)t * p.K;
    W = static_cast<const bf16*>(p.ws);
    out = static_cast<bf16*>(p.mids) + (long)t * p.Fs;
    F = p.Fs;
    limit = p.limit_s;
  } else {
    bid -= nb_s * p.T;
    const int ent = bid / nb;
    c0 = (bid % nb) * 4 * C;
    A = static_cast<const bf16*>(p.h) + (long)(ent / p.top) * p.K;
    W = static_cast<const bf16*>(p.w) + (long)p.ids[ent] * 2 * p.F * p.K;
    out = static_cast<bf16*>(p.mid) + (long)ent * p.F;
    F = p.F;
    limit = p.limit;
  }
  c0 += w * C;
  if (c0 >= F) return;  // wave-uniform, no barriers
  const bf16* wr[2 * C];
#pragma unroll
  for (int j = 0; j < C; ++j) {
    const int c = min(c0 + j, F - 1);
    wr[2 * j] = W + (long)((c >> 4) * 32 + (c & 15)) * p.K;
    wr[2 * j + 1] = wr[2 * j] + 16L * p.K;
  }
  float acc[2 * C] = {};
#pragma unroll 4
  for (int k = lane * 8; k < p.K; k += 512) {
    const bf16x8 a = ld8(A + k);
#pragma unroll
    for (int j = 0; j < 2 * C; ++j) acc[j] = dot8(a, ld8(wr[j] + k), acc[j]);
  }
#pragma unroll
  for (int j = 0; j < 2 * C; ++j) acc[j] = wave_sum(acc[j]);
#pragma unroll
  for (int j = 0; j < C; ++j)
    if (lane == j && c0 + j < F) out[c0 + j] = f2bf(gg::glu_fast(acc[2 * j], acc[2 * j + 1], limit, p.alpha, p.up_one));
}

// One wave: one column of one token's residual += all its experts.
__global__ __launch_bounds__(256) void moe_gemv_down_kernel(MoeGemvParams p) {
  const int lane = lane_id(), t = blockIdx.y;
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (n >= p.K) return;  // K: the residual's width here
  const int ck = (p.F + 511) / 512, cs = (p.Fs + 511) / 512;
  float* x = p.x + (long)t * p.K + n;
  const float x0 = p.add ? *x : 0.f;
  float acc = 0.f;
  const int items = p.top * ck;
#pragma unroll 8
  for (int i = 0; i < items; ++i) {
    const int k = i / ck, c = (i % ck) * 512 + lane * 8;
    const int ent = t * p.top + k, cc = min(c, p.F - 8);
    const bf16x8 a = ld8(static_cast<const bf16*>(p.mid) + (long)ent * p.F + cc);
    const bf16x8 v = ld8(static_cast<const bf16*>(p.w) + ((long)p.ids[ent] * p.K + n) * p.F + cc);
    const float d = dot8(a, v, 0.f) * p.wts[ent];
    acc += c < p.F ? d : 0.f;
  }
#pragma unroll 4
  for (int i = 0; i < cs; ++i) {
    const int c = i * 512 + lane * 8, cc = min(c, p.Fs - 8);
    const bf16x8 a = ld8(static_cast<const bf16*>(p.mids) + (long)t * p.Fs + cc);
    const bf16x8 v = ld8(static_cast<const bf16*>(p.ws) + (long)n * p.Fs + cc);
    const float d = dot8(a, v, 0.f) * (p.wts_s ? p.wts_s[t] : 1.f);
    acc += c < p.Fs ? d : 0.f;
  }
  acc = wave_sum(acc);
  if (lane == 0) *x = x0 + acc;
}

}  // namespace lsd

using namespace lsd;

static long gg_blocks(const GgParams& p, int mode, int tm, int tn) {
  if (mode == GG_UP || mode == GG_DOWN) {
    long b = (long)((p.n_tiles + p.gr - 1) / p.gr) * p.gr * ((p.N + tn - 1) / tn);
    if (p.Ns > 0) b += (long)(((p.T + tm - 1) / tm + p.gr_s - 1) / p.gr_s) * p.gr_s * ((p.Ns + tn - 1) / tn);
    return b;
  }
  return (long)((p.M + tm - 1) / tm) * ((p.N + tn - 1) / tn) * p.groups;
}

template <int MODE>
static hipError_t gg_launch(const GgParams& p, int tm, hipStream_t st) {
  const int tn = tm == 32 ? 64 : 128;
  const dim3 grid((unsigned)gg_blocks(p, MODE, tm, tn));
  if (grid.x == 0) return hipSuccess;
  switch (tm) {
    case 32: hipLaunchKernelGGL((group_gemm_kernel<MODE, 32, 64, 4>), grid, dim3(256), 0, st, p); break;
    case 64: hipLaunchKernelGGL((group_gemm_kernel<MODE, 64, 128, 3>), grid, dim3(256), 0, st, p); break;
    case 128: hipLaunchKernelGGL((group_gemm_kernel<MODE, 128, 128, 2>), grid, dim3(256), 0, st, p); break;
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

// tm: row-tile rows (32 / 64 / 128; the expert modes' table must use the same)
extern "C" hipError_t lsd_group_gemm(const GgParams* p, int mode, int tm, hipStream_t st) {
  switch (mode) {
    case GG_BATCH: return gg_launch<GG_BATCH>(*p, tm, st);
    case GG_UP: return gg_launch<GG_UP>(*p, tm, st);
    case GG_DOWN: return gg_launch<GG_DOWN>(*p, tm, st);
    default: return hipErrorInvalidValue;
  }
}

// fp32 kernels: 64-row tiles
extern "C" hipError_t lsd_group_gemm_f32(const GgParams* p, int mode, hipStream_t st) {
  const dim3 grid((unsigned)gg_blocks(*p, mode, 64, 64));
  if (grid.x == 0) return hipSuccess;
#define LSD_GG_F32(MODE) \
  case MODE: hipLaunchKernelGGL((group_gemm_f32_kernel<MODE>), grid, dim3(256), 0, st, *p); break;
  switch (mode) {
    LSD_GG_F32(GG_UP)
    LSD_GG_F32(GG_DOWN)
    LSD_GG_F32(GG_F32)
    LSD_GG_F32(GG_ADD)
    default: return hipErrorInvalidValue;
  }
#undef LSD_GG_F32
  return hipGetLastError();
}

// up: K input columns, F / Fs gated columns; down: K residual columns
extern "C" hipError_t lsd_moe_gemv_up(const MoeGemvParams* p, hipStream_t st) {
  constexpr int C = 2;
  const long nb = (long)((p->Fs + 4 * C - 1) / (4 * C)) * p->T + (long)((p->F + 4 * C - 1) / (4 * C)) * p->T * p->top;
  hipLaunchKernelGGL((moe_gemv_up_kernel<C>), dim3((unsigned)nb), dim3(256), 0, st, *p);
  return hipGetLastError();
}

extern "C" hipError_t lsd_moe_gemv_down(const MoeGemvParams* p, hipStream_t st) {
  hipLaunchKernelGGL(moe_gemv_down_kernel, dim3((p->K + 3) / 4, p->T), dim3(256), 0, st, *p);
  return hipGetLastError();
}
