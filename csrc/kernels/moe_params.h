// Launch parameters of the grouped GEMMs and the expert router, shared by
// csrc/kernels/group_gemm.hip, csrc/kernels/moe.hip and csrc/latent_bindings.cpp.
#pragma once

namespace lsd {

// What a grouped GEMM's groups and rows are.
enum GgMode : int {
  GG_BATCH = 0,  // group g: out[m][o_gs g + n] = A[m][a_gs g + :] . W[w_gs g][n]      (T out)
  GG_UP = 1,     // expert e: mid[s] = act(A[token(perm[s])] . W_e gate, up rows)       (T out)
  GG_DOWN = 2,   // expert e: slab[k][token] = weight * (mid[s] . W_e)                  (slab out)
  GG_F32 = 3,    // GG_BATCH with fp32 output
  GG_ADD = 4,    // GG_BATCH into an fp32 residual: out += ...
};

struct GgParams {
  const void* A; long lda;
  const void* W; long ldw, w_gs;  // [group][N][K], K contiguous
  int N, K;                       // K % 64 == 0 and N % 16 == 0 (MFMA kernels)
  void* out; long ldo;
  int M, groups;                  // GG_BATCH rows / groups
  long a_gs, o_gs;
  const float* bias;              // GG_F32: [N] added to every row, or null (fp32 kernels)
  // experts: the row-tile table of moe_group (expert, first sorted row, rows,
  // 0), the sorted (token, choice) entries and their weights
  const int* tiles; int n_tiles;
  const int* perm; const float* wts; int top, T;
  float limit, alpha, up_one;     // g sigmoid(alpha g) (u + up_one), g and u clamped at limit
  int slab_bf16;                  // GG_DOWN output dtype (0: fp32)
  // shared expert: one more group over every token (Ns == 0: none)
  const void* As; long ldas;
  const void* Ws; long ldws;
  int Ns, Ks;
  void* outs; long ldos;
  float limit_s;
  const float* wts_s;             // GG_DOWN: its weight per token, or null (1)
  const float* gate; long ldg;    // GG_BATCH / GG_F32: out *= sigmoid(gate[m][o_gs g + n]), or null
  int gr, gr_s;                   // row tiles per group of the tile order (experts, shared)
};

// Experts of a few tokens (weight streaming): see moe_gemv_*_kernel.
struct MoeGemvParams {
  int T, top, K, F, Fs;      // Fs == 0: no shared expert
  const int* ids; const float* wts;
  const void* h;             // up: [T][K]
  const void* w;             // up [E][2F][K] interleaved, down [E][K][F]
  const void* ws;            // up [2Fs][K], down [K][Fs]
  void* mid; void* mids;     // [T top][F], [T][Fs]
  float limit, limit_s, alpha, up_one;
  const float* wts_s;        // down: weight of the shared expert per token, or null (1)
  float* x; int add;         // down: fp32 rows [T][K], added to or written
};

// A router's logits of one row and what becomes of them: the `top` experts with
// the largest corrected sigmoid scores and their normalised scores, or (no
// correction) with the largest logits and the softmax over these.
struct RouteParams {
  const float* z; long ldz;                         // logits [T][experts]
  int T, experts, top;
  const float* correction;                          // [experts] or null
  int* ids; float* wts;                             // [T][top]
  float* shared;                                    // [T] sigmoid of the column behind the logits, or null
};

// Narrow projections with what follows them: a w^T of rows a [T][K] (bf16), then the
// routing of the logits (r.experts > 0, all columns in one block), or
// out = gelu(.) * table[ids[t]].
struct RowsParams {
  const void* a; long lda;
  const void* w; long ldw;                          // [N][K]
  int T, N, K;                                      // K % 64 == 0, N % 16 == 0
  RouteParams r;                                    // z unused
  int splits; float* part; int* counters;           // router: K splits, [row tiles][splits][16][columns], tickets (zero)
  const int* ids; const void* table; int vocab;     // [vocab][N]
  void* out; long ldo;
};

// One token row behind a layer's input projection y (fp32): the latent columns
// are normed and appended to the paged cache with the turned key part behind them,
// the query columns narrowed and their last `rot` columns per head turned -- or
// normed, where they are a latent of their own -- and the experts chosen.
struct LatentPostParams {
  const float* y; long ldy; int T;
  void* q; int nq;                                  // null: queries stay in y
  const float* q_gain; int q_rank;                  // not null: q = norm of the first q_rank of nq columns
  int q_head, q_rot;                                // columns per head and the first turned one
  const float* rope; int half;                      // [positions][half][2] cos, sin; pairs (i, i + half); half 0: none
  void* cache; int c_off, rank, rank_pad;           // null cache: another layer's latent is used
  const float* gain; float eps;
  const int* table; int tw; const int* tslot; const int* tpos;
  int r_off;                                        // first router column (r.experts == 0: no router)
  RouteParams r;
};

// Attention over the paged latent cache, in the latent space: query row
// (t, head) of `rank_pad` columns, keys the cached rows, values their first
// `v_pad` columns.
struct LatentAttnParams {
  const void* q; void* out;                         // [T][H][rank_pad], [T][H][v_pad]
  const void* cache; const int* table; int tw;      // [pages][64][rank_pad], [slots][tw]
  const int* seq_slots; const int* pos;             // decode: [B] positions; prefill: q_start
  const int* cu_q; const int* tiles; int n_tiles;   // prefill tiles (sequence, first row)
  int B, H, rank_pad, v_pad, window;                // window: keys per query (INT_MAX: all)
  float scale_log2;
  const float* sink;                                // [H] a further score without a value, or null
  float* part_o; float* part_ml; int splits;        // decode, splits > 1
};

// Per-head attention over keys and values expanded from gathered latents: rows
// cu_k[i] .. of k / v are positions k_lo[i] .. of sequence i.
struct LatentExpandedParams {
  const void* q; void* out;                         // [T][H][dim], [T][H][vdim]
  const void* k; const void* v;                     // [rows][H][dim], [rows][H][vdim]
  const int* tiles; int n_tiles;                    // (sequence, first query) of 128 queries
  const int* cu_q; const int* q_start; const int* k_lo; const int* cu_k;
  int H, dim, vdim, window;
  float scale_log2;
  const float* sink;                                // [H] or null
  const float* gate; long ldg;                      // out *= sigmoid(gate[T][H vdim]), or null
};

}  // namespace lsd
