// Launch parameters of the recurrent mixers, of attention over a paged cache and
// of grouped norms, shared by csrc/kernels/recurrence.hip, attention_talk.hip,
// attention_paged.hip, norm_group.hip and csrc/mixer_bindings.cpp.  "Rows" are packed tokens; the element type T is
// bf16 or fp32 (models served in fp32).
#pragma once

namespace lsd {

// Short causal convolution of channels [0, channels), which are columns c0 ..
// of the in-projection rows y [rows][ldy] (T).  `gain` (the norm in front of
// the projection, one number) multiplies what the convolution sums.  The inputs
// of position p are kept at ring[slot][p % taps].
struct ConvParams {
  const void* y; long ldy; int c0;
  const float* w;      // [channels][taps], last column: the current token
  const float* bias;   // [channels] or null
  int taps, channels;
  void* ring;          // [slots][taps][channels]
  float gain;
};

// Sequences of a launch: slot, first position and packed rows of each.
struct SeqParams {
  int B; const int* slots; const int* start; const int* cu;
};

// Recurrence over a state S [rows D][V] per (sequence, head), fp32:
//   delta rule   S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q
//   Mamba-2      S <- a S + k (dt v)^T;                                o = S^T q + skip v
// with q / k / v conv channels (Mamba-2: C / B / x).
struct RecurParams {
  ConvParams c;
  SeqParams s;
  int heads, groups, D, V, Vp;         // Vp: V padded to 4 (row pitch of S)
  int q_ch, k_ch, v_ch;                // first conv channel of each
  int gate_col;                        // y column of beta's logits / dt, one per head
  float* S;                            // [slots][heads][D][Vp]
  const float* A;                      // [heads], -exp(A_log)
  const float* dt_bias;                // delta: [heads D], Mamba-2: [heads]
  // delta: second projections of the decay [heads D] and output gate [heads V]
  const void* low; long ldl; int gate_off;
  const float* norm; float eps;        // delta: output norm [V]
  const float* skip;                   // Mamba-2: [heads]
  float* raw; long ldr;                // delta: outputs before norm and gate [rows][heads V], or null
  void* out; long ldo; int out_cols;   // delta (raw null): normed and gated rows, zeros up to out_cols;
                                       // Mamba-2: y silu(z) rows
  int write_ring;                      // single-token portions: this kernel keeps the ring
};

// Recurrence whose forget gate f also decides what is written:
//   S <- diag(f) S + (1 - f) v^T;  o = S^T q;  out = rms(o) norm
// with q = silu, f = l + (1 - l) sigmoid(z + bias) of the in-projection's columns
// q [heads D] | z [heads D] | v [heads V].
struct ForgetParams {
  const void* y; long ldy;
  SeqParams s;
  int heads, D, V, Vp;                 // Vp: V padded to 4 (row pitch of S)
  float* S;                            // [slots][heads][D][Vp]
  const float* bias; const float* lower;  // [heads D]
  const float* norm; float eps;        // [V]
  float* raw; long ldr;                // outputs before the norm [rows][heads V], or null
  void* out; long ldo; int out_cols;   // zeros behind heads V
  // prompts in `segs` segments of each sequence, run together: what a segment
  // starts from (the first two, as it is; of later ones without the segments before
  // them) [seq][head][seg][D][Vp], and the summed log gates of a segment [..][D]
  int segs;
  float* part; float* decay;
};

// Output norms in a launch of their own.
struct MixOutParams {
  const float* raw; long ldr; int T;
  int heads, V;                        // delta, forget: per (row, head); low null: no gate
  const void* low; long ldl; int gate_off;
  int inner, groups;                   // Mamba-2: per (row, group), in place
  const float* norm; float eps, gain;
  void* out; long ldo; int out_cols;
};

// Attention over a paged cache, K [page][kv head][64][dim], V likewise with
// vdim.  Scores are capped, lessened by slope_h times the distance and mixed over
// the heads, then softmaxed -- or mixed behind the softmax (mix_weights).  A
// query at position i sees keys j <= i with i - j < window or j < keep.
struct TalkParams {
  const void* q;                       // [rows][H][dim]
  const void* k; const void* v;        // pools
  const int* table; int tw;            // [slots][pages of a sequence]
  const float* talk;                   // [H][H] or null
  const void* talk_frag;               // MFMA kernels: fp16 [HP][HP], zero padded (HP: H to 8 / 16 / 32)
  void* out; long ldo; int out_cols;   // [rows][H][vdim], zeros up to out_cols
  int H, G, dim, vdim, window, keep;   // window: keys per query (INT_MAX: all)
  float scale, cap;                    // cap 0: none
  const float* slopes;                 // [H] or null
  int mix_weights;
  const void* gate; long ldg;          // logits of a sigmoid gate per row and head, or null
  float* lse;                          // [rows][H] log2 of the softmax' sum (mix_weights, prompts)
  // one token alone: slot and position per row
  const int* slots; const int* pos; int T;
  // prompt tiles: (sequence, first query); sequences
  const int* tiles; int n_tiles;
  SeqParams s;
  // decode, splits > 1
  float* part_o; float* part_ml; int splits;
};

// Behind the in-projection y [rows][H dim | G dim | G vdim]: short convolution,
// unit RMS norms of q and k, rotation, values mixed with earlier ones, and the
// append to the cache.
struct RopeAppendParams {
  const void* y; long ldy; int T;
  float gain;
  const float* taps; int n_taps;       // [n_taps][channels of y], last: the current token; null: none
  void* ring;                          // [slots][n_taps][channels], inputs of position p at p % n_taps
  int write_ring;                      // one token per sequence: this kernel keeps the ring
  float eps; int dim_own;              // norms over a head's dim_own columns (the rest is padding); eps < 0: none
  const void* v_first; float lam;      // [rows][G vdim]: v <- (1 - lam) v + lam v_first, or null
  void* v_out;                         // [rows][G vdim]: this layer's values, or null
  const float* rope; int half;         // [positions][half][2] cos, sin; half 0: none
  void* q; void* k; void* v;
  const int* table; int tw; const int* tslot; const int* tpos;
  int H, G, dim, vdim;
};

// Norms of a row's `groups` equal parts of `size` columns (rows of H columns, the
// rest padding).  With slabs: x += norm(sum of slabs + bias) w_post, written
// back.  With out: out = norm(x) w_pre, padding zeroed.
struct GroupNormParams {
  float* x; int T, H, groups, size;
  float eps;
  const void* slab; int splits, slab_bf16;   // [splits][T][H] or null
  const void* bias; const void* w_post;      // [H], element type
  const void* w_pre; void* out;              // [H], [rows][H], element type
  const int* rows; int n_rows;               // rows of x that are normed into out (null: all)
};

// Elementwise norm tanh(alpha x) w + b; w, b [H] in the element type.
struct TanhNorm {
  float alpha;
  const void* w; const void* b;
};

// Rows of H columns.  With slabs: x += post(sum of slabs), written back.  With out:
// out = pre(x), or x in the element type (pre.w null).
struct TanhStepParams {
  float* x; int T, H;
  const void* slab; int splits, slab_bf16;   // [splits][T][H] or null
  TanhNorm post, pre;
  void* out;                                 // [rows][H] or null
  const int* rows; int n_rows;               // rows of x that go into out (null: all)
};

// In front of a mixer: x_new = x + rms(sum of slabs) w_side over `size` columns (no
// slabs: x stays), h = pre(x), out = h + (h of the token before - h) mix.  last
// [slots][H] holds the row before a portion.  Rows whose slot is the previous
// row's and whose position follows continue a portion.
struct ShiftNormParams {
  const float* x; float* x_new; int T, H, size;
  const void* slab; int splits, slab_bf16;
  const void* w_side; float eps;
  TanhNorm pre;
  const void* mix;
  float* last;
  const int* tslot; const int* tpos;
  void* out;
  const int* tail; int n_tail;               // rows whose h enters `last` (shift_tail)
};

}  // namespace lsd
