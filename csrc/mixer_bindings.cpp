// PyTorch bindings of the recurrent mixers, of attention over a paged cache and
// of grouped norms (csrc/kernels/recurrence.hip, attention_talk.hip,
// attention_paged.hip, norm_group.hip).
//
// Every entry point checks dtypes, shapes, strides and alignment on the host
// before launching; launches go on the current stream and are graph-capturable.
// Element type: bf16 or fp32, that of the in-projection rows.
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#include <hip/hip_runtime.h>

#include <climits>

#include "kernels/gemm_params.h"
#include "kernels/mixer_params.h"

using lsd::ConvParams;
using lsd::ForgetParams;
using lsd::GroupNormParams;
using lsd::MixOutParams;
using lsd::RecurParams;
using lsd::RopeAppendParams;
using lsd::SeqParams;
using lsd::ShiftNormParams;
using lsd::TanhNorm;
using lsd::TanhStepParams;
using lsd::TalkParams;

extern "C" {
int lsd_recur_block(int D, int V);
hipError_t lsd_recur_seq(const RecurParams* p, int delta, int f32, hipStream_t st);
int lsd_chunk_ok(int delta, int D, int V, int groups, int heads);
hipError_t lsd_conv_silu(const ConvParams* c, const SeqParams* s, int T, lsd_bf16_t* out, long ldo, hipStream_t st);
hipError_t lsd_recur_chunk(const RecurParams* p, int delta, const lsd_bf16_t* x, long ldx, hipStream_t st);
hipError_t lsd_conv_tail(const ConvParams* c, const SeqParams* s, int f32, hipStream_t st);
hipError_t lsd_head_norm_gate(const MixOutParams* p, int f32, hipStream_t st);
hipError_t lsd_group_norm(const MixOutParams* p, int f32, hipStream_t st);
hipError_t lsd_loop_pack(float* x, const float* x0, const float* step, void* out, int T, int H, int f32, hipStream_t st);
hipError_t lsd_glu_f32(const float* y, float* out, int T, int F, long ldo, int glu, float s, hipStream_t st);
hipError_t lsd_rope_append(const RopeAppendParams* p, int f32, hipStream_t st);
long lsd_talk_plain_lds(const TalkParams* p);
hipError_t lsd_talk_plain(const TalkParams* p, int f32, hipStream_t st);
int lsd_talk_heads(int H, int G, int dim, int vdim, float cap);
int lsd_talk_tile(int hp);
hipError_t lsd_talk_prefill(const TalkParams* p, int hp, hipStream_t st);
hipError_t lsd_talk_decode(const TalkParams* p, int hp, hipStream_t st);
long lsd_append_lds(const RopeAppendParams* p);
int lsd_paged_ok(int dim, int vdim);
hipError_t lsd_paged_prefill(const TalkParams* p, int qt, int lse, hipStream_t st);
hipError_t lsd_mix_prefill(const TalkParams* p, int hp, hipStream_t st);
hipError_t lsd_paged_decode(const TalkParams* p, hipStream_t st);
int lsd_mix_decode_gc(int H, int G);
long lsd_mix_combine_lds(const TalkParams* p);
hipError_t lsd_mix_decode(const TalkParams* p, hipStream_t st);
int lsd_forget_ok(int D, int V);
hipError_t lsd_forget_seq(const ForgetParams* p, int vb, int f32, hipStream_t st);
hipError_t lsd_forget_chunk(const ForgetParams* p, hipStream_t st);
hipError_t lsd_tanh_step(const TanhStepParams* p, int f32, hipStream_t st);
hipError_t lsd_shift_norm(const ShiftNormParams* p, int f32, hipStream_t st);
hipError_t lsd_shift_tail(const ShiftNormParams* p, int f32, hipStream_t st);
hipError_t lsd_group_rows_norm(const GroupNormParams* p, int f32, hipStream_t st);
}

namespace {

constexpr int PAGE = 64;
constexpr long MAX_LDS = 160 * 1024;
using Opt = c10::optional<torch::Tensor>;
using torch::Tensor;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

void check_hip(hipError_t e, const char* what) { TORCH_CHECK(e == hipSuccess, what, ": ", hipGetErrorString(e)); }

bool is_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && (t.scalar_type() == torch::kBFloat16 || t.scalar_type() == torch::kFloat32), name,
              " must be a bf16 or fp32 GPU tensor");
  return t.scalar_type() == torch::kFloat32;
}

// contiguous fp32 with exactly n elements
const float* fptr(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kFloat32 && t.is_contiguous() && t.numel() == n, name,
              " must be a contiguous fp32 GPU tensor of ", n, " elements");
  return t.data_ptr<float>();
}

const int* iptr(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt32 && t.is_contiguous() && t.numel() >= n, name,
              " must be contiguous int32 on the GPU with >= ", n, " elements");
  return t.data_ptr<int>();
}

// rows [T, >= cols] with unit last stride, 16-byte aligned
void rows_of(const Tensor& t, c10::ScalarType dt, int64_t T, int64_t cols, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == dt && t.dim() == 2 && t.stride(1) == 1 && t.size(0) == T &&
                  t.size(1) >= cols && t.stride(0) % (16 / t.element_size()) == 0 &&
                  reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0,
              name, " must be [", T, ", >= ", cols, "] rows of 16-byte aligned ", dt);
}

SeqParams seqs(const Tensor& slots, const Tensor& start, const Tensor& cu) {
  SeqParams s{};
  s.B = slots.numel();
  s.slots = iptr(slots, s.B, "seq slots");
  s.start = iptr(start, s.B, "seq starts");
  s.cu = iptr(cu, s.B + 1, "row offsets");
  return s;
}

// [slots, taps, channels], like y
void* ring_of(const Tensor& y, const Tensor& ring, int64_t taps, int64_t channels) {
  TORCH_CHECK(ring.is_cuda() && ring.scalar_type() == y.scalar_type() && ring.is_contiguous() && ring.dim() == 3 &&
                  ring.size(1) == taps && ring.size(2) == channels, "ring must be [slots, taps, channels] like y");
  return ring.data_ptr();
}

// y [T, N]: conv channels are columns c0 ..; taps [channels, n], ring [slots, n, channels]
ConvParams conv(const Tensor& y, int64_t c0, const Tensor& w, const Opt& bias, const Tensor& ring, double gain) {
  is_f32(y, "y");
  TORCH_CHECK(w.dim() == 2 && w.size(1) >= 1, "taps must be [channels, n]");
  ConvParams c{};
  c.channels = w.size(0);
  c.taps = w.size(1);
  rows_of(y, y.scalar_type(), y.size(0), c0 + c.channels, "y");
  c.y = y.data_ptr(); c.ldy = y.stride(0); c.c0 = c0;
  c.w = fptr(w, (int64_t)c.channels * c.taps, "taps");
  if (bias.has_value()) c.bias = fptr(*bias, c.channels, "conv bias");
  c.ring = ring_of(y, ring, c.taps, c.channels);
  c.gain = (float)gain;
  return c;
}

template <typename P>
void state_of(P& p, const Tensor& state, int64_t heads, int64_t D, int64_t V) {
  p.heads = heads; p.D = D; p.V = V; p.Vp = (V + 3) / 4 * 4;
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == torch::kFloat32 && state.is_contiguous() && state.dim() == 4 &&
                  state.size(1) == heads && state.size(2) == D && state.size(3) == p.Vp,
              "state must be contiguous fp32 [slots, heads, ", D, ", ", p.Vp, "]");
  p.S = state.data_ptr<float>();
}

template <typename P>
void out_rows(P& p, const Tensor& out, const Tensor& y) {
  rows_of(out, y.scalar_type(), y.size(0), (int64_t)p.heads * p.V, "out");
  p.out = out.data_ptr(); p.ldo = out.stride(0); p.out_cols = out.size(1);
}

// Rows of SiLU(convolution) (bf16) for the chunked forms, which then run.
void run_chunks(const RecurParams& p, int delta, const Tensor& y) {
  const int64_t T = y.size(0), ld = (p.c.channels + 7) / 8 * 8;
  auto x = torch::empty({T, ld}, y.options());
  auto* xp = reinterpret_cast<lsd_bf16_t*>(x.data_ptr());
  check_hip(lsd_conv_silu(&p.c, &p.s, T, xp, ld, cur_stream()), "conv_silu");
  check_hip(lsd_recur_chunk(&p, delta, xp, ld, cur_stream()), "recur_chunk");
}

// y [T, N] rows of q | k | v conv channels from column c0 and beta's logits from
// gate_col; low [T, >= heads D at 0, heads V at gate_off].  Token by token.
void delta_seq(Tensor y, int64_t c0, int64_t gate_col, Tensor low, int64_t gate_off, Tensor slots, Tensor start,
               Tensor cu, int64_t heads, int64_t groups, int64_t D, int64_t V, Tensor taps, Tensor ring, Tensor state,
               Tensor A, Tensor dt_bias, Tensor norm, double gain, double eps, Tensor out, bool single, bool chunked) {
  const bool f32 = is_f32(y, "y");
  RecurParams p{};
  p.c = conv(y, c0, taps, c10::nullopt, ring, gain);
  p.s = seqs(slots, start, cu);
  TORCH_CHECK(groups >= 1 && heads % groups == 0 && D >= 1 && V >= 1, "delta_seq: heads / groups");
  TORCH_CHECK(p.c.channels == 2 * groups * D + heads * V && gate_col + heads <= y.size(1), "delta_seq: y columns");
  state_of(p, state, heads, D, V);
  p.groups = groups;
  p.q_ch = 0; p.k_ch = groups * D; p.v_ch = 2 * groups * D; p.gate_col = gate_col;
  rows_of(low, y.scalar_type(), y.size(0), std::max(heads * D, gate_off + heads * V), "low");
  p.low = low.data_ptr(); p.ldl = low.stride(0); p.gate_off = gate_off;
  p.A = fptr(A, heads, "A"); p.dt_bias = fptr(dt_bias, heads * D, "dt_bias"); p.norm = fptr(norm, V, "norm");
  p.eps = (float)eps;
  out_rows(p, out, y);
  p.write_ring = single;
  TORCH_CHECK(!single || p.s.B == y.size(0), "delta_seq: one row per sequence");
  if (chunked) {
    TORCH_CHECK(!f32 && !single && lsd_chunk_ok(1, D, V, groups, heads), "delta_seq: no chunked kernel");
    run_chunks(p, 1, y);
    check_hip(lsd_conv_tail(&p.c, &p.s, f32, cur_stream()), "conv_tail");
    return;
  }
  const int vb = lsd_recur_block(D, V);
  TORCH_CHECK(vb > 0, "delta_seq: no kernel for key dimension ", D);
  Tensor raw;
  if (p.Vp > vb) {
    raw = torch::empty({y.size(0), heads * V}, y.options().dtype(torch::kFloat32));
    p.raw = raw.data_ptr<float>(); p.ldr = heads * V;
  }
  check_hip(lsd_recur_seq(&p, 1, f32, cur_stream()), "delta_seq");
  if (p.raw) {
    MixOutParams o{};
    o.raw = p.raw; o.ldr = p.ldr; o.T = y.size(0); o.heads = heads; o.V = V;
    o.low = p.low; o.ldl = p.ldl; o.gate_off = gate_off; o.norm = p.norm; o.eps = p.eps; o.gain = p.c.gain;
    o.out = p.out; o.ldo = p.ldo; o.out_cols = p.out_cols;
    check_hip(lsd_head_norm_gate(&o, f32, cur_stream()), "head_norm_gate");
  }
  if (!single) check_hip(lsd_conv_tail(&p.c, &p.s, f32, cur_stream()), "conv_tail");
}

// y [T, N]: z | x | B | C | dt.  `chunked`: prompts of bf16 models
void ssm_seq(Tensor y, Tensor slots, Tensor start, Tensor cu, int64_t heads, int64_t groups, int64_t N, int64_t V,
             int64_t norm_groups, Tensor taps, Tensor bias, Tensor ring, Tensor state, Tensor A, Tensor dt_bias,
             Tensor skip, Tensor norm, double gain, double eps, Tensor out, bool single, bool chunked) {
  const bool f32 = is_f32(y, "y");
  const int64_t inner = heads * V;
  RecurParams p{};
  p.c = conv(y, inner, taps, bias, ring, gain);
  p.s = seqs(slots, start, cu);
  TORCH_CHECK(groups >= 1 && heads % groups == 0 && N >= 1 && V >= 1, "ssm_seq: heads / groups");
  TORCH_CHECK(p.c.channels == inner + 2 * groups * N, "ssm_seq: channels");
  p.gate_col = inner + p.c.channels;
  TORCH_CHECK(p.gate_col + heads <= y.size(1), "ssm_seq: y columns");
  state_of(p, state, heads, N, V);
  p.groups = groups;
  p.v_ch = 0; p.k_ch = inner; p.q_ch = inner + groups * N;
  p.A = fptr(A, heads, "A"); p.dt_bias = fptr(dt_bias, heads, "dt_bias"); p.skip = fptr(skip, heads, "D");
  out_rows(p, out, y);
  TORCH_CHECK(norm_groups >= 1 && inner % norm_groups == 0, "ssm_seq: norm groups");
  p.write_ring = single;
  TORCH_CHECK(!single || p.s.B == y.size(0), "ssm_seq: one row per sequence");
  if (chunked) {
    TORCH_CHECK(!f32 && !single && lsd_chunk_ok(0, N, V, groups, heads), "ssm_seq: no chunked kernel");
    run_chunks(p, 0, y);
  } else {
    TORCH_CHECK(lsd_recur_block(N, V) > 0, "ssm_seq: no kernel for state size ", N);
    check_hip(lsd_recur_seq(&p, 0, f32, cur_stream()), "ssm_seq");
  }
  MixOutParams o{};
  o.T = y.size(0); o.inner = inner; o.groups = norm_groups;
  o.norm = fptr(norm, inner, "norm"); o.eps = (float)eps;
  o.out = p.out; o.ldo = p.ldo; o.out_cols = p.out_cols;
  check_hip(lsd_group_norm(&o, f32, cur_stream()), "group_norm");
  if (!single) check_hip(lsd_conv_tail(&p.c, &p.s, f32, cur_stream()), "conv_tail");
}

// y [T, N]: q [heads D] | forget gate's logits [heads D] | v [heads V].  chunked:
// prompts of bf16 models, each sequence in `segs` segments that run together
void forget_seq(Tensor y, Tensor slots, Tensor start, Tensor cu, int64_t heads, int64_t D, int64_t V, Tensor bias,
                Tensor lower, Tensor norm, double eps, Tensor state, Tensor out, bool chunked, int64_t segs) {
  const bool f32 = is_f32(y, "y");
  TORCH_CHECK(heads >= 1 && D >= 1 && V >= 1, "forget_seq: sizes");
  ForgetParams p{};
  rows_of(y, y.scalar_type(), y.size(0), heads * (2 * D + V), "y");
  p.y = y.data_ptr(); p.ldy = y.stride(0);
  p.s = seqs(slots, start, cu);
  state_of(p, state, heads, D, V);
  p.bias = fptr(bias, heads * D, "bias"); p.lower = fptr(lower, heads * D, "lower"); p.norm = fptr(norm, V, "norm");
  p.eps = (float)eps;
  out_rows(p, out, y);
  if (chunked) {
    TORCH_CHECK(!f32 && lsd_forget_ok(D, V) && segs >= 1 && segs <= 64, "forget_seq: no chunked kernel");
    p.segs = segs;
    Tensor part, decay;
    if (segs > 1) {
      const int64_t n = p.s.B * heads * segs;
      part = torch::empty({n * D * p.Vp}, y.options().dtype(torch::kFloat32));
      decay = torch::empty({n * D}, y.options().dtype(torch::kFloat32));
      p.part = part.data_ptr<float>(); p.decay = decay.data_ptr<float>();
    }
    check_hip(lsd_forget_chunk(&p, cur_stream()), "forget_chunk");
    return;
  }
  const int vb = lsd_recur_block(D, V);
  TORCH_CHECK(vb > 0 && 2 * D * sizeof(float) <= 48 * 1024, "forget_seq: no kernel for dimension ", D);
  Tensor raw;
  if (p.Vp > vb) {
    raw = torch::empty({y.size(0), heads * V}, y.options().dtype(torch::kFloat32));
    p.raw = raw.data_ptr<float>(); p.ldr = heads * V;
  }
  check_hip(lsd_forget_seq(&p, vb, f32, cur_stream()), "forget_seq");
  if (p.raw) {
    MixOutParams o{};
    o.raw = p.raw; o.ldr = p.ldr; o.T = y.size(0); o.heads = heads; o.V = V; o.norm = p.norm; o.eps = p.eps;
    o.out = p.out; o.ldo = p.ldo; o.out_cols = p.out_cols;
    check_hip(lsd_head_norm_gate(&o, f32, cur_stream()), "head_norm_gate");
  }
}

// rows [x | x0] (fp32 or bf16) of a loop's entry; x <- step
Tensor loop_pack(Tensor x, Tensor x0, Tensor step, bool f32) {
  const int64_t T = x.size(0), H = x.size(1);
  fptr(x0, T * H, "x0");
  fptr(step, H, "step");
  auto out = torch::empty({T, 2 * H}, x.options().dtype(f32 ? torch::kFloat32 : torch::kBFloat16));
  check_hip(lsd_loop_pack(const_cast<float*>(fptr(x, T * H, "x")), x0.data_ptr<float>(), step.data_ptr<float>(),
                          out.data_ptr(), T, H, f32, cur_stream()), "loop_pack");
  return out;
}

// y fp32 [T, 2F] (gate / up in 16-row blocks) -> out [T, F]; glu 1 tanh-GELU, 2 clamped
void glu_f32(Tensor y, Tensor out, int64_t glu, double scale) {
  const int64_t T = y.size(0), F = y.size(1) / 2;
  fptr(y, T * F * 2, "y");
  TORCH_CHECK(F % 16 == 0 && (glu == 1 || glu == 2), "glu_f32: F % 16, GELU or clamped");
  rows_of(out, torch::kFloat32, T, F, "out");
  check_hip(lsd_glu_f32(y.data_ptr<float>(), out.data_ptr<float>(), T, F, out.stride(0), (int)glu, (float)scale,
                        cur_stream()), "glu_f32");
}

void need_pools(const Tensor& k, const Tensor& v, const Tensor& table, c10::ScalarType dt) {
  TORCH_CHECK(k.is_cuda() && k.scalar_type() == dt && v.scalar_type() == dt && k.dim() == 4 && v.dim() == 4 &&
                  k.is_contiguous() && v.is_contiguous() && k.size(2) == PAGE && v.size(2) == PAGE &&
                  k.size(0) == v.size(0) && k.size(1) == v.size(1), "pools must be [pages, kv heads, 64, dim]");
  TORCH_CHECK(table.is_cuda() && table.scalar_type() == torch::kInt32 && table.dim() == 2 && table.is_contiguous(),
              "table must be contiguous [slots, pages per sequence]");
}

// [T, G vdim] rows of values, like y
void* value_rows(const RopeAppendParams& p, const Tensor& t, const Tensor& y, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == y.scalar_type() && t.is_contiguous() && t.dim() == 2 && t.size(0) == p.T &&
                  t.size(1) == (int64_t)p.G * p.vdim && reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0,
              name, " must be contiguous [T, kv heads vdim] like y");
  return t.data_ptr();
}

// y [T, N]: q [heads dim] | k [G dim] | v [G vdim] -> q [T, heads dim]; k, v appended.
// taps [n, channels] and ring [slots, n, channels]: a short convolution of all three
// (write_ring: one row per sequence); eps >= 0: unit norms of q and k over dim_own
// columns; v_first: v <- (1 - lam) v + lam v_first; v_out: v as it was before that
Tensor rope_append(Tensor y, int64_t heads, Tensor k, Tensor v, Tensor table, Tensor tslot, Tensor tpos, Opt rope,
                   double gain, Opt taps, Opt ring, bool write_ring, double eps, int64_t dim_own, Opt v_first, double lam,
                   Opt v_out) {
  const bool f32 = is_f32(y, "y");
  need_pools(k, v, table, y.scalar_type());
  RopeAppendParams p{};
  p.T = y.size(0); p.H = heads; p.G = k.size(1); p.dim = k.size(3); p.vdim = v.size(3);
  const int64_t channels = (int64_t)(p.H + p.G) * p.dim + (int64_t)p.G * p.vdim;
  rows_of(y, y.scalar_type(), p.T, channels, "y");
  p.y = y.data_ptr(); p.ldy = y.stride(0); p.gain = (float)gain;
  if (rope.has_value()) {
    TORCH_CHECK(rope->dim() == 3 && rope->size(2) == 2 && 2 * rope->size(1) <= p.dim &&
                    rope->size(0) >= table.size(1) * (int64_t)PAGE, "rope must be [>= positions, half, 2]");
    p.rope = fptr(*rope, rope->numel(), "rope"); p.half = rope->size(1);
  }
  if (taps.has_value()) {
    TORCH_CHECK(ring.has_value() && taps->dim() == 2 && taps->size(0) >= 1 && taps->size(1) == channels,
                "taps must be [n, ", channels, "], with a ring");
    p.n_taps = taps->size(0);
    p.taps = fptr(*taps, p.n_taps * channels, "taps");
    p.ring = ring_of(y, *ring, p.n_taps, channels);
    p.write_ring = write_ring;
  }
  p.eps = (float)eps;
  p.dim_own = dim_own > 0 ? (int)dim_own : p.dim;
  TORCH_CHECK(p.dim_own <= p.dim, "dim_own");
  if (v_first.has_value()) p.v_first = value_rows(p, *v_first, y, "v_first");
  if (v_out.has_value()) p.v_out = value_rows(p, *v_out, y, "v_out");
  p.lam = (float)lam;
  TORCH_CHECK(lsd_append_lds(&p) <= MAX_LDS, "rope_append: ", channels, " channels do not fit the LDS");
  auto q = torch::empty({p.T, heads * p.dim}, y.options());
  p.q = q.data_ptr(); p.k = k.data_ptr(); p.v = v.data_ptr();
  p.table = table.data_ptr<int>(); p.tw = table.size(1);
  p.tslot = iptr(tslot, p.T, "tslot"); p.tpos = iptr(tpos, p.T, "tpos");
  check_hip(lsd_rope_append(&p, f32, cur_stream()), "rope_append");
  return q;
}

// inputs of a portion's last positions (the first columns of y) enter the convolution's ring
void conv_tail(Tensor y, Tensor ring, Tensor slots, Tensor start, Tensor cu) {
  const bool f32 = is_f32(y, "y");
  TORCH_CHECK(ring.dim() == 3, "ring must be [slots, taps, channels]");
  ConvParams c{};
  c.taps = ring.size(1); c.channels = ring.size(2);
  rows_of(y, y.scalar_type(), y.size(0), c.channels, "y");
  c.y = y.data_ptr(); c.ldy = y.stride(0);
  c.ring = ring_of(y, ring, c.taps, c.channels);
  const SeqParams s = seqs(slots, start, cu);
  check_hip(lsd_conv_tail(&c, &s, f32, cur_stream()), "conv_tail");
}

// what is beside the scores of a head: kept first tokens, distance slopes [H], gate
// logits [T, H] (a range of wider rows)
struct Beside { int64_t keep; Opt slopes, gate; };

TalkParams talk_base(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& table, const Opt& talk, int64_t window,
                     double scale, double cap, const Tensor& out, const Beside& b) {
  is_f32(q, "q");
  need_pools(k, v, table, q.scalar_type());
  TalkParams p{};
  p.G = k.size(1); p.dim = k.size(3); p.vdim = v.size(3); p.H = q.size(1) / p.dim;
  TORCH_CHECK(q.dim() == 2 && q.is_contiguous() && q.size(1) == (int64_t)p.H * p.dim && p.H % p.G == 0,
              "q must be contiguous [T, heads dim]");
  TORCH_CHECK(q.numel() < (1L << 31), "q: at most 2^31 elements");
  TORCH_CHECK(window >= 1, "window must be positive");
  p.T = q.size(0);
  p.q = q.data_ptr(); p.k = k.data_ptr(); p.v = v.data_ptr();
  p.table = table.data_ptr<int>(); p.tw = table.size(1);
  if (talk.has_value()) p.talk = fptr(*talk, (int64_t)p.H * p.H, "talk");
  p.window = (int)std::min<int64_t>(window, INT_MAX);
  p.scale = (float)scale; p.cap = (float)cap;
  rows_of(out, q.scalar_type(), p.T, (int64_t)p.H * p.vdim, "out");
  p.out = out.data_ptr(); p.ldo = out.stride(0); p.out_cols = out.size(1);
  TORCH_CHECK(b.keep >= 0 && b.keep <= INT_MAX - 64, "kept tokens");
  p.keep = (int)b.keep;
  if (b.slopes.has_value()) p.slopes = fptr(*b.slopes, p.H, "slopes");
  if (b.gate.has_value()) {
    TORCH_CHECK(b.gate->is_cuda() && b.gate->scalar_type() == q.scalar_type() && b.gate->dim() == 2 &&
                    b.gate->size(0) == p.T && b.gate->size(1) == p.H && (p.H == 1 || b.gate->stride(1) == 1),
                "gate must be [T, heads] like q");
    p.gate = b.gate->data_ptr(); p.ldg = b.gate->stride(0);
  }
  p.splits = 1;
  return p;
}

// every row is a query of its own: slots / pos [T]
void talk_plain(Tensor q, Tensor k, Tensor v, Tensor table, Tensor slots, Tensor pos, Opt talk, int64_t window,
                double scale, double cap, Tensor out, int64_t keep, Opt slopes, Opt gate, bool mix_weights) {
  TalkParams p = talk_base(q, k, v, table, talk, window, scale, cap, out, {keep, slopes, gate});
  p.mix_weights = mix_weights;
  p.slots = iptr(slots, p.T, "slots"); p.pos = iptr(pos, p.T, "pos");
  TORCH_CHECK(lsd_talk_plain_lds(&p) <= MAX_LDS, "talk_plain: ", p.H, " heads of ", p.dim, " / ", p.vdim,
              " do not fit the LDS");
  check_hip(lsd_talk_plain(&p, is_f32(q, "q"), cur_stream()), "talk_plain");
}

int frag_of(TalkParams& p, const Tensor& q, const Tensor& frag) {
  TORCH_CHECK(q.scalar_type() == torch::kBFloat16, "the MFMA kernels are bf16");
  TORCH_CHECK(frag.is_cuda() && frag.scalar_type() == torch::kFloat16 && frag.is_contiguous() && frag.dim() == 2 &&
                  frag.size(0) == frag.size(1), "talk must be a contiguous fp16 [HP, HP]");
  p.talk_frag = frag.data_ptr();
  const int hp = frag.size(0), need = lsd_talk_heads(p.H, p.G, p.dim, p.vdim, p.mix_weights ? -1.f : p.cap);
  TORCH_CHECK(need > 0 && hp >= need && (hp == 8 || hp == 16 || hp == 32), "no MFMA kernel for ", p.H, " heads of ", p.dim,
              " / ", p.vdim, " with talk padded to ", hp);
  return hp;
}

// fp32 outputs and (maximum, sum) of every key split
void partials(TalkParams& p, int64_t splits, const Tensor& q, Tensor& po, Tensor& pml) {
  TORCH_CHECK(splits >= 1 && splits <= 256, "splits");
  p.splits = splits;
  if (splits == 1) return;
  const int64_t n = (int64_t)p.T * p.H * splits;
  po = torch::empty({n * p.vdim}, q.options().dtype(torch::kFloat32));
  pml = torch::empty({n * 2}, q.options().dtype(torch::kFloat32));
  p.part_o = po.data_ptr<float>(); p.part_ml = pml.data_ptr<float>();
}

// packed ragged queries; tiles [n, 2] = (sequence, first query) of talk_tile(hp) queries
void talk_prefill(Tensor q, Tensor k, Tensor v, Tensor table, Tensor frag, Tensor tiles, Tensor slots, Tensor start,
                  Tensor cu, int64_t window, double scale, double cap, int64_t splits, Tensor out) {
  TalkParams p = talk_base(q, k, v, table, c10::nullopt, window, scale, cap, out, {0, c10::nullopt, c10::nullopt});
  const int hp = frag_of(p, q, frag);
  Tensor po, pml;
  partials(p, splits, q, po, pml);
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles must be [n, 2]");
  p.tiles = iptr(tiles, 0, "tiles"); p.n_tiles = tiles.size(0);
  p.s = seqs(slots, start, cu);
  check_hip(lsd_talk_prefill(&p, hp, cur_stream()), "talk_prefill");
}

// one query per row; slots / pos [T]; hp (talk's padding) 16 or 32, G <= hp / 4
void talk_decode(Tensor q, Tensor k, Tensor v, Tensor table, Tensor frag, Tensor slots, Tensor pos, int64_t window,
                 double scale, double cap, int64_t splits, Tensor out) {
  TalkParams p = talk_base(q, k, v, table, c10::nullopt, window, scale, cap, out, {0, c10::nullopt, c10::nullopt});
  const int hp = frag_of(p, q, frag);
  TORCH_CHECK(hp >= 16 && 4 * p.G <= hp, "talk_decode: ", p.G, " K / V heads need talk padded to ", 4 * p.G);
  p.slots = iptr(slots, p.T, "slots"); p.pos = iptr(pos, p.T, "pos");
  Tensor po, pml;
  partials(p, splits, q, po, pml);
  check_hip(lsd_talk_decode(&p, hp, cur_stream()), "talk_decode");
}

void need_paged(const TalkParams& p, const Tensor& q, const char* what) {
  TORCH_CHECK(q.scalar_type() == torch::kBFloat16 && lsd_paged_ok(p.dim, p.vdim), what, ": bf16 heads up to 128 columns, got ",
              p.dim, " / ", p.vdim);
}

// packed ragged queries; tiles [n, 2] = (sequence, first query) of 64 qt queries.
// lse (fp32 [T, heads]): log2 of the softmax sums only, no output
void paged_prefill(Tensor q, Tensor k, Tensor v, Tensor table, Tensor tiles, int64_t qt, Tensor slots, Tensor start,
                   Tensor cu, int64_t window, double scale, int64_t keep, Opt slopes, Opt gate, Tensor out, Opt lse) {
  TalkParams p = talk_base(q, k, v, table, c10::nullopt, window, scale, 0.0, out, {keep, slopes, gate});
  need_paged(p, q, "paged_prefill");
  if (lse.has_value()) p.lse = const_cast<float*>(fptr(*lse, (int64_t)p.T * p.H, "lse"));
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles must be [n, 2]");
  p.tiles = iptr(tiles, 0, "tiles"); p.n_tiles = tiles.size(0);
  p.s = seqs(slots, start, cu);
  check_hip(lsd_paged_prefill(&p, (int)qt, lse.has_value(), cur_stream()), "paged_prefill");
}

// one query per row; slots / pos [T]; at most 16 query heads per K / V head
void paged_decode(Tensor q, Tensor k, Tensor v, Tensor table, Tensor slots, Tensor pos, int64_t window, double scale,
                  int64_t keep, Opt slopes, Opt gate, int64_t splits, Tensor out) {
  TalkParams p = talk_base(q, k, v, table, c10::nullopt, window, scale, 0.0, out, {keep, slopes, gate});
  need_paged(p, q, "paged_decode");
  TORCH_CHECK(p.H / p.G <= 16, "paged_decode: at most 16 query heads per K / V head");
  p.slots = iptr(slots, p.T, "slots"); p.pos = iptr(pos, p.T, "pos");
  Tensor po, pml;
  partials(p, splits, q, po, pml);
  check_hip(lsd_paged_decode(&p, cur_stream()), "paged_decode");
}

// prompts with weights mixed over the heads: lse (fp32 [T, heads]) from paged_prefill,
// frag the mixing matrix in fp16, padded; tiles of mix_tile(hp) queries
void mix_prefill(Tensor q, Tensor k, Tensor v, Tensor table, Tensor frag, Tensor tiles, Tensor slots, Tensor start,
                 Tensor cu, int64_t window, double scale, int64_t keep, Opt slopes, Opt gate, Tensor lse, int64_t splits,
                 Tensor out) {
  TalkParams p = talk_base(q, k, v, table, c10::nullopt, window, scale, 0.0, out, {keep, slopes, gate});
  need_paged(p, q, "mix_prefill");
  p.mix_weights = 1;
  p.lse = const_cast<float*>(fptr(lse, (int64_t)p.T * p.H, "lse"));
  const int hp = frag_of(p, q, frag);
  Tensor po, pml;
  partials(p, splits, q, po, pml);
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles must be [n, 2]");
  p.tiles = iptr(tiles, 0, "tiles"); p.n_tiles = tiles.size(0);
  p.s = seqs(slots, start, cu);
  check_hip(lsd_mix_prefill(&p, hp, cur_stream()), "mix_prefill");
}

// the same with weights mixed over the heads by talk (fp32 [heads, heads])
void mix_decode(Tensor q, Tensor k, Tensor v, Tensor table, Tensor talk, Tensor slots, Tensor pos, int64_t window,
                double scale, int64_t keep, Opt slopes, Opt gate, int64_t splits, Tensor out) {
  TalkParams p = talk_base(q, k, v, table, talk, window, scale, 0.0, out, {keep, slopes, gate});
  need_paged(p, q, "mix_decode");
  TORCH_CHECK(lsd_mix_decode_gc(p.H, p.G) > 0, "mix_decode: no kernel for ", p.H, " heads on ", p.G);
  p.slots = iptr(slots, p.T, "slots"); p.pos = iptr(pos, p.T, "pos");
  TORCH_CHECK(splits >= 1 && splits <= 64, "splits");
  p.splits = splits;
  const int64_t n = (int64_t)p.T * p.H * splits;
  auto po = torch::empty({n * p.G * p.vdim}, q.options().dtype(torch::kFloat32));
  auto pml = torch::empty({n * 2}, q.options().dtype(torch::kFloat32));
  p.part_o = po.data_ptr<float>(); p.part_ml = pml.data_ptr<float>();
  TORCH_CHECK(lsd_mix_combine_lds(&p) <= 64 * 1024, "mix_decode: heads do not fit the LDS");
  check_hip(lsd_mix_decode(&p, cur_stream()), "mix_decode");
}

// x [T, H] fp32, groups parts over the first `width` columns.  slab [S, T, H]: x +=
// norm(sum + bias) w_post; w_pre: returns norm(x) w_pre (rows of x, all by default)
Opt group_norm(Tensor x, int64_t groups, int64_t width, double eps, Opt slab, Opt bias, Opt w_post, Opt w_pre, Opt rows,
               bool f32) {
  const auto dt = f32 ? torch::kFloat32 : torch::kBFloat16;
  GroupNormParams p{};
  TORCH_CHECK(x.dim() == 2, "x must be [T, H]");
  p.T = x.size(0); p.H = x.size(1);
  p.x = const_cast<float*>(fptr(x, (int64_t)p.T * p.H, "x"));
  TORCH_CHECK(groups >= 1 && width >= 1 && width <= p.H && width % groups == 0 && p.H % 4 == 0, "group_norm: ", width,
              " columns in ", groups, " parts");
  p.groups = groups; p.size = width / groups; p.eps = (float)eps;
  auto vec = [&](const Tensor& t, const char* name) -> const void* {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == dt && t.is_contiguous() && t.numel() == p.H, name, " must be [H]");
    return t.data_ptr();
  };
  if (slab.has_value()) {
    const bool sf = is_f32(*slab, "slab");
    TORCH_CHECK(slab->is_contiguous() && slab->dim() == 3 && slab->size(0) >= 1 && slab->size(1) == p.T &&
                    slab->size(2) == p.H && w_post.has_value() && !rows.has_value(), "slab must be [S, T, H], with w_post");
    p.slab = slab->data_ptr(); p.splits = slab->size(0); p.slab_bf16 = !sf;
    p.w_post = vec(*w_post, "w_post");
    if (bias.has_value()) p.bias = vec(*bias, "bias");
  }
  Opt out;
  if (rows.has_value()) {
    p.n_rows = rows->numel();
    p.rows = iptr(*rows, p.n_rows, "rows");
  }
  if (w_pre.has_value()) {
    p.w_pre = vec(*w_pre, "w_pre");
    out = torch::empty({p.rows ? p.n_rows : p.T, p.H}, x.options().dtype(dt));
    p.out = out->data_ptr();
  }
  check_hip(lsd_group_rows_norm(&p, f32, cur_stream()), "group_norm");
  return out;
}

// weight and bias [H] of an elementwise norm in the element type
TanhNorm tanh_norm(double alpha, const Tensor& w, const Tensor& b, int64_t H, c10::ScalarType dt) {
  for (const Tensor* t : {&w, &b})
    TORCH_CHECK(t->is_cuda() && t->scalar_type() == dt && t->is_contiguous() && t->numel() == H, "norm vectors must be [H]");
  return {(float)alpha, w.data_ptr(), b.data_ptr()};
}

// slabs [S, T, H] (bf16 or fp32)
template <typename P>
void slabs_of(P& p, const Tensor& slab) {
  const bool sf = is_f32(slab, "slab");
  TORCH_CHECK(slab.is_contiguous() && slab.dim() == 3 && slab.size(0) >= 1 && slab.size(1) == p.T && slab.size(2) == p.H,
              "slab must be [S, T, H]");
  p.slab = slab.data_ptr(); p.splits = slab.size(0); p.slab_bf16 = !sf;
}

// x [T, H] fp32.  slab, post: x += tanh(alpha sum) w + b; want_out: returns
// tanh(alpha x) w + b (pre), or x in the element type; rows of x (no slab), all by default
Opt tanh_step(Tensor x, Opt slab, double a_post, Opt w_post, Opt b_post, bool want_out, double a_pre, Opt w_pre, Opt b_pre,
              Opt rows, bool f32) {
  const auto dt = f32 ? torch::kFloat32 : torch::kBFloat16;
  TORCH_CHECK(x.dim() == 2 && x.size(1) % 4 == 0, "x must be [T, H], H % 4");
  TanhStepParams p{};
  p.T = x.size(0); p.H = x.size(1);
  p.x = const_cast<float*>(fptr(x, (int64_t)p.T * p.H, "x"));
  if (slab.has_value()) {
    TORCH_CHECK(w_post.has_value() && b_post.has_value() && !rows.has_value(), "slabs need a norm, and all rows");
    slabs_of(p, *slab);
    p.post = tanh_norm(a_post, *w_post, *b_post, p.H, dt);
  }
  if (rows.has_value()) {
    p.n_rows = rows->numel();
    p.rows = iptr(*rows, p.n_rows, "rows");
  }
  Opt out;
  if (want_out) {
    if (w_pre.has_value()) p.pre = tanh_norm(a_pre, *w_pre, *b_pre, p.H, dt);
    out = torch::empty({p.rows ? p.n_rows : p.T, p.H}, x.options().dtype(dt));
    p.out = out->data_ptr();
  }
  check_hip(lsd_tanh_step(&p, f32, cur_stream()), "tanh_step");
  return out;
}

// x [T, H] fp32 -> (residual, shifted norm rows).  slab, w_side: residual = x + rms(sum
// of slabs) w_side over `width` columns, else x itself; last [slots, H]
std::vector<Tensor> shift_norm(Tensor x, Opt slab, Opt w_side, int64_t width, double eps, double alpha, Tensor w, Tensor b,
                               Tensor mix, Tensor last, Tensor tslot, Tensor tpos, bool f32) {
  const auto dt = f32 ? torch::kFloat32 : torch::kBFloat16;
  TORCH_CHECK(x.dim() == 2 && x.size(1) % 4 == 0, "x must be [T, H], H % 4");
  ShiftNormParams p{};
  p.T = x.size(0); p.H = x.size(1); p.size = width; p.eps = (float)eps;
  p.x = fptr(x, (int64_t)p.T * p.H, "x");
  p.pre = tanh_norm(alpha, w, b, p.H, dt);
  p.mix = tanh_norm(0.0, mix, mix, p.H, dt).w;
  TORCH_CHECK(last.dim() == 2 && last.size(1) == p.H, "last must be [slots, H]");
  p.last = const_cast<float*>(fptr(last, last.numel(), "last"));
  p.tslot = iptr(tslot, p.T, "tslot"); p.tpos = iptr(tpos, p.T, "tpos");
  Tensor x_new = x;
  if (slab.has_value()) {
    TORCH_CHECK(w_side.has_value() && width >= 1 && width <= p.H, "slabs need a norm");
    slabs_of(p, *slab);
    p.w_side = tanh_norm(0.0, *w_side, *w_side, p.H, dt).w;
    x_new = torch::empty_like(x);
    p.x_new = x_new.data_ptr<float>();
  }
  auto out = torch::empty({p.T, p.H}, x.options().dtype(dt));
  p.out = out.data_ptr();
  check_hip(lsd_shift_norm(&p, f32, cur_stream()), "shift_norm");
  return {x_new, out};
}

// last[slot of row] = norm(x[row]) for `rows` of x
void shift_tail(Tensor x, double alpha, Tensor w, Tensor b, Tensor last, Tensor tslot, Tensor rows, bool f32) {
  ShiftNormParams p{};
  p.T = x.size(0); p.H = x.size(1);
  p.x = fptr(x, (int64_t)p.T * p.H, "x");
  p.pre = tanh_norm(alpha, w, b, p.H, f32 ? torch::kFloat32 : torch::kBFloat16);
  TORCH_CHECK(last.dim() == 2 && last.size(1) == p.H && p.H % 4 == 0, "last must be [slots, H]");
  p.last = const_cast<float*>(fptr(last, last.numel(), "last"));
  p.tslot = iptr(tslot, p.T, "tslot");
  p.n_tail = rows.numel();
  p.tail = iptr(rows, p.n_tail, "rows");
  check_hip(lsd_shift_tail(&p, f32, cur_stream()), "shift_tail");
}

}  // namespace

void lsd_register_mixers(pybind11::module& m) {
  m.def("chunk_ok", [](bool delta, int64_t D, int64_t V, int64_t groups, int64_t heads) {
    return lsd_chunk_ok(delta, (int)D, (int)V, (int)groups, (int)heads) != 0; });
  m.def("delta_seq", &delta_seq, py::arg("y"), py::arg("c0"), py::arg("gate_col"), py::arg("low"), py::arg("gate_off"),
        py::arg("slots"), py::arg("start"), py::arg("cu"), py::arg("heads"), py::arg("groups"), py::arg("dim"),
        py::arg("vdim"), py::arg("taps"), py::arg("ring"), py::arg("state"), py::arg("A"), py::arg("dt_bias"),
        py::arg("norm"), py::arg("gain"), py::arg("eps"), py::arg("out"), py::arg("single"), py::arg("chunked") = false);
  m.def("ssm_seq", &ssm_seq, py::arg("y"), py::arg("slots"), py::arg("start"), py::arg("cu"), py::arg("heads"),
        py::arg("groups"), py::arg("state_dim"), py::arg("vdim"), py::arg("norm_groups"), py::arg("taps"), py::arg("bias"),
        py::arg("ring"), py::arg("state"), py::arg("A"), py::arg("dt_bias"), py::arg("skip"), py::arg("norm"),
        py::arg("gain"), py::arg("eps"), py::arg("out"), py::arg("single"), py::arg("chunked") = false);
  m.def("forget_ok", [](int64_t D, int64_t V) { return lsd_forget_ok((int)D, (int)V) != 0; });
  m.def("forget_seq", &forget_seq, py::arg("y"), py::arg("slots"), py::arg("start"), py::arg("cu"), py::arg("heads"),
        py::arg("dim"), py::arg("vdim"), py::arg("bias"), py::arg("lower"), py::arg("norm"), py::arg("eps"),
        py::arg("state"), py::arg("out"), py::arg("chunked"), py::arg("segs"));
  m.def("tanh_step", &tanh_step, py::arg("x"), py::arg("slab"), py::arg("a_post"), py::arg("w_post"), py::arg("b_post"),
        py::arg("want_out"), py::arg("a_pre"), py::arg("w_pre"), py::arg("b_pre"), py::arg("rows"), py::arg("f32"));
  m.def("shift_norm", &shift_norm, py::arg("x"), py::arg("slab"), py::arg("w_side"), py::arg("width"), py::arg("eps"),
        py::arg("alpha"), py::arg("w"), py::arg("b"), py::arg("mix"), py::arg("last"), py::arg("tslot"), py::arg("tpos"),
        py::arg("f32"));
  m.def("shift_tail", &shift_tail, py::arg("x"), py::arg("alpha"), py::arg("w"), py::arg("b"), py::arg("last"),
        py::arg("tslot"), py::arg("rows"), py::arg("f32"));
  m.def("loop_pack", &loop_pack, py::arg("x"), py::arg("x0"), py::arg("step"), py::arg("f32"));
  m.def("glu_f32", &glu_f32, py::arg("y"), py::arg("out"), py::arg("glu"), py::arg("scale"));
  m.def("rope_append", &rope_append, py::arg("y"), py::arg("heads"), py::arg("k"), py::arg("v"), py::arg("table"),
        py::arg("tslot"), py::arg("tpos"), py::arg("rope"), py::arg("gain"), py::arg("taps") = py::none(),
        py::arg("ring") = py::none(), py::arg("write_ring") = false, py::arg("eps") = -1.0, py::arg("dim_own") = 0,
        py::arg("v_first") = py::none(), py::arg("lam") = 0.0, py::arg("v_out") = py::none());
  m.def("conv_tail", &conv_tail, py::arg("y"), py::arg("ring"), py::arg("slots"), py::arg("start"), py::arg("cu"));
  m.def("talk_heads", [](int64_t H, int64_t G, int64_t dim, int64_t vdim, double cap) {
    return lsd_talk_heads(H, G, dim, vdim, (float)cap); });
  m.def("talk_tile", [](int64_t hp) { return lsd_talk_tile((int)hp); });
  m.def("talk_prefill", &talk_prefill, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("frag"),
        py::arg("tiles"), py::arg("slots"), py::arg("start"), py::arg("cu"), py::arg("window"), py::arg("scale"),
        py::arg("cap"), py::arg("splits"), py::arg("out"));
  m.def("talk_decode", &talk_decode, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("frag"),
        py::arg("slots"), py::arg("pos"), py::arg("window"), py::arg("scale"), py::arg("cap"), py::arg("splits"),
        py::arg("out"));
  m.def("talk_plain", &talk_plain, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("slots"),
        py::arg("pos"), py::arg("talk"), py::arg("window"), py::arg("scale"), py::arg("cap"), py::arg("out"),
        py::arg("keep") = 0, py::arg("slopes") = py::none(), py::arg("gate") = py::none(), py::arg("mix_weights") = false);
  m.def("paged_ok", [](int64_t dim, int64_t vdim) { return lsd_paged_ok((int)dim, (int)vdim) != 0; });
  m.def("paged_prefill", &paged_prefill, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("tiles"),
        py::arg("qt"), py::arg("slots"), py::arg("start"), py::arg("cu"), py::arg("window"), py::arg("scale"),
        py::arg("keep"), py::arg("slopes"), py::arg("gate"), py::arg("out"), py::arg("lse") = py::none());
  m.def("paged_decode", &paged_decode, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("slots"),
        py::arg("pos"), py::arg("window"), py::arg("scale"), py::arg("keep"), py::arg("slopes"), py::arg("gate"),
        py::arg("splits"), py::arg("out"));
  m.def("mix_prefill", &mix_prefill, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("frag"),
        py::arg("tiles"), py::arg("slots"), py::arg("start"), py::arg("cu"), py::arg("window"), py::arg("scale"),
        py::arg("keep"), py::arg("slopes"), py::arg("gate"), py::arg("lse"), py::arg("splits"), py::arg("out"));
  m.def("mix_decode_ok", [](int64_t H, int64_t G) { return lsd_mix_decode_gc((int)H, (int)G) > 0; });
  m.def("mix_decode", &mix_decode, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("talk"),
        py::arg("slots"), py::arg("pos"), py::arg("window"), py::arg("scale"), py::arg("keep"), py::arg("slopes"),
        py::arg("gate"), py::arg("splits"), py::arg("out"));
  m.def("group_norm", &group_norm, py::arg("x"), py::arg("groups"), py::arg("width"), py::arg("eps"), py::arg("slab"),
        py::arg("bias"), py::arg("w_post"), py::arg("w_pre"), py::arg("rows"), py::arg("f32"));
}
