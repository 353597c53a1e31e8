// PyTorch bindings of the latent-attention, expert and grouped-GEMM kernels
// (csrc/kernels/attention_latent.hip, moe.hip, group_gemm.hip).
//
// As in bindings.cpp, every entry point checks dtypes, shapes, strides and
// alignment on the host before launching; launches go on the current stream
// and are graph-capturable.  Element type: bf16 (MFMA kernels) or fp32.
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#include <hip/hip_runtime.h>

#include <climits>

#include "kernels/gemm_params.h"
#include "kernels/moe_params.h"

using lsd::GgParams;
using lsd::LatentAttnParams;
using lsd::LatentPostParams;
using lsd::MoeGemvParams;
using lsd::RouteParams;
using lsd::RowsParams;

extern "C" {
hipError_t lsd_group_gemm(const GgParams* p, int mode, int tm, hipStream_t st);
hipError_t lsd_group_gemm_f32(const GgParams* p, int mode, hipStream_t st);
hipError_t lsd_moe_gemv_up(const MoeGemvParams* p, hipStream_t st);
hipError_t lsd_moe_gemv_down(const MoeGemvParams* p, hipStream_t st);
hipError_t lsd_latent_post(const LatentPostParams* p, int f32, hipStream_t st);
hipError_t lsd_route(const RouteParams* p, hipStream_t st);
hipError_t lsd_router(const RowsParams* p, hipStream_t st);
hipError_t lsd_side_gate(const RowsParams* p, hipStream_t st);
hipError_t lsd_side_mul(const void* g, const int* ids, const void* table, void* out, int T, int n, int vocab, int f32,
                        hipStream_t st);
int lsd_latent_value_cols(int rank_pad, int rank);
hipError_t lsd_moe_group(const int* ids, int n, int E, int tm, int* perm, int* tiles, int n_tiles, hipStream_t st);
hipError_t lsd_norm_f32(float* x, const float* slab, int splits, const float* w, float* out, int T, int H, float eps,
                        const int* rows, int nrows, int Hn, float woff, hipStream_t st);
hipError_t lsd_embed_f32(const int* ids, const float* wte, float* out, int T, int H, int vocab, float scale,
                         hipStream_t st);
int lsd_latent_tile_rows(int rank);
hipError_t lsd_latent_prefill(const LatentAttnParams* p, hipStream_t st);
hipError_t lsd_latent_decode(const LatentAttnParams* p, hipStream_t st);
hipError_t lsd_latent_gather(const lsd_bf16_t* cache, const int* table, int tw, const int* seq_slots, const int* k_lo,
                             const int* cu_k, int B, int rows, int rank, lsd_bf16_t* out, hipStream_t st);
hipError_t lsd_latent_expanded(const lsd::LatentExpandedParams* p, hipStream_t st);
hipError_t lsd_latent_plain(const LatentAttnParams* p, int f32, hipStream_t st);
}

namespace {

constexpr int PAGE = 64;
using Opt = c10::optional<torch::Tensor>;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

void check_hip(hipError_t e, const char* what) { TORCH_CHECK(e == hipSuccess, what, ": ", hipGetErrorString(e)); }

void need(const torch::Tensor& t, c10::ScalarType dt, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  TORCH_CHECK(t.scalar_type() == dt, name, " has dtype ", t.scalar_type(), ", expected ", dt);
  TORCH_CHECK(t.numel() == 0 || reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0 || t.element_size() == 4, name,
              " must be 16-byte aligned");
}

const int* iptr(const torch::Tensor& t, long n, const char* name) {
  need(t, torch::kInt32, name);
  TORCH_CHECK(t.is_contiguous() && t.numel() >= n, name, " must be contiguous int32 with >= ", n, " elements");
  return t.data_ptr<int>();
}

// rows of 16-byte aligned vectors
void need_rows(const torch::Tensor& t, const char* name) {
  const int v = 16 / t.element_size();
  TORCH_CHECK(t.dim() == 2 && t.stride(1) == 1 && t.stride(0) % v == 0 &&
                  reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0,
              name, " must be 2-D with unit last stride and 16-byte rows");
}

bool is_f32(const torch::Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && (t.scalar_type() == torch::kBFloat16 || t.scalar_type() == torch::kFloat32), name,
              " must be a bf16 or fp32 GPU tensor");
  return t.scalar_type() == torch::kFloat32;
}

int g_group_rows = 8;  // row tiles per group of the expert tile order above 2048 tokens

void run(GgParams& p, int mode, int tm, bool f32, const char* what) {
  const int tiles_s = std::max(1, (p.T + tm - 1) / tm);
  p.gr_s = std::min(tiles_s, g_group_rows);
  p.gr = p.T <= 2048 ? std::max(1, p.n_tiles) : g_group_rows;
  check_hip(f32 ? lsd_group_gemm_f32(&p, mode, cur_stream()) : lsd_group_gemm(&p, mode, tm, cur_stream()), what);
}

int tile_rows(int64_t tm, bool f32) {
  TORCH_CHECK(f32 ? tm == 64 : (tm == 32 || tm == 64 || tm == 128), "row tile must be 32, 64 or 128 (fp32: 64)");
  return (int)tm;
}

// fp32 gate logits [M, N] (rows of a wider tensor)
const float* gate_rows(const torch::Tensor& t, int64_t M, int64_t N, long& ld) {
  need(t, torch::kFloat32, "gate");
  TORCH_CHECK(t.dim() == 2 && t.size(0) == M && t.size(1) == N && t.stride(1) == 1 && (M <= 1 || t.stride(0) % 4 == 0) &&
                  reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0, "gate must be [", M, ", ", N, "] 16-byte rows");
  ld = t.stride(0);
  return t.data_ptr<float>();
}

// per-head scores of the softmax without values
const float* sink_of(const Opt& sink, int64_t H) {
  if (!sink.has_value()) return nullptr;
  need(*sink, torch::kFloat32, "sink");
  TORCH_CHECK(sink->is_contiguous() && sink->numel() == H, "sink must be [heads]");
  return sink->data_ptr<float>();
}

// Clamped gates have a limit; SiLU ones (limit 0) none.
float glu_limit(double limit) { return limit > 0 ? (float)limit : INFINITY; }

// Per-group projection: out[m][g N + n] = a[m][g K : g K + K] . w[g][n], times the
// sigmoid of gate [M, groups N].  a [M, groups K], w [groups, N, K]; bf16 -> bf16,
// fp32 -> fp32.
torch::Tensor batch_linear(torch::Tensor a, torch::Tensor w, int64_t tm, Opt gate) {
  const bool f32 = is_f32(a, "a");
  need(w, a.scalar_type(), "w");
  need_rows(a, "a");
  TORCH_CHECK(w.dim() == 3 && w.is_contiguous(), "w must be contiguous [groups, N, K]");
  const int64_t G = w.size(0), N = w.size(1), K = w.size(2);
  TORCH_CHECK(a.size(1) >= G * K && K % 64 == 0 && N % 16 == 0, "batch_linear: a [M, >= groups K], K % 64, N % 16");
  auto out = torch::empty({a.size(0), G * N}, a.options());
  GgParams p{};
  p.A = a.data_ptr(); p.lda = a.stride(0); p.a_gs = K;
  p.W = w.data_ptr(); p.ldw = K; p.w_gs = N * K;
  p.N = N; p.K = K; p.M = a.size(0); p.groups = G;
  p.out = out.data_ptr(); p.ldo = G * N; p.o_gs = N;
  if (gate.has_value()) p.gate = gate_rows(*gate, p.M, G * N, p.ldg);
  if (p.M) run(p, f32 ? lsd::GG_F32 : lsd::GG_BATCH, tile_rows(tm, f32), f32, "batch_linear");
  return out;
}

// fp32 linear: out = a w^T + bias (a [M, >= K], w [N, K]), or x += a w^T in place.
torch::Tensor linear_fp32(torch::Tensor a, torch::Tensor w, Opt x, Opt bias) {
  need(a, torch::kFloat32, "a");
  need(w, torch::kFloat32, "w");
  need_rows(a, "a");
  need_rows(w, "w");
  const int64_t N = w.size(0), K = w.size(1);
  TORCH_CHECK(a.size(1) == K && K % 16 == 0, "linear_fp32: K mismatch or K % 16 != 0");
  GgParams p{};
  p.A = a.data_ptr(); p.lda = a.stride(0);
  p.W = w.data_ptr(); p.ldw = w.stride(0);
  p.N = N; p.K = K; p.M = a.size(0); p.groups = 1;
  if (bias.has_value()) {
    need(*bias, torch::kFloat32, "bias");
    TORCH_CHECK(!x.has_value() && bias->is_contiguous() && bias->numel() == N, "bias must be [N], not into a residual");
    p.bias = bias->data_ptr<float>();
  }
  torch::Tensor out;
  if (x.has_value()) {
    need(*x, torch::kFloat32, "x");
    TORCH_CHECK(x->dim() == 2 && x->is_contiguous() && x->size(0) == p.M && x->size(1) == N, "x must be [M, N]");
    out = *x;
  } else {
    out = torch::empty({a.size(0), N}, a.options());
  }
  p.out = out.data_ptr(); p.ldo = N;
  if (p.M) run(p, x.has_value() ? lsd::GG_ADD : lsd::GG_F32, 64, true, "linear_fp32");
  return out;
}

// ids [T, top] -> (perm [T top], tiles [n, 4]) for row tiles of tm rows
std::vector<torch::Tensor> moe_group(torch::Tensor ids, int64_t experts, int64_t tm) {
  TORCH_CHECK(ids.dim() == 2, "ids must be [T, top]");
  const int64_t n = ids.numel();
  const int* ip = iptr(ids, n, "ids");
  TORCH_CHECK(experts >= 1 && experts <= 1024 && tm >= 1, "1 to 1024 experts");
  const int64_t nt = n / tm + std::min<int64_t>(experts, n);  // sum over experts of ceil(rows / tm)
  auto perm = torch::empty({n}, ids.options());
  auto tiles = torch::empty({std::max<int64_t>(nt, 1), 4}, ids.options());
  if (n)
    check_hip(lsd_moe_group(ip, (int)n, (int)experts, (int)tm, perm.data_ptr<int>(), tiles.data_ptr<int>(), (int)nt,
                            cur_stream()), "moe_group");
  return {perm, tiles};
}

void expert_weight(const torch::Tensor& w, c10::ScalarType dt, int64_t dims, const char* name) {
  need(w, dt, name);
  TORCH_CHECK(w.dim() == dims && w.is_contiguous(), name, " must be contiguous with ", dims, " dimensions");
  TORCH_CHECK(w.size(dims - 1) % 64 == 0, name, ": K must be a multiple of 64");
}

// Gated up projections of the routed experts (gathered rows of h) and of the
// shared expert (every row): -> (mid [T top, F], mid_shared [T, Fs]).
// w [E, 2F, K], ws [2Fs, K]: gate / up rows interleaved in 16-row blocks.
std::vector<torch::Tensor> moe_up(torch::Tensor h, torch::Tensor perm, torch::Tensor tiles, int64_t top,
                                  torch::Tensor w, double limit, double alpha, Opt ws, double limit_s, int64_t tm) {
  const bool f32 = is_f32(h, "h");
  need_rows(h, "h");
  expert_weight(w, h.scalar_type(), 3, "w");
  const int64_t T = h.size(0), K = h.size(1), n = T * top;
  TORCH_CHECK(w.size(2) == K && w.size(1) % 32 == 0, "moe_up: w must be [E, 2F, K], F % 16 == 0");
  GgParams p{};
  p.A = h.data_ptr(); p.lda = h.stride(0);
  p.W = w.data_ptr(); p.ldw = K; p.w_gs = w.size(1) * K;
  p.N = w.size(1); p.K = K; p.T = T; p.top = top;
  p.perm = iptr(perm, n, "perm");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 4, "tiles must be [n, 4]");
  p.tiles = iptr(tiles, 0, "tiles"); p.n_tiles = tiles.size(0);
  p.limit = glu_limit(limit); p.alpha = limit > 0 ? alpha : 1.f; p.up_one = limit > 0 ? 1.f : 0.f;
  auto mid = torch::empty({n, w.size(1) / 2}, h.options());
  p.out = mid.data_ptr(); p.ldo = mid.size(1);
  torch::Tensor mids;
  if (ws.has_value()) {
    expert_weight(*ws, h.scalar_type(), 2, "ws");
    TORCH_CHECK(ws->size(1) == K && ws->size(0) % 32 == 0, "moe_up: ws must be [2Fs, K], Fs % 16 == 0");
    mids = torch::empty({T, ws->size(0) / 2}, h.options());
    p.As = p.A; p.ldas = p.lda; p.Ws = ws->data_ptr(); p.ldws = K;
    p.Ns = ws->size(0); p.Ks = K; p.outs = mids.data_ptr(); p.ldos = mids.size(1); p.limit_s = glu_limit(limit_s);
    TORCH_CHECK((limit > 0) == (limit_s > 0), "moe_up: experts and shared expert have gates of one kind");
  } else {
    mids = torch::empty({0}, h.options());
  }
  if (T) run(p, lsd::GG_UP, tile_rows(tm, f32), f32, "moe_up");
  return {mid, mids};
}

const float* token_weights(const torch::Tensor& t, int64_t T) {
  need(t, torch::kFloat32, "wts_s");
  TORCH_CHECK(t.is_contiguous() && t.numel() == T, "wts_s must be [T]");
  return t.data_ptr<float>();
}

// Down projections: slab[k][t] = wts[t][k] * (expert k of token t), and
// slab[top][t] the shared expert's (times wts_s[t]).  slab [>= top (+ 1), T, N], bf16 or fp32.
void moe_down(torch::Tensor mid, Opt mids, torch::Tensor perm, torch::Tensor tiles, torch::Tensor wts,
              torch::Tensor w, Opt ws, torch::Tensor slab, int64_t tm, Opt wts_s) {
  const bool f32 = is_f32(mid, "mid");
  need_rows(mid, "mid");
  expert_weight(w, mid.scalar_type(), 3, "w");
  const int64_t T = wts.size(0), top = wts.size(1), n = T * top, N = w.size(1), K = w.size(2);
  TORCH_CHECK(mid.size(0) == n && mid.size(1) == K && N % 16 == 0, "moe_down: mid [T top, K], w [E, N, K]");
  TORCH_CHECK(n < (1L << 31), "moe_down: too many rows");
  const bool shared = ws.has_value();
  const bool sf32 = is_f32(slab, "slab");
  TORCH_CHECK(sf32 || !f32, "moe_down: fp32 models need fp32 slabs");
  TORCH_CHECK(slab.dim() == 3 && slab.is_contiguous() && slab.size(0) >= top + (shared ? 1 : 0) && slab.size(1) == T &&
                  slab.size(2) == N, "slab must be contiguous [>= top (+ 1), T, N]");
  need(wts, torch::kFloat32, "wts");
  TORCH_CHECK(wts.is_contiguous(), "wts must be contiguous");
  GgParams p{};
  p.A = mid.data_ptr(); p.lda = K;
  p.W = w.data_ptr(); p.ldw = K; p.w_gs = N * K;
  p.N = N; p.K = K; p.T = T; p.top = top;
  p.perm = iptr(perm, n, "perm");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 4, "tiles must be [n, 4]");
  p.tiles = iptr(tiles, 0, "tiles"); p.n_tiles = tiles.size(0);
  p.wts = wts.data_ptr<float>();
  p.slab_bf16 = sf32 ? 0 : 1;
  p.out = slab.data_ptr(); p.ldo = N;
  if (shared) {
    expert_weight(*ws, mid.scalar_type(), 2, "ws");
    TORCH_CHECK(mids.has_value(), "moe_down: the shared expert's rows are missing");
    need(*mids, mid.scalar_type(), "mids");
    need_rows(*mids, "mids");
    TORCH_CHECK(mids->size(0) == T && mids->size(1) == ws->size(1) && ws->size(0) == N, "moe_down: ws [N, Fs]");
    p.As = mids->data_ptr(); p.ldas = mids->size(1);
    p.Ws = ws->data_ptr(); p.ldws = ws->size(1); p.Ns = N; p.Ks = ws->size(1);
    p.outs = static_cast<char*>(slab.data_ptr()) + top * T * N * slab.element_size(); p.ldos = N;
    if (wts_s.has_value()) p.wts_s = token_weights(*wts_s, T);
  }
  if (T) run(p, lsd::GG_DOWN, tile_rows(tm, f32), f32, "moe_down");
}

// x += (add) or = the experts of a few tokens, weights streamed per (token, choice):
// h [T, K] bf16, w_up [E, 2F, K], w_down [E, K, F] (+ shared), x [T, K] fp32.
void moe_few(torch::Tensor h, torch::Tensor ids, torch::Tensor wts, torch::Tensor w_up, torch::Tensor w_down,
             double limit, double alpha, Opt ws_up, Opt ws_down, double limit_s, torch::Tensor x, Opt wts_s, bool add) {
  need(h, torch::kBFloat16, "h");
  TORCH_CHECK(h.dim() == 2 && h.is_contiguous(), "h must be contiguous [T, K]");
  const int64_t T = h.size(0), K = h.size(1), top = ids.size(1);
  TORCH_CHECK(ids.dim() == 2 && ids.size(0) == T && T >= 1 && T <= 64, "moe_few: 1 to 64 tokens");
  expert_weight(w_up, torch::kBFloat16, 3, "w_up");
  expert_weight(w_down, torch::kBFloat16, 3, "w_down");
  const int64_t E = w_up.size(0), F = w_down.size(2);
  TORCH_CHECK(w_up.size(1) == 2 * F && w_up.size(2) == K && w_down.size(0) == E && w_down.size(1) == K,
              "moe_few: w_up [E, 2F, K], w_down [E, K, F]");
  need(wts, torch::kFloat32, "wts");
  need(x, torch::kFloat32, "x");
  TORCH_CHECK(wts.is_contiguous() && wts.sizes() == ids.sizes() && x.is_contiguous() && x.dim() == 2 &&
                  x.size(0) == T && x.size(1) == K, "moe_few: wts [T, top], x [T, K]");
  MoeGemvParams p{};
  p.T = T; p.top = top; p.K = K; p.F = F;
  p.ids = iptr(ids, T * top, "ids"); p.wts = wts.data_ptr<float>();
  auto mid = torch::empty({T * top, F}, h.options());
  torch::Tensor mids;
  if (ws_up.has_value()) {
    TORCH_CHECK(ws_down.has_value(), "moe_few: shared down projection");
    expert_weight(*ws_up, torch::kBFloat16, 2, "ws_up");
    expert_weight(*ws_down, torch::kBFloat16, 2, "ws_down");
    p.Fs = ws_down->size(1);
    TORCH_CHECK(ws_up->size(0) == 2 * p.Fs && ws_up->size(1) == K && ws_down->size(0) == K, "moe_few: shared sizes");
    mids = torch::empty({T, p.Fs}, h.options());
    p.mids = mids.data_ptr();
    p.ws = ws_up->data_ptr();
  }
  p.h = h.data_ptr(); p.w = w_up.data_ptr(); p.mid = mid.data_ptr();
  p.limit = glu_limit(limit); p.limit_s = glu_limit(limit_s);
  p.alpha = limit > 0 ? alpha : 1.f; p.up_one = limit > 0 ? 1.f : 0.f;
  TORCH_CHECK(!ws_up.has_value() || (limit > 0) == (limit_s > 0), "moe_few: gates of one kind");
  if (wts_s.has_value()) p.wts_s = token_weights(*wts_s, T);
  p.add = add;
  check_hip(lsd_moe_gemv_up(&p, cur_stream()), "moe_few up");
  p.w = w_down.data_ptr();
  if (ws_down.has_value()) p.ws = ws_down->data_ptr();
  p.x = x.data_ptr<float>();
  check_hip(lsd_moe_gemv_down(&p, cur_stream()), "moe_few down");
}

void need_cache(const torch::Tensor& cache, const torch::Tensor& table, c10::ScalarType dt) {
  need(cache, dt, "cache");
  TORCH_CHECK(cache.dim() == 3 && cache.is_contiguous() && cache.size(1) == PAGE, "cache must be [pages, 64, rank]");
  need(table, torch::kInt32, "table");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous(), "table must be contiguous [slots, pages per slot]");
}

// See LatentPostParams: -> (q or empty, expert ids, expert weights).  c_off: first
// latent column (-1: behind the queries); rope [positions, half, 2] turns columns
// q_rot .. of every q_head query columns and those behind the latent's rank; q_gain
// [<= nq]: the first columns are normed into q
std::vector<torch::Tensor> latent_post(torch::Tensor y, int64_t nq, bool want_q, bool f32, Opt cache, int64_t rank,
                                       Opt gain, double eps, Opt table, Opt tslot, Opt tpos, Opt correction,
                                       int64_t top, int64_t c_off, Opt rope, int64_t q_head, int64_t q_rot, Opt q_gain) {
  need(y, torch::kFloat32, "y");
  need_rows(y, "y");
  const int64_t T = y.size(0);
  const auto dt = f32 ? torch::kFloat32 : torch::kBFloat16;
  LatentPostParams p{};
  p.y = y.data_ptr<float>(); p.ldy = y.stride(0); p.T = T; p.nq = nq; p.eps = eps;
  int64_t off = c_off >= 0 ? c_off : nq;
  TORCH_CHECK(nq <= y.size(1) && off >= nq, "latent_post: queries come first");
  if (rope.has_value()) {
    need(*rope, torch::kFloat32, "rope");
    TORCH_CHECK(rope->dim() == 3 && rope->size(2) == 2 && rope->is_contiguous() && tpos.has_value(), "rope [positions, half, 2]");
    TORCH_CHECK(!table.has_value() || rope->size(0) >= table->size(1) * (int64_t)PAGE, "rope: too few positions");
    p.rope = rope->data_ptr<float>(); p.half = rope->size(1);
    p.tpos = iptr(*tpos, T, "tpos");
    if (want_q && !q_gain.has_value())
      TORCH_CHECK(q_head >= 4 && q_head % 4 == 0 && nq % q_head == 0 && q_rot >= 0 && q_rot + 2 * p.half <= q_head,
                  "latent_post: turned columns of a head");
    p.q_head = q_head; p.q_rot = q_rot;
  }
  if (q_gain.has_value()) {
    need(*q_gain, torch::kFloat32, "q_gain");
    TORCH_CHECK(want_q && q_gain->is_contiguous() && q_gain->numel() >= 1 && q_gain->numel() <= nq, "q_gain [<= nq]");
    p.q_gain = q_gain->data_ptr<float>(); p.q_rank = q_gain->numel();
  }
  torch::Tensor q = torch::empty({want_q ? T : 0, nq}, y.options().dtype(dt));
  TORCH_CHECK(nq % 4 == 0, "query columns must be a multiple of 4");
  if (want_q) p.q = q.data_ptr();
  if (cache.has_value()) {
    TORCH_CHECK(table.has_value() && tslot.has_value() && tpos.has_value() && gain.has_value(), "latent_post: cache");
    need_cache(*cache, *table, dt);
    need(*gain, torch::kFloat32, "gain");
    TORCH_CHECK(gain->is_contiguous() && gain->numel() == rank && rank >= 1 && rank + 2 * p.half <= cache->size(2),
                "gain [rank], and room for the turned part");
    p.cache = cache->data_ptr(); p.c_off = off; p.rank = rank; p.rank_pad = cache->size(2);
    p.gain = gain->data_ptr<float>();
    p.table = table->data_ptr<int>(); p.tw = table->size(1);
    p.tslot = iptr(*tslot, T, "tslot"); p.tpos = iptr(*tpos, T, "tpos");
    off += rank + 2 * p.half;
  }
  const int64_t E = correction.has_value() ? correction->numel() : 0;
  auto ids = torch::empty({T, E ? top : 0}, y.options().dtype(torch::kInt32));
  auto wts = torch::empty({T, E ? top : 0}, y.options());
  if (E) {
    need(*correction, torch::kFloat32, "correction");
    TORCH_CHECK(correction->is_contiguous() && top >= 1 && top <= E && top <= 128 && E <= 1024, "router sizes");
    p.r_off = off; p.r.experts = E; p.r.top = top; p.r.correction = correction->data_ptr<float>();
    p.r.ids = ids.data_ptr<int>(); p.r.wts = wts.data_ptr<float>();
    off += E;
  }
  TORCH_CHECK(off <= y.size(1), "latent_post: y has ", y.size(1), " columns, needs ", off);
  check_hip(lsd_latent_post(&p, f32 ? 1 : 0, cur_stream()), "latent_post");
  return {q, ids, wts};
}

// z [T, >= experts (+ 1 with a shared gate)] fp32 logits -> (ids [T, top], weights
// [T, top], [T] weights of the shared expert or empty): softmax over the chosen
std::vector<torch::Tensor> route_softmax(torch::Tensor z, int64_t experts, int64_t top, bool shared) {
  need(z, torch::kFloat32, "z");
  const int64_t T = z.size(0);
  TORCH_CHECK(z.dim() == 2 && z.stride(1) == 1 && z.size(1) >= experts + (shared ? 1 : 0), "z [T, experts (+ 1)]");
  TORCH_CHECK(top >= 1 && top <= experts && top <= 128 && experts <= 1024, "router sizes");
  auto ids = torch::empty({T, top}, z.options().dtype(torch::kInt32));
  auto wts = torch::empty({T, top}, z.options());
  auto sh = torch::empty({shared ? T : 0}, z.options());
  RouteParams p{};
  p.z = z.data_ptr<float>(); p.ldz = z.stride(0); p.T = T; p.experts = experts; p.top = top;
  p.ids = ids.data_ptr<int>(); p.wts = wts.data_ptr<float>();
  if (shared) p.shared = sh.data_ptr<float>();
  check_hip(lsd_route(&p, cur_stream()), "route");
  return {ids, wts, sh};
}

// rows a [T, K], w [N, K] of a narrow projection (bf16)
RowsParams rows_of(const torch::Tensor& a, const torch::Tensor& w) {
  need(a, torch::kBFloat16, "a");
  need(w, torch::kBFloat16, "w");
  need_rows(a, "a");
  need_rows(w, "w");
  RowsParams p{};
  p.a = a.data_ptr(); p.lda = a.stride(0); p.w = w.data_ptr(); p.ldw = w.stride(0);
  p.T = a.size(0); p.N = w.size(0); p.K = w.size(1);
  TORCH_CHECK(a.size(1) == p.K && p.K % 64 == 0 && p.N % 16 == 0, "narrow projection: a [T, K], w [N, K], K % 64, N % 16");
  return p;
}

// route_softmax of a w^T in one launch (at most 64 columns); splits of K; counters:
// int32 tickets, zero at rest
std::vector<torch::Tensor> router(torch::Tensor a, torch::Tensor w, int64_t experts, int64_t top, bool shared,
                                  int64_t splits, torch::Tensor counters) {
  RowsParams p = rows_of(a, w);
  TORCH_CHECK(p.N <= 64 && experts >= 1 && experts + (shared ? 1 : 0) <= p.N && top >= 1 && top <= experts, "router sizes");
  auto f32 = a.options().dtype(torch::kFloat32);
  auto ids = torch::empty({p.T, top}, a.options().dtype(torch::kInt32));
  auto wts = torch::empty({p.T, top}, f32);
  auto sh = torch::empty({shared ? p.T : 0}, f32);
  p.r.T = p.T; p.r.experts = experts; p.r.top = top;
  p.r.ids = ids.data_ptr<int>(); p.r.wts = wts.data_ptr<float>();
  if (shared) p.r.shared = sh.data_ptr<float>();
  torch::Tensor part;
  p.splits = std::max<int64_t>(1, std::min<int64_t>(splits, p.K / 64));
  if (p.splits > 1) {
    const int64_t tiles = (p.T + 15) / 16, cols = p.N <= 16 ? 16 : p.N <= 32 ? 32 : 64;
    part = torch::empty({tiles * p.splits * 16 * cols}, f32);
    p.part = part.data_ptr<float>();
    p.counters = const_cast<int*>(iptr(counters, tiles, "counters"));
  }
  check_hip(lsd_router(&p, cur_stream()), "router");
  return {ids, wts, sh};
}

// gelu(a w^T) times rows ids of table [vocab, N] in one launch
torch::Tensor side_gate(torch::Tensor a, torch::Tensor w, torch::Tensor ids, torch::Tensor table) {
  RowsParams p = rows_of(a, w);
  need(table, torch::kBFloat16, "table");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous() && table.size(1) == p.N, "table must be [vocab, N]");
  auto out = torch::empty({p.T, p.N}, a.options());
  p.ids = iptr(ids, p.T, "ids"); p.table = table.data_ptr(); p.vocab = table.size(0);
  p.out = out.data_ptr(); p.ldo = p.N;
  check_hip(lsd_side_gate(&p, cur_stream()), "side_gate");
  return out;
}

// rows g [T, n] times rows ids of table [vocab, n] (fp32: gelu(g) times them)
torch::Tensor side_mul(torch::Tensor g, torch::Tensor ids, torch::Tensor table) {
  const bool f32 = is_f32(g, "g");
  need(table, g.scalar_type(), "table");
  const int64_t T = g.size(0), n = g.size(1);
  TORCH_CHECK(g.dim() == 2 && g.is_contiguous() && table.dim() == 2 && table.is_contiguous() && table.size(1) == n &&
                  n % 4 == 0, "side_mul: g [T, n], table [vocab, n], n % 4");
  auto out = torch::empty_like(g);
  check_hip(lsd_side_mul(g.data_ptr(), iptr(ids, T, "ids"), table.data_ptr(), out.data_ptr(), T, n, table.size(0), f32,
                         cur_stream()), "side_mul");
  return out;
}

// rank: value columns of a cached row (0: all)
LatentAttnParams attn_base(const torch::Tensor& q, const torch::Tensor& cache, const torch::Tensor& table,
                           torch::Tensor& out, int64_t H, int64_t window, double scale, int64_t rank, const Opt& sink) {
  is_f32(q, "q");
  need_rows(q, "q");
  need_cache(cache, table, q.scalar_type());
  TORCH_CHECK(q.is_contiguous() && q.size(1) == H * cache.size(2), "q must be contiguous [T, H rank]");
  TORCH_CHECK(window >= 1, "window must be positive");
  const int64_t cols = lsd_latent_value_cols(cache.size(2), rank > 0 ? rank : cache.size(2));
  out = torch::empty({q.size(0), H * cols}, q.options());
  LatentAttnParams p{};
  p.v_pad = cols;
  p.sink = sink_of(sink, H);
  p.q = q.data_ptr(); p.out = out.data_ptr();
  p.cache = cache.data_ptr(); p.table = table.data_ptr<int>(); p.tw = table.size(1);
  p.H = H; p.rank_pad = cache.size(2); p.window = (int)std::min<int64_t>(window, INT_MAX);
  p.scale_log2 = (float)(scale * 1.4426950408889634);
  return p;
}

// one query token per sequence; slots / pos [B]
torch::Tensor latent_decode(torch::Tensor q, torch::Tensor cache, torch::Tensor table, torch::Tensor slots,
                            torch::Tensor pos, int64_t H, int64_t window, double scale, int64_t splits, int64_t rank,
                            Opt sink) {
  torch::Tensor out, po, pml;
  LatentAttnParams p = attn_base(q, cache, table, out, H, window, scale, rank, sink);
  p.B = q.size(0);
  p.seq_slots = iptr(slots, p.B, "slots"); p.pos = iptr(pos, p.B, "pos");
  if (is_f32(q, "q") || lsd_latent_tile_rows(p.rank_pad) == 0) {
    check_hip(lsd_latent_plain(&p, is_f32(q, "q") ? 1 : 0, cur_stream()), "latent_plain");
    return out;
  }
  TORCH_CHECK(splits >= 1 && splits <= 1024, "splits");
  p.splits = splits;
  if (splits > 1) {
    po = torch::empty({p.B * H * splits * p.v_pad}, q.options().dtype(torch::kFloat32));
    pml = torch::empty({p.B * H * splits * 2}, q.options().dtype(torch::kFloat32));
    p.part_o = po.data_ptr<float>(); p.part_ml = pml.data_ptr<float>();
  }
  check_hip(lsd_latent_decode(&p, cur_stream()), "latent_decode");
  return out;
}

// packed ragged queries; tiles [n, 2] = (sequence, first (token, head) row)
torch::Tensor latent_prefill(torch::Tensor q, torch::Tensor cache, torch::Tensor table, torch::Tensor tiles,
                             torch::Tensor seq_slots, torch::Tensor q_start, torch::Tensor cu_q, int64_t H,
                             int64_t window, double scale, int64_t rank, Opt sink) {
  torch::Tensor out;
  LatentAttnParams p = attn_base(q, cache, table, out, H, window, scale, rank, sink);
  TORCH_CHECK(!is_f32(q, "q") && lsd_latent_tile_rows(p.rank_pad) > 0, "latent_prefill: no kernel for this rank");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles must be [n, 2]");
  p.tiles = iptr(tiles, 0, "tiles"); p.n_tiles = tiles.size(0);
  p.B = seq_slots.numel();
  p.seq_slots = iptr(seq_slots, p.B, "seq_slots"); p.pos = iptr(q_start, p.B, "q_start");
  p.cu_q = iptr(cu_q, p.B + 1, "cu_q");
  check_hip(lsd_latent_prefill(&p, cur_stream()), "latent_prefill");
  return out;
}

// cached latents of sequences' reaches as packed rows [rows, rank] (see the kernel)
torch::Tensor latent_gather(torch::Tensor cache, torch::Tensor table, torch::Tensor seq_slots, torch::Tensor k_lo,
                            torch::Tensor cu_k, int64_t rows) {
  need_cache(cache, table, torch::kBFloat16);
  const int64_t B = seq_slots.numel();
  TORCH_CHECK(B >= 1 && rows >= 0 && rows < (1L << 31) && cache.size(2) % 8 == 0, "latent_gather: sizes");
  auto out = torch::empty({rows, cache.size(2)}, cache.options());
  check_hip(lsd_latent_gather(reinterpret_cast<const lsd_bf16_t*>(cache.data_ptr()), table.data_ptr<int>(),
                              table.size(1), iptr(seq_slots, B, "seq_slots"), iptr(k_lo, B, "k_lo"),
                              iptr(cu_k, B + 1, "cu_k"), (int)B, (int)rows, cache.size(2),
                              reinterpret_cast<lsd_bf16_t*>(out.data_ptr()), cur_stream()), "latent_gather");
  return out;
}

// q [T, H dim] over expanded k [rows, H dim], v [rows, H vdim] -> [T, H vdim], times
// the sigmoid of gate [T, H vdim]
torch::Tensor latent_expanded(torch::Tensor q, torch::Tensor k, torch::Tensor v, torch::Tensor tiles,
                              torch::Tensor cu_q, torch::Tensor q_start, torch::Tensor k_lo, torch::Tensor cu_k,
                              int64_t H, int64_t window, double scale, Opt sink, Opt gate) {
  need(q, torch::kBFloat16, "q");
  need(k, torch::kBFloat16, "k");
  need(v, torch::kBFloat16, "v");
  TORCH_CHECK(q.dim() == 2 && q.is_contiguous() && k.dim() == 2 && k.is_contiguous() && v.dim() == 2 &&
                  v.is_contiguous() && k.size(1) == q.size(1) && v.size(0) == k.size(0), "latent_expanded: shapes");
  const int64_t B = q_start.numel(), dim = q.size(1) / H, vdim = v.size(1) / H;
  TORCH_CHECK(q.size(1) == H * dim && v.size(1) == H * vdim && (dim == 64 || dim == 128 || dim == 192) &&
                  vdim % 16 == 0 && vdim >= 16 && vdim <= 128 && window >= 1,
              "latent_expanded: dim 64 / 128 / 192, vdim % 16, vdim <= 128");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles must be [n, 2]");
  auto out = torch::empty({q.size(0), v.size(1)}, q.options());
  lsd::LatentExpandedParams p{};
  p.q = q.data_ptr(); p.k = k.data_ptr(); p.v = v.data_ptr(); p.out = out.data_ptr();
  p.tiles = iptr(tiles, 0, "tiles"); p.n_tiles = tiles.size(0);
  p.cu_q = iptr(cu_q, B + 1, "cu_q"); p.q_start = iptr(q_start, B, "q_start");
  p.k_lo = iptr(k_lo, B, "k_lo"); p.cu_k = iptr(cu_k, B + 1, "cu_k");
  p.sink = sink_of(sink, H);
  if (gate.has_value()) p.gate = gate_rows(*gate, q.size(0), H * vdim, p.ldg);
  p.H = H; p.dim = dim; p.vdim = vdim; p.window = (int)std::min<int64_t>(window, INT_MAX);
  p.scale_log2 = (float)(scale * 1.4426950408889634);
  check_hip(lsd_latent_expanded(&p, cur_stream()), "latent_expanded");
  return out;
}

Opt norm_fp32(torch::Tensor x, Opt slab, Opt w, double eps, Opt rows, bool want_out, int64_t width, double woff) {
  need(x, torch::kFloat32, "x");
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous(), "x must be contiguous [T, H]");
  const int T = x.size(0), H = x.size(1), Hn = width > 0 ? (int)width : H;
  TORCH_CHECK(Hn <= H, "norm_fp32: width");
  const float* sp = nullptr;
  int splits = 0;
  if (slab.has_value()) {
    need(*slab, torch::kFloat32, "slab");
    TORCH_CHECK(!rows.has_value() && slab->is_contiguous() && slab->dim() == 3 && slab->size(1) == T &&
                    slab->size(2) == H, "slab must be [S, T, H]");
    sp = slab->data_ptr<float>();
    splits = slab->size(0);
  }
  Opt out;
  float* op = nullptr;
  const float* wp = nullptr;
  const int* rp = rows.has_value() ? iptr(*rows, rows->numel(), "rows") : nullptr;
  const int n = rows.has_value() ? (int)rows->numel() : T;
  if (want_out) {
    TORCH_CHECK(w.has_value() && w->numel() == H, "w [H]");
    need(*w, torch::kFloat32, "w");
    wp = w->data_ptr<float>();
    out = torch::empty({n, H}, x.options());
    op = out->data_ptr<float>();
  }
  check_hip(lsd_norm_f32(x.data_ptr<float>(), sp, splits, wp, op, T, H, (float)eps, rp, n, Hn, (float)woff,
                         cur_stream()), "norm_fp32");
  return out;
}

torch::Tensor embed_fp32(torch::Tensor ids, torch::Tensor wte, double scale) {
  need(wte, torch::kFloat32, "wte");
  TORCH_CHECK(wte.dim() == 2 && wte.is_contiguous(), "wte must be contiguous [V, H]");
  const int T = ids.numel();
  auto out = torch::empty({T, wte.size(1)}, wte.options());
  check_hip(lsd_embed_f32(iptr(ids, T, "ids"), wte.data_ptr<float>(), out.data_ptr<float>(), T, wte.size(1),
                          wte.size(0), (float)scale, cur_stream()), "embed_fp32");
  return out;
}

}  // namespace

void lsd_register_latent(pybind11::module& m) {
  m.def("batch_linear", &batch_linear, py::arg("a"), py::arg("w"), py::arg("tm"), py::arg("gate") = py::none());
  m.def("linear_fp32", &linear_fp32, py::arg("a"), py::arg("w"), py::arg("x") = py::none(),
        py::arg("bias") = py::none());
  m.def("moe_group", &moe_group, py::arg("ids"), py::arg("experts"), py::arg("tm"));
  m.def("moe_up", &moe_up, py::arg("h"), py::arg("perm"), py::arg("tiles"), py::arg("top"), py::arg("w"),
        py::arg("limit"), py::arg("alpha"), py::arg("ws"), py::arg("limit_s"), py::arg("tm"));
  m.def("moe_down", &moe_down, py::arg("mid"), py::arg("mids"), py::arg("perm"), py::arg("tiles"), py::arg("wts"),
        py::arg("w"), py::arg("ws"), py::arg("slab"), py::arg("tm"), py::arg("wts_s") = py::none());
  m.def("moe_set_group_rows", [](int64_t v) { g_group_rows = v < 1 ? 1 : (int)v; });
  m.def("moe_few", &moe_few, py::arg("h"), py::arg("ids"), py::arg("wts"), py::arg("w_up"), py::arg("w_down"),
        py::arg("limit"), py::arg("alpha"), py::arg("ws_up"), py::arg("ws_down"), py::arg("limit_s"), py::arg("x"),
        py::arg("wts_s") = py::none(), py::arg("add") = true);
  m.def("latent_post", &latent_post, py::arg("y"), py::arg("nq"), py::arg("want_q"), py::arg("f32"), py::arg("cache"),
        py::arg("rank"), py::arg("gain"), py::arg("eps"), py::arg("table"), py::arg("tslot"), py::arg("tpos"),
        py::arg("correction"), py::arg("top"), py::arg("c_off") = -1, py::arg("rope") = py::none(), py::arg("q_head") = 0,
        py::arg("q_rot") = 0, py::arg("q_gain") = py::none());
  m.def("route_softmax", &route_softmax, py::arg("z"), py::arg("experts"), py::arg("top"), py::arg("shared"));
  m.def("router", &router, py::arg("a"), py::arg("w"), py::arg("experts"), py::arg("top"), py::arg("shared"),
        py::arg("splits"), py::arg("counters"));
  m.def("side_gate", &side_gate, py::arg("a"), py::arg("w"), py::arg("ids"), py::arg("table"));
  m.def("side_mul", &side_mul, py::arg("g"), py::arg("ids"), py::arg("table"));
  m.def("latent_value_cols", [](int64_t rank_pad, int64_t rank) { return lsd_latent_value_cols((int)rank_pad, (int)rank); });
  m.def("latent_tile_rows", [](int64_t rank) { return lsd_latent_tile_rows((int)rank); });
  m.def("latent_decode", &latent_decode, py::arg("q"), py::arg("cache"), py::arg("table"), py::arg("slots"),
        py::arg("pos"), py::arg("heads"), py::arg("window"), py::arg("scale"), py::arg("splits"), py::arg("rank") = 0,
        py::arg("sink") = py::none());
  m.def("latent_prefill", &latent_prefill, py::arg("q"), py::arg("cache"), py::arg("table"), py::arg("tiles"),
        py::arg("seq_slots"), py::arg("q_start"), py::arg("cu_q"), py::arg("heads"), py::arg("window"),
        py::arg("scale"), py::arg("rank") = 0, py::arg("sink") = py::none());
  m.def("latent_gather", &latent_gather, py::arg("cache"), py::arg("table"), py::arg("seq_slots"), py::arg("k_lo"),
        py::arg("cu_k"), py::arg("rows"));
  m.def("latent_expanded", &latent_expanded, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("tiles"),
        py::arg("cu_q"), py::arg("q_start"), py::arg("k_lo"), py::arg("cu_k"), py::arg("heads"), py::arg("window"),
        py::arg("scale"), py::arg("sink") = py::none(), py::arg("gate") = py::none());
  m.def("norm_fp32", &norm_fp32, py::arg("x"), py::arg("slab"), py::arg("w"), py::arg("eps"), py::arg("rows"),
        py::arg("want_out"), py::arg("width"), py::arg("woff"));
  m.def("embed_fp32", &embed_fp32, py::arg("ids"), py::arg("wte"), py::arg("scale"));
}
