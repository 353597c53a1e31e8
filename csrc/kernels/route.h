// Expert choice of one row, shared by the kernels that route (moe.hip, gemm_rows.hip).
#pragma once
#include "common.h"
#include "moe_params.h"

namespace lsd {

// One row's routing by one wave; EPL: experts per lane.
template <int EPL>
__device__ __forceinline__ void route_row(const RouteParams& p, const float* z, int t) {
  const int lane = lane_id();
  float sc[EPL], ch[EPL];
#pragma unroll
  for (int j = 0; j < EPL; ++j) {
    const int e = lane + 64 * j;
    const bool ok = e < p.experts;
    const float v = ok ? z[e] : 0.f;
    sc[j] = p.correction ? 1.f / (1.f + expf(-v)) : v;
    ch[j] = !ok ? -INFINITY : p.correction ? sc[j] + p.correction[e] : sc[j];
  }
  if (p.shared && lane == 0) p.shared[t] = 1.f / (1.f + expf(-z[p.experts]));
  float sum = 0.f, mine = 0.f, best = 0.f;
  for (int k = 0; k < p.top; ++k) {
    // best corrected score of the wave; the lower expert wins a tie
    float b = -INFINITY;
    int be = 0x7fffffff;
#pragma unroll
    for (int j = 0; j < EPL; ++j)
      if (ch[j] > b) {
        b = ch[j];
        be = lane + 64 * j;
      }
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) {
      const float ob = __shfl_xor(b, m, 64);
      const int oe = __shfl_xor(be, m, 64);
      if (ob > b || (ob == b && oe < be)) {
        b = ob;
        be = oe;
      }
    }
    // scores that are not numbers never win: keep the ids in range
    if (be >= p.experts) be = k;
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < EPL; ++j)
      if (be == lane + 64 * j) {
        s = sc[j];
        ch[j] = -INFINITY;
      }
    s = __shfl(s, be & 63, 64);
    if (!p.correction) {  // softmax over the chosen logits, the first the largest
      if (k == 0) best = s;
      s = expf(s - best);
    }
    sum += s;
    if (lane == (k & 63)) {
      if (k >= 64) {  // more choices than lanes: park the earlier ones
        p.wts[(long)t * p.top + k - 64] = mine;
      }
      mine = s;
      p.ids[(long)t * p.top + k] = be;
    }
  }
  // divide by the sum: lane l holds choice k = l (+ 64 when top > 64)
  const float inv = 1.f / (sum + 1e-20f);
  for (int k = lane; k < p.top; k += 64) {
    const bool held = k + 64 >= p.top;
    p.wts[(long)t * p.top + k] = (held ? mine : p.wts[(long)t * p.top + k]) * inv;
  }
}

// At most 64 experts, softmax over the chosen logits: every lane counts the logits in
// front of its own (the lower expert first where two are equal).
__device__ __forceinline__ void route_few(const RouteParams& p, const float* z, int t) {
  const int lane = lane_id();
  const float v = lane < p.experts ? z[lane] : -INFINITY;
  if (p.shared && lane == 0) p.shared[t] = 1.f / (1.f + expf(-z[p.experts]));
  int rank = 0;
  for (int e = 0; e < p.experts; ++e) {
    const float u = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), e));
    rank += u > v || (u == v && e < lane) ? 1 : 0;
  }
  const bool real = v == v;  // what is not a number comes last, its ids stay in range
  const int bad = __popcll(__ballot(!real && lane < p.experts));
  if (bad) {
    const int before = __popcll(__ballot(!real && lane < p.experts) & ((1ull << lane) - 1));
    rank = real ? rank : p.experts - bad + before;
  }
  const bool chosen = lane < p.experts && rank < p.top;
  // the largest logit is the first chosen one's
  const unsigned long long first = __ballot(chosen && rank == 0);
  const float best = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), first ? __ffsll(first) - 1 : 0));
  const float e = chosen && real ? expf(v - best) : 0.f;
  const float sum = wave_sum(e);
  if (chosen) {
    p.ids[(long)t * p.top + rank] = lane;
    p.wts[(long)t * p.top + rank] = e / (sum + 1e-20f);
  }
}

}  // namespace lsd
