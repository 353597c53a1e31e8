// Expert routing and the per-token work behind a latent-attention layer's
// input projection.
//
//  * latent_post: one block per token over the fp32 projection row: RMS norm of
//    the latent and its append to the paged cache with the turned key part, bf16
//    queries for the MFMA projections (turned, or normed where they are a latent of
//    their own), and the routing where the router reads the same row.  A model
//    whose layers have only some of these passes the others as absent.
//  * route: a wave per row of router logits; the `top` experts with the largest
//    corrected sigmoid score and their normalised uncorrected scores, or with the
//    largest logits and their softmax.
//  * side_mul: gated rows times the tokens' own rows of a table.
//  * moe_group: sorts the (token, choice) entries by expert and cuts every
//    expert's rows into tiles for the grouped GEMMs (group_gemm.hip) -- all on
//    the device, so a captured decode graph follows the routing of each replay.
#include "common.h"
#include "moe_params.h"
#include "route.h"

namespace lsd {

template <typename T>
__device__ __forceinline__ T narrow(float v);
template <>
__device__ __forceinline__ bf16 narrow<bf16>(float v) { return f2bf(v); }
template <>
__device__ __forceinline__ float narrow<float>(float v) { return v; }

constexpr int LATENT_PAGE = 64;  // tokens per cache page
constexpr int MAX_EXPERTS = 1024;

// One wave per row of router logits that stand alone
template <int EPL>
__global__ __launch_bounds__(256) void route_kernel(RouteParams p) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= p.T) return;
  if (EPL == 1 && !p.correction) route_few(p, p.z + (long)t * p.ldz, t);
  else route_row<EPL>(p, p.z + (long)t * p.ldz, t);
}

// Column c of a head turned: pairs (rot + i, rot + i + half)
__device__ __forceinline__ float turned(const float* head, int c, int rot, int half, const float* cs) {
  const int j = c - rot;
  const float v = head[c];
  if (j < 0 || j >= 2 * half) return v;
  const int i = j < half ? j : j - half;
  const float co = cs[2 * i], si = cs[2 * i + 1];
  return j < half ? v * co - head[c + half] * si : v * co + head[c - half] * si;
}

template <typename T, int EPL>  // EPL: experts per lane
__global__ __launch_bounds__(256) void latent_post_kernel(LatentPostParams p) {
  // the parts are independent (no block barrier): wave 0 routes, wave 1 appends, and
  // those that have neither, at least the last two, see to the queries
  const int lane = lane_id(), w = threadIdx.x >> 6, t = blockIdx.x;
  const float* y = p.y + (long)t * p.ldy;
  const float* cs = p.half ? p.rope + (long)p.tpos[t] * 2 * p.half : nullptr;
  const int w0 = p.r.experts > 0 ? 2 : p.cache != nullptr ? 1 : 0;  // first wave that may be free
  const bool appends = p.cache != nullptr && w == (w0 == 1 ? 0 : 1);
  if (p.q != nullptr && w >= w0) {
    T* q = static_cast<T*>(p.q) + (long)t * p.nq;
    const int id = threadIdx.x - 64 * w0, step = 256 - 64 * w0;
    if (p.q_gain) {
      if (w == 3) {
        float s = 0.f;
#pragma unroll 8
        for (int i = lane; i < p.q_rank; i += 64) s += y[i] * y[i];
        const float rstd = 1.f / sqrtf(wave_sum(s) / p.q_rank + p.eps);
#pragma unroll 8
        for (int i = lane; i < p.nq; i += 64) q[i] = narrow<T>(i < p.q_rank ? y[i] * rstd * p.q_gain[i] : 0.f);
      }
    } else if (sizeof(T) == 2 && (p.half == 0 || (p.q_rot % 4 == 0 && p.half % 4 == 0))) {
      // a wave takes a head (or 256 columns where nothing turns) at a time: what a lane
      // turns, and by how much, is the same for all of them
      const int span = p.half ? p.q_head : 256, nh = (p.nq + span - 1) / span, nw = 4 - w0;
      for (int at = lane * 4; at < span; at += 256) {
        const int j = at - p.q_rot;
        const bool in = p.half && j >= 0 && j < 2 * p.half;
        const int other = !in ? 0 : j < p.half ? p.half : -p.half;
        f32x4 co = {1.f, 1.f, 1.f, 1.f}, si = {0.f, 0.f, 0.f, 0.f};
        if (in) {
          const float* c = cs + 2 * (j < p.half ? j : j - p.half);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            co[e] = c[2 * e];
            si[e] = j < p.half ? -c[2 * e + 1] : c[2 * e + 1];
          }
        }
        constexpr int FLY = 4;
        for (int h = w - w0; h < nh; h += FLY * nw) {
          f32x4 v[FLY], u[FLY];
#pragma unroll
          for (int i = 0; i < FLY; ++i) {
            const int c = min(min(h + i * nw, nh - 1) * span + at, p.nq - 4);
            v[i] = *reinterpret_cast<const f32x4*>(y + c);
            u[i] = p.half ? *reinterpret_cast<const f32x4*>(y + c + other) : v[i];
          }
#pragma unroll
          for (int i = 0; i < FLY; ++i) {
            const int c = (h + i * nw) * span + at;
            if (h + i * nw < nh && c < p.nq) st4(reinterpret_cast<bf16*>(q) + c, pack4(p.half ? v[i] * co + u[i] * si : v[i]));
          }
        }
      }
    } else {
      for (int c = id; c < p.nq; c += step)
        q[c] = narrow<T>(p.half ? turned(y + c - c % p.q_head, c % p.q_head, p.q_rot, p.half, cs) : y[c]);
    }
  }
  if (appends) {
    const float* c = y + p.c_off;
    const int pos = p.tpos[t];
    const int page = p.table[(long)p.tslot[t] * p.tw + pos / LATENT_PAGE];
    float s = 0.f;
#pragma unroll 8
    for (int i = lane; i < p.rank; i += 64) s += c[i] * c[i];
    s = wave_sum(s);
    const float rstd = 1.f / sqrtf(s / p.rank + p.eps);
    T* o = static_cast<T*>(p.cache) + ((long)page * LATENT_PAGE + pos % LATENT_PAGE) * p.rank_pad;
#pragma unroll 8
    for (int i = lane; i < p.rank_pad; i += 64) {
      float v = i < p.rank ? c[i] * rstd * p.gain[i] : 0.f;
      if (i >= p.rank && i < p.rank + 2 * p.half) v = turned(c, i, p.rank, p.half, cs);
      o[i] = narrow<T>(v);
    }
  }
  if (p.r.experts > 0 && w == 0) route_row<EPL>(p.r, y + p.r_off, t);
}

// One block.  ids [n] -> perm [n] (entries sorted by expert), tiles
// [n_tiles][4] = (expert, first sorted row, rows, 0); rows == 0 past the last.
__global__ __launch_bounds__(1024) void moe_group_kernel(const int* __restrict__ ids, int n, int E, int tm,
                                                         int* __restrict__ perm, int* __restrict__ tiles,
                                                         int n_tiles) {
  __shared__ int cnt[MAX_EXPERTS], off[MAX_EXPERTS], toff[MAX_EXPERTS];
  __shared__ int wsum[16], wtile[16];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  if (tid < E) cnt[tid] = 0;
  __syncthreads();
  for (int i = tid; i < n; i += 1024) atomicAdd(&cnt[ids[i]], 1);
  __syncthreads();
  // exclusive prefix sums of rows and tiles over the experts
  const int c = tid < E ? cnt[tid] : 0;
  const int ct = (c + tm - 1) / tm;
  int a = c, b = ct;
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    const int ua = __shfl_up(a, d, 64), ub = __shfl_up(b, d, 64);
    if (lane >= d) {
      a += ua;
      b += ub;
    }
  }
  if (lane == 63) {
    wsum[w] = a;
    wtile[w] = b;
  }
  __syncthreads();
  int pa = 0, pb = 0, total = 0;
  for (int i = 0; i < 16; ++i) {
    if (i < w) {
      pa += wsum[i];
      pb += wtile[i];
    }
    total += wtile[i];
  }
  if (tid < E) {
    off[tid] = pa + a - c;
    toff[tid] = pb + b - ct;
    for (int k = 0; k < ct; ++k) {
      int* tl = tiles + 4 * (long)(toff[tid] + k);
      tl[0] = tid;
      tl[1] = off[tid] + k * tm;
      tl[2] = min(tm, c - k * tm);
      tl[3] = 0;
    }
  }
  for (int i = total + tid; i < n_tiles; i += 1024) tiles[4 * (long)i + 2] = 0;
  __syncthreads();
  for (int i = tid; i < n; i += 1024) perm[atomicAdd(&off[ids[i]], 1)] = i;
}

// RMS norm of fp32 rows into fp32 (models served in fp32), folding fp32 slabs
// into the residual first: the fp32 twin of norm.hip's kernels.
__global__ __launch_bounds__(256) void norm_f32_kernel(float* x, const float* __restrict__ slab, int splits,
                                                       const float* __restrict__ w, float* out, int T, int H,
                                                       float eps, const int* __restrict__ rows, int Hn, float woff) {
  __shared__ float red[16];
  const int t = blockIdx.x, src = rows ? rows[t] : t;
  float* xr = x + (long)src * H;
  float s = 0.f;
  for (int c = threadIdx.x; c < H; c += 256) {
    float v = xr[c];
    if (slab) {
      for (int k = 0; k < splits; ++k) v += slab[((long)k * T + src) * H + c];
      xr[c] = v;
    }
    s += v * v;
  }
  if (out == nullptr) return;
  const float rstd = 1.f / sqrtf(block_sum(s, red) / Hn + eps);
  for (int c = threadIdx.x; c < H; c += 256) out[(long)t * H + c] = xr[c] * rstd * (w[c] + woff);
}

__global__ __launch_bounds__(256) void embed_f32_kernel(const int* __restrict__ ids, const float* __restrict__ wte,
                                                        float* out, int H, int vocab, float scale) {
  int id = ids[blockIdx.x];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  for (int c = threadIdx.x; c < H; c += 256) out[(long)blockIdx.x * H + c] = wte[(long)id * H + c] * scale;
}

// out[t] = g[t] * table[ids[t]], rows of n columns (fp32: gelu(g[t]) * table[ids[t]])
template <typename T>
__global__ __launch_bounds__(256) void side_mul_kernel(const T* g, const int* __restrict__ ids,
                                                       const T* __restrict__ table, T* out, long items, int n, int vocab) {
  const long at = (long)blockIdx.x * 256 + threadIdx.x;
  if (at >= items) return;
  const long row = at / (n / 4);
  const int c = (int)(at % (n / 4)) * 4;
  int id = ids[row];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  if constexpr (sizeof(T) == 2) {
    const bf16x4 a = ld4(g + row * n + c), e = ld4(table + (long)id * n + c);
    st4(out + row * n + c, pack4(f32x4{bf2f(a[0]) * bf2f(e[0]), bf2f(a[1]) * bf2f(e[1]), bf2f(a[2]) * bf2f(e[2]),
                                       bf2f(a[3]) * bf2f(e[3])}));
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float z = g[row * n + c + i];
      out[row * n + c + i] =
          0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))) * table[(long)id * n + c + i];
    }
  }
}

}  // namespace lsd

using namespace lsd;

template <typename T>
static hipError_t post(const LatentPostParams& p, hipStream_t st) {
  const dim3 grid(p.T), blk(256);
  const int epl = (p.r.experts + 63) / 64;
  if (epl <= 1) hipLaunchKernelGGL((latent_post_kernel<T, 1>), grid, blk, 0, st, p);
  else if (epl <= 4) hipLaunchKernelGGL((latent_post_kernel<T, 4>), grid, blk, 0, st, p);
  else if (epl <= 16) hipLaunchKernelGGL((latent_post_kernel<T, 16>), grid, blk, 0, st, p);
  else return hipErrorInvalidValue;
  return hipGetLastError();
}

extern "C" hipError_t lsd_latent_post(const LatentPostParams* p, int f32, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  if (p->r.top > 128 || p->r.top > p->r.experts) return hipErrorInvalidValue;
  return f32 ? post<float>(*p, st) : post<bf16>(*p, st);
}

extern "C" hipError_t lsd_route(const RouteParams* p, hipStream_t st) {
  if (p->T == 0) return hipSuccess;
  if (p->top > 128 || p->top > p->experts) return hipErrorInvalidValue;
  const dim3 grid((p->T + 3) / 4), blk(256);
  const int epl = (p->experts + 63) / 64;
  if (epl <= 1) hipLaunchKernelGGL((route_kernel<1>), grid, blk, 0, st, *p);
  else if (epl <= 4) hipLaunchKernelGGL((route_kernel<4>), grid, blk, 0, st, *p);
  else if (epl <= 16) hipLaunchKernelGGL((route_kernel<16>), grid, blk, 0, st, *p);
  else return hipErrorInvalidValue;
  return hipGetLastError();
}

extern "C" hipError_t lsd_side_mul(const void* g, const int* ids, const void* table, void* out, int T, int n, int vocab,
                                   int f32, hipStream_t st) {
  if (T == 0) return hipSuccess;
  const long items = (long)T * n / 4;
  const dim3 grid((unsigned)((items + 255) / 256));
  if (f32)
    hipLaunchKernelGGL((side_mul_kernel<float>), grid, dim3(256), 0, st, static_cast<const float*>(g), ids,
                       static_cast<const float*>(table), static_cast<float*>(out), items, n, vocab);
  else
    hipLaunchKernelGGL((side_mul_kernel<bf16>), grid, dim3(256), 0, st, static_cast<const bf16*>(g), ids,
                       static_cast<const bf16*>(table), static_cast<bf16*>(out), items, n, vocab);
  return hipGetLastError();
}

extern "C" hipError_t lsd_moe_group(const int* ids, int n, int E, int tm, int* perm, int* tiles, int n_tiles,
                                    hipStream_t st) {
  if (E > MAX_EXPERTS) return hipErrorInvalidValue;
  hipLaunchKernelGGL(moe_group_kernel, dim3(1), dim3(1024), 0, st, ids, n, E, tm, perm, tiles, n_tiles);
  return hipGetLastError();
}

extern "C" hipError_t lsd_norm_f32(float* x, const float* slab, int splits, const float* w, float* out, int T, int H,
                                   float eps, const int* rows, int nrows, int Hn, float woff, hipStream_t st) {
  const int n = rows ? nrows : T;
  if (n == 0) return hipSuccess;
  hipLaunchKernelGGL(norm_f32_kernel, dim3(n), dim3(256), 0, st, x, slab, splits, w, out, T, H, eps, rows, Hn, woff);
  return hipGetLastError();
}

extern "C" hipError_t lsd_embed_f32(const int* ids, const float* wte, float* out, int T, int H, int vocab, float scale,
                                    hipStream_t st) {
  if (T == 0) return hipSuccess;
  hipLaunchKernelGGL(embed_f32_kernel, dim3(T), dim3(256), 0, st, ids, wte, out, H, vocab, scale);
  return hipGetLastError();
}
