// gfx950 kernels of a mixture of experts (pg_mixers.h): routing, the sorting of (row, expert) pairs
// for grouped products, and the experts of one row as matrix-vector products.
//
// Shapes are checked on the host before any launch (pg_stack.cpp).
#include "pg_mixers.h"

#include <math.h>

#include <algorithm>

namespace pgk {

namespace {

typedef float f4 __attribute__((ext_vector_type(4)));
typedef unsigned u4v __attribute__((ext_vector_type(4)));

constexpr int kPerLane = kMoeMaxExperts / 64;  // logits a lane holds

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, 64));
  return v;
}

// One wavefront: the `top` largest logits of z[experts] in descending order (equal ones: the lower
// index first), each with its softmax over all experts; each(k, expert, weight) in every lane.
// NP: logits per lane, experts <= 64 NP.
template <int NP, typename F>
__device__ __forceinline__ void choose_experts(const float* z, int experts, int top, F each) {
  const int lane = threadIdx.x & 63;
  float v[NP], mx = -INFINITY;
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int e = lane + 64 * p;
    v[p] = e < experts ? z[e] : -INFINITY;
    mx = fmaxf(mx, v[p]);
  }
  mx = wave_max(mx);
  float sum = 0.0f;
#pragma unroll
  for (int p = 0; p < NP; ++p) sum += expf(v[p] - mx);
  sum = wave_sum(sum);
  unsigned taken = 0;  // bit p: logit p of this lane
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int at = kMoeMaxExperts;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int e = lane + 64 * p;
      if (e < experts && !(taken >> p & 1) && (at == kMoeMaxExperts || v[p] > best)) {
        best = v[p];
        at = e;
      }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ob = __shfl_xor(best, off, 64);
      const int oa = __shfl_xor(at, off, 64);
      if (oa != kMoeMaxExperts && (at == kMoeMaxExperts || ob > best || (ob == best && oa < at))) {
        best = ob;
        at = oa;
      }
    }
    at = min(at, experts - 1);  // (logits that are not numbers)
    if ((at & 63) == lane) taken |= 1u << (at >> 6);
    each(k, at, expf(best - mx) / sum);
  }
}
template <typename F>
__device__ __forceinline__ void choose_any(const float* z, int experts, int top, F each) {
  if (experts <= 64) choose_experts<1>(z, experts, top, each);
  else if (experts <= 256) choose_experts<4>(z, experts, top, each);
  else choose_experts<kPerLane>(z, experts, top, each);
}

// Sixteen bytes of a row of a matrix of f32 or bf16 against the values in LDS that they meet.
template <bool BF16>
__device__ __forceinline__ float chunk_dot(const u4v& u, const float* x) {
  const f4 a = *reinterpret_cast<const f4*>(x);
  if (!BF16)
    return __uint_as_float(u.x) * a.x + __uint_as_float(u.y) * a.y + __uint_as_float(u.z) * a.z + __uint_as_float(u.w) * a.w;
  const f4 b = *reinterpret_cast<const f4*>(x + 4);
  return __uint_as_float(u.x << 16) * a.x + __uint_as_float(u.x & 0xffff0000u) * a.y + __uint_as_float(u.y << 16) * a.z +
         __uint_as_float(u.y & 0xffff0000u) * a.w + __uint_as_float(u.z << 16) * b.x +
         __uint_as_float(u.z & 0xffff0000u) * b.y + __uint_as_float(u.w << 16) * b.z + __uint_as_float(u.w & 0xffff0000u) * b.w;
}

constexpr int kRouterRows = 16;  // rows of a router that a wavefront multiplies at most
constexpr int kRouterPre = 4;    // 64-chunk pieces of them asked for at the start

// act[k][j] = silu(gate j . x) * (up j . x) of the row's k-th expert.  Every block brings x up to date
// and routes the row for itself (a wavefront: every fourth row of the router); block (0, k) lists
// the choice.  Grid: x = 4 RJ values of j, y = k.  RR: rows of the router to a wavefront (0: the logits are
// there).
template <bool BF16, int RJ, int RR>
__global__ __launch_bounds__(256) void k_moe_act(Moe m, MoeRow r) {
  extern __shared__ __attribute__((aligned(16))) float xs[];
  __shared__ float zs[4 * kRouterRows], red[4];
  __shared__ int expert;
  constexpr int PER = BF16 ? 8 : 4, IN = 4;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, k = blockIdx.y;
  const int K = r.width_pad, n = K / PER, n4 = K / 4;
  f4 vx[IN], va[IN], vg[IN];
#pragma unroll
  for (int p = 0; p < IN; ++p) {
    vx[p] = va[p] = vg[p] = f4{0.f, 0.f, 0.f, 0.f};
    const int i = tid + 256 * p;
    if (i < n4) {
      vx[p] = reinterpret_cast<const f4*>(r.x)[i];
      if (r.add) {
        va[p] = reinterpret_cast<const f4*>(r.add)[i];
        vg[p] = reinterpret_cast<const f4*>(r.add_gain)[i];
      }
    }
  }
  const u4v* rw = static_cast<const u4v*>(r.router);
  u4v pre[RR > 0 ? RR : 1][kRouterPre];
  if constexpr (RR > 0) {
#pragma unroll
    for (int e = 0; e < RR; ++e)
#pragma unroll
      for (int c = 0; c < kRouterPre; ++c) pre[e][c] = rw[(size_t)min(wave + 4 * e, m.experts - 1) * n + min(lane + 64 * c, n - 1)];
  }
  if (r.add) {
    float ss = 0.0f;
#pragma unroll
    for (int p = 0; p < IN; ++p) ss += (va[p].x * va[p].x + va[p].y * va[p].y) + (va[p].z * va[p].z + va[p].w * va[p].w);
    for (int i = tid + 256 * IN; i < n4; i += 256) {
      const f4 v = reinterpret_cast<const f4*>(r.add)[i];
      ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
    }
    ss = wave_sum(ss);
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    const float f = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)r.width + r.eps);
#pragma unroll
    for (int p = 0; p < IN; ++p) vx[p] += va[p] * f * vg[p];
    for (int i = tid + 256 * IN; i < n4; i += 256) {
      const f4 v = reinterpret_cast<const f4*>(r.x)[i] +
                   reinterpret_cast<const f4*>(r.add)[i] * f * reinterpret_cast<const f4*>(r.add_gain)[i];
      reinterpret_cast<f4*>(xs)[i] = v;
      if (blockIdx.x == 0 && k == 0) reinterpret_cast<f4*>(r.x_out)[i] = v;
    }
  } else {
    for (int i = tid + 256 * IN; i < n4; i += 256) reinterpret_cast<f4*>(xs)[i] = reinterpret_cast<const f4*>(r.x)[i];
  }
#pragma unroll
  for (int p = 0; p < IN; ++p) {
    const int i = tid + 256 * p;
    if (i < n4) {
      reinterpret_cast<f4*>(xs)[i] = vx[p];
      if (r.add && blockIdx.x == 0 && k == 0) reinterpret_cast<f4*>(r.x_out)[i] = vx[p];
    }
  }
  __syncthreads();
  const float* z = r.logits;
  if constexpr (RR > 0) {
#pragma unroll
    for (int e = 0; e < RR; ++e) {
      if (wave + 4 * e >= m.experts) break;
      float s = 0.0f;
#pragma unroll
      for (int c = 0; c < kRouterPre; ++c)
        if (lane + 64 * c < n) s += chunk_dot<BF16>(pre[e][c], xs + PER * (lane + 64 * c));
#pragma unroll 4
      for (int j = lane + 64 * kRouterPre; j < n; j += 64) s += chunk_dot<BF16>(rw[(size_t)(wave + 4 * e) * n + j], xs + PER * j);
      s = wave_sum(s);
      if (lane == 0) zs[wave + 4 * e] = s;
    }
    __syncthreads();
    z = zs;
  }
  if (wave == 0)
    choose_any(z, m.experts, k + 1, [&](int i, int e, float w) {
      if (i == k && tid == 0) {
        expert = e;
        if (blockIdx.x == 0) {
          r.expert[k] = e;
          r.weight[k] = w;
        }
      }
    });
  __syncthreads();
  const int j0 = (blockIdx.x * 4 + wave) * RJ;
  if (j0 >= m.ff_pad) return;
  // rows 2 j and 2 j + 1, RJ values of j (ff_pad is a multiple of 32)
  const u4v* w = static_cast<const u4v*>(m.gate_up) + ((size_t)expert * 2 * m.ff_pad + 2 * j0) * n;
  float s[2 * RJ];
#pragma unroll
  for (int q = 0; q < 2 * RJ; ++q) s[q] = 0.0f;
#pragma unroll 4
  for (int i = lane; i < n; i += 64) {
    u4v u[2 * RJ];
#pragma unroll
    for (int q = 0; q < 2 * RJ; ++q) u[q] = __builtin_nontemporal_load(w + (size_t)q * n + i);
#pragma unroll
    for (int q = 0; q < 2 * RJ; ++q) s[q] += chunk_dot<BF16>(u[q], xs + PER * i);
  }
#pragma unroll
  for (int q = 0; q < 2 * RJ; ++q) s[q] = wave_sum(s[q]);
  if (lane == 0)
#pragma unroll
    for (int q = 0; q < RJ; ++q)
      r.act[(size_t)k * m.ff_pad + j0 + q] = s[2 * q] / (1.0f + expf(-s[2 * q])) * s[2 * q + 1];
}

// out[c] = sum over k of weight k * (down row c of expert k . act): one dot product over the experts'
// rows one after the other, against the weighted activations in LDS (as many experts as fit at a
// time).  Grid: x = 4 values of c.
template <bool BF16>
__global__ __launch_bounds__(256) void k_moe_down(Moe m, MoeRow r, int at_once) {
  extern __shared__ __attribute__((aligned(16))) float as[];
  constexpr int PER = BF16 ? 8 : 4, PRE = 8;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = min((int)blockIdx.x * 4 + wave, r.width_pad - 1);
  const int n = m.ff_pad / PER, n4 = m.ff_pad / 4;
  const u4v* down = static_cast<const u4v*>(m.down);
  float s = 0.0f;
  for (int k0 = 0; k0 < m.top; k0 += at_once) {
    const int nk = min(at_once, m.top - k0), chunks = nk * n;
    auto load = [&](int j) {
      const int k = j / n;
      return __builtin_nontemporal_load(down + ((size_t)r.expert[k0 + k] * r.width_pad + c) * n + (j - k * n));
    };
    u4v pre[PRE];  // the weights' first chunks are on their way while the activations are staged
#pragma unroll
    for (int p = 0; p < PRE; ++p) pre[p] = load(min(lane + 64 * p, chunks - 1));
    __syncthreads();
    const f4* src = reinterpret_cast<const f4*>(r.act + (size_t)k0 * m.ff_pad);
    for (int i = tid; i < nk * n4; i += 256) reinterpret_cast<f4*>(as)[i] = src[i] * r.weight[k0 + i / n4];
    __syncthreads();
#pragma unroll
    for (int p = 0; p < PRE; ++p)
      if (lane + 64 * p < chunks) s += chunk_dot<BF16>(pre[p], as + PER * (lane + 64 * p));
#pragma unroll 4
    for (int j = lane + 64 * PRE; j < chunks; j += 64) s += chunk_dot<BF16>(load(j), as + PER * j);
  }
  s = wave_sum(s);
  if (lane == 0) r.out[c] = s;
}

// ---- several rows: pairs sorted by expert ----
constexpr int kRouteRows = 16;  // rows of a block

__global__ __launch_bounds__(256) void k_moe_clear(MoeRoute r, int experts, int slots) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < experts) r.count[i] = 0;
  if (i < slots) r.slot_row[i] = -1;
  if (i < slots / r.tile_rows) r.tile[i] = -1;
}

// The experts of every row, and the number of each pair within its expert.  (Which pair gets which
// number depends on timing; nothing that is computed from a pair does.)
__global__ __launch_bounds__(256) void k_moe_choose(Moe m, MoeRoute r, const float* logits, int rows) {
  __shared__ int count[kMoeMaxExperts], base[kMoeMaxExperts];
  const int tid = threadIdx.x, wave = tid >> 6, row0 = blockIdx.x * kRouteRows;
  for (int i = tid; i < m.experts; i += 256) count[i] = 0;
  __syncthreads();
  for (int i = wave; i < kRouteRows && row0 + i < rows; i += 4) {
    const int row = row0 + i;
    choose_any(logits + (size_t)row * m.experts_pad, m.experts, m.top, [&](int k, int e, float w) {
      if ((tid & 63) == 0) {
        const size_t p = (size_t)row * m.top + k;
        r.expert[p] = e;
        r.weight[p] = w;
        r.rank[p] = atomicAdd(&count[e], 1);
      }
    });
  }
  __syncthreads();
  for (int i = tid; i < m.experts; i += 256) base[i] = count[i] ? atomicAdd(&r.count[i], count[i]) : 0;
  __syncthreads();
  const int n = min(kRouteRows, rows - row0) * m.top;
  for (int i = tid; i < n; i += 256) {
    const size_t p = (size_t)row0 * m.top + i;
    r.rank[p] += base[r.expert[p]];
  }
}

// One wavefront: running sums of the padded counts.
__device__ void first_slots(const Moe& m, int tile_rows, const int* count, int* first) {
  const int lane = threadIdx.x & 63;
  int at = 0;
  for (int e0 = 0; e0 < m.experts; e0 += 64) {
    const int e = e0 + lane;
    const int n = e < m.experts ? (count[e] + tile_rows - 1) / tile_rows * tile_rows : 0;
    int s = n;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int up = __shfl_up(s, off, 64);
      if (lane >= off) s += up;
    }
    if (e < m.experts) first[e] = at + s - n;
    at += __shfl(s, 63, 64);
  }
  if (lane == 0) first[m.experts] = at;
}

// First slot of every expert, the experts of the tiles, the slots of this block's pairs.
__global__ __launch_bounds__(256) void k_moe_place(Moe m, MoeRoute r, int pairs) {
  __shared__ int first[kMoeMaxExperts + 1];
  const int tid = threadIdx.x;
  if (tid < 64) first_slots(m, r.tile_rows, r.count, first);
  __syncthreads();
  if (blockIdx.x == 0)
    for (int e = tid; e < m.experts; e += 256)
      for (int t = first[e] / r.tile_rows; t < first[e + 1] / r.tile_rows; ++t) r.tile[t] = e;
  const int p = blockIdx.x * 256 + tid;
  if (p >= pairs) return;
  const int s = first[r.expert[p]] + r.rank[p];
  r.slot[p] = s;
  r.slot_row[s] = p / m.top;
}

// All of it in one block, for a few rows.
constexpr int kRouteSmallRows = 128, kRouteSmallPairs = 4096;
__global__ __launch_bounds__(1024) void k_moe_route_small(Moe m, MoeRoute r, const float* logits, int rows) {
  __shared__ int count[kMoeMaxExperts], first[kMoeMaxExperts + 1];
  __shared__ int pair[kRouteSmallPairs];  // expert and number within it
  const int tid = threadIdx.x, wave = tid >> 6;
  for (int i = tid; i < m.experts; i += 1024) count[i] = 0;
  for (int i = tid; i < r.max_slots; i += 1024) r.slot_row[i] = -1;
  for (int i = tid; i < r.max_slots / r.tile_rows; i += 1024) r.tile[i] = -1;
  __syncthreads();
  for (int row = wave; row < rows; row += 16)
    choose_any(logits + (size_t)row * m.experts_pad, m.experts, m.top, [&](int k, int e, float w) {
      if ((tid & 63) == 0) {
        const size_t p = (size_t)row * m.top + k;
        r.weight[p] = w;
        pair[p] = e << 16 | atomicAdd(&count[e], 1);
      }
    });
  __syncthreads();
  if (tid < 64) first_slots(m, r.tile_rows, count, first);
  __syncthreads();
  for (int e = tid; e < m.experts; e += 1024)
    for (int t = first[e] / r.tile_rows; t < first[e + 1] / r.tile_rows; ++t) r.tile[t] = e;
  for (int p = tid; p < rows * m.top; p += 1024) {
    const int s = first[pair[p] >> 16] + (pair[p] & 0xffff);
    r.slot[p] = s;
    r.slot_row[s] = p / m.top;
  }
}

}  // namespace

bool moe_router_fits(const Moe& m, int width_pad) { return m.experts <= 4 * kRouterRows && (long)m.experts * width_pad <= 65536; }

hipError_t launch_moe_row(const Moe& m, const MoeRow& r, hipStream_t s) {
  if (m.experts > kMoeMaxExperts || m.top > kMoeMaxTop || m.top > m.experts || m.ff_pad > kMoeMaxWidth || r.width_pad > kMoeMaxWidth ||
      m.ff_pad % 32 != 0 || r.width_pad % 32 != 0 || (r.logits == nullptr) == (r.router == nullptr) ||
      (r.router && !moe_router_fits(m, r.width_pad)))
    return hipErrorInvalidValue;
  const int rj = (long)m.ff_pad * m.top >= 2048 ? 2 : 1;
  const dim3 up(m.ff_pad / (4 * rj), m.top), down((r.width_pad + 3) / 4);
  const int at_once = std::min(m.top, kMoeMaxWidth / m.ff_pad);
  const size_t xl = (size_t)r.width_pad * sizeof(float), al = (size_t)at_once * m.ff_pad * sizeof(float);
  const int rr = !r.router ? 0 : m.experts <= 8 ? 2 : m.experts <= 16 ? 4 : kRouterRows;
#define PG_ACT(B, J)                                                                                          \
  if (rr == 0) hipLaunchKernelGGL((k_moe_act<B, J, 0>), up, dim3(256), xl, s, m, r);                           \
  else if (rr == 2) hipLaunchKernelGGL((k_moe_act<B, J, 2>), up, dim3(256), xl, s, m, r);                      \
  else if (rr == 4) hipLaunchKernelGGL((k_moe_act<B, J, 4>), up, dim3(256), xl, s, m, r);                      \
  else hipLaunchKernelGGL((k_moe_act<B, J, kRouterRows>), up, dim3(256), xl, s, m, r);
  if (m.w_bf16) {
    if (rj == 2) {
      PG_ACT(true, 2)
    } else {
      PG_ACT(true, 1)
    }
    hipLaunchKernelGGL(k_moe_down<true>, down, dim3(256), al, s, m, r, at_once);
  } else {
    if (rj == 2) {
      PG_ACT(false, 2)
    } else {
      PG_ACT(false, 1)
    }
    hipLaunchKernelGGL(k_moe_down<false>, down, dim3(256), al, s, m, r, at_once);
  }
#undef PG_ACT
  return hipGetLastError();
}

// Every expert that has pairs may leave up to tile_rows - 1 slots of its last tile empty.
int moe_max_slots(const Moe& m, int rows, int tile_rows) {
  const long pairs = (long)rows * m.top, used = std::min<long>(m.experts, pairs);
  return (int)((pairs + used * (tile_rows - 1)) / tile_rows * tile_rows);
}

hipError_t launch_moe_route(const Moe& m, const MoeRoute& r, const float* logits, int rows, hipStream_t s) {
  if (m.experts > kMoeMaxExperts || m.top > kMoeMaxTop || m.top > m.experts || r.max_slots != moe_max_slots(m, rows, r.tile_rows))
    return hipErrorInvalidValue;
  const int pairs = rows * m.top;
  if (rows <= kRouteSmallRows && pairs <= kRouteSmallPairs) {
    hipLaunchKernelGGL(k_moe_route_small, dim3(1), dim3(1024), 0, s, m, r, logits, rows);
    return hipGetLastError();
  }
  hipLaunchKernelGGL(k_moe_clear, dim3((std::max(m.experts, r.max_slots) + 255) / 256), dim3(256), 0, s, r, m.experts,
                     r.max_slots);
  hipLaunchKernelGGL(k_moe_choose, dim3((rows + kRouteRows - 1) / kRouteRows), dim3(256), 0, s, m, r, logits, rows);
  hipLaunchKernelGGL(k_moe_place, dim3((pairs + 255) / 256), dim3(256), 0, s, m, r, pairs);
  return hipGetLastError();
}

}  // namespace pgk
