// gfx950 kernels of a mixture of experts (pg_mixers.h): routing, the sorting of (row, expert) pairs
// for grouped products, and the experts of a few rows as matrix-vector products.
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

// A row of a matrix of f32 or bf16 against a vector in LDS, over the wavefront (n: a multiple of 32).
template <bool BF16>
__device__ __forceinline__ float row_dot(const void* w, size_t at, const float* x, int n) {
  const int lane = threadIdx.x & 63;
  float s = 0.0f;
  if (BF16) {
    const u4v* p = reinterpret_cast<const u4v*>(static_cast<const unsigned short*>(w) + at);
#pragma unroll 4
    for (int j = lane; j < n / 8; j += 64) {
      const u4v u = __builtin_nontemporal_load(p + j);
      const f4 a = *reinterpret_cast<const f4*>(x + 8 * j), b = *reinterpret_cast<const f4*>(x + 8 * j + 4);
      s += __uint_as_float(u.x << 16) * a.x + __uint_as_float(u.x & 0xffff0000u) * a.y + __uint_as_float(u.y << 16) * a.z +
           __uint_as_float(u.y & 0xffff0000u) * a.w + __uint_as_float(u.z << 16) * b.x +
           __uint_as_float(u.z & 0xffff0000u) * b.y + __uint_as_float(u.w << 16) * b.z + __uint_as_float(u.w & 0xffff0000u) * b.w;
    }
  } else {
    const f4* p = reinterpret_cast<const f4*>(static_cast<const float*>(w) + at);
#pragma unroll 4
    for (int j = lane; j < n / 4; j += 64) {
      const f4 u = __builtin_nontemporal_load(p + j);
      const f4 a = *reinterpret_cast<const f4*>(x + 4 * j);
      s += u.x * a.x + u.y * a.y + u.z * a.z + u.w * a.w;
    }
  }
  return s;
}

// act[row * top + k][j] = silu(gate j . x) * (up j . x) of the row's k-th expert.  Every block routes
// its row again: the logits are few.  Grid: x = 4 values of j each, y = (row, k).
template <bool BF16>
__global__ __launch_bounds__(256) void k_moe_act(Moe m, const float* x, const float* logits, float* act, int width) {
  extern __shared__ __attribute__((aligned(16))) float xs[];
  __shared__ int expert;
  const int tid = threadIdx.x, wave = tid >> 6;
  const int row = blockIdx.y / m.top, k = blockIdx.y - row * m.top;
  if (wave == 0)
    choose_any(logits + (size_t)row * m.experts_pad, m.experts, k + 1, [&](int i, int e, float) {
      if (i == k && tid == 0) expert = e;
    });
  for (int i = tid; i < width / 4; i += 256)
    reinterpret_cast<f4*>(xs)[i] = reinterpret_cast<const f4*>(x + (size_t)row * width)[i];
  __syncthreads();
  const int j = blockIdx.x * 4 + wave;
  if (j >= m.ff_pad) return;
  const size_t at = ((size_t)expert * 2 * m.ff_pad + 2 * j) * width;
  float g = row_dot<BF16>(m.gate_up, at, xs, width), u = row_dot<BF16>(m.gate_up, at + width, xs, width);
  g = wave_sum(g);
  u = wave_sum(u);
  if ((tid & 63) == 0) act[(size_t)blockIdx.y * m.ff_pad + j] = g / (1.0f + expf(-g)) * u;
}

// out[row][c] = sum over k of weight k * (down row c of expert k . act).  Grid: x = 4 values of c each,
// y = row.  The activations of as many experts as fit lie in LDS at a time.
template <bool BF16>
__global__ __launch_bounds__(256) void k_moe_down(Moe m, const float* logits, const float* act, float* out, int width,
                                                  int at_once) {
  extern __shared__ __attribute__((aligned(16))) float as[];
  __shared__ int expert[kMoeMaxTop];
  __shared__ float weight[kMoeMaxTop];
  const int tid = threadIdx.x, wave = tid >> 6, row = blockIdx.y, c = blockIdx.x * 4 + wave;
  if (wave == 0)
    choose_any(logits + (size_t)row * m.experts_pad, m.experts, m.top, [&](int i, int e, float w) {
      if (tid == 0) {
        expert[i] = e;
        weight[i] = w;
      }
    });
  float s = 0.0f;
  for (int k0 = 0; k0 < m.top; k0 += at_once) {
    const int nk = min(at_once, m.top - k0);
    __syncthreads();
    const f4* src = reinterpret_cast<const f4*>(act + ((size_t)row * m.top + k0) * m.ff_pad);
    for (int i = tid; i < nk * m.ff_pad / 4; i += 256) reinterpret_cast<f4*>(as)[i] = src[i];
    __syncthreads();
    if (c < width)
      for (int k = 0; k < nk; ++k)
        s += weight[k0 + k] *
             row_dot<BF16>(m.down, ((size_t)expert[k0 + k] * width + c) * m.ff_pad, as + k * m.ff_pad, m.ff_pad);
  }
  s = wave_sum(s);
  if (c < width && (tid & 63) == 0) out[(size_t)row * width + c] = s;
}

// ---- many rows: pairs sorted by expert ----
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

// First slot of every expert, the experts of the tiles, the slots of this block's pairs.
__global__ __launch_bounds__(256) void k_moe_place(Moe m, MoeRoute r, int pairs) {
  __shared__ int first[kMoeMaxExperts + 1];
  const int tid = threadIdx.x;
  if (tid < 64) {  // one wavefront: running sums of the padded counts
    int at = 0;
    for (int e0 = 0; e0 < m.experts; e0 += 64) {
      const int e = e0 + tid;
      const int n = e < m.experts ? (r.count[e] + r.tile_rows - 1) / r.tile_rows * r.tile_rows : 0;
      int s = n;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const int up = __shfl_up(s, off, 64);
        if (tid >= off) s += up;
      }
      if (e < m.experts) first[e] = at + s - n;
      at += __shfl(s, 63, 64);
    }
    if (tid == 0) first[m.experts] = at;
  }
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

}  // namespace

hipError_t launch_moe_few(const Moe& m, const float* x, const float* logits, float* act, float* out, int rows,
                          int width_pad, hipStream_t s) {
  constexpr int kLds = 16000;  // floats of activations at once
  if (m.experts > kMoeMaxExperts || m.top > kMoeMaxTop || m.top > m.experts || m.ff_pad > kLds || width_pad > 16320 ||
      m.ff_pad % 32 != 0 || width_pad % 32 != 0 || rows < 1 || (long)rows * m.top > 65535)
    return hipErrorInvalidValue;
  const dim3 up((m.ff_pad + 3) / 4, rows * m.top), down((width_pad + 3) / 4, rows);
  const int at_once = std::min(m.top, kLds / m.ff_pad);
  const size_t xl = (size_t)width_pad * sizeof(float), al = (size_t)at_once * m.ff_pad * sizeof(float);
  if (m.w_bf16) {
    hipLaunchKernelGGL(k_moe_act<true>, up, dim3(256), xl, s, m, x, logits, act, width_pad);
    hipLaunchKernelGGL(k_moe_down<true>, down, dim3(256), al, s, m, logits, act, out, width_pad, at_once);
  } else {
    hipLaunchKernelGGL(k_moe_act<false>, up, dim3(256), xl, s, m, x, logits, act, width_pad);
    hipLaunchKernelGGL(k_moe_down<false>, down, dim3(256), al, s, m, logits, act, out, width_pad, at_once);
  }
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
  hipLaunchKernelGGL(k_moe_clear, dim3((std::max(m.experts, r.max_slots) + 255) / 256), dim3(256), 0, s, r, m.experts,
                     r.max_slots);
  hipLaunchKernelGGL(k_moe_choose, dim3((rows + kRouteRows - 1) / kRouteRows), dim3(256), 0, s, m, r, logits, rows);
  hipLaunchKernelGGL(k_moe_place, dim3((pairs + 255) / 256), dim3(256), 0, s, m, r, pairs);
  return hipGetLastError();
}

}  // namespace pgk
