// gfx950 kernels of the sequence mixers (pg_mixers.h): chunked sigmoid attention on the f32
// matrix cores, the recurrences, and the element-wise steps around them.  All arithmetic is f32
// (angles: the product position * frequency is reduced to one turn in f64).
//
// Shapes are checked on the host before any launch (pg_stack.cpp); kernels guard ragged tails.
#include "pg_mixers.h"

#include <math.h>

#include <algorithm>

namespace pgk {

namespace {

typedef float f4 __attribute__((ext_vector_type(4)));
typedef float f16v __attribute__((ext_vector_type(16)));

__device__ __forceinline__ float gelu_tanh(float x) {
  return 0.5f * x * (1.0f + tanhf(0.7978846f * (x + 0.044715f * x * x * x)));
}
__device__ __forceinline__ float sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.0f) + log1pf(expf(-fabsf(x))); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
  return v;
}
// Sum over a block of 256 threads; every thread receives the result.  red holds 4 floats.
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

__device__ __forceinline__ void turn(int pos, double freq, float* s, float* c) {
  double a = (double)pos * freq;
  a -= 6.283185307179586476925287 * rint(a * 0.15915494309189533577);
  sincosf((float)a, s, c);
}

// Log of the decay of the gated delta rule and of gated linear attention.
__device__ __forceinline__ float delta_log_decay(float a, float a_log, float dt_bias) {
  return -expf(a_log) * softplus(a + dt_bias);
}
__device__ __forceinline__ float gla_log_decay(float z, float inv_tau) { return -softplus(-z) * inv_tau; }

// ---------------------------------------------------------------------------
// Decode: one token per sequence.
// ---------------------------------------------------------------------------
constexpr int kRG = 8;  // query heads of one key/value head that a block takes

// LDS of a decode block, by role (floats).
constexpr int kDecodeLds = kRG * kMixMaxDim + 2 * kMixMaxDim + kRG * kSplitKeys + 256 * kRG;

// Keys [128 split, ...) of the current chunk against kRG query heads of key/value head g.
__device__ void attn_role(const MixDecode& m, int b, int item, float* lds) {
  const ChunkAttn& a = m.attn;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int R = a.heads / a.kv_heads, groups = (R + kRG - 1) / kRG;
  const int split = item % m.attn_splits, rest = item / m.attn_splits;
  const int rg = rest % groups, g = rest / groups;
  const int r0 = rg * kRG, nr = min(kRG, R - r0);
  const int pos = *m.d_pos, last = pos % a.chunk;  // ring row of the current token
  const int j0 = split * kSplitKeys;
  if (j0 > last) return;
  const int nk = min(last + 1 - j0, kSplitKeys);
  const int dim = a.dim, dp = a.dim_pad, half = a.rot.half;
  float* qs = lds;                       // [kRG][dp]
  float* kn = qs + kRG * dp;             // [dp] the current token's key, rotated
  float* vn = kn + dp;                   // [dp] ... as projected
  float* w = vn + dp;                    // [kRG][kSplitKeys]
  float* red = w + kRG * kSplitKeys;     // [256][kRG]
  const float* y = m.y + (size_t)b * m.ld_y;
  const float* yk = y + a.k_col + g * dim;
  const float* yq = y + a.q_col + (size_t)(g * R + r0) * dim;
  // rotate: one thread per value beyond the pairs' first halves
  for (int i = tid; i < dp; i += 256) {
    if (i < half) {
      float s, c;
      turn(pos, a.rot.freq[i], &s, &c);
      const float u = yk[i], v = yk[i + half];
      kn[i] = u * c - v * s;
      kn[i + half] = v * c + u * s;
      vn[i] = u;
      vn[i + half] = v;
      for (int r = 0; r < nr; ++r) {
        const float qu = yq[r * dim + i], qv = yq[r * dim + i + half];
        qs[r * dp + i] = qu * c - qv * s;
        qs[r * dp + i + half] = qv * c + qu * s;
      }
    } else if (i >= 2 * half) {
      kn[i] = vn[i] = i < dim ? yk[i] : 0.0f;
      for (int r = 0; r < nr; ++r) qs[r * dp + i] = i < dim ? yq[r * dim + i] : 0.0f;
    }
  }
  __syncthreads();
  float* kring = a.kring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;
  float* vring = a.vring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;
  const int own = last - j0;  // the current token's key in this split, if it is below nk
  if (rg == 0 && own < kSplitKeys)
    for (int i = tid; i < dp; i += 256) {
      kring[(size_t)last * dp + i] = kn[i];
      vring[(size_t)last * dp + i] = vn[i];
    }
  // scores: sixteen lanes to a key, four keys to a wavefront
  const int sub = lane >> 4, l16 = lane & 15;
#pragma unroll 2
  for (int j = wave * 4 + sub; j < (nk + 15) / 16 * 16; j += 16) {
    f4 kv[4];
    const bool in = j < nk && j != own;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = 4 * l16 + 64 * i;
      kv[i] = f4{0.f, 0.f, 0.f, 0.f};
      if (e < dp) {
        if (in) kv[i] = *reinterpret_cast<const f4*>(kring + (size_t)(j0 + j) * dp + e);
        else if (j == own) kv[i] = *reinterpret_cast<const f4*>(kn + e);
      }
    }
#pragma unroll
    for (int r = 0; r < kRG; ++r) {
      if (r >= nr) break;
      float s = 0.0f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int e = 4 * l16 + 64 * i;
        if (e < dp) {
          const f4 q = *reinterpret_cast<const f4*>(qs + r * dp + e);
          s += (kv[i].x * q.x + kv[i].y * q.y) + (kv[i].z * q.z + kv[i].w * q.w);
        }
      }
      s += __shfl_xor(s, 8, 64);
      s += __shfl_xor(s, 4, 64);
      s += __shfl_xor(s, 2, 64);
      s += __shfl_xor(s, 1, 64);
      if (l16 == 0 && j < nk) w[r * kSplitKeys + j] = sigmoid(s * a.scale + a.bias[g * R + r0 + r]);
    }
  }
  __syncthreads();
  // weighted values: a thread owns one value column and every kp-th key
  int cols = 1;
  while (cols < dim) cols <<= 1;
  const int parts = 256 / cols, d = tid % cols, part = tid / cols;
  float acc[kRG];
#pragma unroll
  for (int r = 0; r < kRG; ++r) acc[r] = 0.0f;
  if (d < dim) {
#pragma unroll 4
    for (int j = part; j < nk; j += parts) {
      const float v = j == own ? vn[d] : vring[(size_t)(j0 + j) * dp + d];
#pragma unroll
      for (int r = 0; r < kRG; ++r)
        if (r < nr) acc[r] += w[r * kSplitKeys + j] * v;
    }
  }
#pragma unroll
  for (int r = 0; r < kRG; ++r) red[(r * parts + part) * cols + d] = acc[r];
  __syncthreads();
  for (int i = tid; i < nr * cols; i += 256) {
    const int r = i / cols, dd = i - r * cols;
    if (dd >= dim) continue;
    float s = 0.0f;
    for (int p = 0; p < parts; ++p) s += red[(r * parts + p) * cols + dd];
    const int h = g * R + r0 + r;
    if (m.attn_splits > 1)
      m.part[(((size_t)b * m.attn_splits + split) * a.heads + h) * dim + dd] = s;
    else
      m.out[(size_t)b * m.ld_out + a.out_col + h * dim + dd] = s * a.out_scale;
  }
}

// One head of the recurrence.  A thread owns column v of the state and every `parts`-th of its
// rows, RPT of them, in registers.
template <int RPT>
__device__ void recurrence_role(const MixDecode& m, int b, int h, float* lds) {
  const Recurrence& c = m.rec;
  const int tid = threadIdx.x;
  const int dim = c.dim, vdim = c.vdim;
  int cols = 1;
  while (cols < vdim) cols <<= 1;
  const int parts = 256 / cols, v = tid % cols, part = tid / cols;
  float* qs = lds;                 // [256]
  float* ks = qs + 256;            // [256]
  float* vs = ks + 256;            // [256]
  float* al = vs + 256;            // [256] decay per key channel
  float* red = al + 256;           // [256]
  float* red4 = red + 256;         // [4]
  const int pos = *m.d_pos;
  const float* y = m.y + (size_t)b * m.ld_y;
  float* S = c.state + (size_t)b * c.state_seq + (size_t)h * dim * vdim;
  float st[RPT];
  // (at position 0 the state is zero whatever the memory holds)
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    const int i = part + parts * j;
    st[j] = pos > 0 && v < vdim && i < dim ? S[(size_t)i * vdim + v] : 0.0f;
  }
  const int kvh = h / (c.heads / c.kv_heads);
  float beta = 1.0f, g = 1.0f;
  if (c.delta) {
    const ShortConv& cv = c.conv;
    float* ring = cv.ring + (size_t)b * cv.ring_seq;
    const int slot = pos % cv.taps;
    // channel ch of the convolution; the row of this position goes to the ring (no block reads it
    // in this step)
    auto conv = [&](int ch, bool keep) {
      const float cur = y[cv.col + ch];
      float s = cv.w[ch * cv.taps + cv.taps - 1] * cur;
      for (int j = 1; j < cv.taps; ++j)
        if (pos >= j)
          s += cv.w[ch * cv.taps + cv.taps - 1 - j] * ring[(size_t)((pos - j) % cv.taps) * cv.channels + ch];
      if (keep) ring[(size_t)slot * cv.channels + ch] = cur;
      return silu(s);
    };
    const bool first = h % (c.heads / c.kv_heads) == 0;
    float qv = 0.0f, kv = 0.0f;
    if (tid < dim) {
      qv = conv(c.q_col - cv.col + kvh * dim + tid, first);
      kv = conv(c.k_col - cv.col + kvh * dim + tid, first);
    }
    if (tid < vdim) vs[tid] = conv(c.v_col - cv.col + h * vdim + tid, true);
    const float qn = block_sum(qv * qv, red4), kn = block_sum(kv * kv, red4);
    qs[tid] = qv / sqrtf(qn + 1e-6f) * c.q_scale;
    ks[tid] = kv / sqrtf(kn + 1e-6f);
    beta = sigmoid(y[c.b_col + h]);
    g = expf(delta_log_decay(y[c.a_col + h], c.a_log[h], c.dt_bias[h]));
    al[tid] = g;
  } else {
    float qv = 0.0f, kv = 0.0f, av = 1.0f;
    if (tid < dim) {
      qv = y[c.q_col + h * dim + tid] * c.q_scale;
      kv = y[c.k_col + h * dim + tid];
      const float* a2 = c.a2 + (size_t)(h * dim + tid) * c.rank;
      float z = c.a2_bias[h * dim + tid];
      for (int r = 0; r < c.rank; ++r) z += a2[r] * y[c.a_col + r];
      av = expf(gla_log_decay(z, c.inv_tau));
    }
    qs[tid] = qv;
    ks[tid] = kv;
    al[tid] = av;
    if (tid < vdim) vs[tid] = y[c.v_col + h * vdim + tid];
  }
  __syncthreads();
  float u = v < vdim ? vs[v] : 0.0f;
  if (c.delta) {
    float s = 0.0f;
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      const int i = part + parts * j;
      st[j] *= g;
      if (i < dim) s += st[j] * ks[i];
    }
    red[tid] = s;
    __syncthreads();
    s = 0.0f;
    for (int p = 0; p < parts; ++p) s += red[p * cols + v];
    u = beta * (u - s);
    __syncthreads();
  }
  float o = 0.0f;
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    const int i = part + parts * j;
    if (i < dim) {
      st[j] = (c.delta ? st[j] : st[j] * al[i]) + ks[i] * u;
      o += st[j] * qs[i];
      if (v < vdim) S[(size_t)i * vdim + v] = st[j];
    }
  }
  red[tid] = o;
  __syncthreads();
  float out = 0.0f;
  if (tid < vdim)
    for (int p = 0; p < parts; ++p) out += red[p * cols + tid];
  const float ss = block_sum(out * out, red4);
  if (tid < vdim)
    m.out[(size_t)b * m.ld_out + c.out_col + h * vdim + tid] =
        out / sqrtf(ss / (float)vdim + c.eps) * c.norm[tid] * silu(y[c.g_col + h * vdim + tid]) * c.out_scale;
}

template <int RPT>
__global__ __launch_bounds__(256) void k_mix_decode(MixDecode m, int attn_items, int rec_items) {
  __shared__ __attribute__((aligned(16))) float lds[kDecodeLds];
  const int b = blockIdx.y;
  int item = blockIdx.x;
  if (item < rec_items) {
    recurrence_role<RPT>(m, b, item, lds);
    return;
  }
  item -= rec_items;
  if (item < attn_items) {
    attn_role(m, b, item, lds);
    return;
  }
  item -= attn_items;
  const int j = item * 256 + threadIdx.x;
  if (j >= m.mlp.ff_pad) return;
  const float* y = m.y + (size_t)b * m.ld_y;
  m.act[(size_t)b * m.mlp.ff_pad + j] =
      j < m.mlp.ff ? gelu_tanh(y[m.mlp.gate_col + j]) * y[m.mlp.up_col + j] : 0.0f;
}

__global__ __launch_bounds__(256) void k_attn_sum(MixDecode m) {
  const ChunkAttn& a = m.attn;
  const int b = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x, n = a.heads * a.dim;
  if (i >= n) return;
  const int splits = (*m.d_pos % a.chunk) / kSplitKeys + 1;
  const float* p = m.part + (size_t)b * m.attn_splits * n + i;
  float s = 0.0f;
#pragma unroll 4
  for (int k = 0; k < splits; ++k) s += p[(size_t)k * n];
  m.out[(size_t)b * m.ld_out + a.out_col + i] = s * a.out_scale;
}

// ---------------------------------------------------------------------------
// Many rows.
// ---------------------------------------------------------------------------
__global__ __launch_bounds__(256) void k_rotary_rows(MixRows r, ChunkAttn a) {
  __shared__ float cs[kMixMaxDim / 2], sn[kMixMaxDim / 2];
  const int row = blockIdx.x, pos = r.pos0 + row % r.n;
  const int half = a.rot.half, dim = a.dim;
  for (int i = threadIdx.x; i < half; i += 256) turn(pos, a.rot.freq[i], &sn[i], &cs[i]);
  __syncthreads();
  float* y = r.y + (size_t)row * r.ld_y;
  float* kr = r.k_rot + (size_t)row * a.kv_heads * dim;
  const int per = dim - half;  // pairs, then the values that pass
  for (int idx = threadIdx.x; idx < (a.heads + a.kv_heads) * per; idx += 256) {
    const int h = idx / per, e = idx - h * per;
    const bool is_k = h >= a.heads;
    float* src = is_k ? y + a.k_col + (h - a.heads) * dim : y + a.q_col + h * dim;
    float* dst = is_k ? kr + (h - a.heads) * dim : src;
    if (e < half) {
      const float u = src[e], v = src[e + half];
      dst[e] = u * cs[e] - v * sn[e];
      dst[e + half] = v * cs[e] + u * sn[e];
    } else if (is_k) {
      dst[e + half] = src[e + half];
    }
  }
}

// A block of four wavefronts owns 128 queries of one head, 32 to a wavefront, and walks the keys
// from the first query's chunk start to the last query, 32 at a time, staged in LDS:
//   S^T (keys x queries) = K . Q^T, Q in registers (lane (l, half) holds dims half DP/2 ..)
//   weights sigmoid(S scale + bias), 0 outside the query's chunk and after the query
//   O^T (dims x queries) += V^T . P^T, a lane's own weights are the operand
// Keys before pos0 come from the ring, the others from this step's rows.
template <int DP>
__global__ __launch_bounds__(256) void k_chunk_attn_rows(MixRows r, ChunkAttn a) {
  constexpr int KT = 32, LD = DP + 4, NB = DP / 32, NL = KT * DP / 4 / 256;
  __shared__ __attribute__((aligned(16))) float Ks[KT][LD];
  __shared__ __attribute__((aligned(16))) float Vs[KT][LD];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int half = lane >> 5, l32 = lane & 31;
  const int h = blockIdx.x, b = blockIdx.z, g = h / (a.heads / a.kv_heads);
  const int nqb = (r.n + 127) / 128;
  const int t0 = (nqb - 1 - (int)blockIdx.y) * 128;  // first query of the block
  const int tq = t0 + 32 * wave + l32;               // this lane's query
  const int dim = a.dim, dp = a.dim_pad;
  const size_t row0 = (size_t)b * r.n;
  const float* yb = r.y + row0 * r.ld_y;
  const float* krb = r.k_rot + row0 * a.kv_heads * dim + g * dim;
  const float* kring = a.kring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;
  const float* vring = a.vring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;

  float qr[DP / 2];
  {
    const float* q = yb + (size_t)min(tq, r.n - 1) * r.ld_y + a.q_col + h * dim;
#pragma unroll
    for (int s = 0; s < DP / 2; ++s) {
      const int d = half * (DP / 2) + s;
      qr[s] = d < dim ? q[d] : 0.0f;
    }
  }
  f16v o[NB];
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) o[i][v] = 0.0f;

  const int pq = r.pos0 + tq;                 // positions
  const int lo = pq - pq % a.chunk;           // first key this lane's query sees
  const int pb0 = r.pos0 + t0, pb1 = r.pos0 + min(t0 + 128, r.n) - 1;
  const int kfirst = pb0 - pb0 % a.chunk;
  const int tiles = (pb1 - kfirst) / KT + 1;
  // this wavefront's queries
  const int w0 = t0 + 32 * wave, wp0 = r.pos0 + w0, wp1 = r.pos0 + min(w0 + 32, r.n) - 1;
  const int wlo0 = wp0 - wp0 % a.chunk, wlo1 = wp1 - max(wp1, 0) % a.chunk;
  const float bias = a.bias[h];
  const bool vec = (dim & 3) == 0;

  f4 kreg[NL], vreg[NL];
  auto fetch = [&](int tile) {
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int idx = tid + 256 * i, key = idx / (DP / 4), d = (idx % (DP / 4)) * 4;
      const int p = kfirst + tile * KT + key;
      f4 k = f4{0.f, 0.f, 0.f, 0.f}, v = k;
      if (p <= pb1 && d < dp) {
        if (p < r.pos0) {
          const size_t at = (size_t)(p % a.chunk) * dp + d;
          k = *reinterpret_cast<const f4*>(kring + at);
          v = *reinterpret_cast<const f4*>(vring + at);
        } else {
          const int t = p - r.pos0;
          const float* kp = krb + (size_t)t * a.kv_heads * dim + d;
          const float* vp = yb + (size_t)t * r.ld_y + a.k_col + g * dim + d;
          if (vec) {
            k = *reinterpret_cast<const f4*>(kp);
            v = *reinterpret_cast<const f4*>(vp);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (d + e < dim) {
                k[e] = kp[e];
                v[e] = vp[e];
              }
          }
        }
      }
      kreg[i] = k;
      vreg[i] = v;
    }
  };
  fetch(0);
  for (int tile = 0; tile < tiles; ++tile) {
    if (tile) __syncthreads();  // the last tile has been read
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int idx = tid + 256 * i, key = idx / (DP / 4), d = (idx % (DP / 4)) * 4;
      *reinterpret_cast<f4*>(&Ks[key][d]) = kreg[i];
      *reinterpret_cast<f4*>(&Vs[key][d]) = vreg[i];
    }
    __syncthreads();
    if (tile + 1 < tiles) fetch(tile + 1);
    const int k0 = kfirst + tile * KT;
    if (w0 >= r.n || k0 > wp1 || k0 + KT - 1 < wlo0) continue;  // (wavefront-uniform)
    f16v s0, s1;
#pragma unroll
    for (int v = 0; v < 16; ++v) s0[v] = s1[v] = 0.0f;
    const f4* krow = reinterpret_cast<const f4*>(&Ks[l32][half * (DP / 2)]);
#pragma unroll
    for (int j = 0; j < DP / 8; ++j) {
      const f4 k = krow[j];
      s0 = __builtin_amdgcn_mfma_f32_32x32x2f32(k.x, qr[4 * j], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_32x32x2f32(k.y, qr[4 * j + 1], s1, 0, 0, 0);
      s0 = __builtin_amdgcn_mfma_f32_32x32x2f32(k.z, qr[4 * j + 2], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_32x32x2f32(k.w, qr[4 * j + 3], s1, 0, 0, 0);
    }
    s0 += s1;
    // lane holds keys k0 + 8 (v / 4) + 4 half + v % 4 of its query
    const bool edge = k0 + KT - 1 > wp0 || k0 < wlo1;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int key = k0 + 8 * (v >> 2) + 4 * half + (v & 3);
      const float z = s0[v] * a.scale + bias;
      const float wgt = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.44269504088896341f * z));
      s0[v] = !edge || (key <= pq && key >= lo) ? wgt : 0.0f;
    }
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int key = 8 * (v >> 2) + 4 * half + (v & 3);
#pragma unroll
      for (int i = 0; i < NB; ++i)
        o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(Vs[key][32 * i + l32], s0[v], o[i], 0, 0, 0);
    }
  }
  if (tq >= r.n) return;
  float* dst = r.out + (row0 + tq) * r.ld_out + a.out_col + h * dim;
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int d = 32 * i + 8 * (v >> 2) + 4 * half + (v & 3);
      if (d < dim) dst[d] = o[i][v] * a.out_scale;
    }
}

__global__ __launch_bounds__(256) void k_short_conv_rows(MixRows r, ShortConv c) {
  const int ch = blockIdx.x * 256 + threadIdx.x, row = blockIdx.y;
  if (ch >= c.channels) return;
  const int b = row / r.n, t = row - b * r.n, pos = r.pos0 + t;
  const float* w = c.w + ch * c.taps;
  const float* ring = c.ring + (size_t)b * c.ring_seq;
  float s = 0.0f;
  for (int j = 0; j < c.taps; ++j) {
    if (pos < j) break;
    const float x = t >= j ? r.y[(size_t)(row - j) * r.ld_y + c.col + ch]
                           : ring[(size_t)((pos - j) % c.taps) * c.channels + ch];
    s += w[c.taps - 1 - j] * x;
  }
  r.conv_out[(size_t)row * c.channels + ch] = silu(s);
}

// log alpha of gated linear attention
__global__ __launch_bounds__(256) void k_gla_decay_rows(MixRows r, Recurrence c) {
  const int i = blockIdx.x * 256 + threadIdx.x, row = blockIdx.y, n = c.heads * c.dim;
  if (i >= n) return;
  const float* a1 = r.y + (size_t)row * r.ld_y + c.a_col;
  float z = c.a2_bias[i];
  for (int k = 0; k < c.rank; ++k) z += c.a2[(size_t)i * c.rank + k] * a1[k];
  r.decay[(size_t)row * n + i] = gla_log_decay(z, c.inv_tau);
}

// The recurrence token by token; a block owns one head of one sequence (layout of
// recurrence_role).
template <int RPT>
__global__ __launch_bounds__(256) void k_recurrence_scan(MixRows r, Recurrence c) {
  __shared__ float qs[256], ks[256], vs[256], al[256], red[256], red4[4];
  const int tid = threadIdx.x, h = blockIdx.x, b = blockIdx.y;
  const int dim = c.dim, vdim = c.vdim;
  int cols = 1;
  while (cols < vdim) cols <<= 1;
  const int parts = 256 / cols, v = tid % cols, part = tid / cols;
  float* S = c.state + (size_t)b * c.state_seq + (size_t)h * dim * vdim;
  float st[RPT];
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    const int i = part + parts * j;
    st[j] = r.pos0 > 0 && v < vdim && i < dim ? S[(size_t)i * vdim + v] : 0.0f;
  }
  const int kvh = h / (c.heads / c.kv_heads);
  for (int t = 0; t < r.n; ++t) {
    const size_t row = (size_t)b * r.n + t;
    const float* y = r.y + row * r.ld_y;
    float beta = 1.0f, g = 1.0f;
    if (c.delta) {
      const float* x = r.conv_out + row * c.conv.channels;
      float qv = 0.0f, kv = 0.0f;
      if (tid < dim) {
        qv = x[c.q_col - c.conv.col + kvh * dim + tid];
        kv = x[c.k_col - c.conv.col + kvh * dim + tid];
      }
      const float qn = block_sum(qv * qv, red4), kn = block_sum(kv * kv, red4);
      qs[tid] = qv / sqrtf(qn + 1e-6f) * c.q_scale;
      ks[tid] = kv / sqrtf(kn + 1e-6f);
      if (tid < vdim) vs[tid] = x[c.v_col - c.conv.col + h * vdim + tid];
      beta = sigmoid(y[c.b_col + h]);
      g = expf(delta_log_decay(y[c.a_col + h], c.a_log[h], c.dt_bias[h]));
    } else {
      if (tid < dim) {
        qs[tid] = y[c.q_col + h * dim + tid] * c.q_scale;
        ks[tid] = y[c.k_col + h * dim + tid];
        al[tid] = expf(r.decay[row * c.heads * dim + h * dim + tid]);
      }
      if (tid < vdim) vs[tid] = y[c.v_col + h * vdim + tid];
    }
    __syncthreads();
    float u = v < vdim ? vs[v] : 0.0f;
    if (c.delta) {
      float s = 0.0f;
#pragma unroll
      for (int j = 0; j < RPT; ++j) {
        const int i = part + parts * j;
        st[j] *= g;
        if (i < dim) s += st[j] * ks[i];
      }
      red[tid] = s;
      __syncthreads();
      s = 0.0f;
      for (int p = 0; p < parts; ++p) s += red[p * cols + v];
      u = beta * (u - s);
      __syncthreads();
    }
    float o = 0.0f;
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      const int i = part + parts * j;
      if (i < dim) {
        st[j] = (c.delta ? st[j] : st[j] * al[i]) + ks[i] * u;
        o += st[j] * qs[i];
      }
    }
    red[tid] = o;
    __syncthreads();
    if (tid < vdim) {
      float out = 0.0f;
      for (int p = 0; p < parts; ++p) out += red[p * cols + tid];
      r.o[row * c.heads * vdim + h * vdim + tid] = out;
    }
    __syncthreads();
  }
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    const int i = part + parts * j;
    if (v < vdim && i < dim) S[(size_t)i * vdim + v] = st[j];
  }
}

// One wavefront per (row, head).
__global__ __launch_bounds__(256) void k_gated_norm_rows(MixRows r, Recurrence c, int rows) {
  const int lane = threadIdx.x & 63;
  const int item = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= rows * c.heads) return;
  const int row = item / c.heads, h = item - row * c.heads;
  const float* o = r.o + (size_t)item * c.vdim;
  float x[kMixMaxDim / 64], ss = 0.0f;
#pragma unroll
  for (int j = 0; j < kMixMaxDim / 64; ++j) {
    const int e = lane + 64 * j;
    x[j] = e < c.vdim ? o[e] : 0.0f;
    ss += x[j] * x[j];
  }
  const float inv = c.out_scale / sqrtf(wave_sum(ss) / (float)c.vdim + c.eps);
  const float* gate = r.y + (size_t)row * r.ld_y + c.g_col + h * c.vdim;
  float* dst = r.out + (size_t)row * r.ld_out + c.out_col + h * c.vdim;
#pragma unroll
  for (int j = 0; j < kMixMaxDim / 64; ++j) {
    const int e = lane + 64 * j;
    if (e < c.vdim) dst[e] = x[j] * inv * c.norm[e] * silu(gate[e]);
  }
  if (h == 0)
    for (int e = r.out_cols + lane; e < r.ld_out; e += 64) r.out[(size_t)row * r.ld_out + e] = 0.0f;
}

__global__ __launch_bounds__(256) void k_gated_mlp_rows(MixRows r, GatedMlp m) {
  const int j = blockIdx.x * 256 + threadIdx.x;
  const size_t row = blockIdx.y;
  if (j >= m.ff_pad) return;
  const float* y = r.y + row * r.ld_y;
  r.act[row * m.ff_pad + j] = j < m.ff ? gelu_tanh(y[m.gate_col + j]) * y[m.up_col + j] : 0.0f;
}

// x: position in the last rows, y: sequence
__global__ __launch_bounds__(256) void k_commit_rows(MixRows r, ChunkAttn a, ShortConv c, int attn_rows,
                                                     int conv_rows) {
  const int b = blockIdx.y, back = blockIdx.x;  // tokens back from the last one
  const int t = r.n - 1 - back, pos = r.pos0 + t;
  const size_t row = (size_t)b * r.n + t;
  if (back < attn_rows) {
    const int dim = a.dim, dp = a.dim_pad;
    float* kring = a.kring + (size_t)b * a.ring_seq;
    float* vring = a.vring + (size_t)b * a.ring_seq;
    for (int i = threadIdx.x; i < a.kv_heads * dp; i += 256) {
      const int g = i / dp, d = i - g * dp;
      const size_t at = ((size_t)g * a.chunk + pos % a.chunk) * dp + d;
      kring[at] = d < dim ? r.k_rot[row * a.kv_heads * dim + g * dim + d] : 0.0f;
      vring[at] = d < dim ? r.y[row * r.ld_y + a.k_col + g * dim + d] : 0.0f;
    }
  }
  if (back < conv_rows) {
    float* ring = c.ring + (size_t)b * c.ring_seq + (size_t)(pos % c.taps) * c.channels;
    for (int i = threadIdx.x; i < c.channels; i += 256) ring[i] = r.y[row * r.ld_y + c.col + i];
  }
}

__global__ __launch_bounds__(256) void k_rms_rows(const float* src, float* dst, int cols, int ld,
                                                  const float* gain, float eps, float scale,
                                                  const int* rows_at) {
  __shared__ float red[4];
  const size_t at = rows_at ? rows_at[blockIdx.x] : blockIdx.x;
  const float* x = src + at * ld;
  float* y = dst + (size_t)blockIdx.x * ld;
  float ss = 0.0f;
  for (int i = threadIdx.x; i < cols; i += 256) ss += x[i] * x[i];
  const float k = gain[0] * scale / sqrtf(block_sum(ss, red) / (float)cols + eps);
  for (int i = threadIdx.x; i < ld; i += 256) y[i] = i < cols ? x[i] * k : 0.0f;
}

__global__ void k_set_int(int* p, int value) { *p = value; }
__global__ void k_add_one(int* p) { *p += 1; }

// Rows of a state column per thread (kernels with RPT): the next power of two.
int rows_per_thread(int dim, int vdim) {
  int cols = 1;
  while (cols < vdim) cols <<= 1;
  const int need = (dim + 256 / cols - 1) / (256 / cols);
  int rpt = 4;
  while (rpt < need) rpt <<= 1;
  return rpt;
}

}  // namespace

int attn_decode_splits(int chunk) { return (chunk + kSplitKeys - 1) / kSplitKeys; }

hipError_t launch_mix_decode(const MixDecode& a, hipStream_t s) {
  int attn_items = 0;
  if (a.has_attn) {
    const int R = a.attn.heads / a.attn.kv_heads;
    attn_items = a.attn.kv_heads * ((R + kRG - 1) / kRG) * a.attn_splits;
  }
  const int rec_items = a.has_rec ? a.rec.heads : 0;
  const int mlp_items = a.has_mlp ? (a.mlp.ff_pad + 255) / 256 : 0;
  const dim3 grid((unsigned)(attn_items + rec_items + mlp_items), (unsigned)a.nseq);
  if (grid.x == 0) return hipSuccess;
  switch (a.has_rec ? rows_per_thread(a.rec.dim, a.rec.vdim) : 4) {
#define PG_RPT(N)                                                                        \
  case N:                                                                                \
    hipLaunchKernelGGL(k_mix_decode<N>, grid, dim3(256), 0, s, a, attn_items, rec_items); \
    break;
    PG_RPT(4) PG_RPT(8) PG_RPT(16) PG_RPT(32) PG_RPT(64) PG_RPT(128) PG_RPT(256)
#undef PG_RPT
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

hipError_t launch_attn_sum(const MixDecode& a, hipStream_t s) {
  const int n = a.attn.heads * a.attn.dim;
  hipLaunchKernelGGL(k_attn_sum, dim3((n + 255) / 256, a.nseq), dim3(256), 0, s, a);
  return hipGetLastError();
}

hipError_t launch_rotary_rows(const MixRows& r, const ChunkAttn& a, hipStream_t s) {
  hipLaunchKernelGGL(k_rotary_rows, dim3(r.nseq * r.n), dim3(256), 0, s, r, a);
  return hipGetLastError();
}

hipError_t launch_chunk_attn_rows(const MixRows& r, const ChunkAttn& a, hipStream_t s) {
  const dim3 grid(a.heads, (r.n + 127) / 128, r.nseq);
  const int dp = (a.dim + 31) / 32 * 32;
  switch (dp) {
#define PG_DP(N)                                                                   \
  case N:                                                                          \
    hipLaunchKernelGGL(k_chunk_attn_rows<N>, grid, dim3(256), 0, s, r, a);          \
    break;
    PG_DP(32) PG_DP(64) PG_DP(96) PG_DP(128) PG_DP(160) PG_DP(192) PG_DP(224) PG_DP(256)
#undef PG_DP
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

hipError_t launch_short_conv_rows(const MixRows& r, const ShortConv& c, hipStream_t s) {
  hipLaunchKernelGGL(k_short_conv_rows, dim3((c.channels + 255) / 256, r.nseq * r.n), dim3(256), 0, s, r, c);
  return hipGetLastError();
}

hipError_t launch_recurrence_rows(const MixRows& r, const Recurrence& c, hipStream_t s) {
  if (!c.delta)
    hipLaunchKernelGGL(k_gla_decay_rows, dim3((c.heads * c.dim + 255) / 256, r.nseq * r.n), dim3(256), 0, s, r, c);
  const dim3 grid(c.heads, r.nseq);
  switch (rows_per_thread(c.dim, c.vdim)) {
#define PG_RPT(N)                                                              \
  case N:                                                                      \
    hipLaunchKernelGGL(k_recurrence_scan<N>, grid, dim3(256), 0, s, r, c);      \
    break;
    PG_RPT(4) PG_RPT(8) PG_RPT(16) PG_RPT(32) PG_RPT(64) PG_RPT(128) PG_RPT(256)
#undef PG_RPT
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

hipError_t launch_gated_norm_rows(const MixRows& r, const Recurrence& c, hipStream_t s) {
  const int rows = r.nseq * r.n;
  hipLaunchKernelGGL(k_gated_norm_rows, dim3((rows * c.heads + 3) / 4), dim3(256), 0, s, r, c, rows);
  return hipGetLastError();
}

hipError_t launch_gated_mlp_rows(const MixRows& r, const GatedMlp& m, hipStream_t s) {
  hipLaunchKernelGGL(k_gated_mlp_rows, dim3((m.ff_pad + 255) / 256, r.nseq * r.n), dim3(256), 0, s, r, m);
  return hipGetLastError();
}

hipError_t launch_commit_rows(const MixRows& r, const ChunkAttn* a, const ShortConv* c, hipStream_t s) {
  int attn_rows = 0, conv_rows = 0;
  if (a) attn_rows = std::min(r.n, (r.pos0 + r.n - 1) % a->chunk + 1);
  if (c) conv_rows = std::min(r.n, c->taps - 1);
  const int rows = std::max(attn_rows, conv_rows);
  if (rows == 0) return hipSuccess;
  hipLaunchKernelGGL(k_commit_rows, dim3(rows, r.nseq), dim3(256), 0, s, r, a ? *a : ChunkAttn{},
                     c ? *c : ShortConv{}, attn_rows, conv_rows);
  return hipGetLastError();
}

hipError_t launch_rms_rows(const float* src, float* dst, int rows, int cols, int ld, const float* gain,
                           float eps, float scale, const int* rows_at, hipStream_t s) {
  hipLaunchKernelGGL(k_rms_rows, dim3(rows), dim3(256), 0, s, src, dst, cols, ld, gain, eps, scale, rows_at);
  return hipGetLastError();
}

hipError_t launch_set_int(int* p, int value, hipStream_t s) {
  hipLaunchKernelGGL(k_set_int, dim3(1), dim3(1), 0, s, p, value);
  return hipGetLastError();
}
hipError_t launch_add_one(int* p, hipStream_t s) {
  hipLaunchKernelGGL(k_add_one, dim3(1), dim3(1), 0, s, p);
  return hipGetLastError();
}

}  // namespace pgk
