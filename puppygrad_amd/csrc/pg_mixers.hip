// gfx950 kernels of the sequence mixers (pg_mixers.h): chunked sigmoid attention on the f32
// matrix cores, the recurrences, and the element-wise steps around them.  All arithmetic is f32
// (angles: the product position * frequency is reduced to one turn in f64).
//
// Shapes are checked on the host before any launch (pg_stack.cpp); kernels guard ragged tails.
#include "pg_mixers.h"

#include <math.h>

#include <algorithm>
#include <type_traits>

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

__device__ __forceinline__ f4 bf16x4(const unsigned short* p) {
  const uint2 u = *reinterpret_cast<const uint2*>(p);
  return f4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
            __uint_as_float(u.y & 0xffff0000u)};
}

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

// LDS of a decode block of NT threads (floats): the attention role's, the larger of the two.
template <int NT>
constexpr int kDecodeLds = 16 * (kMixMaxDim + 4) + 2 * kMixMaxDim + (NT / 64) * kRG * 64;

// Keys [NT / 4 split, ...) of the current chunk against kRG query heads of key/value head g, sixteen
// keys to a wavefront, on the f32 matrix cores (v_mfma_f32_16x16x4_f32: A operand lane l ->
// A[l % 16][l / 16], B operand lane l -> B[l / 16][l % 16], D lane l, register v -> D[4 (l / 16) + v][l % 16]):
//   S^T (keys x heads) = K . Q^T, lane (key, quarter) holding a quarter of the key's dims;
//   O (heads x dims) += W . V: register v of a lane, the weight of key 4 (l / 16) + v, is the operand
//   of step v as it is, against V's rows 4 (l / 16) + v.
// The wavefronts' sums are added through LDS.  Nothing that is loaded before the first barrier
// depends on another load but on the position.  NV: 64-dim parts of a head.
template <int NT, int NV>
__device__ void attn_role(const MixDecode& m, int b, int item, float* lds) {
  constexpr int SK = NT / 4, NW = NT / 64;
  constexpr int DQ = 16 * NV;           // dims of a lane's quarter, at most
  constexpr bool PREV = NV <= 2;        // values requested together with the keys
  typedef float f4v __attribute__((ext_vector_type(4)));
  const ChunkAttn& a = m.attn;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int l16 = lane & 15, quarter = lane >> 4;
  const int R = a.heads / a.kv_heads, groups = (R + kRG - 1) / kRG;
  const int split = item % m.attn_splits, rest = item / m.attn_splits;
  const int rg = rest % groups, g = rest / groups;
  const int r0 = rg * kRG, nr = min(kRG, R - r0);
  const int dim = a.dim, dp = a.dim_pad, half = a.rot.half;
  const int dq = (dim + 15) / 16 * 4;   // dims of a quarter
  const int j0 = split * SK;
  const float* kring = a.kring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;
  const float* vring = a.vring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;
  const int pos = *m.d_pos, last = pos % a.chunk;  // ring row of the current token
  if (j0 > last) {
    // (every split's sums are added: the ones without keys are 0)
    if (m.attn_splits > 1)
      for (int i = tid; i < nr * dim; i += NT)
        m.part[(((size_t)b * m.attn_splits + split) * a.heads + g * R + r0) * dim + i] = 0.0f;
    return;
  }
  const int nk = min(last + 1 - j0, SK);
  const int own = last - j0;            // the current token's key in this split, if it is below nk
  const int jk = 16 * wave + l16;       // this lane's key (scores)
  const bool active = 16 * wave < nk;   // (wavefront-uniform)
  f4 kv[4 * NV];
  float vv[4 * NV][4];
  auto fetch_v = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const float* row = vring + (size_t)(j0 + min(16 * wave + 4 * quarter + v, nk - 1)) * dp;
#pragma unroll
      for (int t = 0; t < 4 * NV; ++t) vv[t][v] = row[min(16 * t + l16, dp - 1)];
    }
  };
  if (active) {
    const float* row = kring + (size_t)(j0 + min(jk, nk - 1)) * dp;
#pragma unroll
    for (int i = 0; i < DQ / 4; ++i) kv[i] = *reinterpret_cast<const f4*>(row + min(quarter * dq + 4 * min(i, dq / 4 - 1), dp - 4));
    if (PREV) fetch_v();
  }
  constexpr int QLD = 64 * NV + 4;
  float* qs = lds;                      // [16][QLD], rows past nr and columns past dim are 0
  float* kn = qs + 16 * QLD;            // [256] the current token's key, rotated
  float* vn = kn + kMixMaxDim;          // [256] ... as projected
  float* red = vn + kMixMaxDim;         // [NW][kRG][64]
  const float* y = m.y + (size_t)b * m.ld_y;
  const float* yk = y + a.k_col + g * dim;
  const float* yq = y + a.q_col + (size_t)(g * R + r0) * dim;
  // a pair (or values that pass, two apart) per thread; row nr is the key
  const int per = 32 * NV;  // >= half, and 2 per >= dim
  for (int i = tid; i < 17 * per; i += NT) {
    const int r = i / per, e = i - r * per;
    const bool is_k = r == 16, live = r < nr || is_k;
    const float* src = is_k ? yk : yq + r * dim;
    float* dst = is_k ? kn : qs + r * QLD;
    if (e < half) {
      float u = 0.0f, v = 0.0f, s, c;
      if (live) {
        u = src[e];
        v = src[e + half];
      }
      turn(pos, a.rot.freq[e], &s, &c);
      dst[e] = u * c - v * s;
      dst[e + half] = v * c + u * s;
      if (is_k) {
        vn[e] = u;
        vn[e + half] = v;
      }
    }
    // the values past the pairs: 2 half + (e, and e + per)
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const int x = 2 * half + e + k * per;
      if (x < 64 * NV) {
        const float u = live && x < dim ? src[x] : 0.0f;
        dst[x] = u;
        if (is_k) vn[x] = u;
      }
    }
  }
  __syncthreads();
  if (rg == 0 && own < SK) {
    float* kw = a.kring + (size_t)b * a.ring_seq + ((size_t)g * a.chunk + last) * dp;
    float* vw = a.vring + (size_t)b * a.ring_seq + ((size_t)g * a.chunk + last) * dp;
    for (int i = tid; i < dp; i += NT) {
      kw[i] = kn[i];
      vw[i] = vn[i];
    }
  }
  f4v o[4 * NV];
#pragma unroll
  for (int t = 0; t < 4 * NV; ++t) o[t] = f4v{0.f, 0.f, 0.f, 0.f};
  if (active) {
    f4v s = f4v{0.f, 0.f, 0.f, 0.f};
    const float* q = qs + l16 * QLD + quarter * dq;
    const float* ko = kn + quarter * dq;
#pragma unroll
    for (int i = 0; i < DQ / 4; ++i) {
      if (4 * i >= dq) break;
      f4 k4 = kv[i];
      if (jk == own) k4 = *reinterpret_cast<const f4*>(ko + 4 * i);
      const f4 q4 = *reinterpret_cast<const f4*>(q + 4 * i);
#pragma unroll
      for (int e = 0; e < 4; ++e) s = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[e], q4[e], s, 0, 0, 0);
    }
    if (!PREV) fetch_v();
    const float bias = a.bias[g * R + r0 + min(l16, nr - 1)];
    float w[4];
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int j = 16 * wave + 4 * quarter + v;
      w[v] = j < nk ? sigmoid(s[v] * a.scale + bias) : 0.0f;
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const bool mine = 16 * wave + 4 * quarter + v == own;
#pragma unroll
      for (int t = 0; t < 4 * NV; ++t) {
        const float x = mine ? vn[16 * t + l16] : vv[t][v];
        o[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[v], x, o[t], 0, 0, 0);
      }
    }
  }
  // rows (heads) 4 quarter + v, dims 16 t + l16; 64 dims at a time
#pragma unroll
  for (int p = 0; p < NV; ++p) {
    if (64 * p >= dim) break;
    if (p) __syncthreads();
    if (quarter < kRG / 4)
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int v = 0; v < 4; ++v) red[(wave * kRG + 4 * quarter + v) * 64 + 16 * t + l16] = o[4 * p + t][v];
    __syncthreads();
    for (int i = tid; i < nr * 64; i += NT) {
      const int r = i >> 6, d = 64 * p + (i & 63);
      if (d >= dim) continue;
      float sum = 0.0f;
#pragma unroll
      for (int w = 0; w < NW; ++w) sum += red[w * kRG * 64 + i];
      const int h = g * R + r0 + r;
      if (m.attn_splits > 1)
        m.part[(((size_t)b * m.attn_splits + split) * a.heads + h) * dim + d] = sum * a.out_scale;
      else
        m.out[(size_t)b * m.ld_out + a.out_col + h * dim + d] = sum * a.out_scale;
    }
  }
}

// N channels ch[] of a short convolution at position pos, and the ring rows of this position
// (where keep[]; no block reads them in this step).  With up to four taps everything is loaded
// before the first value is used.
template <int N>
__device__ __forceinline__ void conv_channels(const ShortConv& c, const float* y, float* ring, const int (&ch)[N],
                                              const bool (&keep)[N], int pos, float (&out)[N]) {
  float cur[N];
#pragma unroll
  for (int n = 0; n < N; ++n) cur[n] = y[c.col + ch[n]];
  const int slot = pos % c.taps;
  if (c.taps <= 4) {
    float x[N][4], w[N][4];
#pragma unroll
    for (int n = 0; n < N; ++n)
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const int kk = min(k, c.taps - 1);
        x[n][k] = ring[(size_t)kk * c.channels + ch[n]];  // the input whose position is k modulo taps
        w[n][k] = c.w[ch[n] * c.taps + kk];
      }
#pragma unroll
    for (int n = 0; n < N; ++n) {
      float s = c.bias ? c.bias[ch[n]] : 0.0f;
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        int j = slot - k;  // tokens back
        if (j < 0) j += c.taps;
        const float in = k >= c.taps || pos < j ? 0.0f : j == 0 ? cur[n] : x[n][k];
        float wt = w[n][0];
#pragma unroll
        for (int i = 1; i < 4; ++i) wt = i == c.taps - 1 - j ? w[n][i] : wt;
        s += wt * in;
      }
      out[n] = silu(s);
    }
  } else {
#pragma unroll
    for (int n = 0; n < N; ++n) {
      float s = (c.bias ? c.bias[ch[n]] : 0.0f) + c.w[ch[n] * c.taps + c.taps - 1] * cur[n];
      for (int j = 1; j < c.taps; ++j)
        if (pos >= j)
          s += c.w[ch[n] * c.taps + c.taps - 1 - j] * ring[(size_t)((pos - j) % c.taps) * c.channels + ch[n]];
      out[n] = silu(s);
    }
  }
#pragma unroll
  for (int n = 0; n < N; ++n)
    if (keep[n]) ring[(size_t)slot * c.channels + ch[n]] = cur[n];
}

// Rows row0 .. row0 + n - 1 of a low-rank projection, eight lanes to a row: the first 128 rows
// and 128 columns of them are asked for by load() and used by store().  (The two kinds of
// weights part ways around whole runs of loads: a branch per load would wait for each.)
template <int NT>
struct LowRankRows {
  static constexpr int R = 1024 / NT, C = 4, STEP = NT / 8;
  f4 w[R][C], x[C];  // (bf16 weights: in the first two words as they are)
  static __device__ __forceinline__ f4 widened(const f4& raw, int bf16) {
    const unsigned a = __float_as_uint(raw.x), b = __float_as_uint(raw.y);
    return bf16 ? f4{__uint_as_float(a << 16), __uint_as_float(a & 0xffff0000u), __uint_as_float(b << 16),
                     __uint_as_float(b & 0xffff0000u)}
                : raw;
  }
  __device__ __forceinline__ void load(const LowRank& p, const float* y, int row0, int n) {
    const int i0 = threadIdx.x >> 3, k0 = 4 * (threadIdx.x & 7);
#pragma unroll
    for (int c = 0; c < C; ++c) x[c] = *reinterpret_cast<const f4*>(y + p.col + min(k0 + 32 * c, p.rank - 4));
    auto at = [&](int q, int c) __attribute__((always_inline)) {
      return (size_t)(row0 + min(i0 + q * STEP, n - 1)) * p.rank + min(k0 + 32 * c, p.rank - 4);
    };
    if (p.w_bf16) {
#pragma unroll
      for (int q = 0; q < R; ++q)
#pragma unroll
        for (int c = 0; c < C; ++c) {
          const float2 v = *reinterpret_cast<const float2*>(static_cast<const unsigned short*>(p.w) + at(q, c));
          w[q][c].x = v.x;
          w[q][c].y = v.y;
        }
    } else {
#pragma unroll
      for (int q = 0; q < R; ++q)
#pragma unroll
        for (int c = 0; c < C; ++c) w[q][c] = *reinterpret_cast<const f4*>(static_cast<const float*>(p.w) + at(q, c));
    }
  }
  // dst[i] = row row0 + i
  __device__ __forceinline__ void store(const LowRank& p, const float* y, int row0, int n, float* dst) const {
    const int i0 = threadIdx.x >> 3, sub = threadIdx.x & 7;
    auto dot = [](const f4& a, const f4& b) { return (a.x * b.x + a.y * b.y) + (a.z * b.z + a.w * b.w); };
    auto finish = [&](int i, float s) __attribute__((always_inline)) {
#pragma unroll
      for (int off = 4; off > 0; off >>= 1) s += __shfl_xor(s, off, 64);
      if (sub == 0 && i < n) dst[i] = s;
    };
    auto rest = [&](int i, int k0, float s) __attribute__((always_inline)) {
      const size_t at = (size_t)(row0 + min(i, n - 1)) * p.rank;
      for (int k = k0 + 4 * sub; k < p.rank; k += 32) {
        const f4 v = p.w_bf16 ? bf16x4(static_cast<const unsigned short*>(p.w) + at + k)
                              : *reinterpret_cast<const f4*>(static_cast<const float*>(p.w) + at + k);
        s += dot(v, *reinterpret_cast<const f4*>(y + p.col + k));
      }
      return s;
    };
#pragma unroll
    for (int q = 0; q < R; ++q) {
      float s = 0.0f;
#pragma unroll
      for (int c = 0; c < C; ++c)
        if (32 * c < p.rank) s += dot(widened(w[q][c], p.w_bf16), x[c]);
      finish(i0 + q * STEP, p.rank > 32 * C ? rest(i0 + q * STEP, 32 * C, s) : s);
    }
    for (int r0 = R * STEP; r0 < n; r0 += STEP) finish(r0 + i0, rest(r0 + i0, 0, 0.0f));
  }
};

// One head of the recurrence.  A thread owns column v of the state and every `parts`-th of its
// rows, RPT of them, in registers (parts * RPT <= kMixMaxDim; q and k are 0 past dim).
// KIND: a RecurrenceKind, or -1 for REC_GLA or REC_DELTA as m.rec.kind says.
template <int NT, int RPT, int KIND = -1>
__device__ void recurrence_role(const MixDecode& m, int b, int h, float* lds) {
  const Recurrence& c = m.rec;
  const bool delta = KIND < 0 ? c.kind == REC_DELTA : rec_reads_state(KIND);
  constexpr bool kChannel = KIND == REC_CHANNEL_DELTA, kSsd = KIND == REC_SSD;
  const int tid = threadIdx.x;
  const int dim = c.dim, vdim = c.vdim;
  int cols = 1;
  while (cols < vdim) cols <<= 1;
  const int parts = NT / cols, v = tid % cols, part = tid / cols;
  float* qs = lds;                 // [256]
  float* ks = qs + 256;            // [256]
  float* vs = ks + 256;            // [256]
  float* al = vs + 256;            // [256] decay per key channel
  float* red = al + 256;           // [NT]
  float* red2 = red + NT;          // [NT]
  float* redw = red2 + NT;         // [2][NT / 64]
  float* gs = redw + 2 * (NT / 64);  // [256] REC_CHANNEL_DELTA: output gate
  const float* y = m.y + (size_t)b * m.ld_y;
  float* S = c.state + (size_t)b * c.state_seq + (size_t)h * dim * vdim;
  const int pos = *m.d_pos;
  float st[RPT];
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    // (past the state's end: some value of it, which meets zeros of q and k and is not stored)
    st[j] = S[(size_t)min(part + parts * j, dim - 1) * vdim + min(v, vdim - 1)];
  }
  const int tv = min(tid, vdim - 1);
  const float gate = kChannel ? 0.0f : y[c.g_col + h * vdim + tv], norm = kSsd ? 0.0f : c.norm[tv];
  const int kvh = h / (c.heads / c.kv_heads);
  float beta = 1.0f, g = 1.0f, skip = 0.0f;
  if (delta || kSsd) {
    const ShortConv& cv = c.conv;
    float* ring = cv.ring + (size_t)b * cv.ring_seq;
    const bool first = h % (c.heads / c.kv_heads) == 0;
    const float yb = kSsd ? 0.0f : y[c.b_col + h], al0 = c.a_log[h];
    const float ya = kChannel ? 0.0f : y[c.a_col + h], dt = c.dt_bias[kChannel ? h * dim + min(tid, dim - 1) : h];
    typename std::conditional<kChannel, LowRankRows<NT>, int>::type low_a, low_g;
    if constexpr (kChannel) {
      low_a.load(c.low_a, y, h * dim, dim);
      low_g.load(c.low_g, y, h * vdim, vdim);
    }
    const int td = min(tid, dim - 1);
    const int ch[3] = {c.q_col - cv.col + kvh * dim + td, c.k_col - cv.col + kvh * dim + td,
                       c.v_col - cv.col + h * vdim + tv};
    const bool keep[3] = {first && tid < dim, first && tid < dim, tid < vdim};
    float cq[3];
    conv_channels<3>(cv, y, ring, ch, keep, pos, cq);
    if constexpr (kChannel) {
      low_a.store(c.low_a, y, h * dim, dim, al);
      low_g.store(c.low_g, y, h * vdim, vdim, gs);
    }
    float qv = cq[0], kv = cq[1], x = cq[2];
    if (tid >= dim) qv = kv = 0.0f;
    if constexpr (kSsd) {
      const float step = softplus(ya + dt);
      g = expf(-expf(al0) * step);
      skip = c.skip[h] * x;
      if (tid < 256) {
        vs[tid] = step * x;
        qs[tid] = qv;
        ks[tid] = kv;
      }
    } else {
    float qn = wave_sum(qv * qv), kn = wave_sum(kv * kv);
    if ((tid & 63) == 0 && tid < 256) {  // (nothing past kMixMaxDim = 256)
      redw[tid >> 6] = qn;
      redw[4 + (tid >> 6)] = kn;
    }
    __syncthreads();
    qn = (redw[0] + redw[1]) + (redw[2] + redw[3]);
    kn = (redw[4] + redw[5]) + (redw[6] + redw[7]);
    if (tid < 256) {
      vs[tid] = x;
      qs[tid] = qv / sqrtf(qn + 1e-6f) * c.q_scale;
      ks[tid] = kv / sqrtf(kn + 1e-6f);
    }
    beta = sigmoid(yb);
    if constexpr (kChannel) {  // (al was written before the barrier above)
      if (tid < dim) al[tid] = expf(delta_log_decay(al[tid], al0, dt));
    } else {
      g = expf(delta_log_decay(ya, al0, dt));
    }
    }
  } else if constexpr (KIND < 0) {
    float qv = 0.0f, kv = 0.0f, av = 1.0f;
    if (tid < dim) {
      qv = y[c.q_col + h * dim + tid] * c.q_scale;
      kv = y[c.k_col + h * dim + tid];
      const float* a2 = c.a2 + (size_t)(h * dim + tid) * c.rank;
      float z = c.a2_bias[h * dim + tid];
      int r = 0;
      for (; r + 8 <= c.rank; r += 8) {
        float w8[8], x8[8];
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          w8[k] = a2[r + k];
          x8[k] = y[c.a_col + r + k];
        }
#pragma unroll
        for (int k = 0; k < 8; ++k) z += w8[k] * x8[k];
      }
      for (; r < c.rank; ++r) z += a2[r] * y[c.a_col + r];
      av = expf(gla_log_decay(z, c.inv_tau));
    }
    if (tid < 256) {
      qs[tid] = qv;
      ks[tid] = kv;
      al[tid] = av;
      vs[tid] = y[c.v_col + h * vdim + tv];
    }
  }
  // (at position 0 the state is zero whatever the memory holds)
  if (pos == 0) {
#pragma unroll
    for (int j = 0; j < RPT; ++j) st[j] = 0.0f;
  }
  __syncthreads();
  float u = v < vdim ? vs[v] : 0.0f;
  if (delta) {
    float s = 0.0f;
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      st[j] *= kChannel ? al[min(part + parts * j, dim - 1)] : g;
      s += st[j] * ks[part + parts * j];
    }
    red[tid] = s;
    __syncthreads();
    s = 0.0f;
    for (int p = 0; p < parts; ++p) s += red[p * cols + v];
    u = beta * (u - s);
  } else {
#pragma unroll
    for (int j = 0; j < RPT; ++j) st[j] *= kSsd ? g : al[part + parts * j];
  }
  float o = 0.0f;
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    st[j] += ks[part + parts * j] * u;
    o += st[j] * qs[part + parts * j];
  }
  if (v < vdim) {
    float* dst = S + (size_t)part * vdim + v;
    const int n = (dim - part + parts - 1) / parts;  // rows of this thread
    if (n >= RPT) {
#pragma unroll
      for (int j = 0; j < RPT; ++j) dst[(size_t)j * parts * vdim] = st[j];
    } else {
#pragma unroll
      for (int j = 0; j < RPT; ++j)
        if (j < n) dst[(size_t)j * parts * vdim] = st[j];
    }
  }
  red2[tid] = o;
  __syncthreads();
  float out = 0.0f;
  if (tid < vdim)
    for (int p = 0; p < parts; ++p) out += red2[p * cols + tid];
  if constexpr (kSsd) {
    if (tid < vdim) m.out[(size_t)b * m.ld_out + c.out_col + h * vdim + tid] = (out + skip) * silu(gate);
    return;
  }
  float ss = wave_sum(out * out);
  if ((tid & 63) == 0 && tid < 256) redw[tid >> 6] = ss;
  __syncthreads();
  ss = (redw[0] + redw[1]) + (redw[2] + redw[3]);
  if (tid < vdim)
    m.out[(size_t)b * m.ld_out + c.out_col + h * vdim + tid] =
        out / sqrtf(ss / (float)vdim + c.eps) * norm * (kChannel ? sigmoid(gs[tid]) : silu(gate)) * c.out_scale;
}

template <int NT, int RPT, int NV>
__global__ __launch_bounds__(NT) void k_mix_decode(MixDecode m, int attn_items, int rec_items) {
  __shared__ __attribute__((aligned(16))) float lds[kDecodeLds<NT>];
  const int b = blockIdx.y;
  int item = blockIdx.x;
  if (item < rec_items) {
    recurrence_role<NT, RPT>(m, b, item, lds);
    return;
  }
  item -= rec_items;
  if (item < attn_items) {
    attn_role<NT, NV>(m, b, item, lds);
    return;
  }
  item -= attn_items;
  const int j = item * NT + threadIdx.x;
  if (j >= m.mlp.ff_pad) return;
  const float* y = m.y + (size_t)b * m.ld_y;
  m.act[(size_t)b * m.mlp.ff_pad + j] =
      j < m.mlp.ff ? gelu_tanh(y[m.mlp.gate_col + j]) * y[m.mlp.up_col + j] : 0.0f;
}

template <int NT, int RPT, int KIND>
__global__ __launch_bounds__(NT) void k_recurrence_decode(MixDecode m) {
  __shared__ __attribute__((aligned(16))) float lds[kDecodeLds<NT>];
  recurrence_role<NT, RPT, KIND>(m, blockIdx.y, blockIdx.x, lds);
}

__global__ __launch_bounds__(256) void k_attn_sum(MixDecode m) {
  const ChunkAttn& a = m.attn;
  const int b = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x, n = a.heads * a.dim;
  if (i >= n) return;
  const float* p = m.part + (size_t)b * m.attn_splits * n + i;
  float s = 0.0f;
#pragma unroll 8
  for (int k = 0; k < m.attn_splits; ++k) s += p[(size_t)k * n];
  m.out[(size_t)b * m.ld_out + a.out_col + i] = s;
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

// A block owns 32 queries of one head; its NW wavefronts take the key tiles (32 keys) from the
// first query's chunk start to the last query in turn and add their results through LDS at the
// end (the weights are not normalised: the sums simply add).  Per tile:
//   S^T (keys x queries) = K . Q^T, Q in registers (lane (l, half) holds dims half DP/2 ..), K rows
//     from a wavefront-private LDS tile
//   weights sigmoid(S scale + bias), 0 outside the query's chunk and after the query
//   O^T (dims x queries) += V^T . P^T, a lane's own weights are the operand, V rows from LDS
// Keys before pos0 come from the ring, the others from this step's rows.
// Grid: x = head, y = block of queries, z = sequence.
template <int DP, int NW>
__global__ __launch_bounds__(64 * NW, DP <= 64 ? 2 : 1) void k_chunk_attn_rows(MixRows r, ChunkAttn a) {
  constexpr int KT = 32, LD = DP + 4, NB = DP / 32;
  constexpr int NL = KT * DP / 4 / 64;   // float4 loads of K (and V) per lane and tile
  constexpr bool PRE = DP <= 128;        // the next tile waits in registers
  __shared__ __attribute__((aligned(16))) float Ks[NW][KT * LD];
  __shared__ __attribute__((aligned(16))) float Vs[NW][KT * LD];
  static_assert(KT * LD / 2 >= 32 * 33 - 32 || NB == 1, "two merge tiles fit the K tile");
  static_assert(KT * LD >= 32 * 33, "a merge tile fits the K tile");
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int half = lane >> 5, l32 = lane & 31;
  const int h = blockIdx.x, b = blockIdx.z, g = h / (a.heads / a.kv_heads);
  const int nqb = (r.n + 31) / 32;
  const int t0 = (nqb - 1 - (int)blockIdx.y) * 32;  // first query of the block
  const int tq = t0 + l32;                          // this lane's query
  const int dim = a.dim, dp = a.dim_pad;
  const size_t row0 = (size_t)b * r.n;
  const float* yb = r.y + row0 * r.ld_y;
  const float* krb = r.k_rot + row0 * a.kv_heads * dim + g * dim;
  const float* kring = a.kring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;
  const float* vring = a.vring + (size_t)b * a.ring_seq + (size_t)g * a.chunk * dp;
  const bool vec = (dim & 3) == 0;

  float qr[DP / 2];
  {
    const float* q = yb + (size_t)min(tq, r.n - 1) * r.ld_y + a.q_col + h * dim;
    if (vec) {
#pragma unroll
      for (int s = 0; s < DP / 2; s += 4) {
        const int d = half * (DP / 2) + s;
        f4 x = f4{0.f, 0.f, 0.f, 0.f};
        if (d < dim) x = *reinterpret_cast<const f4*>(q + d);
        qr[s] = x.x; qr[s + 1] = x.y; qr[s + 2] = x.z; qr[s + 3] = x.w;
      }
    } else {
#pragma unroll
      for (int s = 0; s < DP / 2; ++s) {
        const int d = half * (DP / 2) + s;
        qr[s] = d < dim ? q[d] : 0.0f;
      }
    }
  }
  f16v o[NB];
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) o[i][v] = 0.0f;

  const int pq = r.pos0 + tq;                 // positions
  const int lo = pq - pq % a.chunk;           // first key this lane's query sees
  const int pb0 = r.pos0 + t0, pb1 = r.pos0 + min(t0 + 32, r.n) - 1;
  const int kfirst = pb0 - pb0 % a.chunk, lo1 = pb1 - pb1 % a.chunk;
  const int tiles = (pb1 - kfirst) / KT + 1;
  const float bias = a.bias[h];
  float* ks = Ks[wave];
  float* vs = Vs[wave];

  auto load_row = [&](int p, int d, f4& k, f4& v) __attribute__((always_inline)) {
    k = v = f4{0.f, 0.f, 0.f, 0.f};
    if (p > pb1 || d >= dp) return;
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
  };
  f4 kreg[PRE ? NL : 1], vreg[PRE ? NL : 1];
  auto fetch = [&](int tile) __attribute__((always_inline)) {
    if constexpr (PRE) {
#pragma unroll
      for (int i = 0; i < NL; ++i) {
        const int idx = lane + 64 * i;
        load_row(kfirst + tile * KT + idx / (DP / 4), (idx % (DP / 4)) * 4, kreg[i], vreg[i]);
      }
    }
  };
  if (wave < tiles) fetch(wave);
  for (int tile = wave; tile < tiles; tile += NW) {
    const int k0 = kfirst + tile * KT;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int idx = lane + 64 * i, key = idx / (DP / 4), d = (idx % (DP / 4)) * 4;
      f4 k, v;
      if constexpr (PRE) {
        k = kreg[i];
        v = vreg[i];
      } else {
        load_row(k0 + key, d, k, v);
      }
      *reinterpret_cast<f4*>(&ks[key * LD + d]) = k;
      *reinterpret_cast<f4*>(&vs[key * LD + d]) = v;
    }
    // (each wavefront has its own tile and LDS executes a wavefront's accesses in order: only the
    // compiler has to be kept from reordering)
    __builtin_amdgcn_wave_barrier();
    if (tile + NW < tiles) fetch(tile + NW);
    f16v s0, s1;
#pragma unroll
    for (int v = 0; v < 16; ++v) s0[v] = s1[v] = 0.0f;
    // V operands of the first 32 dims are read between the MFMAs of the first product
    float vop[16];
    const f4* krow = reinterpret_cast<const f4*>(&ks[l32 * LD + half * (DP / 2)]);
    f4 k = krow[0];
#pragma unroll
    for (int j = 0; j < DP / 8; ++j) {
      const f4 kc = k;
      s0 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.x, qr[4 * j], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.y, qr[4 * j + 1], s1, 0, 0, 0);
      if (j + 1 < DP / 8) k = krow[j + 1];
      constexpr int PER = (16 + DP / 8 - 1) / (DP / 8);
#pragma unroll
      for (int v = j * PER; v < (j + 1) * PER && v < 16; ++v)
        vop[v] = vs[(8 * (v >> 2) + 4 * half + (v & 3)) * LD + l32];
      __builtin_amdgcn_sched_barrier(0);
      s0 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.z, qr[4 * j + 2], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.w, qr[4 * j + 3], s1, 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
    s0 += s1;
    // lane holds keys k0 + 8 (v / 4) + 4 half + v % 4 of its query
    const bool edge = k0 + KT - 1 > pb0 || k0 < lo1;
    const float zs = -1.44269504088896341f * a.scale, zb = -1.44269504088896341f * bias;
#pragma unroll
    for (int v = 0; v < 16; ++v)
      s0[v] = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(fmaf(s0[v], zs, zb)));
    if (edge) {
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        const int key = k0 + 8 * (v >> 2) + 4 * half + (v & 3);
        if (!(key <= pq && key >= lo)) s0[v] = 0.0f;
      }
    }
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      if (i > 0 && !PRE) {
#pragma unroll
        for (int v = 0; v < 16; ++v) vop[v] = vs[(8 * (v >> 2) + 4 * half + (v & 3)) * LD + 32 * i + l32];
        __builtin_amdgcn_sched_barrier(0);
      }
      float nx[16];
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(vop[v], s0[v], o[i], 0, 0, 0);
        if (PRE && i + 1 < NB) nx[v] = vs[(8 * (v >> 2) + 4 * half + (v & 3)) * LD + 32 * (i + 1) + l32];
      }
      if (PRE && i + 1 < NB) {
#pragma unroll
        for (int v = 0; v < 16; ++v) vop[v] = nx[v];
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
  // the wavefronts' sums, in wavefront order: [dim][query] tiles, 32 dims at a time
  float* dst = r.out + (row0 + min(tq, r.n - 1)) * r.ld_out + a.out_col + h * dim;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NB; ++i) {
    float* ob = ks + (i & 1) * (KT * LD / 2);
#pragma unroll
    for (int v = 0; v < 16; ++v) ob[(8 * (v >> 2) + 4 * half + (v & 3)) * 33 + l32] = o[i][v];
    __syncthreads();
    // lane (query l32, half) of wavefront w sums dims [32 / NW w, ..) of the tile
    constexpr int ND = 32 / NW / 2;
#pragma unroll
    for (int e = 0; e < ND; ++e) {
      const int d = (32 / NW) * wave + ND * half + e;
      float sum = 0.0f;
#pragma unroll
      for (int w = 0; w < NW; ++w) sum += Ks[w][(i & 1) * (KT * LD / 2) + d * 33 + l32];
      if (tq < r.n && 32 * i + d < dim) dst[32 * i + d] = sum * a.out_scale;
    }
  }
}

// A thread owns one channel of kConvRows consecutive tokens; up to TAPS - 1 inputs before them.
constexpr int kConvRows = 16;
template <int TAPS>
__global__ __launch_bounds__(256) void k_short_conv_rows(MixRows r, ShortConv c) {
  const int ch = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, t0 = blockIdx.y * kConvRows;
  if (ch >= c.channels) return;
  const float* x = r.y + (size_t)b * r.n * r.ld_y + c.col + ch;
  const float* ring = c.ring + (size_t)b * c.ring_seq + ch;
  float w[TAPS], in[TAPS - 1 + kConvRows];
  const float bias = c.bias ? c.bias[ch] : 0.0f;
#pragma unroll
  for (int j = 0; j < TAPS; ++j) w[j] = j < c.taps ? c.w[ch * c.taps + c.taps - 1 - j] : 0.0f;  // j tokens back
#pragma unroll
  for (int i = 0; i < TAPS - 1 + kConvRows; ++i) {
    const int t = t0 + i - (TAPS - 1), pos = r.pos0 + t;
    in[i] = 0.0f;
    if (t >= 0) {
      in[i] = x[(size_t)min(t, r.n - 1) * r.ld_y];
    } else if (pos >= 0 && -t < c.taps) {
      in[i] = ring[(size_t)(pos % c.taps) * c.channels];
    }
  }
#pragma unroll
  for (int i = 0; i < kConvRows; ++i) {
    if (t0 + i >= r.n) return;
    float s = bias;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) s += w[j] * in[TAPS - 1 + i - j];
    r.conv_out[((size_t)b * r.n + t0 + i) * c.channels + ch] = silu(s);
  }
}

// log alpha of gated linear attention: a thread owns one channel of kDecayRows tokens
constexpr int kDecayRows = 16, kDecayRank = 16;
__global__ __launch_bounds__(256) void k_gla_decay_rows(MixRows r, Recurrence c, int rows) {
  __shared__ float a1[kDecayRows][kDecayRank];
  const int tid = threadIdx.x, i = blockIdx.x * 256 + tid, n = c.heads * c.dim, row0 = blockIdx.y * kDecayRows;
  const int ii = min(i, n - 1);
  float z[kDecayRows];
#pragma unroll
  for (int t = 0; t < kDecayRows; ++t) z[t] = c.a2_bias[ii];
  for (int k0 = 0; k0 < c.rank; k0 += kDecayRank) {
    float w[kDecayRank];
#pragma unroll
    for (int k = 0; k < kDecayRank; ++k) w[k] = k0 + k < c.rank ? c.a2[(size_t)ii * c.rank + k0 + k] : 0.0f;
    __syncthreads();
    {
      const int t = tid / kDecayRank, k = tid % kDecayRank;
      a1[t][k] = k0 + k < c.rank && row0 + t < rows ? r.y[(size_t)(row0 + t) * r.ld_y + c.a_col + k0 + k] : 0.0f;
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < kDecayRows; ++t)
#pragma unroll
      for (int k = 0; k < kDecayRank; ++k) z[t] += w[k] * a1[t][k];
  }
  if (i >= n) return;
#pragma unroll
  for (int t = 0; t < kDecayRows; ++t)
    if (row0 + t < rows) r.decay[(size_t)(row0 + t) * n + i] = gla_log_decay(z[t], c.inv_tau);
}

// ---------------------------------------------------------------------------
// The recurrences over many rows, kChunk tokens at a time.  With G_t the sum of the log decays of
// a chunk's tokens up to t (per head, or per key channel), S0 the state before the chunk and
//   Kd_t = exp(G_end - G_t) k_t,  Qd_t = exp(G_t) q_t,  P_tj = q_t . (exp(G_t - G_j) k_j), j <= t
// the chunk's tokens write U into the state and read it out as
//   S_end = exp(G_end) S0 + Kd^T U,   O = Qd S0 + P U,
// where U = V for gated linear attention and, for the delta rule (whose k_t first reads the state),
//   U = U0 - W S0,  (1 + A) [U0 | W] = [beta V | beta exp(G) K],  A_tj = beta_t exp(G_t - G_j) k_t . k_j, j < t
// (with decays per key channel the exponentials stand inside the dot products).  The state-space
// recurrence is the form without reads, U = dt V.
// All exponents are <= 0.  Three launches: the parts that need no state for every chunk at once,
// the states from chunk to chunk (the only serial part), the read-outs for every chunk at once.
// A chunk's tiles lie in the work area one after the other, 32 rows each, widths padded to
// 32 (pads and rows past the end are zeros).
// ---------------------------------------------------------------------------
constexpr int kChunk = 32;

struct ChunkWork {
  int chunks;            // per sequence
  int dp, ep;            // dim and vdim padded to 32
  float *W, *U0, *Kd, *Qd, *P, *U, *S, *G;
  // tile (sequence, chunk, head): W, Kd, Qd [32][dp]; U0, U [ep / 32][32][32]; P [32][32];
  // S [ep / 32][dp][32]; G [dp] (exp(G_end) per key channel)
  __device__ __forceinline__ size_t tile(int b, int c, int h, int heads) const {
    return ((size_t)b * chunks + c) * heads + h;
  }
};

// Floats of a sequence's work area per chunk and head.
__host__ __device__ inline size_t chunk_floats(int dp, int ep, bool delta) {
  return (size_t)32 * ((delta ? 3 : 2) * dp + (delta ? 2 : 1) * ep + 32) + (size_t)dp * ep + dp;
}

// One tile of 32 x 32 dot products over dp columns: rows x of X against rows of Y (LDS, LD apart),
// columns [k0, k1); lane layout of v_mfma_f32_32x32x2_f32.
__device__ __forceinline__ f16v dots32(const float* X, const float* Y, int LD, int k0, int k1, int lane) {
  const int half = lane >> 5, l32 = lane & 31, n = (k1 - k0) / 2;
  f16v s;
#pragma unroll
  for (int v = 0; v < 16; ++v) s[v] = 0.0f;
  const float* x = X + l32 * LD + k0 + half * n;
  const float* y = Y + l32 * LD + k0 + half * n;
  for (int j = 0; j < n; j += 4) {
    const f4 a = *reinterpret_cast<const f4*>(x + j), b = *reinterpret_cast<const f4*>(y + j);
    s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.x, b.x, s, 0, 0, 0);
    s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.y, b.y, s, 0, 0, 0);
    s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.z, b.z, s, 0, 0, 0);
    s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.w, b.w, s, 0, 0, 0);
  }
  return s;
}

// Delta rule, per (chunk, head, sequence): U0, W, Kd, Qd, P, G.
__global__ __launch_bounds__(256) void k_delta_chunk(MixRows r, Recurrence c, ChunkWork w) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ double Gs[kChunk];
  __shared__ float beta[kChunk], eg[kChunk], ek[kChunk];
  __shared__ float red[4][32 * 33];
  __shared__ __attribute__((aligned(16))) float As[32][36];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int half = lane >> 5, l32 = lane & 31;
  const int ci = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int dim = c.dim, vdim = c.vdim, dp = w.dp, ep = w.ep, LD = dp + 4;
  float* Ks = lds;            // [32][LD]
  float* Qs = lds + 32 * LD;
  const int t0 = ci * kChunk, nt = min(kChunk, r.n - t0);
  const size_t row0 = (size_t)b * r.n + t0;
  const int kvh = h / (c.heads / c.kv_heads);
  const int CH = c.conv.channels;
  const float* xq = r.conv_out + row0 * CH + (c.q_col - c.conv.col) + kvh * dim;
  const float* xk = r.conv_out + row0 * CH + (c.k_col - c.conv.col) + kvh * dim;
  const float* xv = r.conv_out + row0 * CH + (c.v_col - c.conv.col) + h * vdim;
  {
    // eight threads to a row: q and k as unit vectors
    const int t = tid >> 3, sub = tid & 7;
    float qq = 0.0f, kk = 0.0f;
#pragma unroll 4
    for (int i = sub; i < dp; i += 8) {
      float q = 0.0f, k = 0.0f;
      if (t < nt && i < dim) {
        q = xq[(size_t)t * CH + i];
        k = xk[(size_t)t * CH + i];
      }
      Qs[t * LD + i] = q;
      Ks[t * LD + i] = k;
      qq += q * q;
      kk += k * k;
    }
#pragma unroll
    for (int off = 4; off > 0; off >>= 1) {
      qq += __shfl_xor(qq, off, 64);
      kk += __shfl_xor(kk, off, 64);
    }
    const float qm = c.q_scale / sqrtf(qq + 1e-6f), km = 1.0f / sqrtf(kk + 1e-6f);
    for (int i = sub; i < dp; i += 8) {
      Qs[t * LD + i] *= qm;
      Ks[t * LD + i] *= km;
    }
  }
  if (wave == 0) {
    double g = 0.0;
    float bt = 0.0f;
    if (lane < nt) {
      const float* y = r.y + (row0 + lane) * r.ld_y;
      bt = sigmoid(y[c.b_col + h]);
      g = (double)delta_log_decay(y[c.a_col + h], c.a_log[h], c.dt_bias[h]);
    }
#pragma unroll
    for (int off = 1; off < 32; off <<= 1) {
      const double up = __shfl_up(g, off, 64);
      if (lane >= off) g += up;
    }
    const double end = __shfl(g, 31, 64);  // (tokens past the end decay by nothing)
    if (lane < 32) {
      Gs[lane] = g;
      beta[lane] = bt;
      eg[lane] = expf((float)g);
      ek[lane] = expf((float)(end - g));
    }
  }
  __syncthreads();
  const size_t tile = w.tile(b, ci, h, c.heads);
  {
    // wavefronts 0, 1: k . k over half of the columns each; 2, 3: q . k
    const int k0 = (wave & 1) * (dp / 2);
    const f16v s = dots32(wave < 2 ? Ks : Qs, Ks, LD, k0, k0 + dp / 2, lane);
#pragma unroll
    for (int v = 0; v < 16; ++v) red[wave][(8 * (v >> 2) + 4 * half + (v & 3)) * 33 + l32] = s[v];
  }
  __syncthreads();
  for (int i = tid; i < 1024; i += 256) {
    const int t = i >> 5, j = i & 31, at = t * 33 + j;
    const float e = j <= t ? expf((float)(Gs[t] - Gs[j])) : 0.0f;
    As[t][j] = j < t ? beta[t] * e * (red[0][at] + red[1][at]) : 0.0f;
    w.P[tile * 1024 + i] = e * (red[2][at] + red[3][at]);
  }
  __syncthreads();
  // columns of [W | U0] by forward substitution, one per thread
  for (int col = tid; col < dp + ep; col += 256) {
    const bool isw = col < dp;
    const int e = col - dp;
    float x[kChunk];
#pragma unroll
    for (int t = 0; t < kChunk; ++t) {
      float v = 0.0f;
      if (isw) v = eg[t] * Ks[t * LD + col];
      else if (t < nt && e < vdim) v = xv[(size_t)t * CH + e];
      x[t] = beta[t] * v;
    }
#pragma unroll
    for (int t = 1; t < kChunk; ++t) {
      float s = x[t];
#pragma unroll
      for (int j = 0; j < t; j += 4) {
        const f4 a4 = *reinterpret_cast<const f4*>(&As[t][j]);
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (j + k < t) s -= a4[k] * x[j + k];
      }
      x[t] = s;
      __builtin_amdgcn_sched_barrier(0);  // (row by row: all rows of A at once do not fit the registers)
    }
    float* dst = isw ? w.W + tile * 32 * dp + col : w.U0 + tile * 32 * ep + (e >> 5) * 1024 + (e & 31);
    const int ld = isw ? dp : 32;
#pragma unroll
    for (int t = 0; t < kChunk; ++t) dst[t * ld] = x[t];
  }
  for (int i = tid; i < 32 * dp; i += 256) {
    const int t = i / dp, d = i - t * dp;
    w.Kd[tile * 32 * dp + i] = ek[t] * Ks[t * LD + d];
    w.Qd[tile * 32 * dp + i] = eg[t] * Qs[t * LD + d];
  }
  for (int i = tid; i < dp; i += 256) w.G[tile * dp + i] = eg[31];
}

// Gated linear attention, per (chunk, head, sequence): U (= V), Kd, Qd, P, G.
__global__ __launch_bounds__(256) void k_gla_chunk(MixRows r, Recurrence c, ChunkWork w) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x;
  const int ci = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int dim = c.dim, vdim = c.vdim, dp = w.dp, ep = w.ep, LD = dp + 1;
  float* Ks = lds;  // [32][LD] each
  float* Qs = lds + 32 * LD;
  float* Gs = lds + 64 * LD;
  const int t0 = ci * kChunk, nt = min(kChunk, r.n - t0);
  const size_t row0 = (size_t)b * r.n + t0;
  const size_t tile = w.tile(b, ci, h, c.heads);
  for (int i = tid; i < 32 * dp; i += 256) {
    const int t = i / dp, d = i - t * dp;
    float q = 0.0f, k = 0.0f, g = 0.0f;
    if (t < nt && d < dim) {
      const float* y = r.y + (row0 + t) * r.ld_y + h * dim + d;
      q = y[c.q_col] * c.q_scale;
      k = y[c.k_col];
      g = r.decay[(row0 + t) * c.heads * dim + h * dim + d];
    }
    Qs[t * LD + d] = q;
    Ks[t * LD + d] = k;
    Gs[t * LD + d] = g;
  }
  for (int i = tid; i < 32 * ep; i += 256) {
    const int t = (i >> 5) & 31, e = (i >> 10) * 32 + (i & 31);
    w.U[tile * 32 * ep + i] = t < nt && e < vdim ? r.y[(row0 + t) * r.ld_y + c.v_col + h * vdim + e] : 0.0f;
  }
  __syncthreads();
  for (int d = tid; d < dp; d += 256) {
    float s = 0.0f;
#pragma unroll
    for (int t = 0; t < kChunk; ++t) {
      s += Gs[t * LD + d];
      Gs[t * LD + d] = s;
    }
    w.G[tile * dp + d] = expf(s);
  }
  __syncthreads();
  for (int i = tid; i < 1024; i += 256) {
    const int t = i >> 5, j = i & 31;
    float s = 0.0f;
    if (j <= t) {
      const float *q = Qs + t * LD, *k = Ks + j * LD, *gt = Gs + t * LD, *gj = Gs + j * LD;
#pragma unroll 8
      for (int d = 0; d < dim; ++d) s += q[d] * k[d] * __builtin_amdgcn_exp2f(1.44269504088896341f * (gt[d] - gj[d]));
    }
    w.P[tile * 1024 + i] = s;
  }
  for (int i = tid; i < 32 * dp; i += 256) {
    const int t = i / dp, d = i - t * dp;
    const float g = Gs[t * LD + d];
    w.Kd[tile * 32 * dp + i] = expf(Gs[31 * LD + d] - g) * Ks[t * LD + d];
    w.Qd[tile * 32 * dp + i] = expf(g) * Qs[t * LD + d];
  }
}

// State-space recurrence, per (chunk, head, sequence): U (= dt V), Kd, Qd, P, G.
__global__ __launch_bounds__(256) void k_ssd_chunk(MixRows r, Recurrence c, ChunkWork w) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ double Gs[kChunk];
  __shared__ float step[kChunk], eg[kChunk], ek[kChunk];
  __shared__ float red[4][32 * 33];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int half = lane >> 5, l32 = lane & 31;
  const int ci = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int dim = c.dim, vdim = c.vdim, dp = w.dp, ep = w.ep, LD = dp + 4;
  float* Ks = lds;            // [32][LD]
  float* Qs = lds + 32 * LD;
  const int t0 = ci * kChunk, nt = min(kChunk, r.n - t0);
  const size_t row0 = (size_t)b * r.n + t0;
  const int kvh = h / (c.heads / c.kv_heads);
  const int CH = c.conv.channels;
  const float* xq = r.conv_out + row0 * CH + (c.q_col - c.conv.col) + kvh * dim;
  const float* xk = r.conv_out + row0 * CH + (c.k_col - c.conv.col) + kvh * dim;
  const float* xv = r.conv_out + row0 * CH + (c.v_col - c.conv.col) + h * vdim;
  for (int i = tid; i < 32 * dp; i += 256) {
    const int t = i / dp, d = i - t * dp;
    const bool in = t < nt && d < dim;
    Qs[t * LD + d] = in ? xq[(size_t)t * CH + d] : 0.0f;
    Ks[t * LD + d] = in ? xk[(size_t)t * CH + d] : 0.0f;
  }
  if (wave == 0) {
    double g = 0.0;
    float dt = 0.0f;
    if (lane < nt) {
      dt = softplus(r.y[(row0 + lane) * r.ld_y + c.a_col + h] + c.dt_bias[h]);
      g = (double)(-expf(c.a_log[h]) * dt);
    }
#pragma unroll
    for (int off = 1; off < 32; off <<= 1) {
      const double up = __shfl_up(g, off, 64);
      if (lane >= off) g += up;
    }
    const double end = __shfl(g, 31, 64);
    if (lane < 32) {
      Gs[lane] = g;
      step[lane] = dt;
      eg[lane] = expf((float)g);
      ek[lane] = expf((float)(end - g));
    }
  }
  __syncthreads();
  const size_t tile = w.tile(b, ci, h, c.heads);
  {
    const int k0 = wave * (dp / 4);  // q . k over a quarter of the columns each
    const f16v s = dots32(Qs, Ks, LD, k0, k0 + dp / 4, lane);
#pragma unroll
    for (int v = 0; v < 16; ++v) red[wave][(8 * (v >> 2) + 4 * half + (v & 3)) * 33 + l32] = s[v];
  }
  for (int i = tid; i < 32 * ep; i += 256) {
    const int t = (i >> 5) & 31, e = (i >> 10) * 32 + (i & 31);
    w.U[tile * 32 * ep + i] = t < nt && e < vdim ? step[t] * xv[(size_t)t * CH + e] : 0.0f;
  }
  __syncthreads();
  for (int i = tid; i < 1024; i += 256) {
    const int t = i >> 5, j = i & 31, at = t * 33 + j;
    const float e = j <= t ? expf((float)(Gs[t] - Gs[j])) : 0.0f;
    w.P[tile * 1024 + i] = e * ((red[0][at] + red[1][at]) + (red[2][at] + red[3][at]));
  }
  for (int i = tid; i < 32 * dp; i += 256) {
    const int t = i / dp, d = i - t * dp;
    w.Kd[tile * 32 * dp + i] = ek[t] * Ks[t * LD + d];
    w.Qd[tile * 32 * dp + i] = eg[t] * Qs[t * LD + d];
  }
  for (int i = tid; i < dp; i += 256) w.G[tile * dp + i] = eg[31];
}

// Delta rule with a decay per key channel, per (chunk, head, sequence): U0, W, Kd, Qd, P, G.  The
// sums of the log decays (base 2) are kept as two floats each, so that their differences are as
// exact as f32 however strongly the channel has decayed before.
__global__ __launch_bounds__(256) void k_channel_delta_chunk(MixRows r, Recurrence c, ChunkWork w) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float beta[kChunk];
  __shared__ __attribute__((aligned(16))) float As[32][36];
  const int tid = threadIdx.x;
  const int ci = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int dim = c.dim, vdim = c.vdim, dp = w.dp, ep = w.ep, LD = dp + 1;
  float* Ks = lds;  // [32][LD] each
  float* Qs = lds + 32 * LD;
  float* Gh = lds + 64 * LD;
  float* Gl = lds + 96 * LD;
  const int t0 = ci * kChunk, nt = min(kChunk, r.n - t0);
  const size_t row0 = (size_t)b * r.n + t0;
  const size_t tile = w.tile(b, ci, h, c.heads);
  const int kvh = h / (c.heads / c.kv_heads);
  const int CH = c.conv.channels;
  const float* xq = r.conv_out + row0 * CH + (c.q_col - c.conv.col) + kvh * dim;
  const float* xk = r.conv_out + row0 * CH + (c.k_col - c.conv.col) + kvh * dim;
  const float* xv = r.conv_out + row0 * CH + (c.v_col - c.conv.col) + h * vdim;
  {
    // eight threads to a row: q and k as unit vectors
    const int t = tid >> 3, sub = tid & 7;
    float qq = 0.0f, kk = 0.0f;
#pragma unroll 4
    for (int i = sub; i < dp; i += 8) {
      float q = 0.0f, k = 0.0f;
      if (t < nt && i < dim) {
        q = xq[(size_t)t * CH + i];
        k = xk[(size_t)t * CH + i];
      }
      Qs[t * LD + i] = q;
      Ks[t * LD + i] = k;
      qq += q * q;
      kk += k * k;
    }
#pragma unroll
    for (int off = 4; off > 0; off >>= 1) {
      qq += __shfl_xor(qq, off, 64);
      kk += __shfl_xor(kk, off, 64);
    }
    const float qm = c.q_scale / sqrtf(qq + 1e-6f), km = 1.0f / sqrtf(kk + 1e-6f);
    for (int i = sub; i < dp; i += 8) {
      Qs[t * LD + i] *= qm;
      Ks[t * LD + i] *= km;
    }
  }
  if (tid < 32) beta[tid] = tid < nt ? sigmoid(r.y[(row0 + tid) * r.ld_y + c.b_col + h]) : 0.0f;
  {
    // log decays, then their sums down the chunk, a channel per thread
    const float al = c.a_log[h];
    for (int i = tid; i < 32 * dp; i += 256) {
      const int t = i / dp, d = i - t * dp;
      float g = 0.0f;
      if (t < nt && d < dim)
        g = delta_log_decay(r.decay[(row0 + t) * c.heads * dim + h * dim + d], al, c.dt_bias[h * dim + d]);
      Gh[t * LD + d] = g;
    }
    __syncthreads();
    for (int d = tid; d < dp; d += 256) {
      double s = 0.0;
#pragma unroll 8
      for (int t = 0; t < kChunk; ++t) {
        s += (double)Gh[t * LD + d];
        const double s2 = s * 1.4426950408889634074;
        const float hi = (float)s2;
        Gh[t * LD + d] = hi;
        Gl[t * LD + d] = (float)(s2 - (double)hi);
      }
    }
  }
  __syncthreads();
  // the 496 pairs j < t: rows 31 - i and i together have 31 of them
  for (int p = tid; p < 496; p += 256) {
    const int i = p / 31, e = p - 31 * i;
    const bool high = e < 31 - i;
    const int t = high ? 31 - i : i, j = high ? e : e - (31 - i);
    const float *q = Qs + t * LD, *kt = Ks + t * LD, *kj = Ks + j * LD;
    const float *ht = Gh + t * LD, *hj = Gh + j * LD, *lt = Gl + t * LD, *lj = Gl + j * LD;
    float sp = 0.0f, sa = 0.0f;
#pragma unroll 4
    for (int d = 0; d < dim; ++d) {
      const float k = kj[d] * __builtin_amdgcn_exp2f((ht[d] - hj[d]) + (lt[d] - lj[d]));
      sp = fmaf(q[d], k, sp);
      sa = fmaf(kt[d], k, sa);
    }
    w.P[tile * 1024 + t * 32 + j] = sp;
    w.P[tile * 1024 + j * 32 + t] = 0.0f;
    As[t][j] = beta[t] * sa;
    As[j][t] = 0.0f;
  }
  {
    const int t = tid >> 3, sub = tid & 7;
    float s = 0.0f;
    for (int d = sub; d < dim; d += 8) s += Qs[t * LD + d] * Ks[t * LD + d];
#pragma unroll
    for (int off = 4; off > 0; off >>= 1) s += __shfl_xor(s, off, 64);
    if (sub == 0) {
      w.P[tile * 1024 + t * 33] = s;
      As[t][t] = 0.0f;
    }
  }
  __syncthreads();
  // columns of [W | U0] by forward substitution, one per thread
  for (int col = tid; col < dp + ep; col += 256) {
    const bool isw = col < dp;
    const int e = col - dp;
    float x[kChunk];
#pragma unroll
    for (int t = 0; t < kChunk; ++t) {
      float v = 0.0f;
      if (isw) v = __builtin_amdgcn_exp2f(Gh[t * LD + col]) * Ks[t * LD + col];
      else if (t < nt && e < vdim) v = xv[(size_t)t * CH + e];
      x[t] = beta[t] * v;
    }
#pragma unroll
    for (int t = 1; t < kChunk; ++t) {
      float s = x[t];
#pragma unroll
      for (int j = 0; j < t; j += 4) {
        const f4 a4 = *reinterpret_cast<const f4*>(&As[t][j]);
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (j + k < t) s -= a4[k] * x[j + k];
      }
      x[t] = s;
      __builtin_amdgcn_sched_barrier(0);  // (row by row: all rows of A at once do not fit the registers)
    }
    float* dst = isw ? w.W + tile * 32 * dp + col : w.U0 + tile * 32 * ep + (e >> 5) * 1024 + (e & 31);
    const int ld = isw ? dp : 32;
#pragma unroll
    for (int t = 0; t < kChunk; ++t) dst[t * ld] = x[t];
  }
  for (int i = tid; i < 32 * dp; i += 256) {
    const int t = i / dp, d = i - t * dp;
    const float hi = Gh[t * LD + d], lo = Gl[t * LD + d];
    w.Kd[tile * 32 * dp + i] = __builtin_amdgcn_exp2f((Gh[31 * LD + d] - hi) + (Gl[31 * LD + d] - lo)) * Ks[t * LD + d];
    w.Qd[tile * 32 * dp + i] = __builtin_amdgcn_exp2f(hi) * Qs[t * LD + d];
  }
  for (int d = tid; d < dp; d += 256) w.G[tile * dp + d] = __builtin_amdgcn_exp2f(Gh[31 * LD + d]);
}

// The states from chunk to chunk.  A block owns 16 value columns of one head; wavefront w keeps
// the state's rows 32 w .. 32 w + 31 in the accumulator layout of v_mfma_f32_16x16x4_f32, where
// register v of lane (l, quarter) of row tile a is row 16 a + 4 quarter + v of column l.  In that
// layout the state is an operand of W S as it is (step (a, v) multiplies the rows its four lane
// quarters hold), and so is U of Kd^T U.  The wavefronts' parts of W S meet in LDS, two buffers in
// turn.  A chunk's tiles are requested two chunks ahead.
template <bool DELTA, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void k_chunk_states(MixRows r, Recurrence c, ChunkWork w) {
  extern __shared__ __attribute__((aligned(16))) float part[];  // [2][WAVES][2][64][4] (delta)
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int quarter = lane >> 4, l16 = lane & 15;
  const int ct = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  constexpr int dp = 32 * WAVES;
  const int cts = w.ep / 32, dim = c.dim, vdim = c.vdim;
  const int col = 16 * ct + l16;
  const int at = (16 * (ct & 1)) + l16 + 4 * quarter * 32;  // of a [32][32] tile
  float* state = c.state + (size_t)b * c.state_seq + (size_t)h * dim * vdim;
  f4 S[2];
#pragma unroll
  for (int a = 0; a < 2; ++a)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int i = 32 * wave + 16 * a + 4 * quarter + v;
      S[a][v] = r.pos0 > 0 && i < dim && col < vdim ? state[(size_t)i * vdim + col] : 0.0f;
    }
  struct Tiles {  // of one chunk: W by (state row tile, token tile), the others by token tile
    f4 w[2][2], g[2], u[2];
    float k[2][2][4];
  };
  auto fetch = [&](int ci, Tiles& x) __attribute__((always_inline)) {
    const size_t tile = w.tile(b, min(ci, w.chunks - 1), h, c.heads);
    const float* u = (DELTA ? w.U0 : w.U) + (tile * cts + (ct >> 1)) * 1024 + at;
    const float* kd = w.Kd + tile * 32 * dp + 32 * wave + 4 * quarter * dp + l16;
    const float* g = w.G + tile * dp + 32 * wave + 4 * quarter;
    if (DELTA) {
      const float* wt = w.W + tile * 32 * dp + 32 * wave + l16 * dp + 4 * quarter;
#pragma unroll
      for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int t = 0; t < 2; ++t) x.w[a][t] = *reinterpret_cast<const f4*>(wt + 16 * a + 16 * t * dp);
    }
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int v = 0; v < 4; ++v) x.u[t][v] = u[(16 * t + v) * 32];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int v = 0; v < 4; ++v)
#pragma unroll
        for (int a = 0; a < 2; ++a) x.k[a][t][v] = kd[(16 * t + v) * dp + 16 * a];
#pragma unroll
    for (int a = 0; a < 2; ++a) x.g[a] = *reinterpret_cast<const f4*>(g + 16 * a);
  };
  auto chunk = [&](int ci, Tiles& x) __attribute__((always_inline)) {
    __builtin_amdgcn_sched_barrier(0);
    const size_t tile = w.tile(b, ci, h, c.heads) * cts + (ct >> 1);
    float* s0 = w.S + (tile * WAVES + wave) * 1024 + at;
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
      for (int v = 0; v < 4; ++v) s0[(16 * a + v) * 32] = S[a][v];
    if (DELTA) {
      f4 p[2] = {f4{0.f, 0.f, 0.f, 0.f}, f4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
      for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int v = 0; v < 4; ++v)
#pragma unroll
          for (int t = 0; t < 2; ++t) p[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w[a][t][v], S[a][v], p[t], 0, 0, 0);
      f4* mine = reinterpret_cast<f4*>(part) + ((ci & 1) * WAVES + wave) * 128 + lane;
      mine[0] = p[0];
      mine[64] = p[1];
      __syncthreads();
      const f4* all = reinterpret_cast<const f4*>(part) + ((ci & 1) * WAVES) * 128 + lane;
#pragma unroll
      for (int o = 0; o < WAVES; ++o) {
        x.u[0] -= all[o * 128];
        x.u[1] -= all[o * 128 + 64];
      }
      if (wave == ci % WAVES) {
        float* ud = w.U + tile * 1024 + at;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int v = 0; v < 4; ++v) ud[(16 * t + v) * 32] = x.u[t][v];
      }
    }
#pragma unroll
    for (int a = 0; a < 2; ++a) S[a] *= x.g[a];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int v = 0; v < 4; ++v)
#pragma unroll
        for (int a = 0; a < 2; ++a) S[a] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[a][t][v], x.u[t][v], S[a], 0, 0, 0);
    __builtin_amdgcn_sched_barrier(0);
  };
  // (past the end: the last chunk's tiles again, never used)
  Tiles x0, x1, x2;
  int ci = 0;
  fetch(0, x0);
  fetch(1, x1);
  for (; ci + 3 <= w.chunks; ci += 3) {
    fetch(ci + 2, x2);
    chunk(ci, x0);
    fetch(ci + 3, x0);
    chunk(ci + 1, x1);
    fetch(ci + 4, x1);
    chunk(ci + 2, x2);
  }
  if (ci < w.chunks) chunk(ci, x0);
  if (ci + 1 < w.chunks) chunk(ci + 1, x1);
#pragma unroll
  for (int a = 0; a < 2; ++a)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int i = 32 * wave + 16 * a + 4 * quarter + v;
      if (i < dim && col < vdim) state[(size_t)i * vdim + col] = S[a][v];
    }
}

// The read-outs of one (chunk, head, sequence), normalised, gated and written to the mixer outputs.
// KIND: REC_CHANNEL_DELTA, REC_SSD, or REC_GLA for the other two.  A wavefront owns the 32-column tiles wave and wave + 4.
template <int KIND>
__global__ __launch_bounds__(256) void k_chunk_out(MixRows r, Recurrence c, ChunkWork w) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ __attribute__((aligned(16))) float Ps[32][36];
  __shared__ float ss[4][32];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int half = lane >> 5, l32 = lane & 31;
  const int ci = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int dp = w.dp, ep = w.ep, vdim = c.vdim, LD = dp + 4;
  const int t0 = ci * kChunk, nt = min(kChunk, r.n - t0);
  const size_t row0 = (size_t)b * r.n + t0, tile = w.tile(b, ci, h, c.heads);
  float* Qs = lds;
  for (int i = tid; i < 8 * dp; i += 256) {
    const int t = i / (dp / 4), d = (i - t * (dp / 4)) * 4;
    *reinterpret_cast<f4*>(&Qs[t * LD + d]) = *reinterpret_cast<const f4*>(w.Qd + tile * 32 * dp + t * dp + d);
  }
  {
    const int t = tid >> 3, d = (tid & 7) * 4;
    *reinterpret_cast<f4*>(&Ps[t][d]) = *reinterpret_cast<const f4*>(w.P + tile * 1024 + t * 32 + d);
  }
  __syncthreads();
  const int tiles = ep / 32;
  f16v o[2];
#pragma unroll
  for (int v = 0; v < 16; ++v) o[0][v] = o[1][v] = 0.0f;
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    const int ct = wave + 4 * k;
    if (ct >= tiles) break;
    // rows half * dp / 2 + j of the state meet columns half * dp / 2 + j of Qd
    const float* s = w.S + tile * dp * ep + (size_t)ct * dp * 32 + half * (dp / 2) * 32 + l32;
    const float* q = Qs + l32 * LD + half * (dp / 2);
    for (int j = 0; j < dp / 2; j += 16) {
      float sv[16];
#pragma unroll
      for (int e = 0; e < 16; ++e) sv[e] = s[(j + e) * 32];
#pragma unroll
      for (int e = 0; e < 16; e += 4) {
        const f4 a4 = *reinterpret_cast<const f4*>(q + j + e);
#pragma unroll
        for (int k4 = 0; k4 < 4; ++k4) o[k] = __builtin_amdgcn_mfma_f32_32x32x2f32(a4[k4], sv[e + k4], o[k], 0, 0, 0);
      }
    }
    const float* u = w.U + tile * 32 * ep + ct * 1024 + 16 * half * 32 + l32;
    float uv[16];
#pragma unroll
    for (int e = 0; e < 16; ++e) uv[e] = u[e * 32];
#pragma unroll
    for (int e = 0; e < 16; e += 4) {
      const f4 a4 = *reinterpret_cast<const f4*>(&Ps[l32][16 * half + e]);
#pragma unroll
      for (int k4 = 0; k4 < 4; ++k4) o[k] = __builtin_amdgcn_mfma_f32_32x32x2f32(a4[k4], uv[e + k4], o[k], 0, 0, 0);
    }
  }
  // sums of squares per token: over the 32 lanes of a half, then over the wavefronts
#pragma unroll
  for (int v = 0; v < 16; ++v) {
    float x = o[0][v] * o[0][v] + o[1][v] * o[1][v];
#pragma unroll
    for (int off = 16; off > 0; off >>= 1) x += __shfl_xor(x, off, 64);
    if (l32 == 0) ss[wave][8 * (v >> 2) + 4 * half + (v & 3)] = x;
  }
  __syncthreads();
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    const int e = 32 * (wave + 4 * k) + l32;
    if (e >= vdim) break;
    const float norm = KIND == REC_SSD ? 0.0f : c.norm[e] * c.out_scale;
    const float skip = KIND == REC_SSD ? c.skip[h] : 0.0f;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int t = 8 * (v >> 2) + 4 * half + (v & 3);
      if (t >= nt) continue;
      const float sq = (ss[0][t] + ss[1][t]) + (ss[2][t] + ss[3][t]);
      const size_t row = row0 + t;
      if constexpr (KIND == REC_SSD) {
        const float x = r.conv_out[row * c.conv.channels + (c.v_col - c.conv.col) + h * vdim + e];
        r.out[row * r.ld_out + c.out_col + h * vdim + e] =
            (o[k][v] + skip * x) * silu(r.y[row * r.ld_y + c.g_col + h * vdim + e]);
        continue;
      }
      if constexpr (KIND == REC_CHANNEL_DELTA) {
        r.out[row * r.ld_out + c.out_col + h * vdim + e] =
            o[k][v] / sqrtf(sq / (float)vdim + c.eps) * norm * sigmoid(r.gate[(row * c.heads + h) * vdim + e]);
        continue;
      }
      r.out[row * r.ld_out + c.out_col + h * vdim + e] =
          o[k][v] / sqrtf(sq / (float)vdim + c.eps) * norm * silu(r.y[row * r.ld_y + c.g_col + h * vdim + e]);
    }
  }
  if (h == 0) {  // padding columns of the mixer outputs
    const int pad = r.ld_out - r.out_cols;
    for (int i = tid; i < nt * pad; i += 256) r.out[(row0 + i / pad) * r.ld_out + r.out_cols + i % pad] = 0.0f;
  }
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

__global__ __launch_bounds__(256) void k_add_norm_rows(float* dst, const float* src, int cols, int ld, const float* gain,
                                                       float eps, const int* slot, const float* weight, int top) {
  __shared__ float red[4];
  constexpr int PER = 8;  // columns a thread keeps; more are read again
  const size_t row = blockIdx.x;
  float* x = dst + row * ld;
  auto value = [&](int i) -> float {
    if (top == 0) return src[row * ld + i];
    float s = 0.0f;
    for (int k = 0; k < top; ++k) s += weight[row * top + k] * src[(size_t)slot[row * top + k] * ld + i];
    return s;
  };
  float keep[PER], old[PER], g[PER], ss = 0.0f;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int i = threadIdx.x + 256 * p;
    const bool in = i < cols;
    old[p] = in ? x[i] : 0.0f;
    g[p] = in ? gain[i] : 0.0f;
    keep[p] = in ? value(i) : 0.0f;
  }
#pragma unroll
  for (int p = 0; p < PER; ++p) ss += keep[p] * keep[p];
  for (int i = threadIdx.x + 256 * PER; i < cols; i += 256) {
    const float v = value(i);
    ss += v * v;
  }
  const float k = 1.0f / sqrtf(block_sum(ss, red) / (float)cols + eps);
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int i = threadIdx.x + 256 * p;
    if (i < cols) x[i] = old[p] + keep[p] * k * g[p];
  }
  for (int i = threadIdx.x + 256 * PER; i < cols; i += 256) x[i] += value(i) * k * gain[i];
}

// Up to four parts of rows of up to 4096 columns: the row is kept in registers.  Otherwise a
// wavefront takes a part at a time.
__global__ __launch_bounds__(256) void k_group_rms_rows(const float* src, int ld_src, float* dst, int ld_dst, int cols,
                                                        int groups, const float* gain, float eps, const int* rows_at) {
  __shared__ float red[4];
  constexpr int PER = 16;
  const size_t row = rows_at ? rows_at[blockIdx.x] : blockIdx.x;
  const float* x = src + row * ld_src;
  float* y = dst + (size_t)blockIdx.x * ld_dst;
  const int n = cols / groups, tid = threadIdx.x, lane = tid & 63;
  if (groups <= 4 && cols <= 256 * PER) {
    float v[PER], g[PER], ss[4] = {0.f, 0.f, 0.f, 0.f}, k[4];
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int i = tid + 256 * p;
      v[p] = i < cols ? x[i] : 0.0f;
      g[p] = i < cols ? gain[i] : 0.0f;
    }
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int i = tid + 256 * p, part = (i >= n) + (i >= 2 * n) + (i >= 3 * n);
#pragma unroll
      for (int q = 0; q < 4; ++q) ss[q] += q == part ? v[p] * v[p] : 0.0f;
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      k[q] = 0.0f;
      if (q < groups) k[q] = 1.0f / sqrtf(block_sum(ss[q], red) / (float)n + eps);
    }
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int i = tid + 256 * p, part = (i >= n) + (i >= 2 * n) + (i >= 3 * n);
      if (i < cols) y[i] = v[p] * (part == 0 ? k[0] : part == 1 ? k[1] : part == 2 ? k[2] : k[3]) * g[p];
    }
  } else if (groups == 1) {
    float ss = 0.0f;
    for (int i = tid; i < n; i += 256) ss += x[i] * x[i];
    const float k = 1.0f / sqrtf(block_sum(ss, red) / (float)n + eps);
    for (int i = tid; i < n; i += 256) y[i] = x[i] * k * gain[i];
  } else {
    for (int g = tid >> 6; g < groups; g += 4) {
      float ss = 0.0f;
      for (int i = lane; i < n; i += 64) ss += x[g * n + i] * x[g * n + i];
      const float k = 1.0f / sqrtf(wave_sum(ss) / (float)n + eps);
      for (int i = lane; i < n; i += 64) y[g * n + i] = x[g * n + i] * k * gain[g * n + i];
    }
  }
  for (int i = cols + tid; i < ld_dst; i += 256) y[i] = 0.0f;
}

__global__ __launch_bounds__(256) void k_begin_step(float* x, const void* table, int table_bf16, const uint32_t* ids,
                                                    int width, StepWords* words) {
  const int b = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
  const size_t at = (size_t)ids[b] * width + i;
  if (i < width)
    x[(size_t)b * width + i] =
        table_bf16 ? __uint_as_float((unsigned)static_cast<const unsigned short*>(table)[at] << 16)
                   : static_cast<const float*>(table)[at];
  if (blockIdx.x == 0 && b == 0) {  // (no other block touches the words)
    const int n = words->n_out, p = words->next;
    uint32_t* out = words->out;
    if (out)
      for (int k = threadIdx.x; k < (int)gridDim.y; k += 256) out[(size_t)n * gridDim.y + k] = ids[k];
    __syncthreads();
    if (threadIdx.x == 0) {
      words->pos = p;
      words->next = p + 1;
      words->n_out = n + 1;
    }
  }
}
__global__ void k_set_words(StepWords* w, int next, uint32_t* out) {
  w->next = next;
  w->out = out;
  w->n_out = 0;
}

// Rows of a state column per thread (recurrence_role): the next power of two.
int rows_per_thread(int dim, int vdim) {
  int cols = 1;
  while (cols < vdim) cols <<= 1;
  const int need = (dim + 256 / cols - 1) / (256 / cols);
  int rpt = 1;
  while (rpt < need) rpt <<= 1;
  return rpt;
}

}  // namespace

// Threads of a decode block.  rows: rows of a state column per thread of a block of 256; blocks grow
// so that a thread holds at most 32 (128 x 128 states, 32 sequences: 36.6 us with 1024 threads,
// 28.4 with 512, 31.4 with 256).
static int decode_threads(int rows) { return rows <= 16 ? 256 : rows <= 64 ? 512 : 1024; }

int mix_decode_splits(const ChunkAttn& a, const Recurrence* rec) {
  const int keys = decode_threads(rec ? rows_per_thread(rec->dim, rec->vdim) : 1) / 4;
  return (a.chunk + keys - 1) / keys;
}

hipError_t launch_mix_decode(const MixDecode& a, hipStream_t s) {
  int attn_items = 0;
  if (a.has_attn) {
    if (a.attn_splits != mix_decode_splits(a.attn, a.has_rec ? &a.rec : nullptr)) return hipErrorInvalidValue;
    const int R = a.attn.heads / a.attn.kv_heads;
    attn_items = a.attn.kv_heads * ((R + kRG - 1) / kRG) * a.attn_splits;
  }
  const int rec_items = a.has_rec ? a.rec.heads : 0;
  const int rows = a.has_rec ? rows_per_thread(a.rec.dim, a.rec.vdim) : 1, nt = decode_threads(rows);
  const int mlp_items = a.has_mlp ? (a.mlp.ff_pad + nt - 1) / nt : 0;
  const dim3 grid((unsigned)(attn_items + rec_items + mlp_items), (unsigned)a.nseq);
  if (grid.x == 0) return hipSuccess;
  const int nv = !a.has_attn || a.attn.dim_pad <= 64 ? 1 : a.attn.dim_pad <= 128 ? 2 : 4;
  switch (rows) {
#define PG_RPT(R, NT, N)                                                                                             \
  case R:                                                                                                            \
    if (nv == 1) hipLaunchKernelGGL((k_mix_decode<NT, N, 1>), grid, dim3(NT), 0, s, a, attn_items, rec_items);        \
    else if (nv == 2) hipLaunchKernelGGL((k_mix_decode<NT, N, 2>), grid, dim3(NT), 0, s, a, attn_items, rec_items);   \
    else hipLaunchKernelGGL((k_mix_decode<NT, N, 4>), grid, dim3(NT), 0, s, a, attn_items, rec_items);                \
    break;
    PG_RPT(1, 256, 1) PG_RPT(2, 256, 2) PG_RPT(4, 256, 4) PG_RPT(8, 256, 8) PG_RPT(16, 256, 16)
    PG_RPT(32, 512, 16) PG_RPT(64, 512, 32) PG_RPT(128, 1024, 32) PG_RPT(256, 1024, 64)
#undef PG_RPT
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

hipError_t launch_recurrence_decode(const MixDecode& a, hipStream_t s) {
  const dim3 grid((unsigned)a.rec.heads, (unsigned)a.nseq);
  if (a.rec.kind != REC_CHANNEL_DELTA && a.rec.kind != REC_SSD) return launch_mix_decode(a, s);
  switch (rows_per_thread(a.rec.dim, a.rec.vdim)) {
#define PG_RPT(R, NT, N)                                                                                     \
  case R:                                                                                                    \
    if (a.rec.kind == REC_SSD)                                                                               \
      hipLaunchKernelGGL((k_recurrence_decode<NT, N, REC_SSD>), grid, dim3(NT), 0, s, a);                     \
    else                                                                                                     \
      hipLaunchKernelGGL((k_recurrence_decode<NT, N, REC_CHANNEL_DELTA>), grid, dim3(NT), 0, s, a);           \
    break;
    PG_RPT(1, 256, 1) PG_RPT(2, 256, 2) PG_RPT(4, 256, 4) PG_RPT(8, 256, 8) PG_RPT(16, 256, 16)
    PG_RPT(32, 512, 16) PG_RPT(64, 512, 32) PG_RPT(128, 1024, 32) PG_RPT(256, 1024, 64)
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
  const dim3 grid(a.heads, (r.n + 31) / 32, r.nseq);
  int dp = (a.dim + 31) / 32 * 32;
  if (dp > 160) dp = 256;
  // (as many wavefronts as the LDS of a CU holds tiles for)
  switch (dp) {
#define PG_DP(N, W)                                                                      \
  case N:                                                                                \
    hipLaunchKernelGGL((k_chunk_attn_rows<N, W>), grid, dim3(64 * W), 0, s, r, a);        \
    break;
    PG_DP(32, 4) PG_DP(64, 4) PG_DP(96, 4) PG_DP(128, 4) PG_DP(160, 2) PG_DP(256, 2)
#undef PG_DP
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

hipError_t launch_short_conv_rows(const MixRows& r, const ShortConv& c, hipStream_t s) {
  const dim3 grid((c.channels + 255) / 256, (r.n + kConvRows - 1) / kConvRows, r.nseq);
  if (c.taps <= 4)
    hipLaunchKernelGGL(k_short_conv_rows<4>, grid, dim3(256), 0, s, r, c);
  else
    hipLaunchKernelGGL(k_short_conv_rows<kMixMaxTaps>, grid, dim3(256), 0, s, r, c);
  return hipGetLastError();
}

// Key size as the chunk kernels pad it: 32 rows of the state to a wavefront, and numbers of
// wavefronts that k_chunk_states is instantiated for.
static int chunk_dim(int dim) {
  const int waves = (dim + 31) / 32;
  return 32 * (waves == 5 ? 6 : waves == 7 ? 8 : waves);
}

size_t recurrence_work_floats(const Recurrence& c, int nseq, int n) {
  const int dp = chunk_dim(c.dim), ep = (c.vdim + 31) / 32 * 32;
  return chunk_floats(dp, ep, rec_reads_state(c.kind)) * (size_t)nseq * ((n + kChunk - 1) / kChunk) * c.heads;
}

hipError_t launch_recurrence_rows(const MixRows& r, const Recurrence& c, hipStream_t s) {
  ChunkWork w{};
  w.chunks = (r.n + kChunk - 1) / kChunk;
  w.dp = chunk_dim(c.dim);
  w.ep = (c.vdim + 31) / 32 * 32;
  const size_t tiles = (size_t)r.nseq * w.chunks * c.heads;
  if (r.work_floats < recurrence_work_floats(c, r.nseq, r.n)) return hipErrorInvalidValue;
  float* at = r.work;
  auto take = [&](size_t per_tile) {
    float* p = at;
    at += per_tile * tiles;
    return p;
  };
  w.S = take((size_t)w.dp * w.ep);
  w.Kd = take((size_t)32 * w.dp);
  w.Qd = take((size_t)32 * w.dp);
  w.U = take((size_t)32 * w.ep);
  w.P = take(1024);
  w.G = take(w.dp);
  const bool delta = rec_reads_state(c.kind);
  if (delta) {
    w.W = take((size_t)32 * w.dp);
    w.U0 = take((size_t)32 * w.ep);
  }
  const dim3 grid(w.chunks, c.heads, r.nseq);
  const int waves = w.dp / 32;
  // (large heads: more LDS than a launch gets by default)
  if (w.dp > 128) {
    const int most = 100 * 1024;
    const void* kernel = c.kind == REC_DELTA ? reinterpret_cast<const void*>(&k_delta_chunk)
                         : c.kind == REC_SSD ? reinterpret_cast<const void*>(&k_ssd_chunk)
                                             : reinterpret_cast<const void*>(&k_gla_chunk);
    if (c.kind != REC_CHANNEL_DELTA) {
      hipError_t e = hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, most);
      if (e != hipSuccess) return e;
    }
  }
  if (c.kind == REC_CHANNEL_DELTA) {
    const size_t lds = 4 * 32 * (size_t)(w.dp + 1) * sizeof(float);
    if (lds > 48 * 1024) {
      hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_channel_delta_chunk),
                                         hipFuncAttributeMaxDynamicSharedMemorySize, 140 * 1024);
      if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(k_channel_delta_chunk, grid, dim3(256), lds, s, r, c, w);
  } else if (c.kind == REC_SSD) {
    const size_t lds = 2 * 32 * (size_t)(w.dp + 4) * sizeof(float);
    hipLaunchKernelGGL(k_ssd_chunk, grid, dim3(256), lds, s, r, c, w);
  } else if (c.kind == REC_DELTA) {
    const size_t lds = 2 * 32 * (size_t)(w.dp + 4) * sizeof(float);
    hipLaunchKernelGGL(k_delta_chunk, grid, dim3(256), lds, s, r, c, w);
  } else {
    const int rows = r.nseq * r.n;
    hipLaunchKernelGGL(k_gla_decay_rows, dim3((c.heads * c.dim + 255) / 256, (rows + kDecayRows - 1) / kDecayRows),
                       dim3(256), 0, s, r, c, rows);
    const size_t lds = 3 * 32 * (size_t)(w.dp + 1) * sizeof(float);
    hipLaunchKernelGGL(k_gla_chunk, grid, dim3(256), lds, s, r, c, w);
  }
  hipError_t e = hipGetLastError();
  if (e != hipSuccess) return e;
  const dim3 sgrid(w.ep / 16, c.heads, r.nseq);
  const size_t slds = delta ? 2 * waves * 512 * sizeof(float) : 0;
  switch (waves) {
#define PG_WAVES(N)                                                                                          \
  case N:                                                                                                    \
    if (delta) hipLaunchKernelGGL((k_chunk_states<true, N>), sgrid, dim3(64 * N), slds, s, r, c, w);        \
    else hipLaunchKernelGGL((k_chunk_states<false, N>), sgrid, dim3(64 * N), slds, s, r, c, w);               \
    break;
    PG_WAVES(1) PG_WAVES(2) PG_WAVES(3) PG_WAVES(4) PG_WAVES(6) PG_WAVES(8)
#undef PG_WAVES
    default: return hipErrorInvalidValue;
  }
  if ((e = hipGetLastError()) != hipSuccess) return e;
  const size_t olds = 32 * (size_t)(w.dp + 4) * sizeof(float);
  if (c.kind == REC_SSD) hipLaunchKernelGGL(k_chunk_out<REC_SSD>, grid, dim3(256), olds, s, r, c, w);
  else if (c.kind == REC_CHANNEL_DELTA) hipLaunchKernelGGL(k_chunk_out<REC_CHANNEL_DELTA>, grid, dim3(256), olds, s, r, c, w);
  else hipLaunchKernelGGL(k_chunk_out<REC_GLA>, grid, dim3(256), olds, s, r, c, w);
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

hipError_t launch_add_norm_rows(float* dst, const float* src, int rows, int cols, int ld, const float* gain, float eps,
                                const int* slot, const float* weight, int top, hipStream_t s) {
  hipLaunchKernelGGL(k_add_norm_rows, dim3(rows), dim3(256), 0, s, dst, src, cols, ld, gain, eps, slot, weight, top);
  return hipGetLastError();
}

hipError_t launch_group_rms_rows(const float* src, int ld_src, float* dst, int ld_dst, int rows, int cols, int groups,
                                 const float* gain, float eps, const int* rows_at, hipStream_t s) {
  if (groups < 1 || cols % groups != 0) return hipErrorInvalidValue;
  hipLaunchKernelGGL(k_group_rms_rows, dim3(rows), dim3(256), 0, s, src, ld_src, dst, ld_dst, cols, groups, gain, eps,
                     rows_at);
  return hipGetLastError();
}

hipError_t launch_begin_step(float* x, const void* table, int table_bf16, const uint32_t* ids, int nseq, int width,
                             StepWords* words, hipStream_t s) {
  hipLaunchKernelGGL(k_begin_step, dim3((width + 255) / 256, nseq), dim3(256), 0, s, x, table, table_bf16, ids, width,
                     words);
  return hipGetLastError();
}
hipError_t launch_set_words(StepWords* words, int next, uint32_t* out, hipStream_t s) {
  hipLaunchKernelGGL(k_set_words, dim3(1), dim3(1), 0, s, words, next, out);
  return hipGetLastError();
}

}  // namespace pgk
