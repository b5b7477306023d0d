// gfx950 kernels of latent attention (pg_mixers.h): windowed softmax attention with a sink whose keys
// and values are projections of one cached latent row per position.  All arithmetic is f32 (angles:
// the product position * frequency is reduced to one turn in f64).
//
// One token: the queries are brought to the latent space (W_uk^T q), attend the cached rows as they
// are, and the weighted sum of latents goes through W_uv.  Many rows: the latents are expanded to
// keys and values by a product and attended 32 keys at a time.
//
// Shapes are checked on the host before any launch (pg_stack.cpp); kernels guard ragged tails.
#include "pg_mixers.h"

#include <math.h>

#include <algorithm>

namespace pgk {

namespace {

typedef float f4 __attribute__((ext_vector_type(4)));
typedef float f16v __attribute__((ext_vector_type(16)));

constexpr float kLog2e = 1.44269504088896341f;
constexpr float kNone = -1e30f;  // a running maximum before the first key

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
  return v;
}
__device__ __forceinline__ float block_sum(float v, float* red) {  // 256 threads
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
template <bool BF16>
__device__ __forceinline__ f4 load_w4(const void* w, size_t at) {
  if (BF16) {
    const uint2 u = *reinterpret_cast<const uint2*>(static_cast<const unsigned short*>(w) + at);
    return f4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
              __uint_as_float(u.y & 0xffff0000u)};
  }
  return *reinterpret_cast<const f4*>(static_cast<const float*>(w) + at);
}

// The cached row of the position whose projections are src[kv_rank + rot_dim]: the latent normed, the
// rest rotated (a block of 256 threads).
__device__ void latent_row(const LatentAttn& a, const float* src, int pos, float* dst, float* red) {
  float ss = 0.0f;
  for (int i = threadIdx.x; i < a.kv_rank; i += 256) ss += src[i] * src[i];
  const float k = 1.0f / sqrtf(block_sum(ss, red) / (float)a.kv_rank + a.eps);
  for (int i = threadIdx.x; i < a.kv_pad; i += 256) dst[i] = i < a.kv_rank ? src[i] * k * a.c_norm[i] : 0.0f;
  const float* rs = src + a.kv_rank;
  for (int i = threadIdx.x; i < (a.ld - a.kv_pad) / 2; i += 256) {
    float u = 2 * i < a.rot_dim ? rs[2 * i] : 0.0f, v = 2 * i + 1 < a.rot_dim ? rs[2 * i + 1] : 0.0f;
    if (i < a.half) {
      float s, c;
      turn(pos, a.freq[i], &s, &c);
      s *= a.mag;
      c *= a.mag;
      const float u0 = u;
      u = u0 * c - v * s;
      v = v * c + u0 * s;
    }
    dst[a.kv_pad + 2 * i] = u;
    dst[a.kv_pad + 2 * i + 1] = v;
  }
}

// ---- one token per sequence ----
// Queries in the latent space, times scale and log2(e): blocks (h < heads, part of 128 latent
// columns); block (heads, 0) writes the token's row of the cache.
template <bool BF16>
__global__ __launch_bounds__(256) void k_latent_query(LatentDecode m, LatentAttn a) {
  __shared__ float qs[kMixMaxDim], red[4];
  __shared__ __attribute__((aligned(16))) float sums[8][128];
  constexpr int PRE = 16;
  const int tid = threadIdx.x, h = blockIdx.x, b = blockIdx.z, pos = *m.d_pos;
  if (h == a.heads) {
    if (blockIdx.y == 0)
      latent_row(a, m.y + (size_t)b * m.ld_y + a.c_col, pos,
                 a.ring + (size_t)b * a.ring_seq + (size_t)(pos % a.window) * a.ld, red);
    return;
  }
  const float* q = m.q + ((size_t)b * a.heads + h) * (a.dim + a.rot_dim);
  float* qa = m.qa + ((size_t)b * a.heads + h) * a.ld;
  const float mul = a.scale * kLog2e, mine = q[min(tid, a.dim - 1)];
  // 32 threads to the 128 columns, four each; eight groups take every eighth row of W_uk
  const int col = blockIdx.y * 128 + (tid & 31) * 4, grp = tid >> 5;
  const size_t w0 = (size_t)h * a.dim * a.kv_pad + min(col, a.kv_pad - 4);
  f4 w[PRE];
#pragma unroll
  for (int i = 0; i < PRE; ++i) w[i] = load_w4<BF16>(a.up_w, w0 + (size_t)min(grp + 8 * i, a.dim - 1) * a.kv_pad);
  if (tid < a.dim) qs[tid] = mine;
  __syncthreads();
  f4 sum = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < PRE; ++i)
    if (grp + 8 * i < a.dim) sum += w[i] * qs[grp + 8 * i];
#pragma unroll 8
  for (int d = grp + 8 * PRE; d < a.dim; d += 8) sum += load_w4<BF16>(a.up_w, w0 + (size_t)d * a.kv_pad) * qs[d];
  *reinterpret_cast<f4*>(&sums[grp][(tid & 31) * 4]) = sum;
  __syncthreads();
  if (tid < 128 && blockIdx.y * 128 + tid < a.kv_pad) {
    float s = 0.0f;
#pragma unroll
    for (int g = 0; g < 8; ++g) s += sums[g][tid];
    qa[blockIdx.y * 128 + tid] = s * mul;
  }
  if (blockIdx.y == 0) {
    const float* rq = q + a.dim;
    for (int i = tid; i < (a.ld - a.kv_pad) / 2; i += 256) {
      float u = 2 * i < a.rot_dim ? rq[2 * i] : 0.0f, v = 2 * i + 1 < a.rot_dim ? rq[2 * i + 1] : 0.0f;
      if (i < a.half) {
        float s, c;
        turn(pos, a.freq[i], &s, &c);
        s *= a.mag;
        c *= a.mag;
        const float u0 = u;
        u = u0 * c - v * s;
        v = v * c + u0 * s;
      }
      qa[a.kv_pad + 2 * i] = u * mul;
      qa[a.kv_pad + 2 * i + 1] = v * mul;
    }
  }
}

// Sixteen heads against a share of the cached rows, 32 rows at a time, on the f32 matrix cores
// (v_mfma_f32_16x16x4_f32: A operand lane l -> A[l % 16][l / 16], B operand lane l -> B[l / 16][l % 16],
// D lane l, register v -> D[4 (l / 16) + v][l % 16]):
//   S (rows x heads): wavefront w takes rows 16 (w % 2) .. and every second 16 columns of them from
//     16 (w / 2) on; four columns of a lane's quarter per step
//   softmax over the rows in LDS, running maximum and sum per head
//   O (heads x latent columns) += P . C: wavefront w owns the 16-column tiles w, w + 4, ...
// Everything a tile needs is asked for before the first of it is used.  Which position a row of the
// ring holds does not matter: the first min(position + 1, window) rows are the ones that the token
// sees.  Grid: x = share, y = 16 heads, z = sequence.  NT: column tiles of a wavefront; a row has at most
// 64 NT + ROT columns.
constexpr int kShareRows = 32;
constexpr int kLatentGroup = 6;  // steps taken together
constexpr int latent_steps(int nt, int rot) {
  return ((64 * nt + rot) / 32 + kLatentGroup - 1) / kLatentGroup * kLatentGroup;
}
static_assert(32 * kLatentGroup <= kLatentTail, "what a group may read past a row");
template <int NT, int ROT>
__global__ __launch_bounds__(256, NT <= 8 && ROT <= 64 ? 2 : 1) void k_latent_attn(LatentDecode m, LatentAttn a) {
  constexpr int NS = latent_steps(NT, ROT), G = kLatentGroup, LD = 32 * NS + 4;
  extern __shared__ __attribute__((aligned(16))) float qs[];  // [16][LD], zeros past a row's columns
  __shared__ __attribute__((aligned(16))) float ps[2][16][36];
  __shared__ __attribute__((aligned(16))) float ms[16], ls[16], al[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int quarter = lane >> 4, l16 = lane & 15;
  const int split = blockIdx.x, h0 = blockIdx.y * 16, b = blockIdx.z;
  const int nh = min(16, a.heads - h0), ld = a.ld;
  const int pos = *m.d_pos, n = min(pos + 1, a.window);
  const int per = ((a.window + m.splits - 1) / m.splits + kShareRows - 1) / kShareRows * kShareRows;
  const int j0 = split * per, j1 = min(n, j0 + per);
  float* part = m.part + (((size_t)b * a.heads + h0) * m.splits + split) * (a.kv_pad + 2);
  const size_t part_h = (size_t)m.splits * (a.kv_pad + 2);
  if (j0 >= n) {
    if (tid < nh) {
      part[tid * part_h + a.kv_pad] = kNone;
      part[tid * part_h + a.kv_pad + 1] = 0.0f;
    }
    return;
  }
  const float* ring = a.ring + (size_t)b * a.ring_seq;
  const int tiles = a.kv_pad / 16, first = wave >> 1, rows16 = 16 * (wave & 1);
  const int mine = (ld / 16 - first + 1) / 2;  // steps of this wavefront: 16 columns from 16 (first + 2 s) on
  // sixteen threads to a head
  f4 qr[NS / 2];
  {
    const int h = tid >> 4;
    const float* q = m.qa + ((size_t)b * a.heads + h0 + min(h, nh - 1)) * ld + 4 * (tid & 15);
#pragma unroll
    for (int i = 0; i < NS / 2; ++i) {
      qr[i] = f4{0.f, 0.f, 0.f, 0.f};
      if (h < nh && 4 * (tid & 15) + 64 * i < ld) qr[i] = *reinterpret_cast<const f4*>(q + 64 * i);
    }
  }
  f4 kr[NS];
  float cr[NT][8];
  auto fetch = [&](int k0) __attribute__((always_inline)) {
    // (whole groups of steps: past the row's columns lies the next row, or what the ring ends with)
    const float* row = ring + (size_t)min(k0 + rows16 + l16, j1 - 1) * ld + 16 * first + 4 * quarter;
#pragma unroll
    for (int s = 0; s < NS; ++s)
      if (s / G * G < mine) kr[s] = *reinterpret_cast<const f4*>(row + 32 * s);
    const float* col[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) col[k] = ring + (size_t)min(k0 + 4 * k + quarter, j1 - 1) * ld + 16 * wave + l16;
#pragma unroll
    for (int t = 0; t < NT; ++t)
      if (wave + 4 * t < tiles) {
#pragma unroll
        for (int k = 0; k < 8; ++k) cr[t][k] = col[k][64 * t];
      }
  };
  fetch(j0);
#pragma unroll
  for (int i = 0; i < NS / 2; ++i) *reinterpret_cast<f4*>(&qs[(tid >> 4) * LD + 4 * (tid & 15) + 64 * i]) = qr[i];
  if (tid < 16) {
    ms[tid] = kNone;
    ls[tid] = 0.0f;
  }
  f4 o[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) o[t] = f4{0.f, 0.f, 0.f, 0.f};
  __syncthreads();
  for (int k0 = j0; k0 < j1; k0 += kShareRows) {
    {
      const float* q = qs + l16 * LD + 16 * first + 4 * quarter;
      f4 s0 = f4{0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
      for (int g = 0; g < NS / G; ++g) {
        if (g * G >= mine) break;
        f4 q4[G];
#pragma unroll
        for (int s = 0; s < G; ++s) q4[s] = *reinterpret_cast<const f4*>(q + 32 * (g * G + s));
#pragma unroll
        for (int s = 0; s < G; ++s) {
          const f4 k4 = kr[g * G + s];
          s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.x, q4[s].x, s0, 0, 0, 0);
          s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.y, q4[s].y, s1, 0, 0, 0);
          s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.z, q4[s].z, s0, 0, 0, 0);
          s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.w, q4[s].w, s1, 0, 0, 0);
        }
      }
      *reinterpret_cast<f4*>(&ps[first][l16][rows16 + 4 * quarter]) = s0 + s1;
    }
    __syncthreads();
    {
      // sixteen lanes to a head, two rows each
      const int h = 4 * wave + quarter, key = 2 * l16;
      const float2 p0 = *reinterpret_cast<const float2*>(&ps[0][h][key]);
      const float2 p1 = *reinterpret_cast<const float2*>(&ps[1][h][key]);
      const float z0 = k0 + key < j1 ? p0.x + p1.x : -INFINITY, z1 = k0 + key + 1 < j1 ? p0.y + p1.y : -INFINITY;
      float mx = fmaxf(z0, z1);
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
      const float old = ms[h], now = fmaxf(old, mx);
      const float w0 = __builtin_amdgcn_exp2f(z0 - now), w1 = __builtin_amdgcn_exp2f(z1 - now);
      float sum = w0 + w1;
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) sum += __shfl_xor(sum, off, 64);
      *reinterpret_cast<float2*>(&ps[0][h][key]) = float2{w0, w1};
      if (l16 == 0) {
        const float f = __builtin_amdgcn_exp2f(old - now);
        al[h] = f;
        ms[h] = now;
        ls[h] = ls[h] * f + sum;
      }
    }
    __syncthreads();
    {
      float p[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) p[k] = ps[0][l16][4 * k + quarter];
      if (k0 > j0) {
        const f4 f = *reinterpret_cast<const f4*>(&al[4 * quarter]);
#pragma unroll
        for (int t = 0; t < NT; ++t) o[t] *= f;
      }
#pragma unroll
      for (int t = 0; t < NT; ++t)
        if (wave + 4 * t < tiles) {
#pragma unroll
          for (int k = 0; k < 8; ++k) o[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(p[k], cr[t][k], o[t], 0, 0, 0);
        }
    }
    if (k0 + kShareRows < j1) {
      fetch(k0 + kShareRows);
      __syncthreads();
    }
  }
  float* dst[4];
#pragma unroll
  for (int v = 0; v < 4; ++v) dst[v] = part + (4 * quarter + v) * part_h + 16 * wave + l16;
#pragma unroll
  for (int t = 0; t < NT; ++t)
    if (wave + 4 * t < tiles) {
#pragma unroll
      for (int v = 0; v < 4; ++v)
        if (4 * quarter + v < nh) dst[v][64 * t] = o[t][v];
    }
  if (tid < nh) {
    part[tid * part_h + a.kv_pad] = ms[tid];
    part[tid * part_h + a.kv_pad + 1] = ls[tid];
  }
}

// The shares' sums brought together with the sink, and 32 rows of W_uv.  Grid: x = head, y = rows of
// W_uv, z = sequence.  NC: 256-column pieces of a latent.
constexpr int kMaxShares = 64;
template <int NC, bool BF16>
__global__ __launch_bounds__(256) void k_latent_out(LatentDecode m, LatentAttn a) {
  __shared__ __attribute__((aligned(16))) float os[256 * NC];
  __shared__ float ws[kMaxShares];
  constexpr int PRE = 16;  // shares asked for before their weights are known
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, b = blockIdx.z;
  const int e0 = blockIdx.y * 32 + wave, last = m.splits - 1;
  const size_t ps = a.kv_pad + 2;
  const float* part = m.part + ((size_t)b * a.heads + h) * m.splits * ps;
  const float sink = a.sink[h] * kLog2e;
  // a share per lane
  const float* pl = part + min(lane, last) * ps + a.kv_pad;
  const float mx = lane <= last ? pl[0] : kNone, l = lane <= last ? pl[1] : 0.0f;
  float x[NC][PRE];
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int s = 0; s < PRE; ++s) x[c][s] = part[min(s, last) * ps + min(tid + 256 * c, a.kv_pad - 1)];
  f4 w[8][NC];
#pragma unroll
  for (int r = 0; r < 8; ++r)
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const size_t row = (size_t)a.v_row + h * a.vdim + min(e0 + 4 * r, a.vdim - 1);
      w[r][c] = load_w4<BF16>(a.up_w, row * a.kv_pad + min(4 * lane + 256 * c, a.kv_pad - 4));
    }
  if (wave == 0) {
    float top = fmaxf(mx, sink);
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) top = fmaxf(top, __shfl_xor(top, off, 64));
    const float f = l > 0.0f ? exp2f(mx - top) : 0.0f;
    const float sum = wave_sum(l * f) + exp2f(sink - top);
    ws[lane] = f / sum;
  }
  __syncthreads();
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = tid + 256 * c;
    float o = 0.0f;
    // (a share without rows has left its sums unwritten)
#pragma unroll
    for (int s = 0; s < PRE; ++s)
      if (s <= last && ws[s] != 0.0f) o += ws[s] * x[c][s];
    const float* p = part + min(i, a.kv_pad - 1);
#pragma unroll 8
    for (int s = PRE; s <= last; ++s) {
      const float f = ws[s], y = p[s * ps];
      o += f != 0.0f ? f * y : 0.0f;
    }
    os[i] = i < a.kv_pad ? o : 0.0f;
  }
  __syncthreads();
  f4 o[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) o[c] = *reinterpret_cast<const f4*>(&os[4 * lane + 256 * c]);
#pragma unroll
  for (int r = 0; r < 8; ++r) {
    float s = 0.0f;
#pragma unroll
    for (int c = 0; c < NC; ++c)
      s += (w[r][c].x * o[c].x + w[r][c].y * o[c].y) + (w[r][c].z * o[c].z + w[r][c].w * o[c].w);
    s = wave_sum(s);
    if (lane == 0 && e0 + 4 * r < a.vdim) m.out[(size_t)b * m.ld_out + a.out_col + h * a.vdim + e0 + 4 * r] = s;
  }
}

// ---- many rows ----
// x: cached rows of the history, then the step's rows; y: sequence
__global__ __launch_bounds__(256) void k_latent_prepare_rows(MixRows r, LatentAttn a, LatentRows l) {
  __shared__ float red[4];
  const int j = blockIdx.x, b = blockIdx.y, pos = r.pos0 - l.hist + j;
  float* dst = l.lat + ((size_t)b * (l.hist + r.n) + j) * a.ld;
  if (j < l.hist) {
    const float* src = a.ring + (size_t)b * a.ring_seq + (size_t)(pos % a.window) * a.ld;
    for (int i = threadIdx.x; i < a.ld; i += 256) dst[i] = src[i];
    return;
  }
  const size_t row = (size_t)b * r.n + (j - l.hist);
  const float* y = r.y + row * r.ld_y;
  latent_row(a, y + a.c_col, pos, dst, red);
  const float* q = y + a.q_col;
  float* cq = l.cq + row * a.q_pad;
  float ss = 0.0f;
  for (int i = threadIdx.x; i < a.q_rank; i += 256) ss += q[i] * q[i];
  const float k = 1.0f / sqrtf(block_sum(ss, red) / (float)a.q_rank + a.eps);
  for (int i = threadIdx.x; i < a.q_pad; i += 256) cq[i] = i < a.q_rank ? q[i] * k * a.q_norm[i] : 0.0f;
}

__global__ __launch_bounds__(256) void k_latent_rotate_rows(MixRows r, LatentAttn a, LatentRows l) {
  __shared__ float cs[kMixMaxDim / 2], sn[kMixMaxDim / 2];
  const int t = blockIdx.x, b = blockIdx.y, pos = r.pos0 + t;
  const size_t row = (size_t)b * r.n + t;
  for (int i = threadIdx.x; i < a.half; i += 256) {
    float s, c;
    turn(pos, a.freq[i], &s, &c);
    sn[i] = s * a.mag;
    cs[i] = c * a.mag;
  }
  __syncthreads();
  const int per = a.dim + a.rot_dim;
  float* q = l.q + row * a.heads * per + a.dim;
  for (int i = threadIdx.x; i < a.heads * a.half; i += 256) {
    const int h = i / a.half, e = i - h * a.half;
    float* p = q + (size_t)h * per + 2 * e;
    const float u = p[0], v = p[1];
    p[0] = u * cs[e] - v * sn[e];
    p[1] = v * cs[e] + u * sn[e];
  }
  for (int i = r.out_cols + threadIdx.x; i < r.ld_out; i += 256) r.out[row * r.ld_out + i] = 0.0f;
  if (t >= r.n - a.window) {
    const float* src = l.lat + ((size_t)b * (l.hist + r.n) + l.hist + t) * a.ld;
    float* dst = a.ring + (size_t)b * a.ring_seq + (size_t)(pos % a.window) * a.ld;
    for (int i = threadIdx.x; i < a.ld; i += 256) dst[i] = src[i];
  }
}

// Four wavefronts: 4 / KG groups of 32 queries of one head times KG shares of the keys.  The
// wavefronts of a share stage its key tiles (32 keys: unrotated and rotated part side by side, and
// the values) in LDS together; the next tile waits in registers.  Per tile
//   S^T (keys x queries) = K . Q^T, Q in registers (lane (l, half) holds dims half DP / 2 ..)
//   online softmax per query: a lane and the one 32 away hold 16 keys each of query l
//   O^T (dims x queries) += V^T . P^T, a lane's own weights are the operand
// The sink is the first key's predecessor: maximum sink, sum 1, no value.  Shares are merged through
// LDS.  Grid: x = head, y = queries, longest first, z = sequence.
template <int DP, int DV, int KG>
__global__ __launch_bounds__(256, 1) void k_latent_attn_rows(MixRows r, LatentAttn a, LatentRows l) {
  constexpr int KT = 32, LDK = DP + 4, LDV = DV + 4, NB = DV / 32, QG = 4 / KG;
  constexpr int TH = 64 * QG;                 // threads that stage a share's tiles
  constexpr int NK = KT * DP / 4 / TH, NV = KT * DV / 4 / TH;
  constexpr int TILE = KT * (LDK + LDV);
  extern __shared__ __attribute__((aligned(16))) float lds[];  // [KG][K tile, V tile]
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int qg = wave % QG, kg = wave / QG, st = tid % TH;
  const int half = lane >> 5, l32 = lane & 31;
  const int h = blockIdx.x, b = blockIdx.z;
  const int nqb = (r.n + 32 * QG - 1) / (32 * QG);
  const int t0 = (nqb - 1 - (int)blockIdx.y) * 32 * QG;  // first query of the block
  const int tq = t0 + 32 * qg + l32;
  const int dim = a.dim, rot = a.rot_dim, dk = dim + rot, vdim = a.vdim;
  const bool vec = ((dim | rot | vdim) & 3) == 0;  // (rows and heads then start at multiples of 4)
  const size_t rows = (size_t)l.hist + r.n;
  const float* kb = l.kv + (size_t)b * rows * l.ld_kv + h * dim;
  const float* vb = l.kv + (size_t)b * rows * l.ld_kv + a.v_row + h * vdim;
  const float* rb = l.lat + (size_t)b * rows * a.ld + a.kv_pad;

  float qr[DP / 2];
  {
    const float* q = l.q + ((size_t)b * r.n + min(tq, r.n - 1)) * a.heads * dk + (size_t)h * dk;
#pragma unroll
    for (int s = 0; s < DP / 2; ++s) {
      const int d = half * (DP / 2) + s;
      qr[s] = d < dk ? q[min(d, dk - 1)] : 0.0f;
    }
  }
  f16v o[NB];
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) o[i][v] = 0.0f;
  // keys as rows j of kv: query t sees rows hist + t - window + 1 .. hist + t
  const int jq = l.hist + tq;
  const int jl = l.hist + min(t0 + 32 * QG, r.n) - 1;           // last key of the block
  const int jf = max(0, l.hist + t0 - a.window + 1);            // first
  const int lo = jq - a.window + 1;
  const int tiles = (jl - jf) / KT + 1, turns = (tiles + KG - 1) / KG;
  const float zs = a.scale * kLog2e;
  float mx = kg == 0 ? a.sink[h] * kLog2e : kNone, sum = kg == 0 && half == 0 ? 1.0f : 0.0f;
  float* ks = lds + kg * TILE;
  float* vs = ks + KT * LDK;

  // sixteen lanes (eight for narrow values) to 64 (32) columns of a row: column block c, row pass i
  constexpr int VL = DV >= 64 ? 16 : 8;
  constexpr int KC = DP / 64, KR = 32 * 16 / TH, VC = DV / (4 * VL), VR = 32 * VL / TH > 0 ? 32 * VL / TH : 1;
  static_assert(KC * KR == NK && VC * VR == NV, "whole passes");
  const int ki = st >> 4, kd = (st & 15) * 4, vi = st / VL, vd = (st % VL) * 4;
  f4 kreg[NK], vreg[NV];
  auto fetch = [&](int tile) __attribute__((always_inline)) {
    const int j0 = jf + tile * KT;
    if (vec) {
#pragma unroll
      for (int i = 0; i < KR; ++i) {
        const int j = min(j0 + ki + TH / 16 * i, jl);
        const float *k = kb + (size_t)j * l.ld_kv, *x = rb + (size_t)j * a.ld - dim;
#pragma unroll
        for (int c = 0; c < KC; ++c) {
          const int d = kd + 64 * c;
          kreg[i * KC + c] = f4{0.f, 0.f, 0.f, 0.f};
          if (d < dk) kreg[i * KC + c] = *reinterpret_cast<const f4*>((d < dim ? k : x) + d);
        }
      }
#pragma unroll
      for (int i = 0; i < VR; ++i) {
        const float* v = vb + (size_t)min(j0 + vi + TH / VL * i, jl) * l.ld_kv;
#pragma unroll
        for (int c = 0; c < VC; ++c) {
          const int d = vd + 4 * VL * c;
          vreg[i * VC + c] = f4{0.f, 0.f, 0.f, 0.f};
          if (d < vdim) vreg[i * VC + c] = *reinterpret_cast<const f4*>(v + d);
        }
      }
      return;
    }
#pragma unroll
    for (int i = 0; i < KR; ++i) {
      const int j = min(j0 + ki + TH / 16 * i, jl);
      const float *k = kb + (size_t)j * l.ld_kv, *x = rb + (size_t)j * a.ld - dim;
#pragma unroll
      for (int c = 0; c < KC; ++c)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int d = kd + 64 * c + e;
          kreg[i * KC + c][e] = d < dk ? (d < dim ? k : x)[d] : 0.0f;
        }
    }
#pragma unroll
    for (int i = 0; i < VR; ++i) {
      const float* v = vb + (size_t)min(j0 + vi + TH / VL * i, jl) * l.ld_kv;
#pragma unroll
      for (int c = 0; c < VC; ++c)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int d = vd + 4 * VL * c + e;
          vreg[i * VC + c][e] = d < vdim ? v[d] : 0.0f;
        }
    }
  };
  fetch(min(kg, tiles - 1));
  for (int turn = 0; turn < turns; ++turn) {
    const int tile = turn * KG + kg, k0 = jf + tile * KT;
    __syncthreads();  // (the previous tile has been read)
#pragma unroll
    for (int i = 0; i < KR; ++i)
#pragma unroll
      for (int c = 0; c < KC; ++c) *reinterpret_cast<f4*>(&ks[(ki + TH / 16 * i) * LDK + kd + 64 * c]) = kreg[i * KC + c];
#pragma unroll
    for (int i = 0; i < VR; ++i)
#pragma unroll
      for (int c = 0; c < VC; ++c) *reinterpret_cast<f4*>(&vs[(vi + TH / VL * i) * LDV + vd + 4 * VL * c]) = vreg[i * VC + c];
    __syncthreads();
    if (turn + 1 < turns) fetch(min(tile + KG, tiles - 1));
    // (wavefront-uniform: past the share's last tile, or no query of the group sees the tile)
    if (tile >= tiles || k0 > l.hist + t0 + 32 * qg + 31 || k0 + KT - 1 < l.hist + t0 + 32 * qg - a.window + 1) continue;
    f16v s0, s1;
#pragma unroll
    for (int v = 0; v < 16; ++v) s0[v] = s1[v] = 0.0f;
    const f4* krow = reinterpret_cast<const f4*>(&ks[l32 * LDK + half * (DP / 2)]);
    f4 k = krow[0];
#pragma unroll
    for (int j = 0; j < DP / 8; ++j) {
      const f4 kc = k;
      s0 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.x, qr[4 * j], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.y, qr[4 * j + 1], s1, 0, 0, 0);
      if (j + 1 < DP / 8) k = krow[j + 1];
      __builtin_amdgcn_sched_barrier(0);
      s0 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.z, qr[4 * j + 2], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_32x32x2f32(kc.w, qr[4 * j + 3], s1, 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
    // lane holds keys k0 + 8 (v / 4) + 4 half + v % 4 of its query
    float top = -INFINITY;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int key = k0 + 8 * (v >> 2) + 4 * half + (v & 3);
      s0[v] = key <= jq && key >= lo ? (s0[v] + s1[v]) * zs : -INFINITY;
      top = fmaxf(top, s0[v]);
    }
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    const float now = fmaxf(mx, top), f = __builtin_amdgcn_exp2f(mx - now);
    mx = now;
    sum *= f;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      s0[v] = __builtin_amdgcn_exp2f(s0[v] - now);
      sum += s0[v];
    }
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      float vop[16];
#pragma unroll
      for (int v = 0; v < 16; ++v) vop[v] = vs[(8 * (v >> 2) + 4 * half + (v & 3)) * LDV + 32 * i + l32];
      o[i] *= f;
#pragma unroll
      for (int v = 0; v < 16; ++v) o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(vop[v], s0[v], o[i], 0, 0, 0);
    }
  }
  if constexpr (KG == 2) {
    // the second share's sums through LDS, 32 dims at a time
    __syncthreads();
    float* ob = lds + qg * 32 * 33;
    float* om = lds + QG * 32 * 33 + qg * 128;
    if (kg == 1) {
      om[lane] = mx;
      om[64 + lane] = sum;
    }
    __syncthreads();
    float f0 = 1.0f, f1 = 0.0f;
    if (kg == 0) {
      const float m1 = om[lane], now = fmaxf(mx, m1);
      f0 = exp2f(mx - now);
      f1 = exp2f(m1 - now);
      sum = sum * f0 + om[64 + lane] * f1;
    }
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      if (kg == 1)
#pragma unroll
        for (int v = 0; v < 16; ++v) ob[(8 * (v >> 2) + 4 * half + (v & 3)) * 33 + l32] = o[i][v];
      __syncthreads();
      if (kg == 0)
#pragma unroll
        for (int v = 0; v < 16; ++v) o[i][v] = o[i][v] * f0 + ob[(8 * (v >> 2) + 4 * half + (v & 3)) * 33 + l32] * f1;
      __syncthreads();
    }
    if (kg == 1) return;
  }
  sum += __shfl_xor(sum, 32, 64);
  if (tq >= r.n) return;
  const float inv = 1.0f / sum;
  float* dst = r.out + ((size_t)b * r.n + tq) * r.ld_out + a.out_col + h * vdim;
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int d = 32 * i + 8 * (v >> 2) + 4 * half + (v & 3);
      if (d < vdim) dst[d] = o[i][v] * inv;
    }
}

template <int DP, int DV, int KG>
hipError_t launch_attn_rows(const MixRows& r, const LatentAttn& a, const LatentRows& l, hipStream_t s) {
  constexpr int QG = 4 / KG;
  const size_t tiles = (size_t)KG * 32 * (DP + DV + 8), merge = KG == 2 ? (size_t)QG * (32 * 33 + 128) : 0;
  const size_t lds = std::max(tiles, merge) * sizeof(float);
  if (lds > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_latent_attn_rows<DP, DV, KG>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL((k_latent_attn_rows<DP, DV, KG>), dim3(a.heads, (r.n + 32 * QG - 1) / (32 * QG), r.nseq), dim3(256),
                     lds, s, r, a, l);
  return hipGetLastError();
}

}  // namespace

// Shares of the window: 32 rows each, 64 shares at most.
int latent_decode_splits(const LatentAttn& a) { return std::min(kMaxShares, (a.window + kShareRows - 1) / kShareRows); }

hipError_t launch_latent_decode(const LatentDecode& m, const LatentAttn& a, hipStream_t s) {
  if (a.kv_pad > kLatentMaxRank || a.dim + a.rot_dim > kMixMaxDim || a.vdim > kMixMaxDim || a.kv_pad % 32 != 0 ||
      a.ld % 16 != 0 || a.ld > a.kv_pad + kMixMaxDim || m.splits != latent_decode_splits(a))
    return hipErrorInvalidValue;
  const dim3 qgrid(a.heads + 1, (a.kv_pad + 127) / 128, m.nseq);
  if (a.w_bf16) hipLaunchKernelGGL(k_latent_query<true>, qgrid, dim3(256), 0, s, m, a);
  else hipLaunchKernelGGL(k_latent_query<false>, qgrid, dim3(256), 0, s, m, a);
  const dim3 grid(m.splits, (a.heads + 15) / 16, m.nseq);
#define PG_ATTN(T, R)                                                                                                  \
  {                                                                                                                    \
    constexpr int lds = 16 * (32 * latent_steps(T, R) + 4) * (int)sizeof(float);                                       \
    if (lds > 48 * 1024) {                                                                                             \
      hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_latent_attn<T, R>),                          \
                                         hipFuncAttributeMaxDynamicSharedMemorySize, lds);                             \
      if (e != hipSuccess) return e;                                                                                   \
    }                                                                                                                  \
    hipLaunchKernelGGL((k_latent_attn<T, R>), grid, dim3(256), lds, s, m, a);                                          \
  }
  const bool narrow = a.ld - a.kv_pad <= 64;
  if (a.kv_pad <= 256) {
    if (narrow) PG_ATTN(4, 64) else PG_ATTN(4, 256)
  } else if (a.kv_pad <= 512) {
    if (narrow) PG_ATTN(8, 64) else PG_ATTN(8, 256)
  } else {
    PG_ATTN(16, 256)
  }
#undef PG_ATTN
  const dim3 ogrid(a.heads, (a.vdim + 31) / 32, m.nseq);
#define PG_OUT(C)                                                                               \
  if (a.w_bf16) hipLaunchKernelGGL((k_latent_out<C, true>), ogrid, dim3(256), 0, s, m, a);       \
  else hipLaunchKernelGGL((k_latent_out<C, false>), ogrid, dim3(256), 0, s, m, a);
  if (a.kv_pad <= 256) {
    PG_OUT(1)
  } else if (a.kv_pad <= 512) {
    PG_OUT(2)
  } else {
    PG_OUT(4)
  }
#undef PG_OUT
  return hipGetLastError();
}

hipError_t launch_latent_prepare_rows(const MixRows& r, const LatentAttn& a, const LatentRows& l, hipStream_t s) {
  hipLaunchKernelGGL(k_latent_prepare_rows, dim3(l.hist + r.n, r.nseq), dim3(256), 0, s, r, a, l);
  return hipGetLastError();
}

hipError_t launch_latent_rotate_rows(const MixRows& r, const LatentAttn& a, const LatentRows& l, hipStream_t s) {
  hipLaunchKernelGGL(k_latent_rotate_rows, dim3(r.n, r.nseq), dim3(256), 0, s, r, a, l);
  return hipGetLastError();
}

hipError_t launch_latent_attn_rows(const MixRows& r, const LatentAttn& a, const LatentRows& l, hipStream_t s) {
  if (a.dim + a.rot_dim > kMixMaxDim || a.vdim > kMixMaxDim) return hipErrorInvalidValue;
  int dp = (a.dim + a.rot_dim + 63) / 64 * 64, dv = (a.vdim + 31) / 32 * 32;
  if (dv > 128) dv = 256;
  else if (dv == 96) dv = 128;
  // two shares of the keys where whole groups of queries leave CUs idle
  // (values of more than 128: the registers of two do not fit)
  const bool two = (long)a.heads * ((r.n + 127) / 128) * r.nseq < 256;
#define PG_SHAPE(K, V)                                                         \
  if (dp == K && dv == V) {                                                    \
    if constexpr (V <= 128)                                                    \
      if (two) return launch_attn_rows<K, V, 2>(r, a, l, s);                   \
    return launch_attn_rows<K, V, 1>(r, a, l, s);                              \
  }
  PG_SHAPE(64, 32) PG_SHAPE(64, 64) PG_SHAPE(64, 128) PG_SHAPE(64, 256)
  PG_SHAPE(128, 32) PG_SHAPE(128, 64) PG_SHAPE(128, 128) PG_SHAPE(128, 256)
  PG_SHAPE(192, 32) PG_SHAPE(192, 64) PG_SHAPE(192, 128) PG_SHAPE(192, 256)
  PG_SHAPE(256, 32) PG_SHAPE(256, 64) PG_SHAPE(256, 128) PG_SHAPE(256, 256)
#undef PG_SHAPE
  return hipErrorInvalidValue;
}

}  // namespace pgk
