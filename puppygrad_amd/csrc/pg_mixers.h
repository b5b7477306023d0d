// Launchers of the sequence mixers that a layer of a stack model (pg_stack.h) is made of:
// rotary positions, chunked sigmoid attention, short convolution, gated delta rule, gated
// linear attention, gated MLP activation, RMS norm with one gain.  Every constant of a
// mechanism is a field of its argument struct.
//
// Rows: a step brings n tokens of each of nseq sequences, which all stand at the same
// position.  Row b * n + t of an activation matrix is token t of sequence b, at position
// pos0 + t.  All values are f32.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace pgk {

constexpr int kMixMaxDim = 256;   // key and value sizes per head
constexpr int kMixMaxTaps = 16;   // short convolution

// Rotary positions: the pair (i, i + half) of a head turns by position * freq[i], i < half; the
// head's values from 2 * half on pass unchanged.
struct Rotary {
  const double* freq;
  int half;
};

// Attention inside chunks of `chunk` positions counted from position 0, whose weights are
// sigmoid(q . k * scale + bias[head]) without normalisation; query head h reads key/value head
// h / (heads / kv_heads), and the values are the keys as projected, before rotation.
// The cache of a sequence holds one chunk: kring[kv head][position % chunk][dim_pad] (rotated)
// and vring likewise (as projected).
struct ChunkAttn {
  int heads, kv_heads, dim, dim_pad;
  int chunk;
  float scale;
  const float* bias;
  Rotary rot;
  int q_col, k_col;   // first column of q and k in a row of projections
  float *kring, *vring;
  size_t ring_seq;    // floats from one sequence's ring to the next
  int out_col;        // first column of the result in a row of mixer outputs
  float out_scale;    // multiplies the result
};

// Causal convolution of `taps` taps per channel over the projections of `channels` adjacent
// columns, then silu; w[channel][taps], the last tap is the current token's.  ring[position %
// taps][channels] keeps a sequence's last inputs.
struct ShortConv {
  int channels, taps;
  int col;
  const float* w;
  float* ring;
  size_t ring_seq;
};

// One linear recurrence per head with state S[dim][vdim].
//  delta (gated delta rule): S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q with unit
//    vectors q (times q_scale) and k, beta = sigmoid(b), g = exp(-exp(a_log) softplus(a + dt_bias)).
//    q, k and v are the columns of the short convolution (q | k | v), a and b columns of the
//    projections.
//  otherwise (gated linear attention): S <- diag(alpha) S + k v^T; o = S^T q, alpha =
//    sigmoid(z)^inv_tau, z = a2 . a1 + a2_bias with a1 `rank` columns of the projections.
// Then y = o / rms(o) * norm * silu(gate columns) * out_scale.
struct Recurrence {
  int delta;
  int heads, kv_heads, dim, vdim;
  float q_scale;
  float eps;
  int q_col, k_col, v_col;  // of the projections (q, k, v of the delta rule: inputs of the convolution)
  int g_col;                // output gate
  int a_col, b_col;         // delta: decay and step size; otherwise a_col is a1
  const float *a_log, *dt_bias;
  const float *a2, *a2_bias;
  int rank;
  float inv_tau;
  const float* norm;
  ShortConv conv;           // delta only
  float* state;             // [heads][dim][vdim] per sequence
  size_t state_seq;
  int out_col;
  float out_scale;
};

// act[j] = gelu_tanh(gate[j]) * up[j], j < ff; columns [ff, ff_pad) of act are 0
struct GatedMlp {
  int ff, ff_pad;
  int gate_col, up_col;
};

// One decode step of a layer's mixers for all sequences, in one launch: attention, recurrence and
// gated activation side by side (they read the same row of projections).  *d_pos is the
// position.  With more than one key split (attn_splits > 1) the attention leaves partial sums in
// part[b][split][heads][dim] (zeros for splits without keys); they are added into the mixer
// outputs by launch_attn_sum, or by the projection that reads them (GemvPair::part).
struct MixDecode {
  int nseq;
  const int* d_pos;
  const float* y;     // projections [nseq][ld_y]
  int ld_y;
  float* out;         // mixer outputs [nseq][ld_out]
  int ld_out;
  float* act;         // [nseq][ff_pad]
  int has_attn, has_rec, has_mlp;
  ChunkAttn attn;
  Recurrence rec;
  GatedMlp mlp;
  int attn_splits;
  float* part;
};
// Key splits of a layer's attention (rec: the recurrence beside it, or null).
int mix_decode_splits(const ChunkAttn& a, const Recurrence* rec);
hipError_t launch_mix_decode(const MixDecode& a, hipStream_t s);
hipError_t launch_attn_sum(const MixDecode& a, hipStream_t s);

// ---- many rows ----
struct MixRows {
  int nseq, n, pos0;
  float* y;           // projections [rows][ld_y]; q is rotated in place
  int ld_y;
  float* out;         // mixer outputs [rows][ld_out]
  int ld_out, out_cols;  // columns [out_cols, ld_out) are set to 0
  float* act;
  float* k_rot;       // [rows][kv_heads * dim]: rotated keys
  float* conv_out;    // [rows][channels]
  float* decay;       // gated linear attention: log alpha [rows][heads * dim]
  float* work;        // chunk tiles of the recurrence (recurrence_work_floats)
  size_t work_floats;
};
hipError_t launch_rotary_rows(const MixRows& r, const ChunkAttn& a, hipStream_t s);
hipError_t launch_chunk_attn_rows(const MixRows& r, const ChunkAttn& a, hipStream_t s);
hipError_t launch_short_conv_rows(const MixRows& r, const ShortConv& c, hipStream_t s);
// The recurrence of all rows, normalised and gated, into the mixer output columns.
hipError_t launch_recurrence_rows(const MixRows& r, const Recurrence& c, hipStream_t s);
size_t recurrence_work_floats(const Recurrence& c, int nseq, int n);
hipError_t launch_gated_mlp_rows(const MixRows& r, const GatedMlp& m, hipStream_t s);
// The rows that the caches keep: the last chunk's keys and values, the convolution's last inputs
// (a or c may be null).
hipError_t launch_commit_rows(const MixRows& r, const ChunkAttn* a, const ShortConv* c, hipStream_t s);

// dst[r] = src[r] / sqrt(mean(src[r]^2) + eps) * gain[0] * scale over `cols` columns; rows are ld
// floats apart and the columns [cols, ld) of dst are set to 0.  rows_at (may be null): row r of
// src is rows_at[r].
hipError_t launch_rms_rows(const float* src, float* dst, int rows, int cols, int ld, const float* gain,
                           float eps, float scale, const int* rows_at, hipStream_t s);
// What a one-token step keeps on the device: the position of the step that is running, that of the
// next one, and, for generations that run ahead of the host, where the next ids are listed
// (out[n_out][nseq], out may be null).
struct StepWords {
  int pos, next, n_out, unused;
  uint32_t* out;
};
// The start of a step: x[b] = table[ids[b]] ([vocab][width], f32 or bf16), the ids are appended to
// words->out, and the position advances.
hipError_t launch_begin_step(float* x, const void* table, int table_bf16, const uint32_t* ids, int nseq, int width,
                             StepWords* words, hipStream_t s);
hipError_t launch_set_words(StepWords* words, int next, uint32_t* out, hipStream_t s);

}  // namespace pgk
