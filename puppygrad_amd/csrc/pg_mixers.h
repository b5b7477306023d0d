// Launchers of the sequence mixers that a layer of a stack model (pg_stack.h) is made of:
// rotary positions, chunked sigmoid attention, latent attention (windowed, with a sink), short
// convolution, gated delta rule (one decay per head or per key channel), gated linear attention,
// state-space recurrence, gated MLP activation, mixture of experts, RMS norms.  Every constant
// of a mechanism is a field of its argument struct.
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
// columns, then silu; w[channel][taps], the last tap is the current token's; bias[channel] may be
// null.  ring[position % taps][channels] keeps a sequence's last inputs.
struct ShortConv {
  int channels, taps;
  int col;
  const float* w;
  const float* bias;
  float* ring;
  size_t ring_seq;
};

// One linear recurrence per head with state S[dim][vdim].
//  REC_DELTA (gated delta rule): S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q with unit
//    vectors q (times q_scale) and k, beta = sigmoid(b), g = exp(-exp(a_log) softplus(a + dt_bias)).
//    q, k and v are the columns of the short convolution (q | k | v), a and b columns of the
//    projections.
//  REC_CHANNEL_DELTA: the same with one g per key channel: a = a2 . a1, dt_bias[heads * dim].
//  REC_GLA (gated linear attention): S <- diag(alpha) S + k v^T; o = S^T q, alpha =
//    sigmoid(z)^inv_tau, z = a2 . a1 + a2_bias with a1 `rank` columns of the projections.
//  Then y = o / rms(o) * norm * gate * out_scale with gate = silu of the gate columns, or
//  (REC_CHANNEL_DELTA) sigmoid(g2 . g1).
//  REC_SSD (state-space duality): S <- exp(-exp(a_log) dt) S + dt k v^T; y = (S^T q + skip v) *
//    silu(gate columns), dt = softplus(a + dt_bias); v, k and q are the columns of the short
//    convolution (v | k | q).  y is not normalised.
enum RecurrenceKind : int { REC_GLA = 0, REC_DELTA = 1, REC_CHANNEL_DELTA = 2, REC_SSD = 3 };
constexpr bool rec_has_conv(int kind) { return kind != REC_GLA; }
constexpr bool rec_reads_state(int kind) { return kind == REC_DELTA || kind == REC_CHANNEL_DELTA; }

// Second half of a projection through a low rank: rows of w[rows][rank] (f32, or bf16 where
// w_bf16), rank a multiple of 32 (columns past the tensor's rank are zeros), against columns
// [col, col + rank) of a row of projections.
struct LowRank {
  const void* w;
  int w_bf16, rank;
  int col;
};

struct Recurrence {
  int kind;
  int heads, kv_heads, dim, vdim;
  float q_scale;
  float eps;
  int q_col, k_col, v_col;  // of the projections (with a convolution: its inputs)
  int g_col;                // output gate
  int a_col, b_col;         // REC_DELTA: decay and step size; REC_SSD: a; REC_GLA: a_col is a1
  const float *a_log, *dt_bias;
  const float *a2, *a2_bias;  // REC_GLA
  int rank;
  float inv_tau;
  LowRank low_a, low_g;     // REC_CHANNEL_DELTA: decay, output gate
  const float* skip;        // REC_SSD
  const float* norm;
  ShortConv conv;           // all but REC_GLA
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
// The same for a layer whose only mixer is a recurrence of any kind (a.rec).
hipError_t launch_recurrence_decode(const MixDecode& a, hipStream_t s);
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
  float* decay;       // [rows][heads * dim]: log alpha (REC_GLA), a (REC_CHANNEL_DELTA: an input)
  float* gate;        // REC_CHANNEL_DELTA: g2 . g1, [rows][heads * vdim] (an input)
  float* work;        // chunk tiles of the recurrence (recurrence_work_floats)
  size_t work_floats;
};
hipError_t launch_rotary_rows(const MixRows& r, const ChunkAttn& a, hipStream_t s);
hipError_t launch_chunk_attn_rows(const MixRows& r, const ChunkAttn& a, hipStream_t s);
hipError_t launch_short_conv_rows(const MixRows& r, const ShortConv& c, hipStream_t s);
// The recurrence of all rows, normalised (not REC_SSD) and gated, into the mixer output columns.
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
// dst[r] += src[r] / sqrt(mean(src[r]^2) + eps) * gain over `cols` columns (norm of a sublayer's
// output, added to the residual); rows are ld floats apart.  With top > 0 a row of the sublayer's
// output is instead the sum over k < top of weight[r][k] * src[slot[r][k]] (launch_moe_route).
hipError_t launch_add_norm_rows(float* dst, const float* src, int rows, int cols, int ld, const float* gain, float eps,
                                const int* slot, const float* weight, int top, hipStream_t s);
// dst[r] = src[r] / rms * gain, the mean square over each of `groups` equal parts of the `cols`
// columns; columns [cols, ld_dst) of dst are set to 0 (src and dst may be the same rows).
// rows_at (may be null): row r of src is rows_at[r].
hipError_t launch_group_rms_rows(const float* src, int ld_src, float* dst, int ld_dst, int rows, int cols, int groups,
                                 const float* gain, float eps, const int* rows_at, hipStream_t s);

// ---- latent attention (pg_latent.hip) ----
// Keys and values of all heads come from one latent row c[kv_rank] per position and a rotated
// part r[rot_dim] shared by the heads: the score of query head h is (q_h . (W_uk_h c) + q'_h . r) *
// scale, its value W_uv_h c.  Position i sees the `window` positions up to i; the softmax's
// denominator also holds exp(sink[h]).  Only [c | r] is cached: ring[position % window][ld].
// Rotation: the pair (2 i, 2 i + 1) turns by position * freq[i], i < half, and grows by mag; the
// values from 2 * half on pass unchanged.
constexpr int kLatentMaxRank = 1024;
constexpr int kLatentTail = 256;  // floats that the last ring is followed by (read, multiplied by zeros)
struct LatentAttn {
  int heads, dim, rot_dim, vdim;
  int q_rank, q_pad;      // q_pad, kv_pad: multiples of 32
  int kv_rank, kv_pad;
  int ld;                 // floats of a cached row: kv_pad + rot_dim padded to 16
  int window;
  float scale, eps;
  const double* freq;
  int half;
  float mag;
  int q_col, c_col;       // columns of a row of projections: query latent; kv_rank + rot_dim values
  const float *q_norm, *c_norm, *sink;
  const void* up_w;       // [heads * dim | heads * vdim from row v_row][kv_pad], f32 or bf16
  int w_bf16, v_row;
  float* ring;
  size_t ring_seq;
  int out_col;
};
// One token of every sequence.  q: [nseq][heads * (dim + rot_dim)] as projected; qa: [nseq][heads][ld]
// queries brought to the latent space; part: [nseq][heads][splits][kv_pad + 2].
struct LatentDecode {
  int nseq;
  const int* d_pos;
  const float* y;
  int ld_y;
  const float* q;
  float *qa, *part;
  int splits;
  float* out;
  int ld_out;
};
int latent_decode_splits(const LatentAttn& a);
hipError_t launch_latent_decode(const LatentDecode& m, const LatentAttn& a, hipStream_t s);
// Many rows.  hist positions before pos0 are seen (latent_history); row b * (hist + n) + j of lat and
// kv is position pos0 - hist + j of sequence b.
inline int latent_history(const LatentAttn& a, int pos0) { return pos0 < a.window - 1 ? pos0 : a.window - 1; }
struct LatentRows {
  float* cq;    // [rows][q_pad] normed query latents
  float* q;     // [rows][heads * (dim + rot_dim)], rotated in place
  float* lat;   // [nseq * (hist + n)][ld]
  float* kv;    // [nseq * (hist + n)][ld_kv]: unrotated keys, then values from column v_row
  int ld_kv, hist;
};
// Norms and rotates the latents of the step's rows into lat behind the cached ones, and cq.
hipError_t launch_latent_prepare_rows(const MixRows& r, const LatentAttn& a, const LatentRows& l, hipStream_t s);
// Rotates the queries in place, clears the padding columns of the mixer outputs, and keeps the last
// rows of lat in the cache.
hipError_t launch_latent_rotate_rows(const MixRows& r, const LatentAttn& a, const LatentRows& l, hipStream_t s);
hipError_t launch_latent_attn_rows(const MixRows& r, const LatentAttn& a, const LatentRows& l, hipStream_t s);

// ---- mixture of experts (pg_moe.hip) ----
// The `top` largest of softmax(router logits) over all experts are a token's experts and, as they
// are, their weights (equal ones: the lower expert first).  An expert is W_down (silu(gate) * up);
// gate_up[expert][2 ff_pad][width_pad] has the gate rows at 2 j and the up rows at 2 j + 1,
// down[expert][width_pad][ff_pad].
constexpr int kMoeMaxExperts = 1024;
constexpr int kMoeMaxTop = 64;
constexpr int kMoeMaxWidth = 16000;  // of the model and of an expert (rows staged in LDS)
struct Moe {
  int experts, experts_pad, top;  // experts_pad: columns of a row of router logits
  int ff, ff_pad;
  const void *gate_up, *down;
  int w_bf16;
};
// One row.  x, out: [width_pad]; act: [top][ff_pad]; expert, weight: [top], filled by the launch.
// logits: the router's, [experts_pad]; or null and router, [experts_pad][width_pad], and the row to be
// brought up to date: x + add / rms(add) * add_gain (add may be null), written to x_out, which is
// not x.
struct MoeRow {
  const float *x, *logits;
  const void* router;
  const float *add, *add_gain;
  float* x_out;
  int width, width_pad;
  float eps;
  float *act, *out;
  int* expert;
  float* weight;
};
// Whether a router is small enough to be multiplied by every block again.
bool moe_router_fits(const Moe& m, int width_pad);
hipError_t launch_moe_row(const Moe& m, const MoeRow& r, hipStream_t s);
// Several rows: pairs are sorted by expert into slots, each expert's padded to whole tiles of tile_rows.
struct MoeRoute {
  int tile_rows, max_slots;  // max_slots: moe_max_slots
  int* count;      // [experts]
  int* rank;       // [rows * top]: number of the pair within its expert
  int* expert;     // [rows * top]
  float* weight;   // [rows * top]
  int* slot;       // [rows * top]
  int* slot_row;   // [max_slots]: row of a slot, -1 in the padding
  int* tile;       // [max_slots / tile_rows]: expert of a tile, -1 past the end
};
int moe_max_slots(const Moe& m, int rows, int tile_rows);
hipError_t launch_moe_route(const Moe& m, const MoeRoute& r, const float* logits, int rows, hipStream_t s);

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
