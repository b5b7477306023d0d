// Stack models: decoders whose config.json lists their layers one by one, each with the kind and
// the sizes of its sequence mixers.  Two forms of layer:
//  parallel (Tarepel): x <- x + ls1 * mixers(h) + ls2 * mlp(h) with h = RMS norm of x: the sublayers
//    read one norm and are added together, so that a layer is one product with all input
//    projections side by side, the mixers, and the products back to x;
//  post-norm (Movudra): x <- x + norm1(mixer(x)), then x <- x + norm2(ff(x)): a sublayer's output is
//    normed and added by whatever reads x next.
//
// The state of a sequence has a fixed size: one chunk or window of keys and values (or latents) per
// attention, one matrix per recurrent head, the last inputs of the short convolutions.
#pragma once

#include <memory>
#include <string>
#include <vector>

#include "pg_internal.h"
#include "pg_json.h"
#include "pg_mixers.h"
#include "pg_model.h"

namespace pgh {

// Feed-forward of a post-norm layer: max(W_up h + b, 0)^2 -> W_down + b, or a mixture of experts.
struct PostFeedForward {
  enum Kind { kNone, kDense, kMoe } kind = kNone;
  int ff = 0, ff_pad = 0;                        // dense
  float *up_w = nullptr, *up_b = nullptr;        // [ff_pad][width_pad]
  float *down_w = nullptr, *down_b = nullptr;    // [width_pad][ff_pad]
  pgk::Moe moe{};
  float* router_w = nullptr;                     // [experts_pad][width_pad]
};

struct StackLayer {
  bool has_attn = false, has_rec = false, has_mlp = false;
  // post-norm layers: exactly one of has_rec and has_latent
  bool post_norm = false, has_latent = false;
  pgk::LatentAttn latent{};
  float* uq_w = nullptr;                         // [heads * (dim + rot_dim)][q_pad]
  float* low_a_w = nullptr;                      // REC_CHANNEL_DELTA: as rec.low_a.w, low_g.w
  float* low_g_w = nullptr;
  int norm_groups = 0;                           // REC_SSD: norm of the mixer's output, and its gain
  float* mix_norm = nullptr;
  PostFeedForward ffn;
  float *norm1 = nullptr, *norm2 = nullptr;      // gains [width_pad]
  // Cache pointers in these are null; the cache fills them in (StackCache::bind).
  pgk::ChunkAttn attn{};
  pgk::Recurrence rec{};
  pgk::GatedMlp mlp{};
  int n_in = 0;                    // columns of a row of projections (a multiple of 4)
  int mix_cols = 0, mix_pad = 0;   // mixer outputs; mix_pad and ff_pad are multiples of 32
  float *in_w = nullptr;           // [n_in][width_pad]
  float *out_w = nullptr;          // [width_pad][mix_pad]
  float *down_w = nullptr;         // [width_pad][ff_pad]
  float *norm = nullptr, *ls1 = nullptr, *ls2 = nullptr;
};

struct StackModel {
  std::string architecture;
  int width = 0, width_pad = 0;    // width_pad: a multiple of 32; columns past width are zeros
  int vocab = 0;
  float eps = 0.0f, logit_scale = 1.0f;
  std::vector<StackLayer> layers;
  float *embed = nullptr, *head = nullptr, *final_norm = nullptr;
  // largest of each over the layers
  int max_in = 0, max_mix = 0, max_ff = 0, max_keys = 0, max_conv = 0, max_decay = 0, max_part = 0;
  // post-norm layers: final_norm has width_pad gains and logit_scale is 1
  bool post_norm = false;
  int max_q_rank = 0, max_q = 0, max_qa = 0, max_gate = 0;
  std::vector<void*> memory;
  ~StackModel();
};

// State and working memory of a pg_kv_cache of a stack model.
struct StackCache {
  struct Layer {
    float *kring = nullptr, *vring = nullptr, *conv = nullptr, *state = nullptr, *latent = nullptr;
  };
  // Mixture of experts: router logits, activations, outputs by slot, and the route's lists.
  struct MoeBuffers {
    float *logits = nullptr, *act = nullptr, *slot_out = nullptr;
    pgk::MoeRoute route{};
    void bind(float* const (&p)[6]) {
      int** at[6] = {&route.count, &route.rank, &route.expert, &route.slot, &route.slot_row, &route.tile};
      for (int i = 0; i < 6; ++i) *at[i] = reinterpret_cast<int*>(p[i]);
    }
  };
  std::vector<Layer> layers;
  MoeBuffers moe;  // one token of every sequence
  pgk::StepWords* words = nullptr;  // position of the next token, on the device
  bool lists_ids = false;           // ... steps list their ids
  // one token of every sequence
  float *x = nullptr, *h = nullptr, *y = nullptr, *mix = nullptr, *act = nullptr, *part = nullptr;
  // post-norm layers: the residual before and after a sublayer in turn (x, h), a sublayer's output,
  // queries of latent attention (their latents normed, as projected, in the latent space)
  float *sub = nullptr, *cq = nullptr, *q = nullptr, *qa = nullptr;
  // many rows: one block, grown on demand
  float* rows = nullptr;
  size_t rows_floats = 0;
  // Steps of many rows run the recurrence of a layer on the cache's stream and everything that does
  // not depend on it on this one (fork and join are events).
  hipStream_t side = nullptr;
  hipEvent_t forked = nullptr, joined = nullptr;
  int* rows_at = nullptr;     // rows whose logits are wanted
  size_t rows_at_cap = 0;
  hipGraphExec_t graph = nullptr;  // the one-token step
  bool warm = false;               // the step has run once outside a graph
  std::vector<void*> memory;
  ~StackCache();
};

// Whether config.json describes a stack model, and the model of a directory.
bool stack_config_matches(const Json& config);
pg_status stack_create(const std::string& config_path, const Json& config, const pg_tensor_store& store,
                       const pg_hip_options& opts, pg_model** out);
pg_status stack_cache_create(const pg_model* m, pg_kv_cache* c);
// Queues n tokens of every sequence (ids[B][n]) from position pos0.  rows: which of the B * n rows
// have their logits written to dst[n_rows][vocab] (device), in this order.
pg_status stack_rows(const pg_model* m, pg_kv_cache* c, const uint32_t* ids, size_t n, size_t pos0,
                     const std::vector<int>& rows, float* dst, ProfileMarks* marks = nullptr);
// Queues one token of every sequence: ids in c->d_tok, position in StackCache::words (advanced);
// logits to c->logits_buf.
pg_status stack_step(const pg_model* m, pg_kv_cache* c, ProfileMarks* marks = nullptr);
// Sets the position on the device, and where the steps from here on list their ids (device memory,
// [step][B]; null: nowhere).
pg_status stack_set_pos(pg_kv_cache* c, size_t pos, uint32_t* out = nullptr);

}  // namespace pgh
