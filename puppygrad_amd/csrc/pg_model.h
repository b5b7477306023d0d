// The handle types behind the C ABI (pg_model, pg_kv_cache, pg_logits) and what the host-side
// translation units that drive kernels share.
#pragma once

#include <hip/hip_runtime.h>

#include <algorithm>
#include <memory>
#include <string>
#include <vector>

#include "pg_internal.h"
#include "pg_kernels.h"

#define PG_HIP(expr)                                                                  \
  do {                                                                                \
    hipError_t e__ = (expr);                                                          \
    if (e__ != hipSuccess)                                                            \
      return pgh::fail(PG_BACKEND, std::string("HIP error: ") + hipGetErrorString(e__) +   \
                                  " at " #expr);                                      \
  } while (0)

namespace pgh {

struct StackModel;  // pg_stack.h
struct StackCache;

// Sizes every architecture has: vocabulary, positions, width, layers (and GPT-2's heads and
// inner width, 0 where they differ from layer to layer).
struct Cfg {
  size_t V, P, C, L, H, I;
  float eps;
  size_t hd() const { return C / H; }
};

inline size_t round_up(size_t n, size_t a) { return (n + a - 1) / a * a; }

__attribute__((visibility("hidden"))) pg_status select_device(int device);

struct DevBuf {
  float* p = nullptr;
  ~DevBuf() {
    if (p) (void)hipFree(p);
  }
  pg_status alloc(size_t n) {
    PG_HIP(hipMalloc(&p, std::max<size_t>(n, 1) * sizeof(float)));
    return PG_OK;
  }
};

// Time stamps between the launches of one step, for the buckets of Gpt2OperationProfile
// (src/models/gpt2/rust.rs:336-347): an event is recorded on the step's stream after each
// operation; the span since the previous event belongs to that operation's bucket.
struct ProfileMarks {
  enum Bucket { kNone, kLayerNorm, kQkv, kAttention, kAttnProj, kMlpFc, kMlpProj, kLogits };
  std::vector<hipEvent_t> events;
  std::vector<Bucket> bucket;
  size_t used = 0;
  hipError_t mark(hipStream_t s, Bucket b) {
    if (used == events.size()) {
      hipEvent_t e = nullptr;
      hipError_t r = hipEventCreate(&e);
      if (r != hipSuccess) return r;
      events.push_back(e);
      bucket.push_back(kNone);
    }
    bucket[used] = b;
    return hipEventRecord(events[used++], s);
  }
  // Adds the spans of the step just synchronised to `p` and rewinds.
  hipError_t collect(pg_gpt2_operation_profile* p) {
    for (size_t i = 1; i < used; ++i) {
      float ms = 0.0f;
      hipError_t r = hipEventElapsedTime(&ms, events[i - 1], events[i]);
      if (r != hipSuccess) return r;
      const double sec = (double)ms * 1e-3;
      switch (bucket[i]) {
        case kLayerNorm: p->layer_norm_s += sec; break;
        case kQkv: p->qkv_projection_s += sec; break;
        case kAttention: p->attention_s += sec; break;
        case kAttnProj: p->attention_projection_s += sec; break;
        case kMlpFc: p->mlp_fc_projection_s += sec; break;
        case kMlpProj: p->mlp_projection_s += sec; break;
        case kLogits: p->final_logits_s += sec; break;
        case kNone: break;
      }
    }
    used = 0;
    return hipSuccess;
  }
  ~ProfileMarks() {
    for (hipEvent_t e : events) (void)hipEventDestroy(e);
  }
};

}  // namespace pgh

struct pg_model {
  pgh::Cfg cfg;
  int device = 0;
  int num_cus = 0;
  pg_hip_options opts{};
  float* arena = nullptr;  // one allocation holding every tensor
  size_t arena_floats = 0;
  float *wte = nullptr, *wpe = nullptr, *ln_f_g = nullptr, *ln_f_b = nullptr;
  std::vector<pgk::LayerW> layers;
  pgk::LayerW* d_layers = nullptr;  // the same table in device memory
  bool persistent = false;          // batch-1 decode runs as one persistent launch
  int persistent_grid = 0;          // workgroups of that launch (one per CU)
  int attn_splits = 1;              // key splits per head in the persistent kernel
  // tunables (pg_hip_options; defaults filled in at creation)
  int item_keys = 128;              // keys per attention item of the persistent kernel
  bool item_keys_auto = true;       // not set by the caller: 256-key items for launches that stay
                                    // within 256 positions (one split per head: no merge hop)
  bool item_keys_256_ok = false;    // the device holds the grid of the 256-key instance
  int attn_blocks_per_cu = 4;       // per-operation / batched decode attention
  int gemm_split_items = 3;         // tile GEMM split-K
  int gemm_b9_min_rows = 1024;      // f32 rows on the bf16 matrix cores from this many input rows
  size_t seq_gemm_min_tokens = 4;   // prompts at least this long take the GEMM prefill
  int w_bf16 = 0;                   // wte and the block matrices are stored as bf16
  // int8 storage (QuantizedRows, src/models/cpu.rs:26-56): the block matrices hold int8 rows
  // with the scales in LayerW; wte stays f32 for the embedding (rust.rs:966-974 reads the f32
  // table) and lm_w / lm_s are its quantised copy for the lm_head (rust.rs:1815-1849).
  // Otherwise lm_w == wte and lm_s == nullptr.
  int w_i8 = 0;
  float* lm_w = nullptr;
  float* lm_s = nullptr;
  float* lm_f = nullptr;  // [2 V]: LN_f folded into the lm_head rows (pgk::launch_ln_fold)
  // Set for stack models (pg_stack.h); the GPT-2 fields above are then unused.
  std::shared_ptr<pgh::StackModel> stack;
};

struct pg_logits {
  pg_kv_cache* owner;
  float* data;  // device [rows][vocab]
  uint32_t rows;
  uint64_t vocab;
};

struct pg_kv_cache {
  pgh::Cfg cfg;
  int device = 0;
  int num_cus = 0;
  uint32_t B = 1;
  size_t seq_len = 0;
  float* kv = nullptr;  // [L][2][B][H][P][hd]
  // per-sequence activation scratch, [B][...]
  float* seq_scratch = nullptr;  // activations of the full-sequence (GEMM) forward, grown on demand
  size_t seq_scratch_floats = 0;
  float* gemm_ws = nullptr;      // split-K partial tiles of the batched decode step
  size_t gemm_ws_floats = 0;
  float *x = nullptr, *q = nullptr, *hbuf = nullptr, *part_acc = nullptr, *part_m = nullptr,
        *part_l = nullptr, *logits_buf = nullptr;
  float *qkv_b = nullptr, *xn_b = nullptr, *att_b = nullptr;  // batched step: [B][3C], [B][C], [B][C]
  bool pack32 = false;  // batched step: xn_b, att_b and hbuf are packed (pgk::packed32_index)
  // device-side candidate selection for sampling, allocated at first use: kept candidates
  // (ids, then values, then [count]) and the recent ids of the repeat penalty, with pinned
  // host mirrors
  uint32_t* d_cand = nullptr;
  uint32_t* h_cand = nullptr;
  uint32_t* d_recent = nullptr;
  uint32_t* h_recent = nullptr;
  uint32_t* d_tok = nullptr;      // [B] token the next step embeds
  uint32_t* d_out_ids = nullptr;  // [P][B] ids produced by greedy decode
  uint32_t* h_ids = nullptr;      // pinned staging, [P][B]
  // pinned staging of the prompts of full-sequence forwards, used in turn: the copy to the
  // device is queued without waiting, and a buffer is reused once the copy of two calls ago
  // has been made
  uint32_t* h_prompt[2] = {nullptr, nullptr};
  hipEvent_t ev_prompt[2] = {nullptr, nullptr};
  unsigned prompt_turn = 0;
  // streamed greedy generation: ids the persistent kernel writes straight into pinned host
  // memory as it selects them ([P + 1], batch 1), and the device's address of that block
  uint32_t* h_stream = nullptr;
  uint32_t* h_stream_dev = nullptr;
  hipStream_t stream = nullptr;
  hipEvent_t ev0 = nullptr, ev1 = nullptr;
  pg_logits logits{};
  bool logits_valid = false;
  // persistent decode: tagged activation words {epoch, f32} and the launch status
  // One uncached block: the tagged argmax words, then the f32 exchange vectors (two buffers each)
  unsigned long long* best_t = nullptr;
  unsigned* xch = nullptr;
  size_t best_words = 0;  // 64-bit words at best_t
  size_t x_words = 0;     // 32-bit words at xch
  // The exchange words are as a launch expects them: the last persistent launch on this cache
  // ran to its end and the model has an even number of layers (the set a launch's first layer
  // uses was then armed again during the last layer before it, and the other set is armed by
  // the first layer before the second uses it, as between two forwards of one launch), so the
  // next launch needs no k_arm_exchange in front of it.
  bool xch_ready = false;
  unsigned xch_set = 0;   // words from one set of exchange vectors to the other
  // [grid][L + 1][16] time stamps of a profiled forward of the persistent kernel (allocated on
  // first use; pg_gpt2_stream_token_ids_profiled)
  unsigned long long* stamps = nullptr;
  size_t tagged_bytes = 0;  // size of that allocation as the exchange pool counts it
  unsigned* status = nullptr;
  unsigned* h_status = nullptr;  // pinned
  uint32_t* d_force = nullptr;   // [P] prompt ids for a one-launch prefill
  unsigned epoch = 1;            // next unused epoch
  // logits_buf holds the logits that select the next token (row b: sequence b)
  bool next_valid = false;
  float* want_buf = nullptr;     // logits of pg_model_extend, grown on demand
  size_t want_cap = 0;
  size_t ids_cap = 0;            // ids that d_out_ids and h_ids hold
  size_t prompt_cap = 0;         // ids that a buffer of h_prompt holds
  std::shared_ptr<pgh::StackCache> stack;  // stack models: state and working memory
  const pg_model* stack_model = nullptr;

  float* k_panel(size_t l, size_t b) const {
    return kv + (((l * 2 + 0) * B + b) * cfg.H) * cfg.P * cfg.hd();
  }
  float* v_panel(size_t l, size_t b) const {
    return kv + (((l * 2 + 1) * B + b) * cfg.H) * cfg.P * cfg.hd();
  }
};
