// Stack models: configuration, weight upload, per-sequence state and the two ways a step runs
// (pg_stack.h).
#include "pg_stack.h"

#include <cmath>
#include <cstring>
#include <map>

namespace pgh {

namespace {

// ---- configuration --------------------------------------------------------------------------
// A value of config.json by its path, for messages: "layers[3].mixer.dim".
struct Node {
  const Json* v;
  std::string path;
  const std::string* file;

  pg_status bad(const std::string& what) const {
    return fail(PG_INVALID_CONFIG, "config " + *file + ": " + path + " " + what);
  }
  pg_status child(const char* key, Node* out) const {
    const std::string p = path.empty() ? key : path + "." + key;
    const Json* c = v->kind == Json::Obj ? v->find(key) : nullptr;
    if (!c) return fail(PG_ASSET, "failed to parse config " + *file + ": missing field `" + p + "`");
    *out = Node{c, p, file};
    return PG_OK;
  }
  pg_status object(const char* key, Node* out) const {
    if (pg_status s = child(key, out)) return s;
    return out->v->kind == Json::Obj ? PG_OK : out->bad("must be an object");
  }
  pg_status size(const char* key, int lo, int hi, int* out) const {
    Node n;
    if (pg_status s = child(key, &n)) return s;
    if (n.v->kind != Json::Num || !n.v->integral || n.v->u < (uint64_t)lo || n.v->u > (uint64_t)hi)
      return n.bad("must be an integer in [" + std::to_string(lo) + ", " + std::to_string(hi) + "]");
    *out = (int)n.v->u;
    return PG_OK;
  }
  pg_status number(const char* key, double* out) const {
    Node n;
    if (pg_status s = child(key, &n)) return s;
    if (n.v->kind != Json::Num || !std::isfinite(n.v->num)) return n.bad("must be a finite number");
    *out = n.v->num;
    return PG_OK;
  }
  pg_status text(const char* key, std::string* out) const {
    Node n;
    if (pg_status s = child(key, &n)) return s;
    if (n.v->kind != Json::Str) return n.bad("must be a string");
    *out = n.v->str;
    return PG_OK;
  }
};

constexpr int kMaxWidth = 16320;  // a row is staged in LDS by the one-token projections
constexpr int kMaxHeads = 1024;
constexpr uint64_t kMaxPositions = 1ull << 30;

int up(int n, int a) { return (n + a - 1) / a * a; }

pg_status heads_of(const Node& n, int* heads, int* kv_heads) {
  if (pg_status s = n.size("heads", 1, kMaxHeads, heads)) return s;
  if (pg_status s = n.size("kv_heads", 1, kMaxHeads, kv_heads)) return s;
  return *heads % *kv_heads == 0 ? PG_OK : n.bad("heads must be a multiple of kv_heads");
}

// What the reader of a layer collects beside StackLayer.
struct LayerPlan {
  StackLayer layer;
  std::string type;
  double rot_base = 0.0;
  // the tensors of the input projection and the output projection, in column order (rows
  // [from, from + rows) of a tensor of `of` rows; of 0: all)
  struct Part {
    std::string name;
    int rows, col, from = 0, of = 0;
  };
  std::vector<Part> in_parts, out_parts;
  int next_in = 0;
  int add_in(const std::string& name, int rows) {
    const int at = next_in;
    in_parts.push_back({name, rows, at});
    next_in = up(at + rows, 4);  // (columns are read four at a time)
    return at;
  }
  int add_in_slice(const std::string& name, int rows, int from, int of) {
    const int at = add_in(name, rows);
    in_parts.back().from = from;
    in_parts.back().of = of;
    return at;
  }
  // a part whose columns are an operand of a further product: zeros up to a multiple of 32
  int add_in_pad32(const std::string& name, int rows) {
    next_in = up(next_in, 32);
    const int at = add_in(name, rows);
    next_in = up(next_in, 32);
    return at;
  }
  std::vector<double> freq;  // latent attention
  int add_out(const std::string& name, int cols) {
    const int at = layer.mix_cols;
    out_parts.push_back({name, cols, at});
    layer.mix_cols += cols;
    return at;
  }
};

pg_status read_attention(const Node& n, const std::string& prefix, double out_scale, LayerPlan* p) {
  pgk::ChunkAttn& a = p->layer.attn;
  int vdim = 0, rot_dims = 0;
  double scale = 0.0;
  Node mask, rot;
  pg_status s;
  if ((s = heads_of(n, &a.heads, &a.kv_heads))) return s;
  if ((s = n.size("dim", 1, pgk::kMixMaxDim, &a.dim))) return s;
  if ((s = n.size("vdim", 1, pgk::kMixMaxDim, &vdim))) return s;
  if (vdim != a.dim) return n.bad("vdim must equal dim: the values are the keys");
  if ((s = n.number("scale", &scale))) return s;
  if ((s = n.object("mask", &mask))) return s;
  if ((s = mask.size("size", 1, 1 << 20, &a.chunk))) return s;
  if ((s = n.object("rot", &rot))) return s;
  if ((s = rot.size("dims", 0, a.dim, &rot_dims))) return s;
  if (rot_dims % 2) return rot.bad("dims must be even");
  if ((s = rot.number("base", &p->rot_base))) return s;
  if (!(p->rot_base > 0.0)) return rot.bad("base must be > 0");
  a.dim_pad = up(a.dim, 4);
  a.scale = (float)scale;
  a.rot.half = rot_dims / 2;
  a.out_scale = (float)out_scale;
  a.q_col = p->add_in(prefix + "q", a.heads * a.dim);
  a.k_col = p->add_in(prefix + "k", a.kv_heads * a.dim);
  a.out_col = p->add_out(prefix + "o", a.heads * a.dim);
  p->layer.has_attn = true;
  return PG_OK;
}

pg_status read_delta(const Node& n, const std::string& prefix, double out_scale, float eps, LayerPlan* p) {
  pgk::Recurrence& r = p->layer.rec;
  pg_status s;
  r.kind = pgk::REC_DELTA;
  if ((s = heads_of(n, &r.heads, &r.kv_heads))) return s;
  if ((s = n.size("dim", 1, pgk::kMixMaxDim, &r.dim))) return s;
  if ((s = n.size("vdim", 1, pgk::kMixMaxDim, &r.vdim))) return s;
  if ((s = n.size("conv", 1, pgk::kMixMaxTaps, &r.conv.taps))) return s;
  r.q_scale = 1.0f / std::sqrt((float)r.dim);
  r.eps = eps;
  r.out_scale = (float)out_scale;
  const int qk = r.kv_heads * r.dim, vv = r.heads * r.vdim;
  // q, k and v lie next to each other: one convolution covers the columns of all three (and
  // the unused ones between them, whose taps are zeros)
  r.q_col = p->add_in(prefix + "q", qk);
  r.k_col = p->add_in(prefix + "k", qk);
  r.v_col = p->add_in(prefix + "v", vv);
  r.conv.col = r.q_col;
  r.conv.channels = up(r.v_col + vv - r.q_col, 4);
  r.g_col = p->add_in(prefix + "g", vv);
  r.b_col = p->add_in(prefix + "b", r.heads);
  r.a_col = p->add_in(prefix + "a", r.heads);
  r.out_col = p->add_out(prefix + "o", vv);
  p->layer.has_rec = true;
  return PG_OK;
}

pg_status read_gla(const Node& n, const std::string& prefix, int rank, float eps, LayerPlan* p) {
  pgk::Recurrence& r = p->layer.rec;
  double tau = 0.0;
  pg_status s;
  r.kind = pgk::REC_GLA;
  if ((s = n.size("heads", 1, kMaxHeads, &r.heads))) return s;
  r.kv_heads = r.heads;
  if ((s = n.size("dim", 1, pgk::kMixMaxDim, &r.dim))) return s;
  if ((s = n.size("vdim", 1, pgk::kMixMaxDim, &r.vdim))) return s;
  if ((s = n.number("tau", &tau))) return s;
  if (!(tau > 0.0)) return n.bad("tau must be > 0");
  r.q_scale = 1.0f / std::sqrt((float)r.dim);
  r.eps = eps;
  r.out_scale = 1.0f;
  r.inv_tau = (float)(1.0 / tau);
  r.rank = rank;
  const int qk = r.heads * r.dim, vv = r.heads * r.vdim;
  r.q_col = p->add_in(prefix + "q", qk);
  r.k_col = p->add_in(prefix + "k", qk);
  r.v_col = p->add_in(prefix + "v", vv);
  r.g_col = p->add_in(prefix + "g", vv);
  r.a_col = p->add_in(prefix + "a1", rank);
  r.out_col = p->add_out(prefix + "o", vv);
  p->layer.has_rec = true;
  return PG_OK;
}

pg_status read_mlp(const Node& n, const std::string& prefix, LayerPlan* p) {
  pgk::GatedMlp& m = p->layer.mlp;
  std::string kind;
  pg_status s;
  if ((s = n.text("kind", &kind))) return s;
  if (kind != "dense") return n.bad("kind `" + kind + "` is not supported");
  if ((s = n.size("ff", 1, kMaxWidth, &m.ff))) return s;
  m.ff_pad = up(m.ff, 32);
  m.gate_col = p->add_in(prefix + "gate", m.ff);
  m.up_col = p->add_in(prefix + "up", m.ff);
  p->layer.has_mlp = true;
  return PG_OK;
}

// ---- post-norm layers (Movudra) ----
// Rows of a two-dimensional tensor whose first size the config does not give.
pg_status rank_of(const pg_tensor_store& store, const std::string& name, int* rank) {
  TensorView t;
  if (pg_status s = find_tensor(store, name, &t)) return s;
  if (t.shape.size() != 2 || t.shape[0] < 1 || t.shape[0] > (uint64_t)kMaxWidth)
    return fail(PG_INVALID_WEIGHTS, "tensor " + name + " must have two dimensions");
  *rank = (int)t.shape[0];
  return PG_OK;
}

pg_status read_mamba2(const Node& n, const std::string& prefix, float eps, LayerPlan* p) {
  pgk::Recurrence& r = p->layer.rec;
  pg_status s;
  r.kind = pgk::REC_SSD;
  if ((s = n.size("heads", 1, kMaxHeads, &r.heads))) return s;
  if ((s = n.size("groups", 1, kMaxHeads, &r.kv_heads))) return s;
  if (r.heads % r.kv_heads) return n.bad("heads must be a multiple of groups");
  if ((s = n.size("state", 1, pgk::kMixMaxDim, &r.dim))) return s;
  if ((s = n.size("vdim", 1, pgk::kMixMaxDim, &r.vdim))) return s;
  if ((s = n.size("conv", 1, pgk::kMixMaxTaps, &r.conv.taps))) return s;
  if ((s = n.size("norm_groups", 1, 1 << 20, &p->layer.norm_groups))) return s;
  const int inner = r.heads * r.vdim, gn = r.kv_heads * r.dim, all = 2 * inner + 2 * gn + r.heads;
  if (inner % p->layer.norm_groups) return n.bad("heads * vdim must be a multiple of norm_groups");
  r.q_scale = 1.0f;
  r.eps = eps;
  r.out_scale = 1.0f;
  // [z | x | B | C | dt]; the state is written with B and x and read with C
  r.g_col = p->add_in_slice(prefix + "in", inner, 0, all);
  r.v_col = p->add_in_slice(prefix + "in", inner, inner, all);
  r.k_col = p->add_in_slice(prefix + "in", gn, 2 * inner, all);
  r.q_col = p->add_in_slice(prefix + "in", gn, 2 * inner + gn, all);
  r.a_col = p->add_in_slice(prefix + "in", r.heads, 2 * inner + 2 * gn, all);
  r.conv.col = r.v_col;
  r.conv.channels = up(r.q_col + gn - r.v_col, 4);
  r.out_col = p->add_out(prefix + "o", inner);
  p->layer.has_rec = true;
  return PG_OK;
}

pg_status read_channel_delta(const Node& n, const std::string& prefix, const pg_tensor_store& store, float eps,
                             LayerPlan* p) {
  pgk::Recurrence& r = p->layer.rec;
  pg_status s;
  int rank_a = 0, rank_g = 0;
  r.kind = pgk::REC_CHANNEL_DELTA;
  if ((s = heads_of(n, &r.heads, &r.kv_heads))) return s;
  if ((s = n.size("dim", 1, pgk::kMixMaxDim, &r.dim))) return s;
  if ((s = n.size("vdim", 1, pgk::kMixMaxDim, &r.vdim))) return s;
  if ((s = n.size("conv", 1, pgk::kMixMaxTaps, &r.conv.taps))) return s;
  if ((s = rank_of(store, prefix + "a1", &rank_a)) || (s = rank_of(store, prefix + "g1", &rank_g))) return s;
  r.q_scale = 1.0f / std::sqrt((float)r.dim);
  r.eps = eps;
  r.out_scale = 1.0f;
  const int qk = r.kv_heads * r.dim, vv = r.heads * r.vdim;
  r.q_col = p->add_in(prefix + "q", qk);
  r.k_col = p->add_in(prefix + "k", qk);
  r.v_col = p->add_in(prefix + "v", vv);
  r.conv.col = r.q_col;
  r.conv.channels = up(r.v_col + vv - r.q_col, 4);
  r.b_col = p->add_in(prefix + "b", r.heads);
  r.low_a.rank = up(rank_a, 32);
  r.low_a.col = p->add_in_pad32(prefix + "a1", rank_a);
  r.low_g.rank = up(rank_g, 32);
  r.low_g.col = p->add_in_pad32(prefix + "g1", rank_g);
  r.rank = rank_a;
  r.out_col = p->add_out(prefix + "o", vv);
  p->layer.has_rec = true;
  return PG_OK;
}

// Angles per position of the rotated pairs, with YaRN's stretch where `scaling` is given.
pg_status read_rotation(const Node& rot, int max_dims, std::vector<double>* freq, int* half, float* mag) {
  pg_status s;
  int dims = 0;
  double base = 0.0;
  if ((s = rot.size("dims", 0, max_dims, &dims))) return s;
  if (dims % 2) return rot.bad("dims must be even");
  if ((s = rot.number("base", &base))) return s;
  if (!(base > 0.0)) return rot.bad("base must be > 0");
  *half = dims / 2;
  *mag = 1.0f;
  freq->assign(std::max(1, *half), 0.0);
  for (int i = 0; i < *half; ++i) (*freq)[i] = std::pow(base, -2.0 * i / dims);
  const Json* scaling = rot.v->find("scaling");
  if (!scaling || scaling->kind == Json::Null) return PG_OK;
  Node y;
  double factor = 0.0, original = 0.0, fast = 0.0, slow = 0.0;
  if ((s = rot.object("scaling", &y))) return s;
  if ((s = y.number("factor", &factor)) || (s = y.number("original", &original)) || (s = y.number("fast", &fast)) ||
      (s = y.number("slow", &slow)))
    return s;
  if (!(factor > 0.0 && original > 0.0 && fast > 0.0 && slow > 0.0)) return y.bad("must hold numbers > 0");
  if (base == 1.0) return rot.bad("base must not be 1 with scaling");
  // the pair (a real number) that turns t times over `original` positions
  auto pair_of = [&](double t) { return dims * std::log(original / (2.0 * M_PI * t)) / (2.0 * std::log(base)); };
  const double lo = std::max(std::floor(pair_of(fast)), 0.0), hi = std::min(std::ceil(pair_of(slow)), dims - 1.0);
  for (int i = 0; i < *half; ++i) {
    const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
    (*freq)[i] = (*freq)[i] / factor * ramp + (*freq)[i] * (1.0 - ramp);
  }
  *mag = (float)(0.1 * std::log(factor) + 1.0);
  return PG_OK;
}

pg_status read_latent(const Node& n, const std::string& prefix, float eps, LayerPlan* p) {
  pgk::LatentAttn& a = p->layer.latent;
  double scale = 0.0;
  Node mask, rot;
  pg_status s;
  if ((s = n.size("heads", 1, kMaxHeads, &a.heads))) return s;
  if ((s = n.size("dim", 1, pgk::kMixMaxDim, &a.dim))) return s;
  if ((s = n.size("rot_dim", 0, pgk::kMixMaxDim, &a.rot_dim))) return s;
  if (a.dim + a.rot_dim > pgk::kMixMaxDim) return n.bad("dim + rot_dim may be up to " + std::to_string(pgk::kMixMaxDim));
  if ((s = n.size("vdim", 1, pgk::kMixMaxDim, &a.vdim))) return s;
  if ((s = n.size("q_rank", 1, kMaxWidth, &a.q_rank))) return s;
  if ((s = n.size("kv_rank", 1, pgk::kLatentMaxRank, &a.kv_rank))) return s;
  if ((s = n.number("scale", &scale))) return s;
  if ((s = n.object("mask", &mask))) return s;
  if ((s = mask.size("size", 1, 1 << 20, &a.window))) return s;
  if ((s = n.object("rot", &rot))) return s;
  if ((s = read_rotation(rot, a.rot_dim, &p->freq, &a.half, &a.mag))) return s;
  a.scale = (float)scale;
  a.eps = eps;
  a.q_pad = up(a.q_rank, 32);
  a.kv_pad = up(a.kv_rank, 32);
  a.ld = a.kv_pad + up(a.rot_dim, 16);
  a.v_row = up(a.heads * a.dim, 4);
  a.q_col = p->add_in_pad32(prefix + "dq", a.q_rank);
  a.c_col = p->add_in(prefix + "dkv", a.kv_rank + a.rot_dim);
  a.out_col = p->add_out(prefix + "o", a.heads * a.vdim);
  p->layer.has_latent = true;
  return PG_OK;
}

pg_status read_post_ff(const Node& n, LayerPlan* p) {
  PostFeedForward& f = p->layer.ffn;
  std::string kind;
  pg_status s;
  if ((s = n.text("kind", &kind))) return s;
  if (kind == "dense") {
    f.kind = PostFeedForward::kDense;
    if ((s = n.size("ff", 1, kMaxWidth, &f.ff))) return s;
    f.ff_pad = up(f.ff, 32);
    return f.ff_pad <= kMaxWidth ? PG_OK : n.bad("ff is too large");
  }
  if (kind != "moe") return n.bad("kind `" + kind + "` is not supported");
  Node expert, router;
  f.kind = PostFeedForward::kMoe;
  if ((s = n.object("expert", &expert)) || (s = n.object("router", &router))) return s;
  if ((s = expert.size("ff", 1, pgk::kMoeMaxWidth, &f.moe.ff))) return s;
  if ((s = router.size("experts", 1, pgk::kMoeMaxExperts, &f.moe.experts))) return s;
  if ((s = router.size("top", 1, std::min(f.moe.experts, pgk::kMoeMaxTop), &f.moe.top))) return s;
  f.moe.ff_pad = up(f.moe.ff, 32);
  f.moe.experts_pad = up(f.moe.experts, 4);
  return PG_OK;
}

// ---- weights -----------------------------------------------------------------------------------
struct Loader {
  const pg_tensor_store& store;
  StackModel& model;
  bool bf16;                         // how matrices are kept
  std::vector<unsigned char> host;   // staging
  size_t elem() const { return bf16 ? 2 : 4; }

  pg_status get(const std::string& name, const std::vector<uint64_t>& shape, TensorView* t) {
    if (pg_status s = find_tensor(store, name, t)) return s;
    auto text = [](const std::vector<uint64_t>& v) {
      std::string r = "[";
      for (size_t i = 0; i < v.size(); ++i) r += (i ? ", " : "") + std::to_string(v[i]);
      return r + "]";
    };
    if (t->dtype == TensorView::I32) return fail(PG_ASSET, "tensor " + name + " has dtype I32, expected F32 or BF16");
    if (t->shape != shape)
      return fail(PG_INVALID_WEIGHTS, "tensor " + name + " shape " + text(t->shape) + " does not match expected " + text(shape));
    return PG_OK;
  }
  static float value(const TensorView& t, size_t i) {
    if (t.dtype == TensorView::F32) {
      float f;
      std::memcpy(&f, t.data + 4 * i, 4);
      return f;
    }
    uint16_t h;
    std::memcpy(&h, t.data + 2 * i, 2);
    const uint32_t u = (uint32_t)h << 16;
    float f;
    std::memcpy(&f, &u, 4);
    return f;
  }
  static uint16_t to_bf16(float f) {  // nearest, ties to even
    uint32_t u;
    std::memcpy(&u, &f, 4);
    if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x40u);
    return (uint16_t)((u + 0x7fffu + ((u >> 16) & 1u)) >> 16);
  }
  pg_status upload(const void* src, size_t bytes, float** out) {
    void* p = nullptr;
    PG_HIP(hipMalloc(&p, std::max<size_t>(bytes, 16)));
    model.memory.push_back(p);
    PG_HIP(hipMemcpy(p, src, bytes, hipMemcpyHostToDevice));
    *out = static_cast<float*>(p);
    return PG_OK;
  }
  // A matrix of `rows` x `cols` (both padded) in the storage type, zero to begin with.
  void begin(size_t rows, size_t cols) { host.assign(rows * cols * elem(), 0); }
  // Rows [from, from + n) of the tensor name [r][c] at (row, col) of the staged matrix of `cols`
  // columns, `step` rows of it apart (n 0: all rows).
  pg_status place(const std::string& name, int r, int c, size_t row, size_t col, size_t cols, int from = 0, int n = 0,
                  int step = 1) {
    TensorView t;
    if (pg_status s = get(name, {(uint64_t)r, (uint64_t)c}, &t)) return s;
    if (n == 0) n = r;
    for (int i = 0; i < n; ++i) {
      unsigned char* dst = host.data() + ((row + (size_t)i * step) * cols + col) * elem();
      const size_t at = (size_t)(from + i) * c;
      if (bf16 && t.dtype == TensorView::BF16) {
        std::memcpy(dst, t.data + 2 * at, (size_t)c * 2);
      } else if (!bf16 && t.dtype == TensorView::F32) {
        std::memcpy(dst, t.data + 4 * at, (size_t)c * 4);
      } else {
        for (int j = 0; j < c; ++j) {
          const float f = value(t, at + j);
          if (bf16) {
            const uint16_t h = to_bf16(f);
            std::memcpy(dst + 2 * j, &h, 2);
          } else {
            std::memcpy(dst + 4 * j, &f, 4);
          }
        }
      }
    }
    return PG_OK;
  }
  pg_status end(float** out) { return upload(host.data(), host.size(), out); }
  // A small tensor as f32.
  pg_status read(const std::string& name, const std::vector<uint64_t>& shape, std::vector<float>* out) {
    TensorView t;
    if (pg_status s = get(name, shape, &t)) return s;
    out->resize(t.count);
    for (size_t i = 0; i < t.count; ++i) (*out)[i] = value(t, i);
    return PG_OK;
  }
  pg_status vector(const std::string& name, const std::vector<uint64_t>& shape, size_t padded, float** out) {
    std::vector<float> v;
    if (pg_status s = read(name, shape, &v)) return s;
    v.resize(std::max(padded, v.size()), 0.0f);
    return upload(v.data(), v.size() * sizeof(float), out);
  }
};

// What a post-norm layer has beside its input and output projection.
pg_status load_post_norm(Loader& ld, const std::string& name, LayerPlan& p) {
  StackModel& m = ld.model;
  StackLayer& l = p.layer;
  const int C = m.width, Cp = m.width_pad;
  const uint64_t uC = (uint64_t)C;
  const std::string q = name + ".mix.", f = name + ".mlp.";
  float* v = nullptr;
  pg_status s;
  if (l.has_latent) {
    pgk::LatentAttn& a = l.latent;
    if ((s = ld.vector(q + "dq.norm", {(uint64_t)a.q_rank}, a.q_pad, &v))) return s;
    a.q_norm = v;
    if ((s = ld.vector(q + "dkv.norm", {(uint64_t)a.kv_rank}, a.kv_pad, &v))) return s;
    a.c_norm = v;
    if ((s = ld.vector(q + "sink", {(uint64_t)a.heads}, 0, &v))) return s;
    a.sink = v;
    const int nq = a.heads * (a.dim + a.rot_dim), nk = a.heads * a.dim, nv = a.heads * a.vdim;
    ld.begin(nq, a.q_pad);
    if ((s = ld.place(q + "uq", nq, a.q_rank, 0, 0, a.q_pad)) || (s = ld.end(&l.uq_w))) return s;
    ld.begin(up(a.v_row + nv, 4), a.kv_pad);
    if ((s = ld.place(q + "uk", nk, a.kv_rank, 0, 0, a.kv_pad)) ||
        (s = ld.place(q + "uv", nv, a.kv_rank, a.v_row, 0, a.kv_pad)) || (s = ld.end(&v)))
      return s;
    a.up_w = v;
    a.w_bf16 = ld.bf16;
    if ((s = ld.upload(p.freq.data(), p.freq.size() * sizeof(double), &v))) return s;
    a.freq = reinterpret_cast<const double*>(v);
  } else {
    pgk::Recurrence& r = l.rec;
    const uint64_t H = (uint64_t)r.heads;
    const bool ssd = r.kind == pgk::REC_SSD;
    if ((s = ld.vector(q + "A_log", {H}, 0, &v))) return s;
    r.a_log = v;
    if ((s = ld.vector(q + "dt_bias", {ssd ? H : H * r.dim}, 0, &v))) return s;
    r.dt_bias = v;
    // taps (and biases) by column: the columns between the parts keep zeros
    const int taps = r.conv.taps, n_v = r.heads * r.vdim, n_k = r.kv_heads * r.dim;
    std::vector<float> w((size_t)r.conv.channels * taps, 0.0f), b(r.conv.channels, 0.0f), one, bias;
    if (ssd) {
      const uint64_t ch = (uint64_t)n_v + 2 * (uint64_t)n_k;
      if ((s = ld.read(q + "conv", {ch, (uint64_t)taps}, &one)) || (s = ld.read(q + "conv.b", {ch}, &bias))) return s;
      const struct { int col, n, from; } parts[3] = {{r.v_col, n_v, 0}, {r.k_col, n_k, n_v}, {r.q_col, n_k, n_v + n_k}};
      for (const auto& x : parts) {
        std::copy_n(one.begin() + (size_t)x.from * taps, (size_t)x.n * taps, w.begin() + (size_t)(x.col - r.conv.col) * taps);
        std::copy_n(bias.begin() + x.from, x.n, b.begin() + (x.col - r.conv.col));
      }
      if ((s = ld.upload(b.data(), b.size() * sizeof(float), &v))) return s;
      r.conv.bias = v;
      if ((s = ld.vector(q + "D", {H}, 0, &v))) return s;
      r.skip = v;
      if ((s = ld.vector(q + "norm", {(uint64_t)n_v}, l.mix_pad, &l.mix_norm))) return s;
    } else {
      const struct { const char* key; int col, n; } parts[3] = {{"q", r.q_col, n_k}, {"k", r.k_col, n_k}, {"v", r.v_col, n_v}};
      for (const auto& x : parts) {
        if ((s = ld.read(q + x.key + ".conv", {(uint64_t)x.n, (uint64_t)taps}, &one))) return s;
        std::copy(one.begin(), one.end(), w.begin() + (size_t)(x.col - r.conv.col) * taps);
      }
      if ((s = ld.vector(q + "norm", {(uint64_t)r.vdim}, 0, &v))) return s;
      r.norm = v;
      const struct { const char *in, *out; pgk::LowRank* low; int n; float** w; } low[2] = {
          {"a1", "a2", &r.low_a, r.heads * r.dim, &l.low_a_w}, {"g1", "g2", &r.low_g, n_v, &l.low_g_w}};
      for (const auto& x : low) {
        int rank = 0;
        if ((s = rank_of(ld.store, q + x.in, &rank))) return s;
        ld.begin(x.n, x.low->rank);
        if ((s = ld.place(q + x.out, x.n, rank, 0, 0, x.low->rank)) || (s = ld.end(x.w))) return s;
        x.low->w = *x.w;
        x.low->w_bf16 = ld.bf16;
      }
    }
    if ((s = ld.upload(w.data(), w.size() * sizeof(float), &v))) return s;
    r.conv.w = v;
  }
  PostFeedForward& ff = l.ffn;
  if (ff.kind == PostFeedForward::kNone) return PG_OK;
  if ((s = ld.vector(name + ".norm2", {uC}, Cp, &l.norm2))) return s;
  if (ff.kind == PostFeedForward::kDense) {
    ld.begin(ff.ff_pad, Cp);
    if ((s = ld.place(f + "up", ff.ff, C, 0, 0, Cp)) || (s = ld.end(&ff.up_w))) return s;
    if ((s = ld.vector(f + "up.b", {(uint64_t)ff.ff}, ff.ff_pad, &ff.up_b))) return s;
    ld.begin(Cp, ff.ff_pad);
    if ((s = ld.place(f + "down", C, ff.ff, 0, 0, ff.ff_pad)) || (s = ld.end(&ff.down_w))) return s;
    return ld.vector(f + "down.b", {uC}, Cp, &ff.down_b);
  }
  pgk::Moe& e = ff.moe;
  e.w_bf16 = ld.bf16;
  ld.begin(e.experts_pad, Cp);
  if ((s = ld.place(f + "router", e.experts, C, 0, 0, Cp)) || (s = ld.end(&ff.router_w))) return s;
  ld.begin((size_t)e.experts * 2 * e.ff_pad, Cp);
  for (int i = 0; i < e.experts; ++i) {
    const std::string x = f + "e" + std::to_string(i) + ".";
    const size_t row = (size_t)i * 2 * e.ff_pad;
    if ((s = ld.place(x + "gate", e.ff, C, row, 0, Cp, 0, 0, 2)) || (s = ld.place(x + "up", e.ff, C, row + 1, 0, Cp, 0, 0, 2)))
      return s;
  }
  if ((s = ld.end(&v))) return s;
  e.gate_up = v;
  ld.begin((size_t)e.experts * Cp, e.ff_pad);
  for (int i = 0; i < e.experts; ++i)
    if ((s = ld.place(f + "e" + std::to_string(i) + ".down", C, e.ff, (size_t)i * Cp, 0, e.ff_pad))) return s;
  if ((s = ld.end(&v))) return s;
  e.down = v;
  return PG_OK;
}

pg_status load_layer(Loader& ld, const std::string& name, LayerPlan& p) {
  StackModel& m = ld.model;
  StackLayer& l = p.layer;
  const int C = m.width, Cp = m.width_pad;
  const uint64_t uC = (uint64_t)C;
  pg_status s;
  if (l.post_norm) {
    if ((s = ld.vector(name + ".norm1", {uC}, Cp, &l.norm1))) return s;
  } else {
    if ((s = ld.vector(name + ".norm1", {}, 1, &l.norm))) return s;
    if ((s = ld.vector(name + ".ls1", {uC}, Cp, &l.ls1))) return s;
  }
  ld.begin(l.n_in, Cp);
  for (const auto& part : p.in_parts)
    if ((s = ld.place(part.name, part.of ? part.of : part.rows, C, part.col, 0, Cp, part.from, part.rows))) return s;
  if ((s = ld.end(&l.in_w))) return s;
  ld.begin(Cp, l.mix_pad);
  for (const auto& part : p.out_parts)
    if ((s = ld.place(part.name, C, part.rows, 0, part.col, l.mix_pad))) return s;
  if ((s = ld.end(&l.out_w))) return s;
  if (l.post_norm) return load_post_norm(ld, name, p);
  if (l.has_mlp) {
    if ((s = ld.vector(name + ".ls2", {uC}, Cp, &l.ls2))) return s;
    ld.begin(Cp, l.mlp.ff_pad);
    if ((s = ld.place(name + ".mlp.down", C, l.mlp.ff, 0, 0, l.mlp.ff_pad))) return s;
    if ((s = ld.end(&l.down_w))) return s;
  }
  if (l.has_attn) {
    float* bias = nullptr;
    if ((s = ld.vector(name + ".mix.left.pb", {(uint64_t)l.attn.heads}, 0, &bias))) return s;
    l.attn.bias = bias;
    std::vector<double> freq(std::max(1, l.attn.rot.half));
    for (int i = 0; i < l.attn.rot.half; ++i) freq[i] = std::pow(p.rot_base, -(double)i / l.attn.rot.half);
    float* f = nullptr;
    if ((s = ld.upload(freq.data(), freq.size() * sizeof(double), &f))) return s;
    l.attn.rot.freq = reinterpret_cast<const double*>(f);
  }
  if (l.has_rec) {
    pgk::Recurrence& r = l.rec;
    const std::string q = name + (r.kind == pgk::REC_DELTA ? ".mix.right." : ".mix.");
    float* v = nullptr;
    if ((s = ld.vector(q + "norm", {(uint64_t)r.vdim}, 0, &v))) return s;
    r.norm = v;
    if (r.kind == pgk::REC_DELTA) {
      if ((s = ld.vector(q + "A_log", {(uint64_t)r.heads}, 0, &v))) return s;
      r.a_log = v;
      if ((s = ld.vector(q + "dt_bias", {(uint64_t)r.heads}, 0, &v))) return s;
      r.dt_bias = v;
      const int taps = r.conv.taps;
      std::vector<float> w((size_t)r.conv.channels * taps, 0.0f), one;
      const struct { const char* key; int col, n; } parts[3] = {{"q", r.q_col, r.kv_heads * r.dim},
                                                               {"k", r.k_col, r.kv_heads * r.dim},
                                                               {"v", r.v_col, r.heads * r.vdim}};
      for (const auto& part : parts) {
        if ((s = ld.read(q + part.key + ".conv", {(uint64_t)part.n, (uint64_t)taps}, &one))) return s;
        std::copy(one.begin(), one.end(), w.begin() + (size_t)(part.col - r.conv.col) * taps);
      }
      if ((s = ld.upload(w.data(), w.size() * sizeof(float), &v))) return s;
      r.conv.w = v;
    } else {
      const uint64_t n = (uint64_t)r.heads * r.dim;
      if ((s = ld.vector(q + "a2", {n, (uint64_t)r.rank}, 0, &v))) return s;
      r.a2 = v;
      if ((s = ld.vector(q + "a2.b", {n}, 0, &v))) return s;
      r.a2_bias = v;
    }
  }
  return PG_OK;
}

}  // namespace

StackModel::~StackModel() {
  for (void* p : memory) (void)hipFree(p);
}
StackCache::~StackCache() {
  if (graph) (void)hipGraphExecDestroy(graph);
  if (side) {
    (void)hipStreamSynchronize(side);
    (void)hipStreamDestroy(side);
  }
  if (forked) (void)hipEventDestroy(forked);
  if (joined) (void)hipEventDestroy(joined);
  if (rows) (void)hipFree(rows);
  if (rows_at) (void)hipFree(rows_at);
  for (void* p : memory) (void)hipFree(p);
}

namespace {

pg_status read_tarepel_layer(const Node& n, const std::string& name, const pg_tensor_store& store, float eps,
                             LayerPlan* p) {
  Node mixer, mlp;
  pg_status s;
  if ((s = n.object("mixer", &mixer))) return s;
  if (p->type == "parallel") {
    Node left, right;
    double ls = 0.0, rs = 0.0;
    if ((s = mixer.number("left_scale", &ls))) return s;
    if ((s = mixer.number("right_scale", &rs))) return s;
    if ((s = mixer.object("left", &left))) return s;
    if ((s = mixer.object("right", &right))) return s;
    if ((s = read_attention(left, name + ".mix.left.", ls, p))) return s;
    if ((s = read_delta(right, name + ".mix.right.", rs, eps, p))) return s;
  } else if (p->type == "gla") {
    int rank = 0;  // the rank of the decay projection is the tensor's
    if ((s = rank_of(store, name + ".mix.a1", &rank))) return s;
    if ((s = read_gla(mixer, name + ".mix.", rank, eps, p))) return s;
  } else {
    return n.bad("type `" + p->type + "` is not supported");
  }
  const Json* has = n.v->find("mlp");
  if (has && has->kind != Json::Null) {
    if ((s = n.object("mlp", &mlp))) return s;
    if ((s = read_mlp(mlp, name + ".mlp.", p))) return s;
  }
  return PG_OK;
}

pg_status read_movudra_layer(const Node& n, const std::string& name, const pg_tensor_store& store, float eps,
                             LayerPlan* p) {
  Node mixer, mlp;
  pg_status s;
  p->layer.post_norm = true;
  if ((s = n.object("mixer", &mixer))) return s;
  if (p->type == "mamba2") s = read_mamba2(mixer, name + ".mix.", eps, p);
  else if (p->type == "channel_delta") s = read_channel_delta(mixer, name + ".mix.", store, eps, p);
  else if (p->type == "latent_attention") s = read_latent(mixer, name + ".mix.", eps, p);
  else s = n.bad("type `" + p->type + "` is not supported");
  if (s) return s;
  const Json* has = n.v->find("mlp");
  if (has && has->kind != Json::Null) {
    if ((s = n.object("mlp", &mlp))) return s;
    if ((s = read_post_ff(mlp, p))) return s;
  }
  return PG_OK;
}

struct Architecture {
  const char* name;
  bool post_norm;  // vector norms, no logit scale
  pg_status (*read_layer)(const Node&, const std::string&, const pg_tensor_store&, float, LayerPlan*);
};
const Architecture kArchitectures[] = {{"Tarepel", false, read_tarepel_layer}, {"Movudra", true, read_movudra_layer}};

const Architecture* architecture_named(const Json& config) {
  const Json* a = config.find("architecture");
  if (a && a->kind == Json::Str)
    for (const Architecture& x : kArchitectures)
      if (a->str == x.name) return &x;
  return nullptr;
}

}  // namespace

bool stack_config_matches(const Json& config) { return architecture_named(config) != nullptr; }

pg_status stack_create(const std::string& config_path, const Json& config, const pg_tensor_store& store,
                       const pg_hip_options& opts, pg_model** out) {
  *out = nullptr;
  pg_status s;
  const Node root{&config, "", &config_path};
  auto m = std::make_shared<StackModel>();
  double eps = 0.0, logit_scale = 1.0;
  Node norm, layers;
  const Architecture* arch = architecture_named(config);
  if (!arch) return root.bad("architecture is not supported");
  m->post_norm = arch->post_norm;
  if ((s = root.text("architecture", &m->architecture))) return s;
  if ((s = root.size("vocab", 1, 1 << 30, &m->vocab))) return s;
  if ((s = root.size("width", 1, kMaxWidth, &m->width))) return s;
  if (!arch->post_norm && (s = root.number("logit_scale", &logit_scale))) return s;
  if (logit_scale == 0.0) return root.bad("logit_scale must not be 0");
  if ((s = root.object("norm", &norm))) return s;
  if ((s = norm.number("eps", &eps))) return s;
  if (!(eps >= 0.0)) return norm.bad("eps must be >= 0");
  if ((s = root.child("layers", &layers))) return s;
  if (layers.v->kind != Json::Arr || layers.v->arr.empty() || layers.v->arr.size() > 4096)
    return layers.bad("must be a list of 1 to 4096 layers");
  m->width_pad = up(m->width, 32);
  m->eps = (float)eps;
  m->logit_scale = (float)logit_scale;
  if (m->width_pad > kMaxWidth) return root.bad("width is too large");

  std::vector<LayerPlan> plans(layers.v->arr.size());
  for (size_t i = 0; i < plans.size(); ++i) {
    LayerPlan& p = plans[i];
    const Node n{&layers.v->arr[i], "layers[" + std::to_string(i) + "]", &config_path};
    const std::string name = "l" + std::to_string(i);
    if ((s = n.text("type", &p.type))) return s;
    if ((s = arch->read_layer(n, name, store, m->eps, &p))) return s;
    StackLayer& l = p.layer;
    l.n_in = up(p.next_in, 32);
    l.mix_pad = up(l.mix_cols, 32);
    if (l.mix_pad > kMaxWidth || (l.has_mlp && l.mlp.ff_pad > kMaxWidth))
      return n.bad("is too wide: heads * vdim of the mixers and ff may be up to " + std::to_string(kMaxWidth));
    if (l.ffn.kind == PostFeedForward::kMoe && m->width_pad > pgk::kMoeMaxWidth)
      return n.bad("needs a width of at most " + std::to_string(pgk::kMoeMaxWidth));
    m->max_in = std::max(m->max_in, l.n_in);
    m->max_mix = std::max(m->max_mix, l.mix_pad);
    m->max_ff = std::max(m->max_ff, l.has_mlp ? l.mlp.ff_pad : 0);
    if (l.has_attn) {
      m->max_keys = std::max(m->max_keys, up(l.attn.kv_heads * l.attn.dim, 4));
      m->max_part = std::max(m->max_part, pgk::mix_decode_splits(l.attn, l.has_rec ? &l.rec : nullptr) * l.attn.heads * l.attn.dim);
    }
    if (l.has_rec) {
      if (pgk::rec_has_conv(l.rec.kind)) m->max_conv = std::max(m->max_conv, l.rec.conv.channels);
      if (l.rec.kind == pgk::REC_GLA || l.rec.kind == pgk::REC_CHANNEL_DELTA)
        m->max_decay = std::max(m->max_decay, up(l.rec.heads * l.rec.dim, 4));
      if (l.rec.kind == pgk::REC_CHANNEL_DELTA) m->max_gate = std::max(m->max_gate, up(l.rec.heads * l.rec.vdim, 4));
    }
    if (l.has_latent) {
      const pgk::LatentAttn& a = l.latent;
      m->max_q_rank = std::max(m->max_q_rank, a.q_pad);
      m->max_q = std::max(m->max_q, up(a.heads * (a.dim + a.rot_dim), 4));
      m->max_qa = std::max(m->max_qa, a.heads * a.ld);
      m->max_part = std::max(m->max_part, a.heads * pgk::latent_decode_splits(a) * (a.kv_pad + 2));
    }
    if (l.ffn.kind == PostFeedForward::kDense) m->max_ff = std::max(m->max_ff, l.ffn.ff_pad);
  }

  if (opts.weight_storage != PG_STORE_F32 && opts.weight_storage != PG_STORE_BF16)
    return fail(PG_INVALID_CONFIG, "hip backend weight_storage of a " + m->architecture + " model must be f32 or bf16");
  if (opts.decode_path > PG_DECODE_KERNELS)
    return fail(PG_INVALID_CONFIG, "hip backend decode_path of a " + m->architecture + " model must be auto or kernels");
  if (opts.reserved != 0) return fail(PG_INVALID_CONFIG, "hip backend options: reserved must be 0");
  if ((s = select_device(opts.device))) return s;

  auto model = std::make_unique<pg_model>();
  model->device = opts.device;
  model->opts = opts;
  model->w_bf16 = opts.weight_storage == PG_STORE_BF16 ? 1 : 0;
  model->gemm_split_items = opts.gemm_split_items_per_cu ? (int)opts.gemm_split_items_per_cu : 3;
  model->gemm_b9_min_rows = opts.gemm_b9_min_rows == 0 ? 1024
                            : opts.gemm_b9_min_rows > 0x7fffffffu ? 0x7fffffff
                                                                  : (int)opts.gemm_b9_min_rows;
  hipDeviceProp_t prop;
  PG_HIP(hipGetDeviceProperties(&prop, opts.device));
  model->num_cus = prop.multiProcessorCount;
  model->cfg = Cfg{(size_t)m->vocab, kMaxPositions, (size_t)m->width, plans.size(), 0, 0, m->eps};

  Loader ld{store, *m, model->w_bf16 != 0, {}};
  const int C = m->width, Cp = m->width_pad;
  ld.begin(m->vocab, Cp);
  if ((s = ld.place("embed", m->vocab, C, 0, 0, Cp))) return s;
  if ((s = ld.end(&m->embed))) return s;
  for (size_t i = 0; i < plans.size(); ++i) {
    if ((s = load_layer(ld, "l" + std::to_string(i), plans[i]))) return s;
    m->layers.push_back(plans[i].layer);
  }
  if (m->post_norm) s = ld.vector("final.norm", {(uint64_t)C}, Cp, &m->final_norm);
  else s = ld.vector("final.norm", {}, 1, &m->final_norm);
  if (s) return s;
  ld.begin(m->vocab, Cp);
  if ((s = ld.place("head", m->vocab, C, 0, 0, Cp))) return s;
  if ((s = ld.end(&m->head))) return s;
  model->stack = m;
  *out = model.release();
  return PG_OK;
}

namespace {

#define PG_MARK(b) \
  do {             \
    if (marks) PG_HIP(marks->mark(s, ProfileMarks::b)); \
  } while (0)

// Slots to a tile of the sorted pairs: few rows stream the experts' weights, many fill tiles.
int moe_tile_rows(const pgk::Moe& m, int rows) {
  const long pairs = (long)rows * m.top;
  if (pairs <= 32L * m.experts) return 32;
  return m.w_bf16 && pairs >= 512L * m.experts ? 128 : 64;
}

// Working memory of a mixture of experts over `rows` rows, large enough for each layer added.
struct MoeSizes {
  size_t logits = 0, act = 0, slot_out = 0, experts = 0, pairs = 0, slots = 0, tiles = 0;
  void add(const pgk::Moe& m, int rows, int width_pad) {
    logits = std::max(logits, (size_t)rows * m.experts_pad);
    pairs = std::max(pairs, (size_t)rows * m.top);
    act = std::max(act, (size_t)rows * m.top * m.ff_pad);
    if (rows == 1) return;
    const int tile = moe_tile_rows(m, rows);
    const size_t n = (size_t)pgk::moe_max_slots(m, rows, tile);
    experts = std::max(experts, (size_t)m.experts);
    slots = std::max(slots, n);
    tiles = std::max(tiles, n / tile);
    act = std::max(act, n * m.ff_pad);
    slot_out = std::max(slot_out, n * width_pad);
  }
};

// x += norm2 of the experts' output, rows of x whose router logits are in b.logits.  sub: as many rows
// of working memory.
pg_status moe_rows(const pg_model* model, const StackLayer& l, const StackCache::MoeBuffers& b, float* x, float* sub, int rows,
                   hipStream_t s, ProfileMarks* marks) {
  const StackModel& m = *model->stack;
  const pgk::Moe& e = l.ffn.moe;
  const int Cp = m.width_pad;
  if (rows == 1) {
    pgk::MoeRow r{};
    r.x = x; r.logits = b.logits; r.width = m.width; r.width_pad = Cp; r.eps = m.eps;
    r.act = b.act; r.out = sub; r.expert = b.route.expert; r.weight = b.route.weight;
    PG_HIP(pgk::launch_moe_row(e, r, s));
    PG_MARK(kMlpFc);
    PG_HIP(pgk::launch_add_norm_rows(x, sub, rows, m.width, Cp, l.norm2, m.eps, nullptr, nullptr, 0, s));
    return PG_OK;
  }
  pgk::MoeRoute t = b.route;
  t.tile_rows = moe_tile_rows(e, rows);
  t.max_slots = pgk::moe_max_slots(e, rows, t.tile_rows);
  PG_HIP(pgk::launch_moe_route(e, t, b.logits, rows, s));
  pgk::GemmArgs g{};
  g.w_bf16 = e.w_bf16; g.M = t.max_slots;
  g.A = x; g.lda = Cp; g.W = static_cast<const float*>(e.gate_up); g.N = 2 * e.ff_pad; g.K = Cp;
  g.C = b.act; g.ldc = e.ff_pad;
  PG_HIP(pgk::launch_gemm_grouped(g, pgk::GEMM_SILU_PAIR, t.tile_rows, t.tile, t.slot_row, s));
  PG_MARK(kMlpFc);
  g.A = b.act; g.lda = e.ff_pad; g.W = static_cast<const float*>(e.down); g.N = Cp; g.K = e.ff_pad;
  g.C = b.slot_out; g.ldc = Cp;
  PG_HIP(pgk::launch_gemm_grouped(g, pgk::GEMM_BIAS, t.tile_rows, t.tile, nullptr, s));
  PG_HIP(pgk::launch_add_norm_rows(x, b.slot_out, rows, m.width, Cp, l.norm2, m.eps, t.slot, t.weight, e.top, s));
  return PG_OK;
}

}  // namespace

pg_status stack_cache_create(const pg_model* model, pg_kv_cache* c) {
  const StackModel& m = *model->stack;
  auto st = std::make_shared<StackCache>();
  c->stack = st;  // (destroyed with the cache, also when what follows fails)
  c->stack_model = model;
  const size_t B = c->B;
  if (B > 1024) return fail(PG_INVALID_INPUT, "cache batch must be at most 1024 for this architecture");
  auto alloc = [&](size_t floats, float** p) -> pg_status {
    PG_HIP(hipMalloc(p, std::max<size_t>(floats, 4) * sizeof(float)));
    st->memory.push_back(*p);
    // (padding columns of the one-token buffers are read and never written)
    PG_HIP(pgk::launch_fill_zero(*p, std::max<size_t>(floats, 4), c->stream));
    return PG_OK;
  };
  pg_status s;
  st->layers.resize(m.layers.size());
  for (size_t i = 0; i < m.layers.size(); ++i) {
    const StackLayer& l = m.layers[i];
    StackCache::Layer& k = st->layers[i];
    if (l.has_attn) {
      const size_t n = (size_t)l.attn.kv_heads * l.attn.chunk * l.attn.dim_pad;
      if ((s = alloc(B * n, &k.kring)) || (s = alloc(B * n, &k.vring))) return s;
    }
    if (l.has_rec) {
      if (pgk::rec_has_conv(l.rec.kind) && (s = alloc(B * l.rec.conv.taps * l.rec.conv.channels, &k.conv))) return s;
      if ((s = alloc(B * l.rec.heads * l.rec.dim * l.rec.vdim, &k.state))) return s;
    }
    if (l.has_latent && (s = alloc(B * l.latent.window * l.latent.ld + pgk::kLatentTail, &k.latent))) return s;
  }
  float* words = nullptr;
  if ((s = alloc(sizeof(pgk::StepWords) / sizeof(float), &words))) return s;
  st->words = reinterpret_cast<pgk::StepWords*>(words);
  if ((s = alloc(B * m.width_pad, &st->x)) || (s = alloc(B * m.width_pad, &st->h)) ||
      (s = alloc(B * m.max_in, &st->y)) || (s = alloc(B * m.max_mix, &st->mix)) ||
      (s = alloc(B * m.max_ff, &st->act)) || (s = alloc(B * m.max_part, &st->part)))
    return s;
  if (m.post_norm && ((s = alloc(B * m.width_pad, &st->sub)) || (s = alloc(B * m.max_q, &st->q)) ||
                      (s = alloc(B * m.max_qa, &st->qa)) || (s = alloc(B * m.max_q_rank, &st->cq))))
    return s;
  MoeSizes ms;
  for (const StackLayer& l : m.layers)
    if (l.ffn.kind == PostFeedForward::kMoe) ms.add(l.ffn.moe, (int)B, m.width_pad);
  if (ms.logits) {
    float* ints[6];
    const size_t n[6] = {ms.experts, ms.pairs, ms.pairs, ms.pairs, ms.slots, ms.tiles};
    for (int i = 0; i < 6; ++i)
      if ((s = alloc(n[i], &ints[i]))) return s;
    st->moe.bind(ints);
    if ((s = alloc(ms.logits, &st->moe.logits)) || (s = alloc(ms.act, &st->moe.act)) ||
        (s = alloc(ms.slot_out, &st->moe.slot_out)) || (s = alloc(ms.pairs, &st->moe.route.weight)))
      return s;
  }
  PG_HIP(hipStreamCreateWithFlags(&st->side, hipStreamNonBlocking));
  PG_HIP(hipEventCreateWithFlags(&st->forked, hipEventDisableTiming));
  PG_HIP(hipEventCreateWithFlags(&st->joined, hipEventDisableTiming));
  c->gemm_ws_floats = 8 * B * (size_t)std::max(m.max_in, m.width_pad);
  PG_HIP(hipMalloc(&c->gemm_ws, c->gemm_ws_floats * sizeof(float)));
  PG_HIP(hipMalloc(&c->logits_buf, B * m.vocab * sizeof(float)));
  PG_HIP(hipMalloc(&c->d_tok, B * sizeof(uint32_t)));
  PG_HIP(hipStreamSynchronize(c->stream));
  return PG_OK;
}

namespace {

// A layer's argument structs with this cache's memory.
struct Bound {
  pgk::ChunkAttn attn;
  pgk::Recurrence rec;
  pgk::LatentAttn latent;
};
Bound bind(const StackLayer& l, const StackCache::Layer& k) {
  Bound b{l.attn, l.rec, l.latent};
  b.latent.ring = k.latent;
  b.latent.ring_seq = (size_t)l.latent.window * l.latent.ld;
  b.attn.kring = k.kring;
  b.attn.vring = k.vring;
  b.attn.ring_seq = (size_t)l.attn.kv_heads * l.attn.chunk * l.attn.dim_pad;
  b.rec.state = k.state;
  b.rec.state_seq = (size_t)l.rec.heads * l.rec.dim * l.rec.vdim;
  b.rec.conv.ring = k.conv;
  b.rec.conv.ring_seq = (size_t)l.rec.conv.taps * l.rec.conv.channels;
  return b;
}

struct Gemm {
  const pg_model* m;
  float* ws;
  size_t ws_floats;
  int rows;
  hipStream_t s;
  // C[rows][ldc] = A[rows][K] . W[N][K]^T, or C += scale (.) that, with the next norm of C
  hipError_t operator()(const float* A, const float* W, float* C, int N, int K, const float* resid_scale,
                        const float* norm_gain, float* norm_out) const {
    pgk::GemmArgs a{};
    a.A = A; a.w_bf16 = m->w_bf16; a.W = W; a.bias = nullptr; a.C = C;
    a.M = rows; a.N = N; a.K = K; a.lda = K; a.ldc = N;
    a.ws = ws; a.ws_floats = ws_floats;
    a.split_items_per_cu = m->gemm_split_items;
    a.b9_min_rows = m->gemm_b9_min_rows;
    if (resid_scale) {
      a.resid = C;
      a.col_scale = resid_scale;
    }
    if (norm_out) {
      a.ln_out = norm_out; a.ln_g = norm_gain; a.ln_eps = m->stack->eps; a.rms_cols = m->stack->width;
    }
    return pgk::launch_gemm(a, resid_scale ? pgk::GEMM_RESID_SCALED : pgk::GEMM_BIAS, m->num_cus, s);
  }
  // C[n_rows][N] = epilogue(A[n_rows][lda] . W[N][K]^T + bias)
  // (post_x: the rows' norm is added to it instead, C is working memory)
  hipError_t product(int n_rows, const float* A, int lda, const void* W, float* C, int N, int K, const float* bias = nullptr,
                     int epilogue = pgk::GEMM_BIAS, float* post_x = nullptr, const float* post_gain = nullptr) const {
    pgk::GemmArgs a{};
    a.A = A; a.w_bf16 = m->w_bf16; a.W = static_cast<const float*>(W); a.bias = bias; a.C = C;
    a.M = n_rows; a.N = N; a.K = K; a.lda = lda; a.ldc = N;
    a.ws = ws; a.ws_floats = ws_floats;
    a.split_items_per_cu = m->gemm_split_items;
    a.b9_min_rows = m->gemm_b9_min_rows;
    a.post_x = post_x; a.post_gain = post_gain; a.post_n = m->stack->width; a.ln_eps = m->stack->eps;
    return pgk::launch_gemm(a, epilogue, m->num_cus, s);
  }
};

// Logits of rows of x (rows_at: device list, null for rows 0 .. n - 1) into dst.
pg_status head_rows(const pg_model* model, const Gemm& gemm, const float* x, float* h, const int* rows_at,
                    float* dst) {
  const StackModel& m = *model->stack;
  if (m.post_norm)
    PG_HIP(pgk::launch_group_rms_rows(x, m.width_pad, h, m.width_pad, gemm.rows, m.width, 1, m.final_norm, m.eps, rows_at,
                                      gemm.s));
  else
    PG_HIP(pgk::launch_rms_rows(x, h, gemm.rows, m.width, m.width_pad, m.final_norm, m.eps, m.logit_scale, rows_at,
                                gemm.s));
  PG_HIP(gemm(h, m.head, dst, m.vocab, m.width_pad, nullptr, nullptr, nullptr));
  return PG_OK;
}

// Logits of one row.  add: a sublayer's output that has still to be normed (add_gain) and added.
pg_status head_one(const pg_model* model, const float* x, float* dst, hipStream_t s, const float* add = nullptr,
                   const float* add_gain = nullptr) {
  const StackModel& m = *model->stack;
  pgk::GemvArgs a{};
  a.w_bf16 = model->w_bf16; a.W = m.head; a.bias = nullptr; a.x = x; a.y = dst; a.K = m.width_pad; a.nout = m.vocab;
  a.eps = m.eps; a.norm_n = m.width;
  if (m.post_norm) {
    a.gain = m.final_norm;
    a.add = add; a.add_gain = add_gain; a.add_n = m.width;
    PG_HIP(pgk::launch_gemv(a, pgk::PRO_STACK, pgk::EPI_BIAS, s));
    return PG_OK;
  }
  a.ln_g = m.final_norm; a.out_mul = m.logit_scale;
  PG_HIP(pgk::launch_gemv(a, pgk::PRO_RMS, pgk::EPI_BIAS, s));
  return PG_OK;
}

// One token of every sequence through post-norm layers.  With one sequence a sublayer's output is
// normed and added by the first product of the next one (every block does so for itself; the sum
// goes to the other of the two residual buffers); batches have a launch for it.
pg_status post_norm_step(const pg_model* model, pg_kv_cache* c, ProfileMarks* marks) {
  const StackModel& m = *model->stack;
  StackCache& st = *c->stack;
  hipStream_t s = c->stream;
  const int B = (int)c->B, Cp = m.width_pad;
  const Gemm gemm{model, c->gemm_ws, c->gemm_ws_floats, B, s};
  float *x = st.x, *other = st.h;
  const float* pending = nullptr;  // gain of the norm that st.sub still needs
  // y = epilogue(W x + bias), x first brought up to date
  auto enter = [&](const float* W, const float* bias, float* y, int nout, bool sqrelu) -> hipError_t {
    if (B > 1) return gemm.product(B, x, Cp, W, y, nout, Cp, bias, sqrelu ? pgk::GEMM_SQRELU : pgk::GEMM_BIAS);
    pgk::GemvArgs a{};
    a.w_bf16 = model->w_bf16; a.W = W; a.bias = bias; a.x = x; a.y = y; a.K = Cp; a.nout = nout; a.eps = m.eps;
    if (pending) {
      a.add = st.sub; a.add_gain = pending; a.add_n = m.width; a.x_out = other;
    }
    const hipError_t e = pgk::launch_gemv(a, pgk::PRO_STACK, sqrelu ? pgk::EPI_SQRELU : pgk::EPI_BIAS, s);
    if (pending) std::swap(x, other);
    pending = nullptr;
    return e;
  };
  // y = W (norm of in) (one sequence; groups 0: no norm)
  auto inner = [&](const float* in, const float* W, const float* bias, float* y, int nout, int K, const float* gain,
                   int norm_n, int groups) -> hipError_t {
    pgk::GemvArgs a{};
    a.w_bf16 = model->w_bf16; a.W = W; a.bias = bias; a.x = in; a.y = y; a.K = K; a.nout = nout; a.eps = m.eps;
    if (groups == 0) return pgk::launch_gemv(a, pgk::PRO_NONE, pgk::EPI_BIAS, s);
    a.gain = gain; a.norm_n = norm_n; a.groups = groups;
    return pgk::launch_gemv(a, pgk::PRO_STACK, pgk::EPI_BIAS, s);
  };
  // The end of a sublayer: W (norm of in) + bias, normed and added to x (batches norm `in` beforehand).
  auto leave = [&](const float* in, const float* W, const float* bias, int K, const float* gain, int norm_n, int groups,
                   const float* post) -> hipError_t {
    if (B > 1) return gemm.product(B, in, K, W, st.sub, Cp, K, bias, pgk::GEMM_BIAS, x, post);
    pending = post;
    return inner(in, W, bias, st.sub, Cp, K, gain, norm_n, groups);
  };
  PG_HIP(pgk::launch_begin_step(x, m.embed, model->w_bf16, c->d_tok, B, Cp, st.words, s));
  PG_MARK(kNone);
  for (size_t i = 0; i < m.layers.size(); ++i) {
    const StackLayer& l = m.layers[i];
    const Bound b = bind(l, st.layers[i]);
    PG_HIP(enter(l.in_w, nullptr, st.y, l.n_in, false));
    PG_MARK(kQkv);
    int groups = 0;
    if (l.has_latent) {
      const pgk::LatentAttn& a = b.latent;
      const int nq = a.heads * (a.dim + a.rot_dim);
      if (B > 1) {
        PG_HIP(pgk::launch_group_rms_rows(st.y + a.q_col, l.n_in, st.cq, a.q_pad, B, a.q_rank, 1, a.q_norm, m.eps, nullptr, s));
        PG_HIP(gemm.product(B, st.cq, a.q_pad, l.uq_w, st.q, nq, a.q_pad));
      } else {
        PG_HIP(inner(st.y + a.q_col, l.uq_w, nullptr, st.q, nq, a.q_pad, a.q_norm, a.q_rank, 1));
      }
      pgk::LatentDecode d{};
      d.nseq = B; d.d_pos = &st.words->pos;
      d.y = st.y; d.ld_y = l.n_in;
      d.q = st.q; d.qa = st.qa; d.part = st.part;
      d.splits = pgk::latent_decode_splits(a);
      d.out = st.mix; d.ld_out = l.mix_pad;
      PG_HIP(pgk::launch_latent_decode(d, a, s));
    } else {
      pgk::MixDecode d{};
      d.nseq = B; d.d_pos = &st.words->pos;
      d.y = st.y; d.ld_y = l.n_in;
      d.out = st.mix; d.ld_out = l.mix_pad;
      d.has_rec = 1; d.rec = b.rec; d.attn_splits = 1;
      PG_HIP(pgk::launch_recurrence_decode(d, s));
      groups = l.norm_groups;
      if (B > 1 && groups)
        PG_HIP(pgk::launch_group_rms_rows(st.mix, l.mix_pad, st.mix, l.mix_pad, B, l.mix_cols, groups, l.mix_norm, m.eps,
                                          nullptr, s));
    }
    PG_MARK(kAttention);
    PG_HIP(leave(st.mix, l.out_w, nullptr, l.mix_pad, l.mix_norm, l.mix_cols, groups, l.norm1));
    PG_MARK(kAttnProj);
    const PostFeedForward& f = l.ffn;
    if (f.kind == PostFeedForward::kDense) {
      PG_HIP(enter(f.up_w, f.up_b, st.act, f.ff_pad, true));
      PG_MARK(kMlpFc);
      PG_HIP(leave(st.act, f.down_w, f.down_b, f.ff_pad, nullptr, 0, 0, l.norm2));
    } else if (f.kind == PostFeedForward::kMoe) {
      const bool fused = B == 1 && pgk::moe_router_fits(f.moe, Cp);
      if (!fused) PG_HIP(enter(f.router_w, nullptr, st.moe.logits, f.moe.experts_pad, false));
      if (B > 1) {
        if (pg_status e = moe_rows(model, l, st.moe, x, st.sub, B, s, marks)) return e;
      } else {
        pgk::MoeRow r{};
        r.x = x; r.width = m.width; r.width_pad = Cp; r.eps = m.eps;
        r.act = st.moe.act; r.out = st.sub; r.expert = st.moe.route.expert; r.weight = st.moe.route.weight;
        if (fused) {
          r.router = f.router_w;
          r.add = st.sub; r.add_gain = pending; r.x_out = other;
        } else {
          r.logits = st.moe.logits;
        }
        PG_MARK(kMlpFc);
        PG_HIP(pgk::launch_moe_row(f.moe, r, s));
        if (fused) std::swap(x, other);
        pending = l.norm2;
      }
    }
    PG_MARK(kMlpProj);
  }
  const pg_status r = B == 1 ? head_one(model, x, c->logits_buf, s, pending ? st.sub : nullptr, pending)
                             : head_rows(model, gemm, x, other, nullptr, c->logits_buf);
  if (r) return r;
  PG_MARK(kLogits);
  return PG_OK;
}

pg_status step_launches(const pg_model* model, pg_kv_cache* c, ProfileMarks* marks) {
  const StackModel& m = *model->stack;
  if (m.post_norm) return post_norm_step(model, c, marks);
  StackCache& st = *c->stack;
  hipStream_t s = c->stream;
  const int B = (int)c->B, Cp = m.width_pad;
  const Gemm gemm{model, c->gemm_ws, c->gemm_ws_floats, B, s};
  PG_HIP(pgk::launch_begin_step(st.x, m.embed, model->w_bf16, c->d_tok, B, Cp, st.words, s));
  PG_MARK(kNone);
  for (size_t i = 0; i < m.layers.size(); ++i) {
    const StackLayer& l = m.layers[i];
    const Bound b = bind(l, st.layers[i]);
    if (B == 1) {
      pgk::GemvArgs a{};
      a.w_bf16 = model->w_bf16; a.W = l.in_w; a.bias = nullptr; a.x = st.x; a.y = st.y; a.K = Cp; a.nout = l.n_in;
      a.ln_g = l.norm; a.eps = m.eps; a.norm_n = m.width;
      PG_HIP(pgk::launch_gemv(a, pgk::PRO_RMS, pgk::EPI_BIAS, s));
    } else {
      if (i == 0) PG_HIP(pgk::launch_rms_rows(st.x, st.h, B, m.width, Cp, l.norm, m.eps, 1.0f, nullptr, s));
      PG_HIP(gemm(st.h, l.in_w, st.y, l.n_in, Cp, nullptr, nullptr, nullptr));
    }
    PG_MARK(kQkv);
    pgk::MixDecode d{};
    d.nseq = B; d.d_pos = &st.words->pos;
    d.y = st.y; d.ld_y = l.n_in;
    d.out = st.mix; d.ld_out = l.mix_pad;
    d.act = st.act;
    d.has_attn = l.has_attn; d.has_rec = l.has_rec; d.has_mlp = l.has_mlp;
    d.attn = b.attn; d.rec = b.rec; d.mlp = l.mlp;
    d.attn_splits = l.has_attn ? pgk::mix_decode_splits(l.attn, l.has_rec ? &l.rec : nullptr) : 1;
    d.part = st.part;
    PG_HIP(pgk::launch_mix_decode(d, s));
    // the attention's key splits are added by the projection of the one-sequence step, where
    // they are few
    const bool sum_in_pair = B == 1 && l.has_attn && d.attn_splits > 1 && d.attn_splits <= pgk::kPairMaxSplits;
    if (l.has_attn && d.attn_splits > 1 && !sum_in_pair) PG_HIP(pgk::launch_attn_sum(d, s));
    PG_MARK(kAttention);
    const bool more = i + 1 < m.layers.size();
    if (B == 1) {
      pgk::GemvPair p{};
      p.w_bf16 = model->w_bf16;
      p.W1 = l.out_w; p.x1 = st.mix; p.s1 = l.ls1; p.K1 = l.mix_pad;
      p.resid = st.x; p.y = st.x; p.nout = Cp;
      if (sum_in_pair) {
        p.part = st.part; p.part_splits = d.attn_splits; p.part_n = l.attn.heads * l.attn.dim;
        p.part_col = l.attn.out_col;
      }
      const bool both = l.has_mlp && l.mix_pad + l.mlp.ff_pad <= pgk::kPairMaxK;
      if (both) {
        p.W2 = l.down_w; p.x2 = st.act; p.s2 = l.ls2; p.K2 = l.mlp.ff_pad;
      }
      PG_HIP(pgk::launch_gemv_pair(p, s));
      if (l.has_mlp && !both) {  // (too wide for one launch)
        p.W1 = l.down_w; p.x1 = st.act; p.s1 = l.ls2; p.K1 = l.mlp.ff_pad;
        p.part_splits = 0;
        PG_HIP(pgk::launch_gemv_pair(p, s));
      }
      PG_MARK(kMlpProj);
    } else {
      float* next_h = more ? st.h : nullptr;
      const float* next_g = more ? m.layers[i + 1].norm : nullptr;
      PG_HIP(gemm(st.mix, l.out_w, st.x, Cp, l.mix_pad, l.ls1, next_g, l.has_mlp ? nullptr : next_h));
      PG_MARK(kAttnProj);
      if (l.has_mlp) PG_HIP(gemm(st.act, l.down_w, st.x, Cp, l.mlp.ff_pad, l.ls2, next_g, next_h));
      PG_MARK(kMlpProj);
    }
  }
  pg_status r = B == 1 ? head_one(model, st.x, c->logits_buf, s)
                       : head_rows(model, gemm, st.x, st.h, nullptr, c->logits_buf);
  if (r) return r;
  PG_MARK(kLogits);
  return PG_OK;
}

}  // namespace

pg_status stack_set_pos(pg_kv_cache* c, size_t pos, uint32_t* out) {
  c->stack->lists_ids = out != nullptr;
  PG_HIP(pgk::launch_set_words(c->stack->words, (int)pos, out, c->stream));
  return PG_OK;
}

pg_status stack_step(const pg_model* model, pg_kv_cache* c, ProfileMarks* marks) {
  StackCache& st = *c->stack;
  if (marks || model->opts.decode_path == PG_DECODE_KERNELS) return step_launches(model, c, marks);
  if (!st.warm) {  // the first step loads the kernels; a capture must not
    st.warm = true;
    return step_launches(model, c, nullptr);
  }
  if (!st.graph) {
    PG_HIP(hipStreamBeginCapture(c->stream, hipStreamCaptureModeThreadLocal));
    const pg_status s = step_launches(model, c, nullptr);
    hipGraph_t graph = nullptr;
    const hipError_t e = hipStreamEndCapture(c->stream, &graph);
    if (s || e != hipSuccess) {
      if (graph) (void)hipGraphDestroy(graph);
      if (s) return s;
      PG_HIP(e);
    }
    const hipError_t ei = hipGraphInstantiate(&st.graph, graph, nullptr, nullptr, 0);
    (void)hipGraphDestroy(graph);
    PG_HIP(ei);
  }
  PG_HIP(hipGraphLaunch(st.graph, c->stream));
  return PG_OK;
}

namespace {

// Makes the block of working memory of many rows hold these pieces.
struct Piece {
  float** p;
  size_t n;
};
template <size_t N>
pg_status reserve_rows(StackCache& st, const Piece (&pieces)[N], hipStream_t s) {
  auto r64 = [](size_t v) { return round_up(v, 64); };
  size_t total = 0;
  for (const Piece& p : pieces) total += r64(p.n);
  if (st.rows_floats < total) {
    PG_HIP(hipStreamSynchronize(s));
    if (st.rows) (void)hipFree(st.rows);
    st.rows = nullptr;
    st.rows_floats = 0;
    PG_HIP(hipMalloc(&st.rows, total * sizeof(float)));
    st.rows_floats = total;
  }
  float* at = st.rows;
  for (const Piece& p : pieces) {
    *p.p = at;
    at += r64(p.n);
  }
  return PG_OK;
}

// Logits of the wanted rows of x.  h: want.size() rows of working memory.
pg_status wanted_rows(const pg_model* model, StackCache& st, Gemm gemm, const float* x, float* h,
                      const std::vector<int>& want, float* dst) {
  if (want.empty()) return PG_OK;
  hipStream_t s = gemm.s;
  if (want.size() == 1) return head_one(model, x + (size_t)want[0] * model->stack->width_pad, dst, s);
  if (st.rows_at_cap < want.size()) {
    PG_HIP(hipStreamSynchronize(s));
    if (st.rows_at) (void)hipFree(st.rows_at);
    st.rows_at = nullptr;
    st.rows_at_cap = 0;
    PG_HIP(hipMalloc(&st.rows_at, want.size() * sizeof(int)));
    st.rows_at_cap = want.size();
  }
  // (want is pageable memory: the copy is staged before the call returns)
  PG_HIP(hipMemcpyAsync(st.rows_at, want.data(), want.size() * sizeof(int), hipMemcpyHostToDevice, s));
  gemm.rows = (int)want.size();
  return head_rows(model, gemm, x, h, st.rows_at, dst);
}

// rows_segment for post-norm layers.
pg_status post_norm_rows(const pg_model* model, pg_kv_cache* c, const uint32_t* d_ids, size_t n, size_t pos0,
                         const std::vector<int>& want, float* dst, ProfileMarks* marks) {
  const StackModel& m = *model->stack;
  StackCache& st = *c->stack;
  hipStream_t s = c->stream;
  const size_t B = c->B, rows = B * n, Cp = (size_t)m.width_pad;
  size_t work_floats = 0, lat_floats = 0, kv_floats = 0, act_floats = 0;
  MoeSizes ms;
  for (const StackLayer& l : m.layers) {
    if (l.has_rec) work_floats = std::max(work_floats, pgk::recurrence_work_floats(l.rec, (int)B, (int)n));
    if (l.has_latent) {
      const size_t all = B * (n + pgk::latent_history(l.latent, (int)pos0));
      lat_floats = std::max(lat_floats, all * l.latent.ld);
      kv_floats = std::max(kv_floats, all * up(l.latent.v_row + l.latent.heads * l.latent.vdim, 4));
    }
    if (l.ffn.kind == PostFeedForward::kDense) act_floats = std::max(act_floats, rows * l.ffn.ff_pad);
    if (l.ffn.kind == PostFeedForward::kMoe) ms.add(l.ffn.moe, (int)rows, m.width_pad);
  }
  act_floats = std::max(act_floats, ms.act);
  const size_t ws_floats = 8 * rows * Cp;
  float *x, *h, *sub, *y, *mix, *act, *conv, *decay, *gate, *work, *cq, *q, *lat, *kv, *ws, *ints[6];
  StackCache::MoeBuffers moe;
  const Piece pieces[] = {{&x, rows * Cp}, {&h, want.size() * Cp}, {&sub, rows * Cp}, {&y, rows * m.max_in},
                          {&mix, rows * m.max_mix}, {&act, act_floats}, {&conv, rows * m.max_conv},
                          {&decay, rows * m.max_decay}, {&gate, rows * m.max_gate}, {&work, work_floats},
                          {&cq, rows * m.max_q_rank}, {&q, rows * m.max_q}, {&lat, lat_floats}, {&kv, kv_floats},
                          {&ws, ws_floats}, {&moe.logits, ms.logits}, {&moe.slot_out, ms.slot_out},
                          {&moe.route.weight, ms.pairs}, {&ints[0], ms.experts}, {&ints[1], ms.pairs},
                          {&ints[2], ms.pairs}, {&ints[3], ms.pairs}, {&ints[4], ms.slots}, {&ints[5], ms.tiles}};
  if (pg_status e = reserve_rows(st, pieces, s)) return e;
  moe.act = act;
  moe.bind(ints);
  const Gemm gemm{model, ws, ws_floats, (int)rows, s};
  const int R = (int)rows;
  PG_HIP(pgk::launch_embed_rows(x, m.embed, nullptr, d_ids, R, (int)Cp, s, model->w_bf16, (int)n));
  PG_MARK(kNone);
  for (size_t i = 0; i < m.layers.size(); ++i) {
    const StackLayer& l = m.layers[i];
    const Bound b = bind(l, st.layers[i]);
    PG_HIP(gemm.product(R, x, (int)Cp, l.in_w, y, l.n_in, (int)Cp));
    PG_MARK(kQkv);
    pgk::MixRows r{};
    r.nseq = (int)B; r.n = (int)n; r.pos0 = (int)pos0;
    r.y = y; r.ld_y = l.n_in;
    r.out = mix; r.ld_out = l.mix_pad; r.out_cols = l.mix_cols;
    r.conv_out = conv; r.decay = decay; r.gate = gate;
    r.work = work; r.work_floats = work_floats;
    if (l.has_latent) {
      const pgk::LatentAttn& a = b.latent;
      pgk::LatentRows lr{};
      lr.cq = cq; lr.q = q; lr.lat = lat; lr.kv = kv;
      lr.ld_kv = up(a.v_row + a.heads * a.vdim, 4);
      lr.hist = pgk::latent_history(a, (int)pos0);
      PG_HIP(pgk::launch_latent_prepare_rows(r, a, lr, s));
      PG_HIP(gemm.product(R, cq, a.q_pad, l.uq_w, q, a.heads * (a.dim + a.rot_dim), a.q_pad));
      PG_HIP(gemm.product((int)(B * (n + lr.hist)), lat, a.ld, a.up_w, kv, lr.ld_kv, a.kv_pad));
      PG_HIP(pgk::launch_latent_rotate_rows(r, a, lr, s));
      PG_HIP(pgk::launch_latent_attn_rows(r, a, lr, s));
    } else {
      const pgk::Recurrence& k = b.rec;
      if (k.kind == pgk::REC_CHANNEL_DELTA) {
        PG_HIP(gemm.product(R, y + k.low_a.col, l.n_in, k.low_a.w, decay, k.heads * k.dim, k.low_a.rank));
        PG_HIP(gemm.product(R, y + k.low_g.col, l.n_in, k.low_g.w, gate, k.heads * k.vdim, k.low_g.rank));
      }
      PG_HIP(pgk::launch_short_conv_rows(r, k.conv, s));
      PG_HIP(pgk::launch_recurrence_rows(r, k, s));
      PG_HIP(pgk::launch_commit_rows(r, nullptr, &k.conv, s));
      if (l.norm_groups)
        PG_HIP(pgk::launch_group_rms_rows(mix, l.mix_pad, mix, l.mix_pad, R, l.mix_cols, l.norm_groups, l.mix_norm, m.eps,
                                          nullptr, s));
    }
    PG_MARK(kAttention);
    PG_HIP(gemm.product(R, mix, l.mix_pad, l.out_w, sub, (int)Cp, l.mix_pad, nullptr, pgk::GEMM_BIAS, x, l.norm1));
    PG_MARK(kAttnProj);
    const PostFeedForward& f = l.ffn;
    if (f.kind == PostFeedForward::kDense) {
      PG_HIP(gemm.product(R, x, (int)Cp, f.up_w, act, f.ff_pad, (int)Cp, f.up_b, pgk::GEMM_SQRELU));
      PG_MARK(kMlpFc);
      PG_HIP(gemm.product(R, act, f.ff_pad, f.down_w, sub, (int)Cp, f.ff_pad, f.down_b, pgk::GEMM_BIAS, x, l.norm2));
    } else if (f.kind == PostFeedForward::kMoe) {
      PG_HIP(gemm.product(R, x, (int)Cp, f.router_w, moe.logits, f.moe.experts_pad, (int)Cp));
      if (pg_status e = moe_rows(model, l, moe, x, sub, R, s, marks)) return e;
    }
    PG_MARK(kMlpProj);
  }
  if (pg_status e = wanted_rows(model, st, gemm, x, h, want, dst)) return e;
  PG_MARK(kLogits);
  return PG_OK;
}

// Tokens [t0, t0 + n) of every sequence, ids in device memory ([B][n]).
pg_status rows_segment(const pg_model* model, pg_kv_cache* c, const uint32_t* d_ids, size_t n, size_t pos0,
                       const std::vector<int>& want, float* dst, ProfileMarks* marks) {
  const StackModel& m = *model->stack;
  if (m.post_norm) return post_norm_rows(model, c, d_ids, n, pos0, want, dst, marks);
  StackCache& st = *c->stack;
  hipStream_t s = c->stream;
  const size_t B = c->B, rows = B * n, Cp = (size_t)m.width_pad;
  const size_t ws_floats = 8 * rows * Cp;
  float *x, *h, *y, *mix, *act, *krot, *conv, *decay, *work, *ws, *ws_side;
  size_t work_floats = 0;
  for (const StackLayer& l : m.layers)
    if (l.has_rec) work_floats = std::max(work_floats, pgk::recurrence_work_floats(l.rec, (int)B, (int)n));
  const Piece pieces[] = {{&x, rows * Cp}, {&h, std::max(rows, want.size()) * Cp}, {&y, rows * m.max_in},
                          {&mix, rows * m.max_mix}, {&act, rows * m.max_ff}, {&krot, rows * m.max_keys},
                          {&conv, rows * m.max_conv}, {&decay, rows * m.max_decay}, {&work, work_floats},
                          {&ws, ws_floats}, {&ws_side, ws_floats}};
  if (pg_status e = reserve_rows(st, pieces, s)) return e;
  const Gemm gemm{model, ws, ws_floats, (int)rows, s};
  PG_HIP(pgk::launch_embed_rows(x, m.embed, nullptr, d_ids, (int)rows, (int)Cp, s, model->w_bf16, (int)n));
  PG_MARK(kNone);
  PG_HIP(pgk::launch_rms_rows(x, h, (int)rows, m.width, (int)Cp, m.layers[0].norm, m.eps, 1.0f, nullptr, s));
  PG_MARK(kLayerNorm);
  for (size_t i = 0; i < m.layers.size(); ++i) {
    const StackLayer& l = m.layers[i];
    const Bound b = bind(l, st.layers[i]);
    PG_HIP(gemm(h, l.in_w, y, l.n_in, (int)Cp, nullptr, nullptr, nullptr));
    PG_MARK(kQkv);
    pgk::MixRows r{};
    r.nseq = (int)B; r.n = (int)n; r.pos0 = (int)pos0;
    r.y = y; r.ld_y = l.n_in;
    r.out = mix; r.ld_out = l.mix_pad; r.out_cols = l.mix_cols;
    r.act = act; r.k_rot = krot; r.conv_out = conv; r.decay = decay;
    r.work = work; r.work_floats = work_floats;
    const bool more = i + 1 < m.layers.size();
    float* next_h = more ? h : nullptr;
    const float* next_g = more ? m.layers[i + 1].norm : nullptr;
    // The recurrence is a chain over the tokens that leaves most of the chip idle: with enough
    // rows, the attention and the MLP (its result goes straight to the residual) run beside it.
    const bool fork = !marks && rows >= 64 && l.has_rec && (l.has_attn || l.has_mlp);
    hipStream_t side = fork ? st.side : s;
    Gemm side_gemm = gemm;
    side_gemm.s = side;
    side_gemm.ws = fork ? ws_side : ws;
    if (fork) {
      PG_HIP(hipEventRecord(st.forked, s));
      PG_HIP(hipStreamWaitEvent(side, st.forked, 0));
    }
    if (l.has_attn) {
      PG_HIP(pgk::launch_rotary_rows(r, b.attn, side));
      PG_HIP(pgk::launch_chunk_attn_rows(r, b.attn, side));
      PG_HIP(pgk::launch_commit_rows(r, &b.attn, nullptr, side));
    }
    PG_MARK(kAttention);
    if (l.has_mlp) {
      PG_HIP(pgk::launch_gated_mlp_rows(r, l.mlp, side));
      PG_MARK(kMlpFc);
      PG_HIP(side_gemm(act, l.down_w, x, (int)Cp, l.mlp.ff_pad, l.ls2, nullptr, nullptr));
      PG_MARK(kMlpProj);
    }
    if (l.has_rec) {
      if (l.rec.kind == pgk::REC_DELTA) PG_HIP(pgk::launch_short_conv_rows(r, b.rec.conv, s));
      PG_HIP(pgk::launch_recurrence_rows(r, b.rec, s));
      if (l.rec.kind == pgk::REC_DELTA) PG_HIP(pgk::launch_commit_rows(r, nullptr, &b.rec.conv, s));
    }
    if (fork) {
      PG_HIP(hipEventRecord(st.joined, side));
      PG_HIP(hipStreamWaitEvent(s, st.joined, 0));
    }
    PG_MARK(kAttention);
    PG_HIP(gemm(mix, l.out_w, x, (int)Cp, l.mix_pad, l.ls1, next_g, next_h));
    PG_MARK(kAttnProj);
  }
  if (pg_status e = wanted_rows(model, st, gemm, x, h, want, dst)) return e;
  PG_MARK(kLogits);
  return PG_OK;
}
#undef PG_MARK

}  // namespace

pg_status stack_rows(const pg_model* model, pg_kv_cache* c, const uint32_t* ids, size_t n, size_t pos0,
                     const std::vector<int>& rows, float* dst, ProfileMarks* marks) {
  constexpr size_t kSegmentRows = 8192;
  const size_t B = c->B, V = (size_t)model->stack->vocab;
  const size_t seg = std::max<size_t>(32, kSegmentRows / B);  // tokens (the recurrences' chunk at least)
  if (c->prompt_cap < B * std::min(n, seg)) {
    for (int i = 0; i < 2; ++i) {
      if (c->ev_prompt[i]) PG_HIP(hipEventSynchronize(c->ev_prompt[i]));
      if (c->h_prompt[i]) (void)hipHostFree(c->h_prompt[i]);
      c->h_prompt[i] = nullptr;
    }
    c->prompt_cap = B * std::min(n, seg);
  }
  for (size_t t0 = 0; t0 < n; t0 += seg) {
    const size_t nt = std::min(seg, n - t0);
    // ids through pinned staging to the device, behind what is queued
    const unsigned turn = c->prompt_turn++ & 1;
    if (!c->h_prompt[turn])
      PG_HIP(hipHostMalloc(&c->h_prompt[turn], c->prompt_cap * sizeof(uint32_t), hipHostMallocDefault));
    if (!c->ev_prompt[turn]) PG_HIP(hipEventCreateWithFlags(&c->ev_prompt[turn], hipEventDisableTiming));
    else PG_HIP(hipEventSynchronize(c->ev_prompt[turn]));
    if (c->ids_cap < B * nt) return fail(PG_BACKEND, "id buffer is too small");
    for (size_t b = 0; b < B; ++b)
      std::memcpy(c->h_prompt[turn] + b * nt, ids + b * n + t0, nt * sizeof(uint32_t));
    PG_HIP(hipMemcpyAsync(c->d_out_ids, c->h_prompt[turn], B * nt * sizeof(uint32_t), hipMemcpyHostToDevice, c->stream));
    PG_HIP(hipEventRecord(c->ev_prompt[turn], c->stream));
    std::vector<int> want;
    size_t first = 0;
    bool any = false;
    for (size_t k = 0; k < rows.size(); ++k) {
      const size_t b = (size_t)rows[k] / n, t = (size_t)rows[k] % n;
      if (t < t0 || t >= t0 + nt) continue;
      if (!any) first = k;
      any = true;
      want.push_back((int)(b * nt + (t - t0)));
    }
    if (pg_status s = rows_segment(model, c, c->d_out_ids, nt, pos0 + t0, want, dst + first * V, marks)) return s;
  }
  return stack_set_pos(c, pos0 + n);
}

}  // namespace pgh
