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
  // the tensors of the input projection and the output projection, in column order
  struct Part {
    std::string name;
    int rows, col;
  };
  std::vector<Part> in_parts, out_parts;
  int next_in = 0;
  int add_in(const std::string& name, int rows) {
    const int at = next_in;
    in_parts.push_back({name, rows, at});
    next_in = up(at + rows, 4);  // (columns are read four at a time)
    return at;
  }
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
  r.delta = 1;
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
  r.delta = 0;
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
  // Tensor name [r][c] at (row, col) of the staged matrix of `cols` columns.
  pg_status place(const std::string& name, int r, int c, size_t row, size_t col, size_t cols) {
    TensorView t;
    if (pg_status s = get(name, {(uint64_t)r, (uint64_t)c}, &t)) return s;
    for (int i = 0; i < r; ++i) {
      unsigned char* dst = host.data() + ((row + i) * cols + col) * elem();
      const size_t at = (size_t)i * c;
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

pg_status load_layer(Loader& ld, const std::string& name, LayerPlan& p) {
  StackModel& m = ld.model;
  StackLayer& l = p.layer;
  const int C = m.width, Cp = m.width_pad;
  const uint64_t uC = (uint64_t)C;
  pg_status s;
  if ((s = ld.vector(name + ".norm1", {}, 1, &l.norm))) return s;
  if ((s = ld.vector(name + ".ls1", {uC}, Cp, &l.ls1))) return s;
  ld.begin(l.n_in, Cp);
  for (const auto& part : p.in_parts)
    if ((s = ld.place(part.name, part.rows, C, part.col, 0, Cp))) return s;
  if ((s = ld.end(&l.in_w))) return s;
  ld.begin(Cp, l.mix_pad);
  for (const auto& part : p.out_parts)
    if ((s = ld.place(part.name, C, part.rows, 0, part.col, l.mix_pad))) return s;
  if ((s = ld.end(&l.out_w))) return s;
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
    const std::string q = name + (r.delta ? ".mix.right." : ".mix.");
    float* v = nullptr;
    if ((s = ld.vector(q + "norm", {(uint64_t)r.vdim}, 0, &v))) return s;
    r.norm = v;
    if (r.delta) {
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

bool stack_config_matches(const Json& config) {
  const Json* a = config.find("architecture");
  return a && a->kind == Json::Str && a->str == "Tarepel";
}

pg_status stack_create(const std::string& config_path, const Json& config, const pg_tensor_store& store,
                       const pg_hip_options& opts, pg_model** out) {
  *out = nullptr;
  pg_status s;
  const Node root{&config, "", &config_path};
  auto m = std::make_shared<StackModel>();
  double eps = 0.0, logit_scale = 0.0;
  Node norm, layers;
  if ((s = root.text("architecture", &m->architecture))) return s;
  if ((s = root.size("vocab", 1, 1 << 30, &m->vocab))) return s;
  if ((s = root.size("width", 1, kMaxWidth, &m->width))) return s;
  if ((s = root.number("logit_scale", &logit_scale))) return s;
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
    Node mixer, mlp;
    if ((s = n.text("type", &p.type))) return s;
    if ((s = n.object("mixer", &mixer))) return s;
    if (p.type == "parallel") {
      Node left, right;
      double ls = 0.0, rs = 0.0;
      if ((s = mixer.number("left_scale", &ls))) return s;
      if ((s = mixer.number("right_scale", &rs))) return s;
      if ((s = mixer.object("left", &left))) return s;
      if ((s = mixer.object("right", &right))) return s;
      if ((s = read_attention(left, name + ".mix.left.", ls, &p))) return s;
      if ((s = read_delta(right, name + ".mix.right.", rs, m->eps, &p))) return s;
    } else if (p.type == "gla") {
      TensorView t;  // the rank of the decay projection is the tensor's
      if ((s = find_tensor(store, name + ".mix.a1", &t))) return s;
      if (t.shape.size() != 2 || t.shape[0] < 1 || t.shape[0] > (uint64_t)kMaxWidth)
        return fail(PG_INVALID_WEIGHTS, "tensor " + name + ".mix.a1 must have two dimensions");
      if ((s = read_gla(mixer, name + ".mix.", (int)t.shape[0], m->eps, &p))) return s;
    } else {
      return n.bad("type `" + p.type + "` is not supported");
    }
    const Json* has = n.v->find("mlp");
    if (has && has->kind != Json::Null) {
      if ((s = n.object("mlp", &mlp))) return s;
      if ((s = read_mlp(mlp, name + ".mlp.", &p))) return s;
    }
    StackLayer& l = p.layer;
    l.n_in = up(p.next_in, 32);
    l.mix_pad = up(l.mix_cols, 32);
    if (l.mix_pad > kMaxWidth || (l.has_mlp && l.mlp.ff_pad > kMaxWidth))
      return n.bad("is too wide: heads * vdim of the mixers and ff may be up to " + std::to_string(kMaxWidth));
    m->max_in = std::max(m->max_in, l.n_in);
    m->max_mix = std::max(m->max_mix, l.mix_pad);
    m->max_ff = std::max(m->max_ff, l.has_mlp ? l.mlp.ff_pad : 0);
    if (l.has_attn) {
      m->max_keys = std::max(m->max_keys, up(l.attn.kv_heads * l.attn.dim, 4));
      m->max_part = std::max(m->max_part, pgk::mix_decode_splits(l.attn, l.has_rec ? &l.rec : nullptr) * l.attn.heads * l.attn.dim);
    }
    if (l.has_rec) {
      if (l.rec.delta) m->max_conv = std::max(m->max_conv, l.rec.conv.channels);
      else m->max_decay = std::max(m->max_decay, up(l.rec.heads * l.rec.dim, 4));
    }
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
  if ((s = ld.vector("final.norm", {}, 1, &m->final_norm))) return s;
  ld.begin(m->vocab, Cp);
  if ((s = ld.place("head", m->vocab, C, 0, 0, Cp))) return s;
  if ((s = ld.end(&m->head))) return s;
  model->stack = m;
  *out = model.release();
  return PG_OK;
}

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
      if (l.rec.delta && (s = alloc(B * l.rec.conv.taps * l.rec.conv.channels, &k.conv))) return s;
      if ((s = alloc(B * l.rec.heads * l.rec.dim * l.rec.vdim, &k.state))) return s;
    }
  }
  float* words = nullptr;
  if ((s = alloc(sizeof(pgk::StepWords) / sizeof(float), &words))) return s;
  st->words = reinterpret_cast<pgk::StepWords*>(words);
  if ((s = alloc(B * m.width_pad, &st->x)) || (s = alloc(B * m.width_pad, &st->h)) ||
      (s = alloc(B * m.max_in, &st->y)) || (s = alloc(B * m.max_mix, &st->mix)) ||
      (s = alloc(B * m.max_ff, &st->act)) || (s = alloc(B * m.max_part, &st->part)))
    return s;
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
};
Bound bind(const StackLayer& l, const StackCache::Layer& k) {
  Bound b{l.attn, l.rec};
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
};

#define PG_MARK(b) \
  do {             \
    if (marks) PG_HIP(marks->mark(s, ProfileMarks::b)); \
  } while (0)

// Logits of rows of x (rows_at: device list, null for rows 0 .. n - 1) into dst.
pg_status head_rows(const pg_model* model, const Gemm& gemm, const float* x, float* h, const int* rows_at,
                    float* dst) {
  const StackModel& m = *model->stack;
  PG_HIP(pgk::launch_rms_rows(x, h, gemm.rows, m.width, m.width_pad, m.final_norm, m.eps, m.logit_scale, rows_at,
                              gemm.s));
  PG_HIP(gemm(h, m.head, dst, m.vocab, m.width_pad, nullptr, nullptr, nullptr));
  return PG_OK;
}

pg_status head_one(const pg_model* model, const float* x, float* dst, hipStream_t s) {
  const StackModel& m = *model->stack;
  pgk::GemvArgs a{};
  a.w_bf16 = model->w_bf16; a.W = m.head; a.bias = nullptr; a.x = x; a.y = dst; a.K = m.width_pad; a.nout = m.vocab;
  a.ln_g = m.final_norm; a.eps = m.eps; a.norm_n = m.width; a.out_mul = m.logit_scale;
  PG_HIP(pgk::launch_gemv(a, pgk::PRO_RMS, pgk::EPI_BIAS, s));
  return PG_OK;
}

pg_status step_launches(const pg_model* model, pg_kv_cache* c, ProfileMarks* marks) {
  const StackModel& m = *model->stack;
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

// Tokens [t0, t0 + n) of every sequence, ids in device memory ([B][n]).
pg_status rows_segment(const pg_model* model, pg_kv_cache* c, const uint32_t* d_ids, size_t n, size_t pos0,
                       const std::vector<int>& want, float* dst, ProfileMarks* marks) {
  const StackModel& m = *model->stack;
  StackCache& st = *c->stack;
  hipStream_t s = c->stream;
  const size_t B = c->B, rows = B * n, Cp = (size_t)m.width_pad;
  auto r64 = [](size_t v) { return round_up(v, 64); };
  const size_t ws_floats = 8 * rows * Cp;
  struct Piece { float** p; size_t n; };
  float *x, *h, *y, *mix, *act, *krot, *conv, *decay, *work, *ws, *ws_side;
  size_t work_floats = 0;
  for (const StackLayer& l : m.layers)
    if (l.has_rec) work_floats = std::max(work_floats, pgk::recurrence_work_floats(l.rec, (int)B, (int)n));
  const Piece pieces[] = {{&x, rows * Cp}, {&h, std::max(rows, want.size()) * Cp}, {&y, rows * m.max_in},
                          {&mix, rows * m.max_mix}, {&act, rows * m.max_ff}, {&krot, rows * m.max_keys},
                          {&conv, rows * m.max_conv}, {&decay, rows * m.max_decay}, {&work, work_floats},
                          {&ws, ws_floats}, {&ws_side, ws_floats}};
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
  {
    float* at = st.rows;
    for (const Piece& p : pieces) {
      *p.p = at;
      at += r64(p.n);
    }
  }
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
      if (l.rec.delta) PG_HIP(pgk::launch_short_conv_rows(r, b.rec.conv, s));
      PG_HIP(pgk::launch_recurrence_rows(r, b.rec, s));
      if (l.rec.delta) PG_HIP(pgk::launch_commit_rows(r, nullptr, &b.rec.conv, s));
    }
    if (fork) {
      PG_HIP(hipEventRecord(st.joined, side));
      PG_HIP(hipStreamWaitEvent(s, st.joined, 0));
    }
    PG_MARK(kAttention);
    PG_HIP(gemm(mix, l.out_w, x, (int)Cp, l.mix_pad, l.ls1, next_g, next_h));
    PG_MARK(kAttnProj);
  }
  if (want.size() == 1) {
    if (pg_status e = head_one(model, x + (size_t)want[0] * Cp, dst, s)) return e;
  } else if (!want.empty()) {
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
    Gemm g = gemm;
    g.rows = (int)want.size();
    if (pg_status e = head_rows(model, g, x, h, st.rows_at, dst)) return e;
  }
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
