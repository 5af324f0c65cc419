// session_lirulix.hip -- the Lirulix decoder: a list of layers, each with attention over
// all earlier tokens (a sink in the softmax), differential attention through a sliding
// window or a gated delta rule as its mixer, and a dense gated feed-forward or nothing;
// norms with a weight per channel ahead of every sublayer.  A span of the layers runs
// several times in a row.  Sizes, constants and the order of layers come from the
// configuration.
//
// What a sequence keeps, for every run of a layer: keys and values per head, as a row per
// position or, behind a window, as a ring; or the delta rule's state and the last inputs
// of its convolution.
//
// A token: 6 launches in a layer with attention, 5 with the delta rule, 2 less without a
// feed-forward, captured into one graph:
//   [residual + norm -> projections] -> [mixer: 2 or 1] -> [-> output matrix] ->
//   [residual + norm -> gate | up -> activation] -> [-> down]
#include "delta_rule.h"
#include "elementwise.h"
#include "folder_session.h"
#include "head_attn.h"
#include "rotary.h"

#include <cmath>
#include <memory>

namespace bh {
namespace {

enum MixerKind { kAttention, kDifferential, kDelta };

struct LayerConfig {
  MixerKind kind = kAttention;
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  // attention
  int window = 0;
  double scale = 0.0, diff = 0.0;
  Rotary rot{0, 1.0};
  // delta rule
  int taps = 0;
  // feed-forward; 0: none
  int ff = 0;
};

struct LirulixConfig {
  int vocab = 0, width = 0;
  float eps = 0.f;
  std::vector<LayerConfig> layers;
  int loop_start = 0, loop_stop = 0, loop_times = 0; // layers start .. stop - 1, so often

  explicit LirulixConfig(const Json &j) {
    vocab = positive(j, "vocab");
    width = positive(j, "width");
    eps = (float)j.at("norm").at("eps").number();
    for (const Json &e : j.at("layers").array())
      layers.push_back(layer(e));
    if (layers.empty())
      throw std::runtime_error("config: no layers");
    const Json *loop = j.find("loop");
    if (loop && !loop->is_null()) {
      const int64_t start = loop->at("start").integer();
      loop_stop = positive(*loop, "stop");
      loop_times = positive(*loop, "times");
      if (start < 0 || start >= loop_stop || loop_stop > (int)layers.size() || loop_times > 4096)
        throw std::runtime_error("config: \"loop\" names layers that do not exist");
      loop_start = (int)start;
    }
  }

  static LayerConfig layer(const Json &e) {
    LayerConfig c;
    const std::string type = e.at("type").string();
    const Json &m = e.at("mixer");
    c.heads = positive(m, "heads");
    c.kv_heads = positive(m, "kv_heads");
    c.dim = positive(m, "dim");
    c.vdim = positive(m, "vdim");
    if (c.heads % c.kv_heads)
      throw std::runtime_error("config: heads must be a multiple of kv_heads");
    if (type == "attention" || type == "attention_2") {
      c.kind = type == "attention" ? kAttention : kDifferential;
      c.scale = m.at("scale").number();
      const Json &r = m.at("rot");
      const int dims = positive(r, "dims");
      const double base = r.at("base").number();
      if (dims % 2 || dims > c.dim || base <= 0.0)
        throw std::runtime_error("config: a rotation of " + std::to_string(dims) + " dimensions of " +
                                 std::to_string(c.dim));
      c.rot = Rotary(dims, base);
      const Json *s = r.find("scaling");
      auto of = [&](const char *key) { return s->at(key).number(); };
      if (s && !s->is_null()) {
        if (c.kind == kAttention)
          c.rot.yarn(base, of("factor"), of("original"), of("fast"), of("slow"));
        else
          c.rot.banded(of("factor"), of("low"), of("high"), of("original"));
      }
      if (c.kind == kDifferential) {
        c.window = positive(m.at("mask"), "size");
        c.diff = m.at("diff").number();
      }
    } else if (type == "channel_delta") {
      c.kind = kDelta;
      c.taps = positive(m, "conv");
    } else {
      throw std::runtime_error("config: unknown mixer \"" + type + "\"");
    }
    const Json *f = e.find("mlp");
    if (f && !f->is_null()) {
      if (f->at("kind").string() != "dense")
        throw std::runtime_error("config: unknown feed-forward \"" + f->at("kind").string() + "\"");
      c.ff = positive(*f, "ff");
    }
    return c;
  }
};

struct LirulixLayer {
  float *norm1 = nullptr, *norm2 = nullptr;
  Bf16Matrix in; // q | k | v (| gate), or q | k | v | step size | inner decay | inner gate
  Part q, k, v, g, b, a1, g1;
  Bf16Matrix o;
  HeadShape head;
  DeltaShape delta;
  Bf16Matrix gate_up, down; // gate_up: of the first of its two matrices
};

// One run of a layer: a looped layer has several, each with a cache of its own.
struct LirulixRun {
  int layer = 0;
  const float *add = nullptr; // joins the residual ahead of the layer
  void *keys = nullptr, *values_t = nullptr;
  float *ring = nullptr, *state = nullptr;
};

struct LirulixSession : FolderSession {
  LirulixConfig cfg;
  std::vector<LirulixLayer> layers;
  std::vector<LirulixRun> runs;
  uint16_t *embed = nullptr; // [vocab][width] bfloat16
  float *embed_norm = nullptr, *final_norm = nullptr;
  Bf16Matrix head;
  int longest = 1; // visible keys, at most

  // one token
  float *x[2] = {nullptr, nullptr}, *y = nullptr, *proj = nullptr, *mix = nullptr, *mix_gate = nullptr,
        *act = nullptr, *hrow = nullptr, *part_acc = nullptr, *part_ml = nullptr;

  // a block of a prompt
  float *pf_x = nullptr, *pf_y = nullptr, *pf_proj = nullptr, *pf_maps = nullptr, *pf_delta = nullptr,
        *pf_logits = nullptr;
  void *pf_act = nullptr, *pf_mix = nullptr, *pf_queries = nullptr, *pf_ff = nullptr;
  int ld_act = 0, ld_mix = 0, max_proj = 0;
  static constexpr int kScanRows = 12; // the delta rule takes fewer rows token by token

  LirulixSession(const Json &config, const ModelOptions &o) : FolderSession(o), cfg(config) {}

  const char *architecture() const override { return "Lirulix"; }
  int width16() const { return (int)round_up(cfg.width, 16); }

  // ---- loading -------------------------------------------------------------------
  // a norm's weight, stored as its distance from 1
  float *load_norm(const ModelFolder &f, const std::string &name) {
    std::vector<float> w = f.values(name, {cfg.width});
    for (float &v : w)
      v += 1.0f;
    return device_copy(w);
  }

  void load_attention(const ModelFolder &f, const std::string &p, const LayerConfig &c, LirulixLayer &L) {
    HeadShape &s = L.head;
    s.heads = c.heads;
    s.kv_heads = c.kv_heads;
    s.maps = c.kind == kDifferential ? 2 : 1;
    s.dim = c.dim;
    s.vdim = c.vdim;
    s.rot_dims = c.rot.dims();
    s.turns = device_copy(c.rot.turns);
    s.rot_gain = (float)c.rot.gain;
    s.scale = (float)c.scale;
    s.window = c.window;
    s.f32 = opt.f32;
    head_cache_rows(s, opt.max_len, opt.prefill_block);
    longest = std::max(longest, c.window ? std::min(c.window, opt.max_len) : opt.max_len);
    L.q.n = c.heads * s.maps * c.dim;
    L.k.n = c.kv_heads * s.maps * c.dim;
    L.v.n = c.kv_heads * c.vdim;
    std::vector<std::pair<std::string, Part *>> parts = {{"q", &L.q}, {"k", &L.k}, {"v", &L.v}};
    if (c.kind == kAttention) {
      s.sink = device_copy(f.values(p + "sink", {c.heads}));
    } else {
      auto dot = [&](const char *a, const char *b) {
        const std::vector<float> u = f.values(p + a, {c.dim}), v = f.values(p + b, {c.dim});
        double t = 0.0;
        for (size_t i = 0; i < u.size(); ++i)
          t += (double)u[i] * v[i];
        return t;
      };
      s.lambda = (float)(std::exp(dot("lq1", "lk1")) - std::exp(dot("lq2", "lk2")) + c.diff);
      s.eps = cfg.eps;
      s.out_gain = (float)(1.0 - c.diff);
      s.gated = true;
      L.g.n = c.heads * c.vdim;
      parts.emplace_back("g", &L.g);
    }
    L.in = load_parts(f, p, parts, cfg.width);
  }

  void load_delta(const ModelFolder &f, const std::string &p, const LayerConfig &c, LirulixLayer &L) {
    DeltaShape &s = L.delta;
    s.heads = c.heads;
    s.kv_heads = c.kv_heads;
    s.dim = c.dim;
    s.vdim = c.vdim;
    s.taps = c.taps;
    s.eps = cfg.eps;
    s.decay_rank = f.size(p + "a1", 0);
    s.gate_rank = f.size(p + "g1", 0);
    L.q.n = L.k.n = c.kv_heads * c.dim;
    L.v.n = c.heads * c.vdim;
    L.b.n = c.heads;
    L.a1.n = s.decay_rank;
    L.g1.n = s.gate_rank;
    L.in = load_parts(f, p, {{"q", &L.q}, {"k", &L.k}, {"v", &L.v}, {"b", &L.b}, {"a1", &L.a1}, {"g1", &L.g1}},
                      cfg.width);
    s.q_at = L.q.at;
    s.k_at = L.k.at;
    s.v_at = L.v.at;
    s.beta_at = L.b.at;
    s.decay_at = L.a1.at;
    s.gate_at = L.g1.at;
    s.channels = L.b.at;
    std::vector<float> conv((size_t)c.taps * s.channels); // a row per tap
    for (const auto &part : {std::make_pair("q.conv", &L.q), std::make_pair("k.conv", &L.k),
                             std::make_pair("v.conv", &L.v)}) {
      const std::vector<float> w = f.values(p + part.first, {part.second->n, c.taps});
      for (int i = 0; i < part.second->n; ++i)
        for (int t = 0; t < c.taps; ++t)
          conv[(size_t)t * s.channels + part.second->at + i] = w[(size_t)i * c.taps + t];
    }
    s.conv_w = device_copy(conv);
    s.decay_w = device_bf16(f.bf16(p + "a2", {c.heads * c.dim, s.decay_rank}));
    s.gate_w = device_bf16(f.bf16(p + "g2", {c.heads * c.vdim, s.gate_rank}));
    s.decay = load_matrix(f, p + "a2", c.heads * c.dim, s.decay_rank);
    s.gate = load_matrix(f, p + "g2", c.heads * c.vdim, s.gate_rank);
    s.decay_bias = device_copy(f.values(p + "dt_bias", {c.heads * c.dim}));
    std::vector<float> speed = f.values(p + "A_log", {c.heads});
    for (float &v : speed)
      v = (float)-std::exp((double)v);
    s.decay_speed = device_copy(speed);
    s.norm_w = device_copy(f.values(p + "norm", {c.vdim}));
  }

  void load(const ModelFolder &f) {
    const int W = cfg.width;
    embed = device_bf16(f.bf16("embed", {cfg.vocab, W}));
    embed_norm = load_norm(f, "embed.norm");
    final_norm = load_norm(f, "final.norm");
    head = load_matrix(f, "head", cfg.vocab, W);
    int mix_max = 1, ff_max = 16, parts = 0, parts_ml = 0;
    for (size_t i = 0; i < cfg.layers.size(); ++i) {
      const LayerConfig &c = cfg.layers[i];
      const std::string p = "l" + std::to_string(i) + ".";
      layers.emplace_back();
      LirulixLayer &L = layers.back();
      L.norm1 = load_norm(f, p + "norm1");
      if (c.kind == kDelta)
        load_delta(f, p + "mix.", c, L);
      else
        load_attention(f, p + "mix.", c, L);
      max_proj = std::max(max_proj, L.in.N);
      mix_max = std::max(mix_max, c.heads * c.vdim);
      L.o = load_matrix(f, p + "mix.o", W, c.heads * c.vdim);
      if (c.kind != kDelta) {
        const int chunks = head_max_chunks(L.head, opt.max_len) * L.head.map_heads();
        parts = std::max(parts, chunks * L.head.vdim16());
        parts_ml = std::max(parts_ml, chunks * 2);
      }
      if (!c.ff)
        continue;
      L.norm2 = load_norm(f, p + "norm2");
      const int ff16 = (int)round_up(c.ff, 16);
      L.gate_up = matrix(2 * (int64_t)ff16, W);
      {
        Upload g(f.bf16(p + "mlp.gate", {c.ff, W}), stream), u(f.bf16(p + "mlp.up", {c.ff, W}), stream);
        pack(L.gate_up, 0, g.p, W, 1, c.ff);
        pack(L.gate_up, ff16, u.p, W, 1, c.ff);
      }
      L.gate_up.N = ff16;
      L.down = load_matrix(f, p + "mlp.down", W, c.ff);
      ff_max = std::max(ff_max, ff16);
    }
    auto run = [&](int layer, const float *add) {
      const LirulixLayer &L = layers[(size_t)layer];
      LirulixRun r;
      r.layer = layer;
      r.add = add;
      if (cfg.layers[(size_t)layer].kind == kDelta) {
        r.ring = device_zeros<float>((size_t)L.delta.taps * L.delta.channels);
        r.state = device_zeros<float>((size_t)L.delta.heads * L.delta.dim * L.delta.vdim);
      } else {
        r.keys = device_zeros<char>(L.head.key_bytes());
        r.values_t = device_zeros<char>(L.head.value_bytes());
      }
      runs.push_back(r);
    };
    for (int i = 0; i < cfg.loop_start; ++i)
      run(i, nullptr);
    if (cfg.loop_times) {
      const float *steps = device_copy(f.values("loop.step", {cfg.loop_times, W}));
      for (int t = 0; t < cfg.loop_times; ++t)
        for (int i = cfg.loop_start; i < cfg.loop_stop; ++i)
          run(i, i == cfg.loop_start ? steps + (size_t)t * W : nullptr);
    }
    for (int i = cfg.loop_stop; i < (int)layers.size(); ++i)
      run(i, nullptr);

    for (float *&b : x)
      b = device_zeros<float>((size_t)W);
    hrow = device_zeros<float>((size_t)W);
    y = device_zeros<float>((size_t)width16());
    proj = device_zeros<float>((size_t)max_proj);
    mix = device_zeros<float>((size_t)round_up(mix_max, 64));
    mix_gate = device_zeros<float>((size_t)round_up(mix_max, 64));
    act = device_zeros<float>((size_t)round_up(ff_max, 64));
    if (parts) {
      part_acc = device_zeros<float>((size_t)parts);
      part_ml = device_zeros<float>((size_t)parts_ml);
    }
    ld_act = (int)round_up(W, 8);
    ld_mix = (int)round_up(mix_max, 8);
    if (hipStreamSynchronize(stream) != hipSuccess)
      throw std::runtime_error("weight packing failed");
  }

  // ---- the sequence ----------------------------------------------------------------
  int reset() override {
    // caches and rings are only read where positions of this sequence were written
    for (const LirulixRun &r : runs)
      if (r.state) {
        const DeltaShape &s = layers[(size_t)r.layer].delta;
        BH_CHECK_HIP(hipMemsetAsync(r.state, 0, sizeof(float) * (size_t)s.heads * s.dim * s.vdim, stream));
      }
    seq_len = 0;
    return BUDDY_HIP_OK;
  }

  // ---- one token -------------------------------------------------------------------
  int step_span(int pos) const { return key_span(std::min(pos + 1, longest)); }
  std::pair<int, int> step_key(int pos) const override { return {step_span(pos), 0}; }

  int enqueue_step(int pos) override {
    const int span = step_span(pos);
    int rc, cur = 0;
    const float *pending = nullptr; // a sublayer's output that x does not hold yet
    // the residual with what is pending, its norm, a product
    auto norm_gemv = [&](const Bf16Matrix &M, const float *norm, const float *add, float *out, bool gated) {
      RowGemv g;
      g.W = M;
      g.input = kRowResidual;
      g.src = x[cur];
      g.y = pending;
      g.add = add;
      g.norm_w = norm;
      g.eps = cfg.eps;
      if (pending || add) {
        g.x_out = x[1 - cur];
        cur = 1 - cur;
        pending = nullptr;
      }
      g.out = out;
      if (gated) {
        g.gated = true;
        g.W.N *= 2;
      }
      return launch_row_gemv(g, stream);
    };
    auto plain_gemv = [&](const Bf16Matrix &M, const float *src, const DeltaShape *delta = nullptr) {
      RowGemv g;
      if (delta) { // the mixer's norm and gate stand ahead of the product
        g.input = kRowHeadGated;
        g.weight = delta->norm_w;
        g.gate = mix_gate;
        g.head_dim = delta->vdim;
        g.eps = delta->eps;
      }
      g.W = M;
      g.src = src;
      g.src_padded = true;
      g.out = y;
      pending = y;
      return launch_row_gemv(g, stream);
    };
    for (const LirulixRun &r : runs) {
      const LirulixLayer &L = layers[(size_t)r.layer];
      const LayerConfig &c = cfg.layers[(size_t)r.layer];
      if ((rc = norm_gemv(L.in, L.norm1, r.add, proj, false)))
        return rc;
      if (c.kind == kDelta) {
        DeltaRows d;
        d.s = L.delta;
        d.proj = proj;
        d.rows = 1;
        d.pos = state + 1;
        d.ring = r.ring;
        d.state = r.state;
        d.o = mix;
        d.gate = mix_gate;
        rc = launch_delta_scan(d, stream);
      } else {
        HeadStep s;
        s.s = L.head;
        s.proj = proj;
        s.q_at = L.q.at;
        s.k_at = L.k.at;
        s.v_at = L.v.at;
        s.gate_at = L.g.at;
        s.pos = state + 1;
        s.keys = r.keys;
        s.values_t = r.values_t;
        s.part_acc = part_acc;
        s.part_ml = part_ml;
        s.out = mix;
        rc = launch_head_step(s, span, stream);
      }
      if (rc || (rc = plain_gemv(L.o, mix, c.kind == kDelta ? &L.delta : nullptr)))
        return rc;
      if (c.ff && ((rc = norm_gemv(L.gate_up, L.norm2, nullptr, act, true)) || (rc = plain_gemv(L.down, act))))
        return rc;
    }
    RowGemv g;
    g.W = head;
    g.input = kRowResidual;
    g.src = x[cur];
    g.y = pending;
    g.norm_w = final_norm;
    g.eps = cfg.eps;
    g.out = logits;
    g.max_v = group_max_v;
    g.max_i = group_max_i;
    g.valid = cfg.vocab;
    if ((rc = launch_row_gemv(g, stream)))
      return rc;
    return finish(group_max_v, group_max_i, head.groups(), true);
  }

  int finish(const float *cand_v, const int *cand_i, int parts, bool advance) {
    return launch_finish_step_bf16(cand_v, cand_i, parts, state, token_log, embed, 1.0f, embed_norm,
                                   cfg.eps, cfg.width, cfg.vocab, x[0], advance, token_log_cap, stream);
  }
  int prepare_step() override { return finish(nullptr, nullptr, 0, false); }

  // ---- many tokens -----------------------------------------------------------------
  int alloc_block(int rows) override {
    const size_t n = (size_t)rows, T = opt.f32 ? 4 : 2;
    size_t queries = 0, maps = 0, ff = 0, delta = 0;
    for (size_t i = 0; i < layers.size(); ++i) {
      const LirulixLayer &L = layers[i];
      if (cfg.layers[i].kind != kDelta) {
        queries = std::max(queries, (size_t)L.head.map_heads() * L.head.dim32());
        if (L.head.maps > 1 || L.head.gated)
          maps = std::max(maps, (size_t)L.head.map_heads() * L.head.vdim);
      } else {
        delta = std::max({delta, delta_workspace(L.delta, rows), 2 * n * L.delta.heads * L.delta.vdim});
      }
      ff = std::max(ff, (size_t)round_up(cfg.layers[i].ff, 16));
    }
    int rc = block_alloc(&pf_x, 4 * n * cfg.width);
    rc |= block_alloc(&pf_y, 4 * n * width16());
    rc |= block_alloc(&pf_act, T * n * ld_act);
    rc |= block_alloc(&pf_proj, 4 * n * max_proj);
    rc |= block_alloc(&pf_mix, T * n * ld_mix);
    rc |= block_alloc(&pf_queries, T * n * queries);
    rc |= block_alloc(&pf_maps, 4 * n * maps);
    rc |= block_alloc(&pf_delta, 4 * delta);
    rc |= block_alloc(&pf_ff, T * n * ff);
    rc |= block_alloc(&pf_logits, 4 * (size_t)std::min(rows, kLogitRows) * head.N);
    return rc;
  }

  int mixer_rows(const LirulixRun &r, int n, int start) {
    const LirulixLayer &L = layers[(size_t)r.layer];
    if (r.state) {
      DeltaRows d;
      d.s = L.delta;
      d.proj = pf_proj;
      d.ld = L.in.N;
      d.rows = n;
      d.start = start;
      d.ring = r.ring;
      d.state = r.state;
      d.out = pf_mix;
      d.out_ld = ld_mix;
      d.act_f32 = opt.f32;
      if (n >= kScanRows && delta_workspace(L.delta, n))
        return launch_delta_chunks(d, pf_delta, stream);
      const int width = L.delta.heads * L.delta.vdim;
      d.o = pf_delta;
      d.gate = pf_delta + (size_t)n * width;
      const int rc = launch_delta_scan(d, stream);
      return rc ? rc
                : launch_delta_gate(L.delta, d.o, d.gate, width, n, pf_mix, ld_mix, opt.f32, stream);
    }
    HeadRows a;
    a.s = L.head;
    a.proj = pf_proj;
    a.ld = L.in.N;
    a.q_at = L.q.at;
    a.k_at = L.k.at;
    a.v_at = L.v.at;
    a.gate_at = L.g.at;
    a.rows = n;
    a.start = start;
    a.keys = r.keys;
    a.values_t = r.values_t;
    a.queries = pf_queries;
    a.maps_out = pf_maps;
    a.out = pf_mix;
    a.out_ld = ld_mix;
    return launch_head_rows(a, stream);
  }

  int run_block(int n, int start, const int *rows, int n_rows, float *dst) override {
    int rc;
    if ((rc = launch_embed_rows(embed, pf_tokens, n, cfg.width, cfg.vocab, 1.0f, embed_norm, cfg.eps, pf_x,
                                stream)))
      return rc;
    NormRows pend; // residual and norm, with the output x does not hold yet
    pend.x = pf_x;
    pend.plain_y = true;
    pend.eps = cfg.eps;
    pend.width = cfg.width;
    pend.ldy = width16();
    pend.ld_act = ld_act;
    pend.act_f32 = opt.f32;
    auto norm_rows = [&](const float *norm, const float *add) {
      NormRows a = pend;
      a.rows = n;
      a.add = add;
      a.write_x = a.y || a.add;
      a.norm_w = norm;
      a.out_act = pf_act;
      pend.y = nullptr;
      return launch_norm_rows(a, stream);
    };
    auto product = [&](const Bf16Matrix &M, const void *A, int lda) {
      pend.y = pf_y;
      return launch_rows_gemm(gemm(M, A, lda, n, kOutF32, pf_y, M.N), stream);
    };
    for (const LirulixRun &r : runs) {
      const LirulixLayer &L = layers[(size_t)r.layer];
      if ((rc = norm_rows(L.norm1, r.add)) ||
          (rc = launch_rows_gemm(gemm(L.in, pf_act, ld_act, n, kOutF32, pf_proj, L.in.N), stream)) ||
          (rc = mixer_rows(r, n, start)) || (rc = product(L.o, pf_mix, ld_mix)))
        return rc;
      if (!cfg.layers[(size_t)r.layer].ff)
        continue;
      RowsGemm up = gemm(L.gate_up, pf_act, ld_act, n, kOutExpertAct, pf_ff, L.gate_up.N);
      up.act = kActGeluTanh;
      if ((rc = norm_rows(L.norm2, nullptr)) || (rc = launch_rows_gemm(up, stream)) ||
          (rc = product(L.down, pf_ff, L.gate_up.N)))
        return rc;
    }
    if (n_rows == 0)
      return BUDDY_HIP_OK;
    pend.norm_w = final_norm;
    return logit_rows(pend, head, rows, n_rows, hrow, pf_act, pf_logits, dst);
  }
};

Session *create_lirulix(const ModelFolder &folder, const ModelOptions &options) {
  auto s = std::make_unique<LirulixSession>(folder.config(), options);
  if (s->init(s->cfg.vocab, options.max_len, options.stream))
    return nullptr;
  s->load(folder);
  return s.release();
}

const ModelRegistration registered("Lirulix", create_lirulix);

} // namespace
} // namespace bh
