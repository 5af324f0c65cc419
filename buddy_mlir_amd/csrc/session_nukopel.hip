// session_nukopel.hip -- the Nukopel decoder: a list of layers, each with latent
// attention through a sliding window or decaying linear attention as its mixer, a
// short causal convolution in front of the mixer, and a mixture of clamped gated
// experts (or nothing) as its feed-forward; norms with a single gain before and
// after every sublayer.  Sizes, constants and the order of layers come from the
// configuration.
//
// What a sequence keeps: per latent layer a ring of cache rows as long as the
// window (plus the block a prompt goes through the layers in), per linear layer its
// state, and per layer the last rows its convolution reads.  None of it grows with
// the position.
//
// A token: 8 launches in a latent layer, 6 in a linear one, captured into one graph:
//   [residual + norms + convolution -> projections] -> [mixer: 3 or 1] ->
//   [-> output matrix] -> [residual + norms -> router] ->
//   [choice of experts -> gate | up -> activation] -> [down of all of them, summed]
// The residual sum and norms that stand between two matrix products are computed by
// every workgroup of the second one.
#include "elementwise.h"
#include "folder_session.h"
#include "latent_attn.h"
#include "linear_attn.h"

#include <algorithm>
#include <cmath>
#include <cstring>
#include <memory>
#include <new>
#include <stdexcept>
#include <string>
#include <vector>

namespace bh {
namespace {

struct ExpertConfig {
  int ff = 0;
  float limit = 0.f;
};

struct LayerConfig {
  bool latent = false;
  // both mixers
  int heads = 0, dim = 0, vdim = 0;
  // latent attention
  int rot_dim = 0, kv_rank = 0, window = 0;
  double rot_base = 0.0;
  float scale = 0.f;
  // linear attention
  std::vector<double> decay;
  // feed-forward
  bool mlp = false, shared = false;
  int experts = 0, top = 0;
  ExpertConfig expert, shared_expert;
};

struct NukopelConfig {
  int vocab = 0, width = 0, taps = 0;
  float eps = 0.f, embed_scale = 1.f;
  std::vector<LayerConfig> layers;

  explicit NukopelConfig(const Json &j) {
    vocab = positive(j, "vocab");
    width = positive(j, "width");
    taps = positive(j.at("canon"), "taps");
    eps = (float)j.at("norm").at("eps").number();
    embed_scale = (float)j.at("embedding").at("scale").number();
    for (const Json &e : j.at("layers").array()) {
      LayerConfig c;
      const std::string type = e.at("type").string();
      const Json &m = e.at("mixer");
      c.heads = positive(m, "heads");
      c.dim = positive(m, "dim");
      c.vdim = positive(m, "vdim");
      if (type == "latent_attention") {
        c.latent = true;
        c.rot_dim = positive(m, "rot_dim");
        c.kv_rank = positive(m, "kv_rank");
        c.scale = (float)m.at("scale").number();
        c.window = positive(m.at("mask"), "size");
        c.rot_base = m.at("rot").at("base").number();
        if (positive(m.at("rot"), "dims") != c.rot_dim || c.rot_dim % 2)
          throw std::runtime_error("config: the rotation covers the rotated part of a head");
      } else if (type == "lightning") {
        for (const Json &d : m.at("decay").array())
          c.decay.push_back(d.number());
        if ((int)c.decay.size() != c.heads)
          throw std::runtime_error("config: one decay per head");
      } else {
        throw std::runtime_error("config: unknown mixer \"" + type + "\"");
      }
      const Json *f = e.find("mlp");
      if (f && !f->is_null()) {
        if (f->at("kind").string() != "moe")
          throw std::runtime_error("config: unknown feed-forward \"" + f->at("kind").string() + "\"");
        c.mlp = true;
        c.experts = positive(f->at("router"), "experts");
        c.top = positive(f->at("router"), "top");
        c.expert.ff = positive(f->at("expert"), "ff");
        c.expert.limit = (float)f->at("expert").at("limit").number();
        if (c.top > c.experts || c.top > 64 || c.experts > kMaxExperts)
          throw std::runtime_error("config: router of " + std::to_string(c.experts) + " experts, " +
                                   std::to_string(c.top) + " chosen");
        const Json *s = f->find("shared");
        if (s && !s->is_null()) {
          c.shared = true;
          c.shared_expert.ff = positive(*s, "ff");
          c.shared_expert.limit = (float)s->at("limit").number();
        }
      }
      layers.push_back(std::move(c));
    }
    if (layers.empty())
      throw std::runtime_error("config: no layers");
  }
};

struct NukopelLayer {
  float norm1 = 0.f, norm1b = 0.f, norm2 = 0.f, norm2b = 0.f;
  float *conv_w = nullptr, *conv_ring = nullptr; // [taps][width] each
  float *conv_next = nullptr;                    // [2][width]
  Bf16Matrix in;                                 // q | dkv | g, or q | k | v | g
  Part q, k, v, dkv, g;
  int silu_channels = 0;
  float *mix_norm = nullptr; // latent norm, or output norm
  Bf16Matrix o;
  // latent
  LatentShape lat;
  double *turns = nullptr;
  Bf16Matrix uk, uk_t, uv; // head by head
  void *cache = nullptr;
  // linear
  LinearShape lin;
  float *powers = nullptr, *lin_state = nullptr;
  // feed-forward
  Bf16Matrix router;
  ExpertSet experts, shared;
  Bf16Matrix gate_up, down, shared_gate_up, shared_down; // of the first expert
};

struct NukopelSession : FolderSession {
  NukopelConfig cfg;
  std::vector<NukopelLayer> layers;
  uint16_t *embed = nullptr; // [vocab][width] bfloat16
  Bf16Matrix head;
  float final_norm = 1.f;
  int longest_window = 1;

  // one token
  float *x[2] = {nullptr, nullptr}, *hrow = nullptr, *y = nullptr, *proj = nullptr,
        *mix = nullptr, *rlogits = nullptr, *act = nullptr, *chosen_w = nullptr,
        *lat_query = nullptr, *lat_acc = nullptr, *lat_ml = nullptr;
  int *chosen = nullptr;
  int act_stride = 64;

  // a block of a prompt
  int *pf_chosen = nullptr, *pf_counts = nullptr, *pf_lists = nullptr;
  float *pf_x = nullptr, *pf_y = nullptr, *pf_h = nullptr, *pf_proj = nullptr, *pf_lin = nullptr,
        *pf_states = nullptr, *pf_router = nullptr, *pf_weights = nullptr, *pf_experts = nullptr,
        *pf_logits = nullptr;
  void *pf_act = nullptr, *pf_mix = nullptr, *pf_keys = nullptr, *pf_values = nullptr, *pf_queries = nullptr,
       *pf_moe = nullptr, *pf_shared = nullptr;
  int ld_act = 0, ld_mix = 0, max_proj = 0;

  NukopelSession(const Json &config, const ModelOptions &o) : FolderSession(o), cfg(config) {}

  const char *architecture() const override { return "Nukopel"; }
  int width16() const { return (int)round_up(cfg.width, 16); }

  // ---- loading -------------------------------------------------------------------
  void load_mixer(const ModelFolder &f, const std::string &p, const LayerConfig &c, NukopelLayer &L) {
    const int W = cfg.width;
    std::vector<std::pair<std::string, Part *>> parts;
    const int heads_v = c.heads * c.vdim;
    if (c.latent) {
      L.q.n = c.heads * (c.dim + c.rot_dim);
      L.dkv.n = c.kv_rank + c.rot_dim;
      L.g.n = c.heads;
      parts = {{"q", &L.q}, {"dkv", &L.dkv}, {"g", &L.g}};
    } else {
      L.q.n = L.k.n = c.heads * c.dim;
      L.v.n = L.g.n = heads_v;
      parts = {{"q", &L.q}, {"k", &L.k}, {"v", &L.v}, {"g", &L.g}};
    }
    L.in = load_parts(f, p + "mix.", parts, W);
    max_proj = std::max(max_proj, L.in.N);
    L.o = load_matrix(f, p + "mix.o", W, heads_v);
    if (!c.latent) {
      L.silu_channels = L.g.at; // q, k and v, not the gate
      L.mix_norm = device_copy(f.values(p + "mix.norm", {heads_v}));
      L.lin = {c.heads, c.dim, c.vdim};
      std::vector<float> pw;
      for (double d : c.decay)
        for (int j = 0; j <= kLinearChunk; ++j)
          pw.push_back((float)std::pow(d, (double)j));
      L.powers = device_copy(pw);
      L.lin_state = device_zeros<float>((size_t)c.heads * c.dim * c.vdim);
      return;
    }
    L.mix_norm = device_copy(f.values(p + "mix.dkv.norm", {c.kv_rank}));
    L.lat.heads = c.heads;
    L.lat.dim = c.dim;
    L.lat.rot_dim = c.rot_dim;
    L.lat.vdim = c.vdim;
    L.lat.rank = c.kv_rank;
    L.lat.window = c.window;
    L.lat.scale = c.scale;
    L.lat.eps = cfg.eps;
    L.lat.f32 = opt.f32;
    const int64_t rows = std::min<int64_t>(opt.max_len, (int64_t)c.window - 1 + opt.prefill_block);
    L.lat.ring_mask = pow2_at_least(rows) - 1;
    longest_window = std::max(longest_window, std::min(c.window, opt.max_len));
    std::vector<double> turns;
    for (int i = 0; i < c.rot_dim / 2; ++i)
      turns.push_back(std::pow(c.rot_base, -2.0 * i / c.rot_dim) / (2.0 * M_PI));
    L.turns = device_copy(turns);
    // per head, padded to whole channel groups: the key matrix both ways round (a
    // token's query goes through it, a prompt's latents go through it), the value matrix
    const int d16 = L.lat.dim16(), v16 = L.lat.vdim16(), r16 = L.lat.rank16();
    L.uk = matrix((int64_t)c.heads * d16, c.kv_rank);
    L.uk_t = matrix((int64_t)c.heads * r16, c.dim);
    L.uv = matrix((int64_t)c.heads * v16, c.kv_rank);
    Upload uk(f.bf16(p + "mix.uk", {c.heads * c.dim, c.kv_rank}), stream);
    Upload uv(f.bf16(p + "mix.uv", {heads_v, c.kv_rank}), stream);
    for (int h = 0; h < c.heads; ++h) {
      const uint16_t *k = uk.p + (int64_t)h * c.dim * c.kv_rank;
      pack(L.uk, h * d16, k, c.kv_rank, 1, c.dim);
      pack(L.uk_t, h * r16, k, 1, c.kv_rank, c.kv_rank);
      pack(L.uv, h * v16, uv.p + (int64_t)h * c.vdim * c.kv_rank, c.kv_rank, 1, c.vdim);
    }
    L.cache = device_zeros<char>((size_t)(L.lat.ring_mask + 1) * L.lat.row_elems() * (opt.f32 ? 4 : 2));
  }

  ExpertSet load_experts(const ModelFolder &f, const std::vector<std::string> &names,
                         const ExpertConfig &e, Bf16Matrix &gate_up, Bf16Matrix &down) {
    const int64_t W = cfg.width, ff16 = round_up(e.ff, 16), n = (int64_t)names.size();
    gate_up = matrix(n * 2 * ff16, W);
    down = matrix(n * width16(), e.ff);
    for (int64_t i = 0; i < n; ++i) {
      const std::string &p = names[(size_t)i];
      Upload g(f.bf16(p + ".gate", {e.ff, W}), stream), u(f.bf16(p + ".up", {e.ff, W}), stream),
          d(f.bf16(p + ".down", {W, e.ff}), stream);
      pack(gate_up, (int)(i * 2 * ff16), g.p, W, 1, e.ff);
      pack(gate_up, (int)(i * 2 * ff16 + ff16), u.p, W, 1, e.ff);
      pack(down, (int)(i * width16()), d.p, e.ff, 1, W);
    }
    ExpertSet s;
    s.gate_up = gate_up.tiles;
    s.down = down.tiles;
    s.count = (int)n;
    s.ff = e.ff;
    s.limit = e.limit;
    gate_up.N = (int)ff16; // from here on: one matrix of the first expert
    down.N = width16();
    return s;
  }

  void load(const ModelFolder &f) {
    const int W = cfg.width;
    embed = device_bf16(f.bf16("embed", {cfg.vocab, W}));
    head = load_matrix(f, "head", cfg.vocab, W);
    final_norm = f.scalar("final.norm");
    int mix_max = 1, e16 = 16, query = 0, parts = 0, parts_ml = 0, top = 1;
    for (size_t i = 0; i < cfg.layers.size(); ++i) {
      const LayerConfig &c = cfg.layers[i];
      const std::string p = "l" + std::to_string(i) + ".";
      layers.emplace_back();
      NukopelLayer &L = layers.back();
      L.norm1 = f.scalar(p + "norm1");
      L.norm1b = f.scalar(p + "norm1b");
      {
        const std::vector<float> w = f.values(p + "canon1", {W, cfg.taps});
        std::vector<float> t(w.size()); // a row per tap
        for (int ch = 0; ch < W; ++ch)
          for (int j = 0; j < cfg.taps; ++j)
            t[(size_t)j * W + ch] = w[(size_t)ch * cfg.taps + j];
        L.conv_w = device_copy(t);
        L.conv_ring = device_zeros<float>((size_t)cfg.taps * W);
        L.conv_next = device_zeros<float>((size_t)2 * W);
      }
      load_mixer(f, p, c, L);
      mix_max = std::max(mix_max, c.heads * c.vdim);
      if (c.latent) {
        const LatentShape &s = L.lat;
        const int chunks = latent_max_chunks(s);
        query = std::max(query, s.heads16() * s.row_elems());
        parts = std::max(parts, chunks * s.heads16() * s.rank16());
        parts_ml = std::max(parts_ml, chunks * s.heads16() * 2);
      }
      if (!c.mlp)
        continue;
      L.norm2 = f.scalar(p + "norm2");
      L.norm2b = f.scalar(p + "norm2b");
      L.router = load_matrix(f, p + "mlp.router", c.experts, W);
      std::vector<std::string> names;
      for (int e = 0; e < c.experts; ++e)
        names.push_back(p + "mlp.e" + std::to_string(e));
      L.experts = load_experts(f, names, c.expert, L.gate_up, L.down);
      if (c.shared)
        L.shared = load_experts(f, {p + "mlp.shared"}, c.shared_expert, L.shared_gate_up, L.shared_down);
      e16 = std::max(e16, L.router.N);
      top = std::max(top, c.top);
      act_stride = std::max(act_stride, (int)round_up(std::max(c.expert.ff, c.shared_expert.ff), 64));
    }
    for (float *&b : x)
      b = device_zeros<float>((size_t)W);
    hrow = device_zeros<float>((size_t)W);
    y = device_zeros<float>((size_t)width16());
    proj = device_zeros<float>((size_t)max_proj);
    mix = device_zeros<float>((size_t)mix_max);
    rlogits = device_zeros<float>((size_t)e16);
    act = device_zeros<float>((size_t)(top + 1) * act_stride);
    chosen = device_zeros<int>((size_t)top);
    chosen_w = device_zeros<float>((size_t)top);
    if (query) {
      lat_query = device_zeros<float>((size_t)query);
      lat_acc = device_zeros<float>((size_t)parts);
      lat_ml = device_zeros<float>((size_t)parts_ml);
    }
    ld_act = (int)round_up(W, 8);
    ld_mix = (int)round_up(mix_max, 8);
    if (hipStreamSynchronize(stream) != hipSuccess)
      throw std::runtime_error("weight packing failed");
  }

  // ---- the sequence ----------------------------------------------------------------
  int reset() override {
    // caches and rings are only read where positions of this sequence were written
    for (NukopelLayer &L : layers)
      if (L.lin_state)
        BH_CHECK_HIP(hipMemsetAsync(L.lin_state, 0,
                                    sizeof(float) * (size_t)L.lin.heads * L.lin.dim * L.lin.vdim,
                                    stream));
    seq_len = 0;
    return BUDDY_HIP_OK;
  }
  // ---- one token -------------------------------------------------------------------
  int step_span(int pos) const { return key_span(std::min(pos + 1, longest_window)); }
  std::pair<int, int> step_key(int pos) const override { return {step_span(pos), 0}; }

  int enqueue_step(int pos) override {
    const int span = step_span(pos), W = cfg.width;
    int rc, cur = 0;
    const float *pending = nullptr; // a sublayer's output that x does not hold yet
    float pending_gain = 1.f;
    auto norm_gemv = [&](const Bf16Matrix &M, float gain, float *out) {
      RowGemv g;
      g.W = M;
      g.input = kRowNorm;
      g.src = x[cur];
      g.eps = cfg.eps;
      g.y = pending;
      g.out_gain = pending_gain;
      g.gain = gain;
      g.x_out = pending ? x[1 - cur] : nullptr;
      g.out = out;
      return g;
    };
    auto consumed = [&] {
      if (pending)
        cur = 1 - cur;
      pending = nullptr;
    };
    for (size_t i = 0; i < layers.size(); ++i) {
      NukopelLayer &L = layers[i];
      const LayerConfig &c = cfg.layers[i];
      {
        RowGemv g = norm_gemv(L.in, L.norm1, proj);
        g.conv_w = L.conv_w;
        g.conv_ring = L.conv_ring;
        g.conv_next = L.conv_next;
        g.taps = cfg.taps;
        g.pos = state + 1;
        g.silu_channels = L.silu_channels;
        if ((rc = launch_row_gemv(g, stream)))
          return rc;
        consumed();
      }
      RowGemv out;
      out.W = L.o;
      out.src = mix;
      out.out = y;
      if (c.latent) {
        LatentStep s;
        s.s = L.lat;
        s.proj = proj;
        s.dkv_at = L.dkv.at;
        s.gate_at = L.g.at;
        s.norm_w = L.mix_norm;
        s.turns = L.turns;
        s.pos = state + 1;
        s.uk_t = L.uk_t;
        s.uv = L.uv;
        s.cache = L.cache;
        s.query = lat_query;
        s.part_acc = lat_acc;
        s.part_ml = lat_ml;
        s.out = mix;
        if ((rc = launch_latent_step(s, span, stream)))
          return rc;
      } else {
        LinearStep s;
        s.s = L.lin;
        s.q = proj + L.q.at;
        s.k = proj + L.k.at;
        s.v = proj + L.v.at;
        s.powers = L.powers;
        s.state = L.lin_state;
        s.out = mix;
        if ((rc = launch_linear_step(s, stream)))
          return rc;
        out.input = kRowGated;
        out.weight = L.mix_norm;
        out.gate = proj + L.g.at;
        out.eps = cfg.eps;
      }
      if ((rc = launch_row_gemv(out, stream)))
        return rc;
      pending = y;
      pending_gain = L.norm1b;
      if (!c.mlp)
        continue;
      {
        RowGemv g = norm_gemv(L.router, L.norm2, rlogits);
        g.row_out = hrow;
        if ((rc = launch_row_gemv(g, stream)))
          return rc;
        consumed();
      }
      RowMoe m;
      m.h = hrow;
      m.logits = rlogits;
      m.width = W;
      m.top = c.top;
      m.experts = L.experts;
      m.shared = L.shared;
      m.act = act;
      m.act_stride = act_stride;
      m.chosen = chosen;
      m.weights = chosen_w;
      m.out = y;
      if ((rc = launch_row_moe(m, stream)))
        return rc;
      pending = y;
      pending_gain = L.norm2b;
    }
    RowGemv g = norm_gemv(head, final_norm, logits);
    g.x_out = nullptr;
    g.max_v = group_max_v;
    g.max_i = group_max_i;
    g.valid = cfg.vocab;
    if ((rc = launch_row_gemv(g, stream)))
      return rc;
    return launch_finish_step_bf16(group_max_v, group_max_i, head.groups(), state, token_log, embed,
                                   cfg.embed_scale, nullptr, 0.f, W, cfg.vocab, x[0], true, token_log_cap, stream);
  }

  int prepare_step() override {
    return launch_finish_step_bf16(nullptr, nullptr, 0, state, token_log, embed, cfg.embed_scale,
                                   nullptr, 0.f, cfg.width, cfg.vocab, x[0], false, token_log_cap, stream);
  }

  // ---- many tokens -----------------------------------------------------------------
  static int key_cap(const LatentShape &s, int rows) {
    return (int)round_up((int64_t)std::min(s.window - 1, s.ring_mask + 1) + rows, kLatentKeyTile);
  }
  int alloc_block(int rows) override {
    const size_t n = (size_t)rows, T = opt.f32 ? 4 : 2;
    size_t keys = 0, values = 0, queries = 0, lin = 0, states = 0, e16 = 0, top = 0, experts = 0, moe = 0, shared = 0;
    for (size_t i = 0; i < layers.size(); ++i) {
      const NukopelLayer &L = layers[i];
      const LayerConfig &c = cfg.layers[i];
      if (c.latent) {
        const size_t cap = (size_t)key_cap(L.lat, rows);
        keys = std::max(keys, cap * L.uk.N);
        values = std::max(values, cap * L.uv.N);
        queries = std::max(queries, n * c.heads * L.lat.key_elems());
      } else {
        lin = std::max(lin, n * c.heads * c.vdim);
        states = std::max(states, (size_t)linear_chunks(rows) * c.heads * c.dim * c.vdim);
      }
      if (c.mlp) {
        e16 = std::max(e16, (size_t)L.router.N);
        experts = std::max(experts, (size_t)c.experts);
        top = std::max(top, (size_t)c.top);
        moe = std::max(moe, n * c.top * round_up(c.expert.ff, 16));
        shared = std::max(shared, n * round_up(c.shared_expert.ff, 16));
      }
    }
    int rc = block_alloc(&pf_x, 4 * n * cfg.width);
    rc |= block_alloc(&pf_h, 4 * n * cfg.width);
    rc |= block_alloc(&pf_y, 4 * n * width16());
    rc |= block_alloc(&pf_act, T * n * ld_act);
    rc |= block_alloc(&pf_proj, 4 * n * max_proj);
    rc |= block_alloc(&pf_mix, T * n * ld_mix);
    rc |= block_alloc(&pf_keys, T * keys);
    rc |= block_alloc(&pf_values, T * values);
    rc |= block_alloc(&pf_queries, T * queries);
    rc |= block_alloc(&pf_lin, 4 * lin);
    rc |= block_alloc(&pf_states, 4 * states);
    rc |= block_alloc(&pf_router, 4 * n * e16);
    rc |= block_alloc(&pf_chosen, 4 * n * top);
    rc |= block_alloc(&pf_weights, 4 * n * top);
    rc |= block_alloc(&pf_counts, 4 * experts);
    rc |= block_alloc(&pf_lists, 4 * experts * n);
    rc |= block_alloc(&pf_moe, T * moe);
    rc |= block_alloc(&pf_shared, T * shared);
    rc |= block_alloc(&pf_experts, 4 * n * top * width16());
    rc |= block_alloc(&pf_logits, 4 * (size_t)std::min(rows, kLogitRows) * head.N);
    return rc;
  }

  int latent_rows(NukopelLayer &L, int n, int start) {
    int rc;
    LatentRows r;
    r.s = L.lat;
    r.proj = pf_proj;
    r.ld = L.in.N;
    r.dkv_at = L.dkv.at;
    r.gate_at = L.g.at;
    r.rows = n;
    r.start = start;
    r.norm_w = L.mix_norm;
    r.turns = L.turns;
    r.cache = L.cache;
    r.first = latent_first_visible(L.lat, start);
    const int keys = start + n - r.first;
    r.queries = pf_queries;
    r.keys = pf_keys;
    r.values_t = pf_values;
    r.value_ld = (int)round_up(keys, kLatentKeyTile);
    r.out = pf_mix;
    r.out_ld = ld_mix;
    if ((rc = launch_latent_rows(r, stream)))
      return rc;
    const char *latents = static_cast<const char *>(L.cache) + L.lat.rot8() * (opt.f32 ? 4 : 2);
    RowsGemm k = gemm(L.uk, latents, L.lat.row_elems(), keys, kOutAct, pf_keys, L.uk.N);
    k.ring_base = r.first & L.lat.ring_mask;
    k.ring_mask = L.lat.ring_mask;
    if ((rc = launch_rows_gemm(k, stream)))
      return rc;
    RowsGemm v = k;
    v.W = L.uv;
    v.out = kOutActTrans;
    v.C = pf_values;
    v.ldc = r.value_ld;
    if ((rc = launch_rows_gemm(v, stream)))
      return rc;
    return launch_latent_attention(r, stream);
  }

  int linear_rows(NukopelLayer &L, int n) {
    int rc;
    LinearRows r;
    r.s = L.lin;
    r.proj = pf_proj;
    r.ld = L.in.N;
    r.q_at = L.q.at;
    r.k_at = L.k.at;
    r.v_at = L.v.at;
    r.rows = n;
    r.powers = L.powers;
    r.state = L.lin_state;
    r.chunk_states = pf_states;
    r.out = pf_lin;
    if ((rc = launch_linear_rows(r, stream)))
      return rc;
    GatedNormRows g;
    g.x = pf_lin;
    g.w = L.mix_norm;
    g.gate = pf_proj + L.g.at;
    g.ld_gate = L.in.N;
    g.rows = n;
    g.width = L.lin.heads * L.lin.vdim;
    g.eps = cfg.eps;
    g.out = pf_mix;
    g.ld = ld_mix;
    g.act_f32 = opt.f32;
    return launch_gated_norm_rows(g, stream);
  }

  int moe_rows(NukopelLayer &L, const LayerConfig &c, int n) {
    int rc;
    if ((rc = launch_rows_gemm(gemm(L.router, pf_act, ld_act, n, kOutF32, pf_router, L.router.N), stream)))
      return rc;
    RouteRows r;
    r.logits = pf_router;
    r.ld = L.router.N;
    r.rows = n;
    r.experts = c.experts;
    r.top = c.top;
    r.chosen = pf_chosen;
    r.weights = pf_weights;
    r.counts = pf_counts;
    r.lists = pf_lists;
    r.list_cap = n;
    if ((rc = launch_route_rows(r, stream)))
      return rc;
    RowsGemm up = gemm(L.gate_up, pf_act, ld_act, n, kOutExpertAct, pf_moe, L.gate_up.N);
    up.limit = c.expert.limit;
    up.experts = c.experts;
    up.counts = pf_counts;
    up.lists = pf_lists;
    up.list_cap = n;
    up.list_div = c.top; // an assignment reads its token's row ...
    up.list_total = n * c.top;
    up.expert_tiles = (int64_t)2 * L.gate_up.groups() * L.gate_up.ktiles;
    if ((rc = launch_rows_gemm(up, stream)))
      return rc;
    RowsGemm down = gemm(L.down, pf_moe, L.gate_up.N, n, kOutF32, pf_experts, L.down.N);
    down.experts = c.experts;
    down.counts = pf_counts;
    down.lists = pf_lists;
    down.list_cap = n;
    down.list_div = 1; // ... and from there on its own
    down.list_total = n * c.top;
    down.expert_tiles = (int64_t)L.down.groups() * L.down.ktiles;
    if ((rc = launch_rows_gemm(down, stream)))
      return rc;
    if (c.shared) {
      RowsGemm su = gemm(L.shared_gate_up, pf_act, ld_act, n, kOutExpertAct, pf_shared, L.shared_gate_up.N);
      su.limit = c.shared_expert.limit;
      if ((rc = launch_rows_gemm(su, stream)))
        return rc;
      if ((rc = launch_rows_gemm(gemm(L.shared_down, pf_shared, L.shared_gate_up.N, n, kOutF32, pf_y,
                                      L.shared_down.N), stream)))
        return rc;
    }
    return BUDDY_HIP_OK;
  }

  int run_block(int n, int start, const int *rows, int n_rows, float *dst) override {
    int rc;
    if ((rc = launch_embed_rows(embed, pf_tokens, n, cfg.width, cfg.vocab, cfg.embed_scale, nullptr, 0.f, pf_x, stream)))
      return rc;
    NormRows pend; // residual and norm, with the output x does not hold yet
    pend.x = pf_x;
    pend.eps = cfg.eps;
    pend.width = cfg.width;
    pend.ldy = width16();
    pend.lde = width16();
    pend.ld_act = ld_act;
    pend.act_f32 = opt.f32;
    for (size_t i = 0; i < layers.size(); ++i) {
      NukopelLayer &L = layers[i];
      const LayerConfig &c = cfg.layers[i];
      NormRows a = pend;
      a.rows = n;
      a.write_x = a.y || a.expert_out;
      a.gain = L.norm1;
      a.out_f32 = pf_h;
      if ((rc = launch_norm_rows(a, stream)))
        return rc;
      ConvRows cv;
      cv.h = pf_h;
      cv.w = L.conv_w;
      cv.ring = L.conv_ring;
      cv.next = L.conv_next;
      cv.taps = cfg.taps;
      cv.width = cfg.width;
      cv.rows = n;
      cv.start = start;
      cv.out = pf_act;
      cv.ld = ld_act;
      cv.act_f32 = opt.f32;
      if ((rc = launch_conv_rows(cv, stream)))
        return rc;
      RowsGemm in = gemm(L.in, pf_act, ld_act, n, kOutF32, pf_proj, L.in.N);
      in.silu_channels = L.silu_channels;
      if ((rc = launch_rows_gemm(in, stream)))
        return rc;
      if ((rc = c.latent ? latent_rows(L, n, start) : linear_rows(L, n)))
        return rc;
      if ((rc = launch_rows_gemm(gemm(L.o, pf_mix, ld_mix, n, kOutF32, pf_y, L.o.N), stream)))
        return rc;
      pend.y = pf_y;
      pend.expert_out = nullptr;
      pend.top = 0;
      pend.out_gain = L.norm1b;
      if (!c.mlp)
        continue;
      NormRows b = pend;
      b.rows = n;
      b.write_x = true;
      b.gain = L.norm2;
      b.out_act = pf_act;
      if ((rc = launch_norm_rows(b, stream)))
        return rc;
      if ((rc = moe_rows(L, c, n)))
        return rc;
      pend.y = c.shared ? pf_y : nullptr;
      pend.expert_out = pf_experts;
      pend.expert_w = pf_weights;
      pend.top = c.top;
      pend.out_gain = L.norm2b;
    }
    if (n_rows == 0)
      return BUDDY_HIP_OK;
    pend.gain = final_norm;
    return logit_rows(pend, head, rows, n_rows, hrow, pf_act, pf_logits, dst);
  }
};

Session *create_nukopel(const ModelFolder &folder, const ModelOptions &options) {
  auto s = std::make_unique<NukopelSession>(folder.config(), options);
  if (s->init(s->cfg.vocab, options.max_len, options.stream))
    return nullptr;
  s->load(folder);
  return s.release();
}

const ModelRegistration registered("Nukopel", create_nukopel);

} // namespace
} // namespace bh
