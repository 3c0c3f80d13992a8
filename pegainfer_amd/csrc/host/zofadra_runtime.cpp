// C++ host runtime of the Zofadra decoder on MI355X (include/pegainfer_zofadra.h) over StepModel (step_core.h): this file holds what
// is the design's own - its configuration, tensor names, weight layout and the launches of a step.
//
// T = all token rows of the step, prompts' portions and single tokens alike; X = the fp32 streams [T][streams][D].  Between two
// sublayers ONE launch closes the one and opens the other: the output joins the streams, the streams are mixed, the next
// sublayer's weighted sum of them goes through its layer norm into h.
//   start     : X = embed * scale in every stream;  h = ln(sum a X)         one launch
//   latent    : [W_dq ; W_dkv] h;  query latent normed, key latent normed / rotated into the cache (one launch);  W_uq;
//               rotated query parts;  absorb qc = W_uk^T q per head;  attention over the cached latents;  W_uv per head;  W_o
//               (kv_from: no W_dkv, the attention reads the other layer's part of the pages)
//   attention : [W_q ; W_k ; W_v] h;  whole-row norms, k / v into the cache (one launch);  windowed attention with the linear distance
//               bias;  W_o
//   lightning : [W_q ; W_k ; W_v ; W_g] h;  the decayed linear attention over the request's fp32 state;  norm over all heads, weight,
//               sigmoid gate (one launch);  W_o
//   ff        : [W_gate ; W_up] h;  gelu(gate) * up;  W_down
//   logits    : W_head ln(sum X) on the wanted rows, fp32 out
// Cache: page-first [page][layer that caches][latent: slot, rank + rot | k: slot, kv head, dim / v: slot, kv head, vdim].
#include "step_core.h"

#include "pegainfer_zofadra.h"

namespace pzf {

using namespace pstep;

constexpr int kSplitGroups = 512;   // most (tile, kv head, key split) workgroups of an attention launch that cuts its keys
constexpr int kMaxSplits = 16;
constexpr int kFewTiles = 128;      // launches of fewer workgroups deal their keys to several
constexpr int kMaxDeals = 64;
constexpr int kScanMax = 32;        // longest entry whose recurrence runs token by token

enum Kind { kLatent = 1, kAttention = 2, kLightning = 3 };

struct LayerCfg {
  int type = 0, heads = 0, kv = 0, dim = 0, vdim = 0;
  float scale = 1.f;
  int q_rank = 0, kv_rank = 0, rot_dim = 0, kv_from = -1;   // latent attention
  double base = 10000.0;
  int window = 0;                                           // attention
  std::vector<float> decay_pow;                             // lightning: [heads][kPow], g_h^n
  int ff = 0;                                               // 0: no feed-forward
  // columns of the stacked projections
  int o_q = 0, o_k = 0, o_v = 0, o_g = 0, proj_rows = 0, o_up = 0, gu_rows = 0;
  int tiles = -1;
  int64_t c_off = 0, k_off = 0, v_off = 0;                  // parts of a cache page
  int64_t st_off = 0;                                       // part of the request's state region
  int entry() const { return kv_rank + rot_dim; }
};
constexpr int kPow = PEGAINFER_DECAY_CHUNK + 1;

struct Hyper { void *in = nullptr, *out = nullptr, *mix = nullptr; };   // how one sublayer reads and writes the streams
struct LayerW {
  Hyper hc[2];
  void *norm[2] = {nullptr, nullptr};
  void *proj = nullptr, *o = nullptr;
  void *q_norm = nullptr, *k_norm = nullptr;        // attention: whole-row norms; latent: query latent, key latent
  void *uq = nullptr, *uk = nullptr, *uv = nullptr;
  float *inv_freq = nullptr, *slopes = nullptr, *decay_pow = nullptr;
  void *gate_norm = nullptr;                        // lightning
  void *gu = nullptr, *down = nullptr;
};

class Model : public StepModel {
 public:
  Model() {
    const char* e = getenv("PEGAINFER_ZOFADRA_GRAPH");   // 0: decode steps run eagerly
    graphs_on = !(e && e[0] == '0');
  }
  const char* architecture() const override { return "Zofadra"; }
  int layer_runs() const override { return (int)layers.size(); }

  // ------------------------------------------------------------------ configuration
  int parse(const Json& j) override {
    D = geti(&j, "width", 0);
    V = geti(&j, "vocab", 0);
    eps = getf(j.get("norm"), "eps", 1e-5);
    embed_scale = getf(j.get("embedding"), "scale", 1.0);
    residual_mult = getf(&j, "residual_mult", 1.0);
    hyper = j.get("streams") != nullptr;             // without the key: one stream, plain residual sums
    streams = geti(&j, "streams", 1);
    const Json* ls = j.get("layers");
    if (D <= 0 || D > 32768 || V <= 0 || !ls || ls->kind != Json::Arr || ls->arr.empty()) return set_error("config: width / vocab / layers missing");
    if (streams < 1 || streams > 16) return set_error("config: streams outside 1 .. 16");
    for (size_t i = 0; i < ls->arr.size(); ++i) {
      LayerCfg c;
      if (parse_layer(ls->arr[i], (int)i, &c)) return -1;
      layers.push_back(c);
    }
    weights.resize(layers.size());
    for (auto& c : layers) {
      mx_proj = std::max(mx_proj, c.proj_rows);
      mx_mix = std::max(mx_mix, c.heads * c.vdim);
      mx_gu = std::max(mx_gu, c.gu_rows);
      mx_ff = std::max(mx_ff, c.ff);
      if (c.type == kLatent) {
        mx_qr = std::max(mx_qr, c.q_rank);
        mx_q = std::max(mx_q, c.heads * (c.dim + c.rot_dim));
        mx_qf = std::max(mx_qf, c.heads * c.entry());
        mx_of = std::max(mx_of, c.heads * c.kv_rank);
        part_floats = std::max(part_floats, (size_t)kSplitGroups * kFlatRows * (size_t)(c.kv_rank + 2));
      } else if (c.type == kAttention) {
        mx_qf = std::max(mx_qf, c.heads * c.dim);
        part_floats = std::max(part_floats, (size_t)kSplitGroups * kGroupRows * (size_t)(c.vdim + 2));
      } else {
        mx_of = std::max(mx_of, c.heads * c.vdim);
      }
    }
    return 0;
  }
  int parse_layer(const Json& l, int index, LayerCfg* c) {
    const std::string li = std::to_string(index);
    const Json *ty = l.get("type"), *mx = l.get("mixer"), *mlp = l.get("mlp");
    if (!ty || !mx || mx->kind != Json::Obj) return set_error("config: layer " + li + " without type / mixer");
    c->heads = geti(mx, "heads", 0);
    c->dim = geti(mx, "dim", 0);
    c->vdim = geti(mx, "vdim", c->dim);
    if (c->heads <= 0 || c->heads > 65535 || c->dim <= 0 || c->vdim <= 0) return set_error("config: unsupported mixer sizes in layer " + li);
    if (ty->str == "latent_attention") {
      c->type = kLatent;
      c->q_rank = geti(mx, "q_rank", 0);
      c->kv_rank = geti(mx, "kv_rank", 0);
      c->rot_dim = geti(mx, "rot_dim", 0);
      c->scale = getf(mx, "scale", 1.0 / std::sqrt((double)(c->dim + c->rot_dim)));
      const Json* rot = mx->get("rot");
      c->base = rot ? rot->number_or("base", 10000.0) : 10000.0;
      if (c->q_rank <= 0 || c->kv_rank <= 0 || c->kv_rank > 1024 || c->rot_dim < 0 || (c->rot_dim & 1) || geti(rot, "dims", c->rot_dim) != c->rot_dim)
        return set_error("config: unsupported latent attention sizes in layer " + li);
      const Json* from = mx->get("kv_from");
      if (from && from->kind == Json::Num) {
        c->kv_from = (int)from->num;
        if (c->kv_from < 0 || c->kv_from >= index) return set_error("config: kv_from of layer " + li + " names no earlier layer");
        const LayerCfg& s = layers[(size_t)c->kv_from];
        if (s.type != kLatent || s.kv_from >= 0 || s.kv_rank != c->kv_rank || s.rot_dim != c->rot_dim)
          return set_error("config: kv_from of layer " + li + " names a layer without such a latent");
        c->c_off = s.c_off;
      } else {
        c->c_off = add_cache(c->entry());
      }
      c->o_q = 0;                                    // query latent
      c->o_k = pad8(c->q_rank);                      // [key latent | rotated key part], when the layer has its own
      c->proj_rows = pad8(c->kv_from < 0 ? c->o_k + c->entry() : c->q_rank);
      c->tiles = flat_tiles(c->heads);
    } else if (ty->str == "attention") {
      c->type = kAttention;
      c->kv = geti(mx, "kv_heads", c->heads);
      c->scale = getf(mx, "scale", 1.0 / std::sqrt((double)c->dim));
      const Json* mk = mx->get("mask");
      if (mk && mk->kind == Json::Obj) {
        c->window = geti(mk, "size", 0);
        if (c->window < 1) return set_error("config: mask.size must be positive in layer " + li);
      }
      if (c->kv <= 0 || c->heads % c->kv || c->dim > 256 || c->vdim > 256) return set_error("config: unsupported attention sizes in layer " + li);
      c->o_k = c->heads * c->dim;
      c->o_v = c->o_k + c->kv * c->dim;
      c->proj_rows = pad8(c->o_v + c->kv * c->vdim);
      c->k_off = add_cache((int64_t)c->kv * c->dim);
      c->v_off = add_cache((int64_t)c->kv * c->vdim);
      const bool wide = dtype == PEGAINFER_DTYPE_BF16 && pegainfer_paged_attention_rows_ok(c->dim, c->vdim, 0, 0, 0, kPageSize);
      c->tiles = group_tiles(c->heads / c->kv, wide ? c->kv : 0);
    } else if (ty->str == "lightning") {
      c->type = kLightning;
      const Json* g = mx->get("decay");
      if (c->dim > 256 || !g || g->kind != Json::Arr || (int)g->arr.size() != c->heads)
        return set_error("config: layer " + li + " needs dim <= 256 and a decay per head");
      for (auto& d : g->arr)
        for (int n = 0; n < kPow; ++n) c->decay_pow.push_back((float)std::pow(d.num, (double)n));
      c->o_k = pad8(c->heads * c->dim);
      c->o_v = pad8(c->o_k + c->heads * c->dim);
      c->o_g = pad8(c->o_v + c->heads * c->vdim);
      c->proj_rows = pad8(c->o_g + c->heads * c->vdim);
      c->st_off = state_layout.reserve("l" + li + ".state", (int64_t)c->heads * c->dim * c->vdim);
      if (pegainfer_decay_attention_chunked_ok(c->dim, c->vdim)) scan_max = kScanMax;
    } else {
      return set_error("config: layer " + li + " has an unknown mixer type");
    }
    if (mlp && mlp->kind == Json::Obj) {
      const Json* kind = mlp->get("kind");
      if (kind && kind->str != "dense") return set_error("config: unknown feed-forward kind in layer " + li);
      c->ff = geti(mlp, "ff", 0);
      if (c->ff <= 0) return set_error("config: feed-forward without ff in layer " + li);
      c->o_up = pad8(c->ff);
      c->gu_rows = c->o_up + pad8(c->ff);
    }
    return 0;
  }

  // ------------------------------------------------------------------ weights
  TensorList tensor_list() const override {
    TensorList out;
    auto add = [&](const std::string& n, std::vector<int64_t> s) { out.push_back({n, std::move(s)}); };
    add("embed", {V, D});
    for (size_t i = 0; i < layers.size(); ++i) {
      const LayerCfg& c = layers[i];
      const std::string p = "l" + std::to_string(i), m = p + ".mix";
      const int64_t hd = (int64_t)c.heads * c.dim, hv = (int64_t)c.heads * c.vdim;
      for (int q = 1; q <= (c.ff ? 2 : 1); ++q) {
        add(p + ".norm" + std::to_string(q), {D});
        if (!hyper) continue;
        const std::string h = p + ".hc" + std::to_string(q);
        add(h + ".in", {streams});
        add(h + ".out", {streams});
        add(h + ".mix", {streams, streams});
      }
      if (c.type == kLatent) {
        add(m + ".dq", {c.q_rank, D});
        add(m + ".dq.norm", {c.q_rank});
        add(m + ".uq", {(int64_t)c.heads * (c.dim + c.rot_dim), c.q_rank});
        if (c.kv_from < 0) {
          add(m + ".dkv", {c.entry(), D});
          add(m + ".dkv.norm", {c.kv_rank});
        }
        add(m + ".uk", {hd, c.kv_rank});
        add(m + ".uv", {hv, c.kv_rank});
      } else if (c.type == kAttention) {
        add(m + ".q", {hd, D});
        add(m + ".k", {(int64_t)c.kv * c.dim, D});
        add(m + ".v", {(int64_t)c.kv * c.vdim, D});
        add(m + ".q.norm", {hd});
        add(m + ".k.norm", {(int64_t)c.kv * c.dim});
      } else {
        add(m + ".q", {hd, D});
        add(m + ".k", {hd, D});
        add(m + ".v", {hv, D});
        add(m + ".g", {hv, D});
        add(m + ".norm", {hv});
      }
      add(m + ".o", {D, hv});
      if (c.ff) {
        add(p + ".mlp.gate", {c.ff, D});
        add(p + ".mlp.up", {c.ff, D});
        add(p + ".mlp.down", {D, c.ff});
      }
    }
    add("final.norm", {D});
    add("head", {V, D});
    return out;
  }
  float synthetic(const std::string& n, float z, float std) const override {
    if (ends_with(n, ".norm") || ends_with(n, ".norm1") || ends_with(n, ".norm2")) return 1.0f + 0.1f * z;
    if (n.find(".hc") != std::string::npos) return (ends_with(n, ".out") ? 1.0f : 1.0f / (float)streams) + 0.1f * z;
    return std * z;
  }
  int build_weights() override {
    if (up(&embed, "embed", (int64_t)V * D) || up(&head, "head", (int64_t)V * D) || up(&final_norm, "final.norm", D)) return -1;
    const uint16_t one = f2bf(1.0f);
    void* ones = nullptr;
    if (!hyper && upload(&ones, &one, 1)) return -1;
    for (size_t i = 0; i < layers.size(); ++i) {
      const LayerCfg& c = layers[i];
      LayerW& w = weights[i];
      const std::string p = "l" + std::to_string(i), m = p + ".mix";
      const int64_t hd = (int64_t)c.heads * c.dim, hv = (int64_t)c.heads * c.vdim;
      for (int q = 0; q < (c.ff ? 2 : 1); ++q) {
        const std::string qs = std::to_string(q + 1), h = p + ".hc" + qs;
        if (up(&w.norm[q], p + ".norm" + qs, D)) return -1;
        if (!hyper) w.hc[q] = Hyper{ones, ones, ones};
        else if (up(&w.hc[q].in, h + ".in", streams) || up(&w.hc[q].out, h + ".out", streams) || up(&w.hc[q].mix, h + ".mix", (int64_t)streams * streams))
          return -1;
      }
      if (c.type == kLatent) {
        std::vector<Part> parts{{m + ".dq", c.q_rank, 0}};
        if (c.kv_from < 0) parts.push_back({m + ".dkv", c.entry(), c.o_k});
        if (up_stacked(&w.proj, parts, D, c.proj_rows) || up(&w.q_norm, m + ".dq.norm", c.q_rank) ||
            up(&w.uq, m + ".uq", (int64_t)c.heads * (c.dim + c.rot_dim) * c.q_rank) ||
            (c.kv_from < 0 && up(&w.k_norm, m + ".dkv.norm", c.kv_rank)) ||
            up_transposed(&w.uk, m + ".uk", c.heads, c.dim, c.kv_rank) ||     // the absorb GEMM reads it with k contiguous
            up(&w.uv, m + ".uv", hv * c.kv_rank) || upload_f32(&w.inv_freq, rotation_frequencies(c.base, c.rot_dim)))
          return -1;
      } else if (c.type == kAttention) {
        const int64_t kd = (int64_t)c.kv * c.dim;
        std::vector<float> sl((size_t)c.heads);
        for (int h = 0; h < c.heads; ++h) sl[h] = (float)std::pow(2.0, -8.0 * (h + 1) / (double)c.heads);
        if (up_stacked(&w.proj, {{m + ".q", hd, 0}, {m + ".k", kd, c.o_k}, {m + ".v", (int64_t)c.kv * c.vdim, c.o_v}}, D, c.proj_rows) ||
            up(&w.q_norm, m + ".q.norm", hd) || up(&w.k_norm, m + ".k.norm", kd) || upload_f32(&w.slopes, sl))
          return -1;
      } else {
        if (up_stacked(&w.proj, {{m + ".q", hd, 0}, {m + ".k", hd, c.o_k}, {m + ".v", hv, c.o_v}, {m + ".g", hv, c.o_g}}, D, c.proj_rows) ||
            up(&w.gate_norm, m + ".norm", hv) || upload_f32(&w.decay_pow, c.decay_pow))
          return -1;
      }
      if (up(&w.o, m + ".o", (int64_t)D * hv)) return -1;
      if (c.ff && (up_stacked(&w.gu, {{p + ".mlp.gate", c.ff, 0}, {p + ".mlp.up", c.ff, c.o_up}}, D, c.gu_rows) ||
                   up(&w.down, p + ".mlp.down", (int64_t)D * c.ff)))
        return -1;
    }
    return 0;
  }

  // ------------------------------------------------------------------ buffers
  int grow_rows(size_t n) override {
    auto* so = &step_owned;
    return dalloc(&x, n * (size_t)streams * D, so) || dalloc_a(&h, n * D, so) || dalloc_a(&proj, n * (size_t)mx_proj, so) ||
           dalloc_a(&ql, n * (size_t)mx_qr, so) || dalloc_a(&qb, n * (size_t)mx_q, so) || dalloc(&qf, n * (size_t)mx_qf, so) ||
           dalloc(&of, n * (size_t)mx_of, so) || dalloc_a(&mix, n * (size_t)mx_mix, so) || dalloc_a(&y, n * D, so) ||
           dalloc_a(&gu, n * (size_t)mx_gu, so) || dalloc_a(&act, n * (size_t)mx_ff, so) || dalloc(&part, part_floats, so) ? -1 : 0;
  }
  int grow_want(size_t n) override { return dalloc_a(&hw, n * D, &want_owned); }
  int before_step(const StepCtx& c) override {       // chunks of long entries: never part of a captured step
    size_t need = 0;
    if (c.chunks.n_long > 0)
      for (auto& l : layers)
        if (l.type == kLightning) need = std::max(need, (size_t)pegainfer_decay_attention_workspace(c.chunks.n_chunks, l.heads, l.dim, l.vdim));
    if (need <= chunk_cap) return 0;
    PSTEP_HIP(hipStreamSynchronize(stream));
    if (chunk_ws) (void)hipFree(chunk_ws);
    chunk_ws = nullptr;
    chunk_cap = 0;
    PSTEP_HIP(hipMalloc(reinterpret_cast<void**>(&chunk_ws), need * 4));
    chunk_cap = need;
    return 0;
  }
  ~Model() override {
    if (stream) (void)hipStreamSynchronize(stream);
    if (chunk_ws) (void)hipFree(chunk_ws);
  }

  // ------------------------------------------------------------------ one step
  // the end of sublayer q of a layer and the start of the next: y joins the streams, `next` reads them through its norm
  int join(const StepCtx& s, const Hyper& hc, const Hyper* next, const void* next_norm, float* sum_out) {
    pegainfer_stream_mix_desc d = stream_desc(s.T);
    d.x_in = x; d.x_out = x;
    d.y = y; d.y_row_stride = D; d.mix = hc.mix; d.out_w = hc.out; d.mult = residual_mult;
    d.sum_out = sum_out;
    if (next) { d.read_w = next->in; d.gain = next_norm; d.n_out = h; }
    PSTEP_K(pegainfer_stream_mix(&d, S()));
    return 0;
  }
  pegainfer_stream_mix_desc stream_desc(int rows) const {
    pegainfer_stream_mix_desc d{};
    d.eps = eps; d.norm_kind = PEGAINFER_NORM_LAYER;
    d.streams = streams; d.d = D; d.rows = rows; d.dtype = dtype;
    return d;
  }
  int latent_layer(const StepCtx& s, const LayerCfg& c, const LayerW& w) {
    const int H = c.heads, E = c.entry(), qrow = c.dim + c.rot_dim;
    if (linear(w.proj, h, proj, c.proj_rows, s.T, D)) return -1;
    pegainfer_latent_prep_desc p{};
    p.eps = eps; p.inv_freq = w.inv_freq; p.rot_dims = c.rot_dim; p.rot_layout = PEGAINFER_ROT_PAIRS;
    p.positions = s.pos; p.token_req = s.entry; p.page_indptr = s.page_indptr; p.page_ids = s.pages;
    p.cache = cache; p.page_stride = page_stride; p.layer_off = c.c_off; p.page_size = kPageSize;
    p.heads = H; p.nope = c.dim; p.rot = c.rot_dim; p.rank = c.kv_rank; p.n_tokens = s.T; p.dtype = dtype;
    pegainfer_latent_prep_desc p2 = p;
    p.ql = proj; p.ql_stride = c.proj_rows; p.ql_norm_w = w.q_norm; p.ql_out = ql; p.q_rank = c.q_rank;
    if (c.kv_from < 0) { p.dkv = at(proj, (size_t)c.o_k); p.dkv_stride = c.proj_rows; p.c_norm_w = w.k_norm; }
    PSTEP_K(pegainfer_latent_prep_form(&p, S()));
    if (linear(w.uq, ql, qb, H * qrow, s.T, c.q_rank)) return -1;
    p2.q = qb; p2.q_stride = (int64_t)H * qrow; p2.qc = qf;
    PSTEP_K(pegainfer_latent_prep_form(&p2, S()));
    pegainfer_gemm_desc g{};            // absorb: qc[t, h, :rank] = W_uk_h^T q[t, h, :dim]
    g.x = qb; g.w = w.uk; g.y = qf;
    g.x_dtype = g.w_dtype = dtype; g.y_dtype = PEGAINFER_DTYPE_F32;
    g.m = c.kv_rank; g.k = c.dim; g.rows = s.T; g.groups = H;
    g.x_row_stride = (int64_t)H * qrow; g.x_group_stride = qrow;
    g.w_m_stride = c.dim; g.w_k_stride = 1; g.w_group_stride = (int64_t)c.dim * c.kv_rank;
    g.y_row_stride = (int64_t)H * E; g.y_group_stride = E;
    g.plain = plain_kernels;
    PSTEP_K(pegainfer_gemm_strided(&g, S()));
    const TileTable& t = s.flat_tiles[(size_t)c.tiles];
    const bool tiled = !plain_kernels && pegainfer_latent_attention_tiled_ok(c.kv_rank, c.rot_dim, page_stride, c.c_off, dtype);
    const int deals = t.count >= kFewTiles ? 1 : std::max(1, std::min(kMaxDeals, kSplitGroups / t.count));
    PSTEP_K(pegainfer_latent_attention_dealt(qf, of, cache, page_stride, c.c_off, kPageSize, s.pos, s.entry, s.page_indptr, s.pages, H,
                                             c.kv_rank, c.rot_dim, c.scale, s.T, deals, part, tiled ? t.col(0) : nullptr,
                                             tiled ? t.col(1) : nullptr, t.count, dtype, S()));
    pegainfer_gemm_desc v{};            // values: mix[t, h] = W_uv_h o_lat[t, h]
    v.x = of; v.w = w.uv; v.y = mix;
    v.x_dtype = PEGAINFER_DTYPE_F32; v.w_dtype = v.y_dtype = dtype;
    v.m = c.vdim; v.k = c.kv_rank; v.rows = s.T; v.groups = H;
    v.x_row_stride = (int64_t)H * c.kv_rank; v.x_group_stride = c.kv_rank;
    v.w_m_stride = c.kv_rank; v.w_k_stride = 1; v.w_group_stride = (int64_t)c.vdim * c.kv_rank;
    v.y_row_stride = (int64_t)H * c.vdim; v.y_group_stride = c.vdim;
    v.plain = plain_kernels;
    PSTEP_K(pegainfer_gemm_strided(&v, S()));
    return 0;
  }
  int attention_layer(const StepCtx& s, const LayerCfg& c, const LayerW& w) {
    if (linear(w.proj, h, proj, c.proj_rows, s.T, D)) return -1;
    PSTEP_K(pegainfer_qk_prep_paged_form(proj, dtype, c.proj_rows, c.o_q, c.o_k, c.o_v, c.heads, c.kv, c.dim, c.vdim, w.q_norm, w.k_norm,
                                         PEGAINFER_QKNORM_ALL_WEIGHT, eps, nullptr, nullptr, nullptr, 0.f, 0, nullptr, 0, PEGAINFER_ROT_PAIRS,
                                         s.pos, s.entry, s.page_indptr, s.pages, cache, page_stride, c.k_off, c.v_off, kPageSize, qf, nullptr,
                                         s.T, dtype, S()));
    const TileTable& t = s.group_tiles[(size_t)c.tiles];
    const int wgs = t.count * c.kv;     // depends on the step's shape only, never on the contexts' lengths
    pegainfer_attn_options o{};
    o.window = c.window;
    o.dist_slope = w.slopes;
    o.tile_rows = t.rows;
    o.n_split = wgs >= kFewTiles || t.rows > kGroupRows ? 1 : std::max(1, std::min(kMaxSplits, kSplitGroups / wgs));
    o.workspace = part;
    o.plain = plain_kernels ? 1 : 0;
    PSTEP_K(pegainfer_paged_attention_opt(qf, cache, page_stride, c.k_off, c.v_off, kPageSize, s.pos, s.entry, s.page_indptr, s.pages, c.heads,
                                          c.kv, c.dim, c.vdim, c.scale, 1.0f, t.col(0), t.col(1), t.col(2), t.col(3), t.count, mix,
                                          (int64_t)c.heads * c.vdim, &o, dtype, S()));
    return 0;
  }
  int lightning_layer(const StepCtx& s, const LayerCfg& c, const LayerW& w) {
    if (linear(w.proj, h, proj, c.proj_rows, s.T, D)) return -1;
    pegainfer_decay_attention_desc d{};
    d.proj = proj; d.proj_stride = c.proj_rows; d.q_off = c.o_q; d.k_off = c.o_k; d.v_off = c.o_v; d.silu = 1;
    d.decay_pow = w.decay_pow; d.pow_n = kPow;
    d.state = state + c.st_off; d.slot_stride = state_layout.floats_per_slot(); d.o = of;
    d.heads = c.heads; d.dim = c.dim; d.vdim = c.vdim;
    d.entry_row0 = s.row0; d.entry_slot = s.slot; d.n_entries = s.n;
    d.dtype = dtype;
    if (s.chunks.n_long > 0 && pegainfer_decay_attention_chunked_ok(c.dim, c.vdim)) {
      d.scan_max = scan_max;
      d.chunk_row0 = s.chunks.row0; d.chunk_rows = s.chunks.rows; d.n_chunks = s.chunks.n_chunks;
      d.long_chunk0 = s.chunks.long_chunk0; d.long_slot = s.chunks.long_slot; d.n_long = s.chunks.n_long;
      d.workspace = chunk_ws;
    }
    PSTEP_K(pegainfer_decay_attention(&d, S()));
    const int hv = c.heads * c.vdim;    // one norm over all heads: one "head" as wide as the row
    PSTEP_K(pegainfer_head_rms_gate(of, w.gate_norm, 0, at(proj, (size_t)c.o_g), c.proj_rows, 1, 1.0f, eps, mix, hv, 1, hv, s.T, dtype, S()));
    return 0;
  }
  int run_step(const StepCtx& s) override {
    {
      pegainfer_stream_mix_desc d = stream_desc(s.T);
      d.embed = embed; d.token_ids = s.tokens; d.embed_scale = embed_scale;
      d.x_out = x; d.read_w = weights[0].hc[0].in; d.gain = weights[0].norm[0]; d.n_out = h;
      PSTEP_K(pegainfer_stream_mix(&d, S()));
    }
    for (size_t i = 0; i < layers.size(); ++i) {
      const LayerCfg& c = layers[i];
      const LayerW& w = weights[i];
      const LayerW* nx = i + 1 < layers.size() ? &weights[i + 1] : nullptr;
      float* tap = tap_on ? tap_at((int)i) : nullptr;
      if (c.type == kLatent ? latent_layer(s, c, w) : c.type == kAttention ? attention_layer(s, c, w) : lightning_layer(s, c, w)) return -1;
      if (linear(w.o, mix, y, D, s.T, c.heads * c.vdim)) return -1;
      if (c.ff) {
        if (join(s, w.hc[0], &w.hc[1], w.norm[1], nullptr)) return -1;
        if (linear(w.gu, h, gu, c.gu_rows, s.T, D)) return -1;
        PSTEP_K(pegainfer_glu_rows(gu, at(gu, (size_t)c.o_up), c.gu_rows, act, c.ff, c.ff, s.T, PEGAINFER_ACT_GELU_TANH, dtype, S()));
        if (linear(w.down, act, y, D, s.T, c.ff)) return -1;
      }
      if (join(s, w.hc[c.ff ? 1 : 0], nx ? &nx->hc[0] : nullptr, nx ? nx->norm[0] : nullptr, tap)) return -1;
    }
    if (s.W > 0) {
      pegainfer_stream_mix_desc d = stream_desc(s.W);
      d.x_in = x; d.row_index = s.want; d.gain = final_norm; d.n_out = hw;
      PSTEP_K(pegainfer_stream_mix(&d, S()));
      if (linear_strided(head, hw, dtype, D, logits32, PEGAINFER_DTYPE_F32, V, s.W, D)) return -1;
    }
    return 0;
  }

 private:
  int streams = 1;
  bool hyper = false;
  float eps = 1e-5f, embed_scale = 1.f, residual_mult = 1.f;
  std::vector<LayerCfg> layers;
  std::vector<LayerW> weights;
  void *embed = nullptr, *head = nullptr, *final_norm = nullptr;
  int mx_proj = 0, mx_mix = 0, mx_gu = 0, mx_ff = 0, mx_qr = 0, mx_q = 0, mx_qf = 0, mx_of = 0;
  size_t part_floats = 0;
  float *x = nullptr, *qf = nullptr, *of = nullptr, *part = nullptr, *chunk_ws = nullptr;
  size_t chunk_cap = 0;
  void *h = nullptr, *proj = nullptr, *ql = nullptr, *qb = nullptr, *mix = nullptr, *y = nullptr, *gu = nullptr, *act = nullptr, *hw = nullptr;
};

}  // namespace pzf

using pzf::Model;
PEGAINFER_STEP_ENTRIES(pegainfer_zofadra, pzf::Model)
