// C++ host runtime of the Sopanex decoder on MI355X (include/pegainfer_sopanex.h) over StepModel (step_core.h): this file holds what
// is the design's own - its configuration, tensor names, weight layout and the launches of a step.
//
// T = all token rows of the step, prompts' portions and single tokens alike; x = the fp32 stream [T][D].  Between two sublayers ONE
// launch closes the one (its output is normed and joins the stream) and opens the other (the next norm leaves h).
//   start    : x = embed * scale + bigram row of (previous token, token);  h = norm(x)                     one launch
//   parallel : [W_q ; W_k ; W_g | W_q ; W_k ; W_v ; W_g ; W_a1] h of both mixers in ONE GEMM;
//              left : rotation and cache write (one launch), softmax attention with a sink and a gate per head, times left_scale;
//              right: W_a2 (W_a1 h) in fp32, the recurrence over the request's fp32 state, norm * gate * right_scale (one launch);
//              both leave their heads side by side in one row, and ONE GEMM over [W_o | W_o] gives the sum
//   ff       : [router ; shared gate] h in fp32, selection and sort by expert, the experts' two GEMMs (gelu in the first one's
//              epilogue), the shared expert; the weighted sum, with the input's own row for identity experts, is made in the launch that
//              norms it, adds it to the stream and norms for the next layer
//   logits   : W_head norm(x) on the wanted rows, fp32 out
// Cache: page-first [page][layer][k: slot, kv head, rotated values | v: slot, kv head, dim] - the values are the unrotated keys, so the
// part of a key that the rotation does not reach is read from them.
#include "step_core.h"

#include "pegainfer_sopanex.h"

namespace psx {

using namespace pstep;

constexpr int kSplitGroups = 512;   // most (tile, kv head, key split) workgroups of an attention launch that cuts its keys
constexpr int kMaxSplits = 16;
constexpr int kFewTiles = 128;      // launches of fewer workgroups deal their keys to several
constexpr int kFusedRows = 8;       // steps of at most so many rows make the decay inputs inside the scan
constexpr int kScanMax = 32;        // longest entry whose recurrence runs token by token
constexpr int kSyntheticRank = 32;  // of the decays' two-step projection when no tensor tells it
constexpr float kGainOffset = 1.0f; // the stream's norm weights are kept as offsets from one

struct AttnCfg {
  int heads = 0, kv = 0, dim = 0, rot_dims = 0;
  float scale = 1.f, amp = 1.f;
  std::vector<float> freq;
  int o_q = 0, o_k = 0, o_g = 0;    // columns of the stacked projection
  int tail() const { return dim - rot_dims; }
};
struct MemCfg {
  int heads = 0, dim = 0, vdim = 0, rank = 0;
  float tau = 1.f;
  int o_q = 0, o_k = 0, o_v = 0, o_g = 0, o_a = 0;
  int64_t st_off = 0;               // part of the request's state region
};
struct MoeCfg { int ff = 0, experts = 0, identity = 0, top = 0, shared_ff = 0; float scale = 1.f; };   // ff 0: no feed-forward
struct LayerCfg {
  AttnCfg left;
  MemCfg right;
  float left_scale = 1.f, right_scale = 1.f;
  MoeCfg moe;
  int proj_rows = 0, mix_right = 0, mix_cols = 0;
  int tiles = -1;
  int64_t k_off = 0, v_off = 0;     // parts of a cache page
};
struct LayerW {
  void *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr;
  void *proj = nullptr, *o = nullptr, *sink = nullptr, *a2 = nullptr, *a2_bias = nullptr, *mem_norm = nullptr;
  float* inv_freq = nullptr;
  void *router = nullptr, *correction = nullptr, *up_e = nullptr, *down_e = nullptr, *up_s = nullptr, *down_s = nullptr;
};

class Model : public StepModel {
 public:
  Model() {
    const char* e = getenv("PEGAINFER_SOPANEX_GRAPH");   // 0: decode steps run eagerly
    graphs_on = !(e && e[0] == '0');
  }
  const char* architecture() const override { return "Sopanex"; }
  int layer_runs() const override { return (int)layers.size(); }

  // ------------------------------------------------------------------ configuration
  int parse(const Json& j) override {
    D = geti(&j, "width", 0);
    V = geti(&j, "vocab", 0);
    eps = getf(j.get("norm"), "eps", 1e-5);
    const Json* em = j.get("embedding");
    embed_scale = getf(em, "scale", 1.0);
    const Json* bg = em ? em->get("bigram") : nullptr;
    if (bg && bg->kind == Json::Obj) {
      buckets = (int64_t)bg->number_or("buckets", 0);
      mul_prev = (int64_t)bg->number_or("mul_prev", 0);
      mul_cur = (int64_t)bg->number_or("mul_cur", 0);
      if (buckets < 1 || mul_prev < 0 || mul_cur < 0 || mul_prev > (1LL << 31) || mul_cur > (1LL << 31))
        return set_error("config: embedding.bigram needs positive buckets and multipliers of at most 2^31");
    }
    const Json* ls = j.get("layers");
    if (D <= 0 || D > 32768 || V <= 0 || !ls || ls->kind != Json::Arr || ls->arr.empty()) return set_error("config: width / vocab / layers missing");
    for (size_t i = 0; i < ls->arr.size(); ++i) {
      LayerCfg c;
      if (parse_layer(ls->arr[i], (int)i, &c)) return -1;
      layers.push_back(c);
    }
    weights.resize(layers.size());
    return 0;
  }
  int parse_layer(const Json& l, int index, LayerCfg* c) {
    const std::string li = std::to_string(index);
    const Json *ty = l.get("type"), *mx = l.get("mixer"), *mlp = l.get("mlp");
    if (!ty || !mx || mx->kind != Json::Obj) return set_error("config: layer " + li + " without type / mixer");
    if (ty->str != "parallel") return set_error("config: layer " + li + " has an unknown mixer type");
    const Json *lf = mx->get("left"), *rt = mx->get("right");
    if (!lf || !rt || lf->kind != Json::Obj || rt->kind != Json::Obj) return set_error("config: layer " + li + " needs mixer.left and mixer.right");
    c->left_scale = getf(mx, "left_scale", 1.0);
    c->right_scale = getf(mx, "right_scale", 1.0);
    AttnCfg& a = c->left;
    a.heads = geti(lf, "heads", 0);
    a.kv = geti(lf, "kv_heads", a.heads);
    a.dim = geti(lf, "dim", 0);
    a.scale = getf(lf, "scale", 1.0 / std::sqrt((double)std::max(1, a.dim)));
    const Json* rot = lf->get("rot");
    if (rot && rot->kind == Json::Obj) {
      a.rot_dims = geti(rot, "dims", a.dim);
      const double base = rot->number_or("base", 10000.0);
      const RampScaling ramp = parse_ramp(rot->get("scaling"));
      if (a.rot_dims < 0 || a.rot_dims > a.dim || (a.rot_dims & 1) || base <= 1.0 || (ramp.on && !ramp.ok()))
        return set_error("config: unsupported rotation in layer " + li);
      a.freq = rotation_frequencies(base, a.rot_dims, ramp);
      a.amp = ramp.amplitude();
    }
    if (a.heads <= 0 || a.kv <= 0 || a.heads % a.kv || a.dim <= 0 || a.dim > 256 || geti(lf, "vdim", a.dim) != a.dim)
      return set_error("config: unsupported attention sizes in layer " + li + " (values are the keys: vdim is dim)");
    MemCfg& m = c->right;
    m.heads = geti(rt, "heads", 0);
    m.dim = geti(rt, "dim", 0);
    m.vdim = geti(rt, "vdim", m.dim);
    m.tau = getf(rt, "tau", 1.0);
    m.rank = geti(rt, "rank", 0);
    if (m.heads <= 0 || m.heads > 65535 || m.dim <= 0 || m.dim > 256 || m.vdim <= 0 || !(m.tau > 0.f) || m.rank < 0)
      return set_error("config: unsupported linear attention sizes in layer " + li);
    c->mix_right = pad8(a.heads * a.dim);
    c->mix_cols = pad8(c->mix_right + m.heads * m.vdim);
    c->k_off = add_cache((int64_t)a.kv * a.rot_dims);
    c->v_off = add_cache((int64_t)a.kv * a.dim);
    const bool wide = dtype == PEGAINFER_DTYPE_BF16 && pegainfer_paged_attention_rows_ok(a.dim, a.dim, a.tail(), 0, 0, kPageSize);
    c->tiles = group_tiles(a.heads / a.kv, wide ? a.kv : 0);
    m.st_off = state_layout.reserve("l" + li + ".memory", (int64_t)m.heads * m.dim * m.vdim);
    if (pegainfer_gated_linear_chunked_ok(m.dim, m.vdim)) scan_max = kScanMax;
    if (mlp && mlp->kind == Json::Obj) {
      const Json *kind = mlp->get("kind"), *r = mlp->get("router"), *sh = mlp->get("shared");
      if (kind && kind->str != "moe") return set_error("config: unknown feed-forward kind in layer " + li);
      MoeCfg& f = c->moe;
      f.ff = geti(mlp->get("expert"), "ff", 0);
      f.experts = geti(r, "experts", 0);
      f.identity = geti(r, "identity", 0);
      f.top = geti(r, "top", 0);
      f.scale = getf(r, "scale", 1.0);
      if (f.ff <= 0 || f.experts <= 0 || f.identity < 0 || f.experts + f.identity > 1024 || f.top <= 0 || f.top > f.experts + f.identity)
        return set_error("config: unsupported router in layer " + li);
      if (sh && sh->kind == Json::Obj) {
        f.shared_ff = geti(sh, "ff", 0);
        if (f.shared_ff <= 0) return set_error("config: shared expert without ff in layer " + li);
      }
    }
    return 0;
  }
  // the rank of the decays' two-step projection is a tensor's shape; with it the stacked projection is laid out
  int resolve_sizes(const std::function<int64_t(const std::string&)>& numel_of) override {
    for (size_t i = 0; i < layers.size(); ++i) {
      LayerCfg& c = layers[i];
      AttnCfg& a = c.left;
      MemCfg& m = c.right;
      const int64_t n = numel_of("l" + std::to_string(i) + ".mix.right.a1");
      if (n > 0 && n % D == 0) m.rank = (int)(n / D);
      if (m.rank <= 0) m.rank = kSyntheticRank;
      a.o_k = a.heads * a.dim;
      a.o_g = pad8(a.o_k + a.kv * a.dim);
      m.o_q = pad8(a.o_g + a.heads);
      m.o_k = pad8(m.o_q + m.heads * m.dim);
      m.o_v = pad8(m.o_k + m.heads * m.dim);
      m.o_g = pad8(m.o_v + m.heads * m.vdim);
      m.o_a = pad8(m.o_g + m.heads * m.vdim);
      c.proj_rows = m.o_a + pad8(m.rank);
    }
    mx_proj = mx_mix = mx_q = mx_o = mx_z = mx_route = mx_top = mx_pair_ff = mx_shared = mx_experts = 0;
    part_floats = 0;
    for (auto& c : layers) {
      mx_proj = std::max(mx_proj, c.proj_rows);
      mx_mix = std::max(mx_mix, c.mix_cols);
      mx_q = std::max(mx_q, c.left.heads * c.left.dim);
      mx_o = std::max(mx_o, c.right.heads * c.right.vdim);
      mx_z = std::max(mx_z, c.right.heads * c.right.dim);
      mx_route = std::max(mx_route, c.moe.experts + c.moe.identity + 1);
      mx_top = std::max(mx_top, c.moe.top);
      mx_pair_ff = std::max(mx_pair_ff, c.moe.top * c.moe.ff);
      mx_shared = std::max(mx_shared, c.moe.shared_ff);
      mx_experts = std::max(mx_experts, c.moe.experts);
      part_floats = std::max(part_floats, (size_t)kSplitGroups * kGroupRows * (size_t)(c.left.dim + 2));
    }
    return 0;
  }

  // ------------------------------------------------------------------ weights
  TensorList tensor_list() const override {
    TensorList out;
    auto add = [&](const std::string& n, std::vector<int64_t> s) { out.push_back({n, std::move(s)}); };
    add("embed", {V, D});
    if (buckets > 0) add("bigram", {buckets + 1, D});
    for (size_t i = 0; i < layers.size(); ++i) {
      const LayerCfg& c = layers[i];
      const AttnCfg& a = c.left;
      const MemCfg& m = c.right;
      const MoeCfg& f = c.moe;
      const std::string p = "l" + std::to_string(i), l = p + ".mix.left", r = p + ".mix.right", e = p + ".mlp";
      const int64_t hd = (int64_t)a.heads * a.dim, rd = (int64_t)m.heads * m.dim, rv = (int64_t)m.heads * m.vdim;
      for (const char* n : {".norm1", ".norm1b"}) add(p + n, {D});
      add(l + ".q", {hd, D});
      add(l + ".k", {(int64_t)a.kv * a.dim, D});
      add(l + ".sink", {a.heads});
      add(l + ".g", {a.heads, D});
      add(l + ".o", {D, hd});
      add(r + ".q", {rd, D});
      add(r + ".k", {rd, D});
      add(r + ".v", {rv, D});
      add(r + ".g", {rv, D});
      add(r + ".o", {D, rv});
      add(r + ".norm", {m.vdim});
      add(r + ".a1", {m.rank, D});
      add(r + ".a2", {rd, m.rank});
      add(r + ".a2.b", {rd});
      if (!f.ff) continue;
      for (const char* n : {".norm2", ".norm2b"}) add(p + n, {D});
      for (int k = 0; k < f.experts; ++k) {
        const std::string ek = e + ".e" + std::to_string(k);
        add(ek + ".up", {f.ff, D});
        add(ek + ".down", {D, f.ff});
      }
      add(e + ".router", {f.experts + f.identity, D});
      add(e + ".correction", {f.experts + f.identity});
      if (f.shared_ff) {
        add(e + ".shared.up", {f.shared_ff, D});
        add(e + ".shared.down", {D, f.shared_ff});
        add(e + ".shared.sg", {1, D});
      }
    }
    add("final.norm", {D});
    add("head", {V, D});
    return out;
  }
  float synthetic(const std::string& n, float z, float std) const override {
    if (ends_with(n, ".right.norm")) return 1.0f + 0.1f * z;
    if (n.find("norm") != std::string::npos) return 0.1f * z;
    if (ends_with(n, ".sink")) return 0.5f * z;
    if (ends_with(n, ".a2.b")) return 2.0f + 0.5f * z;
    if (ends_with(n, ".a2")) return 0.2f * z;
    if (ends_with(n, ".correction")) return 0.01f * z;
    return std * z;
  }
  int build_weights() override {
    if (up(&embed, "embed", (int64_t)V * D) || up(&head, "head", (int64_t)V * D) || up(&final_norm, "final.norm", D) ||
        (buckets > 0 && up(&bigram, "bigram", (buckets + 1) * D)))
      return -1;
    for (size_t i = 0; i < layers.size(); ++i) {
      const LayerCfg& c = layers[i];
      const AttnCfg& a = c.left;
      const MemCfg& m = c.right;
      const MoeCfg& f = c.moe;
      LayerW& w = weights[i];
      const std::string p = "l" + std::to_string(i), l = p + ".mix.left", r = p + ".mix.right", e = p + ".mlp";
      const int64_t hd = (int64_t)a.heads * a.dim, rd = (int64_t)m.heads * m.dim, rv = (int64_t)m.heads * m.vdim;
      if (up(&w.norm1, p + ".norm1", D) || up(&w.norm1b, p + ".norm1b", D) || up(&w.sink, l + ".sink", a.heads) ||
          up_stacked(&w.proj, {{l + ".q", hd, a.o_q}, {l + ".k", (int64_t)a.kv * a.dim, a.o_k}, {l + ".g", a.heads, a.o_g}, {r + ".q", rd, m.o_q},
                               {r + ".k", rd, m.o_k}, {r + ".v", rv, m.o_v}, {r + ".g", rv, m.o_g}, {r + ".a1", m.rank, m.o_a}},
                     D, c.proj_rows) ||
          up_beside(&w.o, {{l + ".o", hd, 0}, {r + ".o", rv, c.mix_right}}, D, c.mix_cols) ||
          up_beside(&w.a2, {{r + ".a2", m.rank, 0}}, rd, pad8(m.rank)) || up(&w.a2_bias, r + ".a2.b", rd) ||
          up(&w.mem_norm, r + ".norm", m.vdim) || upload_f32(&w.inv_freq, a.freq))
        return -1;
      if (!f.ff) continue;
      const int all = f.experts + f.identity;
      std::vector<Part> ups, downs, router{{e + ".router", all, 0}};
      for (int k = 0; k < f.experts; ++k) {
        const std::string ek = e + ".e" + std::to_string(k);
        ups.push_back({ek + ".up", f.ff, (int64_t)k * f.ff});
        downs.push_back({ek + ".down", D, (int64_t)k * D});
      }
      // the router's rows and, after them, the shared expert's gate row: one GEMM gives all of a token's logits
      if (f.shared_ff) router.push_back({e + ".shared.sg", 1, all});
      if (up(&w.norm2, p + ".norm2", D) || up(&w.norm2b, p + ".norm2b", D) || up_stacked(&w.up_e, ups, D, (int64_t)f.experts * f.ff) ||
          up_stacked(&w.down_e, downs, f.ff, (int64_t)f.experts * D) || up_stacked(&w.router, router, D, all + 1) ||
          up(&w.correction, e + ".correction", all) ||
          (f.shared_ff && (up(&w.up_s, e + ".shared.up", (int64_t)f.shared_ff * D) || up(&w.down_s, e + ".shared.down", (int64_t)D * f.shared_ff))))
        return -1;
    }
    return 0;
  }

  // ------------------------------------------------------------------ buffers
  int grow_rows(size_t n) override {
    auto* so = &step_owned;
    max_tiles = (int)((n * (size_t)mx_top + 63) / 64) + mx_experts;
    return dalloc(&x, n * D, so) || dalloc_a(&h, n * D, so) || dalloc_a(&proj, n * (size_t)mx_proj, so) || dalloc(&q32, n * (size_t)mx_q, so) ||
           dalloc(&o32, n * (size_t)mx_o, so) || dalloc(&z32, n * (size_t)mx_z, so) || dalloc_a(&mix, n * (size_t)mx_mix, so) ||
           dalloc_a(&y, n * D, so) || dalloc(&part, part_floats, so) || dalloc(&logits_r, n * (size_t)mx_route, so) ||
           dalloc(&route_e, n * (size_t)mx_top, so) || dalloc(&route_w, n * (size_t)mx_top, so) || dalloc(&pos_pair, n * (size_t)mx_top, so) ||
           dalloc(&pos_row, n * (size_t)mx_top, so) || dalloc(&tiles, 3 * (size_t)max_tiles + 1, so) ||
           dalloc_a(&act_e, n * (size_t)mx_pair_ff, so) || dalloc(&y_pairs, n * (size_t)mx_top * D, so) ||
           dalloc_a(&act_s, n * (size_t)mx_shared, so) || dalloc_a(&y_s, n * (size_t)(mx_shared ? D : 0), so) ? -1 : 0;
  }
  int grow_want(size_t n) override { return dalloc_a(&hw, n * D, &want_owned); }
  int before_step(const StepCtx& c) override {       // chunks of long entries: never part of a captured step
    size_t need = 0;
    if (c.chunks.n_long > 0)
      for (auto& l : layers)
        if (pegainfer_gated_linear_chunked_ok(l.right.dim, l.right.vdim))
          need = std::max(need, (size_t)pegainfer_gated_linear_workspace(c.chunks.n_chunks, l.right.heads, l.right.dim, l.right.vdim));
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
  pegainfer_terms_rms_desc norm_desc(int rows) const {
    pegainfer_terms_rms_desc d{};
    d.eps = eps; d.gain_offset = kGainOffset; d.n_dtype = dtype; d.d = D; d.rows = rows; d.dtype = dtype;
    return d;
  }
  // the end of a sublayer and the start of the next: its output, normed, joins the stream, and `next` (NULL: nothing follows) leaves h
  pegainfer_join_rms_desc join_desc(const StepCtx& s, const void* post, const void* next) const {
    pegainfer_join_rms_desc d{};
    d.x = x; d.post = post; d.gain = next; d.n_out = next ? h : nullptr;
    d.eps = eps; d.gain_offset = kGainOffset; d.d = D; d.rows = s.T; d.dtype = dtype;
    return d;
  }
  int join(const StepCtx& s, const void* post, const void* next) {
    pegainfer_join_rms_desc d = join_desc(s, post, next);
    d.y = y; d.y_row_stride = D;
    PSTEP_K(pegainfer_join_rms(&d, S()));
    return 0;
  }
  int attention(const StepCtx& s, const LayerCfg& c, const LayerW& w) {
    const AttnCfg& a = c.left;
    pegainfer_qk_prep_desc p{};
    p.proj = proj; p.proj_dtype = dtype; p.proj_stride = c.proj_rows; p.q_off = a.o_q; p.k_off = a.o_k; p.v_off = a.o_k;
    p.heads = a.heads; p.kv_heads = a.kv; p.dim = a.dim; p.vdim = a.dim; p.norm_kind = PEGAINFER_QKNORM_HEAD_WEIGHT;
    p.inv_freq = w.inv_freq; p.rot_dims = a.rot_dims; p.rot_layout = PEGAINFER_ROT_HALVES; p.rot_amp = a.amp;
    p.positions = s.pos; p.row_entry = s.entry; p.page_indptr = s.page_indptr; p.page_ids = s.pages;
    p.cache = cache; p.page_stride = page_stride; p.k_cache_off = c.k_off; p.v_cache_off = c.v_off; p.page_size = kPageSize;
    p.shared_tail = a.tail(); p.q_out = q32; p.n_rows = s.T; p.dtype = dtype;
    PSTEP_K(pegainfer_qk_prep(&p, S()));
    const TileTable& t = s.group_tiles[(size_t)c.tiles];
    const int wgs = t.count * a.kv;     // depends on the step's shape only, never on the contexts' lengths
    pegainfer_attn_options o{};
    o.sink = w.sink;
    o.gate = at(proj, (size_t)a.o_g); o.gate_stride = c.proj_rows; o.gate_kind = PEGAINFER_GATE_PER_HEAD;
    o.tile_rows = t.rows;
    o.n_split = wgs >= kFewTiles || t.rows > kGroupRows ? 1 : std::max(1, std::min(kMaxSplits, kSplitGroups / wgs));
    o.workspace = part;
    o.plain = plain_kernels ? 1 : 0;
    o.shared_tail = a.tail();
    PSTEP_K(pegainfer_paged_attention_opt(q32, cache, page_stride, c.k_off, c.v_off, kPageSize, s.pos, s.entry, s.page_indptr, s.pages, a.heads,
                                          a.kv, a.dim, a.dim, a.scale, c.left_scale, t.col(0), t.col(1), t.col(2), t.col(3), t.count, mix,
                                          c.mix_cols, &o, dtype, S()));
    return 0;
  }
  int memory(const StepCtx& s, const LayerCfg& c, const LayerW& w) {
    const MemCfg& m = c.right;
    const int rd = m.heads * m.dim;
    const int rp = pad8(m.rank);
    // few rows: the scan makes the decay inputs itself (its workgroups read W_a2 once per row)
    const bool fused = s.T <= kFusedRows && s.chunks.n_long == 0 && !plain_kernels && pegainfer_gated_linear_fused_ok(m.rank, rp, w.a2);
    if (!fused && linear_strided(w.a2, at(proj, (size_t)m.o_a), dtype, c.proj_rows, z32, PEGAINFER_DTYPE_F32, rd, s.T, rp)) return -1;
    pegainfer_gated_linear_desc d{};
    d.proj = proj; d.proj_stride = c.proj_rows; d.q_off = m.o_q; d.k_off = m.o_k; d.v_off = m.o_v;
    d.q_scale = (float)(1.0 / std::sqrt((double)m.dim));
    if (fused) { d.w_up = w.a2; d.low_off = m.o_a; d.rank = m.rank; d.rank_stride = rp; }
    else { d.z = z32; d.z_stride = rd; }
    d.z_bias = w.a2_bias; d.tau = m.tau;
    d.state = state + m.st_off; d.slot_stride = state_layout.floats_per_slot(); d.o = o32;
    d.heads = m.heads; d.dim = m.dim; d.vdim = m.vdim;
    d.entry_row0 = s.row0; d.entry_slot = s.slot; d.n_entries = s.n;
    d.dtype = dtype;
    if (s.chunks.n_long > 0 && pegainfer_gated_linear_chunked_ok(m.dim, m.vdim)) {
      d.scan_max = scan_max;
      d.chunk_row0 = s.chunks.row0; d.chunk_rows = s.chunks.rows; d.n_chunks = s.chunks.n_chunks;
      d.long_chunk0 = s.chunks.long_chunk0; d.long_slot = s.chunks.long_slot; d.n_long = s.chunks.n_long;
      d.workspace = chunk_ws;
    }
    PSTEP_K(pegainfer_gated_linear(&d, S()));
    PSTEP_K(pegainfer_head_rms_gate(o32, w.mem_norm, 0, at(proj, (size_t)m.o_g), c.proj_rows, 0, c.right_scale, eps,
                                    at(mix, (size_t)c.mix_right), c.mix_cols, m.heads, m.vdim, s.T, dtype, S()));
    return 0;
  }
  // h -> the stream, and h of the next layer
  int feed_forward(const StepCtx& s, const LayerCfg& c, const LayerW& w, const void* next) {
    const MoeCfg& f = c.moe;
    const int T = s.T, P = T * f.top, all = f.experts + f.identity;
    const bool tuned = dtype == PEGAINFER_DTYPE_BF16 && !plain_kernels && T > 8;      // many rows in bf16
    if (linear_strided(w.router, h, dtype, D, logits_r, PEGAINFER_DTYPE_F32, all + 1, T, D)) return -1;
    const int per_tile = tuned && D % 8 == 0 && f.ff % 8 == 0 ? 128 : 64;
    pegainfer_route_plan_desc r{};
    r.logits = logits_r; r.logits_stride = all + 1; r.correction = w.correction; r.out_expert = route_e; r.out_weight = route_w;
    r.experts = all; r.n_groups = 1; r.keep_groups = 1; r.top = f.top; r.rows = T; r.score_kind = PEGAINFER_SCORE_SOFTMAX; r.renorm = 1;
    r.factor = f.scale;
    r.sort_experts = f.experts;
    r.pos_pair = pos_pair; r.pos_row = pos_row;
    r.tile_group = tiles; r.tile_row0 = tiles + max_tiles; r.tile_rows = tiles + 2 * max_tiles; r.n_tiles = tiles + 3 * max_tiles;
    r.max_tiles = std::min(P, (P + per_tile - 1) / per_tile + f.experts); r.rows_per_tile = per_tile; r.dtype = dtype;
    PSTEP_K(pegainfer_route_plan(&r, S()));
    pegainfer_gemm_desc g{};
    g.tile_group = r.tile_group; g.tile_row0 = r.tile_row0; g.tile_rows = r.tile_rows; g.n_tiles = r.n_tiles; g.max_tiles = r.max_tiles;
    g.max_tile_rows = std::min(T, 64);   // a row chooses distinct experts: an expert never gets more pairs than there are rows
    g.tile_rows_cap = per_tile;
    g.w_k_stride = 1;
    g.plain = plain_kernels;
    pegainfer_gemm_desc u = g;           // gelu(W_up h), rows by position
    u.x = h; u.w = w.up_e; u.y = act_e;
    u.x_dtype = u.w_dtype = u.y_dtype = dtype;
    u.m = f.ff; u.k = D; u.x_row_stride = D; u.w_m_stride = D; u.w_group_stride = (int64_t)f.ff * D; u.y_row_stride = f.ff;
    u.x_row_index = pos_row;
    u.epilogue = PEGAINFER_EPI_GELU_ERF;
    PSTEP_K(pegainfer_gemm_strided(&u, S()));
    pegainfer_gemm_desc d = g;           // W_down, rows by (token, choice)
    d.x = act_e; d.w = w.down_e; d.y = y_pairs;
    d.x_dtype = d.w_dtype = dtype; d.y_dtype = PEGAINFER_DTYPE_F32;
    d.m = D; d.k = f.ff; d.x_row_stride = f.ff; d.w_m_stride = f.ff; d.w_group_stride = (int64_t)D * f.ff; d.y_row_stride = D;
    d.y_row_index = pos_pair;
    PSTEP_K(pegainfer_gemm_strided(&d, S()));
    if (f.shared_ff) {
      if (dtype == PEGAINFER_DTYPE_BF16 && !plain_kernels && T > 1) {   // a tuned route and the activation; one row: both in one launch
        if (linear(w.up_s, h, act_s, f.shared_ff, T, D)) return -1;
        PSTEP_K(pegainfer_act_rows(act_s, f.shared_ff, act_s, f.shared_ff, f.shared_ff, T, PEGAINFER_ACT_GELU_ERF, dtype, S()));
      } else if (linear_strided(w.up_s, h, dtype, D, act_s, dtype, f.shared_ff, T, D, PEGAINFER_EPI_GELU_ERF)) {
        return -1;
      }
      if (linear(w.down_s, act_s, y_s, D, T, f.shared_ff)) return -1;
    }
    pegainfer_join_rms_desc j = join_desc(s, w.norm2b, next);
    j.y_pairs = y_pairs; j.weight = route_w; j.expert = route_e; j.top = f.top; j.same_from = f.experts;
    if (f.identity) { j.same = h; j.same_stride = D; }
    if (f.shared_ff) { j.add = y_s; j.add_gate = logits_r + all; j.add_gate_stride = all + 1; }
    PSTEP_K(pegainfer_join_rms(&j, S()));
    return 0;
  }
  int run_step(const StepCtx& s) override {
    {
      pegainfer_terms_rms_desc d = norm_desc(s.T);
      d.embed = embed; d.token_ids = s.tokens; d.embed_scale = embed_scale;
      d.pair_table = bigram; d.prev_ids = s.prev; d.mul_prev = mul_prev; d.mul_cur = mul_cur; d.buckets = buckets;
      d.x_out = x; d.gain = weights[0].norm1; d.n_out = h;
      PSTEP_K(pegainfer_terms_rms(&d, S()));
    }
    for (size_t i = 0; i < layers.size(); ++i) {
      const LayerCfg& c = layers[i];
      const LayerW& w = weights[i];
      const void* next = i + 1 < layers.size() ? weights[i + 1].norm1 : nullptr;
      if (linear(w.proj, h, proj, c.proj_rows, s.T, D) || attention(s, c, w) || memory(s, c, w) || linear(w.o, mix, y, D, s.T, c.mix_cols)) return -1;
      if (join(s, w.norm1b, c.moe.ff ? w.norm2 : next)) return -1;
      if (c.moe.ff && feed_forward(s, c, w, next)) return -1;
      if (tap_on) PSTEP_HIP(hipMemcpyAsync(tap_at((int)i), x, (size_t)s.T * D * 4, hipMemcpyDeviceToDevice, stream));
    }
    if (s.W > 0) {
      pegainfer_terms_rms_desc d = norm_desc(s.W);
      d.x_in = x; d.row_index = s.want; d.gain = final_norm; d.n_out = hw;
      PSTEP_K(pegainfer_terms_rms(&d, S()));
      if (linear_strided(head, hw, dtype, D, logits32, PEGAINFER_DTYPE_F32, V, s.W, D)) return -1;
    }
    return 0;
  }

 private:
  float eps = 1e-5f, embed_scale = 1.f;
  int64_t buckets = 0, mul_prev = 0, mul_cur = 0;
  std::vector<LayerCfg> layers;
  std::vector<LayerW> weights;
  void *embed = nullptr, *bigram = nullptr, *head = nullptr, *final_norm = nullptr;
  int mx_proj = 0, mx_mix = 0, mx_q = 0, mx_o = 0, mx_z = 0, mx_route = 0, mx_top = 0, mx_pair_ff = 0, mx_shared = 0, mx_experts = 0, max_tiles = 0;
  size_t part_floats = 0, chunk_cap = 0;
  float *x = nullptr, *q32 = nullptr, *o32 = nullptr, *z32 = nullptr, *part = nullptr, *logits_r = nullptr, *route_w = nullptr, *y_pairs = nullptr,
        *chunk_ws = nullptr;
  void *h = nullptr, *proj = nullptr, *mix = nullptr, *y = nullptr, *act_e = nullptr, *act_s = nullptr, *y_s = nullptr, *hw = nullptr;
  int32_t *route_e = nullptr, *pos_pair = nullptr, *pos_row = nullptr, *tiles = nullptr;
};

}  // namespace psx

using psx::Model;
PEGAINFER_STEP_ENTRIES(pegainfer_sopanex, psx::Model)
