// What a host runtime with ONE batched step function needs besides its layers (include/pegainfer_zofadra.h and include/pegainfer_sopanex.h
// use it; the older runtimes beside them carry their own copies): device memory, checkpoint tensors waiting to be uploaded, request slots over the
// shared PagePool (kv_pool.h) and the fp32 state arena (seq_state.h), the step's packed metadata block with the tile tables its
// attention launches read, decode steps captured as hipGraphs, logits, sampling, logprobs, the per-layer stream tap - and the
// C entry points over all of that (PEGAINFER_STEP_ENTRIES).  A model derives from StepModel, parses its own layers and provides
//   parse(config)      sizes; add_cache() / state_layout.reserve() for what a request holds; *_tiles() for its launches' tables
//   resolve_sizes(f)   sizes that only the checkpoint's tensors tell (optional)
//   tensor_list()      names and shapes of the checkpoint
//   synthetic(...)     one weight of a seeded random model
//   build_weights()    staged tensors -> device
//   grow_rows(n)       step buffers for n token rows
//   run_step(ctx)      the launches of one step, up to logits32 of the wanted rows
#pragma once

#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <functional>
#include <map>
#include <string>
#include <vector>

#include "kv_pool.h"
#include "seq_state.h"
#include "safetensors_loader.h"
#include "pegainfer_kernels.h"
#include "pegainfer_kernels_blocks.h"
#include "pegainfer_kernels_ext.h"
#include "pegainfer_qwen3.h"     // pegainfer_logprobs_from_logits (pure host)
#include "pegainfer_duguzen.h"   // PEGAINFER_DTYPE_*

namespace pstep {

using pq::KvState;
using pq::PagePool;
using pst::Json;

#define PSTEP_HIP(expr)                                                \
  do {                                                                 \
    hipError_t e_ = (expr);                                            \
    if (e_ != hipSuccess) {                                            \
      set_error(std::string(#expr) + ": " + hipGetErrorString(e_));    \
      return -1;                                                       \
    }                                                                  \
  } while (0)
#define PSTEP_K(expr)                                                  \
  do {                                                                 \
    if ((expr) != 0) {                                                 \
      set_error(std::string(#expr) + " failed");                       \
      return -1;                                                       \
    }                                                                  \
  } while (0)

inline uint16_t f2bf(float f) {
  uint32_t u;
  std::memcpy(&u, &f, 4);
  if ((u & 0x7FFFFFFFu) > 0x7F800000u) return 0x7FC0;
  u += 0x7FFFu + ((u >> 16) & 1u);
  return static_cast<uint16_t>(u >> 16);
}
inline float bf2f(uint16_t h) {
  const uint32_t u = (uint32_t)h << 16;
  float f;
  std::memcpy(&f, &u, 4);
  return f;
}
inline int pad8(int n) { return (n + 7) & ~7; }
inline bool ends_with(const std::string& s, const char* suf) {
  const size_t n = std::strlen(suf);
  return s.size() >= n && s.compare(s.size() - n, n, suf) == 0;
}

constexpr int kPageSize = 16;       // tokens per cache page, as in the other runtimes
constexpr int kGroupRows = 16;      // (token, query head) rows of one workgroup of the paged attention
constexpr int kWideGroups = 256;    // a step whose 64- (32-) row tiles give so many workgroups takes those
constexpr int kFlatRows = 64;       // flattened (token, head) rows of one workgroup of the latent attention

// A table of row tiles on the device.  Group tiles: runs of tokens of one entry times a run of the query heads of one key/value
// head, at most kGroupRows rows - or 32 or 64 in prompts, where a model asks for it - (rows of four arrays: first token row, tokens, first
// query head, query heads).  Flat tiles: runs of
// <= kFlatRows flattened rows token * heads + head of one entry (two arrays: first row, rows).
struct TileTable {
  const int32_t* at = nullptr;
  int count = 0;
  int rows = kGroupRows;        // group tiles: the most rows of a tile
  const int32_t* col(int k) const { return at + (size_t)k * count; }
};
// Long entries (more than scan_max rows) cut into chunks, for recurrences with a chunk form.
struct ChunkTable {
  const int32_t *row0 = nullptr, *rows = nullptr, *long_chunk0 = nullptr, *long_slot = nullptr;
  int n_chunks = 0, n_long = 0;
};

// One step as its launches see it: shapes on the host, contents on the device.
struct StepCtx {
  int T = 0, n = 0, W = 0;         // token rows, entries, wanted rows
  bool single = false;             // every entry brings one token: decoding
  const uint32_t* tokens = nullptr;
  const int32_t* prev = nullptr;   // a row's previous token in its sequence, -1 for the first
  const int32_t *pos = nullptr, *entry = nullptr, *row0 = nullptr, *slot = nullptr, *page_indptr = nullptr, *want = nullptr, *pages = nullptr;
  std::vector<TileTable> group_tiles, flat_tiles;
  ChunkTable chunks;
};

typedef std::vector<std::pair<std::string, std::vector<int64_t>>> TensorList;

class StepModel {
 public:
  int device = 0, dtype = 0, D = 0, V = 0, max_requests = 0, num_pages = 0;
  bool plain_kernels = false, finalized = false, tap_on = false;
  std::string err;
  PagePool pool{0};
  std::vector<KvState> requests;
  std::vector<int32_t> last_token;     // of every request slot, -1 before its first
  pq::StateLayout state_layout;
  int64_t weight_bytes = 0;
  float last_step_ms = 0.f;

  virtual ~StepModel() {
    if (stream) (void)hipStreamSynchronize(stream);
    drop_graphs();
    free_all(&owned);
    free_all(&step_owned);
    free_all(&want_owned);
    if (tap) (void)hipFree(tap);
    if (meta_dev) (void)hipFree(meta_dev);
    if (meta_host) (void)hipHostFree(meta_host);
    if (ev0) (void)hipEventDestroy(ev0);
    if (ev1) (void)hipEventDestroy(ev1);
    if (stream) (void)hipStreamDestroy(stream);
    if (blas) cublas_destroy();
  }

  // ------------------------------------------------------------------ what a model provides
  virtual const char* architecture() const = 0;
  virtual int parse(const Json& config) = 0;
  virtual int layer_runs() const = 0;
  // sizes the configuration leaves to the tensors: numel_of gives a tensor's element count, 0 while it is unknown (a model of
  // synthetic weights then picks a size of its own).  Called before tensor_list() is used and before the weights are built.
  virtual int resolve_sizes(const std::function<int64_t(const std::string&)>&) { return 0; }
  virtual TensorList tensor_list() const = 0;
  virtual float synthetic(const std::string& name, float z, float std) const = 0;   // z: a draw of unit variance
  virtual int build_weights() = 0;
  virtual int grow_rows(size_t n) = 0;       // dalloc(.., &step_owned)
  virtual int grow_want(size_t) { return 0; }   // dalloc(.., &want_owned)
  virtual int run_step(const StepCtx& c) = 0;

  // ------------------------------------------------------------------ set-up
  int set_error(const std::string& e) { err = e; return -1; }
  int init(const std::string& text, int dev, int type, int max_tokens, int max_req) {
    device = dev; dtype = type; max_requests = max_req;
    Json j;
    if (!pst::JsonParser(text.data(), text.size()).parse(&j) || j.kind != Json::Obj) return set_error("config: not a JSON object");
    const Json* arch = j.get("architecture");
    if (!arch || arch->str != architecture()) return set_error(std::string("config: architecture is not ") + architecture());
    if (parse(j)) return -1;
    page_stride = std::max<int64_t>(8, (page_stride + 7) & ~(int64_t)7);
    PSTEP_HIP(hipSetDevice(device));
    cublas_init();
    blas = true;
    PSTEP_HIP(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
    PSTEP_HIP(hipEventCreate(&ev0));
    PSTEP_HIP(hipEventCreate(&ev1));
    num_pages = std::max(1, (max_tokens + kPageSize - 1) / kPageSize);
    pool = PagePool(num_pages);
    requests.assign((size_t)max_requests, KvState());
    last_token.assign((size_t)max_requests, -1);
    if (dalloc_a(&cache, (size_t)num_pages * (size_t)page_stride)) return -1;
    if (dalloc(&state, (size_t)max_requests * (size_t)std::max<int64_t>(1, state_layout.floats_per_slot()))) return -1;
    return dalloc(&probs_scratch, (size_t)V) || dalloc(&top1_value, 1) || dalloc(&row_states, 1024 * 1024) ||
           dalloc(&valid_scratch, 1) || dalloc(&sample_out_d, 1) ? -1 : 0;
  }

  // ------------------------------------------------------------------ weights
  int load_tensor(const std::string& name, const uint16_t* bits, int64_t n) {
    if (finalized) return set_error("load_tensor after finalize");
    staged[name].assign(bits, bits + n);
    return 0;
  }
  int fill_synthetic(uint64_t seed, float std) {
    uint64_t s = seed * 0x9E3779B97F4A7C15ull + 0x7654321ull;
    auto g = [&s]() {   // splitmix64; a unit-variance value = four uniforms summed, centred and scaled
      s += 0x9E3779B97F4A7C15ull;
      uint64_t z = s;
      z = (z ^ (z >> 30)) * 0xBF58476D1CE4E5B9ull;
      z = (z ^ (z >> 27)) * 0x94D049BB133111EBull;
      z ^= z >> 31;
      const float u = (float)(z & 0xFFFF) + (float)((z >> 16) & 0xFFFF) + (float)((z >> 32) & 0xFFFF) + (float)(z >> 48);
      return (u * (1.0f / 65536.0f) - 2.0f) * 1.7320508f;
    };
    if (resolve_sizes([](const std::string&) { return (int64_t)0; })) return -1;
    for (auto& t : tensor_list()) {
      std::vector<uint16_t>& v = staged[t.first];
      v.resize((size_t)numel(t.second));
      for (auto& x : v) x = f2bf(synthetic(t.first, g(), std));
    }
    return 0;
  }
  int load_checkpoint(const std::string& path) {
    pst::Checkpoint ck;
    std::string e;
    if (!ck.open(path, &e)) return set_error(e);
    if (resolve_sizes([&ck](const std::string& n) { const pst::TensorView* v = ck.find(n); return v ? (int64_t)v->numel() : (int64_t)0; }))
      return -1;
    for (auto& t : tensor_list()) {
      const pst::TensorView* v = ck.find(t.first);
      if (!v) return set_error("checkpoint has no tensor " + t.first);
      if (v->numel() != numel(t.second)) return set_error("checkpoint tensor " + t.first + " has another shape than config.json gives");
      std::vector<uint16_t>& dst = staged[t.first];
      dst.resize((size_t)v->numel());
      if (v->dtype == "BF16") {
        std::memcpy(dst.data(), v->data, dst.size() * 2);
      } else if (v->dtype == "F32") {
        const float* f = reinterpret_cast<const float*>(v->data);
        for (size_t k = 0; k < dst.size(); ++k) dst[k] = f2bf(f[k]);
      } else {
        return set_error("checkpoint tensor " + t.first + " has dtype " + v->dtype + " (bf16 expected)");
      }
    }
    return finalize();
  }
  int finalize() {
    if (finalized) return 0;
    if (resolve_sizes([this](const std::string& n) { const auto it = staged.find(n); return it == staged.end() ? (int64_t)0 : (int64_t)it->second.size(); }))
      return -1;
    if (build_weights()) return -1;
    staged.clear();
    finalized = true;
    return 0;
  }

  // ------------------------------------------------------------------ requests
  int new_request() {
    for (size_t i = 0; i < requests.size(); ++i)
      if (!requests[i].live) {
        const size_t n = (size_t)state_layout.floats_per_slot();
        if (n) PSTEP_HIP(hipMemsetAsync(state + i * n, 0, n * sizeof(float), stream));   // a request's state starts from zero
        requests[i].live = true;
        requests[i].seq_len = 0;
        last_token[i] = -1;
        return (int)i;
      }
    return set_error("no free request slot");
  }
  int drop_request(int id) {
    if (!known(id)) return set_error("drop_request: unknown request");
    requests[id].reset(&pool);
    requests[id].live = false;
    return 0;
  }
  bool known(int id) const { return id >= 0 && id < (int)requests.size() && requests[id].live; }

  // ------------------------------------------------------------------ the step
  int step(int n, const int32_t* ids, const int32_t* lens, const uint32_t* tokens, int n_want, const int32_t* want_rows,
           float* out_logits, int32_t* out_tokens) {
    if (!finalized) return set_error("step before finalize");
    if (n <= 0 || n > max_requests) return set_error("step: batch size outside 1 .. max_requests");
    // ---- validate everything before anything changes
    size_t T = 0;
    int need_pages = 0;
    for (int i = 0; i < n; ++i) {
      if (!known(ids[i])) return set_error("step: unknown request");
      for (int k = 0; k < i; ++k)
        if (ids[k] == ids[i]) return set_error("step: a request is listed twice");
      if (lens[i] <= 0) return set_error("step: an entry without tokens");
      const KvState& st = requests[ids[i]];
      need_pages += st.pages_short(st.seq_len + lens[i], kPageSize);
      T += (size_t)lens[i];
    }
    if (need_pages > pool.available()) return set_error("step: not enough free cache pages");
    for (size_t t = 0; t < T; ++t)
      if (tokens[t] >= (uint32_t)V) return set_error("step: token outside the vocabulary");
    std::vector<int32_t> want;
    if (n_want < 0) {
      size_t off = 0;
      for (int i = 0; i < n; ++i) { off += (size_t)lens[i]; want.push_back((int32_t)off - 1); }
    } else {
      for (int i = 0; i < n_want; ++i) {
        if (want_rows[i] < 0 || (size_t)want_rows[i] >= T) return set_error("step: wanted row outside the step");
        want.push_back(want_rows[i]);
      }
    }
    const int W = (int)want.size();
    if (ensure_rows(T) || ensure_want((size_t)std::max(1, W))) return -1;
    for (int i = 0; i < n; ++i)
      if (!requests[ids[i]].ensure_capacity(&pool, requests[ids[i]].seq_len + lens[i], kPageSize)) return set_error("step: page pool ran dry");
    // ---- the packed metadata block; the page lists come last: everything before them sits at offsets that depend on the step's
    //      shape only, which a captured graph relies on
    std::vector<int32_t>& mb = meta;
    mb.clear();
    auto open = [&](size_t len) { const size_t at = mb.size(); mb.resize(at + len); return at; };
    const size_t o_tok = open(T), o_prev = open(T), o_pos = open(T), o_ent = open(T), o_row0 = open((size_t)n + 1), o_slot = open((size_t)n),
                 o_ind = open((size_t)n + 1), o_want = open((size_t)std::max(1, W));
    StepCtx c;
    c.T = (int)T; c.n = n; c.W = W;
    c.single = true;
    {
      size_t t = 0, pg = 0;
      for (int i = 0; i < n; ++i) {
        const KvState& st = requests[ids[i]];
        c.single = c.single && lens[i] == 1;
        mb[o_row0 + i] = (int32_t)t;
        mb[o_slot + i] = ids[i];
        mb[o_ind + i] = (int32_t)pg;
        pg += st.pages.size();
        for (int k = 0; k < lens[i]; ++k, ++t) {
          mb[o_tok + t] = (int32_t)tokens[t];
          mb[o_prev + t] = k ? (int32_t)tokens[t - 1] : last_token[ids[i]];
          mb[o_pos + t] = st.seq_len + k;
          mb[o_ent + t] = i;
        }
      }
      mb[o_row0 + n] = (int32_t)t;
      mb[o_ind + n] = (int32_t)pg;
      for (int i = 0; i < W; ++i) mb[o_want + i] = want[i];
    }
    std::vector<std::pair<size_t, int>> group_at, flat_at;    // (offset, tiles)
    std::vector<int> group_rows;
    for (auto& gt : group_sets) {
      const int rows = gt.wide_kv > 0 && !plain_kernels ? wide_rows(lens, n, (int)T, gt) : kGroupRows;
      group_rows.push_back(rows);
      group_at.push_back(put_group_tiles(&mb, lens, n, gt.per, rows));
    }
    for (int heads : flat_heads) flat_at.push_back(put_flat_tiles(&mb, lens, n, heads));
    size_t o_chunks[4] = {0, 0, 0, 0};
    if (scan_max > 0) put_chunks(&mb, ids, lens, n, &c.chunks, o_chunks);
    const size_t o_pages = mb.size();
    for (int i = 0; i < n; ++i) mb.insert(mb.end(), requests[ids[i]].pages.begin(), requests[ids[i]].pages.end());
    if (ensure_meta(mb.size())) return -1;
    std::memcpy(meta_host, mb.data(), mb.size() * 4);
    PSTEP_HIP(hipEventRecord(ev0, stream));
    PSTEP_HIP(hipMemcpyAsync(meta_dev, meta_host, mb.size() * 4, hipMemcpyHostToDevice, stream));
    const int32_t* md = reinterpret_cast<const int32_t*>(meta_dev);
    c.tokens = reinterpret_cast<const uint32_t*>(md + o_tok);
    c.prev = md + o_prev; c.pos = md + o_pos; c.entry = md + o_ent; c.row0 = md + o_row0; c.slot = md + o_slot; c.page_indptr = md + o_ind;
    c.want = md + o_want; c.pages = md + o_pages;
    for (size_t k = 0; k < group_at.size(); ++k) c.group_tiles.push_back(TileTable{md + group_at[k].first, group_at[k].second, group_rows[k]});
    for (auto& f : flat_at) c.flat_tiles.push_back(TileTable{md + f.first, f.second, kFlatRows});
    if (c.chunks.n_long > 0) {
      c.chunks.row0 = md + o_chunks[0]; c.chunks.rows = md + o_chunks[1];
      c.chunks.long_chunk0 = md + o_chunks[2]; c.chunks.long_slot = md + o_chunks[3];
    }
    if (tap_on && ensure_tap(T)) return -1;
    if (before_step(c)) return -1;
    auto launches = [&]() -> int {
      if (run_step(c)) return -1;
      if (W > 0) {
        PSTEP_K(deepseek_f32_to_bf16_cuda(logits32, logits16, W * V, S()));
        if (out_tokens) PSTEP_K(pegainfer_batched_top1(logits16, V, W, V, top1_state, tokens_d, S()));
      }
      return 0;
    };
    // a step of single tokens only (decoding) is launch-bound: its launches are captured once per shape as a hipGraph and
    // replayed; steps with prompt portions run eagerly
    if (c.single && graphs_on && !tap_on) {
      const GraphKey key{n, W, out_tokens != nullptr, plain_kernels};
      hipGraphExec_t exec = nullptr;
      for (auto& g : graphs)
        if (g.first == key) exec = g.second;
      if (!exec) {
        hipGraph_t g = nullptr;
        PSTEP_HIP(hipStreamBeginCapture(stream, hipStreamCaptureModeThreadLocal));
        const int rc = launches();
        const hipError_t e = hipStreamEndCapture(stream, &g);
        if (rc) return -1;
        if (e != hipSuccess) return set_error("graph capture failed");
        PSTEP_HIP(hipGraphInstantiate(&exec, g, nullptr, nullptr, 0));
        PSTEP_HIP(hipGraphDestroy(g));
        graphs.emplace_back(key, exec);
      }
      PSTEP_HIP(hipGraphLaunch(exec, stream));
    } else if (launches()) {
      return -1;
    }
    last_rows = W;
    PSTEP_HIP(hipEventRecord(ev1, stream));
    if (W > 0 && out_logits) PSTEP_HIP(hipMemcpyAsync(out_logits, logits32, (size_t)W * V * 4, hipMemcpyDeviceToHost, stream));
    if (W > 0 && out_tokens) PSTEP_HIP(hipMemcpyAsync(out_tokens, tokens_d, (size_t)W * 4, hipMemcpyDeviceToHost, stream));
    PSTEP_HIP(hipStreamSynchronize(stream));
    (void)hipEventElapsedTime(&last_step_ms, ev0, ev1);
    for (int i = 0, t = 0; i < n; ++i) {
      t += lens[i];
      requests[ids[i]].seq_len += lens[i];
      last_token[ids[i]] = (int32_t)tokens[t - 1];
    }
    return 0;
  }

  // ------------------------------------------------------------------ sampling over the last step's wanted rows
  int sample(int row, float temperature, int top_k, float top_p, float random_val, int32_t* out) {
    if (row < 0 || row >= last_rows) return set_error("no logits for that row");
    const Half* lg = logits16 + (size_t)row * V;
    if ((temperature <= 0.0f || top_k == 1) && top_p >= 1.0f) {
      flashinfer_top1_cuda(lg, top1_value, row_states, sample_out_d, V, S());
    } else {
      uint32_t bits;
      std::memcpy(&bits, &random_val, 4);
      gpu_sample_flashinfer_cuda(lg, probs_scratch, valid_scratch, sample_out_d, V, 1.0f / temperature, top_k, top_p, (uint64_t)bits, S());
    }
    PSTEP_HIP(hipStreamSynchronize(stream));
    PSTEP_HIP(hipMemcpy(out, sample_out_d, 4, hipMemcpyDeviceToHost));
    return 0;
  }
  int logprobs(int row, uint32_t token, int top_k, float* out_lp, uint32_t* top_ids, float* top_lps) {
    if (row < 0 || row >= last_rows) return set_error("no logits for that row");
    if (token >= (uint32_t)V) return set_error("logprobs: token outside the vocabulary");
    lp_row.resize((size_t)V);
    PSTEP_HIP(hipStreamSynchronize(stream));
    PSTEP_HIP(hipMemcpy(lp_row.data(), logits32 + (size_t)row * V, (size_t)V * 4, hipMemcpyDeviceToHost));
    return pegainfer_logprobs_from_logits(lp_row.data(), V, token, top_k, out_lp, top_ids, top_lps);
  }
  int debug_hidden(int run, float* out, int max_rows) {
    if (!tap || run < 0 || run >= layer_runs()) return set_error("debug_hidden: no tap for that layer run");
    const int rows = std::min(max_rows, tap_rows);
    PSTEP_HIP(hipStreamSynchronize(stream));
    PSTEP_HIP(hipMemcpy(out, tap + (size_t)run * tap_rows * D, (size_t)rows * D * 4, hipMemcpyDeviceToHost));
    return rows;
  }

 protected:
  hipStream_t stream = nullptr;
  void* cache = nullptr;
  int64_t page_stride = 0;           // elements of a page; grows by add_cache
  float* state = nullptr;
  std::vector<void*> step_owned, want_owned, owned;
  float* logits32 = nullptr;         // [wanted, V]: run_step leaves them here
  // distinct parameters of the tile tables a model's launches read.  wide_kv: key/value heads of a layer whose prompts may take wider
  // group tiles (0: never)
  struct GroupSet { int per, wide_kv; bool operator==(const GroupSet& o) const { return per == o.per && wide_kv == o.wide_kv; } };
  std::vector<GroupSet> group_sets;
  std::vector<int> flat_heads;
  int scan_max = 0;                  // > 0: entries with more rows go into the chunk table
  bool graphs_on = true;
  std::map<std::string, std::vector<uint16_t>> staged;

  size_t esize() const { return dtype == PEGAINFER_DTYPE_F32 ? 4 : 2; }
  pegainfer_stream_t S() const { return reinterpret_cast<pegainfer_stream_t>(stream); }
  void* at(void* p, size_t elems) const { return static_cast<uint8_t*>(p) + elems * esize(); }
  const void* at(const void* p, size_t elems) const { return static_cast<const uint8_t*>(p) + elems * esize(); }
  static int64_t numel(const std::vector<int64_t>& s) { int64_t n = 1; for (int64_t d : s) n *= d; return n; }
  static int geti(const Json* j, const char* k, int d) { return j ? (int)j->number_or(k, d) : d; }
  static float getf(const Json* j, const char* k, double d) { return j ? (float)j->number_or(k, d) : (float)d; }

  // device buffers that depend on the step's shape (before a capture begins)
  virtual int before_step(const StepCtx&) { return 0; }

  // a part of every cache page: `per_token` elements for each of its tokens; returns the part's offset inside a page
  int64_t add_cache(int64_t per_token) {
    const int64_t off = page_stride;
    page_stride += kPageSize * per_token;
    return off;
  }
  template <typename X>
  static int index_of(std::vector<X>* v, X x) {
    const auto it = std::find(v->begin(), v->end(), x);
    if (it != v->end()) return (int)(it - v->begin());
    v->push_back(x);
    return (int)v->size() - 1;
  }
  int group_tiles(int heads_per_kv, int wide_kv = 0) { return index_of(&group_sets, GroupSet{heads_per_kv, wide_kv}); }
  int flat_tiles(int heads) { return index_of(&flat_heads, heads); }

  template <typename T>
  int dalloc(T** p, size_t count, std::vector<void*>* into = nullptr) {
    void* raw = nullptr;
    PSTEP_HIP(hipMalloc(&raw, std::max<size_t>(count, 1) * sizeof(T)));
    PSTEP_HIP(hipMemset(raw, 0, std::max<size_t>(count, 1) * sizeof(T)));
    (into ? into : &owned)->push_back(raw);
    *p = static_cast<T*>(raw);
    return 0;
  }
  int dalloc_a(void** p, size_t count, std::vector<void*>* into = nullptr) {
    uint8_t* raw = nullptr;
    if (dalloc(&raw, count * esize(), into)) return -1;
    *p = raw;
    return 0;
  }
  int upload(void** out, const uint16_t* bits, size_t n) {
    if (dalloc_a(out, n)) return -1;
    if (dtype == PEGAINFER_DTYPE_BF16) {
      PSTEP_HIP(hipMemcpy(*out, bits, n * 2, hipMemcpyHostToDevice));
    } else {
      std::vector<float> f(n);
      for (size_t i = 0; i < n; ++i) f[i] = bf2f(bits[i]);
      PSTEP_HIP(hipMemcpy(*out, f.data(), n * 4, hipMemcpyHostToDevice));
    }
    weight_bytes += (int64_t)(n * esize());
    return 0;
  }
  int upload_f32(float** out, const std::vector<float>& v) {
    if (dalloc(out, v.size())) return -1;
    if (!v.empty()) PSTEP_HIP(hipMemcpy(*out, v.data(), v.size() * 4, hipMemcpyHostToDevice));
    return 0;
  }
  const std::vector<uint16_t>* need(const std::string& name, int64_t n) {
    auto it = staged.find(name);
    if (it == staged.end()) { set_error("missing tensor " + name); return nullptr; }
    if ((int64_t)it->second.size() != n) { set_error("tensor " + name + " has the wrong number of elements"); return nullptr; }
    return &it->second;
  }
  int up(void** out, const std::string& name, int64_t n) {
    const auto* v = need(name, n);
    return v ? upload(out, v->data(), v->size()) : -1;
  }
  // [rows_i, cols] tensors stacked by rows, each part's first row at the given row of the stack (zero rows between and after)
  struct Part { std::string name; int64_t rows, at; };
  int up_stacked(void** out, const std::vector<Part>& parts, int64_t cols, int64_t total_rows) {
    std::vector<uint16_t> st((size_t)(total_rows * cols), 0);
    for (auto& p : parts) {
      const auto* v = need(p.name, p.rows * cols);
      if (!v) return -1;
      std::memcpy(&st[(size_t)(p.at * cols)], v->data(), v->size() * 2);
    }
    return upload(out, st.data(), st.size());
  }
  // [rows, cols_i] tensors side by side, each part's first column at the given column (Part.rows = its columns), zeros between and after
  int up_beside(void** out, const std::vector<Part>& parts, int64_t rows, int64_t total_cols) {
    std::vector<uint16_t> st((size_t)(rows * total_cols), 0);
    for (auto& p : parts) {
      const auto* v = need(p.name, rows * p.rows);
      if (!v) return -1;
      for (int64_t r = 0; r < rows; ++r) std::memcpy(&st[(size_t)(r * total_cols + p.at)], v->data() + r * p.rows, (size_t)p.rows * 2);
    }
    return upload(out, st.data(), st.size());
  }
  // [groups][rows][cols] transposed group by group to [groups][cols][rows]
  int up_transposed(void** out, const std::string& name, int groups, int rows, int cols) {
    const auto* v = need(name, (int64_t)groups * rows * cols);
    if (!v) return -1;
    std::vector<uint16_t> tr(v->size());
    for (int g = 0; g < groups; ++g)
      for (int r = 0; r < rows; ++r)
        for (int k = 0; k < cols; ++k) tr[((size_t)g * cols + k) * rows + r] = (*v)[((size_t)g * rows + r) * cols + k];
    return upload(out, tr.data(), tr.size());
  }
  // rotation frequencies base^(-2i / dims), rounded once to fp32
  static std::vector<float> rotation_frequencies(double base, int dims) {
    std::vector<float> f((size_t)std::max(1, dims / 2));
    for (int k = 0; k < dims / 2; ++k) f[k] = (float)std::pow(base, -2.0 * k / (double)dims);
    return f;
  }
  // Long-context scaling by a ramp over the dimensions: pairs whose wave turns more than `fast` times over `original` positions keep
  // their frequency, those that turn fewer than `slow` times have it divided by `factor`, the ones between are mixed linearly; every
  // cosine and sine is multiplied by amplitude().
  struct RampScaling {
    bool on = false;
    double factor = 1.0, original = 1.0, fast = 1.0, slow = 1.0;
    bool ok() const { return factor > 0.0 && original > 0.0 && fast > 0.0 && slow > 0.0; }
    float amplitude() const { return on ? (float)(0.1 * std::log(factor) + 1.0) : 1.0f; }
  };
  static RampScaling parse_ramp(const Json* j) {
    RampScaling r;
    r.on = j && j->kind == Json::Obj;
    if (r.on) {
      r.factor = j->number_or("factor", 1.0);
      r.original = j->number_or("original", 0.0);
      r.fast = j->number_or("fast", 32.0);
      r.slow = j->number_or("slow", 1.0);
    }
    return r;
  }
  static std::vector<float> rotation_frequencies(double base, int dims, const RampScaling& r) {
    if (!r.on) return rotation_frequencies(base, dims);
    auto dim_of = [&](double turns) { return dims * std::log(r.original / (2.0 * M_PI * turns)) / (2.0 * std::log(base)); };
    const double lo = std::max(std::floor(dim_of(r.fast)), 0.0), hi = std::min(std::ceil(dim_of(r.slow)), (double)dims - 1.0);
    std::vector<float> f((size_t)std::max(1, dims / 2));
    for (int k = 0; k < dims / 2; ++k) {
      const double w = std::pow(base, -2.0 * k / (double)dims), t = std::min(std::max((k - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
      f[k] = (float)(w / r.factor * t + w * (1.0 - t));
    }
    return f;
  }

  // Y[T, M] = X[T, K] W[M, K]^T in the model's storage type
  int linear(const void* W, const void* X, void* Y, int M, int T, int K) {
    if (dtype == PEGAINFER_DTYPE_BF16 && !plain_kernels) {
      gemm_cuda(static_cast<const Half*>(W), static_cast<const Half*>(X), static_cast<Half*>(Y), M, T, K, S());
      return 0;
    }
    return linear_strided(W, X, dtype, K, Y, dtype, M, T, K);
  }
  // the same through the strided GEMM: operands that are columns of a wider matrix, outputs that stay in fp32
  int linear_strided(const void* W, const void* X, int x_dtype, int64_t x_stride, void* Y, int y_dtype, int M, int T, int K,
                     int epilogue = PEGAINFER_EPI_NONE) {
    pegainfer_gemm_desc d{};
    d.x = X; d.w = W; d.y = Y;
    d.x_dtype = x_dtype; d.w_dtype = dtype; d.y_dtype = y_dtype;
    d.m = M; d.k = K; d.rows = T; d.groups = 1;
    d.x_row_stride = x_stride; d.w_m_stride = K; d.w_k_stride = 1; d.y_row_stride = M;
    d.epilogue = epilogue;
    d.plain = plain_kernels;
    PSTEP_K(pegainfer_gemm_strided(&d, S()));
    return 0;
  }
  float* tap_at(int run) { return tap + (size_t)run * tap_rows * D; }

 private:
  struct GraphKey {
    int n, want; bool tokens, plain;
    bool operator==(const GraphKey& o) const { return n == o.n && want == o.want && tokens == o.tokens && plain == o.plain; }
  };
  std::vector<std::pair<GraphKey, hipGraphExec_t>> graphs;   // captured decode steps, one per shape
  hipEvent_t ev0 = nullptr, ev1 = nullptr;
  bool blas = false;
  size_t cap_rows = 0, cap_want = 0, cap_meta = 0, tap_cap = 0;
  std::vector<int32_t> meta;
  uint8_t *meta_host = nullptr, *meta_dev = nullptr;
  Half *logits16 = nullptr, *top1_value = nullptr;
  int32_t *tokens_d = nullptr, *sample_out_d = nullptr;
  uint8_t *top1_state = nullptr, *row_states = nullptr, *valid_scratch = nullptr;
  float *probs_scratch = nullptr, *tap = nullptr;
  int last_rows = 0, tap_rows = 0;
  std::vector<float> lp_row;

  static void free_all(std::vector<void*>* v) {
    for (void* p : *v) (void)hipFree(p);
    v->clear();
  }
  void drop_graphs() {   // the buffers a graph was recorded over are about to move
    for (auto& g : graphs) (void)hipGraphExecDestroy(g.second);
    graphs.clear();
  }
  int ensure_rows(size_t T) {
    if (T <= cap_rows) return 0;
    PSTEP_HIP(hipStreamSynchronize(stream));
    drop_graphs();
    free_all(&step_owned);
    cap_rows = 0;
    size_t n = 64;
    while (n < T) n *= 2;
    if (grow_rows(n)) return -1;
    cap_rows = n;
    return 0;
  }
  int ensure_want(size_t n) {
    if (n <= cap_want) return 0;
    PSTEP_HIP(hipStreamSynchronize(stream));
    drop_graphs();
    free_all(&want_owned);
    cap_want = 0;
    size_t c = 16;
    while (c < n) c *= 2;
    auto* wo = &want_owned;
    if (dalloc(&logits32, c * V, wo) || dalloc(&logits16, c * V, wo) || dalloc(&tokens_d, c, wo) || dalloc(&top1_state, c * 16, wo) ||
        grow_want(c))
      return -1;
    cap_want = c;
    return 0;
  }
  int ensure_meta(size_t words) {
    if (words <= cap_meta) return 0;
    PSTEP_HIP(hipStreamSynchronize(stream));
    drop_graphs();
    if (meta_host) (void)hipHostFree(meta_host);
    if (meta_dev) (void)hipFree(meta_dev);
    meta_host = meta_dev = nullptr;
    cap_meta = 0;
    size_t c = 4096;
    while (c < words) c *= 2;
    PSTEP_HIP(hipHostMalloc(reinterpret_cast<void**>(&meta_host), c * 4, hipHostMallocDefault));
    PSTEP_HIP(hipMalloc(reinterpret_cast<void**>(&meta_dev), c * 4));
    cap_meta = c;
    return 0;
  }
  int ensure_tap(size_t T) {
    const size_t needf = (size_t)layer_runs() * T * D;
    if (needf > tap_cap) {
      PSTEP_HIP(hipStreamSynchronize(stream));
      if (tap) (void)hipFree(tap);
      tap = nullptr;
      tap_cap = 0;
      PSTEP_HIP(hipMalloc(reinterpret_cast<void**>(&tap), needf * 4));
      tap_cap = needf;
    }
    tap_rows = (int)T;
    return 0;
  }

  static std::pair<size_t, int> put_columns(std::vector<int32_t>* mb, const std::vector<std::vector<int32_t>>& cols) {
    const size_t at = mb->size();
    for (auto& c : cols) mb->insert(mb->end(), c.begin(), c.end());
    return {at, (int)cols[0].size()};
  }
  // the widest tiles that still fill the chip and are at least half full
  static int wide_rows(const int32_t* lens, int n, int T, const GroupSet& g) {
    for (int rows : {64, 32}) {
      const int tpt = std::max(1, rows / g.per), cuts = (g.per + rows - 1) / rows;
      long tiles = 0;
      for (int i = 0; i < n; ++i) tiles += (long)((lens[i] + tpt - 1) / tpt) * cuts;
      if (tiles * g.wide_kv >= kWideGroups && (long)T * g.per * 2 >= tiles * rows) return rows;
    }
    return kGroupRows;
  }
  static std::pair<size_t, int> put_group_tiles(std::vector<int32_t>* mb, const int32_t* lens, int n, int per, int rows) {
    std::vector<std::vector<int32_t>> c(4);
    auto add = [&](int row0, int ntok, int qh0, int nqh) { c[0].push_back(row0); c[1].push_back(ntok); c[2].push_back(qh0); c[3].push_back(nqh); };
    int r0 = 0;
    for (int i = 0; i < n; r0 += lens[i++]) {
      const int tpt = std::max(1, rows / per);
      for (int t0 = 0; t0 < lens[i]; t0 += tpt)
        for (int q0 = 0; q0 < per; q0 += rows) add(r0 + t0, std::min(tpt, lens[i] - t0), q0, std::min(rows, per - q0));
    }
    return put_columns(mb, c);
  }
  static std::pair<size_t, int> put_flat_tiles(std::vector<int32_t>* mb, const int32_t* lens, int n, int heads) {
    std::vector<std::vector<int32_t>> c(2);
    int tok0 = 0;
    for (int i = 0; i < n; tok0 += lens[i++])
      for (int r = 0; r < lens[i] * heads; r += kFlatRows) {
        c[0].push_back(tok0 * heads + r);
        c[1].push_back(std::min(kFlatRows, lens[i] * heads - r));
      }
    return put_columns(mb, c);
  }
  void put_chunks(std::vector<int32_t>* mb, const int32_t* ids, const int32_t* lens, int n, ChunkTable* t, size_t* off) const {
    std::vector<int32_t> row0, rows, first{0}, slot;
    int r0 = 0;
    for (int i = 0; i < n; r0 += lens[i++]) {
      if (lens[i] <= scan_max) continue;
      for (int k = 0; k < lens[i]; k += PEGAINFER_DECAY_CHUNK) {
        row0.push_back(r0 + k);
        rows.push_back(std::min<int>(PEGAINFER_DECAY_CHUNK, lens[i] - k));
      }
      first.push_back((int32_t)row0.size());
      slot.push_back(ids[i]);
    }
    t->n_chunks = (int)row0.size();
    t->n_long = (int)slot.size();
    const std::vector<int32_t>* v[4] = {&row0, &rows, &first, &slot};
    for (int k = 0; k < 4; ++k) {
      off[k] = mb->size();
      mb->insert(mb->end(), v[k]->begin(), v[k]->end());
    }
  }
};

// create / from_pretrained of a model class; the error of a failed creation is kept per thread
template <class Model>
struct Creator {
  static std::string& error() { static thread_local std::string e; return e; }
  static Model* create(const std::string& config, int device, int dtype, int max_tokens, int max_requests) {
    if (dtype != PEGAINFER_DTYPE_BF16 && dtype != PEGAINFER_DTYPE_F32) { error() = "dtype must be 0 (bf16) or 1 (f32)"; return nullptr; }
    if (max_tokens <= 0 || max_requests <= 0) { error() = "max_tokens and max_requests must be positive"; return nullptr; }
    Model* m = new Model();
    if (m->init(config, device, dtype, max_tokens, max_requests)) { error() = m->err; delete m; return nullptr; }
    return m;
  }
  static Model* load(const char* dir, int device, int dtype, int max_tokens, int max_requests) {
    std::string e;
    auto f = pst::MappedFile::open(std::string(dir) + "/config.json", &e);
    if (!f) { error() = e; return nullptr; }
    Model* m = create(std::string(reinterpret_cast<const char*>(f->data), f->size), device, dtype, max_tokens, max_requests);
    if (m && m->load_checkpoint(dir)) { error() = m->err; delete m; return nullptr; }
    return m;
  }
};

// the C entry points PREFIX_* of a class derived from StepModel (declared in the family's header)
#define PEGAINFER_STEP_ENTRIES(PREFIX, MODEL)                                                                                    \
  static MODEL* PREFIX##_m(void* m) { return static_cast<MODEL*>(m); }                                                           \
  extern "C" {                                                                                                                   \
  PREFIX##_t PREFIX##_create(const char* config_json, int32_t device, int32_t dtype, int32_t max_tokens, int32_t max_requests) { \
    if (!config_json) { pstep::Creator<MODEL>::error() = "no configuration"; return nullptr; }                                   \
    return pstep::Creator<MODEL>::create(config_json, device, dtype, max_tokens, max_requests);                                  \
  }                                                                                                                              \
  PREFIX##_t PREFIX##_from_pretrained(const char* dir, int32_t device, int32_t dtype, int32_t max_tokens, int32_t max_requests) { \
    return pstep::Creator<MODEL>::load(dir, device, dtype, max_tokens, max_requests);                                            \
  }                                                                                                                              \
  void PREFIX##_destroy(PREFIX##_t m) { delete PREFIX##_m(m); }                                                                  \
  const char* PREFIX##_last_error(PREFIX##_t m) { return m ? PREFIX##_m(m)->err.c_str() : pstep::Creator<MODEL>::error().c_str(); } \
  int32_t PREFIX##_load_tensor(PREFIX##_t m, const char* name, const void* bf16, int64_t n) {                                    \
    return PREFIX##_m(m)->load_tensor(name, static_cast<const uint16_t*>(bf16), n);                                              \
  }                                                                                                                              \
  int32_t PREFIX##_fill_synthetic(PREFIX##_t m, uint64_t seed, float std) { return PREFIX##_m(m)->fill_synthetic(seed, std); }   \
  int32_t PREFIX##_finalize(PREFIX##_t m) { return PREFIX##_m(m)->finalize(); }                                                  \
  int32_t PREFIX##_new_request(PREFIX##_t m) { return PREFIX##_m(m)->new_request(); }                                            \
  int32_t PREFIX##_drop_request(PREFIX##_t m, int32_t id) { return PREFIX##_m(m)->drop_request(id); }                            \
  int32_t PREFIX##_request_seq_len(PREFIX##_t m, int32_t id) { return PREFIX##_m(m)->known(id) ? PREFIX##_m(m)->requests[id].seq_len : -1; } \
  int32_t PREFIX##_available_pages(PREFIX##_t m) { return PREFIX##_m(m)->pool.available(); }                                     \
  int32_t PREFIX##_capacity_pages(PREFIX##_t m) { return PREFIX##_m(m)->pool.capacity(); }                                       \
  int32_t PREFIX##_page_size(PREFIX##_t) { return pstep::kPageSize; }                                                            \
  int32_t PREFIX##_max_batch_size(PREFIX##_t m) { return PREFIX##_m(m)->max_requests; }                                          \
  int32_t PREFIX##_vocab_size(PREFIX##_t m) { return PREFIX##_m(m)->V; }                                                         \
  int32_t PREFIX##_width(PREFIX##_t m) { return PREFIX##_m(m)->D; }                                                              \
  int32_t PREFIX##_num_layer_runs(PREFIX##_t m) { return PREFIX##_m(m)->layer_runs(); }                                          \
  int32_t PREFIX##_dtype(PREFIX##_t m) { return PREFIX##_m(m)->dtype; }                                                          \
  int64_t PREFIX##_state_floats(PREFIX##_t m) { return PREFIX##_m(m)->state_layout.floats_per_slot(); }                          \
  int32_t PREFIX##_step(PREFIX##_t m, int32_t n, const int32_t* ids, const int32_t* lens, const uint32_t* tokens, int32_t n_want, \
                        const int32_t* want_rows, float* out_logits, int32_t* out_tokens) {                                      \
    return PREFIX##_m(m)->step(n, ids, lens, tokens, n_want, want_rows, out_logits, out_tokens);                                 \
  }                                                                                                                              \
  int32_t PREFIX##_sample(PREFIX##_t m, int32_t row, float t, int32_t k, float p, float rv, int32_t* out) {                      \
    return PREFIX##_m(m)->sample(row, t, k, p, rv, out);                                                                         \
  }                                                                                                                              \
  int32_t PREFIX##_logprobs(PREFIX##_t m, int32_t row, uint32_t token, int32_t k, float* lp, uint32_t* ids, float* vals) {       \
    return PREFIX##_m(m)->logprobs(row, token, k, lp, ids, vals);                                                                \
  }                                                                                                                              \
  int32_t PREFIX##_debug_hidden_enable(PREFIX##_t m, int32_t on) { PREFIX##_m(m)->tap_on = on != 0; return 0; }                  \
  int32_t PREFIX##_debug_hidden(PREFIX##_t m, int32_t run, float* out, int32_t rows) { return PREFIX##_m(m)->debug_hidden(run, out, rows); } \
  float PREFIX##_last_step_ms(PREFIX##_t m) { return PREFIX##_m(m)->last_step_ms; }                                              \
  int64_t PREFIX##_weight_bytes(PREFIX##_t m) { return PREFIX##_m(m)->weight_bytes; }                                            \
  int32_t PREFIX##_set_plain_kernels(PREFIX##_t m, int32_t on) { PREFIX##_m(m)->plain_kernels = on != 0; return 0; }             \
  }

}  // namespace pstep
