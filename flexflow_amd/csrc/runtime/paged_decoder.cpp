// paged_decoder.cpp -- see paged_decoder.h.
#include "paged_decoder.h"

#include <algorithm>
#include <memory>

namespace ffmi {

PagedDecoder::~PagedDecoder() {
  if (stream) (void)hipStreamSynchronize(stream);
  for (auto &kv : graphs) (void)hipGraphExecDestroy(kv.second);
  for (void *p : allocs) (void)hipFree(p);
  if (tmp) (void)hipFree(tmp);
  if (res_h) (void)hipHostFree(res_h);
  if (stream) (void)hipStreamDestroy(stream);
}

ffmi_status PagedDecoder::alloc_bytes(void **p, size_t bytes) {
  if (hipMalloc(p, bytes ? bytes : 16) != hipSuccess) {
    ffmi_set_last_error("model alloc", __FILE__, __LINE__);
    return FFMI_ERR_OOM;
  }
  allocs.push_back(*p);
  return FFMI_OK;
}

ffmi_status PagedDecoder::bad(const std::string &what) {
  ffmi_set_last_error(("config.json: " + what).c_str(), __FILE__, __LINE__);
  return FFMI_ERR_INVALID;
}

ffmi_status PagedDecoder::configure_common(const Json &c) {
  const Json *n = c.find("norm");
  if (!c.get("vocab", &V) || !c.get("width", &W) || V <= 0 || W <= 0) return bad("vocab and width");
  if (!n || !n->get("eps", &eps)) return bad("norm.eps");
  return FFMI_OK;
}

// ---- weights ----
ffmi_status PagedDecoder::raw(const std::string &name, const std::vector<long> &shape, int kind) {
  size_t n = 1;
  for (long d : shape) n *= (size_t)d;
  if (n > tmp_elems) {
    FFMI_HIP(hipStreamSynchronize(stream));
    if (tmp) (void)hipFree(tmp);
    tmp = nullptr, tmp_elems = 0;
    FFMI_HIP(hipMalloc((void **)&tmp, n * 2));
    tmp_elems = n;
  }
  if (folder.empty()) {
    FFMI_HIP(launch_fill_weight_bf16(tmp, n, weight_key(name.c_str(), o.weight_seed), kind, stream));
    return FFMI_OK;
  }
  const SafeTensors::Tensor *t = file.find(name);
  if (!t || t->shape != shape) {
    ffmi_set_last_error(
        ("model.safetensors: " + name + (t ? " has another shape" : " is missing")).c_str(), __FILE__,
        __LINE__);
    return FFMI_ERR_INVALID;
  }
  FFMI_HIP(hipStreamSynchronize(stream));  // (tmp's previous tensor is packed)
  if (t->dtype == "BF16" && t->bytes == n * 2) {
    FFMI_HIP(hipMemcpy(tmp, t->data, n * 2, hipMemcpyHostToDevice));
  } else if (t->dtype == "F32" && t->bytes == n * 4) {  // rounded to bf16
    std::vector<uint16_t> v(n);
    for (size_t i = 0; i < n; ++i) {
      uint32_t b;
      memcpy(&b, t->data + i * 4, 4);
      v[i] = (uint16_t)((b + 0x7fff + ((b >> 16) & 1)) >> 16);
    }
    FFMI_HIP(hipMemcpy(tmp, v.data(), n * 2, hipMemcpyHostToDevice));
  } else {
    ffmi_set_last_error(("model.safetensors: " + name + " has dtype " + t->dtype).c_str(), __FILE__,
                        __LINE__);
    return FFMI_ERR_UNSUPPORTED;
  }
  return FFMI_OK;
}

ffmi_status PagedDecoder::shape_of(const std::string &name, const std::vector<long> &synthetic,
                                   std::vector<long> *shape) {
  *shape = synthetic;
  if (folder.empty()) return FFMI_OK;
  const SafeTensors::Tensor *t = file.find(name);
  if (!t) {
    ffmi_set_last_error(("model.safetensors: " + name + " is missing").c_str(), __FILE__, __LINE__);
    return FFMI_ERR_INVALID;
  }
  *shape = t->shape;
  return FFMI_OK;
}

ffmi_status PagedDecoder::pack_rows(const PackSpec &p, int ld, void *dst, int row0, int N) {
  if (f32)
    FFMI_HIP(launch_pack_f32(tmp, ld, p, (float *)dst + (size_t)row0 * (p.kt ? p.kt * 32 : p.cols * p.kp), stream));
  else
    FFMI_HIP(launch_pack_bf16(tmp, ld, p, (uint16_t *)dst, row0 / 16, N / 16, false, stream));
  return FFMI_OK;
}

ffmi_status PagedDecoder::linear(void **dst, const std::string &name, int nb, int np, int cols, int kb,
                                 int kp) {
  FFMI_TRY(alloc(dst, (size_t)np * cols * kp * es()));
  FFMI_TRY(raw(name, {nb, (long)cols * kb}));
  return pack_rows(spec(1, nb, np, cols, kb, kp), cols * kb, *dst, 0, np);
}

ffmi_status PagedDecoder::host_vec(std::vector<float> *v, const std::string &name, int n, int kind) {
  FFMI_TRY(raw(name, {n}, kind));
  FFMI_HIP(hipStreamSynchronize(stream));
  std::vector<uint16_t> t(n);
  FFMI_HIP(hipMemcpy(t.data(), tmp, t.size() * 2, hipMemcpyDeviceToHost));
  v->resize(n);
  for (int i = 0; i < n; ++i) {
    const uint32_t bits = (uint32_t)t[i] << 16;
    memcpy(&(*v)[i], &bits, 4);
  }
  return FFMI_OK;
}

ffmi_status PagedDecoder::gate_up(void *dst, const std::string &p, int ff, int fp) {
  const PackSpec gu = spec(1, ff, fp, 1, W, Wp);
  for (int k = 0; k < 2; ++k) {  // bf16: gate and up tiles in turn
    FFMI_TRY(raw(p + (k ? "up" : "gate"), {ff, W}));
    if (f32) FFMI_TRY(pack_rows(gu, W, dst, k * fp, 2 * fp));
    else FFMI_HIP(launch_pack_bf16(tmp, W, gu, (uint16_t *)dst, k, 2 * fp / 16, false, stream, 2));
  }
  return FFMI_OK;
}

ffmi_status PagedDecoder::expert_matrices(const std::string &p, int experts, int ff, int fp, void **gated,
                                          void **down) {
  const size_t gu = (size_t)2 * fp * Wp * es(), dn = (size_t)Wp * fp * es();
  FFMI_TRY(alloc(gated, gu * experts));
  FFMI_TRY(alloc(down, dn * experts));
  for (int e = 0; e < experts; ++e) {
    const std::string pe = p + "e" + std::to_string(e) + ".";
    FFMI_TRY(gate_up((char *)*gated + gu * e, pe, ff, fp));
    FFMI_TRY(raw(pe + "down", {W, ff}));
    FFMI_TRY(pack_rows(spec(1, W, Wp, 1, ff, fp), ff, (char *)*down + dn * e, 0, Wp));
  }
  return FFMI_OK;
}

void PagedDecoder::need_experts(MoeSizes n, int fp) {
  for (n.T = 1; n.T <= Tm; ++n.T) {
    moe.num_units = std::max(moe.num_units, (size_t)n.slots() * fp);
    moe.num_slots = std::max(moe.num_slots, (size_t)n.slots());
    moe.num_picks = std::max(moe.num_picks, (size_t)n.T * n.top);
    moe.num_tiles = std::max(moe.num_tiles, (size_t)(n.expert_tiles(n.tile_rows()) + n.shared_tiles(n.tile_rows())));
  }
}
ffmi_status PagedDecoder::alloc_experts() {
  if (!moe.num_slots) return FFMI_OK;
  MoeLists &l = moe.lists;
  FFMI_TRY(alloc_zero(&moe.units, moe.num_units * es()));
  FFMI_TRY(alloc_zero(&moe.rows, moe.num_slots * Wp * es()));
  FFMI_TRY(alloc_zero(&l.picked, moe.num_picks * 4));
  FFMI_TRY(alloc_zero(&l.at, moe.num_picks * 4));
  FFMI_TRY(alloc_zero(&l.wt, moe.num_picks * 4));
  FFMI_TRY(alloc_zero(&l.gate, (size_t)Tm * 4));
  FFMI_TRY(alloc_zero(&l.own, (size_t)Tm * 4));
  FFMI_TRY(alloc_zero(&l.slot_token, moe.num_slots * 4));
  FFMI_TRY(alloc_zero(&l.tiles, moe.num_tiles * sizeof(MoeTile)));
  return alloc_zero(&l.num_tiles, 16);
}

ffmi_status PagedDecoder::vec(float **dst, const std::string &name, int rows, int n, int np, int kind) {
  FFMI_TRY(alloc(dst, (size_t)rows * np * 4));
  return vec_to(*dst, name, rows, n, np, kind);
}

ffmi_status PagedDecoder::vec_to(float *dst, const std::string &name, int rows, int n, int np, int kind) {
  FFMI_TRY(raw(name, {(long)rows * n}, kind));
  FFMI_HIP(launch_pack_f32(tmp, n, spec(rows, 1, 1, 1, n, np), dst, stream));
  return FFMI_OK;
}

ffmi_status PagedDecoder::table(uint16_t **dst, const std::string &name, int rows) {
  FFMI_TRY(alloc(dst, (size_t)rows * Wp * 2));
  FFMI_TRY(raw(name, {rows, W}));
  if (Wp != W) FFMI_HIP(hipMemsetAsync(*dst, 0, (size_t)rows * Wp * 2, stream));
  FFMI_HIP(hipMemcpy2DAsync(*dst, (size_t)Wp * 2, tmp, (size_t)W * 2, (size_t)W * 2, rows,
                            hipMemcpyDeviceToDevice, stream));
  return FFMI_OK;
}

// ---- set-up ----
ffmi_status PagedDecoder::init() {
  f32 = o.full_precision != 0;
  FFMI_HIP(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
  if (!folder.empty() && !file.open(folder + "/model.safetensors")) {
    ffmi_set_last_error(("cannot read " + folder + "/model.safetensors").c_str(), __FILE__, __LINE__);
    return FFMI_ERR_INVALID;
  }
  Tm = up(o.max_tokens, 16);
  Wp = up(W, 32), Vp = up(V, 32);
  FFMI_TRY(init_layers());
  FFMI_TRY(table(&embed, "embed", V));
  FFMI_TRY(load_final());
  FFMI_TRY(linear(&head, "head", V, Vp, 1, W, Wp));
  FFMI_HIP(hipStreamSynchronize(stream));
  if (tmp) (void)hipFree(tmp);
  tmp = nullptr, tmp_elems = 0;
  return FFMI_OK;
}

ffmi_status PagedDecoder::init_step(const std::vector<RowShape> &shapes, int max_slots,
                                    const std::vector<std::pair<int, int>> &gemms,
                                    double weight_bytes) {
  // weights beyond the Infinity Cache: non-temporal loads, as the LLaMA model
  wstream = weight_bytes + 2.0 * Vp * Wp > 192.0 * (1 << 20) ? FFMI_W_STREAM : 0;
  const int positions = P > 0 ? std::min(P, o.max_seq_len) : o.max_seq_len;
  FFMI_TRY(step.init(Tm, o.max_requests, positions, shapes, max_slots));
  const long want = o.kv_pool_tokens > 0 ? o.kv_pool_tokens
                                         : (long)o.max_requests * up(o.max_seq_len, kPageTokens);
  pool.init((int)((want + kPageTokens - 1) / kPageTokens), kPageTokens, o.max_requests);
  states.init(o.max_requests);
  FFMI_TRY(alloc_zero(&x, (size_t)Tm * Wp * 4));
  FFMI_TRY(alloc_zero(&h, (size_t)Tm * Wp * es()));
  FFMI_TRY(alloc(&logits, (size_t)Tm * Vp * 4));
  ws_bytes = std::max(ws_bytes, (size_t)Tm * Wp * 4);
  for (const auto &g : gemms) ws_bytes = std::max(ws_bytes, sum_bytes(g.first, g.second));
  FFMI_TRY(alloc(&ws, ws_bytes));
  FFMI_HIP(hipHostMalloc((void **)&res_h, (size_t)Tm * 8,
                         hipHostMallocCoherent | hipHostMallocMapped));
  return FFMI_OK;
}

// ---- one step ----
size_t PagedDecoder::sum_bytes(int N, int K) const {
  size_t n = (size_t)Tm * N * 4;
  if (!f32)
    for (int t = 16; t <= Tm; t += 16) n = std::max(n, gemm_bf16_workspace_bytes(t, N, K));
  return n;
}

ffmi_status PagedDecoder::gemm_sum_to(const void *X, const void *Wt, int N, int K, Partials *y, float *to,
                                      size_t to_bytes) {
  if (f32) {
    FFMI_HIP(launch_gemm_f32((const float *)X, (const float *)Wt, to, step.T, N, K, stream));
    y->p = to, y->S = 1, y->NP = N;
    return FFMI_OK;
  }
  FFMI_HIP(launch_gemm_bf16_f32((const uint16_t *)X, (const uint16_t *)Wt, nullptr, to, to_bytes,
                                step.T, N, K, FFMI_X_PACKED | wstream, stream, y));
  return FFMI_OK;
}

ffmi_status PagedDecoder::capture(int i, const float *rows) {
  if (dbg)
    FFMI_HIP(hipMemcpyAsync(dbg_x + (size_t)i * Tm * Wp, rows, (size_t)step.T * Wp * 4,
                            hipMemcpyDeviceToDevice, stream));
  return FFMI_OK;
}

ffmi_status PagedDecoder::output_rows() {
  FFMI_HIP(launch_row_norm(step.dev, step.off_rows, x, final_norm, f32 ? nullptr : (uint16_t *)h,
                           f32 ? (float *)h : nullptr, step.R, Wp, W, eps, stream));
  return FFMI_OK;
}

ffmi_status PagedDecoder::enqueue(bool sample) {
  FFMI_TRY(run_layers());
  const int R = step.R;
  if (R == 0) return FFMI_OK;
  FFMI_TRY(output_rows());
  if (f32)
    FFMI_HIP(launch_gemm_f32((const float *)h, (const float *)head, logits, R, Vp, Wp, stream));
  else
    FFMI_HIP(launch_gemm_bf16_f32((const uint16_t *)h, (const uint16_t *)head, nullptr, logits,
                                  (size_t)Tm * Vp * 4, R, Vp, Wp, FFMI_X_PACKED | wstream, stream));
  if (logit_cap > 0.f) FFMI_HIP(launch_soft_cap(logits, R, V, Vp, logit_cap, stream));
  if (sample)  // greedy: argmax of the softmax, straight into pinned memory
    FFMI_HIP(launch_softmax_topk_f32(logits, R, V, 1, res_h, (float *)(res_h + Tm), stream, Vp));
  return FFMI_OK;
}

ffmi_status PagedDecoder::forward(const BatchConfig &bc, const int *rows, int n, bool sample) {
  if (mode != FFMI_MODEL_INC) return FFMI_ERR_INVALID;
  FFMI_CHECK(bc.num_tokens <= o.max_tokens, FFMI_ERR_INVALID);
  const int positions = P > 0 ? P : o.max_seq_len;
  for (int t = 0; t < bc.num_tokens; ++t) {
    const auto &tk = bc.tokensInfo[t];
    FFMI_CHECK(tk.token_id >= 0 && tk.token_id < V, FFMI_ERR_INVALID);
    FFMI_CHECK(tk.abs_depth_in_request >= 0 && tk.abs_depth_in_request < positions, FFMI_ERR_INVALID);
  }
  for (int i = 0; i < n; ++i) FFMI_CHECK(rows[i] >= 0 && rows[i] < bc.num_tokens, FFMI_ERR_INVALID);
  if (recurrent)  // a request's tokens follow each other in a step (checked by stage)
    for (int t = 0; t < bc.num_tokens; ++t) {
      const auto &tk = bc.tokensInfo[t];
      if (t > 0 && bc.tokensInfo[t - 1].request_index == tk.request_index) continue;
      FFMI_CHECK(tk.request_index >= 0 && tk.request_index < o.max_requests, FFMI_ERR_INVALID);
      FFMI_CHECK(states.follows(tk.request_index, bc.requestsInfo[tk.request_index].request_guid,
                                tk.abs_depth_in_request),
                 FFMI_ERR_INVALID);
    }
  FFMI_TRY(step.stage(bc, pool, recurrent ? &states : nullptr, rows, n));
  if (step.T == 0) return FFMI_OK;
  if (recurrent)
    for (int t = 0; t < bc.num_tokens; ++t) {
      const int s = bc.tokensInfo[t].request_index;
      states.begin(s, bc.requestsInfo[s].request_guid);
    }
  if (use_graphs && !dbg && step.T <= 64) {
    std::vector<int> key = step.shape;
    key.push_back(sample);
    auto it = graphs.find(key);
    if (it == graphs.end()) {
      if (graphs.size() >= 256) {
        for (auto &kv : graphs) (void)hipGraphExecDestroy(kv.second);
        graphs.clear();
      }
      hipGraph_t g = nullptr;
      FFMI_HIP(hipStreamBeginCapture(stream, hipStreamCaptureModeThreadLocal));
      const ffmi_status st = enqueue(sample);
      const hipError_t ce = hipStreamEndCapture(stream, &g);
      if (st != FFMI_OK || ce != hipSuccess) {
        if (g) (void)hipGraphDestroy(g);
        if (st != FFMI_OK) return st;
        FFMI_HIP(ce);
      }
      hipGraphExec_t ex = nullptr;
      const hipError_t ie = hipGraphInstantiate(&ex, g, nullptr, nullptr, 0);
      (void)hipGraphDestroy(g);
      FFMI_HIP(ie);
      it = graphs.emplace(key, ex).first;
    }
    FFMI_HIP(hipGraphLaunch(it->second, stream));
  } else {
    FFMI_TRY(enqueue(sample));
  }
  FFMI_HIP(hipStreamSynchronize(stream));
  if (recurrent)
    for (int t = 0; t < bc.num_tokens; ++t) {
      const auto &tk = bc.tokensInfo[t];
      if (t + 1 == bc.num_tokens || bc.tokensInfo[t + 1].request_index != tk.request_index)
        states.done(tk.request_index, tk.abs_depth_in_request + 1, tk.token_id);
    }
  if (dbg) dbg_T = step.T, dbg_R = step.R;
  return FFMI_OK;
}

// the output rows of a generation step are the requests' last tokens: only
// their picks can be a next token
ffmi_status PagedDecoder::run_inc(const BatchConfig &bc, InferenceResult *ir) {
  std::vector<int> rows;
  for (int t = 0; t < bc.num_tokens; ++t)
    if (t + 1 == bc.num_tokens ||
        bc.tokensInfo[t + 1].request_index != bc.tokensInfo[t].request_index)
      rows.push_back(t);
  FFMI_TRY(forward(bc, rows.data(), (int)rows.size(), true));
  for (int t = 0; t < bc.num_tokens; ++t) ir->token_ids[t] = -1;
  for (size_t i = 0; i < rows.size(); ++i) ir->token_ids[rows[i]] = res_h[i];
  return FFMI_OK;
}

ffmi_status PagedDecoder::run_inc_logits(const BatchConfig &bc, const int *rows, int n, float *out) {
  FFMI_TRY(forward(bc, rows, n, false));
  if (n == 0) return FFMI_OK;
  FFMI_HIP(hipMemcpy2D(out, (size_t)V * 4, logits, (size_t)Vp * 4, (size_t)V * 4, n,
                       hipMemcpyDeviceToHost));
  return FFMI_OK;
}

ffmi_status PagedDecoder::set_debug(int enable) {
  if (enable && !dbg_x) FFMI_TRY(alloc(&dbg_x, (size_t)num_layers * Tm * Wp * 4));
  dbg = enable ? 1 : 0;
  dbg_T = -1;
  return FFMI_OK;
}

long PagedDecoder::debug_tensor(int which, int layer, float *out, long cap) {
  const bool hid = which == FFMI_DBG_HIDDEN;
  if (dbg_T < 0 || (!hid && which != FFMI_DBG_LOGITS)) return -1;
  if (hid && (layer < 0 || layer >= num_layers)) return -1;
  const long n = hid ? dbg_T : dbg_R, w = debug_width(which);
  if (cap < n * w) return -1;
  const float *src = hid ? dbg_x + (size_t)layer * Tm * Wp : logits;
  const size_t pitch = (size_t)(hid ? Wp : Vp) * 4;
  if (n > 0 && hipMemcpy2D(out, w * 4, src, pitch, w * 4, n, hipMemcpyDeviceToHost) != hipSuccess)
    return -1;
  return n;
}

ffmi_status PagedDecoder::create(PagedDecoder *m, const Json &config, const ffmi_model_opts *o,
                                 ffmi_model **out) {
  std::unique_ptr<PagedDecoder> own(m);
  FFMI_CHECK(o->mode == FFMI_MODEL_INC && o->tp_size == 1, FFMI_ERR_UNSUPPORTED);
  FFMI_CHECK(o->max_tokens > 0 && o->max_tokens <= BatchConfig::MAX_NUM_TOKENS, FFMI_ERR_INVALID);
  FFMI_CHECK(o->max_requests > 0 && o->max_requests <= BatchConfig::MAX_NUM_REQUESTS,
             FFMI_ERR_INVALID);
  FFMI_CHECK(o->max_seq_len > 0 && o->kv_pool_tokens >= 0, FFMI_ERR_INVALID);
  m->mode = o->mode;
  m->o = *o;
  if (o->weights_folder && o->weights_folder[0]) m->folder = o->weights_folder;
  m->o.weights_folder = nullptr;
  FFMI_TRY(m->configure(config));
  int ndev = 0;
  if (hipGetDeviceCount(&ndev) != hipSuccess || ndev == 0) return FFMI_ERR_NO_DEVICE;
  FFMI_TRY(m->init());
  *out = own.release();
  return FFMI_OK;
}

}  // namespace ffmi
