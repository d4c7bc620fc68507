// vapipel.cpp -- Vapipel: a decoder whose layers attend over a shared latent
// per token (latent attention without positions, learned absolute positions
// at the input, RMS norms on the sublayers' outputs only).
//
//   x = embed[token] + pos[p]
//   per layer:  x += norm1(mixer(x));  x += norm2(ff(x))  (ff optional)
//   mixer:  c = norm(W_dkv x), or another layer's c (kv_from);
//           per head softmax((W_q x)_h . (W_uk c)_h * scale) over the visible
//           positions, applied to (W_uv c)_h, times sigmoid((W_g x)_h); W_o
//   ff:     W_down relu(W_up x)^2
//   logits = head norm(x)
//
// The residual stream, norms, scores and softmax are fp32.  bf16 model:
// products on bf16 operands (kernels/gemm_bf16_*.hip, kernels/latent.hip),
// fp32 accumulation; the sublayers' outputs reach their norm as fp32 sums.
// fp32 model (full_precision): the same graph on fp32 operands.
// The cache holds one latent per token and layer that has its own W_dkv, in
// pages shared by all requests (page_pool.h).
#include <stdio.h>
#include <string.h>

#include <algorithm>
#include <map>
#include <string>
#include <vector>

#include "../kernels/latent.h"
#include "json.h"
#include "model.h"
#include "paged_step.h"
#include "safetensors.h"

namespace ffmi {

namespace {

int up(int v, int m) { return (v + m - 1) / m * m; }

struct VapipelLayer {
  int heads = 0, dim = 0, vdim = 0, rank = 0, kv_from = -1, ff = 0;
  float scale = 0.f;
  // padded sizes: per-head query / value widths, latent, gate columns, ff
  int dp = 0, vp = 0, rp = 0, gp = 0, fp = 0;
  int nq = 0, off_g = 0, off_d = 0;  // columns of the first product: q | gate | down
  void *wq = nullptr, *wuk = nullptr, *wuv = nullptr, *wo = nullptr, *wup = nullptr,
       *wdown = nullptr;
  float *dnorm = nullptr, *norm1 = nullptr, *norm2 = nullptr;
  void *cache = nullptr;  // [pages][kPageTokens][rp]; kv_from: layer kv_from's
};

struct Vapipel : public ffmi_model {
  ffmi_model_opts o{};
  std::string folder;
  int V = 0, W = 0, P = 0;      // vocab, width, positions
  int Vp = 0, Wp = 0, Tm = 0;   // padded; batch capacity
  float eps = 0.f;
  bool f32 = false;
  std::vector<VapipelLayer> layers;
  uint16_t *embed = nullptr, *pos = nullptr;
  float *final_norm = nullptr;
  void *head = nullptr;
  int wstream = 0;
  // activations
  float *x = nullptr, *ws = nullptr, *logits = nullptr;
  size_t ws_bytes = 0;
  uint16_t *xb = nullptr;
  void *qg = nullptr, *ql = nullptr, *ol = nullptr, *att = nullptr, *u = nullptr, *h = nullptr;
  float *slabs = nullptr, *ml = nullptr;
  int32_t *res_h = nullptr;  // pinned: ids [Tm] | probs [Tm]
  PagePool pool;
  PagedStep step;
  hipStream_t stream = nullptr;
  std::vector<void *> allocs;
  SafeTensors file;
  uint16_t *tmp = nullptr;  // one raw tensor while loading
  size_t tmp_elems = 0;
  // decode steps replay a captured graph per launch shape
  std::map<std::vector<int>, hipGraphExec_t> graphs;
  bool use_graphs = getenv("FFMI_NO_GRAPHS") == nullptr;
  // tensor capture (set_debug): the residual stream after every layer
  int dbg = 0, dbg_T = -1, dbg_R = 0;
  float *dbg_x = nullptr;

  static constexpr int kMaxSlots = 512;  // partial results of split attention blocks

  int token_capacity() const override { return o.max_tokens; }
  int vocab_size() const override { return V; }
  PagePool *page_pool() override { return &pool; }

  ~Vapipel() override {
    if (stream) (void)hipStreamSynchronize(stream);
    for (auto &kv : graphs) (void)hipGraphExecDestroy(kv.second);
    for (void *p : allocs) (void)hipFree(p);
    if (res_h) (void)hipHostFree(res_h);
    if (stream) (void)hipStreamDestroy(stream);
  }

  template <class T>
  ffmi_status alloc(T **p, size_t bytes) {
    if (hipMalloc((void **)p, bytes ? bytes : 16) != hipSuccess) {
      ffmi_set_last_error("model alloc", __FILE__, __LINE__);
      return FFMI_ERR_OOM;
    }
    allocs.push_back((void *)*p);
    return FFMI_OK;
  }
  static ffmi_status bad(const std::string &what) {
    ffmi_set_last_error(("config.json: " + what).c_str(), __FILE__, __LINE__);
    return FFMI_ERR_INVALID;
  }

  // ---- configuration ----
  ffmi_status configure(const Json &c) {
    const Json *n = c.find("norm"), *ls = c.find("layers");
    if (!c.get("vocab", &V) || !c.get("width", &W) || !c.get("max_positions", &P) || V <= 0 ||
        W <= 0 || P <= 0)
      return bad("vocab, width and max_positions");
    if (!n || !n->get("eps", &eps)) return bad("norm.eps");
    if (!ls || ls->type != Json::ARR || ls->arr.empty()) return bad("layers");
    for (size_t i = 0; i < ls->arr.size(); ++i) {
      const Json &lj = ls->arr[i];
      const std::string at = "layers[" + std::to_string(i) + "]";
      if (lj.text("type") != "latent_attention") return bad(at + ".type '" + lj.text("type") + "'");
      const Json *m = lj.find("mixer"), *f = lj.find("mlp");
      VapipelLayer L;
      if (!m || !m->get("heads", &L.heads) || !m->get("dim", &L.dim) || !m->get("vdim", &L.vdim) ||
          !m->get("kv_rank", &L.rank) || !m->get("scale", &L.scale) || L.heads <= 0 || L.dim <= 0 ||
          L.vdim <= 0 || L.rank <= 0)
        return bad(at + ".mixer");
      const Json *kf = m->find("kv_from");
      if (kf && !kf->is_null()) {
        if (!m->get("kv_from", &L.kv_from) || L.kv_from < 0 || L.kv_from > (int)i)
          return bad(at + ".mixer.kv_from");
        if (L.kv_from == (int)i) L.kv_from = -1;
        else if (layers[L.kv_from].kv_from >= 0 || layers[L.kv_from].rank != L.rank)
          return bad(at + ".mixer.kv_from: not a layer with a latent of this rank");
      }
      if (f && !f->is_null()) {
        if (f->text("kind") != "dense" || !f->get("ff", &L.ff) || L.ff <= 0) return bad(at + ".mlp");
      }
      layers.push_back(L);
    }
    return FFMI_OK;
  }
  // latent width in the cache: what the attention's MFMA form takes, beyond
  // its largest (and in fp32) whole 32-column steps
  int pad_rank(int r) const {
    if (!f32)
      for (int p = 64; p <= 512; p += 64)
        if (p >= r && latent_rank_supported(p)) return p;
    return up(r, 32);
  }

  // ---- weights ----
  static double elems(const std::vector<long> &shape) {
    double n = 1;
    for (long d : shape) n *= (double)d;
    return n;
  }
  // tensor `name` to tmp as bf16 bits
  ffmi_status raw(const std::string &name, std::vector<long> shape, int kind = 0) {
    const size_t n = (size_t)elems(shape);
    if (n > tmp_elems) {
      FFMI_HIP(hipStreamSynchronize(stream));
      if (tmp) (void)hipFree(tmp);
      tmp = nullptr;
      FFMI_HIP(hipMalloc((void **)&tmp, n * 2));
      tmp_elems = n;
    }
    if (folder.empty()) {
      FFMI_HIP(launch_fill_weight_bf16(tmp, n, weight_key(name.c_str(), o.weight_seed), kind, stream));
      return FFMI_OK;
    }
    const SafeTensors::Tensor *t = file.find(name);
    if (!t || t->shape != shape) {
      ffmi_set_last_error(("model.safetensors: " + name +
                           (t ? " has another shape" : " is missing")).c_str(), __FILE__, __LINE__);
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
      ffmi_set_last_error(("model.safetensors: " + name + " has dtype " + t->dtype).c_str(),
                          __FILE__, __LINE__);
      return FFMI_ERR_UNSUPPORTED;
    }
    return FFMI_OK;
  }
  size_t es() const { return f32 ? 4 : 2; }
  // tmp -> rows of a GEMM weight: tile / row offset `row0` of an N-row matrix
  ffmi_status pack_rows(const PackSpec &p, int ld, void *dst, int row0, int N) {
    if (f32)
      FFMI_HIP(launch_pack_f32(tmp, ld, p, (float *)dst + (size_t)row0 * p.cols * p.kp, stream));
    else
      FFMI_HIP(launch_pack_bf16(tmp, ld, p, (uint16_t *)dst, row0 / 16, N / 16, false, stream));
    return FFMI_OK;
  }
  static PackSpec spec(int rows, int nb, int np, int cols, int kb, int kp, bool tr = false) {
    PackSpec p;
    p.rows = rows, p.nb = nb, p.np = np, p.cols = cols, p.kb = kb, p.kp = kp, p.transpose = tr;
    return p;
  }
  // one whole GEMM weight [nb][kb] -> [np][cols * kp]
  ffmi_status linear(void **dst, const std::string &name, int nb, int np, int cols, int kb, int kp) {
    ffmi_status st = alloc(dst, (size_t)np * cols * kp * es());
    if (st == FFMI_OK) st = raw(name, {nb, (long)cols * kb});
    if (st == FFMI_OK) st = pack_rows(spec(1, nb, np, cols, kb, kp), cols * kb, *dst, 0, np);
    return st;
  }
  ffmi_status vec(float **dst, const std::string &name, int n, int np) {
    ffmi_status st = alloc(dst, (size_t)np * 4);
    if (st == FFMI_OK) st = raw(name, {n}, 1);
    if (st == FFMI_OK) FFMI_HIP(launch_pack_f32(tmp, n, spec(1, 1, 1, 1, n, np), *dst, stream));
    return st;
  }
  // [rows][W] table, bf16 rows of Wp
  ffmi_status table(uint16_t **dst, const std::string &name, int rows) {
    ffmi_status st = alloc(dst, (size_t)rows * Wp * 2);
    if (st == FFMI_OK) st = raw(name, {rows, W});
    if (st != FFMI_OK) return st;
    if (Wp != W) FFMI_HIP(hipMemsetAsync(*dst, 0, (size_t)rows * Wp * 2, stream));
    FFMI_HIP(hipMemcpy2DAsync(*dst, (size_t)Wp * 2, tmp, (size_t)W * 2, (size_t)W * 2, rows,
                              hipMemcpyDeviceToDevice, stream));
    return FFMI_OK;
  }

#define TRY(x_) \
  do { if ((st = (x_)) != FFMI_OK) return st; } while (0)
  ffmi_status init() {
    ffmi_status st;
    f32 = o.full_precision != 0;
    FFMI_HIP(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
    if (!folder.empty() && !file.open(folder + "/model.safetensors")) {
      ffmi_set_last_error(("cannot read " + folder + "/model.safetensors").c_str(), __FILE__, __LINE__);
      return FFMI_ERR_INVALID;
    }
    Tm = up(o.max_tokens, 16);
    Wp = up(W, 32), Vp = up(V, 32);
    int nq = 0, lat = 0, av = 0, fu = 0, rmax = 0;
    double wbytes = (double)Vp * Wp * 2;
    std::vector<int> head_counts;
    for (VapipelLayer &L : layers) {
      L.dp = up(L.dim, 32), L.vp = up(L.vdim, 32), L.rp = pad_rank(L.rank);
      L.gp = up(L.heads, 32), L.fp = up(L.ff, 32);
      FFMI_CHECK(L.rp <= 2048, FFMI_ERR_UNSUPPORTED);  // (the row form's limit)
      L.off_g = L.heads * L.dp, L.off_d = L.off_g + L.gp;
      L.nq = L.off_d + (L.kv_from < 0 ? L.rp : 0);
      L.nq = up(L.nq, 32);
      nq = std::max(nq, L.nq), lat = std::max(lat, L.heads * L.rp);
      av = std::max(av, L.heads * L.vp), fu = std::max(fu, L.fp), rmax = std::max(rmax, L.rp);
      wbytes += 2.0 * ((double)L.nq * Wp + (double)L.heads * L.rp * (L.dp + L.vp) +
                       (double)L.heads * L.vp * Wp + 2.0 * L.fp * Wp);
      if (std::find(head_counts.begin(), head_counts.end(), L.heads) == head_counts.end())
        head_counts.push_back(L.heads);
    }
    // weights beyond the Infinity Cache: non-temporal loads, as the LLaMA model
    wstream = wbytes > 192.0 * (1 << 20) ? FFMI_W_STREAM : 0;
    bool rows_form = f32;  // some layer's attention takes unsplit blocks only
    for (const VapipelLayer &L : layers) rows_form |= !latent_rank_supported(L.rp);
    const int max_slots = rows_form ? 0 : kMaxSlots;
    TRY(step.init(Tm, o.max_requests, std::min(P, o.max_seq_len), head_counts, max_slots));
    // ---- activations ----
    TRY(alloc(&x, (size_t)Tm * Wp * 4));
    if (!f32) TRY(alloc(&xb, (size_t)Tm * Wp * 2));
    TRY(alloc(&qg, (size_t)Tm * nq * es()));
    TRY(alloc(&ql, (size_t)Tm * lat * es()));
    TRY(alloc(&ol, (size_t)Tm * lat * es()));
    TRY(alloc(&att, (size_t)Tm * av * es()));
    TRY(alloc(&u, (size_t)Tm * std::max(fu, 32) * es()));
    TRY(alloc(&h, (size_t)Tm * Wp * es()));
    TRY(alloc(&logits, (size_t)Tm * Vp * 4));
    if (max_slots) {
      TRY(alloc(&slabs, (size_t)max_slots * 64 * rmax * 4));
      TRY(alloc(&ml, (size_t)max_slots * 64 * 2 * 4));
    }
    ws_bytes = (size_t)Tm * Wp * 4;
    if (!f32)
      for (const VapipelLayer &L : layers)
        for (int t = 16; t <= Tm; t += 16) {
          const size_t w[4] = {gemm_bf16_workspace_bytes(t, L.nq, Wp),
                               gemm_bf16_workspace_bytes(t, Wp, L.heads * L.vp),
                               L.fp ? gemm_bf16_workspace_bytes(t, L.fp, Wp) : 0,
                               L.fp ? gemm_bf16_workspace_bytes(t, Wp, L.fp) : 0};
          ws_bytes = std::max(ws_bytes, *std::max_element(w, w + 4));
        }
    TRY(alloc(&ws, ws_bytes));
    // every buffer starts finite: padding columns meet zero weights
    FFMI_HIP(hipMemsetAsync(qg, 0, (size_t)Tm * nq * es(), stream));
    for (void *p : {ql, ol}) FFMI_HIP(hipMemsetAsync(p, 0, (size_t)Tm * lat * es(), stream));
    FFMI_HIP(hipMemsetAsync(att, 0, (size_t)Tm * av * es(), stream));
    if (xb) FFMI_HIP(hipMemsetAsync(xb, 0, (size_t)Tm * Wp * 2, stream));
    FFMI_HIP(hipMemsetAsync(u, 0, (size_t)Tm * std::max(fu, 32) * es(), stream));
    FFMI_HIP(hipMemsetAsync(h, 0, (size_t)Tm * Wp * es(), stream));
    FFMI_HIP(hipHostMalloc((void **)&res_h, (size_t)Tm * 8,
                           hipHostMallocCoherent | hipHostMallocMapped));
    // ---- cache ----
    const long want = o.kv_pool_tokens > 0 ? o.kv_pool_tokens
                                           : (long)o.max_requests * up(o.max_seq_len, kPageTokens);
    const int pages = (int)((want + kPageTokens - 1) / kPageTokens);
    pool.init(pages, kPageTokens, o.max_requests);
    for (VapipelLayer &L : layers) {
      if (L.kv_from >= 0) {
        L.cache = layers[L.kv_from].cache;
        continue;
      }
      // zeroed: positions not yet written are multiplied by zero weights
      const size_t bytes = (size_t)pages * kPageTokens * L.rp * es();
      TRY(alloc(&L.cache, bytes));
      FFMI_HIP(hipMemsetAsync(L.cache, 0, bytes, stream));
    }
    // ---- weights ----
    TRY(table(&embed, "embed", V));
    TRY(table(&pos, "pos", P));
    TRY(vec(&final_norm, "final.norm", W, Wp));
    TRY(linear(&head, "head", V, Vp, 1, W, Wp));
    for (size_t i = 0; i < layers.size(); ++i) {
      VapipelLayer &L = layers[i];
      const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.";
      const int H = L.heads;
      TRY(vec(&L.norm1, p + "norm1", W, Wp));
      TRY(alloc(&L.wq, (size_t)L.nq * Wp * es()));
      TRY(raw(m + "q", {(long)H * L.dim, W}));
      TRY(pack_rows(spec(H, L.dim, L.dp, 1, W, Wp), W, L.wq, 0, L.nq));
      TRY(raw(m + "g", {H, W}));
      TRY(pack_rows(spec(1, H, L.gp, 1, W, Wp), W, L.wq, L.off_g, L.nq));
      if (L.kv_from < 0) {
        TRY(raw(m + "dkv", {L.rank, W}));
        TRY(pack_rows(spec(1, L.rank, L.rp, 1, W, Wp), W, L.wq, L.off_d, L.nq));
        TRY(vec(&L.dnorm, m + "dkv.norm", L.rank, L.rp));
      }
      // head products: W_uk^T [rank][dim] and W_uv [vdim][rank] per head
      TRY(alloc(&L.wuk, (size_t)H * L.rp * L.dp * es()));
      TRY(raw(m + "uk", {(long)H * L.dim, L.rank}));
      if (f32)
        FFMI_HIP(launch_pack_f32(tmp, L.rank, spec(H, L.dim, L.dp, 1, L.rank, L.rp), (float *)L.wuk, stream));
      else
        FFMI_HIP(launch_pack_bf16(tmp, L.rank, spec(H, L.rank, L.rp, 1, L.dim, L.dp, true),
                                  (uint16_t *)L.wuk, 0, 0, true, stream));
      TRY(alloc(&L.wuv, (size_t)H * L.vp * L.rp * es()));
      TRY(raw(m + "uv", {(long)H * L.vdim, L.rank}));
      if (f32)
        FFMI_HIP(launch_pack_f32(tmp, L.rank, spec(H, L.rank, L.rp, 1, L.vdim, L.vp, true),
                                 (float *)L.wuv, stream));
      else
        FFMI_HIP(launch_pack_bf16(tmp, L.rank, spec(H, L.vdim, L.vp, 1, L.rank, L.rp),
                                  (uint16_t *)L.wuv, 0, 0, true, stream));
      TRY(linear(&L.wo, m + "o", W, Wp, H, L.vdim, L.vp));
      if (L.ff) {
        TRY(vec(&L.norm2, p + "norm2", W, Wp));
        TRY(linear(&L.wup, p + "mlp.up", L.ff, L.fp, 1, W, Wp));
        TRY(linear(&L.wdown, p + "mlp.down", W, Wp, 1, L.ff, L.fp));
      }
    }
    FFMI_HIP(hipStreamSynchronize(stream));
    if (tmp) (void)hipFree(tmp);
    tmp = nullptr, tmp_elems = 0;
    return FFMI_OK;
  }

  // ---- one step ----
  // y (fp32 sums) = X . W^T
  ffmi_status gemm_sum(const void *X, const void *Wt, int N, int K, Partials *y) {
    if (f32) {
      FFMI_HIP(launch_gemm_f32((const float *)X, (const float *)Wt, ws, step.T, N, K, stream));
      y->p = ws, y->S = 1, y->NP = N;
      return FFMI_OK;
    }
    FFMI_HIP(launch_gemm_bf16_f32((const uint16_t *)X, (const uint16_t *)Wt, nullptr, ws, ws_bytes,
                                  step.T, N, K, FFMI_X_PACKED | wstream, stream, y));
    return FFMI_OK;
  }
  ffmi_status mixer(const VapipelLayer &L, Partials *y) {
    const int T = step.T;
    const char *blob = step.dev;
    const PagedLists &pl = step.lists(L.heads);
    LatentStore sto;
    sto.w = L.dnorm, sto.ldd = L.nq, sto.rank = L.rp, sto.n = L.rank, sto.eps = eps;
    if (L.kv_from < 0) sto.cache = L.cache, sto.d = (const char *)qg + L.off_d * es();
    HeadGemm uk, uv;
    uk.X = qg, uk.W = L.wuk, uk.Y = ql, uk.T = T, uk.heads = L.heads;
    uk.K = L.dp, uk.N = L.rp, uk.ldx = L.nq;
    uv.X = ol, uv.W = L.wuv, uv.Y = att, uv.T = T, uv.heads = L.heads;
    uv.K = L.rp, uv.N = L.vp, uv.ldx = L.heads * L.rp;
    uv.gate = (const char *)qg + L.off_g * es(), uv.ldg = L.nq, uv.packed = !f32;
    if (f32) {
      FFMI_HIP(launch_gemm_f32(x, (const float *)L.wq, (float *)qg, T, L.nq, Wp, stream));
      if (sto.cache) FFMI_HIP(launch_latent_store_f32(blob, step.off_tokens, T, sto, stream));
      FFMI_HIP(launch_head_gemm_f32(uk, stream));
      FFMI_HIP(launch_latent_attention_rows(blob, pl, ql, L.cache, ol, L.rp, L.scale, false, stream));
      FFMI_HIP(launch_head_gemm_f32(uv, stream));
    } else {
      FFMI_HIP(launch_gemm_bf16_plain(xb, (const uint16_t *)L.wq, (uint16_t *)qg, ws, ws_bytes, T,
                                      L.nq, Wp, FFMI_X_PACKED | wstream, stream));
      FFMI_HIP(launch_latent_prep(blob, step.off_tokens, sto, uk, stream));
      if (latent_rank_supported(L.rp))
        FFMI_HIP(launch_latent_attention(blob, pl, (const uint16_t *)ql, (const uint16_t *)L.cache,
                                         (uint16_t *)ol, slabs, ml, L.rp, L.scale, stream));
      else
        FFMI_HIP(launch_latent_attention_rows(blob, pl, ql, L.cache, ol, L.rp, L.scale, true, stream));
      FFMI_HIP(launch_head_gemm(uv, stream));
    }
    return gemm_sum(att, L.wo, Wp, L.heads * L.vp, y);
  }
  ffmi_status feed_forward(const VapipelLayer &L, Partials *y) {
    const int T = step.T;
    if (f32) {
      FFMI_HIP(launch_gemm_f32(x, (const float *)L.wup, (float *)u, T, L.fp, Wp, stream));
      FFMI_HIP(launch_relu2_f32((float *)u, (size_t)T * L.fp, stream));
    } else {
      FFMI_HIP(launch_gemm_bf16_relu2(xb, (const uint16_t *)L.wup, (uint16_t *)u, ws, ws_bytes, T,
                                      L.fp, Wp, FFMI_X_PACKED | FFMI_Y_PACKED | wstream, stream));
    }
    return gemm_sum(u, L.wdown, Wp, L.fp, y);
  }
  ffmi_status enqueue(bool sample) {
    ffmi_status st;
    const int T = step.T, R = step.R;
    FFMI_HIP(launch_embed_pos(step.host, step.dev, step.bytes, embed, pos, x, xb, T, Wp, stream));
    for (size_t i = 0; i < layers.size(); ++i) {
      const VapipelLayer &L = layers[i];
      Partials y;
      TRY(mixer(L, &y));
      FFMI_HIP(launch_post_norm(y, L.norm1, x, xb, T, Wp, W, eps, stream));
      if (L.ff) {
        TRY(feed_forward(L, &y));
        FFMI_HIP(launch_post_norm(y, L.norm2, x, xb, T, Wp, W, eps, stream));
      }
      if (dbg)
        FFMI_HIP(hipMemcpyAsync(dbg_x + i * (size_t)Tm * Wp, x, (size_t)T * Wp * 4,
                                hipMemcpyDeviceToDevice, stream));
    }
    if (R == 0) return FFMI_OK;
    FFMI_HIP(launch_row_norm(step.dev, step.off_rows, x, final_norm, f32 ? nullptr : (uint16_t *)h,
                             f32 ? (float *)h : nullptr, R, Wp, W, eps, stream));
    if (f32)
      FFMI_HIP(launch_gemm_f32((const float *)h, (const float *)head, logits, R, Vp, Wp, stream));
    else
      FFMI_HIP(launch_gemm_bf16_f32((const uint16_t *)h, (const uint16_t *)head, nullptr, logits,
                                    (size_t)Tm * Vp * 4, R, Vp, Wp, FFMI_X_PACKED | wstream, stream));
    if (sample)  // greedy: argmax of the softmax, straight into pinned memory
      FFMI_HIP(launch_softmax_topk_f32(logits, R, V, 1, res_h, (float *)(res_h + Tm), stream, Vp));
    return FFMI_OK;
  }
  ffmi_status forward(const BatchConfig &bc, const int *rows, int n, bool sample) {
    ffmi_status st;
    if (mode != FFMI_MODEL_INC) return FFMI_ERR_INVALID;
    FFMI_CHECK(bc.num_tokens <= o.max_tokens, FFMI_ERR_INVALID);
    for (int t = 0; t < bc.num_tokens; ++t) {
      const auto &tk = bc.tokensInfo[t];
      FFMI_CHECK(tk.token_id >= 0 && tk.token_id < V, FFMI_ERR_INVALID);
      FFMI_CHECK(tk.abs_depth_in_request >= 0 && tk.abs_depth_in_request < P, FFMI_ERR_INVALID);
    }
    for (int i = 0; i < n; ++i) FFMI_CHECK(rows[i] >= 0 && rows[i] < bc.num_tokens, FFMI_ERR_INVALID);
    TRY(step.stage(bc, pool, rows, n));
    if (step.T == 0) return FFMI_OK;
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
        st = enqueue(sample);
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
      TRY(enqueue(sample));
    }
    FFMI_HIP(hipStreamSynchronize(stream));
    if (dbg) dbg_T = step.T, dbg_R = step.R;
    return FFMI_OK;
  }
#undef TRY

  // the output rows of a generation step are the requests' last tokens: only
  // their picks can be a next token
  ffmi_status run_inc(const BatchConfig &bc, InferenceResult *ir) override {
    std::vector<int> rows;
    for (int t = 0; t < bc.num_tokens; ++t)
      if (t + 1 == bc.num_tokens ||
          bc.tokensInfo[t + 1].request_index != bc.tokensInfo[t].request_index)
        rows.push_back(t);
    ffmi_status st = forward(bc, rows.data(), (int)rows.size(), true);
    if (st != FFMI_OK) return st;
    for (int t = 0; t < bc.num_tokens; ++t) ir->token_ids[t] = -1;
    for (size_t i = 0; i < rows.size(); ++i) ir->token_ids[rows[i]] = res_h[i];
    return FFMI_OK;
  }
  ffmi_status run_inc_logits(const BatchConfig &bc, const int *rows, int n, float *out) override {
    ffmi_status st = forward(bc, rows, n, false);
    if (st != FFMI_OK || n == 0) return st;
    FFMI_HIP(hipMemcpy2D(out, (size_t)V * 4, logits, (size_t)Vp * 4, (size_t)V * 4, n,
                         hipMemcpyDeviceToHost));
    return FFMI_OK;
  }
  ffmi_status run_tree(const TreeVerifyBatchConfig &, InferenceResult *) override {
    return FFMI_ERR_UNSUPPORTED;
  }
  ffmi_status run_beam(const BeamSearchBatchConfig &, BeamInferenceResult *) override {
    return FFMI_ERR_UNSUPPORTED;
  }

  long debug_width(int which) const override {
    return which == FFMI_DBG_LOGITS ? V : which == FFMI_DBG_HIDDEN ? W : -1;
  }
  ffmi_status set_debug(int enable) override {
    if (enable && !dbg_x) {
      ffmi_status st = alloc(&dbg_x, layers.size() * (size_t)Tm * Wp * 4);
      if (st != FFMI_OK) return st;
    }
    dbg = enable ? 1 : 0;
    dbg_T = -1;
    return FFMI_OK;
  }
  long debug_tensor(int which, int layer, float *out, long cap) override {
    const bool hid = which == FFMI_DBG_HIDDEN;
    if (dbg_T < 0 || (!hid && which != FFMI_DBG_LOGITS)) return -1;
    if (hid && (layer < 0 || layer >= (int)layers.size())) return -1;
    const long n = hid ? dbg_T : dbg_R, w = debug_width(which);
    if (cap < n * w) return -1;
    const float *src = hid ? dbg_x + (size_t)layer * Tm * Wp : logits;
    const size_t pitch = (size_t)(hid ? Wp : Vp) * 4;
    if (n > 0 && hipMemcpy2D(out, w * 4, src, pitch, w * 4, n, hipMemcpyDeviceToHost) != hipSuccess)
      return -1;
    return n;
  }
};

ffmi_status create_vapipel(const Json &config, const ffmi_model_opts *o, ffmi_model **out) {
  FFMI_CHECK(o->mode == FFMI_MODEL_INC && o->tp_size == 1, FFMI_ERR_UNSUPPORTED);
  FFMI_CHECK(o->max_tokens > 0 && o->max_tokens <= BatchConfig::MAX_NUM_TOKENS, FFMI_ERR_INVALID);
  FFMI_CHECK(o->max_requests > 0 && o->max_requests <= BatchConfig::MAX_NUM_REQUESTS,
             FFMI_ERR_INVALID);
  FFMI_CHECK(o->max_seq_len > 0 && o->kv_pool_tokens >= 0, FFMI_ERR_INVALID);
  Vapipel *m = new Vapipel();
  m->mode = o->mode;
  m->o = *o;
  if (o->weights_folder && o->weights_folder[0]) m->folder = o->weights_folder;
  m->o.weights_folder = nullptr;
  ffmi_status st = m->configure(config);
  int ndev = 0;
  if (st == FFMI_OK && (hipGetDeviceCount(&ndev) != hipSuccess || ndev == 0)) st = FFMI_ERR_NO_DEVICE;
  if (st == FFMI_OK) st = m->init();
  if (st != FFMI_OK) {
    delete m;
    return st;
  }
  *out = m;
  return FFMI_OK;
}
const ModelRegistrar g_registrar("Vapipel", create_vapipel);

}  // namespace

}  // namespace ffmi
