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
#include <algorithm>

#include "../kernels/latent.h"
#include "paged_decoder.h"

namespace ffmi {

namespace {

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

struct Vapipel : public PagedDecoder {
  std::vector<VapipelLayer> layers;
  uint16_t *pos = nullptr;
  // activations
  uint16_t *xb = nullptr;
  void *qg = nullptr, *ql = nullptr, *ol = nullptr, *att = nullptr, *u = nullptr;
  float *slabs = nullptr, *ml = nullptr;

  static constexpr int kMaxSlots = 512;  // partial results of split attention blocks

  // ---- configuration ----
  ffmi_status configure(const Json &c) override {
    FFMI_TRY(configure_common(c));
    const Json *ls = c.find("layers");
    if (!c.get("max_positions", &P) || P <= 0) return bad("max_positions");
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
    num_layers = (int)layers.size();
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

  ffmi_status init_layers() override {
    int nq = 0, lat = 0, av = 0, fu = 0, rmax = 0;
    double wbytes = 0;
    std::vector<RowShape> shapes;
    std::vector<std::pair<int, int>> gemms;
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
      shapes.push_back(RowShape{L.heads});
      gemms.insert(gemms.end(), {{L.nq, Wp}, {Wp, L.heads * L.vp}});
      if (L.ff) gemms.insert(gemms.end(), {{L.fp, Wp}, {Wp, L.fp}});
    }
    bool rows_form = f32;  // some layer's attention takes unsplit blocks only
    for (const VapipelLayer &L : layers) rows_form |= !latent_rank_supported(L.rp);
    const int max_slots = rows_form ? 0 : kMaxSlots;
    FFMI_TRY(init_step(shapes, max_slots, gemms, wbytes));
    if (!f32) FFMI_TRY(alloc_zero(&xb, (size_t)Tm * Wp * 2));
    FFMI_TRY(alloc_zero(&qg, (size_t)Tm * nq * es()));
    FFMI_TRY(alloc_zero(&ql, (size_t)Tm * lat * es()));
    FFMI_TRY(alloc_zero(&ol, (size_t)Tm * lat * es()));
    FFMI_TRY(alloc_zero(&att, (size_t)Tm * av * es()));
    FFMI_TRY(alloc_zero(&u, (size_t)Tm * std::max(fu, 32) * es()));
    if (max_slots) {
      FFMI_TRY(alloc(&slabs, (size_t)max_slots * 64 * rmax * 4));
      FFMI_TRY(alloc(&ml, (size_t)max_slots * 64 * 2 * 4));
    }
    for (VapipelLayer &L : layers) {
      if (L.kv_from >= 0) L.cache = layers[L.kv_from].cache;
      else FFMI_TRY(alloc_zero(&L.cache, (size_t)cache_pages() * kPageTokens * L.rp * es()));
    }
    // ---- weights ----
    FFMI_TRY(table(&pos, "pos", P));
    for (size_t i = 0; i < layers.size(); ++i) {
      VapipelLayer &L = layers[i];
      const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.";
      const int H = L.heads;
      FFMI_TRY(vec(&L.norm1, p + "norm1", 1, W, Wp));
      FFMI_TRY(alloc(&L.wq, (size_t)L.nq * Wp * es()));
      FFMI_TRY(raw(m + "q", {(long)H * L.dim, W}));
      FFMI_TRY(pack_rows(spec(H, L.dim, L.dp, 1, W, Wp), W, L.wq, 0, L.nq));
      FFMI_TRY(raw(m + "g", {H, W}));
      FFMI_TRY(pack_rows(spec(1, H, L.gp, 1, W, Wp), W, L.wq, L.off_g, L.nq));
      if (L.kv_from < 0) {
        FFMI_TRY(raw(m + "dkv", {L.rank, W}));
        FFMI_TRY(pack_rows(spec(1, L.rank, L.rp, 1, W, Wp), W, L.wq, L.off_d, L.nq));
        FFMI_TRY(vec(&L.dnorm, m + "dkv.norm", 1, L.rank, L.rp));
      }
      // head products: W_uk^T [rank][dim] and W_uv [vdim][rank] per head
      FFMI_TRY(alloc(&L.wuk, (size_t)H * L.rp * L.dp * es()));
      FFMI_TRY(raw(m + "uk", {(long)H * L.dim, L.rank}));
      if (f32)
        FFMI_HIP(launch_pack_f32(raw_tensor(), L.rank, spec(H, L.dim, L.dp, 1, L.rank, L.rp), (float *)L.wuk, stream));
      else
        FFMI_HIP(launch_pack_bf16(raw_tensor(), L.rank, spec(H, L.rank, L.rp, 1, L.dim, L.dp, true),
                                  (uint16_t *)L.wuk, 0, 0, true, stream));
      FFMI_TRY(alloc(&L.wuv, (size_t)H * L.vp * L.rp * es()));
      FFMI_TRY(raw(m + "uv", {(long)H * L.vdim, L.rank}));
      if (f32)
        FFMI_HIP(launch_pack_f32(raw_tensor(), L.rank, spec(H, L.rank, L.rp, 1, L.vdim, L.vp, true),
                                 (float *)L.wuv, stream));
      else
        FFMI_HIP(launch_pack_bf16(raw_tensor(), L.rank, spec(H, L.vdim, L.vp, 1, L.rank, L.rp),
                                  (uint16_t *)L.wuv, 0, 0, true, stream));
      FFMI_TRY(linear(&L.wo, m + "o", W, Wp, H, L.vdim, L.vp));
      if (L.ff) {
        FFMI_TRY(vec(&L.norm2, p + "norm2", 1, W, Wp));
        FFMI_TRY(linear(&L.wup, p + "mlp.up", L.ff, L.fp, 1, W, Wp));
        FFMI_TRY(linear(&L.wdown, p + "mlp.down", W, Wp, 1, L.ff, L.fp));
      }
    }
    return FFMI_OK;
  }

  // ---- one step ----
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
  ffmi_status run_layers() override {
    const int T = step.T;
    FFMI_HIP(launch_embed_pos(step.host, step.dev, step.bytes, embed, pos, x, xb, T, Wp, stream));
    for (size_t i = 0; i < layers.size(); ++i) {
      const VapipelLayer &L = layers[i];
      Partials y;
      FFMI_TRY(mixer(L, &y));
      FFMI_HIP(launch_post_norm(y, L.norm1, x, xb, T, Wp, W, eps, stream));
      if (L.ff) {
        FFMI_TRY(feed_forward(L, &y));
        FFMI_HIP(launch_post_norm(y, L.norm2, x, xb, T, Wp, W, eps, stream));
      }
      FFMI_TRY(capture_layer((int)i));
    }
    return FFMI_OK;
  }
};

ffmi_status create_vapipel(const Json &config, const ffmi_model_opts *o, ffmi_model **out) {
  return PagedDecoder::create(new Vapipel(), config, o, out);
}
const ModelRegistrar g_registrar("Vapipel", create_vapipel);

}  // namespace

}  // namespace ffmi
