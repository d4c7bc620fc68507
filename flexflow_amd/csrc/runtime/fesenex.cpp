// fesenex.cpp -- Fesenex: a pre-norm decoder of softmax-attention layers and
// linear-attention layers with a fixed decay per head.
//
//   x = embed[token] * scale
//   per layer:  x += mixer(norm1(x));  x += ff(norm2(x))  (ff optional)
//   attention:  q, k = rms_norm per head of W x + b, v = W x + b, grouped heads;
//               q *= 1 + coef ln((p + 1) / every + 1); no rotation, scores
//               q . k * scale + rel[bucket(distance)]; the values of later
//               layers are mixed with those of the first mixing layer
//   lightning:  kernels/lightning.h, norm over all heads, sigmoid gate, W_o
//   ff:         W_down clamped_glu(W_gate x, W_up x)
//   logits = head norm(x)
//
// The residual stream, norms, scores, softmax, decays and states are fp32.
// bf16 model: products on bf16 operands, fp32 accumulation; projections reach
// their norms, activations and the residual sum as fp32 sums.  fp32 model
// (full_precision): the same graph on fp32 operands.
// Attention layers keep keys and values in pages shared by all requests
// (page_pool.h), lightning layers a state per request slot (state_slots.h).
#include <math.h>

#include <algorithm>

#include "../kernels/lightning.h"
#include "../kernels/paged_attn.h"
#include "paged_decoder.h"

namespace ffmi {

namespace {

struct FesenexLayer {
  bool attention = false;
  int heads = 0, groups = 0, dim = 0, vdim = 0, ff = 0;
  // attention
  float scale = 0.f, coef = 0.f;
  int every = 1, bias_max = 0;
  bool v_mix = false, v_first = false;
  // lightning
  std::vector<double> decay;
  float limit = 0.f;
  // padded sizes: per-head columns of the products (dg, vg) and of the caches
  // (dp, vp), first product, ff
  int dg = 0, vg = 0, dp = 0, vp = 0, nq = 0, fp = 0;
  void *win = nullptr, *wo = nullptr, *wgu = nullptr, *wdown = nullptr;
  float *norm1 = nullptr, *norm2 = nullptr;
  float *bias = nullptr, *norms = nullptr, *vmix = nullptr, *rel = nullptr;
  float *powers = nullptr, *onorm = nullptr;
  void *kc = nullptr, *vc = nullptr;  // [pages][groups] blocks (kernels/paged_attn.h)
  float *state = nullptr;             // [slots][heads][dg][vg]
};

// Row of the distance-bias table for distance n: one each below half of the
// rows, then logarithmic up to `far`.
int distance_bucket(int n, int rows, int far) {
  const int half = rows / 2;
  if (n < half) return n;
  if (n >= far) return rows - 1;
  const double at = log((double)n / half) / log((double)far / half) * (rows - half);
  return std::min(rows - 1, half + (int)floor(at));
}

struct Fesenex : public PagedDecoder {
  std::vector<FesenexLayer> layers;
  float embed_scale = 1.f;
  bool rows_form = false;  // some layer's attention has no MFMA form
  int max_slots = 0;
  // activations
  void *q = nullptr, *att = nullptr, *u = nullptr;
  uint16_t *qkv = nullptr;
  float *first_v = nullptr, *lin = nullptr, *slabs = nullptr, *ml = nullptr;

  // ---- configuration ----
  ffmi_status configure_attention(const Json &m, const std::string &at, FesenexLayer *L) {
    if (!m.get("kv_heads", &L->groups) || !m.get("scale", &L->scale) || !m.get("bias_max", &L->bias_max) ||
        L->groups <= 0 || L->heads % L->groups || L->bias_max <= 0)
      return bad(at + ".mixer");
    const Json *t = m.find("q_temp"), *vm = m.find("v_mix");
    if (t && !t->is_null() &&
        (!t->get("coef", &L->coef) || !t->get("every", &L->every) || L->every < 1))
      return bad(at + ".mixer.q_temp");
    if (vm && vm->type != Json::BOOL && !vm->is_null()) return bad(at + ".mixer.v_mix");
    L->v_mix = vm && vm->b;
    if (!L->v_mix) return FFMI_OK;
    L->v_first = true;
    for (const FesenexLayer &k : layers) {
      if (!k.v_mix) continue;
      L->v_first = false;
      if (k.groups != L->groups || k.vdim != L->vdim)
        return bad(at + ".mixer.v_mix: other value sizes than the first mixing layer");
    }
    return FFMI_OK;
  }
  ffmi_status configure(const Json &c) override {
    FFMI_TRY(configure_common(c));
    const Json *ls = c.find("layers"), *em = c.find("embedding");
    if (em && !em->is_null() && !em->get("scale", &embed_scale)) return bad("embedding.scale");
    if (!ls || ls->type != Json::ARR || ls->arr.empty()) return bad("layers");
    for (size_t i = 0; i < ls->arr.size(); ++i) {
      const Json &lj = ls->arr[i];
      const std::string at = "layers[" + std::to_string(i) + "]", type = lj.text("type");
      const Json *m = lj.find("mixer"), *f = lj.find("mlp");
      FesenexLayer L;
      L.attention = type == "attention";
      if (!L.attention && type != "lightning") return bad(at + ".type '" + type + "'");
      if (!m || !m->get("heads", &L.heads) || !m->get("dim", &L.dim) || !m->get("vdim", &L.vdim) ||
          L.heads <= 0 || L.dim <= 0 || L.vdim <= 0)
        return bad(at + ".mixer");
      if (L.attention) {
        FFMI_TRY(configure_attention(*m, at, &L));
      } else {
        const Json *d = m->find("decay");
        if (!d || d->type != Json::ARR || (int)d->arr.size() != L.heads) return bad(at + ".mixer.decay");
        for (const Json &v : d->arr) {
          if (v.type != Json::NUM) return bad(at + ".mixer.decay");
          L.decay.push_back(v.num);
        }
      }
      if (f && !f->is_null() &&
          (f->text("kind") != "dense" || !f->get("ff", &L.ff) || !f->get("limit", &L.limit) || L.ff <= 0))
        return bad(at + ".mlp");
      layers.push_back(L);
    }
    num_layers = (int)layers.size();
    return FFMI_OK;
  }

  // ---- buffers and weights ----
  ffmi_status init_layers() override {
    size_t qw = 32, ow = 32, uw = 32, fv = 0, lw = 0, lq = 0;
    double wbytes = 0;
    int min_groups = 1 << 30;
    std::vector<RowShape> shapes;
    std::vector<std::pair<int, int>> gemms;
    for (FesenexLayer &L : layers) {
      const int H = L.heads, G = L.groups;
      L.dg = up(L.dim, 32), L.vg = up(L.vdim, 32), L.fp = up(L.ff, 32);
      if (L.attention) {
        FFMI_CHECK(L.dg <= kAttnRowsMax && L.vg <= kAttnRowsMax, FFMI_ERR_UNSUPPORTED);
        L.dp = L.dg, L.vp = L.vg;
        if (!f32 && attn_width(L.dim) && attn_width(L.vdim))
          L.dp = attn_width(L.dim), L.vp = attn_width(L.vdim);
        else
          rows_form = true;
        L.nq = (H + G) * L.dg + G * L.vg;
        qw = std::max(qw, (size_t)H * L.dp);
        if (L.v_mix) fv = std::max(fv, (size_t)G * L.vg);
        shapes.push_back(RowShape{H / G, G, kAttnTiles, true});
        min_groups = std::min(min_groups, G);
      } else {
        FFMI_CHECK(L.dg <= kLightningMaxDim, FFMI_ERR_UNSUPPORTED);
        L.nq = 2 * H * (L.dg + L.vg);
        lw = std::max(lw, (size_t)H * L.vg);
        lq = std::max(lq, (size_t)H * (2 * L.dg + L.vg));
        recurrent = true;
      }
      ow = std::max(ow, (size_t)H * L.vg), uw = std::max(uw, (size_t)L.fp);
      gemms.insert(gemms.end(), {{L.nq, Wp}, {Wp, H * L.vg}});
      if (L.ff) {
        gemms.push_back({Wp, L.fp});
        if (f32) gemms.push_back({2 * L.fp, Wp});
        else
          for (int t = 16; t <= Tm; t += 16)
            ws_bytes = std::max(ws_bytes, gemm_bf16_glu_workspace_bytes(t, L.fp, Wp));
      }
      wbytes += 2.0 * ((double)L.nq * Wp + (double)H * L.vg * Wp + 3.0 * L.fp * Wp);
    }
    // 16-row slots for the splits of a step whose blocks do not fill the chip
    max_slots = rows_form || shapes.empty() ? 0 : 512 * kAttnTiles / min_groups;
    FFMI_TRY(init_step(shapes, max_slots, gemms, wbytes));
    FFMI_TRY(alloc_zero(&q, (size_t)Tm * qw * es()));
    FFMI_TRY(alloc_zero(&att, (size_t)Tm * ow * es()));
    FFMI_TRY(alloc_zero(&u, (size_t)Tm * uw * es()));
    if (fv) FFMI_TRY(alloc_zero(&first_v, (size_t)Tm * fv * 4));
    if (lw) FFMI_TRY(alloc_zero(&lin, (size_t)Tm * lw * 4));
    if (lq && !f32) FFMI_TRY(alloc_zero(&qkv, (size_t)Tm * lq * 2));
    size_t part = 0, rows = 0;
    for (FesenexLayer &L : layers) {
      if (!L.attention) {
        FFMI_TRY(alloc_zero(&L.state, (size_t)o.max_requests * L.heads * L.dg * L.vg * 4));
        continue;
      }
      const size_t cells = (size_t)cache_pages() * L.groups * kPageTokens;
      FFMI_TRY(alloc_zero(&L.kc, cells * L.dp * es()));
      FFMI_TRY(alloc_zero(&L.vc, cells * L.vp * es()));
      rows = std::max(rows, (size_t)max_slots * L.groups * 16);
      part = std::max(part, (size_t)max_slots * L.groups * 16 * L.vp);
    }
    if (part) {
      FFMI_TRY(alloc(&slabs, part * 4));
      FFMI_TRY(alloc(&ml, rows * 2 * 4));
    }
    for (size_t i = 0; i < layers.size(); ++i) FFMI_TRY(load_layer("l" + std::to_string(i) + ".", layers[i]));
    return FFMI_OK;
  }
  // rows [row0, row0 + heads * np) of the first product's weight
  ffmi_status in_rows(FesenexLayer &L, const std::string &name, int heads, int n, int np, int row0) {
    FFMI_TRY(raw(name, {(long)heads * n, W}));
    return pack_rows(spec(heads, n, np, 1, W, Wp), W, L.win, row0, L.nq);
  }
  ffmi_status load_layer(const std::string &p, FesenexLayer &L) {
    const std::string m = p + "mix.";
    const int H = L.heads, G = L.groups;
    FFMI_TRY(vec(&L.norm1, p + "norm1", 1, W, Wp));
    FFMI_TRY(alloc(&L.win, (size_t)L.nq * Wp * es()));
    FFMI_TRY(in_rows(L, m + "q", H, L.dim, L.dg, 0));
    if (L.attention) {
      const int off_k = H * L.dg, off_v = off_k + G * L.dg;
      FFMI_TRY(in_rows(L, m + "k", G, L.dim, L.dg, off_k));
      FFMI_TRY(in_rows(L, m + "v", G, L.vdim, L.vg, off_v));
      FFMI_TRY(alloc(&L.bias, (size_t)L.nq * 4));
      FFMI_TRY(vec_to(L.bias, m + "q.b", H, L.dim, L.dg, 0));
      FFMI_TRY(vec_to(L.bias + off_k, m + "k.b", G, L.dim, L.dg, 0));
      FFMI_TRY(vec_to(L.bias + off_v, m + "v.b", G, L.vdim, L.vg, 0));
      FFMI_TRY(alloc(&L.norms, (size_t)2 * L.dg * 4));
      FFMI_TRY(vec_to(L.norms, m + "q.norm", 1, L.dim, L.dg));
      FFMI_TRY(vec_to(L.norms + L.dg, m + "k.norm", 1, L.dim, L.dg));
      if (L.v_mix && !L.v_first) {
        std::vector<long> s;
        FFMI_TRY(shape_of(m + "vmix", {}, &s));
        FFMI_TRY(alloc(&L.vmix, 16));
        FFMI_TRY(raw(m + "vmix", s.empty() ? std::vector<long>() : std::vector<long>{1}));
        FFMI_HIP(launch_pack_f32(raw_tensor(), 1, spec(1, 1, 1, 1, 1, 1), L.vmix, stream));
      }
      FFMI_TRY(load_distance_bias(m + "rel", L));
    } else {
      const int off_k = H * L.dg, off_v = 2 * off_k, off_g = off_v + H * L.vg;
      FFMI_TRY(in_rows(L, m + "k", H, L.dim, L.dg, off_k));
      FFMI_TRY(in_rows(L, m + "v", H, L.vdim, L.vg, off_v));
      FFMI_TRY(in_rows(L, m + "g", H, L.vdim, L.vg, off_g));
      FFMI_TRY(vec(&L.onorm, m + "norm", H, L.vdim, L.vg));
      std::vector<float> pw;
      for (double d : L.decay)
        for (int i = 0; i <= kLightningChunk; ++i) pw.push_back((float)pow(d, i));
      FFMI_TRY(alloc(&L.powers, pw.size() * 4));
      FFMI_HIP(hipMemcpy(L.powers, pw.data(), pw.size() * 4, hipMemcpyHostToDevice));
    }
    FFMI_TRY(linear(&L.wo, m + "o", W, Wp, H, L.vdim, L.vg));
    if (!L.ff) return FFMI_OK;
    FFMI_TRY(vec(&L.norm2, p + "norm2", 1, W, Wp));
    FFMI_TRY(alloc(&L.wgu, (size_t)2 * L.fp * Wp * es()));
    FFMI_TRY(gate_up(L.wgu, p + "mlp.", L.ff, L.fp));
    return linear(&L.wdown, p + "mlp.down", W, Wp, 1, L.ff, L.fp);
  }
  // the bias of every distance, per head, in the attention's order (AttnArgs)
  ffmi_status load_distance_bias(const std::string &name, FesenexLayer &L) {
    std::vector<long> s;
    FFMI_TRY(shape_of(name, {32, L.heads}, &s));
    FFMI_CHECK(s.size() == 2 && s[0] >= 2 && s[1] == L.heads && L.bias_max > s[0] / 2, FFMI_ERR_INVALID);
    FFMI_TRY(raw(name, s));
    FFMI_HIP(hipStreamSynchronize(stream));
    std::vector<uint16_t> t((size_t)s[0] * s[1]);
    FFMI_HIP(hipMemcpy(t.data(), raw_tensor(), t.size() * 2, hipMemcpyDeviceToHost));
    const int D = L.bias_max, H = L.heads;
    std::vector<float> out((size_t)H * (D + 8), 0.f);
    for (int n = 0; n <= D + 3; ++n) {
      const int row = distance_bucket(n, (int)s[0], D);
      for (int h = 0; h < H; ++h) {
        const uint32_t bits = (uint32_t)t[(size_t)row * H + h] << 16;
        float v;
        memcpy(&v, &bits, 4);
        out[(size_t)h * (D + 8) + D + 3 - n] = f32 ? v : v * 1.4426950408889634f;
      }
    }
    FFMI_TRY(alloc(&L.rel, out.size() * 4));
    FFMI_HIP(hipMemcpy(L.rel, out.data(), out.size() * 4, hipMemcpyHostToDevice));
    return FFMI_OK;
  }

  // ---- one step ----
  ffmi_status attention(const FesenexLayer &L, Partials *y) {
    const int H = L.heads, G = L.groups;
    FFMI_TRY(gemm_sum(h, L.win, L.nq, Wp, y));
    AttnPrep p;
    p.y = *y, p.bias = L.bias, p.norms = L.norms;
    if (L.v_mix) p.first = first_v, p.vmix = L.vmix;
    p.q = q, p.kc = L.kc, p.vc = L.vc;
    p.H = H, p.G = G, p.dim = L.dim, p.dg = L.dg, p.dp = L.dp, p.vg = L.vg, p.vp = L.vp;
    p.eps = eps, p.coef = L.coef, p.every = L.every;
    const PagedLists &pl = step.lists(H / G, G);
    const bool rows = f32 || !attn_width(L.dim) || !attn_width(L.vdim);
    // decoding and short portions: in the attention's launch
    const bool fused = !rows && pl.row_tiles == 1;
    if (!fused) FFMI_HIP(launch_attn_prep(step.dev, step.off_tokens, step.T, p, f32, stream));
    AttnArgs a;
    a.q = q, a.kc = L.kc, a.vc = L.vc, a.bias = L.rel, a.o = att;
    a.H = H, a.G = G, a.dp = L.dp, a.vg = L.vg, a.vp = L.vp, a.D = L.bias_max;
    a.scale = f32 ? L.scale : L.scale * 1.4426950408889634f;
    if (rows) FFMI_HIP(launch_paged_attn_rows(step.dev, pl, a, f32, stream));
    else FFMI_HIP(launch_paged_attn(step.dev, pl, a, slabs, ml, stream, fused ? &p : nullptr, step.T));
    return gemm_sum(att, L.wo, Wp, H * L.vg, y);
  }
  ffmi_status lightning(const FesenexLayer &L, Partials *y) {
    const int H = L.heads;
    FFMI_TRY(gemm_sum(h, L.win, L.nq, Wp, y));
    Lightning a;
    a.y = *y, a.powers = L.powers, a.state = L.state, a.qkv = qkv, a.o = lin;
    a.H = H, a.dg = L.dg, a.vg = L.vg, a.T = step.T;
    // short spans token by token, long ones in chunks (bf16)
    const bool chunks = !f32 && L.dg <= kLightningMaxChunkDim;
    const int limit = chunks ? kShortSpan : BatchConfig::MAX_NUM_TOKENS;
    if (step.short_spans || !chunks)
      FFMI_HIP(launch_lightning_recurrent(step.dev, step.off_spans, step.num_spans, a, limit, stream));
    if (step.long_spans && chunks)
      FFMI_HIP(launch_lightning_chunks(step.dev, step.off_spans, step.num_spans, a, limit, stream));
    FFMI_HIP(launch_gated_norm(lin, *y, H * (2 * L.dg + L.vg), L.onorm, f32 ? nullptr : (uint16_t *)att,
                               f32 ? (float *)att : nullptr, step.T, H * L.vg, H * L.vdim, eps, stream));
    return gemm_sum(att, L.wo, Wp, H * L.vg, y);
  }
  ffmi_status feed_forward(const FesenexLayer &L, Partials *y) {
    const int T = step.T;
    if (f32) {
      FFMI_HIP(launch_gemm_f32((const float *)h, (const float *)L.wgu, ws, T, 2 * L.fp, Wp, stream));
      FFMI_HIP(launch_glu_f32(ws, (float *)u, T, L.fp, L.limit, stream));
    } else {
      FFMI_HIP(launch_gemm_bf16_glu((const uint16_t *)h, (const uint16_t *)L.wgu, (uint16_t *)u, ws, ws_bytes,
                                    T, L.fp, Wp, FFMI_X_PACKED | FFMI_Y_PACKED | wstream, L.limit, stream));
    }
    return gemm_sum(u, L.wdown, Wp, L.fp, y);
  }
  // x += y, then the next sublayer's input (w null: none follows)
  ffmi_status add_norm(const Partials &y, const float *w) {
    FFMI_HIP(launch_add_norm(y, w, x, f32 ? nullptr : (uint16_t *)h, f32 ? (float *)h : nullptr, step.T, Wp,
                             W, eps, stream));
    return FFMI_OK;
  }
  ffmi_status run_layers() override {
    FFMI_HIP(launch_embed_norm(step.host, step.dev, step.bytes, embed, embed_scale, layers[0].norm1, x,
                               f32 ? nullptr : (uint16_t *)h, f32 ? (float *)h : nullptr, step.T, Wp, W, eps,
                               stream));
    for (size_t i = 0; i < layers.size(); ++i) {
      const FesenexLayer &L = layers[i];
      const float *next = i + 1 < layers.size() ? layers[i + 1].norm1 : nullptr;
      Partials y;
      FFMI_TRY(L.attention ? attention(L, &y) : lightning(L, &y));
      FFMI_TRY(add_norm(y, L.ff ? L.norm2 : next));
      if (L.ff) {
        FFMI_TRY(feed_forward(L, &y));
        FFMI_TRY(add_norm(y, next));
      }
      FFMI_TRY(capture_layer((int)i));
    }
    return FFMI_OK;
  }
};

ffmi_status create_fesenex(const Json &config, const ffmi_model_opts *o, ffmi_model **out) {
  return PagedDecoder::create(new Fesenex(), config, o, out);
}
const ModelRegistrar g_registrar("Fesenex", create_fesenex);

}  // namespace

}  // namespace ffmi
