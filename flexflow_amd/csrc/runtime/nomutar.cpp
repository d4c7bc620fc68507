// nomutar.cpp -- Nomutar: a decoder of parallel layers (mixer and feed-forward read
// the same norm) with rotary attention of three types, dense or mixture-of-experts
// feed-forwards, a short convolution at every mixer's input and a stretch of layers
// that may run several times over.
//
//   x = embed[token] * scale + bigram[hash(previous token, token)]
//   per layer:  h = group norm(x);  x += m (mixer(h + conv(h)) + ff(h))  (ff optional)
//   mixer:  q, k, v = W h (+ b), grouped heads; optional norm of the whole q and k
//           rows; rotation (frequencies as they are, scaled by wavelength, or YaRN);
//           scores cap tanh(q . k * scale / cap) over a window; softmax, optionally
//           with a sink; optionally values that turn with their positions; W_o
//   ff:     W_down (silu(W_gate h) * (W_up h)); or the `top` of many such, weighted,
//           beside a shared one with a sigmoid gate (on its units, so that its W_down
//           joins W_o)
//   logits = cap tanh(head group norm(x) / cap)
//
// 32-bit in either precision: residual stream, norms, convolution and its carried
// rows, angles, scores, softmax, router.  bf16 model: products on bf16 operands with
// fp32 accumulation, q, cached k and v, gated units and experts' outputs in bf16.
// fp32 model (full_precision): the same graph on fp32 operands.
// Every run of a layer has its own pages and carried rows; the request slot also
// remembers the last token (state_slots.h).
//
// Head columns are kept in pairs: where a rotation pairs m with m + half, the rows of
// W_q, W_k, W_v (and the columns of W_o) are interleaved when they are loaded.
#include <math.h>

#include <algorithm>

#include "../kernels/conv_norm.h"
#include "../kernels/moe.h"
#include "../kernels/paged_attn.h"
#include "paged_decoder.h"

namespace ffmi {

namespace {

// what a mixer's type fixes
struct MixerType {
  const char *name;
  bool norm, bias, halves, turn_values, sink, learned_sink, yarn;
};
constexpr MixerType kMixers[] = {
    // norm, bias, halves, turn_values, sink, learned_sink, yarn
    {"attention", true, false, true, true, true, true, false},
    {"attention_2", false, true, false, false, true, false, true},
    {"attention_3", true, false, true, false, false, false, false},
};

struct NomutarLayer {
  const MixerType *type = nullptr;
  int heads = 0, groups = 0, dim = 0, vdim = 0, window = 0;
  float scale = 0.f, cap = 0.f;
  int rot = 0;
  float rot_mult = 1.f;
  double rot_base = 1.0;
  std::vector<double> freq;  // turns per position
  // feed-forward: dense (ff) or experts
  int ff = 0, experts = 0, top = 0, eff = 0, sff = 0;
  // padded sizes: per-head columns of the products (dg, vg) and of the caches (dp,
  // vp), first product, attention output, feed-forwards, router; units (dense or the
  // shared expert's) beside the attention output in the layer's last product
  int dg = 0, vg = 0, dp = 0, vp = 0, nq = 0, na = 0, fp = 0, efp = 0, gate_col = 0, nr = 0;
  void *win = nullptr, *wout = nullptr, *wgu = nullptr, *wrouter = nullptr;
  void *egu = nullptr, *edown = nullptr;
  float *norm = nullptr, *bias = nullptr, *norms = nullptr, *sink = nullptr, *conv = nullptr, *rbias = nullptr;
  double *dfreq = nullptr, *dvfreq = nullptr;
};

struct NomutarRun {  // one pass through a layer
  int layer = 0;
  void *kc = nullptr, *vc = nullptr;  // [pages][groups] blocks (kernels/paged_attn.h)
  float *carry = nullptr;             // [slots][2][taps - 1][Wp]
};

constexpr double kTwoPi = 6.283185307179586476925286766559;
constexpr float kLog2e = 1.4426950408889634f;

struct Nomutar : public PagedDecoder {
  std::vector<NomutarLayer> layers;
  std::vector<NomutarRun> runs;
  EmbedPairs em;
  float mult = 1.f;
  int groups = 1, taps = 0;
  bool rows_form = false;  // some layer's attention has no MFMA form
  int max_slots = 0;
  // activations: second residual buffer, mixer input, rows for the experts
  float *x2 = nullptr, *xs[2] = {}, *rms = nullptr;
  void *c = nullptr, *q = nullptr, *cat = nullptr;
  uint16_t *hrow = nullptr;
  float *slabs = nullptr, *ml = nullptr;

  // ---- configuration ----
  ffmi_status configure_rotation(const Json &r, const std::string &at, NomutarLayer *L) {
    if (!r.get("base", &L->rot_base) || !r.get("dims", &L->rot) || L->rot_base <= 0 || L->rot < 0 ||
        L->rot % 2 || L->rot > L->dim)
      return bad(at);
    std::vector<double> f;
    for (int i = 0; i < L->rot / 2; ++i) f.push_back(pow(L->rot_base, -2.0 * i / L->rot));
    const Json *s = r.find("scaling");
    if (s && !s->is_null()) {
      double factor = 1, original = 1;
      if (!s->get("factor", &factor) || !s->get("original", &original) || factor <= 0 || original <= 0)
        return bad(at + ".scaling");
      if (L->type->yarn) {
        double fast = 0, slow = 0;
        if (!s->get("fast", &fast) || !s->get("slow", &slow) || fast <= 0 || slow <= 0 || L->rot_base == 1.0)
          return bad(at + ".scaling");
        const auto dim_of = [&](double turns) {
          return L->rot * log(original / (kTwoPi * turns)) / (2.0 * log(L->rot_base));
        };
        const double lo = std::max(floor(dim_of(fast)), 0.0), hi = std::min(ceil(dim_of(slow)), L->rot - 1.0);
        for (size_t i = 0; i < f.size(); ++i) {
          const double ramp = std::min(1.0, std::max(0.0, ((double)i - lo) / std::max(hi - lo, 0.001)));
          f[i] = f[i] / factor * ramp + f[i] * (1.0 - ramp);
        }
        L->rot_mult = (float)(0.1 * log(factor) + 1.0);
      } else {
        double low = 0, high = 0;
        if (!s->get("low", &low) || !s->get("high", &high) || low <= 0 || high < low) return bad(at + ".scaling");
        for (double &v : f) {
          const double wave = kTwoPi / v;
          if (wave < original / high) continue;
          if (wave > original / low) {
            v /= factor;
            continue;
          }
          const double t = high > low ? (original / wave - low) / (high - low) : 1.0;
          v = (1.0 - t) * v / factor + t * v;
        }
      }
    }
    for (double v : f) L->freq.push_back(v / kTwoPi);
    return FFMI_OK;
  }
  ffmi_status configure_ff(const Json &f, const std::string &at, NomutarLayer *L) {
    const std::string kind = f.text("kind");
    if (kind == "dense") return f.get("ff", &L->ff) && L->ff > 0 ? FFMI_OK : bad(at);
    if (kind != "moe") return bad(at + ".kind '" + kind + "'");
    const Json *e = f.find("expert"), *r = f.find("router"), *s = f.find("shared");
    if (!e || !e->get("ff", &L->eff) || L->eff <= 0) return bad(at + ".expert");
    if (!r || !r->get("experts", &L->experts) || !r->get("top", &L->top) || L->experts < 1 ||
        L->experts > kMoeMaxExperts || L->top < 1 || L->top > std::min(L->experts, kMoeMaxTop))
      return bad(at + ".router");
    if (s && !s->is_null() && (!s->get("ff", &L->sff) || L->sff <= 0)) return bad(at + ".shared");
    return FFMI_OK;
  }
  ffmi_status configure(const Json &cf) override {
    FFMI_TRY(configure_common(cf));
    const Json *ls = cf.find("layers"), *e = cf.find("embedding"), *cn = cf.find("canon"), *lp = cf.find("loop");
    const Json *gr = cf.find("norm")->find("groups");
    if (gr && !gr->is_null() && (!cf.find("norm")->get("groups", &groups) || groups < 1 || W % groups))
      return bad("norm.groups");
    if (!cf.get("residual_mult", &mult)) return bad("residual_mult");
    if (!cn || !cn->get("taps", &taps) || taps < 1) return bad("canon.taps");
    const Json *cap = cf.find("logit_softcap");
    if (cap && !cap->is_null() && (!cf.get("logit_softcap", &logit_cap) || logit_cap <= 0))
      return bad("logit_softcap");
    if (e && !e->is_null()) {
      if (!e->get("scale", &em.scale)) return bad("embedding.scale");
      const Json *b = e->find("bigram");
      double mp = 0, mc = 0;
      if (b && !b->is_null()) {
        if (!b->get("buckets", &em.buckets) || !b->get("mul_prev", &mp) || !b->get("mul_cur", &mc) ||
            em.buckets < 1 || mp < 0 || mc < 0 || mp != floor(mp) || mc != floor(mc) || (mp + mc) * V > 9e18)
          return bad("embedding.bigram");
        em.mul_prev = (int64_t)mp, em.mul_cur = (int64_t)mc;
      }
    }
    if (!ls || ls->type != Json::ARR || ls->arr.empty()) return bad("layers");
    for (size_t i = 0; i < ls->arr.size(); ++i) {
      const Json &lj = ls->arr[i];
      const std::string at = "layers[" + std::to_string(i) + "]", type = lj.text("type");
      const Json *m = lj.find("mixer"), *f = lj.find("mlp");
      NomutarLayer L;
      for (const MixerType &t : kMixers)
        if (type == t.name) L.type = &t;
      if (!L.type) return bad(at + ".type '" + type + "'");
      if (!m || !m->get("heads", &L.heads) || !m->get("kv_heads", &L.groups) || !m->get("dim", &L.dim) ||
          !m->get("vdim", &L.vdim) || !m->get("scale", &L.scale) || L.heads <= 0 || L.dim <= 0 || L.vdim <= 0 ||
          L.groups <= 0 || L.heads % L.groups || (L.type->turn_values && L.vdim % 2))
        return bad(at + ".mixer");
      const Json *mask = m->find("mask"), *sc = m->find("softcap"), *rot = m->find("rot");
      if (mask && !mask->is_null() && (!mask->get("size", &L.window) || L.window < 1)) return bad(at + ".mixer.mask");
      if (sc && !sc->is_null() && (!m->get("softcap", &L.cap) || L.cap <= 0)) return bad(at + ".mixer.softcap");
      if (!rot) return bad(at + ".mixer.rot");
      FFMI_TRY(configure_rotation(*rot, at + ".mixer.rot", &L));
      if (f && !f->is_null()) FFMI_TRY(configure_ff(*f, at + ".mlp", &L));
      layers.push_back(L);
    }
    const int n = (int)layers.size();
    int start = 0, stop = 0, times = 1;
    if (lp && !lp->is_null() &&
        (!lp->get("start", &start) || !lp->get("stop", &stop) || !lp->get("times", &times) || start < 0 ||
         stop < start || stop > n || times < 1))
      return bad("loop");
    for (int i = 0; i < start; ++i) runs.push_back({i});
    for (int k = 0; k < times; ++k)
      for (int i = start; i < stop; ++i) runs.push_back({i});
    for (int i = stop; i < n; ++i) runs.push_back({i});
    num_layers = (int)runs.size();
    recurrent = true;
    return FFMI_OK;
  }

  // ---- buffers and weights ----
  ffmi_status init_layers() override {
    size_t qw = 32, cw = 32;
    double wbytes = 0;
    int min_groups = 1 << 30;
    std::vector<RowShape> shapes;
    std::vector<std::pair<int, int>> gemms;
    FFMI_CHECK((taps <= 4 && Wp <= 8192) || (size_t)taps * Wp * 4 <= 150 * 1024, FFMI_ERR_UNSUPPORTED);
    for (NomutarLayer &L : layers) {
      const int H = L.heads, G = L.groups;
      L.dg = up(L.dim, 32), L.vg = up(L.vdim, 32), L.fp = up(L.ff + L.sff, 32);
      FFMI_CHECK(L.dg <= kAttnRowsMax && L.vg <= kAttnRowsMax, FFMI_ERR_UNSUPPORTED);
      L.dp = L.dg, L.vp = L.vg;
      if (!f32 && attn_width(L.dim) && attn_width(L.vdim)) L.dp = attn_width(L.dim), L.vp = attn_width(L.vdim);
      else rows_form = true;
      L.nq = (H + G) * L.dg + G * L.vg, L.na = H * L.vg;
      shapes.push_back(RowShape{H / G, G, kAttnTiles, true, L.window});
      min_groups = std::min(min_groups, G);
      qw = std::max(qw, (size_t)H * L.dp), cw = std::max(cw, (size_t)L.na + L.fp);
      gemms.insert(gemms.end(), {{L.nq, Wp}, {Wp, L.na + L.fp}});
      wbytes += 2.0 * ((double)L.nq * Wp + ((double)L.na + 3.0 * L.fp) * Wp);
      if (L.ff && f32) gemms.push_back({2 * L.fp, Wp});
      if (L.ff && !f32)
        for (int t = 16; t <= Tm; t += 16)
          ws_bytes = std::max(ws_bytes, gemm_bf16_swiglu_workspace_bytes(t, L.fp, Wp));
      if (!L.experts) continue;
      L.efp = up(L.eff, 32), L.gate_col = up(L.experts, 16);
      L.nr = up(L.gate_col + 1, 32);
      gemms.push_back({L.nr, Wp});
      wbytes += 6.0 * Wp * L.experts * L.efp;
      need_experts(sizes(L, 0), L.efp);
    }
    // 16-row slots for the splits of a step whose blocks do not fill the chip
    max_slots = rows_form ? 0 : 512 * kAttnTiles / min_groups;
    FFMI_TRY(init_step(shapes, max_slots, gemms, wbytes));
    FFMI_TRY(alloc_zero(&x2, (size_t)Tm * Wp * 4));
    xs[0] = x, xs[1] = x2;
    FFMI_TRY(alloc_zero(&rms, (size_t)Tm * groups * 4));
    FFMI_TRY(alloc_zero(&c, (size_t)Tm * Wp * es()));
    FFMI_TRY(alloc_zero(&q, (size_t)Tm * qw * es()));
    FFMI_TRY(alloc_zero(&cat, (size_t)Tm * cw * es()));
    if (moe.num_slots && !f32) FFMI_TRY(alloc_zero(&hrow, (size_t)Tm * Wp * 2));
    FFMI_TRY(alloc_experts());
    size_t part = 0, rows = 0;
    for (NomutarRun &r : runs) {
      const NomutarLayer &L = layers[r.layer];
      const size_t cells = (size_t)cache_pages() * L.groups * kPageTokens;
      FFMI_TRY(alloc_zero(&r.kc, cells * L.dp * es()));
      FFMI_TRY(alloc_zero(&r.vc, cells * L.vp * es()));
      FFMI_TRY(alloc_zero(&r.carry, (size_t)o.max_requests * 2 * (taps - 1) * Wp * 4));
      rows = std::max(rows, (size_t)max_slots * L.groups * 16);
      part = std::max(part, (size_t)max_slots * L.groups * 16 * L.vp);
    }
    if (part) {
      FFMI_TRY(alloc(&slabs, part * 4));
      FFMI_TRY(alloc(&ml, rows * 2 * 4));
    }
    if (em.buckets) {
      uint16_t *t = nullptr;
      FFMI_TRY(table(&t, "bigram", em.buckets + 1));
      em.pairs = t;
    }
    for (size_t i = 0; i < layers.size(); ++i) FFMI_TRY(load_layer("l" + std::to_string(i) + ".", layers[i]));
    return FFMI_OK;
  }
  MoeSizes sizes(const NomutarLayer &L, int T) const {
    MoeSizes n;
    n.T = T, n.experts = L.experts, n.top = L.top, n.shared = L.sff > 0, n.gate_col = L.gate_col;
    return n;
  }
  // rows of the first product's weight: `heads` of n rows, padded to np
  ffmi_status in_rows(NomutarLayer &L, const std::string &name, int heads, int n, int np, int pairs, int row0) {
    FFMI_TRY(raw(name, {(long)heads * n, W}));
    PackSpec p = spec(heads, n, np, 1, W, Wp);
    p.row_pairs = pairs;
    return pack_rows(p, W, L.win, row0, L.nq);
  }
  // a vector with one value per such row
  ffmi_status head_vec(float *dst, const std::string &name, int heads, int n, int np, int pairs) {
    FFMI_TRY(raw(name, {(long)heads * n}, 1));
    PackSpec p = spec(heads, 1, 1, 1, n, np);
    p.col_pairs = pairs;
    FFMI_HIP(launch_pack_f32(raw_tensor(), n, p, dst, stream));
    return FFMI_OK;
  }
  ffmi_status load_layer(const std::string &p, NomutarLayer &L) {
    const std::string m = p + "mix.", f = p + "mlp.";
    const int H = L.heads, G = L.groups, off_k = H * L.dg, off_v = off_k + G * L.dg;
    const int pairs = L.type->halves ? L.rot : 0, vpairs = L.type->halves && L.type->turn_values ? L.vdim : 0;
    FFMI_TRY(vec(&L.norm, p + "norm1", 1, W, Wp));
    FFMI_TRY(alloc(&L.conv, (size_t)taps * Wp * 4));
    FFMI_TRY(raw(p + "canon1", {W, taps}));
    FFMI_HIP(launch_pack_f32(raw_tensor(), taps, spec(1, taps, taps, 1, W, Wp, true), L.conv, stream));
    FFMI_TRY(alloc(&L.win, (size_t)L.nq * Wp * es()));
    FFMI_TRY(in_rows(L, m + "q", H, L.dim, L.dg, pairs, 0));
    FFMI_TRY(in_rows(L, m + "k", G, L.dim, L.dg, pairs, off_k));
    FFMI_TRY(in_rows(L, m + "v", G, L.vdim, L.vg, vpairs, off_v));
    if (L.type->bias) {
      FFMI_TRY(alloc(&L.bias, (size_t)L.nq * 4));
      FFMI_TRY(head_vec(L.bias, m + "q.b", H, L.dim, L.dg, pairs));
      FFMI_TRY(head_vec(L.bias + off_k, m + "k.b", G, L.dim, L.dg, pairs));
      FFMI_TRY(head_vec(L.bias + off_v, m + "v.b", G, L.vdim, L.vg, vpairs));
    }
    if (L.type->norm) {
      FFMI_TRY(alloc(&L.norms, (size_t)(H + G) * L.dg * 4));
      FFMI_TRY(head_vec(L.norms, m + "q.norm", H, L.dim, L.dg, pairs));
      FFMI_TRY(head_vec(L.norms + off_k, m + "k.norm", G, L.dim, L.dg, pairs));
    }
    FFMI_TRY(upload(&L.dfreq, L.freq));
    if (L.type->turn_values) {
      std::vector<double> v(L.vg / 2, 0.0);
      for (int i = 0; i < L.vdim / 2; ++i) v[i] = pow(L.rot_base, -2.0 * i / L.vdim) / kTwoPi;
      FFMI_TRY(upload(&L.dvfreq, v));
    }
    if (L.type->sink) {
      std::vector<float> s(H, 0.f);
      if (L.type->learned_sink) {
        FFMI_TRY(host_vec(&s, m + "sink", H));
        if (!f32)
          for (float &v : s) v *= kLog2e;
      }
      FFMI_TRY(upload(&L.sink, s));
    }
    // one product for the sublayers' outputs: W_o and a W_down that every token takes
    // (dense or the shared expert's) side by side
    FFMI_TRY(alloc(&L.wout, (size_t)Wp * (L.na + L.fp) * es()));
    PackSpec so = spec(1, W, Wp, H, L.vdim, L.vg);
    so.col_pairs = vpairs, so.kt = (L.na + L.fp) / 32;
    FFMI_TRY(raw(m + "o", {W, (long)H * L.vdim}));
    FFMI_TRY(pack_rows(so, H * L.vdim, L.wout, 0, Wp));
    if (L.fp) {
      const std::string d = L.ff ? f : f + "shared.";
      const int ff = L.ff + L.sff;  // (one of the two)
      PackSpec sd = spec(1, W, Wp, 1, ff, L.fp);
      sd.k0 = L.na / 32, sd.kt = so.kt;
      FFMI_TRY(raw(d + "down", {W, ff}));
      FFMI_TRY(pack_rows(sd, ff, L.wout, 0, Wp));
      FFMI_TRY(alloc(&L.wgu, (size_t)2 * L.fp * Wp * es()));
      FFMI_TRY(gate_up(L.wgu, d, ff, L.fp));
    }
    return L.experts ? load_experts(f, L) : FFMI_OK;
  }
  ffmi_status load_experts(const std::string &f, NomutarLayer &L) {
    FFMI_TRY(alloc_zero(&L.wrouter, (size_t)L.nr * Wp * es()));
    FFMI_TRY(raw(f + "router", {L.experts, W}));
    FFMI_TRY(pack_rows(spec(1, L.experts, L.gate_col, 1, W, Wp), W, L.wrouter, 0, L.nr));
    FFMI_TRY(vec(&L.rbias, f + "router.b", 1, L.experts, L.gate_col));
    FFMI_TRY(expert_matrices(f, L.experts, L.eff, L.efp, &L.egu, &L.edown));
    if (!L.sff) return FFMI_OK;
    FFMI_TRY(raw(f + "shared.sg", {1, W}));
    return pack_rows(spec(1, 1, 16, 1, W, Wp), W, L.wrouter, L.gate_col, L.nr);
  }

  // ---- one step ----
  ffmi_status attention(const NomutarLayer &L, const NomutarRun &r) {
    const int H = L.heads, G = L.groups;
    AttnPrep p;
    FFMI_TRY(gemm_sum(c, L.win, L.nq, Wp, &p.y));
    p.bias = L.bias, p.norms = L.norms, p.eps = eps;
    p.freq = L.dfreq, p.vfreq = L.dvfreq, p.rot = L.rot, p.rot_mult = L.rot_mult;
    p.q = q, p.kc = r.kc, p.vc = r.vc;
    p.H = H, p.G = G, p.dim = L.dim, p.dg = L.dg, p.dp = L.dp, p.vg = L.vg, p.vp = L.vp;
    const PagedLists &pl = step.lists(H / G, G, L.window);
    const bool rows = f32 || !attn_width(L.dim) || !attn_width(L.vdim);
    // decoding and short portions: in the attention's launch
    const bool fused = !rows && pl.row_tiles == 1;
    if (!fused) FFMI_HIP(launch_rotary_prep(step.dev, step.off_tokens, step.T, p, f32, stream));
    AttnArgs a;
    a.q = q, a.kc = r.kc, a.vc = r.vc, a.o = cat, a.ldo = L.na + L.fp;
    a.H = H, a.G = G, a.dp = L.dp, a.vg = L.vg, a.vp = L.vp;
    a.scale = f32 ? L.scale : L.scale * kLog2e;
    if (L.cap > 0.f) {
      a.cap_in = f32 ? L.scale / L.cap : 2.f * kLog2e * L.scale / L.cap;
      a.cap_out = f32 ? L.cap : L.cap * kLog2e;
    }
    if (L.window) a.window = L.window;
    a.sink = L.sink, a.vfreq = L.dvfreq, a.off_tokens = step.off_tokens;
    if (rows) FFMI_HIP(launch_rotary_attn_rows(step.dev, pl, a, f32, stream));
    else FFMI_HIP(launch_rotary_attn(step.dev, pl, a, slabs, ml, stream, fused ? &p : nullptr, step.T));
    return FFMI_OK;
  }
  // the columns after the attention output
  void *units_of(const NomutarLayer &L) {
    return (char *)cat + (f32 ? (size_t)L.na * 4 : (size_t)L.na / 32 * 512 * 2);
  }
  ffmi_status dense(const NomutarLayer &L) {
    const int T = step.T, ld = L.na + L.fp;
    if (f32) {
      FFMI_HIP(launch_gemm_f32((const float *)h, (const float *)L.wgu, ws, T, 2 * L.fp, Wp, stream));
      FFMI_HIP(launch_swiglu_f32(ws, (float *)units_of(L), T, L.fp, ld, stream));
    } else {
      FFMI_HIP(launch_gemm_bf16_swiglu((const uint16_t *)h, (const uint16_t *)L.wgu,
                                       (uint16_t *)units_of(L), ws, ws_bytes, T, L.fp, Wp,
                                       FFMI_X_PACKED | FFMI_Y_PACKED | wstream, ld, stream));
    }
    return FFMI_OK;
  }
  ffmi_status experts(const NomutarLayer &L) {
    const MoeSizes n = sizes(L, step.T);
    Partials z;
    FFMI_TRY(gemm_sum(h, L.wrouter, L.nr, Wp, &z));
    FFMI_HIP(launch_moe_route(z, L.rbias, n, moe.lists, stream));
    MoeGemm a;
    const MoeLists &l = moe.lists;
    a.experts = L.experts, a.slot_token = l.slot_token, a.tiles = l.tiles, a.num_tiles = l.num_tiles;
    a.gate = l.gate;
    const void *rows = f32 ? h : hrow;
    a.g[0] = {rows, L.egu, moe.units, L.efp, Wp, L.efp, (size_t)2 * L.efp * Wp};
    a.g[1] = {rows, L.wgu, units_of(L), L.fp, Wp, L.na + L.fp, 0};
    FFMI_HIP(launch_moe_gemm(a, n, true, f32, wstream != 0, stream));
    a.g[0] = {moe.units, L.edown, moe.rows, Wp, L.efp, 0, (size_t)L.efp * Wp};
    FFMI_HIP(launch_moe_gemm(a, n, false, f32, wstream != 0, stream));
    return FFMI_OK;
  }
  // x of the sums that layer `prev` (null: none) left, for the norm `w`
  ConvNorm sum_norm(const NomutarLayer *prev, const Partials &y, const float *w) {
    ConvNorm n;
    n.H = Wp, n.n = W, n.groups = groups, n.eps = eps, n.mult = mult, n.w = w, n.x_in = xs[0], n.inv = rms;
    if (prev) n.y = y;
    if (prev && prev->experts) {
      n.rows = moe.rows, n.rows_f32 = f32, n.at = moe.lists.at, n.wt = moe.lists.wt, n.top = prev->top;
    }
    return n;
  }
  const NomutarLayer *last = nullptr;  // the layer whose sums are not in x yet
  Partials last_y;

  ffmi_status run_layers() override {
    const int T = step.T;
    xs[0] = x2, xs[1] = x;
    em.embed = embed;
    last = nullptr;
    for (size_t i = 0; i < runs.size(); ++i) {
      const NomutarRun &r = runs[i];
      const NomutarLayer &L = layers[r.layer];
      ConvNorm n = sum_norm(last, last_y, L.norm);
      n.x = xs[1], n.conv = L.conv, n.taps = taps, n.carry = r.carry;
      if (f32) {
        n.cf = (float *)c;
        if (L.ff || L.experts) n.hf = (float *)h;
      } else {
        n.cb = (uint16_t *)c;
        if (L.ff || L.experts) n.hb = (uint16_t *)h;
        if (L.experts) n.hrow = hrow;
      }
      FFMI_HIP(launch_conv_norm(i ? step.dev : step.host, step.dev, step.bytes, step.off_tokens, n,
                                i ? nullptr : &em, T, stream));
      std::swap(xs[0], xs[1]);
      if (i) FFMI_TRY(capture((int)i - 1, xs[0]));
      FFMI_TRY(attention(L, r));
      if (L.ff) FFMI_TRY(dense(L));
      if (L.experts) FFMI_TRY(experts(L));
      FFMI_TRY(gemm_sum(cat, L.wout, Wp, L.na + L.fp, &last_y));
      last = &L;
    }
    if (capturing()) {
      ConvNorm n = sum_norm(last, last_y, nullptr);
      n.x = xs[1];
      FFMI_HIP(launch_conv_norm(step.dev, nullptr, 0, step.off_tokens, n, nullptr, T, stream));
      FFMI_TRY(capture(num_layers - 1, n.x));
    }
    return FFMI_OK;
  }
  ffmi_status output_rows() override {
    ConvNorm n = sum_norm(last, last_y, final_norm);
    if (f32) n.hf = (float *)h;
    else n.hb = (uint16_t *)h;
    FFMI_HIP(launch_conv_norm_rows(step.dev, step.off_tokens, step.off_rows, n, step.T, step.R, stream));
    return FFMI_OK;
  }
};

ffmi_status create_nomutar(const Json &config, const ffmi_model_opts *o, ffmi_model **out) {
  return PagedDecoder::create(new Nomutar(), config, o, out);
}
const ModelRegistrar g_registrar("Nomutar", create_nomutar);

}  // namespace

}  // namespace ffmi
