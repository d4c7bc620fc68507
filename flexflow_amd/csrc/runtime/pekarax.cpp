// pekarax.cpp -- Pekarax: a post-norm decoder whose layers mix tokens by matrix memories
// (gated or delta rule) or by softmax attention beside a normalised matrix memory, each
// followed by a mixture of experts.
//
//   x = embed[token]
//   per layer:  x = norm1(alpha x + mixer(x));  x = norm2(alpha x + ff(x))  (ff optional)
//               norms x / rms(x) * (1 + w)
//   gla, channel_delta:  kernels/memory.h, rules gated and delta
//   parallel:   ls attention(x) + rs memory(x), rule normed; attention: q, k, v through a
//               short convolution over time, q and k rotated by halves and put over their
//               rms per head, grouped heads, scores q . k * scale over all keys so far
//   ff:         `top` of many clamped gated units chosen by corrected softmax scores within
//               the best groups; the last outputs of the router stand for the row itself
//   logits = head norm(x)
//
// 32-bit in either precision: residual stream, norms, convolutions and their carried rows,
// angles, scores, softmax, router scores, and everything of a recurrence but the products
// it reads.  bf16 model: products on bf16 operands with fp32 accumulation; long portions
// of a memory take bf16 operands besides the state and the solved values, which go in as
// two terms (memory_chunks.hip).  fp32 model (full_precision): the same graph on fp32
// operands, memories token by token.
// Attention keeps keys and values in pages shared by all requests (page_pool.h); states,
// maxima and carried rows lie in the request's slot (state_slots.h).
#include <math.h>

#include <algorithm>

#include "../kernels/conv_rows.h"
#include "../kernels/memory.h"
#include "../kernels/moe.h"
#include "../kernels/paged_attn.h"
#include "paged_decoder.h"

namespace ffmi {

namespace {

constexpr double kTwoPi = 6.283185307179586476925286766559;
constexpr float kLog2e = 1.4426950408889634f;

struct PekaraxAttention {
  int heads = 0, groups = 0, dim = 0, vdim = 0, rot = 0, taps = 0;
  float scale = 0.f, mult = 1.f;
  double rot_base = 1.0;
  // padded: per-head columns of the products (dg, vg) and of the caches (dp, vp)
  int dg = 0, vg = 0, dp = 0, vp = 0, cols = 0;
  double *freq = nullptr;
  float *conv = nullptr, *carry = nullptr;
  void *kc = nullptr, *vc = nullptr;  // [pages][groups] blocks (kernels/paged_attn.h)
};

struct PekaraxLayer {
  bool attention = false;
  PekaraxAttention att;
  Memory mem;  // a step's fields (T, y, z, out) aside
  float mem_mult = 1.f;
  int low = 0;  // columns of the second product's input, decay | gate (0: none)
  int nz = 0;   // its outputs
  // feed-forward
  int experts = 0, top = 0, identity = 0, eff = 0;
  float limit = 0.f;
  MoeScores scores;
  // padded sizes: first product, output product's input, experts' units, router
  int nq = 0, na = 0, no = 0, efp = 0, nr = 0;
  void *win = nullptr, *wout = nullptr, *wlow = nullptr, *wrouter = nullptr, *egu = nullptr, *edown = nullptr;
  float *norm1 = nullptr, *norm2 = nullptr;
};

struct Pekarax : public PagedDecoder {
  std::vector<PekaraxLayer> layers;
  float alpha = 1.f;
  bool rows_form = false;  // some layer's attention has no MFMA form
  int max_slots = 0;
  void *q = nullptr, *cat = nullptr;
  uint16_t *hrow = nullptr, *low = nullptr;
  float *crows = nullptr;  // an attention's convolved product
  float *zs = nullptr, *slabs = nullptr, *ml = nullptr;
  size_t zs_bytes = 0;
  MemoryScratch scratch;

  // ---- configuration ----
  static bool sizes_of(const Json *m, int *heads, int *dim, int *vdim) {
    return m && m->get("heads", heads) && m->get("dim", dim) && m->get("vdim", vdim) && *heads > 0 && *dim > 0 &&
           *vdim > 0;
  }
  ffmi_status configure_attention(const Json *m, const std::string &at, PekaraxAttention *A) {
    if (!sizes_of(m, &A->heads, &A->dim, &A->vdim) || !m->get("kv_heads", &A->groups) || A->groups <= 0 ||
        A->heads % A->groups || !m->get("scale", &A->scale))
      return bad(at);
    if (!m->get("conv", &A->taps) || A->taps < 1) return bad(at + ".conv");
    const Json *r = m->find("rot");
    if (!r || !r->get("base", &A->rot_base) || !r->get("dims", &A->rot) || A->rot_base <= 0 || A->rot < 0 ||
        A->rot % 2 || A->rot > A->dim)
      return bad(at + ".rot");
    return FFMI_OK;
  }
  ffmi_status configure_mixer(const std::string &type, const Json *m, const std::string &at, PekaraxLayer *L) {
    Memory &M = L->mem;
    if (type == "parallel") {
      L->attention = true;
      if (!m || !m->get("left_scale", &L->att.mult) || !m->get("right_scale", &L->mem_mult)) return bad(at);
      FFMI_TRY(configure_attention(m->find("left"), at + ".left", &L->att));
      const Json *r = m->find("right");
      if (!sizes_of(r, &M.H, &M.dim, &M.vdim) || !r->get("gate_cap", &M.cap) || M.cap <= 0) return bad(at + ".right");
      M.rule = kMemoryNormed, M.G = M.H, M.norm_heads = true;
    } else if (type == "gla") {
      float tau = 0;
      if (!sizes_of(m, &M.H, &M.dim, &M.vdim) || !m->get("tau", &tau) || tau <= 0) return bad(at);
      M.rule = kMemoryGated, M.G = M.H, M.inv_tau = 1.f / tau, M.gate_silu = true;
    } else {
      if (!sizes_of(m, &M.H, &M.dim, &M.vdim) || !m->get("kv_heads", &M.G) || M.G <= 0 || M.H % M.G) return bad(at);
      if (!m->get("conv", &M.taps) || M.taps < 1) return bad(at + ".conv");
      M.rule = kMemoryDelta, M.silu = M.unit = true;
    }
    M.q_scale = (float)(1.0 / sqrt((double)M.dim));
    return FFMI_OK;
  }
  ffmi_status configure_experts(const Json &f, const std::string &at, PekaraxLayer *L) {
    if (f.text("kind") != "moe") return bad(at + ".kind '" + f.text("kind") + "'");
    const Json *e = f.find("expert"), *r = f.find("router");
    if (!e || !e->get("ff", &L->eff) || L->eff <= 0 || !e->get("limit", &L->limit) || L->limit <= 0)
      return bad(at + ".expert");
    if (!r || !r->get("experts", &L->experts) || !r->get("top", &L->top) || L->experts < 1 || L->top < 1)
      return bad(at + ".router");
    const Json *id = r->find("identity"), *sc = r->find("scale"), *g = r->find("groups");
    if (id && !id->is_null() && (!r->get("identity", &L->identity) || L->identity < 0)) return bad(at + ".router.identity");
    if (sc && !sc->is_null() && !r->get("scale", &L->scores.scale)) return bad(at + ".router.scale");
    const int outs = L->experts + L->identity;
    if (g && !g->is_null() &&
        (!g->get("count", &L->scores.groups) || !g->get("keep", &L->scores.keep) || L->scores.groups < 1 ||
         outs % L->scores.groups || L->scores.keep < 1 || L->scores.keep > L->scores.groups))
      return bad(at + ".router.groups");
    if (outs > kMoeMaxExperts || L->top > std::min(kMoeMaxTop, outs / L->scores.groups * L->scores.keep))
      return bad(at + ".router");
    return FFMI_OK;
  }
  ffmi_status configure(const Json &c) override {
    FFMI_TRY(configure_common(c));
    if (!c.get("postln_alpha", &alpha)) return bad("postln_alpha");
    const Json *ls = c.find("layers");
    if (!ls || ls->type != Json::ARR || ls->arr.empty()) return bad("layers");
    for (size_t i = 0; i < ls->arr.size(); ++i) {
      const Json &lj = ls->arr[i];
      const std::string at = "layers[" + std::to_string(i) + "]", type = lj.text("type");
      if (type != "parallel" && type != "gla" && type != "channel_delta") return bad(at + ".type '" + type + "'");
      PekaraxLayer L;
      FFMI_TRY(configure_mixer(type, lj.find("mixer"), at + ".mixer", &L));
      const Json *f = lj.find("mlp");
      if (f && !f->is_null()) FFMI_TRY(configure_experts(*f, at + ".mlp", &L));
      layers.push_back(L);
    }
    num_layers = (int)layers.size();
    recurrent = true;
    return FFMI_OK;
  }

  // ---- buffers and weights ----
  MoeSizes sizes(const PekaraxLayer &L, int T) const {
    MoeSizes n;
    n.T = T, n.experts = L.experts, n.top = L.top, n.identity = L.identity;
    return n;
  }
  bool mfma_form(const PekaraxAttention &A) const { return !f32 && attn_width(A.dim) && attn_width(A.vdim); }
  bool chunk_form(const Memory &M) const { return !f32 && M.dg <= kMemoryMaxChunkDim; }
  // columns of the first product, and what the padded sizes give
  ffmi_status place(const std::string &p, PekaraxLayer &L) {
    PekaraxAttention &A = L.att;
    Memory &M = L.mem;
    int at = 0;
    const auto take = [&at](int n) {
      const int a = at;
      at += up(n, 16);
      return a;
    };
    if (L.attention) {
      A.dg = up(A.dim, 32), A.vg = up(A.vdim, 32), A.dp = A.dg, A.vp = A.vg;
      FFMI_CHECK(A.dg <= kAttnRowsMax && A.vg <= kAttnRowsMax, FFMI_ERR_UNSUPPORTED);
      if (mfma_form(A)) A.dp = attn_width(A.dim), A.vp = attn_width(A.vdim);
      else rows_form = true;
      A.cols = (A.heads + A.groups) * A.dg + A.groups * A.vg;
      take(A.cols);
      L.na = A.heads * A.vg;
    }
    M.dg = up(M.dim, 32), M.vg = up(M.vdim, 32), M.vs = memory_state_columns(M.rule, M.vdim);
    FFMI_CHECK(M.dg <= kMemoryMaxDim && M.vg <= kMemoryMaxVdim, FFMI_ERR_UNSUPPORTED);
    M.col = take(2 * M.G * M.dg + M.H * M.vg);
    if (M.rule != kMemoryDelta) M.col_gate = take(M.H * M.vg);
    if (M.rule == kMemoryNormed) M.col_i = take(M.H), M.col_f = take(M.H);
    if (M.rule != kMemoryNormed) {
      std::vector<long> s;
      FFMI_TRY(shape_of(p + "mix.a1", {M.rule == kMemoryDelta ? M.dim : 16, W}, &s));
      FFMI_CHECK(s.size() == 2 && s[0] > 0 && s[0] <= 1024, FFMI_ERR_UNSUPPORTED);
      M.decay.r = up((int)s[0], 32), M.decay.col = take(M.decay.r);
      L.nz = M.H * M.dg;
    }
    if (M.rule == kMemoryDelta) {
      std::vector<long> s;
      FFMI_TRY(shape_of(p + "mix.g1", {M.vdim, W}, &s));
      FFMI_CHECK(s.size() == 2 && s[0] > 0 && s[0] <= 1024, FFMI_ERR_UNSUPPORTED);
      M.gate.r = up((int)s[0], 32), M.gate.col = take(M.gate.r);  // (beside the decay's)
      M.gate.zcol = L.nz, L.nz += M.H * M.vg;
      M.col_beta = take(M.H);
    }
    L.low = M.decay.r + M.gate.r;
    L.nq = up(at, 32), L.no = L.na + M.H * M.vg;
    M.eps = eps, M.ldo = L.no, M.out_col = L.na;
    L.efp = up(L.eff, 32), L.nr = up(L.experts + L.identity, 32);
    return FFMI_OK;
  }
  ffmi_status init_layers() override {
    size_t qw = 32, cw = 32, lw = 0, rw = 0;
    double wbytes = 0;
    int min_groups = 1 << 30;
    std::vector<RowShape> shapes;
    std::vector<std::pair<int, int>> gemms;
    for (size_t i = 0; i < layers.size(); ++i) {
      PekaraxLayer &L = layers[i];
      FFMI_TRY(place("l" + std::to_string(i) + ".", L));
      if (L.attention) {
        shapes.push_back(RowShape{L.att.heads / L.att.groups, L.att.groups, kAttnTiles, true});
        min_groups = std::min(min_groups, L.att.groups);
        qw = std::max(qw, (size_t)L.att.heads * L.att.dp), rw = std::max(rw, (size_t)L.att.cols);
      }
      cw = std::max(cw, (size_t)L.no);
      gemms.insert(gemms.end(), {{L.nq, Wp}, {Wp, L.no}});
      wbytes += 2.0 * ((double)L.nq + L.no) * Wp;
      if (chunk_form(L.mem) && L.low) {
        lw = std::max(lw, (size_t)L.low);
        zs_bytes = std::max(zs_bytes, sum_bytes(L.nz, L.low));
      }
      if (!L.experts) continue;
      gemms.push_back({L.nr, Wp});
      wbytes += 6.0 * Wp * L.experts * L.efp;
      need_experts(sizes(L, 0), L.efp);
    }
    // 16-row slots for the splits of a step whose blocks do not fill the chip
    max_slots = rows_form || shapes.empty() ? 0 : 512 * kAttnTiles / min_groups;
    FFMI_TRY(init_step(shapes, max_slots, gemms, wbytes));
    FFMI_TRY(alloc_zero(&q, (size_t)Tm * qw * es()));
    FFMI_TRY(alloc_zero(&cat, (size_t)Tm * cw * es()));
    if (rw) FFMI_TRY(alloc(&crows, (size_t)Tm * rw * 4));
    if (lw) {
      FFMI_TRY(alloc_zero(&low, (size_t)Tm * lw * 2));
      FFMI_TRY(alloc(&zs, zs_bytes));
    }
    if (moe.num_slots && !f32) FFMI_TRY(alloc_zero(&hrow, (size_t)Tm * Wp * 2));
    FFMI_TRY(alloc_experts());
    FFMI_TRY(alloc_states());
    for (size_t i = 0; i < layers.size(); ++i) FFMI_TRY(load_layer("l" + std::to_string(i) + ".", layers[i]));
    return FFMI_OK;
  }
  ffmi_status alloc_states() {
    const size_t n = o.max_requests, chunks = memory_chunks_max(Tm, o.max_requests);
    size_t part = 0, rows = 0, keys = 0, solved = 0, pairs = 0, values = 0, last = 0, gates = 0, outs = 0, cols = 0;
    for (PekaraxLayer &L : layers) {
      PekaraxAttention &A = L.att;
      Memory &M = L.mem;
      if (L.attention) {
        const size_t cells = (size_t)cache_pages() * A.groups * kPageTokens;
        FFMI_TRY(alloc_zero(&A.kc, cells * A.dp * es()));
        FFMI_TRY(alloc_zero(&A.vc, cells * A.vp * es()));
        FFMI_TRY(alloc_zero(&A.carry, n * 2 * (A.taps - 1) * A.cols * 4));
        rows = std::max(rows, (size_t)max_slots * A.groups * 16);
        part = std::max(part, (size_t)max_slots * A.groups * 16 * A.vp);
      }
      FFMI_TRY(alloc_zero(&M.state, n * M.H * M.dg * M.vs * 4));
      if (M.rule == kMemoryNormed) FFMI_TRY(alloc_zero(&M.peak, n * 2 * M.H * 4));
      if (M.taps > 1) FFMI_TRY(alloc_zero(&M.carry, n * 2 * (M.taps - 1) * (2 * M.G * M.dg + M.H * M.vg) * 4));
      if (!chunk_form(M)) continue;
      const size_t c = chunks * M.H, wide = memory_chunk_width(M.dg);
      const bool delta = M.rule == kMemoryDelta;
      keys = std::max(keys, c * kMemoryChunk * wide * 2);
      if (delta) {
        cols = std::max(cols, (size_t)Tm * (2 * M.G * M.dg + M.H * M.vg) * 2);
        solved = std::max(solved, c * kMemoryChunk * wide * 2);
        values = std::max(values, c * kMemoryChunk * M.vs * 4);
      }
      pairs = std::max(pairs, c * kMemoryChunk * kMemoryChunk * 2);
      last = std::max(last, c * wide * 4);
      if (M.rule == kMemoryNormed) gates = std::max(gates, (size_t)Tm * M.H * 12);
      outs = std::max(outs, (size_t)Tm * M.H * M.vs * 4);
    }
    if (part) {
      FFMI_TRY(alloc(&slabs, part * 4));
      FFMI_TRY(alloc(&ml, rows * 2 * 4));
    }
    if (!keys) return FFMI_OK;
    FFMI_TRY(alloc(&scratch.qg, keys));
    FFMI_TRY(alloc(&scratch.kd, keys));
    if (solved) {
      FFMI_TRY(alloc(&scratch.rows, cols));
      FFMI_TRY(alloc(&scratch.w, solved));
      FFMI_TRY(alloc(&scratch.u, values));
    }
    FFMI_TRY(alloc(&scratch.p, pairs));
    FFMI_TRY(alloc(&scratch.last, last));
    if (gates) FFMI_TRY(alloc(&scratch.gates, gates));
    return alloc(&scratch.o, outs);
  }
  // rows of the first product's weight: `heads` of n rows, padded to np
  ffmi_status in_rows(PekaraxLayer &L, const std::string &name, int heads, int n, int np, int row0, int pairs = 0) {
    FFMI_TRY(raw(name, {(long)heads * n, W}));
    PackSpec p = spec(heads, n, np, 1, W, Wp);
    p.row_pairs = pairs;
    return pack_rows(p, W, L.win, row0, L.nq);
  }
  // taps of `heads` of n channels as columns [col, col + heads * np) of rows of `cols`
  ffmi_status conv_columns(float *dst, const std::string &name, int taps, int heads, int n, int np, int col, int cols,
                           int pairs = 0) {
    FFMI_TRY(raw(name, {(long)heads * n, taps}));
    PackSpec p = spec(1, taps, taps, heads, n, np, true);
    p.col_pairs = pairs, p.k0 = col / 32, p.kt = cols / 32;
    FFMI_HIP(launch_pack_f32(raw_tensor(), taps, p, dst, stream));
    return FFMI_OK;
  }
  // a norm's weight, stored around zero
  ffmi_status norm_weight(float **dst, const std::string &name) {
    FFMI_TRY(alloc(dst, (size_t)Wp * 4));
    FFMI_TRY(raw(name, {W}));
    PackSpec p = spec(1, 1, 1, 1, W, Wp);
    p.plus = 1.f;
    FFMI_HIP(launch_pack_f32(raw_tensor(), W, p, *dst, stream));
    return FFMI_OK;
  }
  // the narrow second matrix: rows for the tokens in turn, and its block of the product
  // that long steps take
  ffmi_status low_rank(PekaraxLayer &L, const std::string &m, const std::string &first, const std::string &second,
                       int n, int np, LowRank *l, int k0) {
    const int H = L.mem.H;
    std::vector<long> s;
    FFMI_TRY(shape_of(m + first, {L.mem.rule == kMemoryDelta ? n : 16, W}, &s));
    const int r = (int)s[0];
    FFMI_TRY(in_rows(L, m + first, 1, r, l->r, l->col));
    FFMI_TRY(raw(m + second, {(long)H * n, r}));
    void *rows = nullptr;
    FFMI_TRY(alloc_zero(&rows, (size_t)H * n * l->r * es()));
    if (f32) FFMI_HIP(launch_pack_f32(raw_tensor(), r, spec(1, H * n, H * n, 1, r, l->r), (float *)rows, stream));
    else
      FFMI_HIP(hipMemcpy2DAsync(rows, (size_t)l->r * 2, raw_tensor(), (size_t)r * 2, (size_t)r * 2, (size_t)H * n,
                                hipMemcpyDeviceToDevice, stream));
    l->w = rows;
    if (!L.wlow) return FFMI_OK;
    PackSpec p = spec(H, n, np, 1, r, l->r);
    p.k0 = k0 / 32, p.kt = L.low / 32;
    return pack_rows(p, r, L.wlow, l->zcol, L.nz);
  }
  ffmi_status load_attention(const std::string &m, PekaraxLayer &L) {
    PekaraxAttention &A = L.att;
    const int off_k = A.heads * A.dg, off_v = off_k + A.groups * A.dg;
    FFMI_TRY(in_rows(L, m + "q", A.heads, A.dim, A.dg, 0, A.rot));
    FFMI_TRY(in_rows(L, m + "k", A.groups, A.dim, A.dg, off_k, A.rot));
    FFMI_TRY(in_rows(L, m + "v", A.groups, A.vdim, A.vg, off_v));
    FFMI_TRY(alloc(&A.conv, (size_t)A.taps * A.cols * 4));
    FFMI_TRY(conv_columns(A.conv, m + "q.conv", A.taps, A.heads, A.dim, A.dg, 0, A.cols, A.rot));
    FFMI_TRY(conv_columns(A.conv, m + "k.conv", A.taps, A.groups, A.dim, A.dg, off_k, A.cols, A.rot));
    FFMI_TRY(conv_columns(A.conv, m + "v.conv", A.taps, A.groups, A.vdim, A.vg, off_v, A.cols));
    std::vector<double> f;
    for (int i = 0; i < A.rot / 2; ++i) f.push_back(pow(A.rot_base, -2.0 * i / A.rot) / kTwoPi);
    return upload(&A.freq, f);
  }
  ffmi_status load_memory(const std::string &m, PekaraxLayer &L) {
    Memory &M = L.mem;
    const int off_k = M.G * M.dg, off_v = 2 * off_k, cols = off_v + M.H * M.vg;
    FFMI_TRY(in_rows(L, m + "q", M.G, M.dim, M.dg, M.col));
    FFMI_TRY(in_rows(L, m + "k", M.G, M.dim, M.dg, M.col + off_k));
    FFMI_TRY(in_rows(L, m + "v", M.H, M.vdim, M.vg, M.col + off_v));
    if (M.rule != kMemoryDelta) FFMI_TRY(in_rows(L, m + "g", M.H, M.vdim, M.vg, M.col_gate));
    if (M.taps > 0) {
      float *conv = nullptr;
      FFMI_TRY(alloc(&conv, (size_t)M.taps * cols * 4));
      FFMI_TRY(conv_columns(conv, m + "q.conv", M.taps, M.G, M.dim, M.dg, 0, cols));
      FFMI_TRY(conv_columns(conv, m + "k.conv", M.taps, M.G, M.dim, M.dg, off_k, cols));
      FFMI_TRY(conv_columns(conv, m + "v.conv", M.taps, M.H, M.vdim, M.vg, off_v, cols));
      M.conv = conv;
    }
    float *norm = nullptr, *dbias = nullptr, *v = nullptr;
    if (M.norm_heads) {  // (with the mixer's share of the sum)
      std::vector<float> w, wp((size_t)M.H * M.vg, 0.f);
      FFMI_TRY(host_vec(&w, m + "norm", M.H * M.vdim, 1));
      for (int h = 0; h < M.H; ++h)
        for (int c = 0; c < M.vdim; ++c) wp[(size_t)h * M.vg + c] = w[(size_t)h * M.vdim + c] * L.mem_mult;
      FFMI_TRY(upload(&norm, wp));
    } else {
      FFMI_TRY(vec(&norm, m + "norm", 1, M.vdim, M.vg));
    }
    M.norm = norm;
    if (M.rule == kMemoryNormed) {
      FFMI_TRY(in_rows(L, m + "i", 1, M.H, up(M.H, 16), M.col_i));
      FFMI_TRY(in_rows(L, m + "f", 1, M.H, up(M.H, 16), M.col_f));
      FFMI_TRY(vec(&v, m + "i.b", 1, M.H, M.H, 0));
      M.bi = v;
      FFMI_TRY(vec(&v, m + "f.b", 1, M.H, M.H, 1));
      M.bf = v;
      return FFMI_OK;
    }
    if (chunk_form(M)) FFMI_TRY(alloc_zero(&L.wlow, (size_t)L.nz * L.low * 2));
    FFMI_TRY(low_rank(L, m, "a1", "a2", M.dim, M.dg, &M.decay, 0));
    const bool delta = M.rule == kMemoryDelta;
    FFMI_TRY(vec(&dbias, m + (delta ? "dt_bias" : "a2.b"), M.H, M.dim, M.dg, delta ? 0 : 1));
    M.dbias = dbias;
    if (!delta) return FFMI_OK;
    FFMI_TRY(low_rank(L, m, "g1", "g2", M.vdim, M.vg, &M.gate, M.decay.r));
    FFMI_TRY(in_rows(L, m + "b", 1, M.H, up(M.H, 16), M.col_beta));
    std::vector<float> rate;
    FFMI_TRY(host_vec(&rate, m + "A_log", M.H));
    for (float &x : rate) x = (float)exp((double)x);
    FFMI_TRY(upload(&v, rate));
    M.rate = v;
    return FFMI_OK;
  }
  ffmi_status load_layer(const std::string &p, PekaraxLayer &L) {
    const std::string m = p + "mix.", f = p + "mlp.";
    const Memory &M = L.mem;
    FFMI_TRY(norm_weight(&L.norm1, p + "norm1"));
    FFMI_TRY(alloc_zero(&L.win, (size_t)L.nq * Wp * es()));
    if (L.attention) FFMI_TRY(load_attention(m + "left.", L));
    FFMI_TRY(load_memory(L.attention ? m + "right." : m, L));
    // one product for the mixers' outputs, side by side
    FFMI_TRY(alloc(&L.wout, (size_t)Wp * L.no * es()));
    PackSpec so = spec(1, W, Wp, L.att.heads, L.att.vdim, L.att.vg);
    so.kt = L.no / 32;
    if (L.attention) {
      FFMI_TRY(raw(m + "left.o", {W, (long)L.att.heads * L.att.vdim}));
      FFMI_TRY(pack_rows(so, L.att.heads * L.att.vdim, L.wout, 0, Wp));
    }
    so.cols = M.H, so.kb = M.vdim, so.kp = M.vg, so.k0 = L.na / 32;
    FFMI_TRY(raw(m + (L.attention ? "right.o" : "o"), {W, (long)M.H * M.vdim}));
    FFMI_TRY(pack_rows(so, M.H * M.vdim, L.wout, 0, Wp));
    if (!L.experts) return FFMI_OK;
    FFMI_TRY(norm_weight(&L.norm2, p + "norm2"));
    const int outs = L.experts + L.identity;
    float *correction = nullptr;
    FFMI_TRY(linear(&L.wrouter, f + "router", outs, L.nr, 1, W, Wp));
    FFMI_TRY(vec(&correction, f + "correction", 1, outs, outs, 0));
    L.scores.correction = correction;
    return expert_matrices(f, L.experts, L.eff, L.efp, &L.egu, &L.edown);
  }
  ffmi_status load_final() override { return norm_weight(&final_norm, "final.norm"); }

  // ---- one step ----
  const void *rows_in() const { return f32 ? (const void *)x : h; }
  ffmi_status attention(const PekaraxLayer &L, const Partials &y) {
    const PekaraxAttention &A = L.att;
    const int H = A.heads, G = A.groups;
    AttnPrep p;
    p.y = y, p.eps = eps, p.freq = A.freq, p.rot = A.rot, p.unit = true;
    p.conv = A.conv, p.taps = A.taps, p.carry = A.carry, p.off_tokens = step.off_tokens;
    p.q = q, p.kc = A.kc, p.vc = A.vc;
    p.H = H, p.G = G, p.dim = A.dim, p.dg = A.dg, p.dp = A.dp, p.vg = A.vg, p.vp = A.vp;
    const PagedLists &pl = step.lists(H / G, G);
    const bool rows = !mfma_form(A);
    // decoding and short portions: in the attention's launch
    const bool fused = !rows && pl.row_tiles == 1;
    if (!fused) {
      ConvRows c;
      c.u = y, c.T = step.T, c.cols = A.cols, c.taps = A.taps, c.conv = A.conv, c.carry = A.carry, c.hf = crows;
      c.off_tokens = step.off_tokens;
      FFMI_HIP(launch_conv_rows(step.dev, c, stream));
      p.y.p = crows, p.y.S = 1, p.y.NP = A.cols, p.taps = 0;
    }
    if (!fused) FFMI_HIP(launch_rotary_prep(step.dev, step.off_tokens, step.T, p, f32, stream));
    AttnArgs a;
    a.q = q, a.kc = A.kc, a.vc = A.vc, a.o = cat, a.ldo = L.no;
    a.H = H, a.G = G, a.dp = A.dp, a.vg = A.vg, a.vp = A.vp;
    a.scale = f32 ? A.scale : A.scale * kLog2e, a.mult = A.mult, a.off_tokens = step.off_tokens;
    if (rows) FFMI_HIP(launch_rotary_attn_rows(step.dev, pl, a, f32, stream));
    else FFMI_HIP(launch_rotary_attn(step.dev, pl, a, slabs, ml, stream, fused ? &p : nullptr, step.T));
    return FFMI_OK;
  }
  ffmi_status memory(const PekaraxLayer &L, const Partials &y) {
    Memory a = L.mem;
    a.T = step.T, a.y = y, a.out = cat, a.off_tokens = step.off_tokens;
    // short spans token by token, long ones in chunks
    const bool chunks = chunk_form(a);
    const int limit = chunks ? std::max(kShortSpan, a.taps) : BatchConfig::MAX_NUM_TOKENS;
    const bool longs = chunks && step.long_spans, shorts = !chunks || step.short_spans || limit > kShortSpan;
    if (longs && L.low) {
      FFMI_HIP(launch_pack_sums(y, a.decay.col, low, step.T, L.low, stream));
      FFMI_TRY(gemm_sum_to(low, L.wlow, L.nz, L.low, &a.z, zs, zs_bytes));
    }
    bool left = false;
    if (shorts)
      FFMI_HIP(launch_memory_steps(step.dev, step.off_spans, step.num_spans, a, chunks ? &scratch : nullptr, f32,
                                   limit, &left, stream));
    if (longs)
      FFMI_HIP(launch_memory_chunks(step.dev, step.off_spans, step.num_spans, step.num_chunks, a, scratch, limit,
                                    stream));
    if (left || longs) FFMI_HIP(launch_memory_out(step.dev, a, scratch, left ? 0 : limit, stream));
    return FFMI_OK;
  }
  ffmi_status experts(const PekaraxLayer &L) {
    const MoeSizes n = sizes(L, step.T);
    const MoeLists &l = moe.lists;
    Partials z;
    FFMI_TRY(gemm_sum(rows_in(), L.wrouter, L.nr, Wp, &z));
    FFMI_HIP(launch_moe_route_scores(z, L.scores, n, l, stream));
    MoeGemm a;
    a.experts = L.experts, a.slot_token = l.slot_token, a.tiles = l.tiles, a.num_tiles = l.num_tiles;
    a.limit = L.limit;
    a.g[0] = {f32 ? (const void *)x : hrow, L.egu, moe.units, L.efp, Wp, L.efp, (size_t)2 * L.efp * Wp};
    FFMI_HIP(launch_moe_gemm(a, n, true, f32, wstream != 0, stream));
    a.g[0] = {moe.units, L.edown, moe.rows, Wp, L.efp, 0, (size_t)L.efp * Wp};
    FFMI_HIP(launch_moe_gemm(a, n, false, f32, wstream != 0, stream));
    return FFMI_OK;
  }
  // x = norm(alpha x + what the sublayer left)
  SumNorm sum_norm(const float *w) {
    SumNorm n;
    n.alpha = alpha, n.eps = eps, n.w = w, n.x = x, n.T = step.T, n.H = Wp, n.n = W;
    if (!f32) n.hb = (uint16_t *)h;
    return n;
  }
  ffmi_status run_layers() override {
    FFMI_HIP(launch_embed_pos(step.host, step.dev, step.bytes, embed, nullptr, x, f32 ? nullptr : (uint16_t *)h,
                              step.T, Wp, stream));
    for (size_t i = 0; i < layers.size(); ++i) {
      const PekaraxLayer &L = layers[i];
      Partials y;
      FFMI_TRY(gemm_sum(rows_in(), L.win, L.nq, Wp, &y));
      if (L.attention) FFMI_TRY(attention(L, y));
      FFMI_TRY(memory(L, y));
      SumNorm n = sum_norm(L.norm1);
      FFMI_TRY(gemm_sum(cat, L.wout, Wp, L.no, &n.y));
      if (L.experts) n.hrow = hrow;
      FFMI_HIP(launch_sum_norm(n, stream));
      if (L.experts) {
        FFMI_TRY(experts(L));
        n = sum_norm(L.norm2);
        n.rows = moe.rows, n.rows_f32 = f32, n.at = moe.lists.at, n.wt = moe.lists.wt, n.top = L.top;
        if (L.identity) n.own = moe.lists.own;
        FFMI_HIP(launch_sum_norm(n, stream));
      }
      FFMI_TRY(capture_layer((int)i));
    }
    return FFMI_OK;
  }
};

ffmi_status create_pekarax(const Json &config, const ffmi_model_opts *o, ffmi_model **out) {
  return PagedDecoder::create(new Pekarax(), config, o, out);
}
const ModelRegistrar g_registrar("Pekarax", create_pekarax);

}  // namespace

}  // namespace ffmi
