// paged_decoder.h -- what the model families over a paged cache have in common:
// weight loading, the cache pool and the step's metadata, the output product
// and greedy pick, captured decode graphs, tensor capture.  A family gives its
// configuration, its buffers and weights, and the layers of a step.
#pragma once
#include <stdio.h>
#include <string.h>

#include <map>
#include <string>
#include <vector>

#include "../kernels/moe.h"
#include "../kernels/packing.h"
#include "../kernels/residual.h"
#include "json.h"
#include "model.h"
#include "paged_step.h"
#include "safetensors.h"
#include "state_slots.h"

namespace ffmi {

inline int up(int v, int m) { return (v + m - 1) / m * m; }

#define FFMI_TRY(x_)                                      \
  do {                                                    \
    const ffmi_status st_ = (x_);                         \
    if (st_ != FFMI_OK) return st_;                       \
  } while (0)

struct PagedDecoder : public ffmi_model {
  // ---- a family's part ----
  virtual ffmi_status configure(const Json &c) = 0;
  // buffers, cache, layer weights; calls init_step()
  virtual ffmi_status init_layers() = 0;
  // the layers of a step: token rows to the residual stream x
  virtual ffmi_status run_layers() = 0;
  // the output product's rows: h = norm(x) of the step's output rows
  virtual ffmi_status output_rows();
  // "final.norm"
  virtual ffmi_status load_final() { return vec(&final_norm, "final.norm", 1, W, Wp); }

  ffmi_model_opts o{};
  std::string folder;
  int V = 0, W = 0;            // vocab, width
  int P = 0;                   // positions of the position table (0: none)
  int Vp = 0, Wp = 0, Tm = 0;  // padded; batch capacity
  int num_layers = 0;
  float eps = 0.f;
  float logit_cap = 0.f;  // soft cap of the logits (0: none)
  bool f32 = false;
  bool recurrent = false;  // some layer keeps a state per request slot
  float *final_norm = nullptr;
  void *head = nullptr;
  uint16_t *embed = nullptr;
  int wstream = 0;
  // activations every family has: residual stream, fp32 sums, output rows
  float *x = nullptr, *ws = nullptr, *logits = nullptr;
  size_t ws_bytes = 0;
  void *h = nullptr;           // normed rows [Tm][Wp] (bf16: packed tiles)
  int32_t *res_h = nullptr;    // pinned: ids [Tm] | probs [Tm]
  PagePool pool;
  StateSlots states;
  PagedStep step;
  hipStream_t stream = nullptr;

  int token_capacity() const override { return o.max_tokens; }
  int vocab_size() const override { return V; }
  PagePool *page_pool() override { return &pool; }
  ~PagedDecoder() override;

  ffmi_status init();
  static ffmi_status bad(const std::string &what);  // a refused configuration
  // "vocab", "width" and "norm.eps"
  ffmi_status configure_common(const Json &c);

  // ---- memory ----
  ffmi_status alloc_bytes(void **p, size_t bytes);
  template <class T>
  ffmi_status alloc(T **p, size_t bytes) {
    return alloc_bytes((void **)p, bytes);
  }
  // zeroed: padding columns and unwritten cache rows meet zero weights
  template <class T>
  ffmi_status alloc_zero(T **p, size_t bytes) {
    FFMI_TRY(alloc_bytes((void **)p, bytes));
    FFMI_HIP(hipMemsetAsync((void *)*p, 0, bytes, stream));
    return FFMI_OK;
  }
  size_t es() const { return f32 ? 4 : 2; }
  // the page pool, the step's metadata and the buffers above; gemms: the
  // products (N, K) whose fp32 sums pass through ws (ws_bytes: its least size)
  ffmi_status init_step(const std::vector<RowShape> &shapes, int max_slots,
                        const std::vector<std::pair<int, int>> &gemms, double weight_bytes);
  int cache_pages() const { return pool.pages(); }

  // ---- weights ----
  // tensor `name` to tmp as bf16 bits
  ffmi_status raw(const std::string &name, const std::vector<long> &shape, int kind = 0);
  // shape of a tensor of the checkpoint (`synthetic` without one)
  ffmi_status shape_of(const std::string &name, const std::vector<long> &synthetic,
                       std::vector<long> *shape);
  // tmp -> rows of a GEMM weight: tile / row offset `row0` of an N-row matrix
  ffmi_status pack_rows(const PackSpec &p, int ld, void *dst, int row0, int N);
  static PackSpec spec(int rows, int nb, int np, int cols, int kb, int kp, bool tr = false) {
    PackSpec p;
    p.rows = rows, p.nb = nb, p.np = np, p.cols = cols, p.kb = kb, p.kp = kp, p.transpose = tr;
    return p;
  }
  // one whole GEMM weight [nb][cols * kb] -> [np][cols * kp]
  ffmi_status linear(void **dst, const std::string &name, int nb, int np, int cols, int kb, int kp);
  // an fp32 vector of `rows` blocks of n values, each padded to np
  ffmi_status vec(float **dst, const std::string &name, int rows, int n, int np, int kind = 1);
  ffmi_status vec_to(float *dst, const std::string &name, int rows, int n, int np, int kind = 1);
  // [rows][W] table, bf16 rows of Wp
  ffmi_status table(uint16_t **dst, const std::string &name, int rows);
  const uint16_t *raw_tensor() const { return tmp; }
  // a vector's n values on the host
  ffmi_status host_vec(std::vector<float> *v, const std::string &name, int n, int kind = 0);
  template <class T>
  ffmi_status upload(T **dst, const std::vector<T> &v) {
    FFMI_TRY(alloc(dst, v.size() * sizeof(T)));
    if (!v.empty()) FFMI_HIP(hipMemcpy(*dst, v.data(), v.size() * sizeof(T), hipMemcpyHostToDevice));
    return FFMI_OK;
  }
  // "<p>gate" and "<p>up" [ff][W] as one gated product's weight
  ffmi_status gate_up(void *dst, const std::string &p, int ff, int fp);
  // "<p>e0.", "<p>e1.", ...: the experts' gated and down matrices, expert after expert
  ffmi_status expert_matrices(const std::string &p, int experts, int ff, int fp, void **gated, void **down);

  // ---- mixture of experts: a step's buffers, sized for every layer (kernels/moe.h) ----
  struct ExpertBuffers {
    void *units = nullptr, *rows = nullptr;  // the first product's, the second's
    MoeLists lists;
    size_t num_units = 0, num_slots = 0, num_picks = 0, num_tiles = 0;
  } moe;
  // room for a layer's steps of 1 .. Tm tokens (n: its sizes, T aside; fp: padded units)
  void need_experts(MoeSizes n, int fp);
  ffmi_status alloc_experts();

  // ---- steps ----
  // y (fp32 sums) = X . W^T
  ffmi_status gemm_sum(const void *X, const void *Wt, int N, int K, Partials *y) {
    return gemm_sum_to(X, Wt, N, K, y, ws, ws_bytes);
  }
  ffmi_status gemm_sum_to(const void *X, const void *Wt, int N, int K, Partials *y, float *to, size_t to_bytes);
  // least bytes of the sums of a product with N columns
  size_t sum_bytes(int N, int K) const;
  ffmi_status capture_layer(int i) { return capture(i, x); }  // (tensor capture) x after layer i
  ffmi_status capture(int i, const float *rows);
  bool capturing() const { return dbg != 0; }
  ffmi_status enqueue(bool sample);
  ffmi_status forward(const BatchConfig &bc, const int *rows, int n, bool sample);

  ffmi_status run_inc(const BatchConfig &bc, InferenceResult *ir) override;
  ffmi_status run_inc_logits(const BatchConfig &bc, const int *rows, int n, float *out) override;
  ffmi_status run_tree(const TreeVerifyBatchConfig &, InferenceResult *) override {
    return FFMI_ERR_UNSUPPORTED;
  }
  ffmi_status run_beam(const BeamSearchBatchConfig &, BeamInferenceResult *) override {
    return FFMI_ERR_UNSUPPORTED;
  }
  long debug_width(int which) const override {
    return which == FFMI_DBG_LOGITS ? V : which == FFMI_DBG_HIDDEN ? W : -1;
  }
  ffmi_status set_debug(int enable) override;
  long debug_tensor(int which, int layer, float *out, long cap) override;

  // a factory's body: options checked, `m` configured and initialised
  static ffmi_status create(PagedDecoder *m, const Json &config, const ffmi_model_opts *o,
                            ffmi_model **out);

 private:
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
};

}  // namespace ffmi
