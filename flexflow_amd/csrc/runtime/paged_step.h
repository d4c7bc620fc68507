// paged_step.h -- one step's metadata for models over a paged cache: tokens
// with their cache rows, page tables, and per head count the attention's
// workgroup list (kernels/latent.h).
#pragma once
#include <vector>

#include "../kernels/latent.h"
#include "batch_config.h"
#include "page_pool.h"

namespace ffmi {

struct PagedStep {
  // head_counts: the distinct head counts of the model's layers; max_slots:
  // partial results the slab buffer holds (0: blocks are never split)
  ffmi_status init(int max_tokens, int max_requests, int max_positions,
                   const std::vector<int> &head_counts, int max_slots);
  ~PagedStep();
  // one request's consecutive tokens in the batch: positions pos0 .. pos0 + n
  struct Seg {
    int n, pos0;
    const int32_t *table;  // pages of positions 0 .. pos0 + n
  };
  // Fills the pinned staging: the segments' tokens in order (token_ids), the
  // output rows and the attention's lists.
  ffmi_status stage(const int32_t *token_ids, const std::vector<Seg> &segs, const int *rows,
                    int num_rows);
  // The same from an INC batch: takes the pages its tokens
  // need (a slot whose request changed gives its old pages back first) and
  // lists rows[0, num_rows) for the output.
  ffmi_status stage(const BatchConfig &bc, PagePool &pool, const int *rows, int num_rows);
  const PagedLists &lists(int heads) const;

  char *host = nullptr, *dev = nullptr;
  size_t bytes = 0;
  int T = 0, R = 0, off_tokens = 0, off_rows = 0;
  std::vector<int> shape;  // everything a captured graph of this step depends on

 private:
  int max_tokens_ = 0, max_requests_ = 0, max_pages_ = 0, max_slots_ = 0;
  size_t cap_ = 0;
  std::vector<PagedLists> lists_;
  std::vector<LatentBlock> blocks_;
  std::vector<LatentMerge> merges_;
  std::vector<int32_t> ids_;
};

}  // namespace ffmi
