// paged_step.h -- one step's metadata for models over a paged cache: tokens
// with their cache rows, page tables, the requests' spans, and per row shape of
// the attention its workgroup list (kernels/paged.h).
#pragma once
#include <vector>

#include "../kernels/paged.h"
#include "batch_config.h"
#include "page_pool.h"
#include "state_slots.h"

namespace ffmi {

// The row shape of an attention's launches: `heads` rows per token, `groups`
// copies of the list (key/value heads), blocks of at most 16 * max_tiles rows.
//   per_block == false: all blocks of a step have the size that the longest
//     request asks for (1, 2 or 4 tiles)
//   per_block == true: a request of one tile gets blocks of 16 rows, others of
//     16 * max_tiles, side by side
struct RowShape {
  int heads = 1, groups = 1, max_tiles = 4;
  bool per_block = false;
  int window = 0;  // positions a query sees, itself included: earlier pages are left out (0: all)
};

struct PagedStep {
  // shapes: the distinct row shapes of the model's layers; max_slots: partial
  // results of split blocks that the slab buffer holds (0: never split), one
  // per block, or one per 16 rows of a block where the shape is per_block
  ffmi_status init(int max_tokens, int max_requests, int max_positions,
                   const std::vector<RowShape> &shapes, int max_slots);
  ~PagedStep();
  // one request's consecutive tokens in the batch: positions pos0 .. pos0 + n
  struct Seg {
    int n, pos0;
    const int32_t *table;  // pages of positions 0 .. pos0 + n
    int slot = 0;          // request slot
    int prev = -1;         // the token before the first (-1: none or not wanted)
    int bank = 0;          // of the slot's carried rows (kernels/paged.h)
  };
  // Fills the pinned staging: the segments' tokens in order (token_ids), the
  // output rows and the attention's lists.
  ffmi_status stage(const int32_t *token_ids, const std::vector<Seg> &segs, const int *rows,
                    int num_rows);
  // The same from an INC batch: takes the pages its tokens
  // need (a slot whose request changed gives its old pages back first) and
  // lists rows[0, num_rows) for the output.  states: where the requests' last
  // tokens and banks come from (null: no layer asks for them).
  ffmi_status stage(const BatchConfig &bc, PagePool &pool, const StateSlots *states, const int *rows,
                    int num_rows);
  const PagedLists &lists(int heads, int groups = 1, int window = 0) const;

  char *host = nullptr, *dev = nullptr;
  size_t bytes = 0;
  int T = 0, R = 0, off_tokens = 0, off_rows = 0, off_spans = 0, num_spans = 0;
  bool short_spans = false, long_spans = false;  // spans of either kind in the step
  int num_chunks = 0;                            // of the long ones
  std::vector<int> shape;  // everything a captured graph of this step depends on

 private:
  int max_tokens_ = 0, max_requests_ = 0, max_pages_ = 0, max_slots_ = 0;
  size_t cap_ = 0;
  std::vector<RowShape> shapes_;
  std::vector<PagedLists> lists_;
  std::vector<PagedBlock> blocks_;
  std::vector<PagedMerge> merges_;
  std::vector<int32_t> ids_;
};

}  // namespace ffmi
