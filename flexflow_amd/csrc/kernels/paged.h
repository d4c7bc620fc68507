// paged.h -- a step's metadata for layers over a paged cache.
//
// The cache is a pool of pages of kPageTokens tokens; a request's page table
// lists the pages of its positions in order.
#pragma once
#include "../ffmi_internal.h"

namespace ffmi {

constexpr int kPageTokens = 64;

struct PagedToken {
  int32_t token, pos;  // embedding row, position in the sequence
  int32_t row;         // cache row: page * kPageTokens + offset
  int32_t prev;        // the token before it in the sequence (-1: none)
  // its place among its request's tokens in the batch: so many before and after
  int32_t back, ahead;
  // rows that a layer carries from step to step lie in two banks per request
  // slot: this step reads one and writes the other
  int32_t slot, bank;
};

// One workgroup of the attention: `nrows` consecutive (token, head) rows of a
// request (row = batch token * heads + head) against cache tiles (= pages)
// [tile0, tile0 + ntiles).  slot >= 0: a partial result for a PagedMerge.
struct PagedBlock {
  int32_t row0, nrows;   // nrows == 0: padding, nothing to do
  int32_t seg_row, pos0;  // first row of the request's tokens, its position
  int32_t table;          // offset of the request's page table (int32 units)
  int32_t tile0, ntiles;
  int32_t slot;
  int32_t page0;          // the page of tile0: one dependent load less at the start
  int32_t pad[3];
};
struct PagedMerge {
  int32_t row0, nrows, slot0, nslots;
};

// A request's consecutive tokens in the batch, for layers that keep a state
// per request slot instead of cached tokens: batch tokens [t0, t0 + n) at
// positions pos0 ...
struct PagedSpan {
  int32_t t0, n, pos0, slot;
  int32_t bank;    // of the slot's carried rows, as a token's
  int32_t chunk0;  // its first chunk among those of all spans beyond kShortSpan
  int32_t pad[2];
};
// spans up to this length take the token-by-token form of a recurrence
constexpr int kShortSpan = 16;
constexpr int kSpanChunk = 64;  // tokens of a chunk of the others

// Layout of a step's metadata, packed by runtime/paged_step.cpp.  Offsets in
// bytes from the start of the blob.
struct PagedLists {  // the block lists of the layers with one row shape
  int heads = 0;      // rows per token
  int groups = 1;     // copies of the list a launch runs (key/value heads)
  int window = 0;     // the last positions that a query sees, itself included (0: all)
  int row_tiles = 0;  // rows of the largest block / 16
  int num_blocks = 0, num_merges = 0, off_blocks = 0, off_merges = 0;
};

}  // namespace ffmi
