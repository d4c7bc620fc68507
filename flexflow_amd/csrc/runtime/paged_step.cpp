// paged_step.cpp -- BatchConfig -> paged step metadata (paged_step.h).
#include "paged_step.h"

#include <string.h>

#include <algorithm>

namespace ffmi {

static size_t up16(size_t v) { return (v + 15) & ~(size_t)15; }
// workgroups that fill the chip; fewer blocks than this are split over keys --
// from kSplitTiles pages on (a page costs a workgroup ~1.6 us, the merge of the
// partials ~5 us).  The per-block form shares half-pages out to a workgroup's
// waves: it is split later, into whole rounds of them.
constexpr int kTargetBlocks = 256, kSplitTiles = 5;
constexpr int kBlockSplitTiles = 32, kBlockRound = 8;

ffmi_status PagedStep::init(int max_tokens, int max_requests, int max_positions,
                            const std::vector<RowShape> &shapes, int max_slots) {
  max_tokens_ = max_tokens, max_requests_ = max_requests, max_slots_ = max_slots;
  max_pages_ = (max_positions + kPageTokens - 1) / kPageTokens;
  cap_ = up16((size_t)max_tokens * sizeof(PagedToken)) + up16((size_t)max_tokens * 4) +
         (size_t)max_requests * ((max_pages_ + 16) * 4 + sizeof(PagedSpan)) + 256;
  for (const RowShape &h : shapes) {
    bool known = false;
    for (const RowShape &k : shapes_) known |= k.heads == h.heads && k.groups == h.groups && k.window == h.window;
    if (known) continue;
    PagedLists l;
    l.heads = h.heads, l.groups = h.groups, l.window = h.window;
    lists_.push_back(l);
    shapes_.push_back(h);
    const size_t nb = ((size_t)max_tokens * h.heads + 15) / 16 + max_requests + max_slots + 128;
    cap_ += nb * sizeof(PagedBlock) + (size_t)(max_slots + 64) * sizeof(PagedMerge) + 64;
  }
  // mapped: the step's first kernel copies it into device memory
  if (hipHostMalloc((void **)&host, cap_, hipHostMallocCoherent | hipHostMallocMapped) !=
          hipSuccess ||
      hipMalloc((void **)&dev, cap_) != hipSuccess) {
    ffmi_set_last_error("paged step alloc", __FILE__, __LINE__);
    return FFMI_ERR_OOM;
  }
  memset(host, 0, cap_);
  return FFMI_OK;
}

PagedStep::~PagedStep() {
  if (host) (void)hipHostFree(host);
  if (dev) (void)hipFree(dev);
}

const PagedLists &PagedStep::lists(int heads, int groups, int window) const {
  for (const auto &l : lists_)
    if (l.heads == heads && l.groups == groups && l.window == window) return l;
  return lists_.front();
}

ffmi_status PagedStep::stage(const BatchConfig &bc, PagePool &pool, const StateSlots *states, const int *rows,
                             int num_rows) {
  const int n = bc.num_tokens;
  FFMI_CHECK(n >= 0 && n <= max_tokens_, FFMI_ERR_INVALID);
  std::vector<Seg> segs;
  std::vector<bool> seen(pool.num_slots(), false);
  ids_.resize(n);
  for (int t = 0; t < n;) {
    const int slot = bc.tokensInfo[t].request_index;
    FFMI_CHECK(slot >= 0 && slot < pool.num_slots() && !seen[slot], FFMI_ERR_INVALID);
    seen[slot] = true;
    const int64_t guid = bc.requestsInfo[slot].request_guid;
    if (pool.owner(slot) != guid) {
      pool.release(slot);
      pool.set_owner(slot, guid);
    }
    Seg s{0, bc.tokensInfo[t].abs_depth_in_request, nullptr, slot};
    if (states) {
      if (s.pos0 > 0) s.prev = states->last(slot);
      s.bank = states->bank(slot);
    }
    for (; t < n && bc.tokensInfo[t].request_index == slot; ++t, ++s.n) {
      FFMI_CHECK(bc.tokensInfo[t].abs_depth_in_request == s.pos0 + s.n, FFMI_ERR_INVALID);
      ids_[t] = bc.tokensInfo[t].token_id;
    }
    // positions before the portion must already be in the cache
    FFMI_CHECK(s.pos0 >= 0 && (int)pool.table(slot).size() >= pool.pages_for(s.pos0),
               FFMI_ERR_INVALID);
    FFMI_CHECK(pool.ensure(slot, s.pos0 + s.n), FFMI_ERR_OOM);
    s.table = pool.table(slot).data();
    segs.push_back(s);
  }
  return stage(ids_.data(), segs, rows, num_rows);
}

ffmi_status PagedStep::stage(const int32_t *token_ids, const std::vector<Seg> &in, const int *rows,
                             int num_rows) {
  struct Placed {
    int t0, n, pos0, table;
  };
  std::vector<Placed> segs;
  T = 0, R = num_rows, off_tokens = 0;
  int max_used = 0;
  for (const Seg &s : in) {
    const int end = s.pos0 + s.n;
    FFMI_CHECK(s.n > 0 && s.pos0 >= 0 && T + s.n <= max_tokens_ &&
                   (end + kPageTokens - 1) / kPageTokens <= max_pages_,
               FFMI_ERR_INVALID);
    segs.push_back({T, s.n, s.pos0, 0});
    T += s.n;
    max_used = std::max(max_used, (end + kPageTokens - 1) / kPageTokens);
  }
  FFMI_CHECK((int)segs.size() <= max_requests_ && R >= 0 && R <= T, FFMI_ERR_INVALID);
  PagedToken *tok = reinterpret_cast<PagedToken *>(host);
  for (size_t i = 0; i < in.size(); ++i)
    for (int j = 0; j < in[i].n; ++j) {
      const int p = in[i].pos0 + j, t = segs[i].t0 + j;
      tok[t] = {token_ids[t], p, in[i].table[p / kPageTokens] * kPageTokens + p % kPageTokens,
                j > 0 ? token_ids[t - 1] : in[i].prev, j, in[i].n - 1 - j, in[i].slot, in[i].bank};
    }
  size_t off = up16((size_t)T * sizeof(PagedToken));
  off_rows = (int)off;
  if (R) memcpy(host + off, rows, (size_t)R * 4);
  off = up16(off + (size_t)R * 4);
  // page tables, one stride for all (16-page steps: decode steps keep their
  // layout for 1024 tokens)
  const int stride = (max_used + 15) & ~15;
  for (size_t i = 0; i < in.size(); ++i) {
    segs[i].table = (int)(off / 4);
    memcpy(host + off, in[i].table,
           (size_t)((in[i].pos0 + in[i].n + kPageTokens - 1) / kPageTokens) * 4);
    off += (size_t)stride * 4;
  }
  off_spans = (int)(off = up16(off));
  num_spans = (int)segs.size();
  short_spans = long_spans = false;
  num_chunks = 0;
  for (size_t i = 0; i < segs.size(); ++i, off += sizeof(PagedSpan)) {
    const PagedSpan sp{segs[i].t0, segs[i].n, segs[i].pos0, in[i].slot, in[i].bank, num_chunks, {0, 0}};
    memcpy(host + off, &sp, sizeof(sp));
    (sp.n <= kShortSpan ? short_spans : long_spans) = true;
    if (sp.n > kShortSpan) num_chunks += (sp.n + kSpanChunk - 1) / kSpanChunk;
  }
  off = up16(off);
  shape.assign({T, R, num_spans, stride, short_spans, long_spans, num_chunks});
  for (size_t li = 0; li < lists_.size(); ++li) {
    PagedLists &l = lists_[li];
    const RowShape &rs = shapes_[li];
    blocks_.clear();
    merges_.clear();
    int max_rows = 0;
    for (const Placed &s : segs) max_rows = std::max(max_rows, s.n * l.heads);
    const auto tiles_for = [&](int rows) {
      if (rs.per_block) return rows <= 16 ? 1 : rs.max_tiles;
      return rows <= 16 ? 1 : rows <= 32 ? 2 : rs.max_tiles;
    };
    l.row_tiles = tiles_for(max_rows);
    const auto block_rows = [&](const Placed &s) {
      return 16 * (rs.per_block ? tiles_for(s.n * l.heads) : l.row_tiles);
    };
    long base = 0;
    for (const Placed &s : segs)
      base += ((long)s.n * l.heads + block_rows(s) - 1) / block_rows(s) * rs.groups;
    const int want = std::max(1L, kTargetBlocks * (rs.per_block ? 2 : 1) / std::max(1L, base));
    int slots = 0;
    for (const Placed &s : segs) {
      const int nrows = s.n * l.heads, row0 = s.t0 * l.heads, br = block_rows(s);
      for (int r = 0; r < nrows; r += br) {
        PagedBlock b{};
        b.row0 = row0 + r, b.nrows = std::min(br, nrows - r);
        b.seg_row = row0, b.pos0 = s.pos0, b.table = s.table;
        const int last = s.pos0 + (r + b.nrows - 1) / l.heads;  // last visible position
        // the first page that the block's first row sees
        const int first = l.window ? std::max(0, s.pos0 + r / l.heads - l.window + 1) / kPageTokens : 0;
        const int tiles = last / kPageTokens + 1 - first;
        const int units = rs.per_block && b.nrows > 16 ? rs.max_tiles : 1;  // slots of a partial
        int ns = tiles < (rs.per_block ? kBlockSplitTiles : kSplitTiles) ? 1 : std::min(want, tiles);
        int per = (tiles + ns - 1) / ns;
        if (rs.per_block && ns > 1) per = (per + kBlockRound - 1) / kBlockRound * kBlockRound;
        ns = (tiles + per - 1) / per;
        if (slots + ns * units > max_slots_) ns = 1, per = tiles;
        if (ns > 1) merges_.push_back({b.row0, b.nrows, slots, ns});
        for (int i = 0; i < ns; ++i) {
          b.tile0 = first + i * per, b.ntiles = std::min(per, tiles - i * per);
          b.slot = ns > 1 ? slots : -1;
          if (ns > 1) slots += units;
          b.page0 = reinterpret_cast<const int32_t *>(host)[s.table + b.tile0];
          blocks_.push_back(b);
        }
      }
    }
    // longest first: the causal triangle's short blocks fill the end
    std::stable_sort(blocks_.begin(), blocks_.end(),
                     [](const PagedBlock &a, const PagedBlock &b) { return a.ntiles > b.ntiles; });
    // padded counts: a decode step's launch shape changes every 32 blocks
    blocks_.resize((blocks_.size() + 31) & ~(size_t)31, PagedBlock{});
    if (!merges_.empty()) merges_.resize((merges_.size() + 7) & ~(size_t)7, PagedMerge{});
    l.num_blocks = (int)blocks_.size(), l.num_merges = (int)merges_.size();
    l.off_blocks = (int)off;
    off += blocks_.size() * sizeof(PagedBlock);
    l.off_merges = (int)(off = up16(off));
    off = up16(off + merges_.size() * sizeof(PagedMerge));
    FFMI_CHECK(off <= cap_, FFMI_ERR_INVALID);
    memcpy(host + l.off_blocks, blocks_.data(), blocks_.size() * sizeof(PagedBlock));
    if (!merges_.empty())
      memcpy(host + l.off_merges, merges_.data(), merges_.size() * sizeof(PagedMerge));
    shape.insert(shape.end(), {l.row_tiles, l.num_blocks, l.num_merges});
  }
  bytes = off;
  return FFMI_OK;
}

}  // namespace ffmi
