// page_pool.h -- pages of a token cache shared by the request slots.
//
// A request slot reserves the pages its longest length needs when it is
// admitted (so that it can never run out on the way) and takes them one by
// one as its tokens arrive; a finished slot gives all of them back.
#pragma once
#include <stdint.h>

#include <vector>

namespace ffmi {

class PagePool {
 public:
  void init(int pages, int page_tokens, int slots) {
    page_tokens_ = page_tokens;
    slots_.assign(slots, Slot());
    free_.clear();
    for (int p = pages - 1; p >= 0; --p) free_.push_back(p);
    total_ = pages, promised_ = 0;
  }
  int page_tokens() const { return page_tokens_; }
  int pages() const { return total_; }
  int free_pages() const { return (int)free_.size(); }
  int pages_for(int tokens) const { return (tokens + page_tokens_ - 1) / page_tokens_; }
  // pages neither taken nor promised to an admitted request
  int available() const { return (int)free_.size() - promised_; }
  bool can_reserve(int tokens) const { return pages_for(tokens) <= available(); }
  // slot `s` now belongs to request `owner`, with room for `tokens` promised
  bool reserve(int s, int64_t owner, int tokens) {
    release(s);
    if (!can_reserve(tokens)) return false;
    slots_[s].owner = owner;
    slots_[s].promised = pages_for(tokens);
    promised_ += slots_[s].promised;
    return true;
  }
  // pages for positions [0, tokens) of the slot; false: none left
  bool ensure(int s, int tokens) {
    Slot &q = slots_[s];
    while ((int)q.table.size() < pages_for(tokens)) {
      if (q.promised > 0) --q.promised, --promised_;
      else if (available() <= 0) return false;
      q.table.push_back(free_.back());
      free_.pop_back();
    }
    return true;
  }
  void release(int s) {
    Slot &q = slots_[s];
    promised_ -= q.promised;
    for (size_t i = q.table.size(); i > 0; --i) free_.push_back(q.table[i - 1]);
    q = Slot();
  }
  int64_t owner(int s) const { return slots_[s].owner; }
  void set_owner(int s, int64_t id) { slots_[s].owner = id; }
  int num_slots() const { return (int)slots_.size(); }
  const std::vector<int32_t> &table(int s) const { return slots_[s].table; }

 private:
  struct Slot {
    int64_t owner = -1;
    int promised = 0;
    std::vector<int32_t> table;
  };
  std::vector<Slot> slots_;
  std::vector<int32_t> free_;
  int page_tokens_ = 64, total_ = 0, promised_ = 0;
};

}  // namespace ffmi
