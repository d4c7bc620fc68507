// state_slots.h -- which request's state each slot of a recurrent layer holds,
// how many of its tokens the state has taken in, the last of them, and which of
// the slot's two banks holds rows that layers carry from step to step.
//
// A state cannot be rewound: a step must bring exactly the token after the
// last one.  Position 0 starts a state afresh (the kernels take zeros for it),
// so a slot that is used again needs no clearing.
#pragma once
#include <stdint.h>

#include <vector>

namespace ffmi {

class StateSlots {
 public:
  void init(int slots) { slots_.assign(slots, Slot()); }
  // may request `owner` bring its token at position pos0 next?
  bool follows(int s, int64_t owner, int pos0) const {
    return pos0 == 0 || (slots_[s].owner == owner && slots_[s].len == pos0);
  }
  // a step is under way: until done() the slot's state is neither old nor new
  void begin(int s, int64_t owner) { slots_[s].owner = owner, slots_[s].len = -1; }
  void done(int s, int len, int last) { slots_[s].len = len, slots_[s].last = last, slots_[s].bank ^= 1; }
  int last(int s) const { return slots_[s].last; }
  int bank(int s) const { return slots_[s].bank; }

 private:
  struct Slot {
    int64_t owner = -1;
    int len = -1;
    int last = -1, bank = 0;
  };
  std::vector<Slot> slots_;
};

}  // namespace ffmi
