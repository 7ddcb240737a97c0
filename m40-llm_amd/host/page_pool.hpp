// Pages of a paged sequence cache and what the sequences hold: a fixed pool of pages, shared by all sequences and given back
// when a sequence ends; per sequence slot its length, its pages and the token before the next one.  One page number stands for
// the same page of every layer that keeps entries.
#pragma once

#include <cstdint>
#include <stdexcept>
#include <vector>

namespace m40host {

class SequencePages {
public:
    static constexpr uint32_t kNoToken = 0xffffffffu;
    SequencePages(uint32_t n_pages, uint32_t page_tokens, uint32_t n_slots)
        : page_tokens_(page_tokens), n_pages_(n_pages), slots_(n_slots) {
        for (uint32_t p = n_pages; p > 0; --p) free_.push_back(p - 1);
    }
    uint32_t slots() const { return (uint32_t)slots_.size(); }
    uint32_t total_pages() const { return n_pages_; }
    uint32_t free_pages() const { return (uint32_t)free_.size(); }
    uint32_t pages_for(uint64_t tokens) const { return (uint32_t)((tokens + page_tokens_ - 1) / page_tokens_); }
    uint32_t length(uint32_t slot) const { return at(slot).length; }
    uint32_t previous_token(uint32_t slot) const { return at(slot).prev; }
    const std::vector<uint32_t>& pages(uint32_t slot) const { return at(slot).pages; }

    // Sets pages aside for a sequence that may grow to `tokens`; false where they are not there.
    bool reserve(uint32_t slot, uint64_t tokens) {
        Slot& s = at(slot);
        const uint32_t want = pages_for(tokens), have = (uint32_t)s.pages.size();
        const uint32_t more = want > have ? want - have : 0;
        if (more > free_.size() - (promised_ - s.promised)) return false;
        promised_ = promised_ - s.promised + more;
        s.promised = more;
        return true;
    }
    // Makes room for `tokens` tokens in all; throws, with nothing changed, where the pool cannot give the pages.
    void grow(uint32_t slot, uint64_t tokens) {
        Slot& s = at(slot);
        const uint32_t want = pages_for(tokens);
        if (want <= s.pages.size()) return;
        const uint32_t more = want - (uint32_t)s.pages.size();
        if (more > free_.size() - (promised_ - s.promised)) throw std::runtime_error("the cache pool has no page left");
        for (uint32_t i = 0; i < more; ++i) {
            s.pages.push_back(free_.back());
            free_.pop_back();
        }
        const uint32_t used = more < s.promised ? more : s.promised;
        s.promised -= used;
        promised_ -= used;
    }
    void advance(uint32_t slot, uint32_t tokens, uint32_t last_token) {
        Slot& s = at(slot);
        s.length += tokens;
        s.prev = last_token;
    }
    // back to an earlier length (entries past it are rewritten by what follows); pages are kept
    void rewind(uint32_t slot, uint32_t length, uint32_t prev) {
        Slot& s = at(slot);
        if (length > s.length) throw std::out_of_range("cannot rewind forwards");
        s.length = length;
        s.prev = prev;
    }
    void release(uint32_t slot) {
        Slot& s = at(slot);
        while (!s.pages.empty()) {
            free_.push_back(s.pages.back());
            s.pages.pop_back();
        }
        promised_ -= s.promised;
        s = Slot{};
    }

private:
    struct Slot {
        uint32_t length = 0, prev = kNoToken, promised = 0;
        std::vector<uint32_t> pages;
    };
    Slot& at(uint32_t slot) {
        if (slot >= slots_.size()) throw std::out_of_range("sequence slot out of range");
        return slots_[slot];
    }
    const Slot& at(uint32_t slot) const { return const_cast<SequencePages*>(this)->at(slot); }
    uint32_t page_tokens_, n_pages_, promised_ = 0;
    std::vector<Slot> slots_;
    std::vector<uint32_t> free_;
};

}  // namespace m40host
