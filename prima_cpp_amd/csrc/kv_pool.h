// kv_pool.h — pages of a KV cache shared by the open sequences of a model (host side only). A sequence's pages are found through its table: page index (position / 64)
// -> pool page, or -1 in front of what its layers can still see. Pages come back in LIFO order, so a freed page is the next one handed out.
#pragma once
#include "../../include/prima_mi355.h"
#include <utility>
#include <vector>

struct pm355_page_pool {
    static constexpr int PAGE = 64;
    struct Seq { bool open = false; int lo = 0, hi = 0; std::vector<int> page; };      // pages [lo, hi) are held
    int n_pages, max_seq_pages;
    std::vector<int> free_list;
    std::vector<Seq> seqs;
    std::vector<std::pair<int, int>> changes;              // (seq * max_seq_pages + index, page) since the owner last took them

    pm355_page_pool(int pages, int n_seqs, int max_pages) : n_pages(pages), max_seq_pages(max_pages), seqs((size_t) n_seqs) {
        for (int i = pages - 1; i >= 0; --i) free_list.push_back(i);
    }
    bool valid(int s) const { return s >= 0 && s < (int) seqs.size() && seqs[s].open; }
    int open() {
        for (size_t s = 0; s < seqs.size(); ++s) if (!seqs[s].open) { seqs[s] = Seq(); seqs[s].open = true; return (int) s; }
        return PM355_E_NOMEM;
    }
    int close(int s) {
        if (!valid(s)) return PM355_E_RANGE;
        for (int i = seqs[s].hi - 1; i >= seqs[s].lo; --i) free_list.push_back(seqs[s].page[i]);
        seqs[s] = Seq();
        return 0;
    }
    int missing(int s, int n_tokens) const { const int need = (n_tokens + PAGE - 1) / PAGE; return need > seqs[s].hi ? need - seqs[s].hi : 0; }
    int grow(int s, int n_tokens) {
        if (!valid(s)) return PM355_E_RANGE;
        const int n = missing(s, n_tokens);
        if (seqs[s].hi + n > max_seq_pages) return PM355_E_RANGE;
        if (n > (int) free_list.size()) return PM355_E_NOMEM;
        for (int i = 0; i < n; ++i) {
            seqs[s].page.push_back(free_list.back());
            free_list.pop_back();
            changes.push_back({s * max_seq_pages + seqs[s].hi++, seqs[s].page.back()});
        }
        return 0;
    }
    int drop_before(int s, int position) {
        if (!valid(s)) return PM355_E_RANGE;
        Seq & q = seqs[s];
        for (; q.lo < q.hi && (q.lo + 1) * PAGE <= position; ++q.lo) { free_list.push_back(q.page[q.lo]); q.page[q.lo] = -1; }
        return 0;
    }
    int page(int s, int i) const { return valid(s) && i >= 0 && i < seqs[s].hi ? seqs[s].page[i] : -1; }
};
