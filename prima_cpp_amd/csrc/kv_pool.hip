// kv_pool.hip — C entry points of the page pool (kv_pool.h); no device code.
#include "kv_pool.h"

extern "C" {
pm355_page_pool * pm355_page_pool_new(int n_pages, int n_seqs, int max_seq_pages) {
    return n_pages > 0 && n_seqs > 0 && max_seq_pages > 0 ? new pm355_page_pool(n_pages, n_seqs, max_seq_pages) : nullptr;
}
void pm355_page_pool_free(pm355_page_pool * p) { delete p; }
int pm355_page_pool_open(pm355_page_pool * p) { return p->open(); }
int pm355_page_pool_close(pm355_page_pool * p, int seq) { return p->close(seq); }
int pm355_page_pool_grow(pm355_page_pool * p, int seq, int n_tokens) { return p->grow(seq, n_tokens); }
int pm355_page_pool_drop_before(pm355_page_pool * p, int seq, int position) { return p->drop_before(seq, position); }
int pm355_page_pool_page(const pm355_page_pool * p, int seq, int index) { return p->page(seq, index); }
int pm355_page_pool_free_pages(const pm355_page_pool * p) { return (int) p->free_list.size(); }
}
