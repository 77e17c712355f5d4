// Host side of a KV cache whose cells are shared between sequences (llama_kv_cell / llama_kv_cache, llama.cpp:1381-1420, 1683-1848): a cell
// holds a position (-1: free) and a set of sequence ids (bit s); `head` is where the search for free cells starts.
#pragma once
#include <limits.h>
#include <stdint.h>

#include <algorithm>
#include <vector>

struct KvCells {
    int n = 0, head = 0, n_used = 0;
    std::vector<int32_t>  pos;
    std::vector<uint32_t> seq;
    std::vector<int32_t>  delta;                   // position shifts not yet applied to the stored rows
    bool has_shift = false;
    uint32_t edited = 0;                           // sequences whose set of cells changed other than by take() since the owner cleared its bit

    void init(int n_cells) {
        n = n_cells; head = 0; n_used = 0; has_shift = false;
        pos.assign(n, -1); seq.assign(n, 0u); delta.assign(n, 0);
        edited = ~0u;
    }
    void grow(int n_cells) {                       // further free cells behind the ones there are
        n = n_cells;
        pos.resize(n, -1); seq.resize(n, 0u); delta.resize(n, 0);
        edited = ~0u;
    }
    void take(int cell, int32_t p, uint32_t seqs) {
        if (pos[cell] < 0) ++n_used;
        pos[cell] = p;
        seq[cell] |= seqs;
    }
    void release(int cell) {
        if (pos[cell] >= 0) --n_used;
        pos[cell] = -1; seq[cell] = 0; delta[cell] = 0;
    }
    // llama_kv_cache_find_slot (llama.cpp:1683-1730): k contiguous free cells, searched from the ring's head, wrapping once
    bool find_run(int k) {
        if (k > n) return false;
        int n_tested = 0;
        while (true) {
            if (head + k > n) { n_tested += n - head; head = 0; continue; }
            bool found = true;
            for (int i = 0; i < k; ++i)
                if (pos[head + i] >= 0) { found = false; head += i + 1; n_tested += i + 1; break; }
            if (found) return true;
            if (n_tested >= n) return false;
        }
    }
    // any k free cells, searched from the ring's head; nothing is taken when there are fewer
    bool find_free(int k, int32_t * out) {
        if (k > n - n_used) return false;
        int c = head, got = 0;
        for (int i = 0; i < n && got < k; ++i, c = c + 1 == n ? 0 : c + 1)
            if (pos[c] < 0) out[got++] = c;
        return got == k;
    }
    // the cells a step looks at: up to the last one in use, at least 32 (llama_kv_cache_cell_max, llama.cpp:1735-1743, 6842)
    int n_kv() const {
        int cell_max = 0;
        for (int i = n - 1; i > 0; --i) if (pos[i] >= 0 && seq[i]) { cell_max = i + 1; break; }
        return std::min(n, std::max(32, cell_max));
    }
    void move_head(int to) { head = to >= n ? 0 : to; }          // llama_decode moves the ring's head past a step's cells (llama.cpp:6936-6943)

    // llama_kv_cache_seq_rm (llama.cpp:1757-1785): s < 0 removes the range from every sequence; p1 < 0: to the end
    void seq_rm(int s, int p0, int p1) {
        int new_head = n;
        range(p0, p1);
        edited |= s < 0 ? ~0u : 1u << s;
        for (int i = 0; i < n; ++i) {
            if (pos[i] < p0 || pos[i] >= p1) continue;
            if (s < 0) seq[i] = 0;
            else if (seq[i] >> s & 1u) seq[i] &= ~(1u << s);
            else continue;
            if (seq[i] == 0) { release(i); if (new_head == n) new_head = i; }
        }
        if (new_head != n) head = new_head;
    }
    // llama_kv_cache_seq_cp (llama.cpp:1787-1803): the cells of src in [p0, p1) join dst as well; nothing is copied
    void seq_cp(int src, int dst, int p0, int p1) {
        range(p0, p1);
        head = 0;
        edited |= 1u << dst;
        for (int i = 0; i < n; ++i)
            if ((seq[i] >> src & 1u) && pos[i] >= p0 && pos[i] < p1) seq[i] |= 1u << dst;
    }
    // llama_kv_cache_seq_keep (llama.cpp:1805-1822)
    void seq_keep(int s) {
        int new_head = n;
        edited = ~0u;
        for (int i = 0; i < n; ++i) {
            if (!(seq[i] >> s & 1u)) { release(i); if (new_head == n) new_head = i; }
            else seq[i] = 1u << s;
        }
        if (new_head != n) head = new_head;
    }
    // llama_kv_cache_seq_shift (llama.cpp:1824-1848): the positions move now, the stored rows at the start of the next step
    void seq_shift(int s, int p0, int p1, int by) {
        int new_head = n;
        range(p0, p1);
        edited = ~0u;                              // shared cells move for every sequence that holds them
        for (int i = 0; i < n; ++i) {
            if (!(seq[i] >> s & 1u) || pos[i] < p0 || pos[i] >= p1) continue;
            has_shift = true;
            if (pos[i] + by < 0) { release(i); if (new_head == n) new_head = i; continue; }
            pos[i] += by;
            delta[i] += by;
        }
        head = new_head != n ? new_head : 0;
    }
    void clear() {                                 // llama_kv_cache_clear (llama.cpp:1745-1751)
        std::fill(pos.begin(), pos.end(), -1);
        std::fill(seq.begin(), seq.end(), 0u);
        std::fill(delta.begin(), delta.end(), 0);
        head = 0; n_used = 0; has_shift = false; edited = ~0u;
    }
    void shift_done() { has_shift = false; std::fill(delta.begin(), delta.end(), 0); }

private:
    static void range(int & p0, int & p1) { if (p0 < 0) p0 = 0; if (p1 < 0) p1 = INT32_MAX; }
};
