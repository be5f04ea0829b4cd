// step_arrays.h -- device copies of the host-side description of one ragged batch.
#pragma once
#include <algorithm>
#include <vector>

#include "nvllm_internal.h"

namespace nvllm {

struct StepArrays {
    int T, B;
    int n_seqs;
    int max_pos;      // largest position in the batch
    int write_limit;  // tokens [0, write_limit) get their K/V stored (see attention.c:159-162)
    bool table_short; // some token's logical block lies beyond its sequence's table
    int* d_tokens;    // [T]        (null when not supplied)
    int* d_tok_src;   // [T]        (null unless supplied) -1, or the output row of the previous pass whose arg-max is the token
    int* d_pos;       // [T]
    int* d_seq;       // [T]
    int* d_out_idx;   // [B]
    int* d_tbl_off;   // [n_seqs]   start of each sequence's table inside d_tables
    int* d_tables;    // concatenated logical->physical block maps
    int* d_kv_row;    // [T] pool row (block * block_size + slot) where the token's K/V go, -1: not stored
    int* d_runs;      // [n_runs][4] (first token, count, last position, table offset): attention work items
    int n_runs;
    long kv_positions;
    long kv_rows;            // sum over the batch's sequences of the positions their last token sees
    long qk_pairs;           // sum over tokens of the positions they see
    int max_run;             // tokens of the longest run
    int n_multi;             // with `multi_first`: the first n_multi runs have several tokens, the others one each
    long kv_rows_single;     // ... positions those others see
    int runs_in_tb[4];       // runs that touch each of the first four 16-token blocks
    bool one_token_per_seq;  // no sequence contributes more than one token (a pure decode step)
    // with `spans`: every sequence's portion of the batch as a whole (models whose layers carry a state from token to token)
    int* d_spans;            // [n_spans][4] (first token, count, first position, sequence); portions of several tokens come first
    int* d_span_of;          // [T] the span of each token
    int n_spans, n_spans_multi;
    int max_span;            // tokens of the longest
    bool seq_split;          // some sequence's tokens do not lie side by side at consecutive positions
    // chunk_len > 0: the portions of several tokens cut into chunks of that many
    int chunk_len, n_chunks;
    int* d_chunks;           // [n_chunks][2] (span, its chunk)
    int* d_first_chunk;      // [n_spans_multi]
    std::vector<int> host_spans;
    // Kernel timing, when a token sees at most `limit` positions: rows of K/V that the portions of several tokens (of one
    // token) see, each counted once, and (token, position) pairs of the former.
    long multi_rows(long limit) const { return count(0, n_spans_multi, limit, false); }
    long multi_pairs(long limit) const { return count(0, n_spans_multi, limit, true); }
    long single_rows(long limit) const { return count(n_spans_multi, n_spans, limit, false); }

private:
    long count(int from, int to, long limit, bool pairs) const {
        long n = 0;
        for (int i = from; i < to; i++) {
            const long toks = host_spans[4 * i + 1], p0 = host_spans[4 * i + 2], last = p0 + toks;   // sees p0 + 1 .. last positions
            const long rising = std::max(0L, std::min(last, limit) - p0);                          // tokens below the limit
            n += pairs ? rising * p0 + rising * (rising + 1) / 2 + (toks - rising) * limit : std::min(last, limit + toks - 1);
        }
        return n;
    }
};

// Copies the arrays into the pinned ring, lays the block tables of the sequences
// that occur in the batch end to end, and enqueues ONE host-to-HBM copy.
// `tables` (indexed by seq id) or `single` (one table, positions pos0 + t) may be
// null for operators that do not touch the pool.  attn_ct > 0 also cuts the batch into
// attention work items: runs of at most attn_ct tokens of one sequence at
// consecutive positions.  multi_first: runs of several tokens come before those of one.
StepArrays stage_step(const int* tokens, const int* pos_arr, const int* seq_ids, int T,
                      const int* output_indices, int B, BlockTable** tables, const BlockTable* single,
                      int pos0, int block_size, int attn_ct = 0, const int* token_src = nullptr, bool multi_first = false,
                      bool spans = false, int chunk_len = 0);

KvPoolView pool_view(const KVCacheManager* mgr, int n_kv_heads, int head_dim);

}  // namespace nvllm
