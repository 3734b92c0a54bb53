// Attention over a paged context whose scores are more than q . k, and whose keys and values may have sizes of their own or
// be one tensor:
//     score(i, j) = cap tanh(scale q_i . k_j / cap) + bias[h][min(i - j, bias_n - 1)]       (cap 0: without it)
//     out_i = sum over visible j of e^score(i, j) v_j / (sum over visible j of e^score(i, j) + e^sink[h])
// A query row is two pieces side by side (a latent part and a rotated part), or one.
#pragma once
#include "row_common.h"

typedef uint32_t scored_u4 __attribute__((ext_vector_type(4)));

struct ScoredArgs {
    const void *q1, *q2;  // pieces of n1 and n2 elements, head h of row r at r * q*_row + h * q*_head
    int64_t q1_row, q1_head, q2_row, q2_head;
    int n1, n2;
    const void *k, *v;  // pool rows of a token: [hkv][k_dim], [hkv][v_dim]; v may lie inside k
    int k_dim, v_dim, vdim;
    const int32_t *bt;
    int64_t bt_stride, num_blocks;
    int bs;
    const int32_t *ctx_lens, *q_lens, *q_starts;  // (q_lens NULL: one row per sequence)
    int64_t n_rows;
    int batch, max_q_len, heads, hkv, n_rep, window;
    float scale, cap;
    const float *bias;  // [heads][bias_n], or NULL
    int bias_n;
    const float *sink;  // [heads], or NULL
    void *out;          // [rows][heads][vdim]
    int splits;         // decode: pieces of a sequence's keys
    float *part_o, *part_ml;
};

struct ScoredPortion {
    int n, pos0;
    int64_t row0;
};
__device__ __forceinline__ bool scored_portion(const ScoredArgs &a, int b, ScoredPortion &p) {
    p.n = a.q_lens ? a.q_lens[b] : 1;
    p.row0 = a.q_starts ? a.q_starts[b] : b;
    p.pos0 = a.ctx_lens[b] - p.n;
    return p.n > 0 && p.pos0 >= 0 && p.row0 >= 0 && p.row0 + p.n <= a.n_rows;
}
__device__ __forceinline__ int scored_first_key(const ScoredArgs &a, int pos) {
    return a.window > 0 && pos >= a.window ? pos - a.window + 1 : 0;
}
// Pool row of a key, -1 when its block is missing
__device__ __forceinline__ int64_t scored_slot(const ScoredArgs &a, const int32_t *table, int key) {
    const int blk = key / a.bs;
    const int64_t id = blk < a.bt_stride ? table[blk] : -1;
    return id >= 0 && id < a.num_blocks ? id * a.bs + key % a.bs : -1;
}

// For loops that fetch a tile ahead: the block id of a key, loaded without a branch, and, when the tile is fetched, the key's
// pool row.  (bt_stride > 0.)
__device__ __forceinline__ int scored_block_id(const ScoredArgs &a, const int32_t *table, int key) {
    return table[min((int64_t)(key / a.bs), a.bt_stride - 1)];
}
__device__ __forceinline__ int scored_slot_of(const ScoredArgs &a, int id, int key, int end) {
    return key < end && key / a.bs < a.bt_stride && (uint32_t)id < (uint64_t)a.num_blocks ? id * a.bs + key % a.bs : -1;
}
// 16 bytes of a row, zeros where there is none: always one load, so that nothing waits for it before it is used.
static __device__ const uint32_t kScoredZeros[4] __attribute__((aligned(16))) = {0, 0, 0, 0};
__device__ __forceinline__ scored_u4 scored_load16(const uint16_t *p, bool there) {
    return *reinterpret_cast<const scored_u4 *>(there ? p : reinterpret_cast<const uint16_t *>(kScoredZeros));
}

constexpr float kScoredLog2e = 1.4426950408889634f;
constexpr float kScoredNone = -1.0e30f;  // finite stand-in for minus infinity

// Value columns that the decode kernel for these sizes holds, 0: there is none.
inline int scored_value_cols(int keys, int vdim, bool one) {
    if (one) return keys <= 160 && vdim <= 128 ? 128 : keys <= 320 && vdim <= 256 ? 256 : keys <= 576 && vdim <= 512 ? 512 : 0;
    const int most = keys > vdim ? keys : vdim;
    return most <= 64 ? 64 : most <= 128 ? 128 : most <= 256 ? 256 : 0;
}

// Pieces that a decode step's sequences are cut into: two workgroups per compute unit (`full`: one, which has its LDS to
// itself, and none of which waits for another's end), of at least 256 keys each.
inline int scored_splits(int64_t workgroups, int cus, int64_t span, bool full) {
    int64_t n = full ? cus / workgroups : (2 * (int64_t)cus + workgroups - 1) / workgroups;
    if (n > span / 256) n = span / 256;
    return n < 1 ? 1 : n > 16 ? 16 : (int)n;
}

// false: no matrix-core kernel for these sizes
bool pa_scored_decode_launch(const ScoredArgs &a, int dtype, hipStream_t s, int &rc);
bool pa_scored_prefill_launch(const ScoredArgs &a, int dtype, hipStream_t s, int &rc);
