// Attention whose heads' weights are mixed before they meet the values, over a paged context:
//     s_g(i, j) = scale q_i . k_j - size[g] ln(1 + rate[g] (i - j)),   p_g(i, j) = e^s_g(i, j) / sum over visible j' of e^s_g(i, j')
//     out_h(i) = sum over visible j of (sum_g talk[h][g] p_g(i, j)) v_j        (v of h's own kv head)
// A weight enters the mixture normalised, so every head's sum comes first: a pass over the keys alone leaves
// lse = log2 of the sum of 2^(s log2 e) per row and head.
#pragma once
#include "scored_attn.h"

struct TalkArgs : ScoredArgs {  // (q1, n1: the queries; cap, bias, sink, window unused)
    const float *size, *rate;   // [heads], or NULL: no distance bias
    const float *talk;          // [heads][heads]
    float *lse;                 // [rows][heads], base 2
    float *scores;              // decode: [batch][heads][keys_cap], base 2
    int64_t keys_cap;
    int bs_shift;               // log2 of the block size, -1: it is no power of two
};

// scored_block_id and scored_slot_of without a division where the block size allows it (key < 2^31, bt_stride > 0)
__device__ __forceinline__ int talk_block(const TalkArgs &a, int key) { return a.bs_shift >= 0 ? key >> a.bs_shift : key / a.bs; }
__device__ __forceinline__ int talk_block_id(const TalkArgs &a, const int32_t *table, int key) {
    return table[min((int64_t)talk_block(a, key), a.bt_stride - 1)];
}
__device__ __forceinline__ int talk_slot_of(const TalkArgs &a, int id, int key, int end) {
    const int blk = talk_block(a, key);
    return key < end && blk < a.bt_stride && (uint32_t)id < (uint64_t)a.num_blocks ? id * a.bs + (key - blk * a.bs) : -1;
}

// The distance bias in units of the base-2 exponential.
__device__ __forceinline__ float talk_bias(float size, float rate, int dist) {
    return -size * __builtin_amdgcn_logf(fmaf(rate, (float)dist, 1.f));
}

// The same, and nothing where the key lies behind the row.
__device__ __forceinline__ float talk_masked_bias(float size, float rate, int dist) {
    return dist >= 0 ? talk_bias(size, rate, dist) : kScoredNone;
}

constexpr int kTalkMaxHeads = 128;

// false: no matrix-core kernels for these sizes
bool pa_talking_decode_launch(const TalkArgs &a, int dtype, void *workspace, size_t workspace_bytes, hipStream_t s, int &rc);
bool pa_talking_prefill_launch(const TalkArgs &a, int dtype, hipStream_t s, int &rc);
size_t pa_talking_decode_bytes(int batch, int heads, int kv_heads, int vdim, int64_t max_keys);
