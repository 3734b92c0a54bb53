// Host-testable arithmetic of the linear-recurrence kernels: padded state sizes, value slices and the segments a long
// portion is cut into.  Plain C++.
#pragma once
#include <stddef.h>
#include <stdint.h>

constexpr int kLaChunk = 64;      // rows multiplied at once
constexpr int kLaMinSegChunks = 8;  // a segment is at least this many chunks long
constexpr int kLaMaxSegments = 64;

static inline int la_pad16(int n) { return (n + 15) / 16 * 16; }

// Columns of the value dimension that one workgroup of the chunked kernel owns: 16 for each of its four or eight waves.
static inline int la_value_cols(int vdim) { return vdim <= 64 ? 64 : 128; }

// Segments of a portion of up to max_len rows: as many as (sequences x heads x value slices) leave compute units for,
// one workgroup each, but no shorter than kLaMinSegChunks chunks (a segment's start state costs a second reading of
// its keys and values and two passes over a state's bytes).
static inline int la_segments(int64_t workgroups, int cus, int max_len) {
    if (workgroups <= 0 || max_len <= 0) return 1;
    const int64_t chunks = (max_len + kLaChunk - 1) / kLaChunk;
    int64_t want = cus / workgroups;
    const int64_t most = chunks / kLaMinSegChunks;
    if (want > most) want = most;
    if (want > kLaMaxSegments) want = kLaMaxSegments;
    return want < 1 ? 1 : (int)want;
}

// Rows per segment: whole chunks.
static inline int la_segment_rows(int max_len, int segments) {
    const int chunks = (max_len + kLaChunk - 1) / kLaChunk;
    return (chunks + segments - 1) / segments * kLaChunk;
}

static inline size_t la_state_floats(int dim, int vdim) { return (size_t)la_pad16(dim) * la_pad16(vdim); }
static inline size_t la_workspace_bytes(int64_t batch, int heads, int dim, int vdim, int segments) {
    return segments <= 1 ? 0 : (size_t)batch * heads * segments * la_state_floats(dim, vdim) * sizeof(float);
}

// Gated recurrences: a head's floats in the pool (with a normaliser: S, and n and the running maximum once per 64 value
// columns) and the segments' states (S, n, and three scalars).
static inline size_t gl_state_floats(bool normaliser, int dim, int vdim) {
    return la_state_floats(dim, vdim) + (normaliser ? (size_t)((vdim + 63) / 64) * (la_pad16(dim) + 16) : 0);
}
static inline size_t gl_workspace_bytes(int64_t batch, int heads, int dim, int vdim, int segments) {
    return segments <= 1 ? 0 : (size_t)batch * heads * segments * (la_state_floats(dim, vdim) + la_pad16(dim) + 16) * sizeof(float);
}
