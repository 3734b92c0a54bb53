// Host-testable arithmetic of the expert products: how many tiles the lists can make and which kernel runs them.  Plain C++.
#pragma once
#include <stdint.h>

// Tiles of `bm` items that `items` items of at most `experts` lists can make: every list leaves one tile part-filled, and
// no more lists than items are non-empty.
static inline int64_t moe_max_tiles(int64_t items, int experts, int bm) {
    const int64_t lists = items < experts ? items : experts;
    return lists + (items - lists) / bm;
}

enum MoeShape { kMoeStream, kMoeTile64, kMoeTile256 };

// By the items an expert has on average (lists of unequal length fill the next tile up).
static inline MoeShape moe_shape(int64_t items, int experts) {
    const int64_t mean = items / experts;
    return mean <= 4 ? kMoeStream : mean <= 160 ? kMoeTile64 : kMoeTile256;
}

// Rows of a part of the choice of experts (one workgroup): few parts, so that a part's place behind the others is quickly
// summed, but one row per wave (sixteen per workgroup) while there are few rows; a part's items fit LDS.
static inline int moe_part_rows(int64_t rows, int top) {
    int64_t n = (rows + 255) / 256;
    if (n < 16) n = 16;
    const int64_t most = 8192 / top;
    return (int)(n < most ? n : most);
}
static inline int64_t moe_parts(int64_t rows, int top) { return (rows + moe_part_rows(rows, top) - 1) / moe_part_rows(rows, top); }
