// Host-testable arithmetic of the expert products: how many tiles the lists can make and which kernel runs them.  Plain C++.
#pragma once
#include <stdint.h>

// Tiles of `bm` items that `items` items of at most `experts` lists can make: every list leaves one tile part-filled, and
// no more lists than items are non-empty.
static inline int64_t moe_max_tiles(int64_t items, int experts, int bm) {
    const int64_t lists = items < experts ? items : experts;
    return lists + (items - lists) / bm;
}

enum MoeShape { kMoeStream16, kMoeStream32, kMoeStream64, kMoeTile64, kMoeTile256 };

// By the items an expert has on average (lists of unequal length fill the next tile up).
static inline MoeShape moe_shape(int64_t items, int experts) {
    const int64_t mean = items / experts;
    return mean <= 8 ? kMoeStream16 : mean <= 20 ? kMoeStream32 : mean <= 48 ? kMoeStream64 : mean <= 160 ? kMoeTile64 : kMoeTile256;
}
