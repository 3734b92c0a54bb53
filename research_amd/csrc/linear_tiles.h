// What the chunked linear-recurrence kernels share: 64-row tiles of bf16 rows loaded in 4 x 4 blocks and laid out in LDS
// row-major and transposed, 32-bit factors as a sum of two bf16 terms, states as buffers.
#pragma once
#include "lightning_plan.h"
#include "row_common.h"

namespace {

typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 la_bf4 __attribute__((ext_vector_type(4)));
typedef float f4 __attribute__((ext_vector_type(4)));
typedef uint32_t la_u2 __attribute__((ext_vector_type(2)));
typedef uint32_t la_u4 __attribute__((ext_vector_type(4)));

// LDS layouts.  Row-major [64][KD + 8] for Q and K (the pad moves a row by 16 bytes over the banks).  Transposed
// [rows][64 s] for K^T and V^T: eight 16-byte chunks per row, chunk c of row r at position c ^ la_hash(r), so that
// both the transposing 8-byte writes (rows 4 apart) and the 16-byte operand reads (consecutive rows) spread over the
// banks without a pad.
// (Of the row bits that change over the lanes of an access - 0 to 3 in reads, 2 to 6 in writes - bit 0 picks half of the
// banks, and three more have to reach all eight chunks.)
__device__ __forceinline__ int la_hash(int r) { return ((r >> 1) & 7) ^ ((r >> 4) & 1); }
__device__ __forceinline__ int la_tr(int r, int s) { return r * 64 + ((((s >> 3) ^ la_hash(r)) << 3) | (s & 7)); }

__device__ __forceinline__ f4 la_mfma(bf8 x, bf8 y, f4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, y, c, 0, 0, 0); }

__device__ __forceinline__ bf8 la_read8(const __bf16 *p) { return *reinterpret_cast<const bf8 *>(p); }
__device__ __forceinline__ bf8 la_join(la_bf4 x, la_bf4 y) { return bf8{x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]}; }
__device__ __forceinline__ bf8 la_read44(const __bf16 *p, const __bf16 *q) {
    return la_join(*reinterpret_cast<const la_bf4 *>(p), *reinterpret_cast<const la_bf4 *>(q));
}
// Lane i of 16 gets column i of four rows from a 4 x 16 block in LDS whose lane s points at row s / 4, columns 4 (s % 4) ..
__device__ __forceinline__ la_bf4 la_read_tr(const __bf16 *p) {
    typedef short s4 __attribute__((ext_vector_type(4)));
    return __builtin_bit_cast(la_bf4, __builtin_amdgcn_ds_read_tr16_b64_v4i16((s4 __attribute__((address_space(3))) *)p));
}
// Pairs x = hi + lo, packed bf16
__device__ __forceinline__ void la_split2(float x0, float x1, uint32_t &hi, uint32_t &lo) {
    hi = row_pack_bf16(x0, x1);
    lo = row_pack_bf16(x0 - __builtin_bit_cast(float, hi << 16), x1 - __builtin_bit_cast(float, hi & 0xffff0000u));
}
struct LaSplit {  // eight values as two operands
    uint32_t hi[4], lo[4];
    __device__ __forceinline__ bf8 high() const { return __builtin_bit_cast(bf8, la_u4{hi[0], hi[1], hi[2], hi[3]}); }
    __device__ __forceinline__ bf8 low() const { return __builtin_bit_cast(bf8, la_u4{lo[0], lo[1], lo[2], lo[3]}); }
};

struct LaBlock {  // four rows of four consecutive columns, raw bf16
    uint2 r[4];
};

// A tile of `rows` rows of `cols` columns at row stride `ld` as a buffer: loads past its end give zeros, stores past it
// are dropped.  (Columns past `cols` inside a row are the caller's: it gives such lanes the offset kLaOutside.)
constexpr uint32_t kLaOutside = 0x40000000u;
__device__ __forceinline__ __amdgpu_buffer_rsrc_t la_tile(const uint16_t *base, int64_t ld, int rows, int cols) {
    return __builtin_amdgcn_make_buffer_rsrc((void *)base, 0, (int)(((rows - 1) * ld + cols) * 2), 0x00020000);
}
// Byte offset of the 4 x 4 block at (row s, column c)
__device__ __forceinline__ uint32_t la_block_off(int64_t ld, int s, int c, int cols) {
    return c < cols ? (uint32_t)(s * ld + c) * 2u : kLaOutside;
}
__device__ __forceinline__ LaBlock la_load_block(__amdgpu_buffer_rsrc_t tile, uint32_t off, uint32_t row_bytes) {
    LaBlock b;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const la_u2 x = __builtin_amdgcn_raw_buffer_load_b64(tile, off + i * row_bytes, 0, 0);
        b.r[i] = make_uint2(x[0], x[1]);
    }
    return b;
}

// silu of a raw pair, packed again
__device__ __forceinline__ uint32_t la_silu2(uint32_t w) {
    return row_pack_bf16(row_silu<pa_bf16>(__builtin_bit_cast(float, w << 16)),
                         row_silu<pa_bf16>(__builtin_bit_cast(float, w & 0xffff0000u)));
}

// The block, or with ACT its silu, to a row-major tile (when `rm` is given) and, transposed, to a [column][64] tile
template <bool ACT> __device__ __forceinline__ void la_put_block(LaBlock b, int s, int c, __bf16 *rm, int ld_rm, __bf16 *tr) {
    if constexpr (ACT) {
#pragma unroll
        for (int i = 0; i < 4; ++i) b.r[i] = make_uint2(la_silu2(b.r[i].x), la_silu2(b.r[i].y));
    }
    if (rm) {
#pragma unroll
        for (int i = 0; i < 4; ++i) *reinterpret_cast<uint2 *>(rm + (s + i) * ld_rm + c) = b.r[i];
    }
    if (!tr) return;
    // columns 0/1 and 2/3 of rows 0..3 as pairs over rows (v_perm picks the low or the high halves)
    auto low = [](uint32_t x, uint32_t y) { return __builtin_amdgcn_perm(y, x, 0x05040100u); };
    auto high = [](uint32_t x, uint32_t y) { return __builtin_amdgcn_perm(y, x, 0x07060302u); };
    *reinterpret_cast<uint2 *>(tr + la_tr(c, s)) = make_uint2(low(b.r[0].x, b.r[1].x), low(b.r[2].x, b.r[3].x));
    *reinterpret_cast<uint2 *>(tr + la_tr(c + 1, s)) = make_uint2(high(b.r[0].x, b.r[1].x), high(b.r[2].x, b.r[3].x));
    *reinterpret_cast<uint2 *>(tr + la_tr(c + 2, s)) = make_uint2(low(b.r[0].y, b.r[1].y), low(b.r[2].y, b.r[3].y));
    *reinterpret_cast<uint2 *>(tr + la_tr(c + 3, s)) = make_uint2(high(b.r[0].y, b.r[1].y), high(b.r[2].y, b.r[3].y));
}

constexpr int kLaPitchA = 72;  // bf16 per row of the decayed scores

int la_cus() {
    static int cached[64];
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return 256;
    int n = __atomic_load_n(&cached[dev], __ATOMIC_RELAXED);
    if (n == 0) {
        if (hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || n <= 0) n = 256;
        __atomic_store_n(&cached[dev], n, __ATOMIC_RELAXED);
    }
    return n;
}

template <typename K> int la_big_lds(K kernel, size_t bytes, const char *what) {
    if (bytes > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
        if (e != hipSuccess) return pa_fail(PA_ERR_HIP, "%s: %s", what, hipGetErrorString(e));
    }
    return PA_OK;
}

}  // namespace
