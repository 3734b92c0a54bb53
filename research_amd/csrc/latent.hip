// Latent attention's operands.  pa_latent_append: from the joint projection of a row to rotated queries and to the one row
// the pool keeps per token, [normed latent | rotated key part shared by all heads].  pa_latent_gather: stretches of those
// rows, contiguous, from which keys and values per head are made again for prompts.  HBM-bound.
#include "row_common.h"

namespace {

constexpr int kLatTile = PA_QKV_TILE_ROWS;

struct LatentArgs {
    const void *u;  // [rows][ldu]: heads of dim + rot, then rank + rot
    int64_t ldu, n_rows;
    const float *norm_w;  // [rank]
    const float2 *rope;   // [rope_rows][rot / 2]
    int64_t rope_rows;
    const int32_t *ctx_lens, *q_lens, *q_starts, *tiles;
    const int64_t *slots;
    int64_t total_slots;
    void *q_out;  // [rows][heads][d]
    void *pool;   // [total_slots][row]
    int batch, heads, dim, rot, rank, d, row, heads_per_wg;
    float eps, q_scale;
};

// V consecutive elements from element e of a part whose rotation starts at `first` (a multiple of V, like e and rot; V = 1:
// the partner is read beside it).
template <typename T, int V> __device__ __forceinline__ void load_turned(const T *p, int e, int first, int rot, const float2 *cs, float *f) {
    if constexpr (V > 1) {
        row_load<T, V>(p + e, f);
        if (e >= first && e < first + rot) {
#pragma unroll
            for (int j = 0; j < V / 2; ++j) {
                const float2 t = cs[(e - first) / 2 + j];
                const float x = f[2 * j], y = f[2 * j + 1];
                f[2 * j] = x * t.x - y * t.y;
                f[2 * j + 1] = y * t.x + x * t.y;
            }
        }
    } else {
        f[0] = pa_scalar<T>::load(p + e);
        if (e >= first && e < first + rot) {
            const int r = e - first;
            const float2 t = cs[r / 2];
            const float other = pa_scalar<T>::load(p + first + (r ^ 1));
            f[0] = r & 1 ? f[0] * t.x + other * t.y : f[0] * t.x - other * t.y;
        }
    }
}

template <typename T, int V> __global__ __launch_bounds__(256) void latent_append_kernel(const LatentArgs a) {
    int b = blockIdx.x, i0 = 0, n = 1;
    int64_t row0 = b;
    if (a.tiles) {
        b = a.tiles[2 * blockIdx.x];
        i0 = a.tiles[2 * blockIdx.x + 1];
        if (b < 0 || b >= a.batch) return;
        n = a.q_lens[b];
        row0 = a.q_starts[b];
    }
    const int pos0 = a.ctx_lens[b] - n;
    if (pos0 < 0 || i0 < 0 || i0 >= n || row0 < 0 || row0 + n > a.n_rows) return;
    const int rows = n - i0 < kLatTile ? n - i0 : kLatTile, tid = threadIdx.x;
    const T *u = reinterpret_cast<const T *>(a.u);
    auto turns = [&](int i) {
        int64_t pos = pos0 + i0 + i;
        if (pos >= a.rope_rows) pos = a.rope_rows - 1;  // (the caller sizes the table; never read past it)
        return a.rope + pos * (a.rot / 2);
    };
    if (blockIdx.y > 0) {  // some of the query heads
        const int h0 = (blockIdx.y - 1) * a.heads_per_wg, hn = a.heads - h0 < a.heads_per_wg ? a.heads - h0 : a.heads_per_wg;
        const int per = (a.d + V - 1) / V, size = a.dim + a.rot;
        for (int item = tid; item < rows * hn * per; item += 256) {
            const int e = item % per * V, h = item / per % hn, i = item / per / hn;
            const int64_t row = row0 + i0 + i;
            float f[V];
            row_zero<V>(f);
            if (e < size) load_turned<T, V>(u + row * a.ldu + (int64_t)(h0 + h) * size, e, a.dim, a.rot, turns(i), f);
#pragma unroll
            for (int j = 0; j < V; ++j) f[j] *= a.q_scale;
            row_store<T, V>(reinterpret_cast<T *>(a.q_out) + (row * a.heads + h0 + h) * a.d + e, f);
        }
        return;
    }
    const int lane = tid & 63;
    for (int i = tid / 64; i < rows; i += 4) {  // a wave per row
        const int64_t row = row0 + i0 + i, slot = a.slots[row];
        if (slot < 0 || slot >= a.total_slots) continue;
        const T *src = u + row * a.ldu + (int64_t)a.heads * (a.dim + a.rot);
        T *dst = reinterpret_cast<T *>(a.pool) + slot * a.row;
        float ss = 0.f;
        for (int e = lane * V; e < a.rank; e += 64 * V) {
            float f[V];
            row_load<T, V>(src + e, f);
#pragma unroll
            for (int j = 0; j < V; ++j) ss = fmaf(f[j], f[j], ss);
        }
        const float inv = 1.f / sqrtf(pa_group_sum<64>(ss) / (float)a.rank + a.eps);
        const float2 *cs = turns(i);
        for (int e = lane * V; e < a.row; e += 64 * V) {
            float f[V], w[V];
            row_zero<V>(f);
            if (e < a.rank) {
                row_load<T, V>(src + e, f);
                row_load<float, V>(a.norm_w + e, w);
#pragma unroll
                for (int j = 0; j < V; ++j) f[j] *= inv * w[j];
            } else if (e < a.rank + a.rot) {
                load_turned<T, V>(src, e, a.rank, a.rot, cs, f);
            }
            row_store<T, V>(dst + e, f);
        }
    }
}

// out row r = pool row slots[r], zeros for a slot out of range; rows of `vecs` 16-byte vectors
__global__ __launch_bounds__(256) void latent_gather_kernel(const uint4 *pool, const int64_t *slots, int64_t total_slots, uint4 *out,
                                                            int64_t rows, int vecs) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int64_t r = i / vecs;
    if (r >= rows) return;
    const int64_t slot = slots[r];
    out[i] = slot >= 0 && slot < total_slots ? pool[slot * vecs + (i - r * vecs)] : make_uint4(0, 0, 0, 0);
}

}  // namespace

extern "C" int pa_latent_append(const void *u, int64_t u_stride, int64_t n_rows, const float *norm_weight, float eps,
                                const float *rope, int64_t rope_rows, const int32_t *ctx_lens, const int32_t *q_lens,
                                const int32_t *q_starts, const int32_t *tiles, int n_tiles, int batch, const int64_t *slots,
                                int64_t total_slots, void *q_out, void *pool, int num_heads, int dim, int rot_dim, int rank,
                                int q_dim, int pool_row, float q_scale, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && n_tiles >= 0 && total_slots >= 0 && rope_rows >= 0, "pa_latent_append: a count is negative");
    PA_REQUIRE(num_heads > 0 && dim >= 0 && rot_dim >= 0 && rot_dim % 2 == 0 && dim + rot_dim > 0 && rank > 0,
               "pa_latent_append: heads / dim / rot_dim / rank out of range");
    PA_REQUIRE(q_dim >= dim + rot_dim && q_dim % 8 == 0 && pool_row >= rank + rot_dim && pool_row % 8 == 0,
               "q_dim=%d / pool_row=%d must be multiples of 8 that hold their parts", q_dim, pool_row);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_latent_append: dtype=%d is not F32 or BF16", dtype);
    PA_REQUIRE(u_stride >= (int64_t)num_heads * (dim + rot_dim) + rank + rot_dim, "u_stride=%lld is shorter than its row", (long long)u_stride);
    PA_REQUIRE(tiles || (n_tiles == batch && n_rows >= batch), "without tiles every sequence brings one row");
    if (n_rows == 0 || n_tiles == 0) return PA_OK;
    PA_REQUIRE(u && norm_weight && ctx_lens && slots && q_out && pool, "pa_latent_append: NULL argument");
    PA_REQUIRE(!tiles || (q_lens && q_starts), "tiles without q_lens / q_starts");
    PA_REQUIRE(rot_dim == 0 || (rope && rope_rows > 0), "rot_dim=%d without a table", rot_dim);
    PA_REQUIRE(pa_aligned16(q_out) && pa_aligned16(pool), "pointers must be 16-byte aligned");
    LatentArgs a{u, u_stride, n_rows, norm_weight, (const float2 *)rope, rope_rows, ctx_lens, q_lens, q_starts, tiles, slots, total_slots,
                 q_out, pool, batch, num_heads, dim, rot_dim, rank, q_dim, pool_row, 0, eps, q_scale};
    const bool vec = dim % 8 == 0 && rot_dim % 8 == 0 && rank % 8 == 0 && u_stride % 8 == 0 && pa_aligned16(u) && pa_aligned16(norm_weight);
    // (about one pass of a workgroup's threads over its heads)
    const int per_head = (tiles ? kLatTile : 1) * (q_dim / (vec ? 8 : 1));
    a.heads_per_wg = per_head >= 2048 ? 1 : 2048 / per_head;
    const int parts = (num_heads + a.heads_per_wg - 1) / a.heads_per_wg;
    PA_REQUIRE(parts < 65535, "pa_latent_append: too many heads for one launch");
    const dim3 grid((unsigned)n_tiles, (unsigned)(1 + parts)), block(256);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) {
        if (vec) latent_append_kernel<float, 8><<<grid, block, 0, s>>>(a);
        else latent_append_kernel<float, 1><<<grid, block, 0, s>>>(a);
    } else {
        if (vec) latent_append_kernel<pa_bf16, 8><<<grid, block, 0, s>>>(a);
        else latent_append_kernel<pa_bf16, 1><<<grid, block, 0, s>>>(a);
    }
    PA_CHECK_LAUNCH("pa_latent_append");
    return PA_OK;
}

extern "C" int pa_latent_gather(const void *pool, const int64_t *slots, int64_t total_slots, void *out, int64_t rows, int pool_row,
                                int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && total_slots >= 0 && pool_row > 0 && pool_row % 8 == 0, "pa_latent_gather: sizes out of range");
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_latent_gather: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(pool && slots && out && pa_aligned16(pool) && pa_aligned16(out), "pa_latent_gather: NULL or unaligned argument");
    const int vecs = pool_row / (dtype == PA_F32 ? 4 : 8);
    const int64_t grid = (rows * vecs + 255) / 256;
    PA_REQUIRE(grid <= 0x7fffffff, "pa_latent_gather: rows=%lld is too large for one launch", (long long)rows);
    latent_gather_kernel<<<dim3((unsigned)grid), dim3(256), 0, (hipStream_t)stream>>>((const uint4 *)pool, slots, total_slots, (uint4 *)out,
                                                                                   rows, vecs);
    PA_CHECK_LAUNCH("pa_latent_gather");
    return PA_OK;
}
