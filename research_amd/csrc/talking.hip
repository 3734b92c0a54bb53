// Entry points of attention with mixed heads, and its kernels on the vector units: 32-bit rows, and sizes that the matrix-core
// kernels (talking_decode.hip, talking_prefill.hip) do not have.
#include "talking.h"

namespace {

// The score of a key in units of the base-2 exponential (T float: library functions throughout)
template <typename T> __device__ __forceinline__ float talk_score(const TalkArgs &a, int h, const T *q, const T *k, int dist) {
    float s = 0.f;
    for (int e = 0; e < a.n1; ++e) s = fmaf(pa_scalar<T>::load(q + e), pa_scalar<T>::load(k + e), s);
    s *= a.scale;
    if (a.size) s -= a.size[h] * logf(fmaf(a.rate[h], (float)dist, 1.f));
    return s * kScoredLog2e;
}

// A wave per (row, head), a key per lane.
template <typename T> __global__ __launch_bounds__(256) void talk_lse_vector_kernel(const TalkArgs a) {
    const int b = blockIdx.z, i = blockIdx.y, lane = threadIdx.x & 63, h = blockIdx.x * 4 + threadIdx.x / 64;
    ScoredPortion p;
    if (h >= a.heads || !scored_portion(a, b, p) || i >= p.n) return;
    const int64_t row = p.row0 + i;
    const int pos = p.pos0 + i;
    const T *q = reinterpret_cast<const T *>(a.q1) + row * a.q1_row + h * a.q1_head;
    const T *k = reinterpret_cast<const T *>(a.k) + (int64_t)(h / a.n_rep) * a.k_dim;
    const int32_t *table = a.bt + b * a.bt_stride;
    float m = kScoredNone, l = 0.f;
    for (int j = lane; j <= pos; j += 64) {
        const int64_t slot = scored_slot(a, table, j);
        const float s = slot >= 0 ? talk_score<T>(a, h, q, k + slot * ((int64_t)a.hkv * a.k_dim), pos - j) : kScoredNone;
        const float next = fmaxf(m, s);
        l = l * exp2f(m - next) + exp2f(s - next);
        m = next;
    }
    float top = m;
#pragma unroll
    for (int d = 32; d > 0; d /= 2) top = fmaxf(top, __shfl_xor(top, d, 64));
    l = pa_group_sum<64>(l * exp2f(m - top));
    if (lane == 0) a.lse[row * a.heads + h] = top + log2f(l);
}

// A workgroup per row: weights of 64 keys for all heads, their mixture, then the value columns of all heads.
constexpr int kTalkKeys = 64;
template <typename T, int VPT> __global__ __launch_bounds__(256) void talk_mix_vector_kernel(const TalkArgs a) {
    extern __shared__ float talk_lds[];
    float *p_s = talk_lds, *w_s = p_s + a.heads * kTalkKeys;
    __shared__ int64_t slots[kTalkKeys];
    const int b = blockIdx.z, i = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    ScoredPortion p;
    if (!scored_portion(a, b, p) || i >= p.n) return;
    const int64_t row = p.row0 + i;
    const int pos = p.pos0 + i, columns = a.heads * a.vdim;
    const int32_t *table = a.bt + b * a.bt_stride;
    const T *q = reinterpret_cast<const T *>(a.q1) + row * a.q1_row;
    float acc[VPT];
    row_zero<VPT>(acc);
    for (int j0 = 0; j0 <= pos; j0 += kTalkKeys) {
        const int j = j0 + lane, keys = pos + 1 - j0 < kTalkKeys ? pos + 1 - j0 : kTalkKeys;
        const int64_t slot = j <= pos ? scored_slot(a, table, j) : -1;
        if (wave == 0) slots[lane] = slot;
        for (int h = wave; h < a.heads; h += 4) {
            const T *k = reinterpret_cast<const T *>(a.k) + (slot < 0 ? 0 : slot) * ((int64_t)a.hkv * a.k_dim) + (h / a.n_rep) * a.k_dim;
            p_s[h * kTalkKeys + lane] =
                slot >= 0 ? exp2f(talk_score<T>(a, h, q + h * a.q1_head, k, pos - j) - a.lse[row * a.heads + h]) : 0.f;
        }
        __syncthreads();
        for (int n = tid; n < a.heads * kTalkKeys; n += 256) {
            const float *t = a.talk + (n / kTalkKeys) * a.heads;
            float w = 0.f;
            for (int g = 0; g < a.heads; ++g) w = fmaf(t[g], p_s[g * kTalkKeys + lane], w);
            w_s[n] = w;
        }
        __syncthreads();
#pragma unroll
        for (int c = 0; c < VPT; ++c) {
            const int n = tid + 256 * c;
            if (n >= columns) break;
            const int h = n / a.vdim;
            const T *v = reinterpret_cast<const T *>(a.v) + (h / a.n_rep) * a.v_dim + (n - h * a.vdim);
            for (int t = 0; t < keys; ++t)
                if (slots[t] >= 0) acc[c] = fmaf(w_s[h * kTalkKeys + t], pa_scalar<T>::load(v + slots[t] * ((int64_t)a.hkv * a.v_dim)), acc[c]);
        }
        __syncthreads();
    }
    T *out = reinterpret_cast<T *>(a.out) + row * columns;
#pragma unroll
    for (int c = 0; c < VPT; ++c)
        if (tid + 256 * c < columns) pa_scalar<T>::store(out + tid + 256 * c, acc[c]);
}

template <typename T> int launch_vector(const TalkArgs &a, hipStream_t s) {
    talk_lse_vector_kernel<T><<<dim3((unsigned)((a.heads + 3) / 4), (unsigned)a.max_q_len, (unsigned)a.batch), dim3(256), 0, s>>>(a);
    PA_CHECK_LAUNCH("pa_talking_attention (sums)");
    const dim3 grid(1, (unsigned)a.max_q_len, (unsigned)a.batch), block(256);
    const size_t lds = (size_t)2 * a.heads * kTalkKeys * sizeof(float);
    const int columns = a.heads * a.vdim;
    if (lds > 60 * 1024) {
        const void *kernels[3] = {reinterpret_cast<const void *>(talk_mix_vector_kernel<T, 8>), reinterpret_cast<const void *>(talk_mix_vector_kernel<T, 32>),
                                  reinterpret_cast<const void *>(talk_mix_vector_kernel<T, 128>)};
        for (const void *k : kernels) {
            const hipError_t e = hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            if (e != hipSuccess) return pa_fail(PA_ERR_HIP, "pa_talking_attention: %s", hipGetErrorString(e));
        }
    }
    if (columns <= 8 * 256) talk_mix_vector_kernel<T, 8><<<grid, block, lds, s>>>(a);
    else if (columns <= 32 * 256) talk_mix_vector_kernel<T, 32><<<grid, block, lds, s>>>(a);
    else talk_mix_vector_kernel<T, 128><<<grid, block, lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_talking_attention");
    return PA_OK;
}

size_t lse_bytes(int64_t rows, int heads) { return ((size_t)rows * heads * sizeof(float) + 255) / 256 * 256; }

}  // namespace

extern "C" size_t pa_talking_workspace_bytes(int64_t n_rows, int batch, int num_q_heads, int num_kv_heads, int vdim, int64_t max_keys,
                                             int decode) {
    if (n_rows < 0 || batch < 0 || num_q_heads <= 0 || num_kv_heads <= 0 || vdim <= 0 || max_keys < 0) return 0;
    return lse_bytes(n_rows, num_q_heads) + (decode ? pa_talking_decode_bytes(batch, num_q_heads, num_kv_heads, vdim, max_keys) : 0);
}

extern "C" int pa_talking_attention(const void *q, int64_t q_row, int64_t q_head, int dim, const void *k_cache, int k_dim,
                                    const void *v_cache, int v_dim, int vdim, const int32_t *block_tables, int64_t bt_stride, int block_size,
                                    int64_t num_blocks, const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
                                    int64_t n_rows, int batch, int max_q_len, int num_q_heads, int num_kv_heads, float scale,
                                    const float *bias_size, const float *bias_rate, const float *talk, void *out, int dtype,
                                    void *workspace, size_t workspace_bytes, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && max_q_len >= 0 && num_blocks >= 0 && bt_stride >= 0, "pa_talking_attention: a count is negative");
    PA_REQUIRE(dim > 0 && vdim > 0 && k_dim >= dim && v_dim >= vdim, "pa_talking_attention: dim / vdim do not fit the pool");
    PA_REQUIRE(num_q_heads > 0 && num_kv_heads > 0 && num_q_heads % num_kv_heads == 0,
               "num_q_heads=%d must be a positive multiple of num_kv_heads=%d", num_q_heads, num_kv_heads);
    PA_REQUIRE(block_size > 0, "block_size=%d out of range", block_size);
    PA_REQUIRE((q_lens == nullptr) == (q_starts == nullptr), "q_lens and q_starts come together");
    PA_REQUIRE((bias_size == nullptr) == (bias_rate == nullptr), "bias_size and bias_rate come together");
    PA_REQUIRE(batch <= 65535 && max_q_len <= 65535, "batch=%d / max_q_len=%d above 65535", batch, max_q_len);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_talking_attention: dtype=%d is not F32 or BF16", dtype);
    if (num_q_heads > kTalkMaxHeads || dim > 256 || vdim > 256)
        return pa_fail(PA_ERR_UNSUPPORTED, "pa_talking_attention: heads=%d above %d, or dim=%d / vdim=%d above 256", num_q_heads, kTalkMaxHeads, dim, vdim);
    if (n_rows == 0 || batch == 0 || (q_lens && max_q_len == 0)) return PA_OK;
    PA_REQUIRE(q && k_cache && v_cache && ctx_lens && talk && out && (block_tables || bt_stride == 0), "pa_talking_attention: NULL argument");
    PA_REQUIRE(q_lens || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    const size_t lse = lse_bytes(n_rows, num_q_heads);
    if (!workspace || workspace_bytes < lse) return pa_fail(PA_ERR_WORKSPACE, "pa_talking_attention: %zu bytes of workspace needed", lse);
    PA_REQUIRE(pa_aligned16(workspace), "the workspace must be 16-byte aligned");
    TalkArgs a{};
    a.q1 = a.q2 = q; a.q1_row = a.q2_row = q_row; a.q1_head = a.q2_head = q_head; a.n1 = dim;
    a.k = k_cache; a.v = v_cache; a.k_dim = k_dim; a.v_dim = v_dim; a.vdim = vdim;
    a.bt = block_tables; a.bt_stride = bt_stride; a.num_blocks = num_blocks; a.bs = block_size;
    a.ctx_lens = ctx_lens; a.q_lens = q_lens; a.q_starts = q_starts; a.n_rows = n_rows; a.batch = batch;
    a.max_q_len = q_lens ? max_q_len : 1; a.heads = num_q_heads; a.hkv = num_kv_heads; a.n_rep = num_q_heads / num_kv_heads;
    a.scale = scale; a.out = out; a.splits = 1;
    a.bs_shift = (block_size & (block_size - 1)) == 0 ? __builtin_ctz((unsigned)block_size) : -1;
    a.size = bias_size; a.rate = bias_rate; a.talk = talk; a.lse = (float *)workspace;
    hipStream_t s = (hipStream_t)stream;
    int rc = PA_OK;
    if (pa_talking_decode_launch(a, dtype, (char *)workspace + lse, workspace_bytes - lse, s, rc) || pa_talking_prefill_launch(a, dtype, s, rc))
        return rc;
    return dtype == PA_F32 ? launch_vector<float>(a, s) : launch_vector<pa_bf16>(a, s);
}
