// Queries and keys turned by their position and brought to unit root mean square a head, and the page write of
// keys and values, from one product's float results.
//
//   of every query and key head the first 2 * half coordinates are turned (i with i + half) by position * freq[i],
//   then the head is divided by sqrt(mean over its `key_dim` coordinates of their squares + eps);
//   queries are also multiplied by their head's factor (optional) -> out_q [T, heads, pad] in the storage type
//   keys   -> the token's entry of the key pool, values as projected -> its entry of the value pool
//
// A row of `qkv` is q (heads x key_dim) | k (kv_heads x key_dim) | v (kv_heads x value_dim), floats; whatever lies
// behind (a gate's logits) is not touched.  Heads are followed by zeros up to `pad`, the pools' entry width (the
// attention kernels take one width for keys and values, a multiple of 16).  A wave a (row, head).
#include "api.h"
#include "common.h"

namespace st {

constexpr int kUnitLane = 4;                 // coordinates a lane: heads of up to 256

template <typename T>
__global__ __launch_bounds__(256) void unit_qk_write_kernel(
    T* __restrict__ out_q, T* __restrict__ k_cache, T* __restrict__ v_cache, int64_t page_stride,
    const float* __restrict__ qkv, int64_t stride, const float* __restrict__ freq, int half,
    const float* __restrict__ factor, const int* __restrict__ token_item, const int* __restrict__ positions,
    const int* __restrict__ block_table, int max_pages, int page_size, int64_t waves, int heads, int kv_heads, int key_dim,
    int value_dim, int pad, float eps, int write) {
    const int64_t u = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (u >= waves) return;
    const int lane = threadIdx.x & 63;
    const int per_row = heads + 2 * kv_heads;
    const int64_t t = u / per_row;
    const int unit = (int)(u - t * per_row);
    const bool is_q = unit < heads, is_v = unit >= heads + kv_heads;
    const int item = token_item[t], pos = positions[t];
    const bool padding = item < 0 || pos < 0;
    if (!is_q && (padding || !write)) return;
    T* dst;
    if (is_q) {
        dst = out_q + (t * heads + unit) * pad;
    } else {
        const int page = block_table[(int64_t)item * max_pages + pos / page_size];
        if (page < 0) return;
        const int h = is_v ? unit - heads - kv_heads : unit - heads;
        dst = (is_v ? v_cache : k_cache) + (int64_t)page * page_stride + ((int64_t)h * page_size + pos % page_size) * pad;
    }
    const int dim = is_v ? value_dim : key_dim;
    const float* src = qkv + t * stride + (is_v ? (int64_t)(heads + kv_heads) * key_dim + (int64_t)(unit - heads - kv_heads) * value_dim
                                                : (int64_t)unit * key_dim);
    float y[kUnitLane];
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < kUnitLane; ++e) {
        const int d = lane + 64 * e;
        y[e] = 0.f;
        if (d < dim && !padding) {
            y[e] = src[d];
            if (!is_v && d < 2 * half) {
                const int i = d < half ? d : d - half;
                const float other = src[d < half ? d + half : i];
                const float a = (float)pos * freq[i];
                const float c = cosf(a), s = sinf(a);
                y[e] = d < half ? y[e] * c - other * s : y[e] * c + other * s;
            }
        }
        ss = fmaf(y[e], y[e], ss);
    }
    float r = 1.f;
    if (!is_v) {
        r = 1.f / sqrtf(wave_sum(ss) / (float)dim + eps);
        if (is_q && factor) r *= factor[unit];
    }
#pragma unroll
    for (int e = 0; e < kUnitLane; ++e) {
        const int d = lane + 64 * e;
        if (d < pad) Elem<T>::store(dst + d, y[e] * r);
    }
}

}  // namespace st

using namespace st;

// Pools [pages, kv_heads, page_size, pad] of `dtype`; freq [half] (half 0: nothing turns); factor [heads] or null;
// write == 0: the queries only.
extern "C" int st_unit_qk_write(void* out_q, void* k_cache, void* v_cache, int64_t page_stride, const float* qkv,
                                int64_t stride, const float* freq, int half, const float* factor, const int* token_item,
                                const int* positions, const int* block_table, int max_pages, int page_size,
                                int num_tokens, int heads, int kv_heads, int key_dim, int value_dim, int pad, float eps,
                                int write, int dtype, hipStream_t stream) {
    ST_CHECK(num_tokens >= 0 && heads > 0 && kv_heads > 0 && key_dim > 0 && value_dim > 0 && page_size > 0 && max_pages > 0,
             "unit_qk_write: bad sizes");
    ST_CHECK(pad >= key_dim && pad >= value_dim && pad <= 64 * kUnitLane, "unit_qk_write: heads of %d and %d in entries of %d "
             "(up to %d)", key_dim, value_dim, pad, 64 * kUnitLane);
    ST_CHECK(half >= 0 && 2 * half <= key_dim && (freq || half == 0), "unit_qk_write: %d turned coordinates in heads of %d",
             2 * half, key_dim);
    ST_CHECK(stride >= (int64_t)(heads + kv_heads) * key_dim + (int64_t)kv_heads * value_dim, "unit_qk_write: rows shorter than q, k and v");
    ST_CHECK(eps > 0.f, "unit_qk_write: eps must be positive");
    if (num_tokens == 0) return 0;
    ST_CHECK(out_q && qkv && token_item && positions && (!write || (k_cache && v_cache && block_table)),
             "unit_qk_write: null operand");
    const int64_t waves = (int64_t)num_tokens * (heads + 2 * kv_heads);
    const unsigned grid = (unsigned)((waves + 3) / 4);
#define ST_UQ(T)                                                                                                     \
    unit_qk_write_kernel<T><<<grid, 256, 0, stream>>>((T*)out_q, (T*)k_cache, (T*)v_cache, page_stride, qkv, stride, freq, \
        half, factor, token_item, positions, block_table, max_pages, page_size, waves, heads, kv_heads, key_dim, value_dim, \
        pad, eps, write)
    if (dtype == kF32) ST_UQ(float);
    else if (dtype == kBF16) ST_UQ(bf16_t);
    else ST_CHECK(false, "unit_qk_write: unknown dtype %d", dtype);
#undef ST_UQ
    ST_LAUNCH_CHECK("unit_qk_write");
    return 0;
}
