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
// attention kernels take one width for keys and values, a multiple of 16).
#include "api.h"
#include "common.h"

namespace st {

constexpr int kUnitMax = 256;                // coordinates a head

// Grid (rows, parts of a row's heads): the turn's cosines and sines once a workgroup in LDS, then LPH lanes a head, V
// neighbouring coordinates a lane and turn (4: 16-byte loads; sizes and addresses allow them), E turns.  A row's heads
// are its query heads, then key heads, then value heads.
template <typename T, int V, int LPH, int E>
__global__ __launch_bounds__(256) void unit_qk_write_kernel(
    T* __restrict__ out_q, T* __restrict__ k_cache, T* __restrict__ v_cache, int64_t page_stride,
    const float* __restrict__ qkv, int64_t stride, const float* __restrict__ freq, int half,
    const float* __restrict__ factor, const int* __restrict__ token_item, const int* __restrict__ positions,
    const int* __restrict__ block_table, int max_pages, int page_size, int heads, int kv_heads, int key_dim,
    int value_dim, int pad, float eps, int write) {
    extern __shared__ __attribute__((aligned(16))) float uq_turn[];     // cosines [half] | sines [half]
    const int64_t t = blockIdx.x;
    const int lane = threadIdx.x % LPH;
    const int item = token_item[t], pos = positions[t];
    const bool padding = item < 0 || pos < 0;
    const int page = (!padding && write) ? block_table[(int64_t)item * max_pages + pos / page_size] : -1;
    const float* row = qkv + t * stride;
    const float* v_row = row + (int64_t)(heads + kv_heads) * key_dim;
    const int units = heads + 2 * kv_heads, step = gridDim.y * (256 / LPH);
    bool turned = half == 0;
    for (int u = blockIdx.y * (256 / LPH) + threadIdx.x / LPH; u < units || !turned; u += step) {
        const int uc = min(u, units - 1);
        const bool is_q = uc < heads, is_v = uc >= heads + kv_heads;
        const float* src = is_v ? v_row + (int64_t)(uc - heads - kv_heads) * value_dim : row + (int64_t)uc * key_dim;
        const int dim = is_v ? value_dim : key_dim;
        float y[E][V], z[E][V];
#pragma unroll
        for (int e = 0; e < E; ++e) {
            const int d = (lane + LPH * e) * V, dc = min(d, dim - V);
            // the coordinates these turn with (a stand-in where they do not turn)
            const int other = d < half ? d + half : d < 2 * half ? d - half : dc;
            if (V == 4) {
                const float4 a = *reinterpret_cast<const float4*>(src + dc), b = *reinterpret_cast<const float4*>(src + min(other, dim - V));
                y[e][0] = a.x; y[e][1 % V] = a.y; y[e][2 % V] = a.z; y[e][3 % V] = a.w;
                z[e][0] = b.x; z[e][1 % V] = b.y; z[e][2 % V] = b.z; z[e][3 % V] = b.w;
            } else {
                y[e][0] = src[dc];
                z[e][0] = src[min(other, dim - V)];
            }
#pragma unroll
            for (int v = 0; v < V; ++v) y[e][v] = d < dim && !padding ? y[e][v] : 0.f;
        }
        if (!turned) {                            // every thread's first time round
            for (int i = threadIdx.x; i < half; i += 256) {
                const float a = (float)max(pos, 0) * freq[i];
                uq_turn[i] = cosf(a);
                uq_turn[half + i] = sinf(a);
            }
            __syncthreads();
            turned = true;
        }
        if (u >= units) break;
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < E; ++e) {
            const int d = (lane + LPH * e) * V;
            if (!is_v && d < 2 * half && !padding) {
                const int i = d < half ? d : d - half;
                const float sign = d < half ? -1.f : 1.f;
#pragma unroll
                for (int v = 0; v < V; ++v) y[e][v] = y[e][v] * uq_turn[i + v] + sign * z[e][v] * uq_turn[half + i + v];
            }
#pragma unroll
            for (int v = 0; v < V; ++v) ss = fmaf(y[e][v], y[e][v], ss);
        }
        float r = 1.f;
        if (!is_v) {
#pragma unroll
            for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
            r = 1.f / sqrtf(ss / (float)key_dim + eps);
            if (is_q && factor) r *= factor[uc];
        }
        if (!is_q && page < 0) continue;
        T* dst;
        if (is_q) {
            dst = out_q + (t * heads + uc) * pad;
        } else {
            const int h = is_v ? uc - heads - kv_heads : uc - heads;
            dst = (is_v ? v_cache : k_cache) + (int64_t)page * page_stride + ((int64_t)h * page_size + pos % page_size) * pad;
        }
#pragma unroll
        for (int e = 0; e < E; ++e) {
            const int d = (lane + LPH * e) * V;
            if (d >= pad) continue;
#pragma unroll
            for (int v = 0; v < V; ++v) y[e][v] *= r;
            if (V == 4) Elem<T>::store4(dst + d, y[e]); else Elem<T>::store(dst + d, y[e][0]);
        }
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
    ST_CHECK(pad >= key_dim && pad >= value_dim && pad <= kUnitMax, "unit_qk_write: heads of %d and %d in entries of %d "
             "(up to %d)", key_dim, value_dim, pad, kUnitMax);
    ST_CHECK(half >= 0 && 2 * half <= key_dim && (freq || half == 0), "unit_qk_write: %d turned coordinates in heads of %d",
             2 * half, key_dim);
    ST_CHECK(stride >= (int64_t)(heads + kv_heads) * key_dim + (int64_t)kv_heads * value_dim, "unit_qk_write: rows shorter than q, k and v");
    ST_CHECK(eps > 0.f, "unit_qk_write: eps must be positive");
    if (num_tokens == 0) return 0;
    ST_CHECK(out_q && qkv && token_item && positions && (!write || (k_cache && v_cache && block_table)),
             "unit_qk_write: null operand");
    const bool vec = key_dim % 4 == 0 && value_dim % 4 == 0 && half % 4 == 0 && stride % 4 == 0 && page_stride % 4 == 0 &&
                     (((uintptr_t)qkv | (uintptr_t)out_q | (uintptr_t)k_cache | (uintptr_t)v_cache) & 15) == 0;
    const size_t lds = sizeof(float) * 2 * half;
    // a workgroup walks over all of a row's heads where there are rows enough, else a row's heads are dealt to several
#define ST_UQ(T, V, LPH, E) do {                                                                                      \
        const int passes = (heads + 2 * kv_heads + 256 / LPH - 1) / (256 / LPH);                                       \
        const int parts = num_tokens >= 2 * device_compute_units() ? 1 : passes;                                       \
        ST_CHECK(parts <= 65535, "unit_qk_write: too many heads");                                                     \
        unit_qk_write_kernel<T, V, LPH, E><<<dim3(num_tokens, parts), 256, lds, stream>>>((T*)out_q, (T*)k_cache, (T*)v_cache, \
            page_stride, qkv, stride, freq, half, factor, token_item, positions, block_table, max_pages, page_size, heads, \
            kv_heads, key_dim, value_dim, pad, eps, write); } while (0)
#define ST_UQ_T(T) do {                                                                                               \
        if (vec) { if (pad <= 64) ST_UQ(T, 4, 16, 1); else if (pad <= 128) ST_UQ(T, 4, 32, 1); else ST_UQ(T, 4, 64, 1); } \
        else { if (pad <= 64) ST_UQ(T, 1, 64, 1); else if (pad <= 128) ST_UQ(T, 1, 64, 2); else ST_UQ(T, 1, 64, 4); } } while (0)
    if (dtype == kF32) ST_UQ_T(float);
    else if (dtype == kBF16) ST_UQ_T(bf16_t);
    else ST_CHECK(false, "unit_qk_write: unknown dtype %d", dtype);
#undef ST_UQ_T
#undef ST_UQ
    ST_LAUNCH_CHECK("unit_qk_write");
    return 0;
}
