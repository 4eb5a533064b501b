// The cache of a latent attention: per token one normalised vector that every head's keys and
// values are linear functions of.  It lives in a page pool of one "head" whose entries are the
// latent vectors (padded with zeros to the width the attention kernels take), so the paged
// attention kernels read it as the keys and as the values of one shared head.
#include "api.h"
#include "common.h"

namespace st {

// One wave per token: c = x * rsqrt(mean(x^2) + eps) * gain in float, stored in the pool's type.
template <typename T>
__global__ __launch_bounds__(256) void latent_write_kernel(
    T* __restrict__ cache, int64_t page_stride, const float* __restrict__ x, int64_t x_stride,
    const float* __restrict__ gain, const int* __restrict__ token_item, const int* __restrict__ positions,
    const int* __restrict__ block_table, int max_pages, int page_size, int num_tokens, int rank, int entry,
    float eps, int tail, const float* __restrict__ freq, float tail_mult) {
    const int lane = threadIdx.x & 63;
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= num_tokens) return;
    const int item = token_item[t], pos = positions[t];
    if (item < 0 || pos < 0) return;                 // a padding row
    const int page = block_table[(int64_t)item * max_pages + pos / page_size];
    if (page < 0) return;
    const float* xp = x + (int64_t)t * x_stride;
    float ss = 0.f;
    for (int j = lane; j < rank; j += 64) { const float v = xp[j]; ss = fmaf(v, v, ss); }
    ss = wave_sum(ss);
    const float r = 1.f / sqrtf(ss / (float)rank + eps);
    T* dst = cache + (int64_t)page * page_stride + (int64_t)(pos % page_size) * entry;
    for (int j = lane; j < entry; j += 64) {
        float v = 0.f;
        if (j < rank) {
            v = xp[j] * r * gain[j];
        } else if (j < rank + tail) {
            v = xp[j];
            if (freq) {                               // pairs (2i, 2i + 1) of the tail turn with the position
                const int i = (j - rank) >> 1;
                const float a = (float)pos * freq[i];
                const float c = cosf(a) * tail_mult, s = sinf(a) * tail_mult;
                const int ju = rank + 2 * i;
                const float u = xp[ju], w = xp[ju + 1];
                v = ((j - rank) & 1) ? w * c + u * s : u * c - w * s;
            }
        }
        Elem<T>::store(dst + j, v);
    }
}

// What a latent attention makes of its input products' float rows, in one launch (blockIdx.y): the query latent,
// normalised with its gain, for the product that makes queries of it (0; columns past its rank are zeros), and the cached
// entry (1): the latent, normalised with its gain, at [0, rank), zeros up to `tail_off`, the turned key part there, zeros
// to the end.  A wave a token and job, NP numbers a lane of the vector to normalise in registers.
template <typename T, int NP>
__global__ __launch_bounds__(256) void latent_inputs_kernel(
    T* __restrict__ cq, int cq_width, const float* __restrict__ gain_q, int q_rank, T* __restrict__ cache, int64_t page_stride,
    const float* __restrict__ gain, int rank, int tail_off, int tail, const float* __restrict__ freq, int half, float tail_mult,
    int entry, const float* __restrict__ x, int64_t x_stride, const int* __restrict__ token_item,
    const int* __restrict__ positions, const int* __restrict__ block_table, int max_pages, int page_size, int num_tokens,
    float eps) {
    const int lane = threadIdx.x & 63, t = blockIdx.x * 4 + (threadIdx.x >> 6), job = blockIdx.y;
    if (t >= num_tokens) return;
    const float* xp = x + (int64_t)t * x_stride + (job ? q_rank : 0);
    const int n = job ? rank : q_rank;
    const float* gn = job ? gain : gain_q;
    float v[NP], w[NP], ss = 0.f;
#pragma unroll
    for (int i = 0; i < NP; ++i) {
        const int j = min(lane + 64 * i, n - 1);
        v[i] = xp[j];
        w[i] = gn[j];
    }
    T* dst;
    int pos = 0;
    if (job) {
        const int item = token_item[t];
        pos = positions[t];
        if (item < 0 || pos < 0) return;                 // a padding row
        const int page = block_table[(int64_t)item * max_pages + pos / page_size];
        if (page < 0) return;
        dst = cache + (int64_t)page * page_stride + (int64_t)(pos % page_size) * entry;
    } else {
        dst = cq + (int64_t)t * cq_width;
    }
#pragma unroll
    for (int i = 0; i < NP; ++i)
        if (lane + 64 * i < n) ss = fmaf(v[i], v[i], ss);
    for (int j = lane + 64 * NP; j < n; j += 64) ss = fmaf(xp[j], xp[j], ss);
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)n + eps);
#pragma unroll
    for (int i = 0; i < NP; ++i)
        if (lane + 64 * i < n) Elem<T>::store(dst + lane + 64 * i, v[i] * r * w[i]);
    for (int j = lane + 64 * NP; j < n; j += 64) Elem<T>::store(dst + j, xp[j] * r * gn[j]);
    const int end = job ? entry : cq_width;
    for (int j = n + lane; j < end; j += 64) {
        const int k = j - tail_off;
        float z = 0.f;
        if (job && k >= 0 && k < tail) {
            const float* tp = xp + rank;
            z = tp[k];
            const int i = k >> 1;
            if (i < half) {                              // pairs (2i, 2i + 1) turn with the position
                const float a = (float)pos * freq[i], c = cosf(a) * tail_mult, s = sinf(a) * tail_mult;
                const float u = tp[2 * i], x2 = tp[2 * i + 1];
                z = (k & 1) ? x2 * c + u * s : u * c - x2 * s;
            }
        }
        Elem<T>::store(dst + j, z);
    }
}

}  // namespace st

using namespace st;

// x: float rows q latent [q_rank] | latent [rank] | key part [tail] (the last two absent where cache is null).  cq
// [tokens, cq_width]; cache [pages, page_size, entry].
extern "C" int st_latent_inputs(void* cq, int cq_width, const float* gain_q, int q_rank, void* cache, int64_t page_stride,
                                const float* gain, int rank, int tail_off, int tail, const float* freq, int half,
                                float tail_mult, int entry, const float* x, int64_t x_stride, const int* token_item,
                                const int* positions, const int* block_table, int max_pages, int page_size, int num_tokens,
                                float eps, int dtype, hipStream_t stream) {
    ST_CHECK(num_tokens >= 0 && q_rank > 0 && cq_width >= q_rank && eps > 0.f, "latent_inputs: bad sizes");
    ST_CHECK(cq && gain_q && x && x_stride >= q_rank, "latent_inputs: null operand or short rows");
    if (cache) {
        ST_CHECK(rank > 0 && tail >= 0 && tail_off >= rank && entry >= tail_off + tail && 2 * half <= tail && page_size > 0 &&
                 max_pages > 0 && x_stride >= (int64_t)q_rank + rank + tail && (half == 0 || freq),
                 "latent_inputs: a latent of %d and a part of %d from %d on in an entry of %d", rank, tail, tail_off, entry);
        ST_CHECK(gain && token_item && positions && block_table, "latent_inputs: null operand");
    }
    if (num_tokens == 0) return 0;
    const dim3 grid((num_tokens + 3) / 4, cache ? 2 : 1);
#define ST_LI(T, NP)                                                                                                   \
    latent_inputs_kernel<T, NP><<<grid, 256, 0, stream>>>((T*)cq, cq_width, gain_q, q_rank, (T*)cache, page_stride, gain, rank, \
        tail_off, tail, freq, half, tail_mult, entry, x, x_stride, token_item, positions, block_table, max_pages, page_size,    \
        num_tokens, eps)
    const int most = cache && rank > q_rank ? rank : q_rank;
#define ST_LI_T(T) do { if (most <= 128) ST_LI(T, 2); else if (most <= 256) ST_LI(T, 4); else if (most <= 512) ST_LI(T, 8); \
                        else if (most <= 1024) ST_LI(T, 16); else ST_LI(T, 24); } while (0)
    if (dtype == kF32) ST_LI_T(float);
    else if (dtype == kBF16) ST_LI_T(bf16_t);
    else ST_CHECK(false, "latent_inputs: unknown dtype %d", dtype);
#undef ST_LI_T
#undef ST_LI
    ST_LAUNCH_CHECK("latent_inputs");
    return 0;
}

extern "C" int st_latent_write(void* cache, int64_t page_stride, const float* x, int64_t x_stride, const float* gain,
                               const int* token_item, const int* positions, const int* block_table, int max_pages,
                               int page_size, int num_tokens, int rank, int entry, float eps, int tail,
                               const float* freq, float tail_mult, int dtype, hipStream_t stream) {
    ST_CHECK(num_tokens >= 0 && rank > 0 && tail >= 0 && entry >= rank + tail && page_size > 0 && max_pages > 0,
             "latent_write: bad sizes");
    ST_CHECK(!freq || tail % 2 == 0, "latent_write: a turned tail has an even size");
    ST_CHECK(cache && x && gain && token_item && positions && block_table, "latent_write: null operand");
    ST_CHECK(eps > 0.f, "latent_write: eps must be positive");
    if (num_tokens == 0) return 0;
    const unsigned grid = (unsigned)((num_tokens + 3) / 4);
    if (dtype == kF32)
        latent_write_kernel<float><<<grid, 256, 0, stream>>>((float*)cache, page_stride, x, x_stride, gain, token_item,
            positions, block_table, max_pages, page_size, num_tokens, rank, entry, eps, tail, freq, tail_mult);
    else if (dtype == kBF16)
        latent_write_kernel<bf16_t><<<grid, 256, 0, stream>>>((bf16_t*)cache, page_stride, x, x_stride, gain, token_item,
            positions, block_table, max_pages, page_size, num_tokens, rank, entry, eps, tail, freq, tail_mult);
    else ST_CHECK(false, "latent_write: unknown dtype %d", dtype);
    ST_LAUNCH_CHECK("latent_write");
    return 0;
}
