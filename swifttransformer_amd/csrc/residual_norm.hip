// A branch's result on its way into the residual stream through a root-mean-square norm, and what the next branch reads:
//
//   x' = x + y / sqrt(mean(y^2) + eps) * gain;     h = x' / sqrt(mean(x'^2) + eps2) * gain2
//
// in one pass over the row: x, y, x', the statistics and the gains are float, h has the storage type.
#include "api.h"
#include "common.h"

namespace st {

// A workgroup a row; NP pieces of V neighbouring columns a thread stay in registers between the sums.
template <typename T, int V, int NP>
__global__ __launch_bounds__(256) void rms_onto_kernel(
    float* __restrict__ out32, T* __restrict__ out_t, const float* __restrict__ y, const float* __restrict__ x,
    const float* __restrict__ gain, const float* __restrict__ gain2, int width, float eps, float eps2) {
    __shared__ float red[16];
    const int64_t row = (int64_t)blockIdx.x * width;
    float a[NP][V], b[NP][V];
    auto load = [&](const float* p, float (*v)[V]) {
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int c = (threadIdx.x + 256 * i) * V, cc = min(c, width - V);
            if (V == 4) {
                const float4 z = *reinterpret_cast<const float4*>(p + cc);
                v[i][0] = z.x; v[i][1 % V] = z.y; v[i][2 % V] = z.z; v[i][3 % V] = z.w;
            } else {
                v[i][0] = p[cc];
            }
            if (c >= width) {
#pragma unroll
                for (int e = 0; e < V; ++e) v[i][e] = 0.f;
            }
        }
    };
    auto mean_square = [&](float (*v)[V]) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NP; ++i)
#pragma unroll
            for (int e = 0; e < V; ++e) ss = fmaf(v[i][e], v[i][e], ss);
        return block_sum(ss, red) / (float)width;
    };
    float w[NP][V];
    load(y + row, a);
    load(x + row, b);
    load(gain, w);
    const float r = 1.f / sqrtf(mean_square(a) + eps);
#pragma unroll
    for (int i = 0; i < NP; ++i) {
        const int c = (threadIdx.x + 256 * i) * V;
#pragma unroll
        for (int e = 0; e < V; ++e) b[i][e] = fmaf(a[i][e] * r, w[i][e], b[i][e]);
        if (c < width) {
            if (V == 4) *reinterpret_cast<float4*>(out32 + row + c) = make_float4(b[i][0], b[i][1 % V], b[i][2 % V], b[i][3 % V]);
            else out32[row + c] = b[i][0];
        }
    }
    if (!gain2) return;
    load(gain2, w);
    const float r2 = 1.f / sqrtf(mean_square(b) + eps2);
#pragma unroll
    for (int i = 0; i < NP; ++i) {
        const int c = (threadIdx.x + 256 * i) * V;
        if (c >= width) continue;
        float h[V];
#pragma unroll
        for (int e = 0; e < V; ++e) h[e] = b[i][e] * r2 * w[i][e];
        if (V == 4) Elem<T>::store4(out_t + row + c, h);
        else Elem<T>::store(out_t + row + c, h[0]);
    }
}

// Rows too long for registers: three passes over memory.
template <typename T>
__global__ __launch_bounds__(256) void rms_onto_long_kernel(
    float* out32, T* __restrict__ out_t, const float* __restrict__ y, const float* x, const float* __restrict__ gain,
    const float* __restrict__ gain2, int width, float eps, float eps2) {
    __shared__ float red[16];
    const int64_t row = (int64_t)blockIdx.x * width;
    float ss = 0.f;
    for (int c = threadIdx.x; c < width; c += 256) ss = fmaf(y[row + c], y[row + c], ss);
    const float r = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
    ss = 0.f;
    for (int c = threadIdx.x; c < width; c += 256) {
        const float v = fmaf(y[row + c] * r, gain[c], x[row + c]);
        out32[row + c] = v;
        ss = fmaf(v, v, ss);
    }
    if (!gain2) return;
    const float r2 = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps2);
    for (int c = threadIdx.x; c < width; c += 256) Elem<T>::store(out_t + row + c, out32[row + c] * r2 * gain2[c]);
}

}  // namespace st

using namespace st;

// out32 [rows, width] = x + rms_norm(y) * gain; with gain2, out_t (the storage type) = rms_norm(out32) * gain2.
extern "C" int st_rms_onto(float* out32, void* out_t, const float* y, const float* x, const float* gain, const float* gain2,
                           int num_rows, int width, float eps, float eps2, int dtype, hipStream_t stream) {
    ST_CHECK(num_rows >= 0 && width > 0, "rms_onto: bad sizes");
    ST_CHECK(eps > 0.f && (!gain2 || eps2 > 0.f), "rms_onto: eps must be positive");
    ST_CHECK(dtype == kF32 || dtype == kBF16, "rms_onto: unknown dtype %d", dtype);
    if (num_rows == 0) return 0;
    ST_CHECK(out32 && y && x && gain && (!gain2 || out_t), "rms_onto: null operand");
    const bool vec = width % 4 == 0 && (((uintptr_t)out32 | (uintptr_t)out_t | (uintptr_t)y | (uintptr_t)x | (uintptr_t)gain |
                                         (uintptr_t)gain2) & 15) == 0;
#define ST_RO(T, V, NP) rms_onto_kernel<T, V, NP><<<num_rows, 256, 0, stream>>>(out32, (T*)out_t, y, x, gain, gain2, width, eps, eps2)
#define ST_RO_T(T)                                                                                                     \
    do {                                                                                                               \
        if (vec && width <= 1024) ST_RO(T, 4, 1);                                                                      \
        else if (vec && width <= 2048) ST_RO(T, 4, 2);                                                                 \
        else if (vec && width <= 4096) ST_RO(T, 4, 4);                                                                 \
        else if (vec && width <= 8192) ST_RO(T, 4, 8);                                                                 \
        else if (width <= 1024) ST_RO(T, 1, 4);                                                                        \
        else rms_onto_long_kernel<T><<<num_rows, 256, 0, stream>>>(out32, (T*)out_t, y, x, gain, gain2, width, eps, eps2); \
    } while (0)
    if (dtype == kF32) ST_RO_T(float); else ST_RO_T(bf16_t);
#undef ST_RO_T
#undef ST_RO
    ST_LAUNCH_CHECK("rms_onto");
    return 0;
}
