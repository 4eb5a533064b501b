// Routed experts: every token sends its vector, scaled by a routing weight, through `top` of
// `experts` small gated feed-forward layers.
//
// Everything stays on the device and has a fixed launch shape, so a step can be recorded:
//   route    per token the `top` best experts and their weights (five rules, see st_moe_route);
//   align    the (token, choice) pairs sorted by expert into tiles of 16, 64 or 128 places, a tile
//            holding pairs of one expert only (places left over are marked -1);
//   up       per tile and 64 inner features: both input products on the matrix cores, rows
//            gathered through the sorted list, then clamp, gate and product of the two halves (experts
//            without a gate: one product and the exact GELU);
//   down     per tile and 64 output features: the output product; with one expert a token the
//            result goes straight into the residual stream, otherwise to a row per pair that
//   combine  sums in the order of the token's choices.  Router outputs past the experts stand for identity
//            experts: a choice of one has no place in the tiles, and its result is the token's own vector.
// A wave computes 16 x 16 blocks of results with operands read straight from memory in the
// matrix instruction's own layout (16 bytes a lane and step): with 16 rows a tile the products
// are bound by the stream of expert weights, which every tile reads once.
#include "api.h"
#include "common.h"
#include "activation.h"
#include "fragment.h"

#include <type_traits>

namespace st {

template <int N> using Steps = std::integral_constant<int, N>;
constexpr int kRows = 16;            // rows of one matrix-instruction block
constexpr int kMaxTop = 16;

__global__ __launch_bounds__(256) void moe_route_kernel(
    int* __restrict__ ids, float* __restrict__ weights, const float* __restrict__ logits,
    int logit_stride, const int* __restrict__ token_item, const float* __restrict__ correction, float scale, int num_tokens,
    int experts, int top, int mode, int groups, int keep, int stage) {
    // The rows of the workgroup's tokens go to LDS first, read side by side (a thread that walked its own row in
    // memory would wait for every logit by itself, several times over); rows are experts + 1 floats apart.
    extern __shared__ float s_z[];
    const int t0 = blockIdx.x * blockDim.x, t = t0 + threadIdx.x;
    if (stage) {
        const int n = min((int)blockDim.x, num_tokens - t0);
        const float* src = logits + (int64_t)t0 * logit_stride;
        for (int i = threadIdx.x; i < n * experts; i += blockDim.x) {
            const int r = i / experts;
            // (mode 3 chooses by the sigmoid of a logit plus the expert's correction: formed here, side by side)
            const float z = src[(int64_t)r * logit_stride + (i - r * experts)];
            s_z[r * (experts + 1) + (i - r * experts)] = mode == 3 ? 1.f / (1.f + expf(-z)) + correction[i - r * experts] : z;
        }
        __syncthreads();
    }
    if (t >= num_tokens) return;
    if (token_item && token_item[t] < 0) {
        for (int j = 0; j < top; ++j) { ids[(int64_t)t * top + j] = -1; weights[(int64_t)t * top + j] = 0.f; }
        return;
    }
    const float* z = stage ? s_z + threadIdx.x * (experts + 1) : logits + (int64_t)t * logit_stride;
    // mode 2: only the experts of the `keep` groups (of `groups` equal groups of neighbours) whose largest
    // logit is largest can be chosen; bit g of `open` says that group g is one of them
    uint64_t open = ~0ull;
    const int per = experts / groups;
    if (mode == 2 && keep < groups) {
        open = 0;
        for (int j = 0; j < keep; ++j) {
            int best = -1;
            float bv = 0.f;
            for (int g = 0; g < groups; ++g) {
                if ((open >> g) & 1) continue;
                float gv = z[g * per];
                for (int e = 1; e < per; ++e) gv = fmaxf(gv, z[g * per + e]);
                if (best < 0 || gv > bv) { best = g; bv = gv; }
            }
            open |= 1ull << best;
        }
    }
    // modes 2 and 4: the weights are the chosen experts' shares of the softmax over all experts, as they are
    float m_all = 0.f, inv_sum = 1.f;
    if (mode == 2 || mode == 4) {
        m_all = z[0];
        for (int e = 1; e < experts; ++e) m_all = fmaxf(m_all, z[e]);
        float sum = 0.f;
        for (int e = 0; e < experts; ++e) sum += expf(z[e] - m_all);
        inv_sum = 1.f / sum;
    }
    // mode 4: the share plus the expert's correction chooses; staged, it takes the logit's place in this thread's own row
    if (mode == 4 && stage) {
        float* own = s_z + threadIdx.x * (experts + 1);
        for (int e = 0; e < experts; ++e) own[e] = expf(own[e] - m_all) * inv_sum + correction[e];
    }
    // modes 3 and 4: what an expert is chosen by, where it was not staged
    auto choice = [&](int e) {
        if (stage || mode < 3) return z[e];
        return (mode == 3 ? 1.f / (1.f + expf(-z[e])) : expf(z[e] - m_all) * inv_sum) + correction[e];
    };
    auto weight_of = [&](float v) { return mode == 0 ? 1.f / (1.f + expf(-v)) : mode == 2 ? expf(v - m_all) * inv_sum : v; };
    if (experts <= 64) {
        // which experts can still be chosen, a bit each: no list of the chosen ones to walk
        uint64_t free_ = experts == 64 ? ~0ull : (1ull << experts) - 1;
        if (mode == 2 && keep < groups) {
            const uint64_t one_group = per == 64 ? ~0ull : (1ull << per) - 1;
            free_ = 0;
            for (int g = 0; g < groups; ++g)
                if ((open >> g) & 1) free_ |= one_group << (g * per);
        }
        for (int j = 0; j < top; ++j) {
            int best = -1;
            float bv = 0.f;
            for (int e = 0; e < experts; ++e) {
                const float v = choice(e);
                if (((free_ >> e) & 1) && (best < 0 || v > bv)) { best = e; bv = v; }
            }
            free_ &= ~(1ull << best);
            ids[(int64_t)t * top + j] = best;
            weights[(int64_t)t * top + j] = weight_of(bv);
        }
    } else {
        int chosen[kMaxTop];
        for (int j = 0; j < top; ++j) {
            int best = -1;
            float bv = 0.f;
            for (int e = 0; e < experts; ++e) {
                bool taken = mode == 2 && !((open >> (e / per)) & 1);
                for (int u = 0; u < j; ++u) taken |= chosen[u] == e;
                const float v = choice(e);
                if (!taken && (best < 0 || v > bv)) { best = e; bv = v; }
            }
            chosen[j] = best;
            ids[(int64_t)t * top + j] = best;
            weights[(int64_t)t * top + j] = weight_of(bv);
        }
    }
    if (mode == 1) {
        // softmax over the chosen logits alone; the first chosen is the largest
        float* w = weights + (int64_t)t * top;
        const float m = w[0];
        float sum = 0.f;
        for (int j = 0; j < top; ++j) { w[j] = expf(w[j] - m); sum += w[j]; }
        for (int j = 0; j < top; ++j) w[j] /= sum;
    } else if (mode == 3) {
        // the chosen experts' sigmoids, without the correction, over their sum
        float* w = weights + (int64_t)t * top;
        const float* raw = logits + (int64_t)t * logit_stride;
        float sum = 0.f;
        for (int j = 0; j < top; ++j) {
            w[j] = 1.f / (1.f + expf(-raw[ids[(int64_t)t * top + j]]));
            sum += w[j];
        }
        for (int j = 0; j < top; ++j) w[j] = w[j] / (sum + 1e-20f) * scale;
    } else if (mode == 4) {
        // the shares themselves, without the correction
        const float* raw = logits + (int64_t)t * logit_stride;
        for (int j = 0; j < top; ++j) weights[(int64_t)t * top + j] = expf(raw[ids[(int64_t)t * top + j]] - m_all) * inv_sum;
    }
}

// One workgroup: counts, padded offsets, then places.  Which place of its expert's tiles a pair
// gets depends on the order of the atomics; a pair's result does not depend on its place.
__global__ __launch_bounds__(1024) void moe_align_kernel(
    int* __restrict__ sorted, int* __restrict__ place_of_pair, int* __restrict__ tile_expert,
    const int* __restrict__ ids, int num_pairs, int experts, int capacity, int kTile) {
    extern __shared__ int lds[];
    int* count = lds;                  // [experts]
    int* offset = lds + experts;       // [experts + 1]
    const int tid = threadIdx.x;
    for (int e = tid; e < experts; e += 1024) count[e] = 0;
    for (int i = tid; i < capacity; i += 1024) sorted[i] = -1;
    for (int i = tid; i < capacity / kTile; i += 1024) tile_expert[i] = -1;
    __syncthreads();
    for (int p = tid; p < num_pairs; p += 1024) {
        const int e = ids[p];                          // (an identity expert has no tiles)
        if (e >= 0 && e < experts) atomicAdd(&count[e], 1);
    }
    __syncthreads();
    if (tid == 0) {
        int run = 0;
        for (int e = 0; e < experts; ++e) {
            offset[e] = run;
            run += (count[e] + kTile - 1) / kTile * kTile;
        }
        offset[experts] = run;
    }
    __syncthreads();
    for (int e = tid; e < experts; e += 1024) {
        for (int i = offset[e] / kTile; i < offset[e + 1] / kTile; ++i) tile_expert[i] = e;
        count[e] = offset[e];          // from here on: the next free place of the expert
    }
    __syncthreads();
    for (int p = tid; p < num_pairs; p += 1024) {
        const int e = ids[p];
        int place = -1;
        if (e >= 0 && e < experts) {
            place = atomicAdd(&count[e], 1);
            sorted[place] = p;
        }
        place_of_pair[p] = place;
    }
}

// ---- few rows an expert: tiles of 16 places, where only the weights' stream counts.  A workgroup takes 16 features; its
// four waves share the depth, so that a wave's part is one or a few batches of loads that are all on their way at once and
// that the waves' rows, which lie a whole row of weights apart, start at different offsets (equal offsets meet in the
// same memory channels); the waves' sums meet in LDS.  The addresses of rows and features that do not exist stand for
// row and feature 0: their results are not stored.
template <typename T, int MATS>
__device__ inline void moe_depth_share(floatx4* acc, const T* xr, const T* const* wr, int K, int vec) {
    constexpr int D = Frag<T>::kDepth, L = Frag<T>::kLane;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4;
    const int steps = (K + D - 1) / D, share = (steps + 3) / 4;
    int k0 = wave * share * D;
    const int end = min(K, k0 + share * D);
    auto batches = [&](auto count) {
        constexpr int U = decltype(count)::value;
        for (; k0 + U * D <= end; k0 += U * D) {
            Frag<T> a[U], b[MATS][U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int k = k0 + u * D + L * g;
#pragma unroll
                for (int m = 0; m < MATS; ++m) b[m][u].load_whole(wr[m] + k);
                a[u].load_whole(xr + k);
            }
            __builtin_amdgcn_sched_barrier(0);    // (left to itself the compiler keeps a few of the loads on their way)
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int m = 0; m < MATS; ++m) acc[m] = Frag<T>::mma(a[u], b[m][u], acc[m]);
        }
    };
    if (vec) {
        batches(Steps<MATS == 1 ? 16 : 8>());
        batches(Steps<4>());
    }
    for (; k0 < end; k0 += D) {
        Frag<T> a, b;
        a.load(xr, k0 + L * g, K, true, vec);
#pragma unroll
        for (int m = 0; m < MATS; ++m) {
            b.load(wr[m], k0 + L * g, K, true, vec);
            acc[m] = Frag<T>::mma(a, b, acc[m]);
        }
    }
}

// the waves' blocks of 16 x 16 summed: thread t of the workgroup gets row t / 16, feature t % 16
template <int MATS>
__device__ inline void moe_sum_shares(float* sum, const floatx4* acc, float* lds) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
    for (int m = 0; m < MATS; ++m) *reinterpret_cast<floatx4*>(lds + ((wave * MATS + m) * 64 + lane) * 4) = acc[m];
    __syncthreads();
    const int row = threadIdx.x >> 4, from = ((row >> 2) * 16 + (threadIdx.x & 15)) * 4 + (row & 3);
#pragma unroll
    for (int m = 0; m < MATS; ++m) {
        sum[m] = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) sum[m] += lds[(w * MATS + m) * 256 + from];
    }
}

// grid (tiles, ceil(inner / 16))
template <typename T, bool GATED>
__global__ __launch_bounds__(256) void moe_up_few_kernel(
    T* __restrict__ y, const T* __restrict__ x, const T* __restrict__ w_gate, const T* __restrict__ w_up,
    const int* __restrict__ sorted, const int* __restrict__ tile_expert, const float* __restrict__ weights,
    int top, int width, int inner, float limit, int style, int vec) {
    constexpr int MATS = GATED ? 2 : 1;
    __shared__ __attribute__((aligned(16))) float lds[4 * MATS * 256];
    const int tile = blockIdx.x, e = tile_expert[tile];
    if (e < 0) return;
    const int r16 = threadIdx.x & 15, f0 = blockIdx.y * 16, base = tile * kRows;
    const int64_t feature = (int64_t)e * inner + min(f0 + r16, inner - 1);
    const int pair = sorted[base + r16];
    const T* wr[MATS];
    wr[0] = w_up + feature * width;
    if (GATED) wr[MATS - 1] = w_gate + feature * width;
    floatx4 acc[MATS];
#pragma unroll
    for (int m = 0; m < MATS; ++m) acc[m] = floatx4{0.f, 0.f, 0.f, 0.f};
    moe_depth_share<T, MATS>(acc, x + (int64_t)(pair >= 0 ? pair / top : 0) * width, wr, width, vec);
    float sum[MATS];
    moe_sum_shares<MATS>(sum, acc, lds);
    const int place = base + (threadIdx.x >> 4), f = f0 + r16;
    if (f >= inner) return;
    const int p = sorted[place];
    float out = 0.f;
    if (p >= 0 && !GATED) {
        out = apply_activation(kActGeluErf, sum[0]);
    } else if (p >= 0 && style == 1) {
        const float gv = sum[MATS - 1];
        out = gv / (1.f + expf(-gv)) * sum[0];
    } else if (p >= 0) {
        const float s = style == 0 ? weights[p] : 1.f;
        const float gv = fminf(s * sum[MATS - 1], limit);
        const float uv = fminf(fmaxf(s * sum[0], -limit), limit);
        out = gv / (1.f + expf(-1.702f * gv)) * (uv + 1.f);
    }
    Elem<T>::store(y + (int64_t)place * inner + f, out);
}

// grid (tiles, ceil(width / 16))
template <typename T>
__global__ __launch_bounds__(256) void moe_down_few_kernel(
    float* out, const float* residual, float* __restrict__ pair_out, const T* __restrict__ y, const T* __restrict__ w_down,
    const int* __restrict__ sorted, const int* __restrict__ tile_expert, int top, int width, int inner, float out_scale,
    int vec) {
    __shared__ __attribute__((aligned(16))) float lds[4 * 256];
    const int tile = blockIdx.x, e = tile_expert[tile];
    if (e < 0) return;
    const int r16 = threadIdx.x & 15, n0 = blockIdx.y * 16, base = tile * kRows;
    const T* wr[1] = {w_down + ((int64_t)e * width + min(n0 + r16, width - 1)) * inner};
    floatx4 acc[1] = {floatx4{0.f, 0.f, 0.f, 0.f}};
    moe_depth_share<T, 1>(acc, y + (int64_t)(base + r16) * inner, wr, inner, vec);
    float sum[1];
    moe_sum_shares<1>(sum, acc, lds);
    const int place = base + (threadIdx.x >> 4), n = n0 + r16;
    const int p = sorted[place];
    if (n >= width || p < 0) return;
    if (pair_out) {
        pair_out[(int64_t)place * width + n] = sum[0];
    } else {                                           // one expert a token: p is the token
        const int64_t at = (int64_t)p * width + n;
        out[at] = fmaf(out_scale, sum[0], residual[at]);
    }
}

// grid (tiles, ceil(inner / 64)); wave w of the workgroup takes inner features f0 + 16 w .. +15 of
// the tile's RT blocks of 16 rows: a step's weight operands are loaded once and meet RT blocks of
// rows (4 or 8, for prompts, where every tile reads its expert's weights again from the L2).
// Result layout of a block: lane (r16, g) holds rows 4g .. 4g+3 of feature r16.
// GATED false: one weight matrix (w_up) and the exact GELU of its product (style 2).
template <typename T, int RT, bool GATED>
__global__ __launch_bounds__(256) void moe_up_kernel(
    T* __restrict__ y, const T* __restrict__ x, const T* __restrict__ w_gate, const T* __restrict__ w_up,
    const int* __restrict__ sorted, const int* __restrict__ tile_expert, const float* __restrict__ weights,
    int top, int width, int inner, float limit, int style, int vec) {
    const int tile = blockIdx.x;
    const int e = tile_expert[tile];
    if (e < 0) return;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
    const int f = blockIdx.y * 64 + wave * 16 + r16;           // this lane's feature as an operand row
    const bool f_ok = f < inner;
    const int base = tile * (kRows * RT);
    const T* xr[RT];
    bool p_ok[RT];
#pragma unroll
    for (int b = 0; b < RT; ++b) {
        const int pair = sorted[base + b * kRows + r16];       // this lane's token row as an operand row
        p_ok[b] = pair >= 0;
        xr[b] = x + (int64_t)(p_ok[b] ? pair / top : 0) * width;
    }
    const T* gr = (GATED ? w_gate : w_up) + ((int64_t)e * inner + (f_ok ? f : 0)) * width;
    const T* ur = w_up + ((int64_t)e * inner + (f_ok ? f : 0)) * width;
    floatx4 cg[RT], cu[RT];
#pragma unroll
    for (int b = 0; b < RT; ++b) { cg[b] = floatx4{0.f, 0.f, 0.f, 0.f}; cu[b] = floatx4{0.f, 0.f, 0.f, 0.f}; }
    constexpr int D = Frag<T>::kDepth, L = Frag<T>::kLane;

    // (the addresses of rows and features that do not exist stand for row and feature 0: their results are not stored)
    int k0 = 0;
    auto batches = [&](auto steps) {
        constexpr int U = decltype(steps)::value;
        for (; k0 + U * D <= width; k0 += U * D) {
            Frag<T> a[U][RT], bg[U], bu[U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int k = k0 + u * D + L * g;
                if (GATED) bg[u].load_whole(gr + k);
                bu[u].load_whole(ur + k);
#pragma unroll
                for (int b = 0; b < RT; ++b) a[u][b].load_whole(xr[b] + k);
            }
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int b = 0; b < RT; ++b) {
                    if (GATED) cg[b] = Frag<T>::mma(a[u][b], bg[u], cg[b]);
                    cu[b] = Frag<T>::mma(a[u][b], bu[u], cu[b]);
                }
        }
    };
    if (vec && RT == 4) batches(Steps<2>());
    for (; k0 < width; k0 += D) {
        Frag<T> a[RT], bg, bu;
        const int k = k0 + L * g;
        if (GATED) bg.load(gr, k, width, f_ok, vec);
        bu.load(ur, k, width, f_ok, vec);
#pragma unroll
        for (int b = 0; b < RT; ++b) a[b].load(xr[b], k, width, p_ok[b], vec);
#pragma unroll
        for (int b = 0; b < RT; ++b) {
            if (GATED) cg[b] = Frag<T>::mma(a[b], bg, cg[b]);
            cu[b] = Frag<T>::mma(a[b], bu, cu[b]);
        }
    }
    if (!f_ok) return;
#pragma unroll
    for (int b = 0; b < RT; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int place = base + b * kRows + 4 * g + r;
            const int p = sorted[place];
            float out = 0.f;
            if (p >= 0 && !GATED) {
                out = apply_activation(kActGeluErf, cu[b][r]);
            } else if (p >= 0 && style == 1) {
                const float gv = cg[b][r];
                out = gv / (1.f + expf(-gv)) * cu[b][r];
            } else if (p >= 0) {
                const float s = style == 0 ? weights[p] : 1.f;
                const float gv = fminf(s * cg[b][r], limit);
                const float uv = fminf(fmaxf(s * cu[b][r], -limit), limit);
                out = gv / (1.f + expf(-1.702f * gv)) * (uv + 1.f);
            }
            Elem<T>::store(y + (int64_t)place * inner + f, out);
        }
}

// grid (tiles, ceil(width / 64)).
template <typename T, int RT>
__global__ __launch_bounds__(256) void moe_down_kernel(
    float* __restrict__ out, const float* __restrict__ residual, float* __restrict__ pair_out,
    const T* __restrict__ y, const T* __restrict__ w_down, const int* __restrict__ sorted,
    const int* __restrict__ tile_expert, int top, int width, int inner, float out_scale, int vec) {
    const int tile = blockIdx.x;
    const int e = tile_expert[tile];
    if (e < 0) return;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
    const int n = blockIdx.y * 64 + wave * 16 + r16;
    const bool n_ok = n < width;
    const int base = tile * (kRows * RT);
    const T* yr = y + (int64_t)(base + r16) * inner;
    const T* wr = w_down + ((int64_t)e * width + (n_ok ? n : 0)) * inner;
    floatx4 c[RT];
#pragma unroll
    for (int b = 0; b < RT; ++b) c[b] = floatx4{0.f, 0.f, 0.f, 0.f};
    constexpr int D = Frag<T>::kDepth, L = Frag<T>::kLane;

    int k0 = 0;
    auto batches = [&](auto steps) {              // (as in moe_up_kernel)
        constexpr int U = decltype(steps)::value;
        for (; k0 + U * D <= inner; k0 += U * D) {
            Frag<T> a[U][RT], bw[U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int k = k0 + u * D + L * g;
                bw[u].load_whole(wr + k);
#pragma unroll
                for (int b = 0; b < RT; ++b) a[u][b].load_whole(yr + (int64_t)b * kRows * inner + k);
            }
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int b = 0; b < RT; ++b) c[b] = Frag<T>::mma(a[u][b], bw[u], c[b]);
        }
    };
    if (vec && RT == 4) batches(Steps<2>());
    for (; k0 < inner; k0 += D) {
        Frag<T> a[RT], bw;
        const int k = k0 + L * g;
        bw.load(wr, k, inner, n_ok, vec);
#pragma unroll
        for (int b = 0; b < RT; ++b) a[b].load(yr + (int64_t)b * kRows * inner, k, inner, true, vec);
#pragma unroll
        for (int b = 0; b < RT; ++b) c[b] = Frag<T>::mma(a[b], bw, c[b]);
    }
    if (!n_ok) return;
#pragma unroll
    for (int b = 0; b < RT; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int place = base + b * kRows + 4 * g + r;
            const int p = sorted[place];
            if (p < 0) continue;
            if (pair_out) {
                pair_out[(int64_t)place * width + n] = c[b][r];
            } else {                                           // one expert a token: p is the token
                const int64_t at = (int64_t)p * width + n;
                out[at] = fmaf(out_scale, c[b][r], residual[at]);
            }
        }
}

// ---- prompts in bfloat16: tiles of 128 places, operands staged through LDS ----------------------
// With a hundred rows and more an expert the products are bound by arithmetic, not by the weights'
// stream, and operands read straight from memory leave the matrix cores waiting.  Here a workgroup
// computes 128 places x 128 weight rows in steps of 64 in depth: all threads bring the two operand
// tiles into registers with 16-byte loads (the next step's while this one is multiplied), store
// them into LDS with the rows' chunks rotated so that the matrix instruction's reads spread over
// the banks, and every wave multiplies a 64 x 64 part (v_mfma_f32_32x32x16_bf16).
// UP: the 128 weight rows are 64 inner features of the gate matrix and the same 64 of the other
// one, dealt so that a lane holds both halves of a result; rows of x are gathered through the
// sorted list.  Otherwise: 128 output features of the expert's output matrix over the rows of y.
typedef float floatx16 __attribute__((ext_vector_type(16)));
__device__ inline int rot(int row, int chunk) { return row * 8 + (chunk ^ ((row >> 1) & 7)); }

// GELU: as UP, but the 128 weight rows are 128 inner features of the one input matrix of experts without a gate.
enum TiledKind : int { kTiledDown = 0, kTiledUp = 1, kTiledGelu = 2 };
template <int KIND>
__global__ __launch_bounds__(256) void moe_tiled_kernel(
    bf16_t* __restrict__ y_out, float* __restrict__ out, const float* __restrict__ residual,
    float* __restrict__ pair_out, const bf16_t* __restrict__ a_rows, const bf16_t* __restrict__ w0,
    const bf16_t* __restrict__ w1, const int* __restrict__ sorted, const int* __restrict__ tile_expert,
    const float* __restrict__ weights, int top, int N, int K, float limit, float out_scale, int style) {
    constexpr bool UP = KIND == kTiledUp, GATHER = KIND != kTiledDown;
    __shared__ uint4 sw[128 * 8];      // weight rows: [row][chunk of 8 in depth]
    __shared__ uint4 sx[128 * 8];      // places
    const int tile = blockIdx.x;
    const int e = tile_expert[tile];
    if (e < 0) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int wn = wave & 1, wm = wave >> 1, l32 = lane & 31, lh = lane >> 5;
    const int base = tile * 128;
    const int n0 = blockIdx.y * (UP ? 64 : 128);
    // the four rows of each tile that this thread brings in, fixed over the steps
    const bf16_t* wrow[4];
    const bf16_t* xrow[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int row = (tid + i * 256) >> 3;
        int n;
        const bf16_t* m;
        if (UP) { n = n0 + (row >> 6) * 32 + (row & 31); m = ((row >> 5) & 1) ? w1 : w0; }
        else { n = n0 + row; m = w0; }
        wrow[i] = n < N ? m + ((int64_t)e * N + n) * K : nullptr;
        const int p = sorted[base + row];
        xrow[i] = GATHER ? (p >= 0 ? a_rows + (int64_t)(p / top) * K : nullptr) : a_rows + (int64_t)(base + row) * K;
    }
    floatx16 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int q = 0; q < 16; ++q) acc[i][j][q] = 0.f;
    uint4 rw[4], rx[4];
    auto load_global = [&](int k0) {
        const int k = k0 + (tid & 7) * 8;
        const bool in = k < K;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            // (addresses clamped and values cleared rather than loads behind a branch)
            const bf16_t* pw = wrow[i] ? wrow[i] : w0;
            const bf16_t* px = xrow[i] ? xrow[i] : a_rows;
            const uint4 vw = *reinterpret_cast<const uint4*>(pw + (in ? k : 0));
            const uint4 vx = *reinterpret_cast<const uint4*>(px + (in ? k : 0));
            rw[i] = (in && wrow[i]) ? vw : make_uint4(0, 0, 0, 0);
            rx[i] = (in && xrow[i]) ? vx : make_uint4(0, 0, 0, 0);
        }
    };
    load_global(0);
    for (int k0 = 0; k0 < K; k0 += 64) {
        __syncthreads();               // the step before has been read
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = tid + i * 256;
            sw[rot(c >> 3, c & 7)] = rw[i];
            sx[rot(c >> 3, c & 7)] = rx[i];
        }
        __syncthreads();
        if (k0 + 64 < K) load_global(k0 + 64);
#pragma unroll
        for (int kk = 0; kk < 4; ++kk) {
            const int chunk = kk * 2 + lh;
            bf16x8 a[2], b[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) a[i] = __builtin_bit_cast(bf16x8, sw[rot(wn * 64 + i * 32 + l32, chunk)]);
#pragma unroll
            for (int j = 0; j < 2; ++j) b[j] = __builtin_bit_cast(bf16x8, sx[rot(wm * 64 + j * 32 + l32, chunk)]);
#pragma unroll
            for (int i = 0; i < 2; ++i)
#pragma unroll
                for (int j = 0; j < 2; ++j)
                    acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[i], b[j], acc[i][j], 0, 0, 0);
        }
    }
    // acc[i][j][q]: weight row wn*64 + i*32 + 8*(q/4) + 4*lh + q%4, place base + wm*64 + j*32 + l32
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int place = base + wm * 64 + j * 32 + l32;
        const int p = sorted[place];
        if (UP) {
            const float s = p >= 0 && style == 0 ? weights[p] : 1.f;
#pragma unroll
            for (int q4 = 0; q4 < 4; ++q4) {
                const int f = n0 + wn * 32 + 8 * q4 + 4 * lh;
                if (f >= N) continue;
                float r[4];
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    if (style == 1) {
                        const float gv = acc[0][j][4 * q4 + u];
                        r[u] = p >= 0 ? gv / (1.f + expf(-gv)) * acc[1][j][4 * q4 + u] : 0.f;
                        continue;
                    }
                    const float gv = fminf(s * acc[0][j][4 * q4 + u], limit);
                    const float uv = fminf(fmaxf(s * acc[1][j][4 * q4 + u], -limit), limit);
                    r[u] = p >= 0 ? gv / (1.f + expf(-1.702f * gv)) * (uv + 1.f) : 0.f;
                }
                bf16_t* dst = y_out + (int64_t)place * N + f;
                if (f + 3 < N && (N & 3) == 0) Elem<bf16_t>::store4(dst, r);
                else
                    for (int u = 0; u < 4 && f + u < N; ++u) Elem<bf16_t>::store(dst + u, r[u]);
            }
        } else if (KIND == kTiledGelu) {
#pragma unroll
            for (int i = 0; i < 2; ++i)
#pragma unroll
                for (int q4 = 0; q4 < 4; ++q4) {
                    const int f = n0 + wn * 64 + i * 32 + 8 * q4 + 4 * lh;
                    if (f >= N) continue;
                    float r[4];
#pragma unroll
                    for (int u = 0; u < 4; ++u) r[u] = p >= 0 ? apply_activation(kActGeluErf, acc[i][j][4 * q4 + u]) : 0.f;
                    bf16_t* dst = y_out + (int64_t)place * N + f;
                    if (f + 3 < N && (N & 3) == 0) Elem<bf16_t>::store4(dst, r);
                    else
                        for (int u = 0; u < 4 && f + u < N; ++u) Elem<bf16_t>::store(dst + u, r[u]);
                }
        } else {
            if (p < 0) continue;
#pragma unroll
            for (int i = 0; i < 2; ++i)
#pragma unroll
                for (int q4 = 0; q4 < 4; ++q4) {
                    const int n = n0 + wn * 64 + i * 32 + 8 * q4 + 4 * lh;
#pragma unroll
                    for (int u = 0; u < 4; ++u) {
                        if (n + u >= N) continue;
                        const float v = acc[i][j][4 * q4 + u];
                        if (pair_out) pair_out[(int64_t)place * N + n + u] = v;
                        else {
                            const int64_t at = (int64_t)p * N + n + u;       // one expert a token: p is the token
                            out[at] = fmaf(out_scale, v, residual[at]);
                        }
                    }
                }
        }
    }
}

// V columns a thread and turn (4: 16-byte accesses).  x (or null): the tokens' own vectors, the results of the identity
// experts, whose numbers are `experts` and above.
template <typename T, int V>
__global__ __launch_bounds__(256) void moe_combine_kernel(
    float* out, const float* residual, const float* __restrict__ pair_out,
    const int* __restrict__ place_of_pair, const float* __restrict__ weights, const int* __restrict__ ids,
    const T* __restrict__ x, int experts, int top, int width, float out_scale) {
    const int t = blockIdx.x;
    for (int n = threadIdx.x * V; n < width; n += 256 * V) {
        float sum[V], base[V], own[V];
        bool any = false;
        const int64_t at = (int64_t)t * width + n;
#pragma unroll
        for (int v = 0; v < V; ++v) { sum[v] = 0.f; base[v] = 0.f; own[v] = 0.f; }
        if (residual) {
            if (V == 4) {
                const float4 r = *reinterpret_cast<const float4*>(residual + at);
                base[0] = r.x; base[1 % V] = r.y; base[2 % V] = r.z; base[3 % V] = r.w;
            } else {
                base[0] = residual[at];
            }
        }
        if (x) {
#pragma unroll
            for (int v = 0; v < V; ++v) own[v] = Elem<T>::load(x + at + v);
        }
#pragma unroll 2
        for (int j = 0; j < top; ++j) {
            const int place = place_of_pair[(int64_t)t * top + j];
            const float w = weights ? weights[(int64_t)t * top + j] : 1.f;
            const bool identity = x && ids[(int64_t)t * top + j] >= experts;
            const float* src = pair_out + (int64_t)max(place, 0) * width + n;
            float r[V];
            if (V == 4) {
                const float4 q = *reinterpret_cast<const float4*>(src);
                r[0] = q.x; r[1 % V] = q.y; r[2 % V] = q.z; r[3 % V] = q.w;
            } else {
                r[0] = src[0];
            }
            if (place >= 0 || identity) {
#pragma unroll
                for (int v = 0; v < V; ++v) sum[v] = fmaf(w, identity ? own[v] : r[v], sum[v]);
                any = true;
            }
        }
        if (residual && !any && out == residual) continue;
#pragma unroll
        for (int v = 0; v < V; ++v) sum[v] = any ? fmaf(out_scale, sum[v], base[v]) : base[v];
        if (V == 4) *reinterpret_cast<float4*>(out + at) = make_float4(sum[0], sum[1 % V], sum[2 % V], sum[3 % V]);
        else out[at] = sum[0];
    }
}

}  // namespace st

using namespace st;

extern "C" int st_moe_route(int* ids, float* weights, const float* logits, int logit_stride, const int* token_item,
                            const float* correction, float scale, int num_tokens, int experts, int top, int mode, int groups, int keep,
                            hipStream_t stream) {
    ST_CHECK(mode >= 0 && mode <= 4, "moe_route: mode 0 (sigmoid of each), 1 (softmax over the chosen), 2 (softmax "
             "over all, the choice within the best groups), 3 (sigmoids over their sum, a corrected choice) or 4 (softmax over "
             "all, a corrected choice)");
    ST_CHECK(mode < 3 || correction, "moe_route: modes 3 and 4 choose by corrected scores");
    if (mode != 2) groups = keep = 1;
    ST_CHECK(groups >= 1 && groups <= 64 && experts % groups == 0 && keep >= 1 && keep <= groups,
             "moe_route: %d experts in %d groups of which %d are kept (up to 64 equal groups)", experts, groups, keep);
    ST_CHECK(top <= keep * (experts / groups), "moe_route: %d experts a token do not fit %d groups of %d", top, keep,
             experts / groups);
    ST_CHECK(num_tokens >= 0 && experts > 0, "moe_route: bad sizes");
    ST_CHECK(top >= 1 && top <= kMaxTop && top <= experts, "moe_route: 1 to %d experts a token (of %d), not %d",
             kMaxTop, experts, top);
    ST_CHECK(ids && weights && logits && logit_stride >= experts, "moe_route: null operand or short rows");
    if (num_tokens == 0) return 0;
    // workgroups of as many tokens as have their rows side by side in 48 KB of LDS (256, 64, or none staged)
    const size_t row = (size_t)(experts + 1) * sizeof(float);
    const int threads = 256 * row <= 48 * 1024 ? 256 : 64;
    const int stage = threads * row <= 48 * 1024;
    moe_route_kernel<<<(num_tokens + threads - 1) / threads, threads, stage ? threads * row : 0, stream>>>(
        ids, weights, logits, logit_stride, token_item, correction, scale, num_tokens, experts, top, mode, groups, keep, stage);
    ST_LAUNCH_CHECK("moe_route");
    return 0;
}

extern "C" int st_moe_align(int* sorted, int* place_of_pair, int* tile_expert, const int* ids, int num_pairs,
                            int experts, int capacity, int tile, hipStream_t stream) {
    const int kTile = tile;
    ST_CHECK(num_pairs >= 0 && experts > 0 && experts <= 4096, "moe_align: bad sizes (up to 4096 experts)");
    ST_CHECK(tile == 16 || tile == 64 || tile == 128, "moe_align: tiles of 16, 64 or 128 places, not %d", tile);
    ST_CHECK(capacity % kTile == 0 && capacity >= (num_pairs + kTile - 1) / kTile * kTile + kTile * experts,
             "moe_align: %d places do not hold %d pairs of %d experts in tiles of %d", capacity, num_pairs, experts, kTile);
    ST_CHECK(sorted && place_of_pair && tile_expert && ids, "moe_align: null operand");
    moe_align_kernel<<<1, 1024, (2 * experts + 1) * sizeof(int), stream>>>(sorted, place_of_pair, tile_expert, ids,
                                                                          num_pairs, experts, capacity, tile);
    ST_LAUNCH_CHECK("moe_align");
    return 0;
}

static bool rows_vectorised(const void* a, const void* b, const void* c, int depth, int dtype) {
    const int per = dtype == kF32 ? 4 : 8;
    return depth % per == 0 && ((reinterpret_cast<uintptr_t>(a) | reinterpret_cast<uintptr_t>(b) |
                                 reinterpret_cast<uintptr_t>(c)) & 15) == 0;
}

extern "C" int st_moe_up(void* y, const void* x, const void* w_gate, const void* w_up, const int* sorted,
                         const int* tile_expert, const float* weights, int capacity, int tile, int top, int width,
                         int inner, float limit, int style, int dtype, hipStream_t stream) {
    const int kTile = tile;
    ST_CHECK(style >= 0 && style <= 3, "moe_up: style 0 (weighted, clamped inputs), 1 (plain gated unit), 2 (no gate, GELU) or 3 "
             "(clamped inputs, no weight)");
    if (style == 2) w_gate = w_up;
    ST_CHECK(tile == 16 || tile == 64 || tile == 128, "moe_up: tiles of 16, 64 or 128 places, not %d", tile);
    ST_CHECK(capacity > 0 && capacity % kTile == 0 && top >= 1 && width > 0 && inner > 0, "moe_up: bad sizes");
    ST_CHECK(y && x && w_gate && w_up && sorted && tile_expert && weights, "moe_up: null operand");
    const dim3 grid(capacity / kTile, (inner + 63) / 64);
    ST_CHECK(grid.y <= 65535, "moe_up: too many inner features");
    const int vec = rows_vectorised(x, w_gate, w_up, width, dtype);
    if (dtype == kBF16 && tile == 128 && vec) {
        if (style == 2) {
            moe_tiled_kernel<kTiledGelu><<<dim3(capacity / 128, (inner + 127) / 128), 256, 0, stream>>>((bf16_t*)y, nullptr, nullptr,
                nullptr, (const bf16_t*)x, (const bf16_t*)w_up, nullptr, sorted, tile_expert, weights, top, inner, width, limit, 1.f, style);
            ST_LAUNCH_CHECK("moe_up (tiled, no gate)");
            return 0;
        }
        const dim3 g2(capacity / 128, (inner + 63) / 64);
        moe_tiled_kernel<kTiledUp><<<g2, 256, 0, stream>>>((bf16_t*)y, nullptr, nullptr, nullptr, (const bf16_t*)x,
            (const bf16_t*)w_gate, (const bf16_t*)w_up, sorted, tile_expert, weights, top, inner, width, limit, 1.f, style);
        ST_LAUNCH_CHECK("moe_up (tiled)");
        return 0;
    }
#define ST_UP_G(T, RT, G)                                                                                    \
    moe_up_kernel<T, RT, G><<<grid, 256, 0, stream>>>((T*)y, (const T*)x, (const T*)w_gate, (const T*)w_up, sorted, \
                                                      tile_expert, weights, top, width, inner, limit, style, vec)
    if (tile == 16) {
        const dim3 few(capacity / 16, (inner + 15) / 16);
        ST_CHECK(few.y <= 65535, "moe_up: too many inner features");
#define ST_UP_FEW(T, G)                                                                                      \
    moe_up_few_kernel<T, G><<<few, 256, 0, stream>>>((T*)y, (const T*)x, (const T*)w_gate, (const T*)w_up, sorted, tile_expert, \
                                                     weights, top, width, inner, limit, style, vec)
        if (dtype == kF32) { if (style == 2) ST_UP_FEW(float, false); else ST_UP_FEW(float, true); }
        else if (dtype == kBF16) { if (style == 2) ST_UP_FEW(bf16_t, false); else ST_UP_FEW(bf16_t, true); }
        else ST_CHECK(false, "moe_up: unknown dtype %d", dtype);
#undef ST_UP_FEW
        ST_LAUNCH_CHECK("moe_up (few rows)");
        return 0;
    }
#define ST_UP(T, RT) do { if (style == 2) ST_UP_G(T, RT, false); else ST_UP_G(T, RT, true); } while (0)
    if (dtype == kF32) { if (tile == 64) ST_UP(float, 4); else ST_UP(float, 8); }
    else if (dtype == kBF16) { if (tile == 64) ST_UP(bf16_t, 4); else ST_UP(bf16_t, 8); }
    else ST_CHECK(false, "moe_up: unknown dtype %d", dtype);
#undef ST_UP
#undef ST_UP_G
    ST_LAUNCH_CHECK("moe_up");
    return 0;
}

extern "C" int st_moe_down(float* out, const float* residual, float* pair_out, const void* y, const void* w_down,
                           const int* sorted, const int* tile_expert, int capacity, int tile, int top, int width,
                           int inner, float out_scale, int dtype, hipStream_t stream) {
    const int kTile = tile;
    ST_CHECK(tile == 16 || tile == 64 || tile == 128, "moe_down: tiles of 16, 64 or 128 places, not %d", tile);
    ST_CHECK(capacity > 0 && capacity % kTile == 0 && top >= 1 && width > 0 && inner > 0, "moe_down: bad sizes");
    ST_CHECK(y && w_down && sorted && tile_expert, "moe_down: null operand");
    ST_CHECK(pair_out ? true : (top == 1 && out && residual),
             "moe_down: without a row per pair the result goes to the stream, for one expert a token only");
    const dim3 grid(capacity / kTile, (width + 63) / 64);
    ST_CHECK(grid.y <= 65535, "moe_down: too wide");
    const int vec = rows_vectorised(y, w_down, w_down, inner, dtype);
    if (dtype == kBF16 && tile == 128 && vec) {
        const dim3 g2(capacity / 128, (width + 127) / 128);
        moe_tiled_kernel<kTiledDown><<<g2, 256, 0, stream>>>(nullptr, out, residual, pair_out, (const bf16_t*)y,
            (const bf16_t*)w_down, nullptr, sorted, tile_expert, nullptr, top, width, inner, 0.f, out_scale, 0);
        ST_LAUNCH_CHECK("moe_down (tiled)");
        return 0;
    }
    if (tile == 16) {
        const dim3 few(capacity / 16, (width + 15) / 16);
        ST_CHECK(few.y <= 65535, "moe_down: too wide");
#define ST_DOWN_FEW(T)                                                                                       \
    moe_down_few_kernel<T><<<few, 256, 0, stream>>>(out, residual, pair_out, (const T*)y, (const T*)w_down, sorted, tile_expert, \
                                                    top, width, inner, out_scale, vec)
        if (dtype == kF32) ST_DOWN_FEW(float);
        else if (dtype == kBF16) ST_DOWN_FEW(bf16_t);
        else ST_CHECK(false, "moe_down: unknown dtype %d", dtype);
#undef ST_DOWN_FEW
        ST_LAUNCH_CHECK("moe_down (few rows)");
        return 0;
    }
#define ST_DOWN(T, RT)                                                                                        \
    moe_down_kernel<T, RT><<<grid, 256, 0, stream>>>(out, residual, pair_out, (const T*)y, (const T*)w_down,      \
                                                     sorted, tile_expert, top, width, inner, out_scale, vec)
    if (dtype == kF32) { if (tile == 64) ST_DOWN(float, 4); else ST_DOWN(float, 8); }
    else if (dtype == kBF16) { if (tile == 64) ST_DOWN(bf16_t, 4); else ST_DOWN(bf16_t, 8); }
    else ST_CHECK(false, "moe_down: unknown dtype %d", dtype);
#undef ST_DOWN
    ST_LAUNCH_CHECK("moe_down");
    return 0;
}

// ids and x (both or neither): a choice of `experts` or above is an identity expert, whose result is the token's row of x
// [tokens, width] in the storage type.
extern "C" int st_moe_combine(float* out, const float* residual, const float* pair_out, const int* place_of_pair,
                              const float* weights, const int* ids, const void* x, int experts, int num_tokens, int top,
                              int width, float out_scale, int dtype, hipStream_t stream) {
    ST_CHECK(num_tokens >= 0 && top >= 1 && width > 0, "moe_combine: bad sizes");
    ST_CHECK(out && pair_out && place_of_pair && (!x || ids), "moe_combine: null operand");
    ST_CHECK(dtype == kF32 || dtype == kBF16, "moe_combine: unknown dtype %d", dtype);
    if (num_tokens == 0) return 0;
    const bool vec = width % 4 == 0 && (((uintptr_t)out | (uintptr_t)residual | (uintptr_t)pair_out) & 15) == 0;
#define ST_MC(T, V)                                                                                                    \
    moe_combine_kernel<T, V><<<num_tokens, 256, 0, stream>>>(out, residual, pair_out, place_of_pair, weights, ids, (const T*)x, \
                                                             experts, top, width, out_scale)
    if (dtype == kF32) { if (vec) ST_MC(float, 4); else ST_MC(float, 1); }
    else { if (vec) ST_MC(bf16_t, 4); else ST_MC(bf16_t, 1); }
#undef ST_MC
    ST_LAUNCH_CHECK("moe_combine");
    return 0;
}
