// Root-mean-square norm in groups, alone and with a short causal filter over time behind it.
//
//   n[t, c] = x[t, c] / sqrt(mean of x[t, c']^2 over c's group + eps) * gain[c]      groups: equal consecutive parts
//   y[t, c] = n[t, c] + sum_{j < taps} w[j, c] * n(position p_t - (taps - 1) + j, c)   zeros before the sequence
//
// The filtered form serves one or two readers of one stream: both take the same statistics of x, each has its
// own gain, filter and state ("sides"), and one pass over x makes both results.  The last taps - 1 normed rows of
// a request are its state, float, one a side, in the request's slot.  Rows of the same step are normalised again
// where a later row's filter reaches them (their statistics are formed once a workgroup).  An item of one row
// moves its state on in the same kernel (nothing else of the launch reads that slot); items of several rows have
// it moved by a second kernel after all rows have read it.  Everything is float; the result takes the storage
// type.
#include "api.h"
#include "common.h"

namespace st {

constexpr int kNormMaxTaps = 8;
constexpr int kNormRows = 4;                 // rows a workgroup of the filtered form at prompt sizes

// 1 / sqrt(mean + eps) of one group of one row, by one wave (every lane gets it)
__device__ inline float group_rstd(const float* __restrict__ part, int width, float eps, int vec) {
    const int lane = threadIdx.x & 63;
    float ss = 0.f;
    if (vec) {
        for (int i = lane * 4; i < width; i += 256) {
            const float4 v = *reinterpret_cast<const float4*>(part + i);
            ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
        }
    } else {
        for (int i = lane; i < width; i += 64) ss = fmaf(part[i], part[i], ss);
    }
    return 1.f / sqrtf(wave_sum(ss) / (float)width + eps);
}

template <int V>
__device__ inline void load_columns(const float* __restrict__ p, float* v) {
    if (V == 4) {
        const float4 q = *reinterpret_cast<const float4*>(p);
        v[0] = q.x; v[1 % V] = q.y; v[2 % V] = q.z; v[3 % V] = q.w;
    } else {
        v[0] = p[0];
    }
}
template <int V, typename T>
__device__ inline void store_columns(T* p, const float* v) {
    if (V == 4) Elem<T>::store4(p, v); else Elem<T>::store(p, v[0]);
}

// a wave a (row, group)
template <typename T>
__global__ __launch_bounds__(256) void group_rms_kernel(
    T* __restrict__ out_t, float* __restrict__ out_f32, const float* __restrict__ x, const int* __restrict__ rows,
    const float* __restrict__ gain, int64_t units, int groups, int part, float eps, int vec) {
    const int64_t u = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (u >= units) return;
    const int lane = threadIdx.x & 63;
    const int64_t r = u / groups;
    const int g = (int)(u - r * groups);
    const int64_t src = rows ? rows[r] : r;
    const int64_t at = (r * groups + g) * part;
    if (src < 0) {                               // a padding entry of a row list of fixed length
        for (int i = lane; i < part; i += 64) {
            if (out_t) Elem<T>::store(out_t + at + i, 0.f);
            if (out_f32) out_f32[at + i] = 0.f;
        }
        return;
    }
    const float* p = x + (src * groups + g) * part;
    const float* gp = gain + (int64_t)g * part;
    const float rstd = group_rstd(p, part, eps, vec);
    if (vec) {
        for (int i = lane * 4; i < part; i += 256) {
            const float4 v = *reinterpret_cast<const float4*>(p + i);
            const float4 w = *reinterpret_cast<const float4*>(gp + i);
            const float y[4] = {v.x * rstd * w.x, v.y * rstd * w.y, v.z * rstd * w.z, v.w * rstd * w.w};
            if (out_t) Elem<T>::store4(out_t + at + i, y);
            if (out_f32) Elem<float>::store4(out_f32 + at + i, y);
        }
    } else {
        for (int i = lane; i < part; i += 64) {
            const float y = p[i] * rstd * gp[i];
            if (out_t) Elem<T>::store(out_t + at + i, y);
            if (out_f32) out_f32[at + i] = y;
        }
    }
}

// one reader of the stream: its gain [width], filter [taps, width], state [slots, taps - 1, width] and result
struct NormConvSide {
    const float* gain;
    const float* w;
    float* state;
    int64_t slot_stride;
    void* out;
};

// LDS: statistics [R + TAPS - 1][groups], entry i of them belonging to batch row t0 - (TAPS - 1) + i.  V columns a
// thread and turn (4: 16-byte accesses; groups, width and addresses allow them), R rows a workgroup.  TAPS: 1 to 4, or
// 8 for any number up to that.  What a thread needs (its columns of all the rows, gains, filters, for single tokens
// the state) is asked for before the statistics are formed: few trips to memory, side by side.
template <typename T, int SIDES, int V, int TAPS, int R>
__global__ __launch_bounds__(512) void group_norm_conv_kernel(
    NormConvSide s0, NormConvSide s1, const float* __restrict__ x, const int* __restrict__ token_item,
    const int* __restrict__ item_len, const int* __restrict__ item_tok_off, const int* __restrict__ item_slot,
    int num_tokens, int width, int groups, int num_taps, float eps) {
    extern __shared__ float nc_stat[];
    constexpr int HIST = TAPS - 1;                // rows before the workgroup's own that are kept at hand
    const int hist = TAPS < kNormMaxTaps ? HIST : num_taps - 1, part = width / groups;
    const int t0 = blockIdx.x * R;
    const int n = min(R, num_tokens - t0);
    const NormConvSide side[2] = {s0, s1};
    int slot[R], row[R];                          // slot of the row's request (-1: a padding row), row within its portion
    bool single[R];
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int item = i < n ? token_item[t0 + i] : -1;
        slot[i] = item >= 0 ? item_slot[item] : -1;
        row[i] = slot[i] >= 0 ? t0 + i - item_tok_off[item] : 0;
        single[i] = slot[i] >= 0 && item_len[item] == 1;
    }
    bool have_stats = false;
    for (int c = threadIdx.x * V; c < width || !have_stats; c += blockDim.x * V) {
        const bool live = c < width;
        const int cc = live ? c : 0;              // (a thread without columns still helps with the statistics)
        const int g = cc / part;
        float gain[SIDES][V], w[SIDES][TAPS][V], xv[R + HIST][V], old[SIDES][TAPS][V];
        // (rows before the batch or past it: a stand-in that is not used)
#pragma unroll
        for (int k = 0; k < R + HIST; ++k)
            load_columns<V>(x + (int64_t)min(max(t0 - HIST + k, 0), num_tokens - 1) * width + cc, xv[k]);
#pragma unroll
        for (int s = 0; s < SIDES; ++s) {
            load_columns<V>(side[s].gain + cc, gain[s]);
#pragma unroll
            for (int b = 0; b < TAPS; ++b)        // [rows back]
                load_columns<V>(side[s].w + (int64_t)max(hist - b, 0) * width + cc, w[s][b]);
        }
        auto load_old = [&](int i) {
#pragma unroll
            for (int s = 0; s < SIDES; ++s)
#pragma unroll
                for (int b = 1; b < TAPS; ++b)
                    load_columns<V>(side[s].state + (int64_t)slot[i] * side[s].slot_stride +
                                    (int64_t)min(max(hist + row[i] - b, 0), hist - 1) * width + cc, old[s][b]);
        };
        if (R == 1 && slot[0] >= 0 && row[0] < hist) load_old(0);
        if (!have_stats) {                        // uniform over the workgroup
            // the rows before the workgroup's own that its filters reach: back to where the first row's item starts
            const int before = slot[0] >= 0 ? min(hist, row[0]) : 0;
            const int units = (n + before) * groups, waves = blockDim.x >> 6, lane = threadIdx.x & 63;
            const float* first = x + (int64_t)(t0 - before) * width;
            float* stat = nc_stat + (HIST - before) * groups;
            // (rows side by side in memory: unit u is the part that starts u * part floats behind the first row)
            for (int u = threadIdx.x >> 6; u < units; u += 4 * waves) {
                float ss[4];
                if (part <= 64 * V) {             // a wave covers a part at once: four parts on their way
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        float v[V];
                        const int at = lane * V;
                        load_columns<V>(first + (int64_t)min(u + j * waves, units - 1) * part + min(at, part - V), v);
                        ss[j] = 0.f;
#pragma unroll
                        for (int e = 0; e < V; ++e) ss[j] = at < part ? fmaf(v[e], v[e], ss[j]) : ss[j];
                    }
                } else {
#pragma unroll
                    for (int j = 0; j < 4; ++j) ss[j] = 0.f;
                    for (int at = lane * V; at < part; at += 64 * V) {
#pragma unroll
                        for (int j = 0; j < 4; ++j) {
                            float v[V];
                            load_columns<V>(first + (int64_t)min(u + j * waves, units - 1) * part + at, v);
#pragma unroll
                            for (int e = 0; e < V; ++e) ss[j] = fmaf(v[e], v[e], ss[j]);
                        }
                    }
                }
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    ss[j] = wave_sum(ss[j]);
                    if (lane == 0 && u + j * waves < units) stat[u + j * waves] = 1.f / sqrtf(ss[j] / (float)part + eps);
                }
            }
            __syncthreads();
            have_stats = true;
        }
        if (!live) break;
#pragma unroll
        for (int k = 0; k < R + HIST; ++k) {
            const float rstd = nc_stat[k * groups + g];      // (entries of rows that no filter here reaches: never used)
#pragma unroll
            for (int v = 0; v < V; ++v) xv[k][v] *= rstd;
        }
#pragma unroll
        for (int i = 0; i < R; ++i) {
            if (i >= n) break;
            const int64_t t = t0 + i;
            if (slot[i] < 0) {                    // a padding row of a batch of fixed size
                const float zero[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < SIDES; ++s) store_columns<V>((T*)side[s].out + t * width + cc, zero);
                continue;
            }
            if (R > 1 && row[i] < hist) load_old(i);
#pragma unroll
            for (int s = 0; s < SIDES; ++s) {
                float own[V], acc[V];
#pragma unroll
                for (int v = 0; v < V; ++v) acc[v] = own[v] = xv[HIST + i][v] * gain[s][v];
#pragma unroll
                for (int b = TAPS - 1; b >= 0; --b) {
                    if (b > hist) continue;
#pragma unroll
                    for (int v = 0; v < V; ++v)
                        acc[v] = fmaf(w[s][b][v], b <= row[i] ? xv[HIST + i - b][v] * gain[s][v] : old[s][b][v], acc[v]);
                }
                store_columns<V>((T*)side[s].out + t * width + cc, acc);
                if (single[i]) {                  // its row is 0: what lies b rows back was read from the state above
                    float* st = side[s].state + (int64_t)slot[i] * side[s].slot_stride + cc;
#pragma unroll
                    for (int b = 1; b < TAPS; ++b) {
                        if (b > hist) continue;
                        store_columns<V>(st + (int64_t)(hist - b) * width, b == 1 ? own : old[s][b - 1]);
                    }
                }
            }
        }
    }
}

// a workgroup an item of several rows: the state becomes the last taps - 1 of (old state, the item's normed rows)
template <int SIDES, int V>
__global__ __launch_bounds__(512) void group_norm_conv_state_kernel(
    NormConvSide s0, NormConvSide s1, const float* __restrict__ x, const int* __restrict__ item_len,
    const int* __restrict__ item_tok_off, const int* __restrict__ item_slot, int width, int groups, int taps, float eps) {
    extern __shared__ float nc_stat[];
    const int item = blockIdx.x;
    const int slot = item_slot[item], n = item_len[item];
    if (slot < 0 || n <= 1) return;
    const int hist = taps - 1, part = width / groups;
    const int fresh = min(n, hist), kept = hist - fresh;     // rows from this step, rows that move up in the state
    const float* xi = x + (int64_t)(item_tok_off[item] + n - fresh) * width;
    // (every workgroup of an item forms the statistics of all parts of the rows)
    for (int u = threadIdx.x >> 6; u < fresh * groups; u += blockDim.x >> 6) {
        const float rstd = group_rstd(xi + (int64_t)u * part, part, eps, V == 4);
        if ((threadIdx.x & 63) == 0) nc_stat[u] = rstd;
    }
    const NormConvSide side[2] = {s0, s1};
    const int c = (blockIdx.y * blockDim.x + threadIdx.x) * V;
    const bool live = c < width;
    const int cc = live ? c : 0, g = cc / part;
    float keep[SIDES][kNormMaxTaps][V], gain[SIDES][V];
#pragma unroll
    for (int s = 0; s < SIDES; ++s) {
        const float* st = side[s].state + (int64_t)slot * side[s].slot_stride + cc;
        load_columns<V>(side[s].gain + cc, gain[s]);
#pragma unroll
        for (int i = 0; i < kNormMaxTaps - 1; ++i) {
            if (i >= hist) continue;
            load_columns<V>(i < kept ? st + (int64_t)(i + fresh) * width : xi + (int64_t)(i - kept) * width + cc, keep[s][i]);
        }
    }
    __syncthreads();
    if (!live) return;
#pragma unroll
    for (int s = 0; s < SIDES; ++s) {
        float* st = side[s].state + (int64_t)slot * side[s].slot_stride + cc;
#pragma unroll
        for (int i = 0; i < kNormMaxTaps - 1; ++i) {
            if (i >= hist) continue;
            if (i >= kept) {
                const float rstd = nc_stat[(i - kept) * groups + g];
#pragma unroll
                for (int v = 0; v < V; ++v) keep[s][i][v] *= rstd * gain[s][v];
            }
            store_columns<V>(st + (int64_t)i * width, keep[s][i]);
        }
    }
}

}  // namespace st

using namespace st;

static bool aligned16(const void* a, const void* b = nullptr, const void* c = nullptr, const void* d = nullptr) {
    return (((uintptr_t)a | (uintptr_t)b | (uintptr_t)c | (uintptr_t)d) & 15) == 0;
}

extern "C" int st_group_rms(void* out_t, void* out_f32, const float* x, const int* rows, const float* gain, int num_rows,
                            int width, int groups, float eps, int dtype, hipStream_t stream) {
    ST_CHECK(num_rows >= 0 && width > 0 && groups > 0 && width % groups == 0, "group_rms: %d channels in %d equal groups",
             width, groups);
    ST_CHECK(eps > 0.f, "group_rms: eps must be positive");
    if (num_rows == 0) return 0;
    ST_CHECK((out_t || out_f32) && x && gain, "group_rms: null operand");
    const int part = width / groups;
    const int64_t units = (int64_t)num_rows * groups;
    const int vec = part % 4 == 0 && aligned16(out_t, out_f32, x, gain);
    const unsigned grid = (unsigned)((units + 3) / 4);
    if (dtype == kF32)
        group_rms_kernel<float><<<grid, 256, 0, stream>>>((float*)out_t, (float*)out_f32, x, rows, gain, units, groups, part,
                                                          eps, vec);
    else if (dtype == kBF16)
        group_rms_kernel<bf16_t><<<grid, 256, 0, stream>>>((bf16_t*)out_t, (float*)out_f32, x, rows, gain, units, groups,
                                                           part, eps, vec);
    else ST_CHECK(false, "group_rms: unknown dtype %d", dtype);
    ST_LAUNCH_CHECK("group_rms");
    return 0;
}

// out1 null: one side.  w: [taps, width] (a tap's weights side by side); state: null with one tap.  all_single: no
// item has more than one row (the second kernel is not needed).
extern "C" int st_group_norm_conv(void* out0, const float* gain0, const float* w0, float* state0, int64_t slot_stride0,
                                  void* out1, const float* gain1, const float* w1, float* state1, int64_t slot_stride1,
                                  const float* x, const int* token_item, const int* item_len, const int* item_tok_off,
                                  const int* item_slot, int num_tokens, int num_items, int width, int groups, int taps,
                                  float eps, int all_single, int dtype, hipStream_t stream) {
    ST_CHECK(num_tokens >= 0 && num_items >= 0 && width > 0 && groups > 0 && width % groups == 0,
             "group_norm_conv: %d channels in %d equal groups", width, groups);
    ST_CHECK(taps >= 1 && taps <= kNormMaxTaps, "group_norm_conv: 1 to %d taps, not %d", kNormMaxTaps, taps);
    ST_CHECK(groups <= 1024, "group_norm_conv: up to 1024 groups, not %d", groups);
    ST_CHECK(eps > 0.f, "group_norm_conv: eps must be positive");
    ST_CHECK(dtype == kF32 || dtype == kBF16, "group_norm_conv: unknown dtype %d", dtype);
    if (num_tokens == 0) return 0;
    ST_CHECK(out0 && gain0 && w0 && x && token_item && item_len && item_tok_off && item_slot && (state0 || taps == 1),
             "group_norm_conv: null operand");
    ST_CHECK(!out1 || (gain1 && w1 && (state1 || taps == 1)), "group_norm_conv: null operand of the second side");
    const NormConvSide a{gain0, w0, state0, slot_stride0, out0}, b{gain1, w1, state1, slot_stride1, out1};
    // several rows a workgroup only where that leaves enough workgroups to fill the chip
    // (and where the registers hold several rows' window of a filter)
    const bool many = taps <= 4 && num_tokens >= kNormRows * device_compute_units();
    const int rows = many ? kNormRows : 1;
    const bool vec = (width / groups) % 4 == 0 && aligned16(x, out0, gain0, w0) && aligned16(out1, gain1, w1) &&
                     aligned16(state0, state1) && slot_stride0 % 4 == 0 && slot_stride1 % 4 == 0;
    const unsigned grid = (unsigned)((num_tokens + rows - 1) / rows);
    const int threads = width > 256 * (vec ? 4 : 1) ? 512 : 256;
    const int kept_taps = taps <= 4 ? taps : kNormMaxTaps;
    const size_t lds = sizeof(float) * (size_t)(rows + kept_taps - 1) * groups;
#define ST_NC(T, S, V, K) do {                                                                                        \
        if (many) group_norm_conv_kernel<T, S, V, (K <= 4 ? K : 4), kNormRows><<<grid, threads, lds, stream>>>(a, b, x, token_item,   \
            item_len, item_tok_off, item_slot, num_tokens, width, groups, taps, eps);                                  \
        else group_norm_conv_kernel<T, S, V, K, 1><<<grid, threads, lds, stream>>>(a, b, x, token_item, item_len,      \
            item_tok_off, item_slot, num_tokens, width, groups, taps, eps); } while (0)
#define ST_NC_K(T, S, V) do { switch (taps) { case 1: ST_NC(T, S, V, 1); break; case 2: ST_NC(T, S, V, 2); break;    \
        case 3: ST_NC(T, S, V, 3); break; case 4: ST_NC(T, S, V, 4); break; default: ST_NC(T, S, V, 8); } } while (0)
#define ST_NC_T(T) do { if (out1) { if (vec) ST_NC_K(T, 2, 4); else ST_NC_K(T, 2, 1); }                              \
                        else { if (vec) ST_NC_K(T, 1, 4); else ST_NC_K(T, 1, 1); } } while (0)
    if (dtype == kF32) ST_NC_T(float); else ST_NC_T(bf16_t);
#undef ST_NC_T
#undef ST_NC_K
#undef ST_NC
    ST_LAUNCH_CHECK("group_norm_conv");
    if (all_single || taps == 1 || num_items == 0) return 0;
    const size_t lds2 = sizeof(float) * (size_t)(taps - 1) * groups;
    const int per = 512 * (vec ? 4 : 1);
    ST_CHECK((width + per - 1) / per <= 65535, "group_norm_conv: rows too wide");
    // (a workgroup writes its own columns of the state only, and has read them before)
    const dim3 grid2(num_items, (width + per - 1) / per);
#define ST_NS(S, V) group_norm_conv_state_kernel<S, V><<<grid2, 512, lds2, stream>>>(a, b, x, item_len, item_tok_off, item_slot, \
                                                                                   width, groups, taps, eps)
    if (out1) { if (vec) ST_NS(2, 4); else ST_NS(2, 1); }
    else { if (vec) ST_NS(1, 4); else ST_NS(1, 1); }
#undef ST_NS
    ST_LAUNCH_CHECK("group_norm_conv (state)");
    return 0;
}
