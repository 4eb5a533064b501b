// Attention over a latent cache: every key is its own value, one shared entry a token for all heads.
//
// An entry holds a latent vector (dims [0, out_dim), of which the tail may be another part of the entry or zeros), and
// optionally, from dim `rot_off` on, a key part that was turned by its token's position when it was cached; the queries'
// dims there are turned here (pairs 2i, 2i + 1).  A head's result is the weighted sum of the latents, `out_dim` dims; what
// the heads make of it (a product with a matrix of their own, a gate) follows in `latent_up`.
//
// With one key head the queries of all heads of a token read the same keys, so rows of the products are (token, head)
// pairs, flattened in memory order:
//   tiles   64 tokens of one item are 64 * heads rows, cut into workgroups of 64 rows (prompts and portions);
//   rows    the heads of one token, keys split over workgroups and over the waves of one (decoded tokens): every entry is
//           read once for all heads; partial results (normalised, with their log-sum-exps) are merged by the reader.
// A block of entries lies in LDS once and serves both products: S^T = K Q^T reads its rows, O^T += V^T P^T reads it
// transposed (ds_read_b64_tr_b16).  The blocks come by direct loads (global_load_lds_dwordx4), the next one while this one
// is consumed; softmax is online, float, in units of log2.  A learned number a head may stand in the denominator beside
// the keys (`sink`): it is the softmax's start state, in the first split only.
#include "api.h"
#include "common.h"
#include "fragment.h"

#include <mutex>
#include <set>

namespace st {

typedef short short4v __attribute__((ext_vector_type(4)));

#define ST_LDS_PTR(T, p) ((__attribute__((address_space(3))) T*)(p))
#define ST_GLOBAL_PTR(p) ((const __attribute__((address_space(1))) void*)(p))

constexpr float kLog2e = 1.44269504088896340736f, kLn2 = 0.69314718055994530942f;
constexpr int kTileTokens = 64;

struct LatentArgs {
    void* out;                    // tiles: [tokens, heads, out_dim]
    float* part_o;                // rows: [list, heads, splits, out_dim]
    float* part_lse;              // rows: [list, heads, splits]
    const void* q;                // [tokens, heads, entry], rows of q_stride elements
    const void* cache;            // [pages, page_size, entry]
    const int *tile_item, *tile_q0, *item_tok_off, *item_start, *item_len;
    const int *row_ids, *token_item, *positions, *block_table;
    const float *sink, *freq;
    int64_t q_stride, page_stride;
    int max_pages, page_size, page_shift, heads, entry, out_dim, rot_off, rot_half, window, num_tiles, deal_period,
        num_splits;
    float scale, rot_mult;
};

// The rows of a workgroup: flattened (token, head) pairs fr0 .. of the `total` that its tile (or token) has.
struct LatentRows {
    int item, pos0, fr0, total;
    int64_t token0;               // batch row of the tile's first token
    int list;                     // rows: place in the list
};

template <bool TILES>
__device__ inline bool latent_find_rows(const LatentArgs& a, int rows, LatentRows& r) {
    r.fr0 = blockIdx.x * rows;
    if (TILES) {
        // grid row -> tile, serpentine over rows of `deal_period` tiles from the list's heavy end: a launch is resident
        // all at once, and every compute unit should get long and short tiles
        const int slot = blockIdx.y, line = slot / a.deal_period, base = line * a.deal_period;
        const int in_line = min(a.deal_period, a.num_tiles - base), c = slot - base;
        const int tile = a.num_tiles - 1 - (base + ((line & 1) ? in_line - 1 - c : c));
        r.item = a.tile_item[tile];
        if (r.item < 0) return false;                // a padding entry of a list of fixed length
        const int q0 = a.tile_q0[tile];
        r.total = min(kTileTokens, a.item_len[r.item] - q0) * a.heads;
        r.pos0 = a.item_start[r.item] + q0;
        r.token0 = (int64_t)a.item_tok_off[r.item] + q0;
        r.list = 0;
    } else {
        r.list = blockIdx.y;
        const int t = a.row_ids ? a.row_ids[r.list] : r.list;
        if (t < 0) return false;
        r.item = a.token_item[t];
        r.pos0 = a.positions[t];
        if (r.item < 0 || r.pos0 < 0) return false;
        r.total = a.heads;
        r.token0 = t;
    }
    return r.fr0 < r.total;
}

// The keys of a workgroup: blocks of `block` keys from kb_first on, all keys in [key_lo, key_hi).
struct LatentKeys { int kb_first, key_lo, key_hi, blocks; };

template <bool TILES>
__device__ inline LatentKeys latent_keys(const LatentArgs& a, const LatentRows& r, int rows, int block) {
    LatentKeys k;
    const int last = min(rows, r.total - r.fr0) - 1;
    const int pos_first = r.pos0 + r.fr0 / a.heads, pos_last = r.pos0 + (r.fr0 + last) / a.heads;
    k.key_lo = a.window > 0 && pos_first + 1 > a.window ? pos_first + 1 - a.window : 0;
    k.key_hi = pos_last + 1;
    k.kb_first = k.key_lo / block * block;
    k.blocks = (k.key_hi - k.kb_first + block - 1) / block;
    if (!TILES) {
        const int per = (k.blocks + a.num_splits - 1) / a.num_splits;
        k.kb_first += (int)blockIdx.z * per * block;
        k.key_lo = max(k.key_lo, k.kb_first);
        k.key_hi = min(k.key_hi, k.kb_first + per * block);
        k.blocks = k.key_hi > k.kb_first ? (k.key_hi - k.kb_first + block - 1) / block : 0;
    }
    return k;
}

// XOR of the 16-byte chunk index within a row of CH chunks (a multiple of 4): the 16 lanes of a ds_read_b128 phase (16
// rows, one chunk) and the 32 lanes of a transposing read's phase (8 rows, two neighbouring chunks each) fall on distinct
// banks.  It depends on row % 16 only and stays inside aligned groups of 16, 8 or 4 chunks.
template <int CH> __device__ inline int latent_swizzle(int row) {
    if (CH % 16 == 0) return ((row & 7) << 1) | ((row >> 3) & 1);
    if (CH % 8 == 0) return (((row >> 1) & 3) << 1) | ((row >> 3) & 1);
    return (((row >> 2) & 1) << 1) | ((row >> 3) & 1);
}

// cosine and sine (times rot_mult) of the turning pairs at the positions of a workgroup's tokens: [tokens][rot_half] in LDS.
// (Once a position in LDS instead of once a lane: the accurate functions, inlined at every place of a query that may
// turn, were four fifths of the kernel's code, and a short launch is as long as its code takes to arrive.)
template <int THREADS>
__device__ inline void latent_turns(const LatentArgs& a, const LatentRows& r, int rows, float2* turns) {
    const int last = min(rows, r.total - r.fr0) - 1, first = r.fr0 / a.heads, tokens = (r.fr0 + last) / a.heads - first + 1;
#pragma unroll 1
    for (int i = threadIdx.x; i < tokens * a.rot_half; i += THREADS) {
        const int t = i / a.rot_half;
        const float ang = (float)(r.pos0 + first + t) * a.freq[i - t * a.rot_half];
        turns[i] = make_float2(cosf(ang) * a.rot_mult, sinf(ang) * a.rot_mult);
    }
}
// tokens of a workgroup at most
__host__ __device__ inline int latent_tokens(int rows, int heads) {
    const int n = (rows - 1 + heads - 1) / heads + 1;
    return n < kTileTokens ? n : kTileTokens;
}

__device__ inline float lo_half(uint32_t w) { return __uint_as_float(w << 16); }
__device__ inline float hi_half(uint32_t w) { return __uint_as_float(w & 0xffff0000u); }

// HDP: 32-wide steps over the entry; QT: subtiles of 16 rows a wave; NKT: 16-key subtiles of a block; RW: waves over the
// rows; KW: groups of RW waves, each with its own share of the key blocks and its own LDS, merged at the end.
template <bool TILES, int HDP, int QT, int NKT, int RW, int KW>
__global__ __launch_bounds__(64 * RW * KW) void latent_attn_kernel(const LatentArgs a) {
    constexpr int CH = 4 * HDP, ROWB = CH * 16, DK = 16 * NKT, DT = 2 * HDP, ROWS = RW * QT * 16, BUF = DK * ROWB;
    constexpr int NI = DK * CH / (64 * RW);          // direct loads (1 KB each) a wave and block
    static_assert(NI * 64 * RW == DK * CH && NKT % 2 == 0, "whole loads");
    extern __shared__ uint4 dyn[];
    char* lds_all = reinterpret_cast<char*>(dyn);    // a group of waves: [2 buffers][DK rows][ROWB]
    float2* turns = reinterpret_cast<float2*>(lds_all + KW * 2 * BUF);
    int* s_bt = reinterpret_cast<int*>(turns + (a.rot_half ? (TILES ? latent_tokens(ROWS, a.heads) : 1) * a.rot_half + 4 : 0));
    LatentRows rows;
    if (!latent_find_rows<TILES>(a, ROWS, rows)) return;
    const LatentKeys keys = latent_keys<TILES>(a, rows, ROWS, DK);
    const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, r16 = lane & 15;
    const int wave_all = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int part = wave_all / RW, wave = wave_all % RW;
    char* lds = lds_all + part * 2 * BUF;
    const bf16_t* cache = reinterpret_cast<const bf16_t*>(a.cache);
    const int shift = a.page_shift, psize = a.page_size;
    auto page_of = [&](int key) { return shift >= 0 ? key >> shift : key / psize; };
    const int p_lo = page_of(keys.kb_first);
    if (keys.blocks > 0) {                           // the pages of these keys -> LDS
        const int p_n = page_of(keys.key_hi - 1) - p_lo + 1;
        const int* bt = a.block_table + (int64_t)rows.item * a.max_pages + p_lo;
        for (int i = tid; i < p_n; i += 64 * RW * KW) s_bt[i] = bt[i];
    }
    // ---- queries: lane (row r16 of a subtile, group g) holds dims 32 s + 8 g .. + 7, turned where they meet the turned part
    uint4 qraw[QT][HDP];
    bf16x8 qf[QT][HDP];
    int qpos[QT], qhead[QT];
    bool qvalid[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const int i = rows.fr0 + (wave * QT + t) * 16 + r16;
        qvalid[t] = i < rows.total;
        const int ii = qvalid[t] ? i : rows.fr0, token = ii / a.heads;
        qhead[t] = ii - token * a.heads;
        qpos[t] = rows.pos0 + token;
        const bf16_t* qrow = reinterpret_cast<const bf16_t*>(a.q) + (rows.token0 + token) * a.q_stride + (int64_t)qhead[t] * a.entry;
#pragma unroll
        for (int s = 0; s < HDP; ++s) {
            const int d = 32 * s + 8 * g;
            const uint4 v = *reinterpret_cast<const uint4*>(qrow + min(d, a.entry - 8));
            qraw[t][s] = qvalid[t] && d < a.entry ? v : make_uint4(0, 0, 0, 0);
        }
    }
    if (a.rot_half) {
        latent_turns<64 * RW * KW>(a, rows, ROWS, turns);
        __syncthreads();
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const float2* mine = turns + (qpos[t] - rows.pos0 - rows.fr0 / a.heads) * a.rot_half;
#pragma unroll
        for (int s = 0; s < HDP; ++s) {
            const int d = 32 * s + 8 * g;
            uint4 v = qraw[t][s];
            const int pair0 = (d - a.rot_off) >> 1;
            if (d >= a.rot_off && pair0 < a.rot_half) {
                uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float2 cs = mine[pair0 + e];           // (past the last pair: whatever follows, not used)
                    const float u = lo_half(w[e]), x = hi_half(w[e]);
                    const uint32_t turned = pack_bf16x2(u * cs.x - x * cs.y, x * cs.x + u * cs.y);
                    w[e] = pair0 + e < a.rot_half ? turned : w[e];
                }
                v = make_uint4(w[0], w[1], w[2], w[3]);
            }
            if (a.scale < 0.f) v = make_uint4(v.x ^ 0x80008000u, v.y ^ 0x80008000u, v.z ^ 0x80008000u, v.w ^ 0x80008000u);
            else if (a.scale == 0.f) v = make_uint4(0, 0, 0, 0);
            qf[t][s] = __builtin_bit_cast(bf16x8, v);
        }
    }
    // (the maximum is kept as block maximum times a positive factor: a negative scale has turned the queries around)
    const float sl = (a.scale == 0.f ? 1.f : fabsf(a.scale)) * kLog2e;

    // ---- direct loads: load j of this wave fills LDS bytes [(wave * NI + j) * 1024, + 1024) of a buffer in lane order;
    // slot (row, chunk) takes the entry's chunk (chunk ^ swizzle(row)); chunks past the entry stay the zeros they are
    const int chunks = a.entry >> 3;
    auto issue = [&](int kb, int buf) {
        char* dst = lds + buf * BUF + wave * (NI * 1024);
        const bool whole = kb >= keys.key_lo && kb + DK <= keys.key_hi;
#pragma unroll
        for (int j = 0; j < NI; ++j) {
            const int slot = (wave * NI + j) * 64 + lane, row = slot / CH, c = (slot % CH) ^ latent_swizzle<CH>(row);
            int key = kb + row;
            if (!whole) key = min(max(key, keys.key_lo), keys.key_hi - 1);     // (an address that exists; masked below)
            const int p = page_of(key);
            const int64_t off = (int64_t)s_bt[p - p_lo] * a.page_stride + (int64_t)(key - p * psize) * a.entry + 8 * c;
            if (c < chunks)
                __builtin_amdgcn_global_load_lds(ST_GLOBAL_PTR(cache + off), ST_LDS_PTR(void, dst + j * 1024), 16, 0, 0);
        }
    };
    // ---- readers' offsets.  As keys: row r16 of a subtile, chunk 4 s + g.  Transposed: a lane of 16 reads 4 dims (8 bytes)
    // of row 4 g + r16 / 4, chunk 2 dt + (r16 % 4) / 2, and receives dim r16 of four rows
    const int sw_k = latent_swizzle<CH>(r16), vrow = 4 * g + (r16 >> 2), sw_v = latent_swizzle<CH>(vrow);
    int koff[HDP], voff[DT];
#pragma unroll
    for (int s = 0; s < HDP; ++s) koff[s] = r16 * ROWB + (((4 * s + g) ^ sw_k) << 4);
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) voff[dt] = vrow * ROWB + (((2 * dt + ((r16 & 3) >> 1)) ^ sw_v) << 4) + ((r16 & 1) << 3);

    // running maximum (log2 units, from a finite floor), accumulators, and the normaliser as one more row of the product
    float ms[QT];
    floatx4 acc[QT][DT], accl[QT];
    const bool with_sink = a.sink && part == 0 && (TILES || blockIdx.z == 0);
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        ms[t] = with_sink ? a.sink[qhead[t]] * kLog2e : -1.0e30f;
        const float one = with_sink ? 1.f : 0.f;
        accl[t] = floatx4{one, one, one, one};
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) acc[t][dt] = floatx4{0.f, 0.f, 0.f, 0.f};
    }
    const bf16x8 ones = __builtin_bit_cast(bf16x8, make_uint4(0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u));
    int sub_first[QT], sub_last[QT];                 // first and last position of a subtile's rows
    int wave_last = -1;
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const int i0 = rows.fr0 + (wave * QT + t) * 16, i1 = min(rows.total - 1, i0 + 15);
        sub_first[t] = rows.pos0 + min(i0, rows.total - 1) / a.heads;
        sub_last[t] = i0 < rows.total ? rows.pos0 + i1 / a.heads : -1;
        wave_last = max(wave_last, sub_last[t]);
    }

    auto consume = [&](int kb, int buf) {
        if (kb > wave_last) return;                  // beyond the last row of this wave
        const char* ks = lds + buf * BUF;
        // S^T: st[t][kt][r] = score of key kb + 16 kt + 4 g + r with this lane's row of subtile t
        floatx4 st[QT][NKT];
#pragma unroll
        for (int t = 0; t < QT; ++t)
#pragma unroll
            for (int kt = 0; kt < NKT; ++kt) st[t][kt] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < HDP; ++s) {
            bf16x8 k8[NKT];
#pragma unroll
            for (int kt = 0; kt < NKT; ++kt)
                k8[kt] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(
                    ks + kt * 16 * ROWB + koff[s]));
#pragma unroll
            for (int t = 0; t < QT; ++t)
#pragma unroll
                for (int kt = 0; kt < NKT; ++kt) st[t][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k8[kt], qf[t][s], st[t][kt], 0, 0, 0);
        }
        bf16x8 pf[QT][NKT / 2];
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            const bool interior = kb + DK - 1 <= sub_first[t] && kb >= keys.key_lo && (a.window <= 0 || kb > sub_last[t] - a.window);
            if (!interior) {
#pragma unroll
                for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const int j = kb + 16 * kt + 4 * g + r;
                        const bool ok = qvalid[t] && j <= qpos[t] && j >= keys.key_lo && (a.window <= 0 || j > qpos[t] - a.window);
                        st[t][kt][r] = ok ? st[t][kt][r] : -INFINITY;
                    }
            }
            float bmax = st[t][0][0];
#pragma unroll
            for (int kt = 0; kt < NKT; ++kt) {
                bmax = max3_raw(bmax, st[t][kt][0], st[t][kt][1]);
                bmax = max3_raw(bmax, st[t][kt][2], st[t][kt][3]);
            }
            bmax = rows4_max(bmax);
            const float mc = max_raw(ms[t], bmax * sl);
            const float alpha = __builtin_amdgcn_exp2f(ms[t] - mc);
            ms[t] = mc;
            if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {    // (no row of the wave has moved its maximum: alpha is 1)
#pragma unroll
                for (int dt = 0; dt < DT; ++dt) acc[t][dt] *= alpha;
                accl[t] *= alpha;
            }
#pragma unroll
            for (int u = 0; u < NKT / 2; ++u) {
                uint32_t packed[4];
#pragma unroll
                for (int half = 0; half < 2; ++half) {
                    float p[4];
#pragma unroll
                    for (int r = 0; r < 4; ++r) p[r] = __builtin_amdgcn_exp2f(fmaf(st[t][2 * u + half][r], sl, -mc));
                    packed[2 * half] = pack_bf16x2(p[0], p[1]);
                    packed[2 * half + 1] = pack_bf16x2(p[2], p[3]);
                }
                pf[t][u] = __builtin_bit_cast(bf16x8, make_uint4(packed[0], packed[1], packed[2], packed[3]));
            }
        }
#pragma unroll
        for (int u = 0; u < NKT / 2; ++u) {
#pragma unroll
            for (int t = 0; t < QT; ++t) accl[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pf[t][u], accl[t], 0, 0, 0);
#pragma unroll
            for (int dt = 0; dt < DT; ++dt) {
                if (16 * dt >= a.out_dim) continue;  // uniform
                const char* at = ks + 32 * u * ROWB + voff[dt];
                const short4v lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(ST_LDS_PTR(short4v, at));
                const short4v hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(ST_LDS_PTR(short4v, at + 16 * ROWB));
                const uint2 lo2 = __builtin_bit_cast(uint2, lo), hi2 = __builtin_bit_cast(uint2, hi);
                const bf16x8 v8 = __builtin_bit_cast(bf16x8, make_uint4(lo2.x, lo2.y, hi2.x, hi2.y));
#pragma unroll
                for (int t = 0; t < QT; ++t) acc[t][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v8, pf[t][u], acc[t][dt], 0, 0, 0);
            }
        }
    };

    // group `part` takes blocks part, part + KW, ...; every group goes through the loop the same number of times
    if (a.entry < 32 * HDP) {                        // chunks that no load fills are zeros for good
        for (int i = tid; i < KW * 2 * BUF / 16; i += 64 * RW * KW) dyn[i] = make_uint4(0, 0, 0, 0);
    }
    __syncthreads();
    const int rounds = (keys.blocks + KW - 1) / KW;
    if (part < keys.blocks) issue(keys.kb_first + part * DK, 0);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    for (int it = 0; it < rounds; ++it) {
        const int b = it * KW + part;
        if (b + KW < keys.blocks) issue(keys.kb_first + (b + KW) * DK, (it + 1) & 1);
        if (b < keys.blocks) consume(keys.kb_first + b * DK, it & 1);
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
    }
    if (KW > 1) {                                    // the groups' partial results meet in LDS
        constexpr int E = QT * (2 + 4 * DT);         // floats a lane
        float* mg = reinterpret_cast<float*>(lds_all);
        if (part > 0) {
            float* dst = mg + (size_t)((part - 1) * RW + wave) * E * 64 + lane;
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                dst[(t * (2 + 4 * DT)) * 64] = ms[t];
                dst[(t * (2 + 4 * DT) + 1) * 64] = accl[t][0];
#pragma unroll
                for (int dt = 0; dt < DT; ++dt) {
                    if (16 * dt >= a.out_dim) continue;
#pragma unroll
                    for (int r = 0; r < 4; ++r) dst[(t * (2 + 4 * DT) + 2 + 4 * dt + r) * 64] = acc[t][dt][r];
                }
            }
        }
        __syncthreads();
        if (part > 0) return;
#pragma unroll
        for (int p = 1; p < KW; ++p) {
            const float* src = mg + (size_t)((p - 1) * RW + wave) * E * 64 + lane;
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                const float mo = src[(t * (2 + 4 * DT)) * 64], lo = src[(t * (2 + 4 * DT) + 1) * 64];
                const float mn = max_raw(ms[t], mo);
                const float wa = __builtin_amdgcn_exp2f(ms[t] - mn), wb = __builtin_amdgcn_exp2f(mo - mn);
                accl[t][0] = accl[t][0] * wa + lo * wb;
#pragma unroll
                for (int dt = 0; dt < DT; ++dt) {
                    if (16 * dt >= a.out_dim) continue;
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        acc[t][dt][r] = acc[t][dt][r] * wa + src[(t * (2 + 4 * DT) + 2 + 4 * dt + r) * 64] * wb;
                }
                ms[t] = mn;
            }
        }
    }
    // acc[t][dt][r] = O[this lane's row of subtile t][dim 16 dt + 4 g + r]
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        if (!qvalid[t]) continue;
        const float lsum = accl[t][0], inv = lsum > 0.f ? 1.0f / lsum : 0.f;
        if (TILES) {
            bf16_t* orow = reinterpret_cast<bf16_t*>(a.out) + ((rows.token0 + qpos[t] - rows.pos0) * a.heads + qhead[t]) * a.out_dim;
#pragma unroll
            for (int dt = 0; dt < DT; ++dt) {
                if (16 * dt >= a.out_dim) continue;
                *reinterpret_cast<uint2*>(orow + 16 * dt + 4 * g) =
                    make_uint2(pack_bf16x2(acc[t][dt][0] * inv, acc[t][dt][1] * inv), pack_bf16x2(acc[t][dt][2] * inv, acc[t][dt][3] * inv));
            }
        } else {
            const int64_t at = ((int64_t)rows.list * a.heads + qhead[t]) * a.num_splits + blockIdx.z;
            float* orow = a.part_o + at * a.out_dim;
#pragma unroll
            for (int dt = 0; dt < DT; ++dt) {
                if (16 * dt >= a.out_dim) continue;
                *reinterpret_cast<float4*>(orow + 16 * dt + 4 * g) =
                    make_float4(acc[t][dt][0] * inv, acc[t][dt][1] * inv, acc[t][dt][2] * inv, acc[t][dt][3] * inv);
            }
            if (g == 0) a.part_lse[at] = lsum > 0.f ? ms[t] * kLn2 + logf(lsum) : -INFINITY;
        }
    }
}

// The float twin: v_mfma_f32_16x16x4_f32 (true 32-bit), accurate exponentials; four waves of 16 rows, blocks of 32 keys that
// all waves share.  ET: 16-wide steps over the entry.
constexpr int kLatentF32Keys = 32;
template <bool TILES, int ET>
__global__ __launch_bounds__(256) void latent_attn_f32_kernel(const LatentArgs a) {
    constexpr int DK = kLatentF32Keys, KS = 16 * ET + 4, ROWS = 64;
    extern __shared__ uint4 dyn[];
    float* ks = reinterpret_cast<float*>(dyn);       // [DK][KS]
    float2* turns = reinterpret_cast<float2*>(ks + DK * KS);
    int* s_bt = reinterpret_cast<int*>(turns + (a.rot_half ? (TILES ? latent_tokens(ROWS, a.heads) : 1) * a.rot_half + 4 : 0));
    LatentRows rows;
    if (!latent_find_rows<TILES>(a, ROWS, rows)) return;
    const LatentKeys keys = latent_keys<TILES>(a, rows, ROWS, DK);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, r16 = lane & 15;
    const float* cache = reinterpret_cast<const float*>(a.cache);
    const int psize = a.page_size, p_lo = keys.kb_first / psize;
    if (keys.blocks > 0) {
        const int p_n = (keys.key_hi - 1) / psize - p_lo + 1;
        const int* bt = a.block_table + (int64_t)rows.item * a.max_pages + p_lo;
        for (int i = tid; i < p_n; i += 256) s_bt[i] = bt[i];
    }
    const int i = rows.fr0 + wave * 16 + r16;
    const bool qvalid = i < rows.total;
    const int ii = qvalid ? i : rows.fr0, token = ii / a.heads, qhead = ii - token * a.heads, qpos = rows.pos0 + token;
    floatx4 qf[ET];                                  // dims 16 j + 4 g .. + 3
    if (a.rot_half) {
        latent_turns<256>(a, rows, ROWS, turns);
        __syncthreads();
    }
    {
        const float2* mine = turns + (token - rows.fr0 / a.heads) * a.rot_half;
        const float* qrow = reinterpret_cast<const float*>(a.q) + (rows.token0 + token) * a.q_stride + (int64_t)qhead * a.entry;
#pragma unroll
        for (int j = 0; j < ET; ++j) {
            const int d = 16 * j + 4 * g;
            floatx4 v = floatx4{0.f, 0.f, 0.f, 0.f};
            if (qvalid && d < a.entry) v = *reinterpret_cast<const floatx4*>(qrow + d);
            const int pair0 = (d - a.rot_off) >> 1;
            if (d >= a.rot_off && pair0 < a.rot_half) {
#pragma unroll
                for (int e = 0; e < 2; ++e) {
                    if (pair0 + e >= a.rot_half) continue;
                    const float2 cs = mine[pair0 + e];
                    const float u = v[2 * e], x = v[2 * e + 1];
                    v[2 * e] = u * cs.x - x * cs.y;
                    v[2 * e + 1] = x * cs.x + u * cs.y;
                }
            }
            qf[j] = v;
        }
    }
    const bool with_sink = a.sink && (TILES || blockIdx.z == 0);
    // (l: this lane's share of the normaliser; the sink's belongs to one of the row's four lanes)
    float m = with_sink ? a.sink[qhead] : -INFINITY, l = with_sink && g == 0 ? 1.f : 0.f;
    floatx4 acc[ET];
#pragma unroll
    for (int dt = 0; dt < ET; ++dt) acc[dt] = floatx4{0.f, 0.f, 0.f, 0.f};
    for (int b = 0; b < keys.blocks; ++b) {
        const int kb = keys.kb_first + b * DK;
        __syncthreads();                             // the page list is there; the block before has been read
        for (int e = tid; e < DK * ET * 4; e += 256) {
            const int row = e / (ET * 4), d = 4 * (e % (ET * 4)), key = kb + row;
            floatx4 v = floatx4{0.f, 0.f, 0.f, 0.f};
            if (d < a.entry && key >= keys.key_lo && key < keys.key_hi) {
                const int p = key / psize;
                v = *reinterpret_cast<const floatx4*>(cache + (int64_t)s_bt[p - p_lo] * a.page_stride + (int64_t)(key - p * psize) * a.entry + d);
            }
            *reinterpret_cast<floatx4*>(ks + row * KS + d) = v;
        }
        __syncthreads();
        floatx4 st[2] = {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int j = 0; j < ET; ++j)
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const floatx4 k4 = *reinterpret_cast<const floatx4*>(ks + (16 * t + r16) * KS + 16 * j + 4 * g);
#pragma unroll
                for (int e = 0; e < 4; ++e) st[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[e], qf[j][e], st[t], 0, 0, 0);
            }
        float bmax = -INFINITY;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int j = kb + 16 * t + 4 * g + r;
                const bool ok = qvalid && j <= qpos && j >= keys.key_lo && j < keys.key_hi && (a.window <= 0 || j > qpos - a.window);
                st[t][r] = ok ? st[t][r] * a.scale : -INFINITY;
                bmax = fmaxf(bmax, st[t][r]);
            }
        bmax = rows4_max(bmax);
        const float mn = fmaxf(m, bmax), msafe = mn == -INFINITY ? 0.f : mn, alpha = expf(m - msafe);
        float psum = 0.f;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                st[t][r] = expf(st[t][r] - msafe);
                psum += st[t][r];
            }
        l = l * alpha + psum;
        m = mn;
#pragma unroll
        for (int dt = 0; dt < ET; ++dt) acc[dt] *= alpha;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float* vr = ks + (16 * t + 4 * g + r) * KS + r16;
#pragma unroll
                for (int dt = 0; dt < ET; ++dt) {
                    if (16 * dt >= a.out_dim) continue;
                    acc[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(vr[16 * dt], st[t][r], acc[dt], 0, 0, 0);
                }
            }
    }
    l = rows4_sum(l);
    if (!qvalid) return;
    const float inv = l > 0.f ? 1.0f / l : 0.f;
    float* orow;
    if (TILES) {
        orow = reinterpret_cast<float*>(a.out) + ((rows.token0 + token) * a.heads + qhead) * a.out_dim;
    } else {
        const int64_t at = ((int64_t)rows.list * a.heads + qhead) * a.num_splits + blockIdx.z;
        orow = a.part_o + at * a.out_dim;
        if (g == 0) a.part_lse[at] = l > 0.f ? m + logf(l) : -INFINITY;
    }
#pragma unroll
    for (int dt = 0; dt < ET; ++dt) {
        if (16 * dt >= a.out_dim) continue;
        *reinterpret_cast<floatx4*>(orow + 16 * dt + 4 * g) = acc[dt] * inv;
    }
}

// ---- partial results -> o[token, head, :] in the storage type (a workgroup a list entry and head)
template <typename T>
__global__ __launch_bounds__(64) void latent_merge_kernel(T* __restrict__ out, const float* __restrict__ part_o,
                                                          const float* __restrict__ part_lse, const int* __restrict__ row_ids,
                                                          int heads, int out_dim, int splits) {
    const int list = blockIdx.y, h = blockIdx.x;
    const int t = row_ids ? row_ids[list] : list;
    if (t < 0) return;
    const int64_t at = ((int64_t)list * heads + h) * splits;
    float M = -INFINITY;
    for (int s = 0; s < splits; ++s) M = fmaxf(M, part_lse[at + s]);
    for (int d = threadIdx.x; d < out_dim; d += 64) {
        float W = 0.f, o = 0.f;
        for (int s = 0; s < splits; ++s) {
            const float w = M > -INFINITY ? expf(part_lse[at + s] - M) : 0.f;
            W += w;
            o = fmaf(w, part_o[(at + s) * out_dim + d], o);
        }
        Elem<T>::store(out + ((int64_t)t * heads + h) * out_dim + d, W > 0.f ? o / W : 0.f);
    }
}

// ---- y[t, h, v] = sigmoid(gate[t, h, v]) * sum_r W[h, v, r] o[t, h, r]
// Decoded tokens: a workgroup a (head, token) merges the key splits in float and takes its head's product; groups of 8
// lanes a value dim.
template <typename T>
__global__ __launch_bounds__(256) void latent_up_rows_kernel(
    T* __restrict__ y, const float* __restrict__ part_o, const float* __restrict__ part_lse, const T* __restrict__ w,
    const float* __restrict__ gate, int64_t gate_stride, const int* __restrict__ token_item, int heads, int value_dim,
    int out_dim, int splits) {
    extern __shared__ __attribute__((aligned(16))) float s_o[];        // [out_dim] | weights [splits]
    float* s_w = s_o + out_dim;
    const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x;
    if (token_item[t] < 0) return;
    const int64_t at = ((int64_t)t * heads + h) * splits;
    if (tid < 64) {
        float M = -INFINITY;
        for (int s = tid; s < splits; s += 64) M = fmaxf(M, part_lse[at + s]);
        M = wave_max(M);
        float W = 0.f;
        for (int s = tid; s < splits; s += 64) {
            const float e = M > -INFINITY ? expf(part_lse[at + s] - M) : 0.f;
            s_w[s] = e;
            W += e;
        }
        W = wave_sum(W);
        for (int s = tid; s < splits; s += 64) s_w[s] = W > 0.f ? s_w[s] / W : 0.f;
    }
    __syncthreads();
    for (int d = tid; d < out_dim; d += 256) {
        float o = 0.f;
#pragma unroll 4
        for (int s = 0; s < splits; ++s) o = fmaf(s_w[s], part_o[(at + s) * out_dim + d], o);
        s_o[d] = o;
    }
    __syncthreads();
    constexpr int VEC = Elem<T>::kVec;
    const int sub = tid & 7;
    const T* wh = w + (int64_t)h * value_dim * out_dim;
    for (int v0 = 0; v0 < value_dim; v0 += 32) {
        const int v = v0 + (tid >> 3), vv = min(v, value_dim - 1);
        float dot = 0.f;
#pragma unroll 2
        for (int d = sub * VEC; d < out_dim; d += 8 * VEC) {
            float x[VEC];
            Elem<T>::load_vec(wh + (int64_t)vv * out_dim + d, x);
#pragma unroll
            for (int e = 0; e < VEC; ++e) dot = fmaf(x[e], s_o[d + e], dot);
        }
#pragma unroll
        for (int o = 4; o > 0; o >>= 1) dot += __shfl_xor(dot, o, 64);
        if (sub == 0 && v < value_dim) {
            if (gate) dot /= 1.f + expf(-gate[(int64_t)t * gate_stride + (int64_t)h * value_dim + v]);
            Elem<T>::store(y + ((int64_t)t * heads + h) * value_dim + v, dot);
        }
    }
}

// Prompts: a wave takes 16 tokens of a head on the matrix cores; DS steps over out_dim at most.
template <typename T, int DS>
__global__ __launch_bounds__(256) void latent_up_kernel(
    T* __restrict__ y, const T* __restrict__ o, const T* __restrict__ w, const float* __restrict__ gate, int64_t gate_stride,
    int num_tokens, int heads, int value_dim, int out_dim) {
    using F = Frag<T>;
    const int h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, r16 = lane & 15;
    const int t = blockIdx.x * 64 + wave * 16 + r16;
    if (blockIdx.x * 64 + wave * 16 >= num_tokens) return;             // uniform over the wave
    const int64_t row = (int64_t)min(t, num_tokens - 1) * heads + h;
    F fo[DS];
#pragma unroll
    for (int s = 0; s < DS; ++s) {
        const int d = F::kDepth * s + F::kLane * g;
        fo[s].load(o + row * out_dim, d, out_dim, true, true);
    }
    const T* wh = w + (int64_t)h * value_dim * out_dim;
    const bool quads = value_dim % 4 == 0 && gate_stride % 4 == 0 && ((reinterpret_cast<uintptr_t>(gate) | reinterpret_cast<uintptr_t>(y)) & 15) == 0;
    for (int v0 = 0; v0 < value_dim; v0 += 16) {
        floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
        const T* wr = wh + (int64_t)min(v0 + r16, value_dim - 1) * out_dim;
#pragma unroll
        for (int s = 0; s < DS; ++s) {
            if (F::kDepth * s >= out_dim) continue;                    // uniform
            F fw;
            fw.load(wr, F::kDepth * s + F::kLane * g, out_dim, true, true);
            acc = F::mma(fw, fo[s], acc);
        }
        // acc[r]: value dim v0 + 4 g + r of token t
        const int v = v0 + 4 * g;
        if (t >= num_tokens || v >= value_dim) continue;
        float out[4] = {acc[0], acc[1], acc[2], acc[3]};
        T* dst = y + row * value_dim + v;
        const float* gp = gate + (int64_t)t * gate_stride + (int64_t)h * value_dim + v;
        if (quads) {
            if (gate) {
                const float4 z = *reinterpret_cast<const float4*>(gp);
                out[0] /= 1.f + expf(-z.x); out[1] /= 1.f + expf(-z.y); out[2] /= 1.f + expf(-z.z); out[3] /= 1.f + expf(-z.w);
            }
            Elem<T>::store4(dst, out);
        } else {
            for (int r = 0; r < 4 && v + r < value_dim; ++r) {
                if (gate) out[r] /= 1.f + expf(-gp[r]);
                Elem<T>::store(dst + r, out[r]);
            }
        }
    }
}

}  // namespace st

using namespace st;

static constexpr size_t kLatentMaxLds = 156 * 1024;
static constexpr int kLatentMaxEntry = 576;

static int latent_raise_lds(const void* kernel, size_t bytes) {
    static std::mutex mutex;
    static std::set<const void*> raised;
    ST_CHECK(bytes <= kLatentMaxLds, "latent_attention: %zu bytes of LDS (a page list this long does not fit)", bytes);
    if (bytes <= 48 * 1024) return 0;
    std::lock_guard<std::mutex> lock(mutex);
    if (raised.count(kernel)) return 0;
    ST_CHECK(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLatentMaxLds) == hipSuccess,
             "latent_attention: cannot raise the LDS limit");
    raised.insert(kernel);
    return 0;
}

// Page numbers a workgroup may hold: those of all keys (tiles), or of a split's share of the longest sequence.
static int64_t latent_table(const LatentArgs& a, bool tiles, int block) {
    if (tiles || a.num_splits == 1) return a.max_pages;
    const int64_t blocks = ((int64_t)a.max_pages * a.page_size + block - 1) / block + 1;
    const int64_t per = (blocks + a.num_splits - 1) / a.num_splits;
    const int64_t pages = per * block / a.page_size + 2;
    return pages < a.max_pages ? pages : a.max_pages;
}

static size_t latent_turn_bytes(const LatentArgs& a, bool tiles, int rows) {
    return a.rot_half ? ((size_t)(tiles ? latent_tokens(rows, a.heads) : 1) * a.rot_half + 4) * sizeof(float2) : 0;
}

template <bool TILES, int HDP, int QT, int NKT, int RW, int KW>
static int launch_latent(const LatentArgs& a, int list, hipStream_t stream) {
    auto kernel = latent_attn_kernel<TILES, HDP, QT, NKT, RW, KW>;
    constexpr size_t bufs = (size_t)KW * 2 * 16 * NKT * HDP * 64;
    constexpr size_t merge = (size_t)(KW - 1) * RW * 64 * QT * (2 + 8 * HDP) * sizeof(float);
    constexpr int rows = RW * QT * 16;
    const size_t table = (size_t)latent_table(a, TILES, 16 * NKT) * sizeof(int) + latent_turn_bytes(a, TILES, rows);
    const size_t lds = bufs + table > merge ? bufs + table : merge;
    if (latent_raise_lds(reinterpret_cast<const void*>(kernel), lds)) return 1;
    const int x = ((TILES ? kTileTokens : 1) * a.heads + rows - 1) / rows;
    LatentArgs args = a;
    if (TILES) {
        const int period = device_compute_units() / x;
        args.deal_period = period > 0 ? period : 1;
        args.num_tiles = list;
    }
    kernel<<<dim3(x, list, TILES ? 1 : a.num_splits), 64 * RW * KW, lds, stream>>>(args);
    ST_LAUNCH_CHECK("latent_attention");
    return 0;
}

template <bool TILES, int ET>
static int launch_latent_f32(const LatentArgs& a, int list, hipStream_t stream) {
    auto kernel = latent_attn_f32_kernel<TILES, ET>;
    const size_t lds = sizeof(float) * ((size_t)kLatentF32Keys * (16 * ET + 4)) + (size_t)latent_table(a, TILES, kLatentF32Keys) * sizeof(int) +
                       latent_turn_bytes(a, TILES, 64);
    if (latent_raise_lds(reinterpret_cast<const void*>(kernel), lds)) return 1;
    const int x = ((TILES ? kTileTokens : 1) * a.heads + 63) / 64;
    LatentArgs args = a;
    if (TILES) {
        const int period = device_compute_units() / x;
        args.deal_period = period > 0 ? period : 1;
        args.num_tiles = list;
    }
    kernel<<<dim3(x, list, TILES ? 1 : a.num_splits), 256, lds, stream>>>(args);
    ST_LAUNCH_CHECK("latent_attention (float)");
    return 0;
}

template <bool TILES>
static int latent_dispatch(const LatentArgs& a, int list, int dtype, hipStream_t stream) {
    if (dtype == kF32) {
        const int et = (a.entry + 15) / 16;
#define ST_LF(E) if (et <= E) return launch_latent_f32<TILES, E>(a, list, stream)
        ST_LF(4); ST_LF(8); ST_LF(10); ST_LF(16); ST_LF(24); ST_LF(36);
#undef ST_LF
        return 1;
    }
    // (an entry runs in the next larger instance, its missing chunks zeros in LDS)
    const int hdp = (a.entry + 31) / 32;
    // tiles: four waves of 16 rows, blocks of 64 keys (32 where entries are large); rows: one or two waves of 16 rows,
    // four (two) shares of the keys, blocks of 32 keys
#define ST_LT(H)                                                                                                       \
    if (hdp <= H) {                                                                                                    \
        if constexpr (TILES) return launch_latent<TILES, H, 1, 4, 4, 1>(a, list, stream);                              \
        else return a.heads <= 16 ? launch_latent<TILES, H, 1, 2, 1, 4>(a, list, stream) : launch_latent<TILES, H, 1, 2, 2, 4>(a, list, stream); \
    }
#define ST_LB(H)                                                                                                       \
    if (hdp <= H) {                                                                                                    \
        if constexpr (TILES) return launch_latent<TILES, H, 1, 2, 4, 1>(a, list, stream);                              \
        else return launch_latent<TILES, H, 1, 2, 1, 2>(a, list, stream);                                                   \
    }
    ST_LT(2) ST_LT(4) ST_LT(5) ST_LT(6) ST_LT(8) ST_LB(12) ST_LB(18)
#undef ST_LT
#undef ST_LB
    return 1;
}

extern "C" int st_latent_max_entry() { return kLatentMaxEntry; }

// Common arguments of both forms: q [tokens, heads, entry] with rows of q_stride elements; cache [pages, page_size, entry];
// out_dim: dims of a result (a multiple of 16, at most entry); rot_off / rot_half / freq / rot_mult: pairs (rot_off + 2i,
// rot_off + 2i + 1), i < rot_half, of every query turn by position * freq[i] (rot_half 0: none; rot_off a multiple of 8);
// sink (or null): a number a head in the denominator.
static int latent_args(LatentArgs& a, const void* q, int64_t q_stride, const void* cache, int64_t page_stride,
                       const int* block_table, const float* sink, const float* freq, int max_pages, int page_size, int heads,
                       int entry, int out_dim, int rot_off, int rot_half, float rot_mult, float scale, int window, int dtype) {
    ST_CHECK(dtype == kBF16 || dtype == kF32, "latent_attention: unknown dtype %d", dtype);
    ST_CHECK(heads > 0 && page_size > 0 && max_pages > 0, "latent_attention: bad sizes");
    ST_CHECK(entry > 0 && entry % 16 == 0 && entry <= kLatentMaxEntry, "latent_attention: entries of up to %d dims in "
             "multiples of 16, not %d", kLatentMaxEntry, entry);
    ST_CHECK(out_dim > 0 && out_dim % 16 == 0 && out_dim <= entry, "latent_attention: %d result dims of an entry of %d", out_dim, entry);
    ST_CHECK(rot_half == 0 || (freq && rot_off >= 0 && rot_off % 8 == 0 && rot_off + 2 * rot_half <= entry),
             "latent_attention: %d turned pairs from dim %d on", rot_half, rot_off);
    ST_CHECK(scale == scale && scale >= -3.0e38f && scale <= 3.0e38f, "latent_attention: the scale must be finite");
    ST_CHECK(q && cache && block_table, "latent_attention: null operand");
    ST_CHECK((((uintptr_t)q | (uintptr_t)cache) & 15) == 0 && q_stride % 8 == 0 && q_stride >= (int64_t)heads * entry &&
             page_stride >= (int64_t)page_size * entry && page_stride % 8 == 0, "latent_attention: rows of queries and pages are "
             "whole and 16-byte aligned");
    a.q = q; a.q_stride = q_stride; a.cache = cache; a.page_stride = page_stride; a.block_table = block_table;
    a.sink = sink; a.freq = freq; a.max_pages = max_pages; a.page_size = page_size; a.heads = heads; a.entry = entry;
    a.out_dim = out_dim; a.rot_off = rot_half ? rot_off : entry; a.rot_half = rot_half; a.rot_mult = rot_mult;
    a.scale = scale; a.window = window > 0 ? window : 0;
    a.page_shift = -1;
    if ((page_size & (page_size - 1)) == 0)
        for (a.page_shift = 0; (1 << a.page_shift) < page_size; ++a.page_shift) {}
    a.num_splits = 1;
    return 0;
}

// Tile i: tokens [tile_q0[i], + 64) of item tile_item[i] (-1: skipped).  out [tokens, heads, out_dim], the storage type.
extern "C" int st_latent_tiles(void* out, const void* q, int64_t q_stride, const void* cache, int64_t page_stride,
                               const int* tile_item, const int* tile_q0, int num_tiles, const int* item_tok_off,
                               const int* item_start, const int* item_len, const int* block_table, const float* sink,
                               const float* freq, int max_pages, int page_size, int heads, int entry, int out_dim, int rot_off,
                               int rot_half, float rot_mult, float scale, int window, int dtype, hipStream_t stream) {
    LatentArgs a = {};
    if (latent_args(a, q, q_stride, cache, page_stride, block_table, sink, freq, max_pages, page_size, heads, entry, out_dim,
                    rot_off, rot_half, rot_mult, scale, window, dtype)) return 1;
    ST_CHECK(num_tiles >= 0 && num_tiles <= 65535, "latent_attention: %d tiles", num_tiles);
    if (num_tiles == 0) return 0;
    ST_CHECK(out && tile_item && tile_q0 && item_tok_off && item_start && item_len && ((uintptr_t)out & 15) == 0, "latent_attention: null operand");
    a.out = out; a.tile_item = tile_item; a.tile_q0 = tile_q0; a.item_tok_off = item_tok_off; a.item_start = item_start;
    a.item_len = item_len;
    return latent_dispatch<true>(a, num_tiles, dtype, stream);
}

// List entry i: batch row row_ids[i] (null: i; -1: skipped).  part_o [list, heads, splits, out_dim], part_lse [list, heads,
// splits]; entries of skipped rows are left as they are.
extern "C" int st_latent_rows(float* part_o, float* part_lse, const void* q, int64_t q_stride, const void* cache,
                              int64_t page_stride, const int* row_ids, const int* token_item, const int* positions, int num_rows,
                              int num_splits, const int* block_table, const float* sink, const float* freq, int max_pages,
                              int page_size, int heads, int entry, int out_dim, int rot_off, int rot_half, float rot_mult,
                              float scale, int window, int dtype, hipStream_t stream) {
    LatentArgs a = {};
    if (latent_args(a, q, q_stride, cache, page_stride, block_table, sink, freq, max_pages, page_size, heads, entry, out_dim,
                    rot_off, rot_half, rot_mult, scale, window, dtype)) return 1;
    ST_CHECK(num_rows >= 0 && num_rows <= 65535 && num_splits >= 1 && num_splits <= 4096, "latent_attention: %d rows, %d splits", num_rows, num_splits);
    if (num_rows == 0) return 0;
    ST_CHECK(part_o && part_lse && token_item && positions && ((uintptr_t)part_o & 15) == 0, "latent_attention: null operand");
    a.part_o = part_o; a.part_lse = part_lse; a.row_ids = row_ids; a.token_item = token_item; a.positions = positions;
    a.num_splits = num_splits;
    return latent_dispatch<false>(a, num_rows, dtype, stream);
}

extern "C" int st_latent_merge(void* out, const float* part_o, const float* part_lse, const int* row_ids, int num_rows, int heads,
                               int out_dim, int num_splits, int dtype, hipStream_t stream) {
    ST_CHECK(num_rows >= 0 && num_rows <= 65535 && heads > 0 && out_dim > 0 && num_splits >= 1, "latent_merge: bad sizes");
    if (num_rows == 0) return 0;
    ST_CHECK(out && part_o && part_lse, "latent_merge: null operand");
    const dim3 grid(heads, num_rows);
    if (dtype == kF32) latent_merge_kernel<float><<<grid, 64, 0, stream>>>((float*)out, part_o, part_lse, row_ids, heads, out_dim, num_splits);
    else if (dtype == kBF16) latent_merge_kernel<bf16_t><<<grid, 64, 0, stream>>>((bf16_t*)out, part_o, part_lse, row_ids, heads, out_dim, num_splits);
    else ST_CHECK(false, "latent_merge: unknown dtype %d", dtype);
    ST_LAUNCH_CHECK("latent_merge");
    return 0;
}

// y [tokens, heads, value_dim] = sigmoid(gate) * W o (gate null: W o); w [heads, value_dim, out_dim]; gate: float rows of
// gate_stride with [heads, value_dim] logits.  o [tokens, heads, out_dim] in the storage type, or (o null) the partial
// results of st_latent_rows for all tokens in order (rows of negative token_item are left as they are).
extern "C" int st_latent_up(void* y, const void* o, const float* part_o, const float* part_lse, int num_splits, const void* w,
                            const float* gate, int64_t gate_stride, const int* token_item, int num_tokens, int heads,
                            int value_dim, int out_dim, int dtype, hipStream_t stream) {
    ST_CHECK(dtype == kBF16 || dtype == kF32, "latent_up: unknown dtype %d", dtype);
    ST_CHECK(num_tokens >= 0 && heads > 0 && heads <= 65535 && value_dim > 0 && out_dim > 0 && out_dim % 16 == 0 && out_dim <= kLatentMaxEntry,
             "latent_up: bad sizes");
    if (num_tokens == 0) return 0;
    ST_CHECK(y && w && ((uintptr_t)w & 15) == 0 && (o || (part_o && part_lse && token_item && num_splits >= 1)), "latent_up: null operand");
    ST_CHECK(!gate || gate_stride >= (int64_t)heads * value_dim, "latent_up: the gate has a logit a value");
    if (!o) {
        ST_CHECK(num_tokens <= 65535, "latent_up: %d decoded tokens", num_tokens);
        const size_t lds = sizeof(float) * ((size_t)out_dim + num_splits);
        const dim3 grid(heads, num_tokens);
        if (dtype == kF32)
            latent_up_rows_kernel<float><<<grid, 256, lds, stream>>>((float*)y, part_o, part_lse, (const float*)w, gate, gate_stride, token_item, heads, value_dim, out_dim, num_splits);
        else
            latent_up_rows_kernel<bf16_t><<<grid, 256, lds, stream>>>((bf16_t*)y, part_o, part_lse, (const bf16_t*)w, gate, gate_stride, token_item, heads, value_dim, out_dim, num_splits);
        ST_LAUNCH_CHECK("latent_up (rows)");
        return 0;
    }
    ST_CHECK(((uintptr_t)o & 15) == 0, "latent_up: rows are 16-byte aligned");
    const dim3 grid((num_tokens + 63) / 64, heads);
#define ST_LU(T, S) latent_up_kernel<T, S><<<grid, 256, 0, stream>>>((T*)y, (const T*)o, (const T*)w, gate, gate_stride, num_tokens, heads, value_dim, out_dim)
    if (dtype == kF32) {
        const int s = (out_dim + 15) / 16;
        if (s <= 4) ST_LU(float, 4); else if (s <= 8) ST_LU(float, 8); else if (s <= 16) ST_LU(float, 16); else ST_LU(float, 36);
    } else {
        const int s = (out_dim + 31) / 32;
        if (s <= 2) ST_LU(bf16_t, 2); else if (s <= 4) ST_LU(bf16_t, 4); else if (s <= 8) ST_LU(bf16_t, 8); else ST_LU(bf16_t, 18);
    }
#undef ST_LU
    ST_LAUNCH_CHECK("latent_up");
    return 0;
}
