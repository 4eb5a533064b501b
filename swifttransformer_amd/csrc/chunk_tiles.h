// Pieces of the recurrences that go by chunks of rows: which rows a chunk has, and tiles of rows on their way to LDS.
#pragma once

#include "common.h"

namespace st {

constexpr int kChunkRows = 64;       // counted from an item's first row of the step

// the chunk of an item that a global chunk index means; false past the last one
__device__ inline bool find_chunk(int idx, const int* __restrict__ item_len, const int* __restrict__ item_slot,
                                         int num_items, int& item, int& chunk) {
    int base = 0;
    for (int b = 0; b < num_items; ++b) {
        const int len = item_len[b];
        const int n = (item_slot[b] >= 0 && len > 0) ? (len + kChunkRows - 1) / kChunkRows : 0;
        if (idx < base + n) {
            item = b;
            chunk = idx - base;
            return true;
        }
        base += n;
    }
    return false;
}

// Four neighbouring floats of a row, zeros past its `limit` numbers or where the row does not exist.  VEC: the row starts
// on 16 bytes and the limit is a multiple of 4.  (Addresses are clamped and values cleared rather than loads behind a
// branch: the loads of a tile are then all on their way at once.)
template <bool VEC>
__device__ inline float4 load_piece(const float* __restrict__ row, int c, int limit, bool ok) {
    float4 v;
    if (VEC) {
        v = *reinterpret_cast<const float4*>(row + min(c, limit - 4));
    } else {
        v.x = row[min(c, limit - 1)];
        v.y = row[min(c + 1, limit - 1)];
        v.z = row[min(c + 2, limit - 1)];
        v.w = row[min(c + 3, limit - 1)];
    }
    v.x = ok && c < limit ? v.x : 0.f;
    v.y = ok && c + 1 < limit ? v.y : 0.f;
    v.z = ok && c + 2 < limit ? v.z : 0.f;
    v.w = ok && c + 3 < limit ? v.w : 0.f;
    return v;
}

// A tile of 64 rows x 4 * P4 floats (P4 a power of two) by 256 threads: piece i of a thread is row e / P4, floats 4 (e % P4)
// on, e = thread + 256 i; P4 / 4 pieces a thread.
template <int P4>
struct Tile {
    static constexpr int kPieces = P4 / 4;
    float4 v[kPieces];
    template <bool VEC>
    __device__ inline void load(const float* __restrict__ base, int64_t stride, int rows, int first, int limit) {
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int e = threadIdx.x + 256 * i, j = e / P4, c = 4 * (e % P4);
            v[i] = load_piece<VEC>(base + (int64_t)min(j, rows - 1) * stride, first + c, limit, j < rows);
        }
    }
    __device__ inline void store(float* lds, int lds_stride) const {
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int e = threadIdx.x + 256 * i;
            *reinterpret_cast<float4*>(lds + (e / P4) * lds_stride + 4 * (e % P4)) = v[i];
        }
    }
    __device__ inline void store_weighted(float* lds, int lds_stride, const float* w) const {
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int e = threadIdx.x + 256 * i;
            const float f = w[e / P4];
            *reinterpret_cast<float4*>(lds + (e / P4) * lds_stride + 4 * (e % P4)) = make_float4(v[i].x * f, v[i].y * f, v[i].z * f, v[i].w * f);
        }
    }
};

}  // namespace st
