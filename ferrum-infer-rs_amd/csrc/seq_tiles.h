// Row tiles of a batch's sequences and rotation of interleaved pairs: what the attention kernels share.
#pragma once
#include "common.h"
#include "layer_ops.h"

namespace fh {

// cosines and sines of the four pairs (2i, 2i + 1) starting at dimension d0, position `pos`; pairs past rot_dims pass unchanged
struct Rot4 { float c[4], s[4]; };
__device__ __forceinline__ Rot4 rot_load(int d0, int rot_dims, const float* __restrict__ cos_t, const float* __restrict__ sin_t, long pos) {
    const int half = rot_dims >> 1;
    Rot4 r;
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const int i = (d0 >> 1) + j;
        r.c[j] = 1.f;
        r.s[j] = 0.f;
        if (half > 0) {                                  // (uniform; the loads themselves are unconditional, clamped)
            const long o = pos * half + (i < half ? i : half - 1);
            const float cv = cos_t[o], sv = sin_t[o];
            r.c[j] = i < half ? cv : 1.f;
            r.s[j] = i < half ? sv : 0.f;
        }
    }
    return r;
}
template <typename V>
__device__ __forceinline__ V rot_apply(V x, const Rot4& r) {
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const float u = (float)x[2 * j], w = (float)x[2 * j + 1];
        x[2 * j] = u * r.c[j] - w * r.s[j];
        x[2 * j + 1] = w * r.c[j] + u * r.s[j];
    }
    return x;
}

struct SeqTile { int seq, tile, tok0, q_len, pos0; };
__device__ __forceinline__ int seq_row_tiles(const BatchView& v, int q_len, int heads, int rows) {
    return v.long_min > 0 && q_len >= v.long_min ? 0 : (q_len * heads + rows - 1) / rows;
}
// tiles of `rows` (16 or 32) (token, head) pairs, numbered sequence by sequence; every wave finds tile w by a scan of cu_seqlens
__device__ __forceinline__ bool find_seq_tile(const BatchView& v, int heads, int rows, int w, SeqTile* o) {
    if (v.single) {
        const int per = (heads + rows - 1) / rows;
        o->seq = w / per; o->tile = w % per; o->tok0 = o->seq; o->q_len = 1;
        if (o->seq >= v.num_seqs) return false;
        o->pos0 = (int)v.pos[o->seq];
        return true;
    }
    const int lane = threadIdx.x & 63;
    int base = 0;
    for (int s0 = 0; s0 < v.num_seqs; s0 += 64) {
        const int s = s0 + lane;
        const int units = s < v.num_seqs ? seq_row_tiles(v, (int)(v.cu[s + 1] - v.cu[s]), heads, rows) : 0;
        int incl = units;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const int t = __shfl_up(incl, off, 64);
            if (lane >= off) incl += t;
        }
        const int total = __builtin_amdgcn_readlane(incl, 63);       // (uniform, and with it everything found)
        if (w < base + total) {
            const int src = __ffsll((unsigned long long)__ballot(w < base + incl)) - 1;
            o->seq = __builtin_amdgcn_readfirstlane(s0 + src);
            o->tile = __builtin_amdgcn_readfirstlane(w - (base + __shfl(incl - units, src, 64)));
            o->tok0 = (int)v.cu[o->seq];
            o->q_len = (int)v.cu[o->seq + 1] - o->tok0;
            o->pos0 = (int)v.pos[o->seq];
            return true;
        }
        base += total;
    }
    return false;
}

// The same tiles with the last ones of every sequence, which see the most keys, first: tile w is the k-th from the end of some sequence, for k = 0,
// then 1, and so on, so that long and short ones fill the chip evenly.
__device__ __forceinline__ bool find_seq_tile_last_first(const BatchView& v, int heads, int rows, int w, SeqTile* o) {
    const int lane = threadIdx.x & 63;
    auto tiles = [&](int s) { return s < v.num_seqs ? seq_row_tiles(v, v.single ? 1 : (int)(v.cu[s + 1] - v.cu[s]), heads, rows) : 0; };
    const int own = tiles(lane);
    // tiles among the last k of their sequence (counts are exact in fp32)
    auto among = [&](int k) {
        float n = (float)min(own, k);
        for (int s = lane + 64; s < v.num_seqs; s += 64) n += (float)min(tiles(s), k);
        return __builtin_amdgcn_readfirstlane((int)wave_reduce_sum(n));
    };
    float most = (float)own;
    for (int s = lane + 64; s < v.num_seqs; s += 64) most = fmaxf(most, (float)tiles(s));
    int lo = 0, hi = __builtin_amdgcn_readfirstlane((int)wave_reduce_max(most));       // among(lo) ≤ w < among(hi)
    if (w >= among(hi)) return false;
    while (hi - lo > 1) {
        const int mid = (lo + hi) / 2;
        if (among(mid) <= w) lo = mid; else hi = mid;
    }
    int rank = w - among(lo);                                                           // among the sequences of more than lo tiles
    for (int s0 = 0; s0 < v.num_seqs; s0 += 64) {
        const int n = s0 ? tiles(s0 + lane) : own;
        const unsigned long long more = __ballot(n > lo);
        const int here = __popcll(more);
        if (rank < here) {
            const bool it = n > lo && __popcll(more & ((1ull << lane) - 1)) == rank;
            const int src = __ffsll((unsigned long long)__ballot(it)) - 1;
            o->seq = s0 + src;
            o->tile = __builtin_amdgcn_readlane(n, src) - 1 - lo;
            o->tok0 = (int)v.cu[o->seq];
            o->q_len = (int)v.cu[o->seq + 1] - o->tok0;
            o->pos0 = (int)v.pos[o->seq];
            return true;
        }
        rank -= here;
    }
    return false;
}

}  // namespace fh
