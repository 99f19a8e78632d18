// Dense projections of the layered models (tiled_gemm.h): one kernel for few rows (K split over the waves of a workgroup, summed in
// LDS, no second launch) and one for prompts (128 × 128 tiles, both operands copied to LDS as fragments by the load unit itself).
// Every activation, bias and per-row factor of a projection is applied to the fp32 accumulator in the epilogue.
#include <algorithm>

#include "common.h"
#include "knobs.h"
#include "tiled_gemm.h"

namespace fh {

template <typename E, bool RARE = false>
__device__ __forceinline__ float gemm_act(const GemmSection& sec, float v) {
    if (sec.act == GEMM_ACT_SIGMOID) return ActMath<E>::sigmoid(v);
    if (sec.act == GEMM_ACT_GELU_TANH) return gelu_tanh_f32<E>(v);
    if (sec.act == GEMM_ACT_XIELU) return xielu_f32<E>(v, sec.p, sec.q);
    if (sec.act == GEMM_ACT_RELU2) { v = fmaxf(v, 0.f); return v * v; }
    if (sec.act == GEMM_ACT_SILU) return v * ActMath<E>::sigmoid(v);
    if (RARE && sec.act == GEMM_ACT_SOFTPLUS) return softplus_f32<E>(v);
    if (RARE && sec.act == GEMM_ACT_LOG_SIGMOID) return sec.p * log_sigmoid_f32<E>(v);
    if (RARE && sec.act == GEMM_ACT_SOFTCAP) return sec.p * ActMath<E>::tanh(v / sec.p);
    return v;
}
// output row of place r, −1: none
template <typename E>
__device__ __forceinline__ int gemm_out_row(const TiledGemm<E>& p, int r) {
    if (p.rows.id) r = p.rows.id[r];
    return r < p.m ? r : -1;
}
template <typename E>
__device__ __forceinline__ void gemm_store(const TiledGemm<E>& p, int g, int row, int col, float v) {
    if (p.row_scale) v *= (float)p.row_scale[row * p.ld_scale + g];
    if (p.col_scale) v *= (float)p.col_scale[p.col_scale_row[row] * p.ld_col_scale + col];
    const long o = row * p.ldo + (p.rows.id ? 0 : g * p.out_group) + col;
    if (p.out_f32) p.out_f32[o] = v; else p.out[o] = (E)v;
}
template <typename E, bool RARE>
__device__ __forceinline__ void gemm_epilogue(const TiledGemm<E>& p, const GemmSection& sec, int g, int place, int col, float v) {
    const int row = gemm_out_row(p, place);
    if (row < 0 || col >= p.n_store) return;
    v *= sec.mul;
    if (p.bias) v += p.bias[(long)g * p.n + col];
    gemm_store(p, g, row, col, gemm_act<E, RARE>(sec, v));
}
template <typename E>
__device__ __forceinline__ float gemm_glu(const GemmSection& sec, float gate, float up) {
    if (sec.act == GEMM_ACT_SILU_GLU) return gate * ActMath<E>::sigmoid(gate) * up;
    if (sec.act == GEMM_ACT_GELU_GLU) return gelu_tanh_f32<E>(gate) * up;
    return clamped_glu_f32<E>(gate, up, sec.p, sec.q);
}
// accumulators of a (gate, up) pair of tiles; col: the gate's column
template <typename E>
__device__ __forceinline__ float gemm_gated(const TiledGemm<E>& p, const GemmSection& sec, int col, float gate, float up) {
    gate *= sec.mul;
    up *= sec.mul;
    if (p.bias) { gate += p.bias[col]; up += p.bias[col + 16]; }
    return gemm_glu<E>(sec, gate, up);
}
__device__ __forceinline__ int gemm_gated_col(const GemmSection& sec, int col) { return sec.begin + ((col - sec.begin) >> 5) * 16 + (col & 15); }
template <typename E>
__device__ __forceinline__ GemmSection gemm_section(const TiledGemm<E>& p, int col) {
    GemmSection s = {0, GEMM_ACT_NONE, 0.f, 0.f, 1.f};
#pragma unroll
    for (int i = 0; i < GEMM_MAX_SECTIONS; i++)
        if (i < p.nsec && col >= p.sec[i].begin) s = p.sec[i];
    return s;
}

// address of lane (a, b)'s 8 values of row tile t at k-step 0, and the distance between k-steps
template <typename E>
__device__ __forceinline__ const E* gemm_row(const TiledGemm<E>& p, int t, int g, int a, int b) {
    if (p.x_blocks) {
        const int tiles = (p.m + 15) >> 4;
        return p.x + (long)p.x_blocks[t < tiles ? t : tiles - 1] * p.x_block_elems + (a * 16 + b) * 8;
    }
    int r = t * 16 + b;
    if (p.rows.id) {
        r = p.rows.id[r];
        return p.x + (long)((unsigned)(r < p.m ? r : p.m - 1) / (unsigned)p.rows.div) * p.ldx + 8 * a;
    }
    return p.x + (long)(r < p.m ? r : p.m - 1) * p.ldx + g * p.x_group + 8 * a;
}
template <typename E>
__device__ __forceinline__ int gemm_row_step(const TiledGemm<E>& p) { return p.x_blocks ? 512 : 32; }

// grid (column blocks, row blocks, groups or K slabs); NW waves = (NW / kw) column groups × kw parts of K.  Two register buffers of U
// k-steps: the next one is requested before the current one is multiplied; loads past the part's end repeat its last k-step.
// EXT: with sorted rows, column factors, gated sections or rare activations (each is a branch on the latency-bound path of the launches without).
template <typename E, int MT, int J, bool EXT>
__global__ __launch_bounds__(512) void tiled_gemm_kernel(TiledGemm<E> p, int kw) {
    typedef typename Frag<E>::v8 v8;
    if (!EXT) { p.rows.id = nullptr; p.col_scale = nullptr; }
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    floatx4* red = reinterpret_cast<floatx4*>(smem);            // [NW][MT·J][64]
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int a = lane >> 4, b = lane & 15;
    const int cw = (blockDim.x >> 6) / kw, part = wave % kw, cg = wave / kw;
    const int n0 = (blockIdx.x * cw + cg) * 16 * J, rb = blockIdx.y;
    const int z = p.slabs > 1 ? blockIdx.z : 0;
    int g = p.slabs > 1 ? 0 : blockIdx.z;
    if (p.rows.id) {
        if (rb * 16 * MT >= *p.rows.total) return;
        g = p.rows.group[rb];
    }
    const int ksteps = p.k >> 5, parts = kw * p.slabs, mine = z * kw + part;
    const bool live = n0 < p.n;
    const int s0 = live ? ksteps * mine / parts : 0, s1 = live ? ksteps * (mine + 1) / parts : 0;
    const E* xrow[MT];
    const int xs = gemm_row_step(p);
#pragma unroll
    for (int mt = 0; mt < MT; mt++) xrow[mt] = gemm_row(p, rb * MT + mt, g, a, b);
    const E* wt = p.w + ((long)g * (p.n >> 4) + (live ? n0 >> 4 : 0)) * ksteps * 512 + lane * 8;
    floatx4 acc[MT][J];
#pragma unroll
    for (int mt = 0; mt < MT; mt++)
#pragma unroll
        for (int j = 0; j < J; j++) acc[mt][j] = (floatx4){0.f, 0.f, 0.f, 0.f};
    constexpr int U = sizeof(E) == 2 ? (MT * J == 1 ? 8 : 4) : 1;
    v8 bw[2][U][J], ax[2][U][MT];
    auto load = [&](v8 (&bq)[U][J], v8 (&aq)[U][MT], int s) {
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int ss = min(s + u, s1 - 1);
#pragma unroll
            for (int j = 0; j < J; j++) bq[u][j] = __builtin_nontemporal_load(reinterpret_cast<const v8*>(wt + ((long)j * ksteps + ss) * 512));
#pragma unroll
            for (int mt = 0; mt < MT; mt++) aq[u][mt] = *reinterpret_cast<const v8*>(xrow[mt] + (long)ss * xs);
        }
    };
    auto mul = [&](v8 (&bq)[U][J], v8 (&aq)[U][MT], int s) {
#pragma unroll
        for (int u = 0; u < U; u++)
            if (s + u < s1) {
#pragma unroll
                for (int j = 0; j < J; j++)
#pragma unroll
                    for (int mt = 0; mt < MT; mt++) acc[mt][j] = Frag<E>::mma(aq[u][mt], bq[u][j], acc[mt][j]);
            }
    };
    // every buffer is requested in the block that multiplies the other one, so each wait counts exactly the loads it needs
    if (s0 < s1) {
        int s = s0;
        load(bw[0], ax[0], s);
        while (true) {
            if (s + U >= s1) { mul(bw[0], ax[0], s); break; }
            load(bw[1], ax[1], s + U);
            mul(bw[0], ax[0], s);
            s += U;
            if (s + U >= s1) { mul(bw[1], ax[1], s); break; }
            load(bw[0], ax[0], s + U);
            mul(bw[1], ax[1], s);
            s += U;
        }
    }
    if (p.slabs > 1) p.out_f32 += z * p.slab_stride;
    const GemmSection sec = gemm_section(p, n0);
    const bool gated = EXT && J == 2 && gemm_gated_act(sec.act);
    if (kw == 1) {
        if (!live) return;
        if constexpr (J == 2)
            if (gated) {
#pragma unroll
                for (int mt = 0; mt < MT; mt++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const int row = gemm_out_row(p, (rb * MT + mt) * 16 + 4 * a + r);
                        if (row >= 0) gemm_store(p, g, row, gemm_gated_col(sec, n0 + b), gemm_gated(p, sec, n0 + b, acc[mt][0][r], acc[mt][J - 1][r]));
                    }
                return;
            }
#pragma unroll
        for (int mt = 0; mt < MT; mt++)
#pragma unroll
            for (int j = 0; j < J; j++)
#pragma unroll
                for (int r = 0; r < 4; r++) gemm_epilogue<E, EXT>(p, sec, g, (rb * MT + mt) * 16 + 4 * a + r, n0 + 16 * j + b, acc[mt][j][r]);
        return;
    }
#pragma unroll
    for (int mt = 0; mt < MT; mt++)
#pragma unroll
        for (int j = 0; j < J; j++) red[(wave * MT * J + mt * J + j) * 64 + lane] = acc[mt][j];
    __syncthreads();
    if (!live) return;
    auto summed = [&](int t) {
        floatx4 v = red[(cg * kw * MT * J + t) * 64 + lane];
        for (int q = 1; q < kw; q++) v += red[((cg * kw + q) * MT * J + t) * 64 + lane];
        return v;
    };
    if (gated) {
        for (int mt = part; mt < MT; mt += kw) {
            const floatx4 gate = summed(mt * J), up = summed(mt * J + 1);
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int row = gemm_out_row(p, (rb * MT + mt) * 16 + 4 * a + r);
                if (row >= 0) gemm_store(p, g, row, gemm_gated_col(sec, n0 + b), gemm_gated(p, sec, n0 + b, gate[r], up[r]));
            }
        }
        return;
    }
    // tile t of the column group is summed (in the order of the K parts) and finished by part t mod kw
    for (int t = part; t < MT * J; t += kw) {
        const floatx4 v = summed(t);
        const int mt = t / J, j = t % J;
#pragma unroll
        for (int r = 0; r < 4; r++) gemm_epilogue<E, EXT>(p, sec, g, (rb * MT + mt) * 16 + 4 * a + r, n0 + 16 * j + b, v[r]);
    }
}

// Prompts, 16-bit: WM × WN waves hold MI × NJ tiles of 16 × 16 each, 64 of K per stage, a ring of S stages.  A fragment (16 rows × 32 of K, or 16
// columns × 32 of K) is one 1-KiB load straight into LDS in lane order, read back as one conflict-free ds_read_b128.
__device__ const bf16 zero_fragment[512] = {};
template <int WM, int WN, int MI, int NJ, int S>
struct BigTile {
    static constexpr int WAVES = WM * WN, RT = WM * MI, CT = WN * NJ, ROWS = 16 * RT, COLS = 16 * CT, FRAGS = 2 * (RT + CT);
    static constexpr size_t LDS = (size_t)S * FRAGS * 1024;
    static_assert(RT % WAVES == 0 && CT % WAVES == 0 && MI % 2 == 0 && NJ == 4, "every wave copies whole tiles");
    static_assert(LDS >= (size_t)WAVES * 32 * 68 * 4, "the epilogue's rows fit the stages");
};
template <int WM, int WN, int MI, int NJ, int S>
__global__ __launch_bounds__(64 * WM * WN, 2) void tiled_gemm_big_kernel(TiledGemm<bf16> p, int mtiles, int ntiles) {
    typedef BigTile<WM, WN, MI, NJ, S> T;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    bf16* lds = reinterpret_cast<bf16*>(smem);                          // per stage: A fragments, then B fragments
    constexpr int STAGE = T::FRAGS * 512, AT = T::RT / T::WAVES, BT = T::CT / T::WAVES;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int a = lane >> 4, b = lane & 15;
    // workgroups go round-robin over 8 XCDs: give each XCD a contiguous run of tiles, and walk 8 row tiles per column tile
    if (p.rows.id) mtiles = *p.rows.total / T::ROWS;
    const int total = mtiles * ntiles, l = blockIdx.x;
    if (l >= total) return;
    const int q8 = total / 8, r8 = total % 8, xcd = l % 8;
    const int id = (xcd < r8 ? xcd * (q8 + 1) : r8 * (q8 + 1) + (xcd - r8) * q8) + l / 8;
    const int band = id / (8 * ntiles), rows_in = min(8, mtiles - band * 8), in = id - band * 8 * ntiles;
    const int mt = band * 8 + in % rows_in, m0 = mt * T::ROWS, n0 = (in / rows_in) * T::COLS;
    const int ksteps = p.k >> 5, ntl = p.n >> 4, g = p.rows.id ? p.rows.group[mt] : blockIdx.z;
    const int wm = wave / WN, wn = wave % WN;
    // this wave's fragments of a stage: AT row tiles and BT column tiles, two k-steps each
    const bf16 *ap[AT], *bp[BT];
#pragma unroll
    for (int i = 0; i < AT; i++) ap[i] = gemm_row(p, (m0 >> 4) + AT * wave + i, g, a, b);
#pragma unroll
    for (int i = 0; i < BT; i++) {
        const int t = (n0 >> 4) + BT * wave + i;
        bp[i] = p.w + ((long)g * ntl + (t < ntl ? t : ntl - 1)) * ksteps * 512 + lane * 8;
    }
    const int xs = gemm_row_step(p);
#define BIG_COPY(src, dst) __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src), (__attribute__((address_space(3))) void*)(dst), 16, 0, 0)
    auto issue = [&](int st, int ks) {
#pragma unroll
        for (int h = 0; h < 2; h++) {
            const int kk = ks + h < ksteps ? ks + h : ksteps - 1;         // (past the end of an odd count: rows of zeros)
#pragma unroll
            for (int i = 0; i < AT; i++) BIG_COPY(ks + h < ksteps ? ap[i] + (long)kk * xs : zero_fragment + lane * 8, lds + st * STAGE + ((AT * wave + i) * 2 + h) * 512);
#pragma unroll
            for (int i = 0; i < BT; i++) BIG_COPY(bp[i] + (long)kk * 512, lds + st * STAGE + ((T::RT + BT * wave + i) * 2 + h) * 512);
        }
    };
#undef BIG_COPY
    floatx4 acc[MI][NJ];
#pragma unroll
    for (int i = 0; i < MI; i++)
#pragma unroll
        for (int j = 0; j < NJ; j++) acc[i][j] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < S - 1; i++)
        if (2 * i < ksteps) issue(i, 2 * i);
    auto multiply = [&](const bf16* la, const bf16* lb, int h) {
        bf16x8 af[MI], bf[NJ];
#pragma unroll
        for (int j = 0; j < NJ; j++) bf[j] = *reinterpret_cast<const bf16x8*>(lb + (j * 2 + h) * 512);
#pragma unroll
        for (int i = 0; i < MI; i++) af[i] = *reinterpret_cast<const bf16x8*>(la + (i * 2 + h) * 512);
#pragma unroll
        for (int i = 0; i < MI; i++)
#pragma unroll
            for (int j = 0; j < NJ; j++) acc[i][j] = Frag<bf16>::mma(af[i], bf[j], acc[i][j]);
    };
    int st = 0;
    for (int ks = 0; ks < ksteps; ks += 2) {
        // this stage has arrived (the S − 2 after it may be on their way) and every wave is done with the one before it, whose place the
        // next request takes
        if (S > 2 && ks + 2 * (S - 2) < ksteps) asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"((S - 2) * 2 * (AT + BT)) : "memory");
        else asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
        if (ks + 2 * (S - 1) < ksteps) issue(st ? st - 1 : S - 1, ks + 2 * (S - 1));
        const bf16 *la = lds + st * STAGE + wm * MI * 1024 + lane * 8, *lb = lds + st * STAGE + (T::RT + wn * NJ) * 1024 + lane * 8;
        multiply(la, lb, 0);
        multiply(la, lb, 1);
        // operands a few MFMAs ahead of their use
        constexpr int AHEAD = NJ + 2, LEFT = 2 * (MI + NJ) - AHEAD, PER = 2 * MI * NJ / (LEFT + 2);
        __builtin_amdgcn_sched_group_barrier(0x100, AHEAD, 0);
#pragma unroll
        for (int i = 0; i < LEFT; i++) {
            __builtin_amdgcn_sched_group_barrier(0x008, PER, 0);
            __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
        }
        __builtin_amdgcn_sched_group_barrier(0x008, 2 * MI * NJ - LEFT * PER, 0);
        st = st + 1 < S ? st + 1 : 0;
    }
    __syncthreads();
    // epilogue: 32 rows of a wave's accumulators at a time through LDS (the stages are free, the rows its own, LDS operations of a wave
    // complete in order), then a lane finishes 8 columns of a row: bias, activation and factors, and rows leave in 16-byte pieces.  In a
    // gated section the lanes of the up tiles have nothing to do, those of the gate tiles read both.
    float* lf = reinterpret_cast<float*>(smem) + wave * 32 * 68;
    const int cl = (lane & 7) * 8, col = n0 + wn * 64 + cl;
    const GemmSection sec = gemm_section(p, min(col, p.n - 1));
    const bool gated = gemm_gated_act(sec.act), vec = p.n_store % 8 == 0 && p.ldo % 8 == 0 && p.out_group % 8 == 0;
    const bool active = gated ? col < p.n && !(col & 16) : col < p.n_store;
    const int oc = gated ? gemm_gated_col(sec, col) : col;
    float bias[8], bias_up[8];
#pragma unroll
    for (int e = 0; e < 8; e++) {
        bias[e] = p.bias && active ? p.bias[(long)g * p.n + col + e] : 0.f;
        bias_up[e] = p.bias && active && gated ? p.bias[(long)g * p.n + col + 16 + e] : 0.f;
    }
#pragma unroll
    for (int ch = 0; ch < MI / 2; ch++) {
#pragma unroll
        for (int i = 0; i < 2; i++)
#pragma unroll
            for (int j = 0; j < NJ; j++)
#pragma unroll
                for (int r = 0; r < 4; r++) lf[(i * 16 + 4 * a + r) * 68 + j * 16 + b] = acc[2 * ch + i][j][r];
        const int row0 = m0 + (wm * MI + 2 * ch) * 16;
#pragma unroll 1
        for (int q = 0; q < 4; q++) {
            const int row = q * 8 + (lane >> 3), gr = gemm_out_row(p, row0 + row);
            if (gr < 0 || !active) continue;
            float v[8];
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = lf[row * 68 + cl + e] * sec.mul + bias[e];
            if (gated) {
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = gemm_glu<bf16>(sec, v[e], lf[row * 68 + cl + 16 + e] * sec.mul + bias_up[e]);
            } else if (sec.act != GEMM_ACT_NONE) {
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = gemm_act<bf16, true>(sec, v[e]);
            }
            if (!vec) {
                for (int e = 0; e < 8; e++)
                    if (gated || col + e < p.n_store) gemm_store(p, g, gr, oc + e, v[e]);
                continue;
            }
            if (p.row_scale) {
                const float f = (float)p.row_scale[gr * p.ld_scale + g];
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] *= f;
            }
            if (p.col_scale) {
                const bf16x8 f = *reinterpret_cast<const bf16x8*>(p.col_scale + p.col_scale_row[gr] * p.ld_col_scale + oc);
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] *= (float)f[e];
            }
            const long o = gr * p.ldo + (p.rows.id ? 0 : g * p.out_group) + oc;
            if (p.out_f32) {
                *reinterpret_cast<floatx4*>(p.out_f32 + o) = (floatx4){v[0], v[1], v[2], v[3]};
                *reinterpret_cast<floatx4*>(p.out_f32 + o + 4) = (floatx4){v[4], v[5], v[6], v[7]};
            } else {
                bf16x8 y;
#pragma unroll
                for (int e = 0; e < 8; e++) y[e] = (bf16)v[e];
                *reinterpret_cast<bf16x8*>(p.out + o) = y;
            }
        }
    }
}

template <int WM, int WN, int MI, int NJ, int S>
static int launch_big(const TiledGemm<bf16>& g, hipStream_t s) {
    typedef BigTile<WM, WN, MI, NJ, S> T;
    static bool attr = false;
    if (!attr) {
        FH_CHECK_HIP(hipFuncSetAttribute((const void*)tiled_gemm_big_kernel<WM, WN, MI, NJ, S>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)T::LDS));
        attr = true;
    }
    const int mtiles = g.rows.id ? g.rows.max_blocks : cdiv(g.m, T::ROWS), ntiles = cdiv(g.n, T::COLS);
    form_hit(g.rows.id ? FORM_TILED_GEMM_GROUPED_BIG : FORM_TILED_GEMM_BIG);
    if (T::ROWS == 256) form_hit(FORM_TILED_GEMM_256);
    hipLaunchKernelGGL((tiled_gemm_big_kernel<WM, WN, MI, NJ, S>), dim3(mtiles * ntiles, 1, g.groups), dim3(64 * T::WAVES), T::LDS, s, g, mtiles, ntiles);
    FH_CHECK_LAUNCH();
    return 0;
}
static int launch_big(const TiledGemm<bf16>& g, hipStream_t s) {
    // one 256 × 256 tile per CU, or two of 128 × 128: the large one halves the bytes per product, as long as there are enough of them
    const long tiles = (long)cdiv(g.m, 256) * cdiv(g.n, 256) * g.groups;
    // (few stages: the epilogues are most of the work, and two workgroups per CU hide one's behind the other's)
    const bool wide = g.rows.id ? g.rows.block == 256 : tiles >= knobs().tiled_wide_min_tiles && g.k >= knobs().tiled_wide_min_k;
    if (wide) return launch_big<2, 4, 8, 4, 2>(g, s);
    // few tiles: rows in halves so that every CU has one, or one workgroup per CU, and a deeper ring in place of the second workgroup
    const long tiles128 = (long)cdiv(g.m, 128) * cdiv(g.n, 128) * g.groups;
    if (!g.rows.id && tiles128 <= knobs().tiled_half_max_tiles) return launch_big<2, 2, 2, 4, 5>(g, s);
    return !g.rows.id && tiles128 <= 256 ? launch_big<2, 2, 4, 4, 4>(g, s) : launch_big<2, 2, 4, 4, 2>(g, s);
}
static int launch_big(const TiledGemm<float>&, hipStream_t) { return 2; }      // (never taken: 16-bit only)

int tiled_gemm_slabs(int m, int n, int k) {
    if (m > 64) return 1;
    // narrow outputs: enough (column group, K part) workgroups to cover the chip, two k-steps or more per wave
    int S = 1;
    while (S < GEMM_MAX_SLABS && (n / 32) * S < 256 && k / 32 >= 2 * 8 * 2 * S) S *= 2;
    return S;
}

template <typename E, int MT, int J, bool EXT>
static int launch_small(const TiledGemm<E>& g, dim3 grid, int nw, int kw, hipStream_t s) {
    const size_t lds = kw == 1 ? 0 : (size_t)nw * MT * J * 1024;
    hipLaunchKernelGGL((tiled_gemm_kernel<E, MT, J, EXT>), grid, dim3(64 * nw), lds, s, g, kw);
    FH_CHECK_LAUNCH();
    return 0;
}

template <typename E>
int tiled_gemm(const TiledGemm<E>& gin, hipStream_t s) {
    TiledGemm<E> g = gin;
    if (g.m <= 0) return 0;
    if (!g.n_store) g.n_store = g.n;
    FH_REQUIRE(g.n > 0 && g.k > 0 && g.n % 32 == 0 && g.k % 32 == 0, "tiled_gemm: n=%d k=%d must be multiples of 32", g.n, g.k);
    FH_REQUIRE(g.ldx % 8 == 0 && g.x_group % 8 == 0 && g.n_store <= g.n && g.groups >= 1, "tiled_gemm: ldx=%ld group stride=%ld", g.ldx, g.x_group);
    FH_REQUIRE((g.out != nullptr) != (g.out_f32 != nullptr), "tiled_gemm: exactly one output");
    FH_REQUIRE(g.slabs == 1 || (g.groups == 1 && g.out_f32 && !g.bias && !g.nsec && !g.row_scale), "tiled_gemm: slabs are plain fp32 partial sums");
    bool gated = false, rare = false;
    for (int i = 0; i < g.nsec; i++) {
        gated |= gemm_gated_act(g.sec[i].act);
        rare |= gemm_rare_act(g.sec[i].act);
        FH_REQUIRE(g.sec[i].begin % 32 == 0, "tiled_gemm: section at column %d", g.sec[i].begin);
    }
    FH_REQUIRE(!gated || (g.groups == 1 && !g.col_scale), "tiled_gemm: gated sections take one group and no column factors");
    FH_REQUIRE(!g.col_scale || (g.out && g.ld_col_scale % 8 == 0), "tiled_gemm: column factors with rows of %ld", g.ld_col_scale);
    const GemmRows& rows = g.rows;
    if (rows.id) {
        FH_REQUIRE(g.slabs == 1 && !g.bias && !g.x_blocks && !g.row_scale && rows.div > 0 && rows.max_blocks > 0 && rows.group && rows.total,
                   "tiled_gemm: sorted rows take plain sections");
        FH_REQUIRE(rows.block == 16 || rows.block == 32 || rows.block == 64 || ((rows.block == 128 || rows.block == 256) && sizeof(E) == 2), "tiled_gemm: blocks of %d rows", rows.block);
    }
    const long tiles = (long)cdiv(g.m, 128) * cdiv(g.n, 128) * g.groups;
    if (rows.id ? rows.block >= 128 : sizeof(E) == 2 && g.m > 64 && g.n >= 128 && g.slabs == 1 && tiles >= knobs().tiled_big_min_tiles) return launch_big(g, s);
    // rows per workgroup: as many as there are, fewer where narrow outputs would leave CUs idle
    int mt = rows.id ? rows.block / 16 : g.m <= 16 ? 1 : (g.m <= 32 ? 2 : 4);
    while (!rows.id && mt > 1 && (long)cdiv(g.m, 16 * mt) * (g.n / 16) * g.groups * g.slabs < knobs().tiled_min_tiles) mt /= 2;
    const int rbs = rows.id ? rows.max_blocks : cdiv(g.m, 16 * mt), ksteps = g.k / 32, zs = rows.id ? 1 : g.groups * g.slabs;
    // 32 columns per wave, 16 where 32 would leave CUs without a workgroup; K split over the waves until the launch has enough of them
    int J = (long)rbs * (g.n / 32) * zs < (g.slabs > 1 ? 256 : g.n <= 96 && g.m > 64 ? 513 : 257) ? 1 : 2;       // (narrow outputs of prompts: two workgroups per CU)
    if (knobs().tiled_j > 0) J = knobs().tiled_j == 1 ? 1 : 2;
    if (gated) J = 2;
    const long cols = g.n / (16 * J);
    int nw = mt == 1 ? 8 : 4, kw = 1;
    if (knobs().tiled_nw > 0) nw = std::min(8, knobs().tiled_nw);
    while (kw < nw && (long)rbs * cols * zs * kw < (rows.id ? 8192 : 4096) && ksteps >= 8 * kw * g.slabs) kw *= 2;
    if (knobs().tiled_kw > 0) kw = std::min(nw, knobs().tiled_kw);
    const dim3 grid(cdiv(cols, nw / kw), rbs, zs);
    form_hit(rows.id ? FORM_TILED_GEMM_GROUPED : FORM_TILED_GEMM);
#define SMALL(J_, EXT_) \
    (mt == 1 ? launch_small<E, 1, J_, EXT_>(g, grid, nw, kw, s) : mt == 2 ? launch_small<E, 2, J_, EXT_>(g, grid, nw, kw, s) : launch_small<E, 4, J_, EXT_>(g, grid, nw, kw, s))
    if (rows.id || g.col_scale || gated || rare) return J == 1 ? SMALL(1, true) : SMALL(2, true);
    return J == 1 ? SMALL(1, false) : SMALL(2, false);
#undef SMALL
}
template int tiled_gemm<bf16>(const TiledGemm<bf16>&, hipStream_t);
template int tiled_gemm<float>(const TiledGemm<float>&, hipStream_t);

}  // namespace fh
