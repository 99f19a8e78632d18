// Kernels of the layered models' mixers and residual stream (latent_attention.hip, grouped_attention.hip, rglru.hip, linear_attention.hip,
// selective_scan.hip, short_conv.hip, residual_stream.hip).
// E is bf16 or float; all leading dimensions are padded to multiples of 32 (tiled_gemm.h).
#pragma once
#include <algorithm>
#include <initializer_list>

#include "tiled_gemm.h"

namespace fh {

// What a forward's kernels know about the batch (device pointers into the index block; scalars for sizing).
struct BatchView {
    int T = 0, num_seqs = 0, max_blocks = 0;
    int max_keys = 0;                            // longest context of the batch, new tokens included (upper bound)
    bool single = false;                         // every sequence brings one token
    const uint32_t* tokens = nullptr;            // [T]
    const uint32_t* cu = nullptr;                // [num_seqs + 1]
    const uint32_t* pos = nullptr;               // [num_seqs] position of a sequence's first new token
    const int32_t* bt = nullptr;                 // [num_seqs][max_blocks]
    const int32_t* tok_seq = nullptr;            // [T] sequence of a token
    const int32_t* prev = nullptr;               // [num_seqs] token before the first new one, −1: none
    const int32_t* slots = nullptr;              // [num_seqs] recurrent state slot
    const int32_t* units = nullptr;              // [num_units][2] (sequence, first token of the chunk within the batch)
    int num_units = 0;
    const uint32_t *host_cu = nullptr, *host_pos = nullptr;      // the same arrays and the block tables on the host (portions only)
    const int32_t* host_bt = nullptr;
    int long_min = 0;                            // > 0: sequences that bring at least this many tokens are not attended by latent_attention
};

// ── residual stream (residual_stream.hip) ──
// x = factor · embed[token] (+ bigram[(prev·mul_prev + token·mul_cur) mod buckets], or the extra row for a first token) (+ positions[position]),
// fp32; xb = E(x)
template <typename E>
struct Embedding {
    const E *table = nullptr, *bigram = nullptr, *positions = nullptr;
    int buckets = 0;
    int64_t mul_prev = 0, mul_cur = 0;
    float factor = 1.f;
};
template <typename E> int embed_tokens(const Embedding<E>& e, const BatchView& v, float* x, E* xb, int dim, int ldb, hipStream_t s);
// x += sub + Σ_j weights[row][j] · pairs[row·top + j] (top 0: none); xb = E(x); sub is the sum of `slabs` partial sums
template <typename E>
int branch_add(const float* sub, long ld_sub, int slabs, long slab_stride, const E* pairs, long ld_pair, const float* weights, int top, float* x, E* xb,
               int rows, int dim, int ldb, hipStream_t s);
// x += mult · rms(sub · gate) · w (gate null: none); xb = E(x), with next_norm E(rms(x)); sub is the sum of `slabs` partial sums
template <typename E>
int post_norm_add(const float* sub, long ld_sub, int slabs, long slab_stride, const E* gate, long ld_gate, const float* w, float mult, float eps, bool next_norm,
                  float* x, E* xb, int rows, int dim, int ldb, hipStream_t s);
// Blocks whose sublayers follow one another: x ← [keep · x +] branch + add + Σ_j weights[row][j] · pairs[row·top + j], where the branch is sub, or with a second one the mean
// (sub·rms⁻¹·w + sub2·rms⁻¹·w2) / 2; with post_w x ← rms(x) · post_w; then out = E(rms(x) · next_w), or E(x) without next_w.  sub and sub2 are sums
// of `slabs` partial sums.  With post_w only: sub is taken times sub_scale[row], pairs with an id of pair_limit or more stand for the stream itself,
// and gate[row] = σ(x · gate_w) of the new stream is left for whoever reads it next.
template <typename E>
struct StreamUpdate {
    // sub null: zero
    const float *sub = nullptr, *sub2 = nullptr; long ld_sub = 0, slab_stride = 0, slab_stride2 = 0; int slabs = 1, slabs2 = 1;
    const float *w = nullptr, *w2 = nullptr;      // norms of the two branches (with sub2)
    const float* add = nullptr;                   // a vector for every row
    const E* pairs = nullptr; long ld_pair = 0; const float* weights = nullptr; int top = 0;
    const int32_t* pair_ids = nullptr; int pair_limit = 0;
    const float *sub_scale = nullptr, *gate_w = nullptr; float* gate = nullptr;
    bool replace = false;                         // x ← branch + add
    float keep = 1.f;
    const float *post_w = nullptr, *next_w = nullptr;
    float eps = 0.f;
    float* x = nullptr; E* out = nullptr; long ldo = 0;     // out null: the last update of a forward
    int rows = 0, dim = 0;
};
template <typename E> int stream_update(const StreamUpdate<E>& u, hipStream_t s);
template <typename E> int copy_rows(const E* x, long ldx, E* out, long ldo, int rows, int cols, hipStream_t s);
// out[i] = E(rms(x[row_idx[i]]) · w); row_idx null: row i; w null: ones
template <typename E>
int rms_norm_rows(const float* x, const int32_t* row_idx, const float* w, float eps, E* out, int rows, int dim, int ldo, hipStream_t s);

// ── latent attention (latent_attention.hip) ──
// Cache of a layer: [blocks][(kp + rp) / 8 chunks][16 tokens][8]: the normed latent, then the rotated shared key part, zero-padded.
// Padded sizes (heads' plain query / key dimensions dp, rotated rp, values vp, latent kp) are rounded to what the matrix-core kernels are
// instantiated for, so that they loop over compile-time extents.
struct LatentDims { int heads, kv_rank, q_rank, rot_dim, rot_dims, vdim, dp, rp, kp, qp, vp, window; float scale; };
inline int latent_pad(int n, std::initializer_list<int> sizes) {
    for (int s : sizes) if (n <= s) return s;
    return pad32(n);
}
inline int latent_pad_rank(int n) { return latent_pad(n, {32, 64, 128, 256, 384, 512}); }
inline int latent_pad_rot(int n) { return latent_pad(n, {32, 64}); }
inline int latent_pad_head(int dim, int vdim, int n) { return std::max(dim, vdim) <= 128 ? latent_pad(std::max(dim, vdim), {32, 64, 128}) : pad32(n); }
inline size_t latent_block_elems(const LatentDims& d) { return (size_t)16 * (d.kp + d.rp); }
template <typename E>
struct LatentBuffers {
    const float *cos_t = nullptr, *sin_t = nullptr;   // [positions][rot_dims / 2]
    E* pool = nullptr;
    const E* q = nullptr; long ldq = 0;    // [T][ldq ≥ heads·(dp + rp)]: per head the plain part, then the part to rotate
    const float* sink = nullptr;       // [heads] score-like numbers that take part in the softmax denominator only; null: none
    const E* q_lat = nullptr;          // [T][heads][kp]: plain part taken through the key projection
    E* o_lat = nullptr;                // [T][heads][kp]
    float* partial = nullptr; size_t partial_bytes = 0;
};
// q latent (q_rank 0: none): RMS norm → cq [T][qp]; kv latent: RMS norm, shared key part: rotation → cache.  `dq` / `dkv`: their columns in the
// fused projection's rows (ld); dkv = [kp latent | rp key part].
template <typename E>
int latent_prepare(const E* dq, const E* dkv, long ld, const float* dq_norm, const float* dkv_norm, float eps, const LatentDims& d,
                   const LatentBuffers<E>& b, const BatchView& v, E* cq, hipStream_t s);
template <typename E>
int latent_attention(const LatentDims& d, const LatentBuffers<E>& b, const BatchView& v, hipStream_t s);
// Portions over expanded keys and values (16-bit): blocks [nblocks] lists the cache blocks whose keys ke [16·nblocks][heads·dp] and
// values ve [16·nblocks][heads·vp] were expanded; units [nunits][4] = (sequence, first token of the tile within the portion, index in
// `blocks` of the sequence's first listed block, that block's number in the sequence).  out [T][ldo ≥ heads·vp], times the head gate if any.
struct LatentExpanded {
    const int32_t *blocks = nullptr, *units = nullptr;
    int nblocks = 0, nunits = 0;
    const bf16 *ke = nullptr, *ve = nullptr;
    long ldk = 0, ldv = 0;
    const bf16* gate = nullptr; long ld_gate = 0;
    bf16* out = nullptr; long ldo = 0;
};
constexpr int LATENT_NO_WINDOW = 1 << 30;
constexpr int LATENT_TILE_TOKENS = 128;          // tokens of a portion per workgroup
bool latent_expanded_supports(const LatentDims& d);
int latent_attention_expanded(const LatentDims& d, const LatentBuffers<bf16>& b, const BatchView& v, const LatentExpanded& x, hipStream_t s);

// ── grouped attention (grouped_attention.hip, talking_attention.hip) ──
// Keys and values of a layer: per block and key / value head [dp / 8 chunks][16 tokens][8] and, for the values, [vp / 32][4 token quads]
// [16 dims][2 halves][4 tokens]: both products' operands are contiguous loads.  Heads are padded with zeros to dp, vp.
struct GroupedDims { int heads, kv_heads, dim, vdim, dp, vp, rot_dims, window; float scale; };
inline int grouped_pad_head(int dim, int vdim, int n) { return std::max(dim, vdim) <= 256 ? latent_pad(std::max(dim, vdim), {32, 64, 96, 128, 192, 256}) : pad32(n); }
inline size_t grouped_k_elems(const GroupedDims& d) { return (size_t)16 * d.kv_heads * d.dp; }
inline size_t grouped_v_elems(const GroupedDims& d) { return (size_t)16 * d.kv_heads * d.vp; }
template <typename E>
struct GroupedBuffers {
    const float *cos_t = nullptr, *sin_t = nullptr;   // [positions][rot_dims / 2]
    E *k_pool = nullptr, *v_pool = nullptr;
    const E *q_in = nullptr, *k_in = nullptr, *v_in = nullptr; long ld = 0;      // columns of the fused projection
    const float *q_norm = nullptr, *k_norm = nullptr;     // [heads·dp], [kv_heads·dp]; norms of one head each: [dp]
    bool head_norm = false;                               // one root mean square per head instead of one for all
    float eps = 0.f;
    E* q = nullptr;                                   // [T][heads][dp]: normed and rotated
    const E* gate = nullptr; long ld_gate = 0;        // [T][heads]: factor per head; null: none
    const E* value_gate = nullptr; long ld_value_gate = 0;       // [T][heads·vp]: factor per element; null: none
    float mult = 1.f;                                 // factor of the result
    const float *r1 = nullptr, *r2 = nullptr;         // [heads]: scores lose r1 · ln(1 + r2 · distance); null: none
    const float* sink = nullptr;                      // [heads]: score-like numbers that take part in the denominator only; null: none
    const float* talk = nullptr;                      // [heads][heads]: weight_h = Σ_g talk[h][g] · weight_g ahead of the values; null: none
    float* offset = nullptr;                          // [T][heads]: scratch for the rows' statistics (talk)
    E* out = nullptr; long ldo = 0;
    float* partial = nullptr; size_t partial_bytes = 0;
};
// norms, rotation, cache write (k_in null: another layer caches the keys and values)
template <typename E> int grouped_prepare(const GroupedDims& d, const GroupedBuffers<E>& b, const BatchView& v, hipStream_t s);
template <typename E> int grouped_attention(const GroupedDims& d, const GroupedBuffers<E>& b, const BatchView& v, hipStream_t s);
// … with mixed heads (talk); grouped_attention takes these launches there
template <typename E> int talking_attention(const GroupedDims& d, const GroupedBuffers<E>& b, const BatchView& v, hipStream_t s);
size_t talking_partial_bytes(const GroupedDims& d, int max_tokens);      // scratch for split keys

// ── linear attention with decay (linear_attention.hip) ──
// Per head S ← diag(decay) S + k vᵀ, o = Sᵀ q; o over its root mean square (· norm), · gate · mult.  The state is fp32 [slots][heads][dp][vp].
struct LinearDims { int heads, dim, vdim, dp, vp, rot_dims; float q_scale, k_scale; };
inline int linear_pad_vdim(int n) { return latent_pad(n, {32, 64, 128, 256}); }
// what the state registers of a workgroup of 1024 threads hold
inline bool linear_supports(int dim, int vdim) { return vdim <= 256 && pad32(dim) <= 16 * (4096 / linear_pad_vdim(vdim)); }
template <typename E>
struct LinearBuffers {
    const float *cos_t = nullptr, *sin_t = nullptr;                     // rotation in halves of the first rot_dims dimensions
    const E *q = nullptr, *k = nullptr, *v = nullptr, *g = nullptr; long ld = 0;      // columns of the fused projection (g with its activation)
    const float* log_decay = nullptr; long ld_decay = 0;               // [T][heads·dp]; null: head_decay
    const float* head_decay = nullptr;                                 // [heads] logarithms
    const float* norm = nullptr;                                       // [vp]; null: ones
    float eps = 0.f, mult = 1.f;
    float* state = nullptr;
    float *chunk_s = nullptr, *chunk_b = nullptr;                      // portions: [units][heads][dp][vp] and [units][heads][dp]
    E* out = nullptr; long ldo = 0;
};
template <typename E> int linear_attention(const LinearDims& d, const LinearBuffers<E>& b, const BatchView& v, hipStream_t s);

// ── short convolution (short_conv.hip) ──
template <typename E>
struct ShortConv {
    const E* x; long ld;                 // [T][ld ≥ wp]
    const float *w, *b;                  // [taps][wp], [wp]
    E* state;                            // [slots][taps − 1][wp]
    E* out;                              // [T][wp]
    int wp, taps;
    bool silu;
};
template <typename E> int short_conv(const ShortConv<E>& p, const BatchView& v, hipStream_t s);

// ── selective scan (selective_scan.hip) ──
// Per channel c and state n: S ← exp(dt_c A[c, n]) S + dt_c u_c B_n; y_c = Σ_n S C_n + D_c u_c; out = y · z.
struct ScanDims { int wp, state, sp, bc; };      // channels (padded), states, states of the kernels' layout (a power of two), columns of B (and of C)
inline int scan_pad_state(int n) { int p = 8; while (p < n) p *= 2; return p; }
constexpr int SCAN_MAX_STATE = 256;
template <typename E>
struct ScanBuffers {
    ShortConv<E> conv{};
    const E* low = nullptr; long ld_low = 0; int c_b = 0;     // [T]: …, B [bc] at c_b, C [bc] behind it
    const float* dt = nullptr;                                // [T][wp]
    const E* z = nullptr; long ld_z = 0;                      // with its activation
    const float *a = nullptr, *d = nullptr;                   // [wp][sp] A · log2 e, [wp]
    float* state = nullptr;                                   // [slots][wp][sp]
    float *chunk_s = nullptr, *chunk_dt = nullptr;            // [units][wp][sp], [units][wp]
    E* out = nullptr;                                         // [T][wp]
};
template <typename E> int selective_scan(const ScanDims& d, const ScanBuffers<E>& b, const BatchView& v, hipStream_t s);

// ── real-gated linear recurrent unit (rglru.hip) ──
// Channels live in a block-padded layout: blocks · bp with bp = pad32(width / blocks); padded channels are zero throughout.
struct RglruDims { int blocks, bp, wp, taps; };
template <typename E>
struct RglruBuffers {
    const E* x = nullptr; const E* y = nullptr; long ld = 0;      // columns of the fused projection (bias and gelu applied)
    const float *conv_w = nullptr, *conv_b = nullptr;              // [taps][wp], [wp]
    const E* gate_w = nullptr; const float *ra_b = nullptr, *ri_b = nullptr;    // fragment tiles [blocks][bp / 16][ra, ri], biases [wp]
    const float* lam = nullptr;                                    // softplus(lam) [wp]
    E* conv_state = nullptr; float* state = nullptr;               // [slots][taps − 1][wp], [slots][wp]
    E* u = nullptr;                                                // [T][wp]
    float *decay = nullptr, *drive = nullptr;                      // [T][wp]
    float *chunk_a = nullptr, *chunk_h = nullptr;                  // [units][wp]
    E* out = nullptr;                                              // [T][wp]
};
constexpr int RGLRU_CHUNK = 64;        // tokens per scan chunk (BatchView::units)
template <typename E>
int rglru_forward(const RglruDims& d, const RglruBuffers<E>& b, const BatchView& v, hipStream_t s);

}  // namespace fh
