// Layered models (layered.h): weight packing and the forward pass.
//
// A layer is a mixer and, optionally, a feed-forward, in one of two blocks.
// Gated post-norm block: both sublayers read the residual stream itself; their result is multiplied by a sigmoid gate of the same input,
// normed (weight stored around zero) and added with a constant factor:
//     x ← x + m · norm(sub(x) · σ(W x + b))
// Everything that reads x is ONE projection per sublayer — the gate's rows, then the mixer's (or feed-forward's) input rows, each
// section with its own activation in the epilogue:
//     latent attention : [gate σ | q latent | kv latent + shared key part | head gates σ] → norms, rotation, cache write → query up-projection
//                        → query through W_ukᵀ (per head) → attention over the latents → W_uv (per head, × head gate) → W_o → add + norm
//                        (long portions: keys and values of the visible cache blocks expanded → flash attention × head gate → W_o)
//     linear recurrence: [gate σ | y gelu | x] → convolution → gates + state (one token) or scan (portions) → W_o → add + norm
//     feed-forward     : [gate σ | up xIELU] → down → add + norm
// Parallel pre-norm block: both sublayers read x̂ = x / rms(x) times a gain of their own that is a single number, so x̂ is written once,
// the gains are factors of the projections' sections, and mixer and dense feed-forward share the projection in and the projection out:
//     [q | kv latent + shared key part | (gate, up) pairs → y] → attention as above → [W_down | W_o]·[y ; attention] → add
//     mixture of experts: router → top-k → rows sorted by expert → up (relu²) → down, summed with its weights by the residual add
// and may end with a per-layer view of the token: x ← x + norm(W_p (gelu(W_g x) · e_layer[token])); the kernel that adds it writes the
// next layer's x̂.  A latent attention layer may read the latents that an earlier layer has cached.
// Pre-norm block: x ← x + mixer(norm1(x)), x ← x + ff(norm2(x)), each sublayer again behind one projection of everything that reads the
// norm's output; the kernel that adds a sublayer's result writes the next sublayer's normed input.
//     two mixers side by side: [q | k | v | q' | k' | v' | decay rank | head gates σ | gate' silu] → norms, rotation, cache write → attention;
//                        decays (from their rank) → linear attention; W_o over both results, or one each where the results are normed
//     selective scan   : [x | z silu] → convolution silu → [dt rank | B | C] → dt softplus → scan × z → W_o
//     feed-forward     : (gate, up) pairs → y → down, or experts of that form behind a grouped router
// A range of its layers may run several times in a row, each pass with caches and states of its own.
// Post-norm block: x ← norm1(α x + mixer(x)), x ← norm2(α x + ff(x)): the same sublayers behind the same projections, which read x itself; the
// kernel that adds a sublayer's result norms the sum.
//     attention        : [q | k | v | value gates σ] → norms per head, cache write → attention, its heads mixed or not → W_o
//     experts          : corrected softmax router → experts of clamped gates; those past the last one hand x on, inside the sum; beside them
//                        (gate, up) pairs → y → down of the shared expert, times a factor per token in the sum; the previous sum leaves the factor
#include <math.h>

#include <algorithm>
#include <functional>
#include <unordered_map>

#include "common.h"
#include "kernels.h"
#include "knobs.h"
#include "layered.h"

namespace fh {

namespace {

uint16_t bf16_bits(float f) {
    uint32_t u;
    memcpy(&u, &f, 4);
    return (uint16_t)((u + 0x7FFFu + ((u >> 16) & 1u)) >> 16);       // round to nearest even (finite weights)
}
void store(bf16* dst, float f) { const uint16_t h = bf16_bits(f); memcpy(dst, &h, 2); }
void store(float* dst, float f) { *dst = f; }

constexpr int MOE_MAX_BLOCK = 256;
constexpr float GLU_SLOPE = 1.702f;              // of the clamped GLUs' sigmoid

struct HostTensor { std::vector<float> data; std::vector<int64_t> shape; };

// Device memory owned by a model.
class Arena {
public:
    ~Arena() { for (void* p : mem_) (void)hipFree(p); }
    template <typename T> int alloc(T** p, size_t n) {
        *p = nullptr;
        if (!n) return 0;
        FH_CHECK_HIP(hipMalloc((void**)p, n * sizeof(T)));
        mem_.push_back(*p);
        FH_CHECK_HIP(hipMemset(*p, 0, n * sizeof(T)));
        return 0;
    }
    template <typename T> int upload(T** p, const std::vector<T>& v) {
        if (int rc = alloc(p, v.size())) return rc;
        FH_CHECK_HIP(hipMemcpy(*p, v.data(), v.size() * sizeof(T), hipMemcpyHostToDevice));
        return 0;
    }
private:
    std::vector<void*> mem_;
};

double softplus(double z) { return z > 0 ? z + log1p(exp(-z)) : log1p(exp(z)); }

__device__ __forceinline__ uint64_t mix64(uint64_t x) {
    x += 0x9E3779B97F4A7C15ull;
    x = (x ^ (x >> 30)) * 0xBF58476D1CE4E5B9ull;
    x = (x ^ (x >> 27)) * 0x94D049BB133111EBull;
    return x ^ (x >> 31);
}
// uniform with the given standard deviation
template <typename E>
__global__ void synth_kernel(E* p, size_t n, uint64_t seed, float std) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) p[i] = (E)(((float)(mix64(seed + i) >> 40) / 8388608.0f - 1.0f) * 1.7320508f * std);
}

#define FH_TRY(call) do { if (int rc_ = (call)) return rc_; } while (0)
// a kernel of the forward `run` (Layered::Run), announced and waited for when launches are traced
#define RUN(call)                                                                                        \
    do {                                                                                                 \
        if (run.trace) fprintf(stderr, "[ferrum_hip] layer %d T=%d %.60s\n", run.li, run.v.T, #call);    \
        FH_TRY(call);                                                                                    \
        if (run.trace) FH_CHECK_HIP(hipStreamSynchronize(run.s));                                        \
    } while (0)

template <typename E>
class Layered final : public LayeredModel {
    struct Linear { E* w = nullptr; float* bias = nullptr; int n = 0, k = 0, groups = 1; };
    struct Layer {
        FerrumHipLayerSpec s;
        // fused input projection of the mixer: sections in the order of the comment at the top
        Linear in, uq, uk, uv, expand, o, ff_in, down;
        GemmSection in_sec[GEMM_MAX_SECTIONS], ff_sec[2];
        int in_nsec = 0, ld_in = 0;
        int c0 = 0, c1 = 0, c2 = 0;        // columns of the mixer's sections: latent attention: q (latent), kv latent, head gates; recurrence: y, x
        int c_glu = -1, c_att = -1;        // parallel block: columns of the feed-forward's gated product and, behind it, of the attention's result
        float *norm1 = nullptr, *norm2 = nullptr;
        float g2 = 1.f;
        Linear router, up, side_gate, side_proj, shared_in, shared_down;
        GemmSection shared_sec;
        float* shared_gate = nullptr;
        E* side_table = nullptr;
        float* side_norm = nullptr;
        // pre-norm block: the second mixer's W_o where its result is normed by itself, and the two norms
        Linear o2, decay, conv_in, dt;
        float *out1 = nullptr, *out2 = nullptr, *down_bias = nullptr, *correction = nullptr, *o_bias = nullptr;
        int c_v = 0, c_q2 = 0, c_k2 = 0, c_v2 = 0, c_g2 = 0, c_rank = 0, c_gate = 0;
        GroupedDims gd{};
        LinearDims nd{};
        ScanDims sd{};
        std::vector<GroupedBuffers<E>> gb;      // one per pass
        std::vector<LinearBuffers<E>> nb;
        std::vector<ScanBuffers<E>> sb;
        LatentDims ld{};
        float *dq_norm = nullptr, *dkv_norm = nullptr;
        LatentBuffers<E> lb{};
        RglruDims rd{};
        RglruBuffers<E> rb{};
    };

public:
    Layered(const FerrumHipModelConfig& c, const FerrumHipLayeredConfig& lc, const FerrumHipLayerSpec* layers, int slots)
        : c_(c), lc_(lc), slots_(slots), D_(c.hidden), Dp_(pad32(c.hidden)) {
        for (int i = 0; i < c.num_layers; i++) { Layer L; L.s = layers[i]; dims(L); layers_.push_back(L); }
    }
    ~Layered() override {
        if (plan_host_) (void)hipHostFree(plan_host_);
        if (fork_) (void)hipEventDestroy(fork_);
        if (join_) (void)hipEventDestroy(join_);
        if (side_stream_) (void)hipStreamDestroy(side_stream_);
    }
    bool has_state() const override {
        return std::any_of(layers_.begin(), layers_.end(), [](const Layer& L) {
            return L.s.mixer2 || (L.s.mixer != FERRUM_HIP_MIXER_LATENT_ATTENTION && L.s.mixer != FERRUM_HIP_MIXER_GROUPED_ATTENTION); });
    }
    int layer_runs() const override { return c_.num_layers + (loops() ? (lc_.loop_times - 1) * (lc_.loop_stop - lc_.loop_start) : 0); }
    bool reads_previous_token() const override { return lc_.bigram_buckets > 0; }

    int set_tensor(const char* name, const float* data, const int64_t* shape, int ndim) override {
        HostTensor t;
        t.shape.assign(shape, shape + ndim);
        size_t n = 1;
        for (int64_t d : t.shape) n *= (size_t)d;
        t.data.assign(data, data + n);
        host_[name] = std::move(t);
        return 0;
    }

    int init_synthetic(uint64_t seed, hipStream_t) override { synth_ = true; seed_ = seed; return 0; }

    int finalize(hipStream_t s) override {
        stream_ = s;
        const size_t T = c_.max_tokens;
        // embedding table (gather) and the same table as vocabulary projection; bigram table
        FH_TRY(table("embed", c_.vocab, &embed_));
        if (lc_.bigram_buckets > 0) FH_TRY(table("bigram", lc_.bigram_buckets + 1, &bigram_));
        if (lc_.position_rows > 0) FH_TRY(table("pos", lc_.position_rows, &positions_));
        FH_TRY(pack(&head_, {{lc_.untied_head ? "head" : "embed", 0, c_.vocab, pad32(c_.vocab)}}, D_));
        if (parallel()) {
            float g = 1.f;
            FH_TRY(scalar("final.norm", &g));
            FH_TRY(arena_.upload(&final_norm_, std::vector<float>(pad32(D_), g)));
        } else if (in_turn()) {
            FH_TRY(vec("final.norm", {D_}, pad32(D_), &final_norm_));
        } else {
            FH_TRY(unit_offset("final.norm", &final_norm_));
        }
        if (loops()) {
            FH_TRY(need("loop.in", {D_, 2 * (int64_t)D_}));
            FH_TRY(pack_fn(&loop_in_, 1, Dp_, 2 * Dp_, "loop.in", [&](const float* w, int, int n, int k) {
                const int half = k / Dp_, c = k % Dp_;
                return n < D_ && c < D_ ? w[(size_t)n * 2 * D_ + half * D_ + c] : 0.f; }));
            FH_TRY(matrix("loop.step", lc_.loop_times, D_, Dp_, &loop_step_));
        }
        long in_cols = 0, q_cols = 0, lat_cols = 0, attn_cols = 0, cq_cols = 0, rnn_cols = 0, side_cols = 0, decay_cols = 0, u_cols = 0, chunk_cols = 0, talk_cols = 0;
        size_t chunk_elems = 0;
        bool joined = false, gated = false;
        size_t units = T / RGLRU_CHUNK + c_.max_seqs, partial = 0, pairs = 0, sorted = 0, expert_cols = 0, logit_cols = 0;
        for (int li = 0; li < c_.num_layers; li++) {
            Layer& L = layers_[li];
            const FerrumHipLayerSpec& sp = L.s;
            const std::string p = "l" + std::to_string(li) + ".";
            Input in;
            float g1 = 1.f;
            if (parallel()) {
                FH_TRY(scalar(p + "norm1", &g1));
                if (sp.ff != FERRUM_HIP_FF_NONE) FH_TRY(scalar(p + "norm2", &L.g2));
            } else if (in_turn()) {
                FH_TRY(vec(p + "norm1", {D_}, Dp_, &L.norm1));
                if (sp.ff != FERRUM_HIP_FF_NONE) FH_TRY(vec(p + "norm2", {D_}, Dp_, &L.norm2));
            } else {
                FH_TRY(unit_offset(p + "norm1", &L.norm1));
                section(L, in, GEMM_ACT_SIGMOID);
                in.add(p + "rg1", 0, D_, Dp_, p + "rg1.b");
            }
            if (sp.mixer == FERRUM_HIP_MIXER_LATENT_ATTENTION) {
                FH_TRY(latent_weights(L, in, p + "mix.", g1));
                const LatentDims& d = L.ld;
                lat_cols = std::max<long>(lat_cols, (long)d.heads * d.kp);
                cq_cols = std::max<long>(cq_cols, d.qp);
                if (d.q_rank) q_cols = std::max<long>(q_cols, L.uq.n);
                // split attention: (row tile, split) pairs stay below 1024
                partial = std::max<size_t>(partial, (size_t)1024 * 16 * (d.kp + 4) * 4);
            } else if (in_turn()) {
                if (sp.mixer == FERRUM_HIP_MIXER_SELECTIVE_SCAN) FH_TRY(scan_weights(L, in, p + "mix.", li));
                else FH_TRY(pair_weights(L, in, p + "mix.", li));
                attn_cols = std::max<long>(attn_cols, L.o.k + L.o2.k);
                if (L.gd.heads) {
                    q_cols = std::max<long>(q_cols, (long)L.gd.heads * L.gd.dp);
                    partial = std::max<size_t>(partial, (size_t)1024 * 16 * (L.gd.vp + 4) * 4);
                    if (sp.attn_flags & FERRUM_HIP_ATTN_TALK) {
                        partial = std::max(partial, talking_partial_bytes(L.gd, c_.max_tokens));
                        talk_cols = std::max<long>(talk_cols, L.gd.heads);
                    }
                }
                decay_cols = std::max<long>(decay_cols, L.decay.n);
                if (L.nd.heads) {
                    chunk_elems = std::max(chunk_elems, (size_t)L.nd.heads * L.nd.dp * L.nd.vp);
                    chunk_cols = std::max<long>(chunk_cols, (long)L.nd.heads * L.nd.dp);
                }
                if (L.sd.wp) {
                    u_cols = std::max<long>(u_cols, L.sd.wp);
                    decay_cols = std::max<long>(decay_cols, L.sd.wp);
                    cq_cols = std::max<long>(cq_cols, L.conv_in.n);
                    chunk_elems = std::max(chunk_elems, (size_t)L.sd.wp * L.sd.sp);
                    chunk_cols = std::max<long>(chunk_cols, L.sd.wp);
                }
                joined |= L.o2.n > 0;
            } else {
                FH_TRY(recurrent_weights(L, in, p + "mix."));
                rnn_cols = std::max<long>(rnn_cols, L.rd.wp);
            }
            FH_TRY(feed_forward_weights(L, in, p));
            FH_TRY(pack(&L.in, in.rows, D_));
            if (in.biased()) FH_TRY(bias(&L.in, in.rows, in.bias));
            L.ld_in = L.in.n;
            if (sp.mixer == FERRUM_HIP_MIXER_LATENT_ATTENTION) {
                const long att = (long)L.ld.heads * L.ld.vp;
                if (L.c_att >= 0) L.ld_in = (int)std::max<long>(L.ld_in, L.c_att + att);
                else attn_cols = std::max(attn_cols, att);
            }
            in_cols = std::max<long>({in_cols, L.ld_in, L.ff_in.n, L.shared_in.n});
            if (moe(sp)) {
                const size_t n = T * sp.top;
                pairs = std::max(pairs, n);
                sorted = std::max(sorted, n + (size_t)MOE_MAX_BLOCK * (std::min<size_t>(sp.experts, n) + 1));
                expert_cols = std::max(expert_cols, n * (size_t)L.down.k);
                logit_cols = std::max<size_t>(logit_cols, sp.experts + sp.identity_experts);
                gated |= L.shared_gate != nullptr;
            }
            if (lc_.token_side_dim) {
                FH_TRY(side_weights(L, p, li));
                side_cols = L.side_gate.n;
            }
        }
        host_.clear();
        FH_TRY(arena_.alloc(&x_, T * D_));
        FH_TRY(arena_.alloc(&xb_, T * Dp_));
        FH_TRY(arena_.alloc(&in_, T * in_cols));
        FH_TRY(arena_.alloc(&sub_, std::max<size_t>(T, (size_t)GEMM_MAX_SLABS * std::min<size_t>(T, 64)) * Dp_));
        if (joined) FH_TRY(arena_.alloc(&sub2_, std::max<size_t>(T, (size_t)GEMM_MAX_SLABS * std::min<size_t>(T, 64)) * Dp_));
        if (loops()) FH_TRY(arena_.alloc(&cat_, T * 2 * Dp_));
        FH_TRY(arena_.alloc(&cq_, T * cq_cols));
        FH_TRY(arena_.alloc(&q_, T * q_cols));
        FH_TRY(arena_.alloc(&talk_offset_, T * talk_cols));
        FH_TRY(arena_.alloc(&row_gate_, gated ? T : 0));
        FH_TRY(arena_.alloc(&q_lat_, T * lat_cols));
        FH_TRY(arena_.alloc(&o_lat_, T * lat_cols));
        FH_TRY(arena_.alloc(&attn_, T * attn_cols));
        partial_bytes_ = partial;
        FH_TRY(arena_.alloc(&partial_, partial / 4));
        FH_TRY(arena_.alloc(&u_, T * std::max(rnn_cols, u_cols)));
        FH_TRY(arena_.alloc(&rnn_out_, T * rnn_cols));
        FH_TRY(arena_.alloc(&decay_, T * std::max(rnn_cols, decay_cols)));
        FH_TRY(arena_.alloc(&drive_, T * rnn_cols));
        FH_TRY(arena_.alloc(&chunk_a_, units * std::max(rnn_cols, chunk_cols)));
        FH_TRY(arena_.alloc(&chunk_h_, units * std::max<size_t>(rnn_cols, chunk_elems)));
        FH_TRY(arena_.alloc(&side_, T * side_cols));
        FH_TRY(arena_.alloc(&router_logits_, T * logit_cols));
        FH_TRY(arena_.alloc(&expert_ids_, pairs));
        FH_TRY(arena_.alloc(&expert_weights_, pairs));
        FH_TRY(arena_.alloc(&sorted_, sorted));
        FH_TRY(arena_.alloc(&sorted_expert_, pairs));
        FH_TRY(arena_.alloc(&sorted_total_, pairs ? 4 : 0));
        FH_TRY(arena_.alloc(&expert_h_, expert_cols));
        FH_TRY(arena_.alloc(&expert_y_, pairs * Dp_));
        FH_TRY(arena_.alloc(&head_in_, (size_t)c_.max_seqs * Dp_));
        FH_TRY(finalize_expansion());
        if (pairs) {
            FH_CHECK_HIP(hipStreamCreateWithFlags(&side_stream_, hipStreamNonBlocking));
            FH_CHECK_HIP(hipEventCreateWithFlags(&fork_, hipEventDisableTiming));
            FH_CHECK_HIP(hipEventCreateWithFlags(&join_, hipEventDisableTiming));
        }
        for (Layer& L : layers_) {
            wire(L);
            if (L.s.kv_source) L.lb.pool = layers_[L.s.kv_source - 1].lb.pool;
            L.lb.q = L.ld.q_rank ? q_ : in_ + L.c0;
            L.lb.ldq = L.ld.q_rank ? L.uq.n : L.ld_in;
            L.lb.q_lat = q_lat_; L.lb.o_lat = o_lat_; L.lb.partial = partial_; L.lb.partial_bytes = partial_bytes_;
            L.rb.x = in_ + L.c1; L.rb.y = in_ + L.c0; L.rb.ld = L.ld_in;
            L.rb.u = u_; L.rb.out = rnn_out_; L.rb.decay = decay_; L.rb.drive = drive_; L.rb.chunk_a = chunk_a_; L.rb.chunk_h = chunk_h_;
        }
        FH_CHECK_HIP(hipStreamSynchronize(s));
        return 0;
    }

    int forward(const BatchView& v, float* taps, bool trace, hipStream_t s) override {
        Run run{v, v, true, trace, s, -1};
        run.any_short = plan_expansion(&run.short_view);
        if (run.short_view.long_min > 0)
            FH_CHECK_HIP(hipMemcpyAsync(plan_dev_, plan_host_, plan_used_ * 4, hipMemcpyHostToDevice, s));
        Embedding<E> e;
        e.table = embed_; e.bigram = bigram_; e.positions = positions_;
        e.buckets = lc_.bigram_buckets; e.mul_prev = lc_.bigram_mul_prev; e.mul_cur = lc_.bigram_mul_cur;
        if (lc_.embed_scale != 0.f) e.factor = lc_.embed_scale;
        RUN(embed_tokens<E>(e, v, x_, xb_, D_, Dp_, s));
        if (in_turn()) return in_turn_forward(run, taps);
        if (parallel()) RUN(rms_norm_rows<E>(x_, nullptr, nullptr, c_.rms_eps, xb_, v.T, D_, Dp_, s));
        for (run.li = 0; run.li < c_.num_layers; run.li++) {
            Layer& L = layers_[run.li];
            FH_TRY(parallel() ? parallel_layer(L, run) : gated_layer(L, run));
            if (taps) FH_CHECK_HIP(hipMemcpyAsync(taps + (size_t)run.li * c_.max_tokens * D_, x_, (size_t)v.T * D_ * 4, hipMemcpyDeviceToDevice, s));
        }
        return 0;
    }

    int head(const int32_t* row_idx, int rows, float* logits, hipStream_t s) override {
        FH_TRY(rms_norm_rows<E>(x_, row_idx, final_norm_, c_.rms_eps, head_in_, rows, D_, Dp_, s));
        TiledGemm<E> g = linear_f32(head_, head_in_, Dp_, rows, logits, c_.vocab);
        g.n_store = c_.vocab;
        if (lc_.logit_softcap > 0.f) { g.nsec = 1; g.sec[0] = {0, GEMM_ACT_SOFTCAP, lc_.logit_softcap, 0}; }
        return tiled_gemm(g, s);
    }

private:
    // one forward: the batch, the part of it that latent_attention takes, and the layer at hand
    struct Run { const BatchView& v; BatchView short_view; bool any_short, trace; hipStream_t s; int li; };

    int gated_layer(Layer& L, const Run& run) {
        const int T = run.v.T;
        hipStream_t s = run.s;
        const float eps = c_.rms_eps;
        int slabs = 1;
        RUN(tiled_gemm(input_projection(L, T), s));
        if (L.s.mixer == FERRUM_HIP_MIXER_LATENT_ATTENTION) {
            FH_TRY(attend(L, run, attn_, (long)L.ld.heads * L.ld.vp));
            RUN(tiled_gemm(linear_slabs(L.o, attn_, (long)L.ld.heads * L.ld.vp, T, &slabs), s));
        } else {
            RUN(rglru_forward<E>(L.rd, L.rb, run.v, s));
            RUN(tiled_gemm(linear_slabs(L.o, rnn_out_, L.rd.wp, T, &slabs), s));
        }
        RUN(post_norm_add<E>(sub_, Dp_, slabs, (long)T * Dp_, in_, L.ld_in, L.norm1, lc_.residual_mult, eps, false, x_, xb_, T, D_, Dp_, s));
        if (L.s.ff != FERRUM_HIP_FF_NONE) {
            TiledGemm<E> f = linear(L.ff_in, xb_, Dp_, T, in_, L.ff_in.n);
            f.nsec = 2; f.sec[0] = L.ff_sec[0]; f.sec[1] = L.ff_sec[1];
            RUN(tiled_gemm(f, s));
            RUN(tiled_gemm(linear_slabs(L.down, in_ + Dp_, L.ff_in.n, T, &slabs), s));
            RUN(post_norm_add<E>(sub_, Dp_, slabs, (long)T * Dp_, in_, L.ff_in.n, L.norm2, lc_.residual_mult, eps, false, x_, xb_, T, D_, Dp_, s));
        }
        return 0;
    }

    int parallel_layer(Layer& L, const Run& run) {
        const int T = run.v.T;
        hipStream_t s = run.s;
        const bool moe = L.s.ff == FERRUM_HIP_FF_MOE_RELU2, last = run.li + 1 == c_.num_layers;
        int slabs = 1;
        // few tokens: the experts, bound by their weights' bytes, beside the mixer, bound by the latency of its chain of launches
        const bool beside = moe && few_tokens(run);
        if (moe) FH_TRY(beside ? experts_beside(L, run) : experts(L, run));
        RUN(tiled_gemm(input_projection(L, T), s));
        E* att = L.c_att >= 0 ? in_ + L.c_att : attn_;
        const long ld_att = L.c_att >= 0 ? L.ld_in : (long)L.ld.heads * L.ld.vp;
        FH_TRY(attend(L, run, att, ld_att));
        RUN(tiled_gemm(linear_slabs(L.o, L.c_glu >= 0 ? in_ + L.c_glu : att, ld_att, T, &slabs), s));
        if (beside) FH_CHECK_HIP(hipStreamWaitEvent(s, join_, 0));
        RUN(branch_add<E>(sub_, Dp_, slabs, (long)T * Dp_, expert_y_, Dp_, expert_weights_, moe ? L.s.top : 0, x_, xb_, T, D_, Dp_, s));
        if (lc_.token_side_dim) {
            TiledGemm<E> g = linear(L.side_gate, xb_, Dp_, T, side_, L.side_gate.n);
            g.nsec = 1; g.sec[0] = {0, GEMM_ACT_GELU_TANH, 0, 0};
            g.col_scale = L.side_table; g.col_scale_row = run.v.tokens; g.ld_col_scale = L.side_gate.n;
            RUN(tiled_gemm(g, s));
            RUN(tiled_gemm(linear_slabs(L.side_proj, side_, L.side_gate.n, T, &slabs), s));
            RUN(post_norm_add<E>(sub_, Dp_, slabs, (long)T * Dp_, nullptr, 0, L.side_norm, 1.f, c_.rms_eps, true, x_, xb_, T, D_, Dp_, s));
        } else if (!last) {
            RUN(rms_norm_rows<E>(x_, nullptr, nullptr, c_.rms_eps, xb_, T, D_, Dp_, s));
        }
        return 0;
    }

    // layers in the order they run; pass −1: outside the loop
    struct LayerRun { int layer, pass; };
    std::vector<LayerRun> order() const {
        std::vector<LayerRun> r;
        const int a = loops() ? lc_.loop_start : c_.num_layers, b = loops() ? lc_.loop_stop : c_.num_layers;
        for (int i = 0; i < a; i++) r.push_back({i, -1});
        for (int t = 0; loops() && t < lc_.loop_times; t++)
            for (int i = a; i < b; i++) r.push_back({i, t});
        for (int i = b; i < c_.num_layers; i++) r.push_back({i, -1});
        return r;
    }
    bool opens_pass(const LayerRun& r) const { return r.pass >= 0 && r.layer == lc_.loop_start; }

    int in_turn_forward(Run& run, float* taps) {
        const int T = run.v.T;
        hipStream_t s = run.s;
        const std::vector<LayerRun> runs = order();
        if (loops()) RUN(copy_rows<E>(xb_, Dp_, cat_ + Dp_, 2 * Dp_, T, Dp_, s));
        if (opens_pass(runs[0])) RUN(copy_rows<E>(xb_, Dp_, cat_, 2 * Dp_, T, Dp_, s));
        else if (pre_norm()) RUN(rms_norm_rows<E>(x_, nullptr, layers_[0].norm1, c_.rms_eps, xb_, T, D_, Dp_, s));
        for (size_t i = 0; i < runs.size(); i++) {
            run.li = runs[i].layer;
            if (opens_pass(runs[i])) {
                StreamUpdate<E> u = update(T);
                RUN(tiled_gemm(linear_slabs(loop_in_, cat_, 2 * Dp_, T, &u.slabs), s));
                u.replace = true;
                u.add = loop_step_ + (size_t)runs[i].pass * Dp_;
                u.next_w = layers_[run.li].norm1;
                RUN(stream_update(u, s));
            }
            // what the layer's last update leaves for the next run: its normed input, or the stream itself ahead of a pass
            StreamUpdate<E> next = update(T);
            if (i + 1 == runs.size()) next.out = nullptr;
            else if (opens_pass(runs[i + 1])) { next.out = cat_; next.ldo = 2 * Dp_; }
            else if (pre_norm()) next.next_w = layers_[runs[i + 1].layer].norm1;
            FH_TRY(in_turn_layer(layers_[run.li], std::max(runs[i].pass, 0), run, next));
            if (taps) FH_CHECK_HIP(hipMemcpyAsync(taps + i * c_.max_tokens * D_, x_, (size_t)T * D_ * 4, hipMemcpyDeviceToDevice, s));
        }
        return 0;
    }
    StreamUpdate<E> update(int T) const {
        StreamUpdate<E> u;
        u.sub = sub_; u.ld_sub = Dp_; u.slab_stride = u.slab_stride2 = (long)T * Dp_; u.ld_pair = Dp_;
        u.eps = c_.rms_eps; u.x = x_; u.out = xb_; u.ldo = Dp_; u.rows = T; u.dim = D_;
        return u;
    }

    // `next`: the layer's last update, up to what it adds
    int in_turn_layer(Layer& L, int pass, const Run& run, const StreamUpdate<E>& next) {
        const int T = run.v.T;
        hipStream_t s = run.s;
        const bool ff = L.s.ff != FERRUM_HIP_FF_NONE;
        StreamUpdate<E> u = ff ? update(T) : next;
        if (post_norm()) { u.post_w = L.norm1; u.keep = lc_.stream_mult; }
        if (L.shared_gate) { u.gate_w = L.shared_gate; u.gate = row_gate_; }
        else if (ff) u.next_w = L.norm2;
        u.add = L.o_bias;
        RUN(tiled_gemm(input_projection(L, T), s));
        if (L.sd.wp) {
            ScanBuffers<E>& b = L.sb[pass];
            RUN(short_conv(b.conv, run.v, s));
            RUN(tiled_gemm(linear(L.conv_in, u_, L.sd.wp, T, cq_, L.conv_in.n), s));
            TiledGemm<E> g = linear_f32(L.dt, cq_, L.conv_in.n, T, decay_, L.sd.wp);
            g.nsec = 1; g.sec[0] = {0, GEMM_ACT_SOFTPLUS, 0, 0};
            RUN(tiled_gemm(g, s));
            RUN(selective_scan(L.sd, b, run.v, s));
            RUN(tiled_gemm(linear_slabs(L.o, attn_, L.o.k, T, &u.slabs), s));
        } else {
            if (L.gd.heads) {
                RUN(grouped_prepare(L.gd, L.gb[pass], run.v, s));
                RUN(grouped_attention(L.gd, L.gb[pass], run.v, s));
            }
            if (L.nd.heads) {
                if (L.decay.n) {
                    TiledGemm<E> g = linear_f32(L.decay, in_ + L.c_rank, L.ld_in, T, decay_, L.decay.n);
                    g.nsec = 1; g.sec[0] = {0, GEMM_ACT_LOG_SIGMOID, 1.0f / L.s.lin_tau, 0};
                    RUN(tiled_gemm(g, s));
                }
                RUN(linear_attention(L.nd, L.nb[pass], run.v, s));
            }
            const long ld = L.o.k + L.o2.k;
            RUN(tiled_gemm(linear_slabs(L.o, attn_, ld, T, &u.slabs), s));
            if (L.o2.n) {
                TiledGemm<E> g = linear_slabs(L.o2, attn_ + L.o.k, ld, T, &u.slabs2);
                g.out_f32 = sub2_;
                RUN(tiled_gemm(g, s));
                u.sub2 = sub2_; u.w = L.out1; u.w2 = L.out2;
            }
        }
        RUN(stream_update(u, s));
        if (!ff) return 0;
        StreamUpdate<E> f = next;
        if (post_norm()) { f.post_w = L.norm2; f.keep = lc_.stream_mult; }
        if (moe(L.s)) {
            // few tokens: the experts beside the shared one
            const bool shared = L.s.shared_width > 0, beside = shared && few_tokens(run);
            FH_TRY(beside ? experts_beside(L, run) : experts(L, run));
            f.sub = nullptr;
            f.pairs = expert_y_; f.weights = expert_weights_; f.top = L.s.top;
            if (L.s.identity_experts) { f.pair_ids = expert_ids_; f.pair_limit = L.s.experts; }
            if (shared) {
                TiledGemm<E> g = linear(L.shared_in, xb_, Dp_, T, in_, L.shared_in.n);
                g.nsec = 1; g.sec[0] = L.shared_sec;
                RUN(tiled_gemm(g, s));
                RUN(tiled_gemm(linear_slabs(L.shared_down, in_, L.shared_in.n, T, &f.slabs), s));
                f.sub = sub_;
                f.sub_scale = row_gate_;
            }
            if (beside) FH_CHECK_HIP(hipStreamWaitEvent(s, join_, 0));
        } else {
            TiledGemm<E> g = linear(L.ff_in, xb_, Dp_, T, in_, L.down.k);
            g.nsec = 1; g.sec[0] = L.ff_sec[0];
            RUN(tiled_gemm(g, s));
            RUN(tiled_gemm(linear_slabs(L.down, in_, L.down.k, T, &f.slabs), s));
            f.add = L.down_bias;
        }
        RUN(stream_update(f, s));
        return 0;
    }

    TiledGemm<E> input_projection(const Layer& L, int T) const {
        TiledGemm<E> g = linear(L.in, xb_, Dp_, T, in_, L.ld_in);
        g.nsec = L.in_nsec;
        std::copy(L.in_sec, L.in_sec + L.in_nsec, g.sec);
        return g;
    }

    // latent attention from the input projection's columns to the heads' values, out [T][ldo ≥ heads·vp]
    int attend(Layer& L, const Run& run, E* out, long ldo) {
        const LatentDims& d = L.ld;
        const int T = run.v.T;
        hipStream_t s = run.s;
        const bool gates = !(L.s.attn_flags & FERRUM_HIP_ATTN_NO_HEAD_GATE);
        if (d.q_rank || !L.s.kv_source)
            RUN(latent_prepare<E>(in_ + L.c0, L.s.kv_source ? nullptr : in_ + L.c1, L.ld_in, L.dq_norm, L.dkv_norm, c_.rms_eps, d, L.lb, run.v, cq_, s));
        if (d.q_rank) RUN(tiled_gemm(linear(L.uq, cq_, d.qp, T, q_, L.uq.n), s));
        if (run.any_short) {
            TiledGemm<E> k = linear(L.uk, L.lb.q, L.lb.ldq, T, q_lat_, (long)d.heads * d.kp);
            k.x_group = d.dp + d.rp; k.out_group = d.kp;
            RUN(tiled_gemm(k, s));
            RUN(latent_attention<E>(d, L.lb, run.short_view, s));
            TiledGemm<E> u = linear(L.uv, o_lat_, (long)d.heads * d.kp, T, out, ldo);
            u.x_group = d.kp; u.out_group = d.vp;
            if (gates) { u.row_scale = in_ + L.c2; u.ld_scale = L.ld_in; }
            RUN(tiled_gemm(u, s));
        }
        if (run.short_view.long_min > 0) RUN(attend_expanded(L, run.v, out, ldo, s));        // (writes the rows of the long portions only)
        return 0;
    }

    bool few_tokens(const Run& run) const { return run.v.T <= knobs().layer_overlap_max_tokens && !run.trace; }
    // the experts on a stream of their own; join_ is recorded behind them
    int experts_beside(Layer& L, const Run& run) {
        Run other = run;
        other.s = side_stream_;
        FH_CHECK_HIP(hipEventRecord(fork_, run.s));
        FH_CHECK_HIP(hipStreamWaitEvent(side_stream_, fork_, 0));
        FH_TRY(experts(L, other));
        FH_CHECK_HIP(hipEventRecord(join_, side_stream_));
        return 0;
    }
    // how a layer's router scores and chooses, beyond the softmax over the chosen logits
    static MoeCorrectedRule route_rule(const FerrumHipLayerSpec& s, const float* correction) {
        MoeCorrectedRule r{correction, s.route_groups, s.route_keep, s.route_scale};
        r.softmax = r.raw = s.ff == FERRUM_HIP_FF_MOE_CLAMPED_GLU;
        r.unlisted = s.identity_experts;
        return r;
    }
    // expert_y_ [T·top][Dp], expert_weights_ and expert_ids_ [T·top] of the chosen experts
    int experts(Layer& L, const Run& run) {
        const int T = run.v.T, E_ = L.s.experts, routed = E_ + L.s.identity_experts, pairs = T * L.s.top;
        hipStream_t s = run.s;
        TiledGemm<E> z = linear_f32(L.router, xb_, Dp_, T, router_logits_, routed);
        z.n_store = routed; z.nsec = 1; z.sec[0] = {0, GEMM_ACT_NONE, 0, 0, L.g2};
        RUN(tiled_gemm(z, s));
        GemmRows rows;
        rows.block = moe_block(pairs, E_);
        rows.max_blocks = std::min(pairs, pairs / rows.block + std::min(E_, pairs));
        rows.id = sorted_; rows.group = sorted_expert_; rows.total = sorted_total_;
        const bool corrected = L.s.ff != FERRUM_HIP_FF_MOE_RELU2;
        const MoeCorrectedRule rule = route_rule(L.s, L.correction);
        if (moe_route_sort_supports(T, routed, L.s.top)) {
            RUN(moe_route_sort_f32(router_logits_, expert_ids_, expert_weights_, sorted_, sorted_expert_, sorted_total_, T, routed, L.s.top, 1, rows.block, s, corrected ? &rule : nullptr));
        } else if (corrected) {
            RUN(moe_route_corrected_f32(router_logits_, rule, expert_ids_, expert_weights_, T, routed, L.s.top, s));
            RUN(moe_align_block_size(expert_ids_, sorted_, sorted_expert_, sorted_total_, pairs, E_, rows.block, rows.max_blocks * rows.block, s));
        } else {
            RUN(moe_route_topk_softmax_f32(router_logits_, expert_ids_, expert_weights_, T, E_, L.s.top, 1, s));
            RUN(moe_align_block_size(expert_ids_, sorted_, sorted_expert_, sorted_total_, pairs, E_, rows.block, rows.max_blocks * rows.block, s));
        }
        TiledGemm<E> u = linear(L.up, xb_, Dp_, pairs, expert_h_, L.down.k);
        u.groups = 1; u.rows = rows; u.rows.div = L.s.top;
        u.nsec = 1; u.sec[0] = L.ff_sec[0];
        RUN(tiled_gemm(u, s));
        TiledGemm<E> y = linear(L.down, expert_h_, L.down.k, pairs, expert_y_, Dp_);
        y.groups = 1; y.rows = rows;
        RUN(tiled_gemm(y, s));
        return 0;
    }
    // rows per block of the sorted list: a large block shares an expert's weights between more rows, a small one pads less
    static int moe_block(int pairs, int experts) {
        const int mean = pairs / experts, forced = knobs().moe_rows_block;
        if (forced > 0 && (sizeof(E) == 2 || forced <= 64)) return forced;
        if (sizeof(E) == 2 && mean >= 48) return mean >= 384 ? 256 : 128;
        return mean >= 32 ? 64 : mean >= 12 ? 32 : 16;
    }

    void dims(Layer& L) {
        const FerrumHipLayerSpec& s = L.s;
        if (s.mixer == FERRUM_HIP_MIXER_LATENT_ATTENTION)
            L.ld = {s.heads, s.kv_rank, s.q_rank, s.rot_dim, s.rot_dims, s.vdim, latent_pad_head(s.dim, s.vdim, s.dim), latent_pad_rot(s.rot_dim),
                    latent_pad_rank(s.kv_rank), pad32(s.q_rank), latent_pad_head(s.dim, s.vdim, s.vdim), s.window == FERRUM_HIP_WINDOW_NONE ? LATENT_NO_WINDOW : s.window, s.scale};
        else if (s.mixer == FERRUM_HIP_MIXER_SELECTIVE_SCAN)
            L.sd = {pad32(s.scan_inner), s.scan_state, scan_pad_state(s.scan_state), pad32(s.scan_state)};
        else if (in_turn()) {
            if (s.mixer == FERRUM_HIP_MIXER_GROUPED_ATTENTION)
                L.gd = {s.heads, s.kv_heads, s.dim, s.vdim, grouped_pad_head(s.dim, s.vdim, s.dim), grouped_pad_head(s.dim, s.vdim, s.vdim), s.rot_dims,
                        s.window == FERRUM_HIP_WINDOW_NONE ? LATENT_NO_WINDOW : s.window, s.scale};
            if (linear_mixer(s)) {
                const float root = 1.0f / sqrtf((float)s.lin_dim);
                const bool gated = linear_mixer(s) == FERRUM_HIP_MIXER_GATED_LINEAR;
                L.nd = {s.lin_heads, s.lin_dim, s.lin_vdim, pad32(s.lin_dim), linear_pad_vdim(s.lin_vdim), gated ? 0 : s.lin_rot_dims, gated ? root : 1.f, gated ? 1.f : root};
            }
        } else
            L.rd = {s.rnn_blocks, pad32(s.rnn_width / s.rnn_blocks), s.rnn_blocks * pad32(s.rnn_width / s.rnn_blocks), s.conv_taps};
    }
    static TiledGemm<E> linear(const Linear& w, const E* x, long ldx, int m, E* out, long ldo) {
        TiledGemm<E> g;
        g.x = x; g.ldx = ldx; g.w = w.w; g.bias = w.bias; g.m = m; g.n = w.n; g.k = w.k; g.groups = w.groups; g.out = out; g.ldo = ldo;
        return g;
    }
    static TiledGemm<E> linear_f32(const Linear& w, const E* x, long ldx, int m, float* out, long ldo) {
        TiledGemm<E> g = linear(w, x, ldx, m, nullptr, ldo);
        g.out_f32 = out;
        return g;
    }

    // ── portions over expanded keys and values (16-bit models) ──
    // Every latent layer must take the form, so one decision per sequence serves the whole forward.
    int finalize_expansion() {
        if (sizeof(E) != 2) return 0;
        long cols = 0;
        int widest = 0;
        for (const Layer& L : layers_)
            if (L.s.mixer == FERRUM_HIP_MIXER_LATENT_ATTENTION) {
                if (!latent_expanded_supports(L.ld)) return 0;
                cols = std::max<long>(cols, L.expand.n);
                widest = std::max(widest, L.ld.window);
                if (std::none_of(plans_.begin(), plans_.end(), [&](const Plan& q) { return q.window == L.ld.window; })) plans_.push_back(Plan{L.ld.window});
            }
        if (plans_.empty()) return 0;
        const long per_seq = std::min<long>(widest, c_.max_seq_len) / 16 + 2;
        expand_blocks_ = (int)std::min<long>((c_.max_tokens + 15) / 16 + c_.max_seqs * per_seq, std::max(c_.kv_num_blocks, 1));
        const size_t ints = plans_.size() * ((size_t)expand_blocks_ + 4 * ((size_t)c_.max_tokens / LATENT_TILE_TOKENS + c_.max_seqs));
        FH_TRY(arena_.alloc(&expanded_, (size_t)expand_blocks_ * 16 * cols));
        FH_TRY(arena_.alloc(&plan_dev_, ints));
        FH_CHECK_HIP(hipHostMalloc((void**)&plan_host_, ints * 4, hipHostMallocDefault));
        return 0;
    }
    // Which cache blocks to expand and which tiles to run, per distinct window.  Sets v->long_min when some sequence takes the form;
    // returns whether any does not.
    bool plan_expansion(BatchView* v) {
        const int min_rows = knobs().latent_expand_min_rows;
        if (v->single || !plan_host_ || min_rows <= 0 || knobs().latent_plain) return true;
        bool any_short = false, any_long = false;
        plan_used_ = 0;
        for (Plan& q : plans_) {
            q.blocks0 = plan_used_;
            q.nblocks = q.nunits = 0;
            std::vector<int32_t> units;
            for (int i = 0; i < v->num_seqs; i++) {
                const int n = (int)(v->host_cu[i + 1] - v->host_cu[i]), pos = (int)v->host_pos[i];
                if (n < min_rows) { any_short = true; continue; }
                any_long = true;
                const int lo = std::max(0, pos + 1 - q.window) / 16, hi = (pos + n + 15) / 16;
                if (q.nblocks + hi - lo > expand_blocks_) return true;           // (shared prefix blocks listed more often than the pool holds)
                for (int t = 0; t < n; t += LATENT_TILE_TOKENS) units.insert(units.end(), {i, t, q.nblocks, lo});
                for (int b = lo; b < hi; b++) plan_host_[plan_used_++] = v->host_bt[(size_t)i * v->max_blocks + b];
                q.nblocks += hi - lo;
            }
            q.units0 = plan_used_;
            q.nunits = (int)units.size() / 4;
            std::copy(units.begin(), units.end(), plan_host_ + plan_used_);
            plan_used_ += units.size();
        }
        if (any_long) v->long_min = min_rows;
        return any_short;
    }
    int attend_expanded(Layer& L, const BatchView& v, E* out, long ldo, hipStream_t s) {
        if constexpr (sizeof(E) == 2) {
            const Plan& q = *std::find_if(plans_.begin(), plans_.end(), [&](const Plan& x) { return x.window == L.ld.window; });
            const LatentDims& d = L.ld;
            TiledGemm<E> g = linear(L.expand, L.lb.pool, 0, q.nblocks * 16, expanded_, L.expand.n);
            g.x_blocks = plan_dev_ + q.blocks0; g.x_block_elems = (long)latent_block_elems(d);
            FH_TRY(tiled_gemm(g, s));
            LatentExpanded x;
            x.blocks = plan_dev_ + q.blocks0; x.units = plan_dev_ + q.units0; x.nblocks = q.nblocks; x.nunits = q.nunits;
            x.ke = expanded_; x.ve = expanded_ + (size_t)d.heads * d.dp; x.ldk = x.ldv = L.expand.n;
            if (!(L.s.attn_flags & FERRUM_HIP_ATTN_NO_HEAD_GATE)) { x.gate = in_ + L.c2; x.ld_gate = L.ld_in; }
            x.out = out; x.ldo = ldo;
            return latent_attention_expanded(d, L.lb, v, x, s);
        }
        return 0;
    }
    struct Plan { int window; size_t blocks0 = 0, units0 = 0; int nblocks = 0, nunits = 0; };

    // projection whose consumer is the residual update: partial sums over K, as many as fill the chip
    TiledGemm<E> linear_slabs(const Linear& w, const E* x, long ldx, int m, int* slabs) const {
        TiledGemm<E> g = linear_f32(w, x, ldx, m, sub_, Dp_);
        g.slabs = *slabs = tiled_gemm_slabs(m, w.n, w.k);
        g.slab_stride = (long)m * Dp_;
        return g;
    }

    // ── weights ──
    bool parallel() const { return lc_.block == FERRUM_HIP_BLOCK_PARALLEL_PRE_NORM; }
    bool pre_norm() const { return lc_.block == FERRUM_HIP_BLOCK_PRE_NORM; }
    bool post_norm() const { return lc_.block == FERRUM_HIP_BLOCK_POST_NORM; }
    bool in_turn() const { return pre_norm() || post_norm(); }       // plain sublayers one after the other
    bool loops() const { return lc_.loop_times > 0; }
    int passes(int li) const { return loops() && li >= lc_.loop_start && li < lc_.loop_stop ? lc_.loop_times : 1; }
    static bool moe(const FerrumHipLayerSpec& s) { return s.ff == FERRUM_HIP_FF_MOE_RELU2 || s.ff == FERRUM_HIP_FF_MOE_SILU_GLU || s.ff == FERRUM_HIP_FF_MOE_CLAMPED_GLU; }
    // the layer's linear attention: its second mixer, or its only one
    static int linear_mixer(const FerrumHipLayerSpec& s) {
        return s.mixer2 ? s.mixer2 : s.mixer == FERRUM_HIP_MIXER_GATED_LINEAR || s.mixer == FERRUM_HIP_MIXER_RETENTION ? s.mixer : 0;
    }
    struct Input;
    // opens a section of the layer's input projection; returns its first column
    static int section(Layer& L, const Input& in, GemmAct act, float mul = 1.f, float p = 0.f, float q = 0.f) {
        L.in_sec[L.in_nsec++] = {in.cols(), act, p, q, mul};
        return in.cols();
    }
    int latent_weights(Layer& L, Input& in, const std::string& m, float g1) {
        const FerrumHipLayerSpec& sp = L.s;
        const LatentDims& d = L.ld;
        const int H = d.heads, dim = sp.dim, kr = d.kv_rank, vd = d.vdim, dp = d.dp, vp = d.vp;
        std::vector<Rows> q;
        const std::string qn = m + (d.q_rank ? "uq" : "q");
        for (int h = 0; h < H; h++) {
            const int r0 = h * (dim + d.rot_dim);
            q.push_back({qn, r0, dim, dp});
            q.push_back({qn, r0 + dim, d.rot_dim, d.rp});
        }
        L.c0 = section(L, in, GEMM_ACT_NONE, g1);
        if (d.q_rank) {
            in.add(m + "dq", 0, d.q_rank, d.qp);
            FH_TRY(pack(&L.uq, q, d.q_rank));
            FH_TRY(vec(m + "dq.norm", {d.q_rank}, d.qp, &L.dq_norm));
        } else {
            for (const Rows& r : q) in.add(r.name, r.row0, r.rows, r.rows_pad);
        }
        if (!sp.kv_source) {
            L.c1 = in.cols();
            in.add(m + "dkv", 0, kr, d.kp);
            in.add(m + "dkv", kr, d.rot_dim, d.rp);
            FH_TRY(vec(m + "dkv.norm", {kr}, d.kp, &L.dkv_norm));
            FH_TRY(arena_.alloc(&L.lb.pool, (size_t)c_.kv_num_blocks * latent_block_elems(d)));
        }
        if (!(sp.attn_flags & FERRUM_HIP_ATTN_NO_HEAD_GATE)) {
            L.c2 = section(L, in, GEMM_ACT_SIGMOID, g1);
            in.add(m + "g", 0, H, pad32(H));
        }
        if (sp.attn_flags & FERRUM_HIP_ATTN_SINK) {
            float* sink = nullptr;
            FH_TRY(vec(m + "sink", {H}, H, &sink));
            L.lb.sink = sink;
        }
        // per head: W_ukᵀ [latent, plain query dims], W_uv [value dims, latent]
        FH_TRY(need(m + "uk", {(int64_t)H * dim, kr}));
        FH_TRY(need(m + "uv", {(int64_t)H * vd, kr}));
        FH_TRY(pack_fn(&L.uk, H, d.kp, dp, m + "uk", [&](const float* w, int g, int n, int k) {
            return n < kr && k < dim ? w[((size_t)g * dim + k) * kr + n] : 0.f; }));
        // [W_uk | W_uv] over the latent: the expansion of keys and values; its second part doubles as the per-head value projection
        const float *uk = data(m + "uk"), *uv = data(m + "uv");
        const int kn = H * dp;
        FH_TRY(pack_fn(&L.expand, 1, kn + H * vp, d.kp, m + "uv", [&](const float*, int, int n, int k) {
            if (k >= kr) return 0.f;
            if (n < kn) return n % dp < dim ? uk[((size_t)(n / dp) * dim + n % dp) * kr + k] : 0.f;
            n -= kn;
            return n % vp < vd ? uv[((size_t)(n / vp) * vd + n % vp) * kr + k] : 0.f; }));
        L.uv.w = L.expand.w + (size_t)kn * d.kp; L.uv.n = vp; L.uv.k = d.kp; L.uv.groups = H;
        FH_TRY(need(m + "o", {D_, (int64_t)H * vd}));
        // W_o, in a parallel block with a dense feed-forward behind W_down: [W_down | W_o]
        const bool glu = sp.ff == FERRUM_HIP_FF_CLAMPED_GLU;
        const std::string dn = m.substr(0, m.size() - 4) + "mlp.down";
        const int F = glu ? sp.ff_width : 0, Fp = pad32(F);
        if (glu) FH_TRY(need(dn, {D_, F}));
        const float* down = data(dn);
        FH_TRY(pack_fn(&L.o, 1, Dp_, Fp + H * vp, m + "o", [&](const float* w, int, int n, int k) {
            if (n >= D_) return 0.f;
            if (k < Fp) return k < F ? down[(size_t)n * F + k] : 0.f;
            k -= Fp;
            return k % vp < vd ? w[(size_t)n * H * vd + (k / vp) * vd + k % vp] : 0.f; }));
        return rope(sp, &L.lb.cos_t, &L.lb.sin_t);
    }
    int recurrent_weights(Layer& L, Input& in, const std::string& m) {
        const RglruDims& d = L.rd;
        const int W = L.s.rnn_width, bs = W / d.blocks, bp = d.bp;
        for (const char* part : {"y", "x"}) {
            (*part == 'y' ? L.c0 : L.c1) = section(L, in, *part == 'y' ? GEMM_ACT_GELU_TANH : GEMM_ACT_NONE);
            for (int g = 0; g < d.blocks; g++) in.add(m + part, g * bs, bs, bp, m + part + ".b");
        }
        FH_TRY(need(m + "ra", {d.blocks, bs, bs}));
        FH_TRY(need(m + "ri", {d.blocks, bs, bs}));
        // gate tiles: [block][16-channel tile][ra, ri] — packed as 2·bp rows per block in that order
        const float *ra = data(m + "ra"), *ri = data(m + "ri");
        Linear gates;
        FH_TRY(pack_fn(&gates, d.blocks, 2 * bp, bp, m + "ra", [&](const float*, int g, int n, int k) {
            const int ch = (n / 32) * 16 + n % 16;
            const float* w = (n / 16) % 2 ? ri : ra;
            return ch < bs && k < bs ? w[((size_t)g * bs + ch) * bs + k] : 0.f; }));
        L.rb.gate_w = gates.w;
        auto padded = [&](const std::string& name, const float** out, bool sp_fold, int taps) -> int {
            const int64_t n = W;
            if (taps > 1 || name == m + "conv") FH_TRY(need(name, {n, taps}));
            else if (name == m + "ra.b" || name == m + "ri.b") FH_TRY(need(name, {d.blocks, bs}));
            else FH_TRY(need(name, {n}));
            const float* src = data(name);
            std::vector<float> v((size_t)taps * d.wp, 0.f);
            for (int j = 0; j < taps; j++)
                for (int ch = 0; ch < W; ch++) {
                    const float x = src ? src[(size_t)ch * taps + j] : 0.25f;
                    v[(size_t)j * d.wp + (ch / bs) * bp + ch % bs] = sp_fold ? (float)softplus(x) : x;
                }
            float* dev = nullptr;
            FH_TRY(arena_.upload(&dev, v));
            *out = dev;
            return 0;
        };
        FH_TRY(padded(m + "conv", &L.rb.conv_w, false, d.taps));
        FH_TRY(padded(m + "conv.b", &L.rb.conv_b, false, 1));
        FH_TRY(padded(m + "ra.b", &L.rb.ra_b, false, 1));
        FH_TRY(padded(m + "ri.b", &L.rb.ri_b, false, 1));
        FH_TRY(padded(m + "lam", &L.rb.lam, true, 1));
        FH_TRY(need(m + "o", {D_, W}));
        FH_TRY(pack_fn(&L.o, 1, Dp_, d.wp, m + "o", [&](const float* w, int, int n, int k) {
            return n < D_ && k % bp < bs ? w[(size_t)n * W + (k / bp) * bs + k % bp] : 0.f; }));
        FH_TRY(arena_.alloc(&L.rb.conv_state, (size_t)slots_ * std::max(d.taps - 1, 1) * d.wp));
        FH_TRY(arena_.alloc(&L.rb.state, (size_t)slots_ * d.wp));
        return 0;
    }
    // grouped attention, linear attention, or the two side by side ("left", "right")
    int pair_weights(Layer& L, Input& in, const std::string& m, int li) {
        const FerrumHipLayerSpec& sp = L.s;
        const bool both = sp.mixer2 != 0, normed = both && sp.join == FERRUM_HIP_JOIN_NORMED_MEAN;
        const std::string a = both ? m + "left." : m, r = both ? m + "right." : m;
        const GroupedDims& g = L.gd;
        const LinearDims& n = L.nd;
        const int lin = linear_mixer(sp), np = passes(li);
        auto heads = [&](const std::string& name, int count, int rows, int pad, bool biased) {
            const int c = in.cols();
            for (int h = 0; h < count; h++) in.add(name, h * rows, rows, pad, biased ? name + ".b" : "");
            return c;
        };
        section(L, in, GEMM_ACT_NONE);
        if (g.heads) {
            const bool biased = sp.attn_flags & FERRUM_HIP_ATTN_QKV_BIAS;
            L.c0 = heads(a + "q", g.heads, g.dim, g.dp, biased);
            if (!sp.kv_source) {
                L.c1 = heads(a + "k", g.kv_heads, g.dim, g.dp, biased);
                L.c_v = heads(a + "v", g.kv_heads, g.vdim, g.vp, biased);
            }
        }
        if (lin) {
            L.c_q2 = heads(r + "q", n.heads, n.dim, n.dp, false);
            L.c_k2 = heads(r + "k", n.heads, n.dim, n.dp, false);
            L.c_v2 = heads(r + "v", n.heads, n.vdim, n.vp, false);
            if (lin == FERRUM_HIP_MIXER_GATED_LINEAR) {
                L.c_rank = in.cols();
                in.add(r + "a1", 0, sp.lin_rank, pad32(sp.lin_rank));
            }
        }
        if (g.heads && !(sp.attn_flags & FERRUM_HIP_ATTN_NO_HEAD_GATE)) {
            L.c2 = section(L, in, GEMM_ACT_SIGMOID);
            in.add(a + "g", 0, g.heads, pad32(g.heads));
        }
        if (g.heads && sp.attn_flags & FERRUM_HIP_ATTN_VALUE_GATE) {
            section(L, in, GEMM_ACT_SIGMOID);
            L.c_gate = heads(a + "g", g.heads, g.vdim, g.vp, false);
        }
        if (lin) {
            section(L, in, GEMM_ACT_SILU);
            L.c_g2 = heads(r + "g", n.heads, n.vdim, n.vp, false);
        }
        GroupedBuffers<E> gb;
        LinearBuffers<E> nb;
        if (g.heads) {
            float *qn = nullptr, *kn = nullptr, *v = nullptr;
            gb.head_norm = sp.attn_flags & FERRUM_HIP_ATTN_HEAD_NORM;
            FH_TRY(head_vec(a + "q.norm", gb.head_norm ? 1 : g.heads, g.dim, g.dp, &qn));
            if (!sp.kv_source) FH_TRY(head_vec(a + "k.norm", gb.head_norm ? 1 : g.kv_heads, g.dim, g.dp, &kn));
            gb.q_norm = qn; gb.k_norm = kn; gb.eps = c_.rms_eps;
            if (sp.attn_flags & FERRUM_HIP_ATTN_LOG_DISTANCE) {
                FH_TRY(vec(a + "r1", {g.heads}, g.heads, &v, 0.5f));
                gb.r1 = v;
                FH_TRY(vec(a + "r2", {g.heads}, g.heads, &v, 0.1f));
                gb.r2 = v;
            }
            if (sp.attn_flags & FERRUM_HIP_ATTN_SINK) {
                FH_TRY(vec(a + "sink", {g.heads}, g.heads, &v, 0.f));
                gb.sink = v;
            }
            if (sp.attn_flags & FERRUM_HIP_ATTN_TALK) {
                FH_TRY(matrix(a + "talk", g.heads, g.heads, g.heads, &v, 1.f));
                gb.talk = v;
            }
            if (sp.attn_flags & FERRUM_HIP_ATTN_OUT_BIAS) FH_TRY(vec(a + "o.b", {D_}, Dp_, &L.o_bias, 0.f));
            gb.mult = both && !normed ? sp.left_scale : 1.f;
            if (g.rot_dims) FH_TRY(rope(sp.rot_dims, sp.rot_base, sp, &gb.cos_t, &gb.sin_t));
            FH_TRY(need(a + "o", {D_, (int64_t)g.heads * g.vdim}));
        }
        if (lin) {
            nb.eps = c_.rms_eps;
            nb.mult = both && !normed ? sp.right_scale : 1.f;
            FH_TRY(need(r + "o", {D_, (int64_t)n.heads * n.vdim}));
            if (lin == FERRUM_HIP_MIXER_GATED_LINEAR) {
                float* w = nullptr;
                FH_TRY(vec(r + "norm", {n.vdim}, n.vp, &w));
                nb.norm = w;
                std::vector<Rows> rows;
                for (int h = 0; h < n.heads; h++) rows.push_back({r + "a2", h * n.dim, n.dim, n.dp});
                FH_TRY(pack(&L.decay, rows, sp.lin_rank));
                FH_TRY(bias(&L.decay, rows, std::vector<std::string>(n.heads, r + "a2.b")));
            } else {
                FH_TRY(need(r + "decay", {n.heads}));
                const float* d = data(r + "decay");
                std::vector<float> logs(n.heads);
                for (int h = 0; h < n.heads; h++) logs[h] = (float)log(d ? (double)d[h] : 1.0 - pow(2.0, -5.0 - h % 8));
                float* dev = nullptr;
                FH_TRY(arena_.upload(&dev, logs));
                nb.head_decay = dev;
                if (n.rot_dims) {
                    FerrumHipLayerSpec plain{};
                    FH_TRY(rope(n.rot_dims, sp.lin_rot_base, plain, &nb.cos_t, &nb.sin_t));
                }
            }
        }
        // W_o over the two results side by side, or each by itself where it is normed
        auto out = [&](Linear* w, bool left, bool right) {
            const int ka = left ? g.heads * g.vp : 0, kb = right ? n.heads * n.vp : 0;
            const float *wa = left ? data(a + "o") : nullptr, *wb = right ? data(r + "o") : nullptr;
            return pack_fn(w, 1, Dp_, ka + kb, "", [&](const float*, int, int row, int k) {
                if (row >= D_) return 0.f;
                if (k < ka) return k % g.vp < g.vdim ? wa[((size_t)row * g.heads + k / g.vp) * g.vdim + k % g.vp] : 0.f;
                k -= ka;
                return k % n.vp < n.vdim ? wb[((size_t)row * n.heads + k / n.vp) * n.vdim + k % n.vp] : 0.f; });
        };
        FH_TRY(out(&L.o, g.heads > 0, lin && !normed));
        if (normed) {
            FH_TRY(out(&L.o2, false, true));
            FH_TRY(vec(m + "left.out", {D_}, Dp_, &L.out1));
            FH_TRY(vec(m + "right.out", {D_}, Dp_, &L.out2));
        }
        for (int t = 0; t < np; t++) {
            if (g.heads && sp.kv_source) {
                gb.k_pool = layers_[sp.kv_source - 1].gb[0].k_pool;
                gb.v_pool = layers_[sp.kv_source - 1].gb[0].v_pool;
                L.gb.push_back(gb);
            } else if (g.heads) {
                FH_TRY(arena_.alloc(&gb.k_pool, (size_t)c_.kv_num_blocks * grouped_k_elems(g)));
                FH_TRY(arena_.alloc(&gb.v_pool, (size_t)c_.kv_num_blocks * grouped_v_elems(g)));
                L.gb.push_back(gb);
            }
            if (lin) {
                FH_TRY(arena_.alloc(&nb.state, (size_t)slots_ * n.heads * n.dp * n.vp));
                L.nb.push_back(nb);
            }
        }
        return 0;
    }
    int scan_weights(Layer& L, Input& in, const std::string& m, int li) {
        const FerrumHipLayerSpec& sp = L.s;
        const ScanDims& d = L.sd;
        const int W = sp.scan_inner, N = sp.scan_state, R = sp.scan_dt_rank, Rp = pad32(R), taps = sp.conv_taps;
        L.c0 = section(L, in, GEMM_ACT_NONE);
        in.add(m + "in", 0, W, d.wp);
        L.c1 = section(L, in, GEMM_ACT_SILU);
        in.add(m + "in", W, W, d.wp);
        FH_TRY(pack(&L.conv_in, {{m + "x", 0, R, Rp}, {m + "x", R, N, d.bc}, {m + "x", R + N, N, d.bc}}, W));
        std::vector<Rows> dt = {{m + "dt", 0, W, d.wp}};
        FH_TRY(pack(&L.dt, dt, R));
        FH_TRY(bias(&L.dt, dt, {m + "dt.b"}));
        FH_TRY(need(m + "conv", {W, taps}));
        FH_TRY(need(m + "A_log", {W, N}));
        FH_TRY(need(m + "o", {D_, W}));
        FH_TRY(pack(&L.o, {{m + "o", 0, D_, Dp_}}, W));
        ScanBuffers<E> b;
        float *cb = nullptr, *skip = nullptr, *dev = nullptr;
        FH_TRY(vec(m + "conv.b", {W}, d.wp, &cb));
        FH_TRY(vec(m + "D", {W}, d.wp, &skip));
        const float *conv = data(m + "conv"), *al = data(m + "A_log");
        std::vector<float> cw((size_t)taps * d.wp, 0.f), A((size_t)d.wp * d.sp, 0.f);
        for (int c = 0; c < W; c++) {
            for (int j = 0; j < taps; j++) cw[(size_t)j * d.wp + c] = conv ? conv[(size_t)c * taps + j] : 0.25f;
            for (int n = 0; n < N; n++) A[(size_t)c * d.sp + n] = (float)(-exp(al ? (double)al[(size_t)c * N + n] : log(1.0 + n)) * M_LOG2E);
        }
        FH_TRY(arena_.upload(&dev, cw));
        b.conv.w = dev;
        b.conv.b = cb; b.d = skip;
        FH_TRY(arena_.upload(&dev, A));
        b.a = dev;
        for (int t = 0; t < passes(li); t++) {
            FH_TRY(arena_.alloc(&b.conv.state, (size_t)slots_ * std::max(taps - 1, 1) * d.wp));
            FH_TRY(arena_.alloc(&b.state, (size_t)slots_ * d.wp * d.sp));
            L.sb.push_back(b);
        }
        return 0;
    }
    // the activations that the kernels of blocks with sublayers in turn read and write
    void wire(Layer& L) {
        const long ld = L.o.k + L.o2.k;
        for (GroupedBuffers<E>& b : L.gb) {
            b.q_in = in_ + L.c0; b.ld = L.ld_in;
            if (!L.s.kv_source) { b.k_in = in_ + L.c1; b.v_in = in_ + L.c_v; }
            if (L.s.attn_flags & FERRUM_HIP_ATTN_VALUE_GATE) { b.value_gate = in_ + L.c_gate; b.ld_value_gate = L.ld_in; }
            b.q = q_; b.out = attn_; b.ldo = ld; b.partial = partial_; b.partial_bytes = partial_bytes_; b.offset = talk_offset_;
            if (!(L.s.attn_flags & FERRUM_HIP_ATTN_NO_HEAD_GATE)) { b.gate = in_ + L.c2; b.ld_gate = L.ld_in; }
        }
        for (LinearBuffers<E>& b : L.nb) {
            b.q = in_ + L.c_q2; b.k = in_ + L.c_k2; b.v = in_ + L.c_v2; b.g = in_ + L.c_g2; b.ld = L.ld_in;
            if (L.decay.n) { b.log_decay = decay_; b.ld_decay = L.decay.n; }
            b.chunk_s = chunk_h_; b.chunk_b = chunk_a_;
            b.out = attn_ + L.gd.heads * L.gd.vp; b.ldo = ld;
        }
        for (ScanBuffers<E>& b : L.sb) {
            ShortConv<E>& c = b.conv;
            c.x = in_ + L.c0; c.ld = L.ld_in; c.out = u_; c.wp = L.sd.wp; c.taps = L.s.conv_taps; c.silu = true;
            b.low = cq_; b.ld_low = L.conv_in.n; b.c_b = pad32(L.s.scan_dt_rank);
            b.dt = decay_; b.z = in_ + L.c1; b.ld_z = L.ld_in; b.chunk_s = chunk_h_; b.chunk_dt = chunk_a_; b.out = attn_;
        }
    }
    int feed_forward_weights(Layer& L, Input& in, const std::string& p) {
        const FerrumHipLayerSpec& sp = L.s;
        const int F = sp.ff_width, Fp = pad32(F);
        if (sp.ff == FERRUM_HIP_FF_XIELU) {
            FH_TRY(unit_offset(p + "norm2", &L.norm2));
            std::vector<Rows> rows = {{p + "rg2", 0, D_, Dp_}, {p + "mlp.up", 0, F, Fp}};
            FH_TRY(pack(&L.ff_in, rows, D_));
            FH_TRY(bias(&L.ff_in, rows, {p + "rg2.b", ""}));
            FH_TRY(pack(&L.down, {{p + "mlp.down", 0, D_, Dp_}}, F));
            FH_TRY(need(p + "mlp.act", {2}));
            const float* act = data(p + "mlp.act");
            L.ff_sec[0] = {0, GEMM_ACT_SIGMOID, 0, 0};
            L.ff_sec[1] = {Dp_, GEMM_ACT_XIELU, (float)softplus(act ? act[0] : 0.5f), (float)softplus(act ? act[1] : 0.5f)};
        } else if (sp.ff == FERRUM_HIP_FF_CLAMPED_GLU) {
            // 16 gate columns, their 16 up columns, and so on; the down projection is part of the projection out
            L.c_glu = section(L, in, GEMM_ACT_CLAMPED_GLU, L.g2, sp.ff_limit, GLU_SLOPE);
            for (int f = 0; f < Fp; f += 16)
                for (const char* part : {"mlp.gate", "mlp.up"}) {
                    const int n = std::min(16, F - f);
                    in.add(p + part, n > 0 ? f : 0, std::max(n, 0), 16);
                }
            L.c_att = L.c_glu + Fp;
        } else if (sp.ff == FERRUM_HIP_FF_GELU_GLU) {
            Input f;
            for (int c = 0; c < Fp; c += 16)
                for (const char* part : {"mlp.gate", "mlp.up"}) {
                    const int n = std::min(16, F - c);
                    f.add(p + part, n > 0 ? c : 0, std::max(n, 0), 16, p + part + ".b");
                }
            FH_TRY(pack(&L.ff_in, f.rows, D_));
            FH_TRY(bias(&L.ff_in, f.rows, f.bias));
            L.ff_sec[0] = {0, GEMM_ACT_GELU_GLU, 0, 0};
            FH_TRY(pack(&L.down, {{p + "mlp.down", 0, D_, Dp_}}, F));
            FH_TRY(vec(p + "mlp.down.b", {D_}, Dp_, &L.down_bias, 0.f));
        } else if (sp.ff == FERRUM_HIP_FF_MOE_SILU_GLU || sp.ff == FERRUM_HIP_FF_MOE_CLAMPED_GLU) {
            const int routed = sp.experts + sp.identity_experts;
            FH_TRY(pack(&L.router, {{p + "mlp.router", 0, routed, pad32(routed)}}, D_));
            FH_TRY(vec(p + "mlp.correction", {routed}, routed, &L.correction, 0.f));
            L.ff_sec[0] = sp.ff == FERRUM_HIP_FF_MOE_SILU_GLU ? GemmSection{0, GEMM_ACT_SILU_GLU, 0, 0, L.g2} : GemmSection{0, GEMM_ACT_CLAMPED_GLU, sp.ff_limit, GLU_SLOPE, L.g2};
            if (const int S = sp.shared_width; S > 0) {
                const std::string x = p + "mlp.shared.";
                Input f;
                for (int c = 0; c < pad32(S); c += 16)
                    for (const char* part : {"gate", "up"}) f.add(x + part, c < S ? c : 0, std::max(std::min(16, S - c), 0), 16);
                L.shared_sec = {0, GEMM_ACT_CLAMPED_GLU, sp.shared_limit, GLU_SLOPE};
                FH_TRY(matrix(x + "sg", 1, D_, Dp_, &L.shared_gate));
                FH_TRY(pack(&L.shared_in, f.rows, D_));
                FH_TRY(pack(&L.shared_down, {{x + "down", 0, D_, Dp_}}, S));
            }
            std::vector<const float*> gate, up, down;
            for (int e = 0; e < sp.experts; e++) {
                const std::string x = p + "mlp.e" + std::to_string(e) + ".";
                FH_TRY(need(x + "gate", {F, D_}));
                FH_TRY(need(x + "up", {F, D_}));
                FH_TRY(need(x + "down", {D_, F}));
                gate.push_back(data(x + "gate"));
                up.push_back(data(x + "up"));
                down.push_back(data(x + "down"));
            }
            FH_TRY(pack_fn(&L.up, sp.experts, 2 * Fp, Dp_, "", [&](const float*, int g, int n, int k) {
                const int f = n / 32 * 16 + n % 16;
                return f < F && k < D_ ? (n / 16 % 2 ? up : gate)[g][(size_t)f * D_ + k] : 0.f; }));
            FH_TRY(pack_fn(&L.down, sp.experts, Dp_, Fp, "", [&](const float*, int g, int n, int k) { return n < D_ && k < F ? down[g][(size_t)n * F + k] : 0.f; }));
        } else if (sp.ff == FERRUM_HIP_FF_MOE_RELU2) {
            std::vector<Rows> r = {{p + "mlp.router", 0, sp.experts, pad32(sp.experts)}};
            FH_TRY(pack(&L.router, r, D_));
            FH_TRY(bias(&L.router, r, {p + "mlp.router.b"}));
            L.ff_sec[0] = {0, GEMM_ACT_RELU2, 0, 0, L.g2};
            std::vector<const float*> up, down;
            for (int e = 0; e < sp.experts; e++) {
                const std::string x = p + "mlp.e" + std::to_string(e) + ".";
                FH_TRY(need(x + "up", {F, D_}));
                FH_TRY(need(x + "down", {D_, F}));
                up.push_back(data(x + "up"));
                down.push_back(data(x + "down"));
            }
            FH_TRY(pack_fn(&L.up, sp.experts, Fp, Dp_, "", [&](const float*, int g, int n, int k) { return n < F && k < D_ ? up[g][(size_t)n * D_ + k] : 0.f; }));
            FH_TRY(pack_fn(&L.down, sp.experts, Dp_, Fp, "", [&](const float*, int g, int n, int k) { return n < D_ && k < F ? down[g][(size_t)n * F + k] : 0.f; }));
        }
        return 0;
    }
    int side_weights(Layer& L, const std::string& p, int li) {
        const int S = lc_.token_side_dim, Sp = pad32(S);
        FH_TRY(pack(&L.side_gate, {{p + "side.gate", 0, S, Sp}}, D_));
        FH_TRY(pack(&L.side_proj, {{p + "side.proj", 0, D_, Dp_}}, S));
        FH_TRY(vec(p + "side.norm", {D_}, Dp_, &L.side_norm));
        // this layer's columns of the side embedding as a table of its own
        return table("side.embed", c_.vocab, (int64_t)c_.num_layers * S, li * S, S, Sp, &L.side_table);
    }

    struct Rows { std::string name; int row0, rows, rows_pad; };      // a run of a matrix's rows, zero-padded
    // rows of a layer's input projection, each run with the name of its bias ("": none)
    struct Input {
        std::vector<Rows> rows;
        std::vector<std::string> bias;
        void add(const std::string& name, int row0, int n, int n_pad, const std::string& b = "") { rows.push_back({name, row0, n, n_pad}); bias.push_back(b); }
        int cols() const { int n = 0; for (const Rows& r : rows) n += r.rows_pad; return n; }
        bool biased() const { return std::any_of(bias.begin(), bias.end(), [](const std::string& b) { return !b.empty(); }); }
    };
    const float* data(const std::string& name) const {
        auto it = host_.find(name);
        return it == host_.end() ? nullptr : it->second.data.data();
    }
    int need(const std::string& name, const std::vector<int64_t>& shape) {
        if (synth_) return 0;
        auto it = host_.find(name);
        FH_REQUIRE(it != host_.end(), "layered model: tensor '%s' missing", name.c_str());
        FH_REQUIRE(it->second.shape == shape, "layered model: tensor '%s' has another shape than the configuration says", name.c_str());
        return 0;
    }
    int upload_tiles(Linear* L, int groups, int n, int k, const std::function<float(int, int, int)>& at) {
        L->n = n; L->k = k; L->groups = groups;
        const size_t total = (size_t)groups * n * k;
        if (synth_) {
            FH_TRY(arena_.alloc(&L->w, total));
            hipLaunchKernelGGL(synth_kernel<E>, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream_, L->w, total, mix(++seed_), 1.0f / sqrtf((float)k));
            FH_CHECK_LAUNCH();
            return 0;
        }
        std::vector<E> v(total);
        const int ks = k / 32;
        for (int g = 0; g < groups; g++)
            for (int r = 0; r < n; r++)
                for (int c = 0; c < k; c++) {
                    const size_t o = ((((size_t)g * (n / 16) + r / 16) * ks + c / 32) * 64 + ((c % 32) / 8) * 16 + r % 16) * 8 + c % 8;
                    store(&v[o], at(g, r, c));
                }
        return arena_.upload(&L->w, v);
    }
    static uint64_t mix(uint64_t x) { return x * 0x9E3779B97F4A7C15ull ^ (x >> 7); }
    int pack_fn(Linear* L, int groups, int n, int k, const std::string& name, const std::function<float(const float*, int, int, int)>& at) {
        const float* w = data(name);
        return upload_tiles(L, groups, n, k, [&](int g, int r, int c) { return at(w, g, r, c); });
    }
    // rows of several matrices, all with `cols` input columns, one below the other
    int pack(Linear* L, const std::vector<Rows>& runs, int cols) {
        std::vector<const float*> row;
        for (const Rows& r : runs) {
            if (!synth_) {
                auto it = host_.find(r.name);
                FH_REQUIRE(it != host_.end(), "layered model: tensor '%s' missing", r.name.c_str());
                const std::vector<int64_t>& sh = it->second.shape;
                FH_REQUIRE(sh.size() == 2 && sh[1] == cols && sh[0] == full_rows(r.name, runs), "layered model: tensor '%s' has another shape than the configuration says", r.name.c_str());
            }
            const float* w = data(r.name);
            for (int i = 0; i < r.rows_pad; i++) row.push_back(w && i < r.rows ? w + (size_t)(r.row0 + i) * cols : nullptr);
        }
        return upload_tiles(L, 1, (int)row.size(), pad32(cols), [&](int, int r, int c) { return row[r] && c < cols ? row[r][c] : 0.f; });
    }
    static int64_t full_rows(const std::string& name, const std::vector<Rows>& runs) {
        int64_t n = 0;
        for (const Rows& r : runs) if (r.name == name) n = std::max<int64_t>(n, r.row0 + r.rows);
        return n;
    }
    int bias(Linear* L, const std::vector<Rows>& runs, const std::vector<std::string>& names) {
        std::vector<float> v;
        for (size_t i = 0; i < runs.size(); i++) {
            if (!names[i].empty()) FH_TRY(need(names[i], {full_rows(runs[i].name, runs)}));
            const float* b = names[i].empty() ? nullptr : data(names[i]);
            for (int r = 0; r < runs[i].rows_pad; r++) v.push_back(b && r < runs[i].rows ? b[runs[i].row0 + r] : 0.f);
        }
        return arena_.upload(&L->bias, v);
    }
    int vec(const std::string& name, const std::vector<int64_t>& shape, int n_pad, float** out, float synth = 1.f) {
        FH_TRY(need(name, shape));
        std::vector<float> v(n_pad, 0.f);
        const float* w = data(name);
        for (int64_t i = 0; i < shape[0]; i++) v[i] = w ? w[i] : synth;
        return arena_.upload(out, v);
    }
    // a vector over heads of `dim`, each padded to `pad`
    int head_vec(const std::string& name, int heads, int dim, int pad, float** out) {
        FH_TRY(need(name, {(int64_t)heads * dim}));
        std::vector<float> v((size_t)heads * pad, 0.f);
        const float* w = data(name);
        for (int i = 0; i < heads * dim; i++) v[(size_t)(i / dim) * pad + i % dim] = w ? w[i] : 1.f;
        return arena_.upload(out, v);
    }
    // fp32 rows, padded; synthetic: `diagonal` times the unit matrix
    int matrix(const std::string& name, int rows, int cols, int pad, float** out, float diagonal = 0.f) {
        FH_TRY(need(name, {rows, cols}));
        std::vector<float> v((size_t)rows * pad, 0.f);
        const float* w = data(name);
        for (int r = 0; r < rows; r++)
            for (int i = 0; i < cols; i++) v[(size_t)r * pad + i] = w ? w[(size_t)r * cols + i] : r == i ? diagonal : 0.f;
        return arena_.upload(out, v);
    }
    int unit_offset(const std::string& name, float** out) {        // stored around zero: 1 + w
        FH_TRY(need(name, {D_}));
        std::vector<float> v(pad32(D_), 0.f);
        const float* w = data(name);
        for (int i = 0; i < D_; i++) v[i] = 1.f + (w ? w[i] : 0.f);
        return arena_.upload(out, v);
    }
    int scalar(const std::string& name, float* out) {
        FH_TRY(need(name, {1}));
        const float* w = data(name);
        *out = w ? w[0] : 1.f;
        return 0;
    }
    int table(const std::string& name, int rows, E** out) { return table(name, rows, D_, 0, D_, D_, out); }
    // columns [col0, col0 + n) of a table of `cols` columns, rows padded to n_pad
    int table(const std::string& name, int rows, int64_t cols, int64_t col0, int n, int n_pad, E** out) {
        FH_TRY(need(name, {rows, cols}));
        const size_t total = (size_t)rows * n_pad;
        if (synth_) {
            FH_TRY(arena_.alloc(out, total));
            hipLaunchKernelGGL(synth_kernel<E>, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream_, *out, total, mix(++seed_), 1.0f);
            FH_CHECK_LAUNCH();
            return 0;
        }
        std::vector<E> v(total);
        const float* w = data(name);
        for (int r = 0; r < rows; r++)
            for (int i = 0; i < n_pad; i++) store(&v[(size_t)r * n_pad + i], i < n ? w[(size_t)r * cols + col0 + i] : 0.f);
        return arena_.upload(out, v);
    }
    // angle tables in double, stored fp32 like the other models'; layers with the same rotation share one
    int rope(const FerrumHipLayerSpec& sp, const float** cos_t, const float** sin_t) { return rope(sp.rot_dims, sp.rot_base, sp, cos_t, sin_t); }
    // (sp: the scaling)
    int rope(int dims, double base, const FerrumHipLayerSpec& sp, const float** cos_t, const float** sin_t) {
        const int half = dims / 2;
        for (const Rope& r : ropes_)
            if (r.dims == dims && r.base == base && r.factor == sp.rot_factor && r.original == sp.rot_original && r.fast == sp.rot_fast && r.slow == sp.rot_slow) {
                *cos_t = r.c; *sin_t = r.s;
                return 0;
            }
        std::vector<double> freq(half);
        for (int i = 0; i < half; i++) freq[i] = pow(base, -2.0 * i / dims);
        double size = 1.0;
        if (sp.rot_factor > 0.0) {
            // pair (not rounded) that turns `turns` times within the original length
            auto pair_of = [&](double turns) { return dims * log(sp.rot_original / (2.0 * M_PI * turns)) / (2.0 * log(base)); };
            const double lo = std::max(floor(pair_of(sp.rot_fast)), 0.0), hi = std::min(ceil(pair_of(sp.rot_slow)), dims - 1.0);
            for (int i = 0; i < half; i++) {
                const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
                freq[i] = freq[i] / sp.rot_factor * ramp + freq[i] * (1.0 - ramp);
            }
            size = 0.1 * log(sp.rot_factor) + 1.0;
        }
        std::vector<float> cs((size_t)c_.max_seq_len * half), sn(cs.size());
        for (int p = 0; p < c_.max_seq_len; p++)
            for (int i = 0; i < half; i++) {
                const double a = (double)p * freq[i];
                cs[(size_t)p * half + i] = (float)(size * cos(a));
                sn[(size_t)p * half + i] = (float)(size * sin(a));
            }
        Rope r{base, sp.rot_factor, sp.rot_original, sp.rot_fast, sp.rot_slow, dims, nullptr, nullptr};
        FH_TRY(arena_.upload(&r.c, cs));
        FH_TRY(arena_.upload(&r.s, sn));
        ropes_.push_back(r);
        *cos_t = r.c; *sin_t = r.s;
        return 0;
    }
    struct Rope { double base, factor, original, fast, slow; int dims; float *c, *s; };

    FerrumHipModelConfig c_;
    FerrumHipLayeredConfig lc_;
    int slots_, D_, Dp_;
    hipStream_t stream_ = nullptr, side_stream_ = nullptr;
    hipEvent_t fork_ = nullptr, join_ = nullptr;
    bool synth_ = false;
    uint64_t seed_ = 0;
    Arena arena_;
    std::unordered_map<std::string, HostTensor> host_;
    std::vector<Layer> layers_;
    std::vector<Rope> ropes_;
    Linear head_, loop_in_;
    float *loop_step_ = nullptr, *sub2_ = nullptr;
    E* cat_ = nullptr;           // [T][stream | embedding], ahead of a pass
    E *embed_ = nullptr, *bigram_ = nullptr, *positions_ = nullptr;
    float* final_norm_ = nullptr;
    // activations of one forward
    float *x_ = nullptr, *sub_ = nullptr, *partial_ = nullptr, *talk_offset_ = nullptr, *row_gate_ = nullptr, *decay_ = nullptr, *drive_ = nullptr, *chunk_a_ = nullptr, *chunk_h_ = nullptr;
    E *xb_ = nullptr, *in_ = nullptr, *cq_ = nullptr, *q_ = nullptr, *q_lat_ = nullptr, *o_lat_ = nullptr, *attn_ = nullptr, *u_ = nullptr,
      *rnn_out_ = nullptr, *head_in_ = nullptr, *side_ = nullptr, *expert_h_ = nullptr, *expert_y_ = nullptr;
    float *router_logits_ = nullptr, *expert_weights_ = nullptr;
    int32_t *expert_ids_ = nullptr, *sorted_ = nullptr, *sorted_expert_ = nullptr, *sorted_total_ = nullptr;
    size_t partial_bytes_ = 0;
    // expansion of keys and values: one plan per distinct window
    std::vector<Plan> plans_;
    int32_t *plan_host_ = nullptr, *plan_dev_ = nullptr;
    size_t plan_used_ = 0;
    int expand_blocks_ = 0;
    E* expanded_ = nullptr;
};

}  // namespace

// a layer of a block whose sublayers follow one another (pre-norm, post-norm)
static int check_in_turn_layer(const FerrumHipLayeredConfig& lc, const FerrumHipLayerSpec* layers, int i) {
    const FerrumHipLayerSpec& s = layers[i];
    const bool post = lc.block == FERRUM_HIP_BLOCK_POST_NORM;
    auto rotated = [](int dims, int of, double base) { return dims >= 0 && dims % 2 == 0 && dims <= of && (dims == 0 || base > 0.0); };
    const bool attention = s.mixer == FERRUM_HIP_MIXER_GROUPED_ATTENTION;
    const int lin = s.mixer2 ? s.mixer2 : attention || s.mixer == FERRUM_HIP_MIXER_SELECTIVE_SCAN ? 0 : s.mixer;
    if (!(attention || s.mixer == FERRUM_HIP_MIXER_SELECTIVE_SCAN || s.mixer == FERRUM_HIP_MIXER_GATED_LINEAR || s.mixer == FERRUM_HIP_MIXER_RETENTION) ||
        !(lin == 0 || lin == FERRUM_HIP_MIXER_GATED_LINEAR || lin == FERRUM_HIP_MIXER_RETENTION)) {
        set_error("layer %d: mixers %d and %d in a pre-norm block", i, s.mixer, s.mixer2);
        return FERRUM_HIP_UNSUPPORTED;
    }
    FH_REQUIRE(!s.mixer2 || (attention && (s.join == FERRUM_HIP_JOIN_SCALED || s.join == FERRUM_HIP_JOIN_NORMED_MEAN)), "layer %d: mixers %d and %d side by side", i, s.mixer, s.mixer2);
    if (attention) {
        FH_REQUIRE(s.heads > 0 && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.vdim > 0 && (s.window > 0 || s.window == FERRUM_HIP_WINDOW_NONE),
                   "layer %d: attention of %d heads on %d, %d / %d dimensions, window %d", i, s.heads, s.kv_heads, s.dim, s.vdim, s.window);
        FH_REQUIRE(rotated(s.rot_dims, s.dim, s.rot_base) && s.rot_factor == 0.0, "layer %d: rotated dimensions %d of %d", i, s.rot_dims, s.dim);
        FH_REQUIRE(!(s.attn_flags & FERRUM_HIP_ATTN_VALUE_GATE) || s.attn_flags & FERRUM_HIP_ATTN_NO_HEAD_GATE, "layer %d: gates per head and per value element share a tensor name", i);
        FH_REQUIRE(!(s.attn_flags & FERRUM_HIP_ATTN_TALK) || !(s.attn_flags & FERRUM_HIP_ATTN_LOG_DISTANCE), "layer %d: mixed heads take scores without a distance", i);
        FH_REQUIRE(!s.mixer2 || !(s.attn_flags & (FERRUM_HIP_ATTN_VALUE_GATE | FERRUM_HIP_ATTN_OUT_BIAS)), "layer %d: value gates and output bias beside a second mixer", i);
        if (s.kv_source) {
            FH_REQUIRE(s.kv_source > 0 && s.kv_source <= i && !lc.loop_times && !s.mixer2 && s.attn_flags & FERRUM_HIP_ATTN_HEAD_NORM, "layer %d: reads the keys of layer %d", i,
                       s.kv_source - 1);
            const FerrumHipLayerSpec& o = layers[s.kv_source - 1];
            FH_REQUIRE(o.mixer == s.mixer && !o.kv_source && o.kv_heads == s.kv_heads && o.dim == s.dim && o.vdim == s.vdim,
                       "layer %d: layer %d caches other keys, or none of its own", i, s.kv_source - 1);
        }
    }
    if (lin) {
        FH_REQUIRE(s.lin_heads > 0 && s.lin_dim > 0 && s.lin_vdim > 0 && linear_supports(s.lin_dim, s.lin_vdim), "layer %d: linear attention of %d heads, a state of %d x %d",
                   i, s.lin_heads, s.lin_dim, s.lin_vdim);
        FH_REQUIRE(lin != FERRUM_HIP_MIXER_GATED_LINEAR || (s.lin_rank > 0 && s.lin_tau > 0.f), "layer %d: decay of rank %d, tau %g", i, s.lin_rank, s.lin_tau);
        FH_REQUIRE(lin != FERRUM_HIP_MIXER_RETENTION || rotated(s.lin_rot_dims, s.lin_dim, s.lin_rot_base), "layer %d: rotated dimensions %d of %d", i, s.lin_rot_dims, s.lin_dim);
    }
    FH_REQUIRE(s.mixer != FERRUM_HIP_MIXER_SELECTIVE_SCAN || (s.scan_inner > 0 && s.scan_state > 0 && s.scan_state <= SCAN_MAX_STATE && s.scan_dt_rank > 0 && s.conv_taps > 0),
               "layer %d: scan of %d channels, %d states, rank %d, %d taps", i, s.scan_inner, s.scan_state, s.scan_dt_rank, s.conv_taps);
    const bool silu = s.ff == FERRUM_HIP_FF_MOE_SILU_GLU, clamped = s.ff == FERRUM_HIP_FF_MOE_CLAMPED_GLU;
    FH_REQUIRE(s.ff == FERRUM_HIP_FF_NONE || ((s.ff == FERRUM_HIP_FF_GELU_GLU || silu || clamped) && s.ff_width > 0), "layer %d: feed-forward %d of width %d", i, s.ff, s.ff_width);
    MoeCorrectedRule rule{nullptr, s.route_groups, s.route_keep, s.route_scale};
    rule.unlisted = s.identity_experts;
    FH_REQUIRE(!(silu || clamped) || (s.experts > 0 && s.identity_experts >= 0 && moe_route_corrected_supports(s.experts + s.identity_experts, s.top, rule)),
               "layer %d: %d of %d experts from %d of %d groups", i, s.top, s.experts + s.identity_experts, s.route_keep, s.route_groups);
    // (the copies of the input and the shared expert's factor are part of the post-norm block's sums)
    FH_REQUIRE(clamped ? s.shared_width >= 0 && (post || (!s.identity_experts && !s.shared_width)) : !s.identity_experts && !s.shared_width,
               "layer %d: %d identity experts, a shared expert of width %d", i, s.identity_experts, s.shared_width);
    return 0;
}

int check_layered_config(const FerrumHipModelConfig& c, const FerrumHipLayeredConfig& lc, const FerrumHipLayerSpec* layers) {
    FH_REQUIRE(c.num_layers > 0 && c.hidden > 0 && c.vocab > 0, "layered model: layers=%d hidden=%d vocab=%d", c.num_layers, c.hidden, c.vocab);
    FH_REQUIRE(c.max_seqs > 0 && c.max_tokens >= c.max_seqs && c.kv_num_blocks > 0 && c.max_seq_len > 0,
               "layered model: max_seqs/max_tokens/kv_num_blocks/max_seq_len must be positive");
    FH_REQUIRE(c.tp_world <= 1, "layered model: tensor parallelism is not available");
    FH_REQUIRE(lc.dtype == FERRUM_HIP_DTYPE_BF16 || lc.dtype == FERRUM_HIP_DTYPE_F32, "layered model: dtype %d", lc.dtype);
    FH_REQUIRE(lc.bigram_buckets >= 0 && lc.state_slots >= 0, "layered model: bigram buckets %d, state slots %d", lc.bigram_buckets, lc.state_slots);
    FH_REQUIRE(lc.block == FERRUM_HIP_BLOCK_GATED_POST_NORM || lc.block == FERRUM_HIP_BLOCK_PARALLEL_PRE_NORM || lc.block == FERRUM_HIP_BLOCK_PRE_NORM ||
                   lc.block == FERRUM_HIP_BLOCK_POST_NORM,
               "layered model: block %d", lc.block);
    const bool pre_norm = lc.block == FERRUM_HIP_BLOCK_PRE_NORM, in_turn = pre_norm || lc.block == FERRUM_HIP_BLOCK_POST_NORM;
    FH_REQUIRE(lc.position_rows == 0 || lc.position_rows >= c.max_seq_len, "layered model: %d learned positions for sequences of %d tokens", lc.position_rows, c.max_seq_len);
    FH_REQUIRE(lc.logit_softcap >= 0.f, "layered model: logits capped at %g", lc.logit_softcap);
    FH_REQUIRE(lc.loop_times == 0 || (pre_norm && lc.loop_times > 0 && lc.loop_start >= 0 && lc.loop_start < lc.loop_stop && lc.loop_stop <= c.num_layers),
               "layered model: layers %d to %d, %d times", lc.loop_start, lc.loop_stop, lc.loop_times);
    FH_REQUIRE(!in_turn || (!lc.bigram_buckets && lc.untied_head), "layered model: a pre-norm or post-norm block takes plain embeddings and a vocabulary projection of its own");
    const bool parallel = lc.block == FERRUM_HIP_BLOCK_PARALLEL_PRE_NORM;
    FH_REQUIRE(lc.token_side_dim >= 0 && (parallel || !lc.token_side_dim), "layered model: per-layer token input of %d dimensions", lc.token_side_dim);
    for (int i = 0; i < c.num_layers; i++) {
        const FerrumHipLayerSpec& s = layers[i];
        if (in_turn) {
            if (int rc = check_in_turn_layer(lc, layers, i)) return rc;
            continue;
        }
        FH_REQUIRE(!s.mixer2, "layer %d: two mixers side by side need a pre-norm or post-norm block", i);
        if (s.mixer == FERRUM_HIP_MIXER_LATENT_ATTENTION) {
            FH_REQUIRE(s.heads > 0 && s.dim > 0 && s.rot_dim > 0 && s.vdim > 0 && s.q_rank >= 0 && s.kv_rank > 0 && (s.window > 0 || s.window == FERRUM_HIP_WINDOW_NONE),
                       "layer %d: latent attention sizes must be positive", i);
            FH_REQUIRE(s.rot_dims >= 0 && s.rot_dims % 2 == 0 && s.rot_dims <= s.rot_dim && (s.rot_dims == 0 || s.rot_base > 0.0),
                       "layer %d: rotated dimensions %d of %d", i, s.rot_dims, s.rot_dim);
            FH_REQUIRE(s.rot_factor == 0.0 || (s.rot_factor > 0.0 && s.rot_original > 0.0 && s.rot_fast > 0.0 && s.rot_slow > 0.0 && s.rot_base > 0.0 && s.rot_base != 1.0),
                       "layer %d: rotation scaling", i);
            if (s.kv_source) {
                FH_REQUIRE(s.kv_source > 0 && s.kv_source <= i, "layer %d: reads the latents of layer %d", i, s.kv_source - 1);
                const FerrumHipLayerSpec& o = layers[s.kv_source - 1];
                FH_REQUIRE(o.mixer == s.mixer && !o.kv_source && o.kv_rank == s.kv_rank && o.rot_dim == s.rot_dim,
                           "layer %d: layer %d caches other latents, or none of its own", i, s.kv_source - 1);
            }
        } else if (s.mixer == FERRUM_HIP_MIXER_RGLRU) {
            FH_REQUIRE(s.rnn_width > 0 && s.rnn_blocks > 0 && s.rnn_width % s.rnn_blocks == 0 && s.conv_taps > 0,
                       "layer %d: recurrence of width %d in %d blocks, %d taps", i, s.rnn_width, s.rnn_blocks, s.conv_taps);
        } else {
            set_error("layer %d: unknown mixer %d", i, s.mixer);
            return FERRUM_HIP_UNSUPPORTED;
        }
        FH_REQUIRE(s.ff == FERRUM_HIP_FF_NONE || ((s.ff == FERRUM_HIP_FF_CLAMPED_GLU || s.ff == FERRUM_HIP_FF_MOE_RELU2 ? parallel : s.ff == FERRUM_HIP_FF_XIELU && !parallel) && s.ff_width > 0),
                   "layer %d: feed-forward %d of width %d", i, s.ff, s.ff_width);
        FH_REQUIRE(s.ff != FERRUM_HIP_FF_MOE_RELU2 || (s.experts > 0 && s.experts <= 512 && s.top > 0 && s.top <= s.experts && s.top <= 64),
                   "layer %d: %d of %d experts", i, s.top, s.experts);
        FH_REQUIRE(!parallel || s.mixer == FERRUM_HIP_MIXER_LATENT_ATTENTION, "layer %d: a parallel block takes latent attention", i);
    }
    return 0;
}

std::unique_ptr<LayeredModel> make_layered_model(const FerrumHipModelConfig& c, const FerrumHipLayeredConfig& lc, const FerrumHipLayerSpec* layers,
                                                 int state_slots) {
    if (lc.dtype == FERRUM_HIP_DTYPE_F32) return std::make_unique<Layered<float>>(c, lc, layers, state_slots);
    return std::make_unique<Layered<bf16>>(c, lc, layers, state_slots);
}

}  // namespace fh
