// Replays a token trace: given ids go through the model step by step, logits at the requested places come out.  Nothing is sampled.
// A thin driver over include/ferrum_hip.h — the step is ferrum_hip_model_unified_forward_rows, the engine's own mixed batch.
//
//   ferrum_hip_trace --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
// stdin, one JSON object a line: {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}; for every step that wants logits
// DIR/<step>.f32 receives [wanted, vocab] little-endian floats, in the order of the entries; "done <step>" follows on stdout.
// Exit code 3: --dtype float32 for a model that only runs in 16 bits.
#include <cstdint>
#include <cstdio>
#include <cstring>
#include <iostream>
#include <map>
#include <string>
#include <vector>

#include "../../include/ferrum_hip.h"
#include "json.h"

namespace {

using fh::json::Value;

constexpr int LIVE_REQUESTS = 4;
constexpr int BLOCK = 16;

int fail(const char* what) {
    std::fprintf(stderr, "%s: %s\n", what, ferrum_hip_last_error());
    return 1;
}

struct Live { uint64_t seq; int len; };

const char* arg(int argc, char** argv, const char* name) {
    for (int i = 1; i + 1 < argc; i++)
        if (!std::strcmp(argv[i], name)) return argv[i + 1];
    return nullptr;
}

bool int_list(const Value* v, std::vector<int64_t>& out) {
    out.clear();
    if (!v) return true;
    if (v->kind != Value::Arr) return false;
    for (const Value& x : v->arr) {
        if (!x.is_u64()) return false;
        out.push_back((int64_t)x.num);
    }
    return true;
}

}  // namespace

int main(int argc, char** argv) {
    const char *dir = arg(argc, argv, "--model"), *dtype = arg(argc, argv, "--dtype"), *out = arg(argc, argv, "--out"), *max_tok = arg(argc, argv, "--max-tokens");
    const bool f32 = dtype && !std::strcmp(dtype, "float32");
    const int max_tokens = max_tok ? std::atoi(max_tok) : 0;
    if (!dir || !out || !dtype || (!f32 && std::strcmp(dtype, "bfloat16")) || max_tokens < 1) {
        std::fprintf(stderr, "usage: %s --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N\n", argv[0]);
        return 2;
    }
    FerrumHipCheckpoint* ck = nullptr;
    if (ferrum_hip_checkpoint_open(&ck, dir)) return fail("checkpoint");
    const int capacity = (max_tokens + BLOCK - 1) / BLOCK * BLOCK;
    FerrumHipModelConfig cfg;
    int layered = 0;
    if (ferrum_hip_checkpoint_model_config(ck, capacity, &cfg, nullptr, 0, nullptr)) return fail("configuration");
    FerrumHipLayeredConfig lc;
    std::vector<FerrumHipLayerSpec> specs((size_t)cfg.num_layers);
    if (ferrum_hip_checkpoint_layered_config(ck, &layered, &lc, specs.data(), cfg.num_layers)) return fail("configuration");
    if (f32 && !layered) {
        std::fprintf(stderr, "this architecture runs in 16 bits only\n");
        return 3;
    }
    cfg.kv_num_blocks = capacity / BLOCK;
    cfg.max_seqs = LIVE_REQUESTS;
    cfg.max_tokens = capacity < LIVE_REQUESTS ? LIVE_REQUESTS : capacity;
    FerrumHipModel* model = nullptr;
    if (layered) {
        lc.dtype = f32 ? FERRUM_HIP_DTYPE_F32 : FERRUM_HIP_DTYPE_BF16;
        lc.state_slots = LIVE_REQUESTS;
        if (ferrum_hip_model_create_layered(&model, &cfg, &lc, specs.data())) return fail("model");
    } else if (ferrum_hip_model_create(&model, &cfg)) {
        return fail("model");
    }
    if (ferrum_hip_model_load_checkpoint(model, ck)) return fail("weights");
    if (ferrum_hip_model_finalize(model)) return fail("finalize");
    ferrum_hip_checkpoint_close(ck);

    std::map<std::string, Live> live;
    uint64_t next_seq = 1;
    std::string line;
    while (std::getline(std::cin, line)) {
        if (line.find_first_not_of(" \t\r\n") == std::string::npos) continue;
        Value step;
        std::string err;
        if (!fh::json::parse(line.data(), line.size(), step, err) || step.kind != Value::Obj || !step.get("step") || !step.get("step")->is_u64()) {
            std::fprintf(stderr, "bad step: %s\n", err.c_str());
            return 2;
        }
        const long long number = (long long)step.get("step")->num;
        std::vector<FerrumHipBatchItem> items;
        std::vector<std::vector<uint32_t>> tokens;
        std::vector<std::string> ids;
        std::vector<int32_t> rows;
        std::vector<int64_t> ints;
        int at = 0;
        const Value* entries = step.get("entries");
        const size_t n = entries && entries->kind == Value::Arr ? entries->arr.size() : 0;
        tokens.reserve(n);
        for (size_t i = 0; i < n; i++) {
            const Value& e = entries->arr[i];
            const Value* id = e.get("id");
            if (!id || id->kind != Value::Str || !int_list(e.get("tokens"), ints)) { std::fprintf(stderr, "bad entry in step %lld\n", number); return 2; }
            if (ints.empty()) continue;
            tokens.emplace_back(ints.begin(), ints.end());
            auto it = live.find(id->str);
            if (it == live.end()) it = live.emplace(id->str, Live{next_seq++, 0}).first;
            FerrumHipBatchItem item;
            std::memset(&item, 0, sizeof(item));
            item.seq_id = it->second.seq;
            item.q_tokens = tokens.back().data();
            item.num_q_tokens = (int)tokens.back().size();
            item.pos_offset = it->second.len;
            items.push_back(item);
            it->second.len += item.num_q_tokens;
            if (!int_list(e.get("want"), ints)) { std::fprintf(stderr, "bad entry in step %lld\n", number); return 2; }
            for (int64_t w : ints) {
                if (w >= item.num_q_tokens) { std::fprintf(stderr, "step %lld asks for place %lld of %d tokens\n", number, (long long)w, item.num_q_tokens); return 2; }
                rows.push_back(at + (int32_t)w);
            }
            at += item.num_q_tokens;
        }
        if (!items.empty()) {
            std::vector<float> logits(rows.size() * (size_t)cfg.vocab);
            if (ferrum_hip_model_unified_forward_rows(model, items.data(), (int)items.size(), rows.data(), (int)rows.size(), logits.data())) return fail("step");
            if (!rows.empty()) {
                const std::string path = std::string(out) + "/" + std::to_string(number) + ".f32";
                FILE* f = std::fopen(path.c_str(), "wb");
                if (!f || std::fwrite(logits.data(), 4, logits.size(), f) != logits.size() || std::fclose(f)) { std::perror(path.c_str()); return 1; }
            }
        }
        if (const Value* end = step.get("end"); end && end->kind == Value::Arr)
            for (const Value& id : end->arr)
                if (auto it = live.find(id.str); it != live.end()) {
                    if (ferrum_hip_model_release(model, it->second.seq)) return fail("release");
                    live.erase(it);
                }
        std::printf("done %lld\n", number);
        std::fflush(stdout);
    }
    return ferrum_hip_model_destroy(model) ? fail("destroy") : 0;
}
