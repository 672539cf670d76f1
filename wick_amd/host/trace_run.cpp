// Replays a trace of token ids through a model folder and writes the logits that are asked for: a step a line of JSON on standard
// input, {"step": n, "entries": [{"id": .., "tokens": [..], "want": [..]}], "end": [..]}, answered by "done n" and, when something is
// wanted, DIR/n.f32 ([wanted][vocab] little-endian floats).  The model handle holds one sequence's state; requests that take turns
// are switched by state snapshots.
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <iostream>
#include <map>
#include <string>
#include <vector>

#include "../../include/wick_rocm_model.h"
#include "../../include/wick_safetensors.h"
#include "../csrc/json.h"

using wick_rocm::Json;
using wick_rocm::JsonParser;

namespace {

[[noreturn]] void die(const std::string& what) {
    std::fprintf(stderr, "trace_run: %s\n", what.c_str());
    std::exit(1);
}

struct Request {
    uint32_t pos = 0;
    std::vector<char> state;  // of a request that waits its turn
};

struct Runner {
    wick_rocm_ctx* ctx = nullptr;
    wick_rocm_model* model = nullptr;
    wick_rocm_model_info info{};
    std::map<std::string, Request> live;
    std::string current;  // whose state the handle holds ("" : nobody's)

    void check(int rc, const char* where) {
        if (rc == WICK_ROCM_OK) return;
        char msg[512] = "";
        if (ctx) wick_rocm_last_error(ctx, msg, sizeof msg);
        die(std::string(where) + ": " + msg + " (status " + std::to_string(rc) + ")");
    }
    // Makes `id` the request whose state the handle holds.
    Request& turn(const std::string& id) {
        Request& r = live[id];
        if (id == current) return r;
        const auto was = live.find(current);
        if (was != live.end() && was->second.pos) {
            Request& w = was->second;
            w.state.resize(wick_rocm_model_state_bytes(model, w.pos));
            check(wick_rocm_model_snapshot_state(ctx, model, w.pos, w.state.data(), w.state.size()), "snapshot");
        }
        if (r.pos)
            check(wick_rocm_model_restore_state(ctx, model, r.pos, r.state.data(), r.state.size()), "restore");
        else
            check(wick_rocm_model_reset(ctx, model), "reset");
        std::vector<char>().swap(r.state);
        current = id;
        return r;
    }
    void finish(const std::string& id) {
        live.erase(id);
        if (id == current) current.clear();
    }
};

std::vector<uint32_t> ids(const Json* j, const char* what) {
    std::vector<uint32_t> v;
    if (!j || j->kind != Json::kArray) die(std::string("a step without ") + what);
    for (const Json& e : j->items) {
        if (e.kind != Json::kNumber || e.number < 0 || e.number > 4294967295.0) die(std::string("bad number in ") + what);
        v.push_back((uint32_t)e.number);
    }
    return v;
}

std::string name_of(const Json& j) {
    if (j.kind == Json::kString) return j.string;
    if (j.kind == Json::kNumber) return std::to_string(j.number);
    die("a request id is neither a string nor a number");
}

}  // namespace

int main(int argc, char** argv) {
    std::string dir, dtype = "bfloat16", out;
    unsigned long max_tokens = 4096;
    for (int i = 1; i < argc; i++) {
        const std::string a = argv[i];
        if (i + 1 >= argc) die("usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N");
        const std::string v = argv[++i];
        if (a == "--model") dir = v;
        else if (a == "--dtype") dtype = v;
        else if (a == "--out") out = v;
        else if (a == "--max-tokens") max_tokens = std::strtoul(v.c_str(), nullptr, 10);
        else die("unknown option " + a);
    }
    if (dir.empty() || out.empty() || max_tokens == 0 || max_tokens > 0x7fffffffu) die("usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N");
    if (dtype != "bfloat16" && dtype != "float32") die("--dtype is bfloat16 or float32");

    Runner r;
    wick_safetensors* folder = nullptr;
    if (wick_safetensors_open(dir.c_str(), &folder) != 0) die(wick_safetensors_last_error());
    if (int rc = wick_rocm_ctx_create(0, &r.ctx)) die("no gfx950 GPU (status " + std::to_string(rc) + ")");
    r.check(wick_rocm_model_from_folder(r.ctx, folder, dtype == "float32" ? WICK_ROCM_MODEL_F32 : WICK_ROCM_MODEL_NATIVE, (uint32_t)max_tokens, &r.model), "load");
    wick_safetensors_close(folder);
    wick_rocm_model_get_info(r.model, &r.info);

    std::string line, err;
    while (std::getline(std::cin, line)) {
        if (line.find_first_not_of(" \t\r\n") == std::string::npos) continue;
        Json step;
        if (!JsonParser::parse(line.data(), line.size(), step, err)) die("step: " + err);
        const Json *number = step.find("step"), *entries = step.find("entries"), *end = step.find("end");
        if (!number || number->kind != Json::kNumber || !entries || entries->kind != Json::kArray) die("a step without a number or entries");
        const long long n = (long long)number->number;
        std::vector<float> logits;
        for (const Json& e : entries->items) {
            const Json* id = e.find("id");
            if (!id) die("an entry without an id");
            const std::vector<uint32_t> tokens = ids(e.find("tokens"), "tokens"), want = ids(e.find("want"), "want");
            if (tokens.empty()) continue;
            Request& q = r.turn(name_of(*id));
            // places in any order: the model returns them ascending
            std::vector<uint32_t> places;
            for (uint32_t w : want) {
                if (w >= tokens.size()) die("a wanted place past the tokens");
                size_t at = 0;
                while (at < places.size() && places[at] < w) at++;
                if (at == places.size() || places[at] != w) places.insert(places.begin() + (long)at, w);
            }
            std::vector<float> got(places.size() * (size_t)r.info.vocab_size);
            r.check(wick_rocm_model_forward(r.ctx, r.model, tokens.data(), (uint32_t)tokens.size(), q.pos, places.data(), (uint32_t)places.size(), got.data()),
                    "forward");
            q.pos += (uint32_t)tokens.size();
            for (uint32_t w : want) {
                size_t at = 0;
                while (places[at] != w) at++;
                logits.insert(logits.end(), got.begin() + (long)(at * r.info.vocab_size), got.begin() + (long)((at + 1) * r.info.vocab_size));
            }
        }
        if (end && end->kind == Json::kArray)
            for (const Json& id : end->items) r.finish(name_of(id));
        if (!logits.empty()) {
            const std::string path = out + "/" + std::to_string(n) + ".f32";
            FILE* f = std::fopen(path.c_str(), "wb");
            if (!f || std::fwrite(logits.data(), sizeof(float), logits.size(), f) != logits.size() || std::fclose(f) != 0) die("cannot write " + path);
        }
        std::printf("done %lld\n", n);
        std::fflush(stdout);
    }
    wick_rocm_model_free(r.ctx, r.model);
    wick_rocm_ctx_destroy(r.ctx);
    return 0;
}
