// Replays a trace of token ids through a model folder and writes logits: steps come as JSON lines on standard input, one
// request at a time, and nothing is sampled.
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
//
// A step's tokens continue the request's sequence in the model's cache (several tokens: a prompt portion; one: a decode step).
// The logits at the places `want` go to OUT/<step>.f32 ([wanted][vocab], 32-bit floats); then "done <step>" is printed.
// `end` names requests whose cache is given back.
#include <errno.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>

#include <iostream>
#include <string>
#include <vector>

#include "checkpoint.h"
#include "forge_hip.h"

namespace {

[[noreturn]] void die(const std::string& msg) {
    fprintf(stderr, "trace_run: %s\n", msg.c_str());
    exit(1);
}
void check(int32_t rc) {
    if (rc) die(forge_hip_last_error());
}
std::vector<uint64_t> numbers(const fh::Json* j, const char* what) {
    std::vector<uint64_t> v;
    if (!j || j->kind != fh::Json::Array) die(std::string(what) + " must be a list");
    for (const fh::Json& x : j->arr) {
        if (x.kind != fh::Json::Number || x.num < 0 || x.num > 4294967295.0) die(std::string(what) + " holds something that is not an index");
        v.push_back((uint64_t)x.num);
    }
    return v;
}
std::string text(const fh::Json* j, const char* what) {
    if (!j) die(std::string(what) + " is missing");
    if (j->kind == fh::Json::Number) return std::to_string((long long)j->num);
    if (j->kind != fh::Json::String) die(std::string(what) + " must be a string");
    return j->str;
}

}  // namespace

int main(int argc, char** argv) {
    std::string dir, dtype = "bfloat16", out;
    uint32_t max_tokens = 0;
    for (int i = 1; i < argc; i++) {
        const std::string a = argv[i];
        if (i + 1 >= argc) die("option " + a + " needs a value");
        const std::string v = argv[++i];
        if (a == "--model") dir = v;
        else if (a == "--dtype") dtype = v;
        else if (a == "--out") out = v;
        else if (a == "--max-tokens") max_tokens = (uint32_t)strtoul(v.c_str(), nullptr, 10);
        else die("unknown option " + a);
    }
    if (dir.empty() || out.empty()) die("usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N");
    if (dtype != "bfloat16" && dtype != "float32") die("--dtype is bfloat16 or float32");

    forge_hip_model* m = nullptr;
    check(forge_hip_model_create_from_folder(dir.c_str(), max_tokens, dtype == "float32" ? FORGE_HIP_F32 : FORGE_HIP_BF16, 0, &m));
    forge_hip_config cfg;
    check(forge_hip_model_config(m, &cfg));

    std::string line, live;                      // live: the request whose tokens the cache holds
    bool has_live = false;
    std::vector<float> logits;
    while (std::getline(std::cin, line)) {
        if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
        fh::Json step;
        check(fh::json_parse(line.data(), line.size(), &step));
        const fh::Json *num = step.get("step"), *entries = step.get("entries"), *end = step.get("end");
        if (!num || num->kind != fh::Json::Number || !entries || entries->kind != fh::Json::Array) die("a step has a number and entries");
        logits.clear();
        for (const fh::Json& e : entries->arr) {
            const std::string id = text(e.get("id"), "id");
            const std::vector<uint64_t> tok64 = numbers(e.get("tokens"), "tokens");
            const std::vector<uint64_t> want = e.get("want") ? numbers(e.get("want"), "want") : std::vector<uint64_t>{};
            std::vector<uint32_t> tok(tok64.begin(), tok64.end());
            if (!has_live) { live = id; has_live = true; }
            else if (live != id) die("request " + id + " begins before request " + live + " has ended");
            for (uint64_t w : want)
                if (w >= tok.size()) die("a wanted place lies past the tokens");
            if (tok.empty()) continue;
            const size_t at = logits.size();
            logits.resize(at + want.size() * cfg.vocab);
            if (tok.size() == 1 && forge_hip_model_pos(m) > 0) {
                std::vector<float> row(cfg.vocab);
                check(forge_hip_forward(m, tok[0], row.data()));
                for (size_t i = 0; i < want.size(); i++) memcpy(logits.data() + at + i * cfg.vocab, row.data(), (size_t)cfg.vocab * 4);
            } else {
                check(forge_hip_prefill_logits(m, tok.data(), tok.size(), want.data(), want.size(), logits.data() + at));
            }
        }
        const std::string name = std::to_string((long long)num->num);
        if (!logits.empty()) {
            const std::string path = out + "/" + name + ".f32";
            FILE* f = fopen(path.c_str(), "wb");
            if (!f || fwrite(logits.data(), 4, logits.size(), f) != logits.size() || fclose(f) != 0) die(path + ": " + strerror(errno));
        }
        if (end && end->kind == fh::Json::Array)
            for (const fh::Json& x : end->arr)
                if (has_live && text(&x, "end") == live) { check(forge_hip_reset(m)); has_live = false; }
        printf("done %s\n", name.c_str());
        fflush(stdout);
    }
    forge_hip_model_destroy(m);
    return 0;
}
