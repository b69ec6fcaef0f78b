// trace_run: feeds given tokens through a model, step by step, and writes logits (the program behind bin/trace_run).
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
// Standard input: one JSON object a line,
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["b"]}
// An entry's tokens continue its request; `want` names the places among them whose logits are asked for; `end` lists the
// requests that are finished after the step.  Logits of a step go to OUT/<step>.f32, f32 [wanted, vocab] in the order of
// the entries and of `want`; every step is answered by a line "done <step>".  A request is a session of the engine.
#include <algorithm>
#include <cstdio>
#include <cstdlib>
#include <iostream>
#include <map>
#include <string>
#include <vector>

#include "../../include/mynn_hip.h"
#include "json.h"

using mynn::Json;

static int die(const char *what) {
    fprintf(stderr, "trace_run: %s: %s\n", what, mynn_last_error());
    return 1;
}
static bool integers(const Json *j, std::vector<int64_t> &out) {
    out.clear();
    if (!j) return true;
    if (j->kind != Json::ARR) return false;
    for (const Json &v : j->arr) {
        if (v.kind != Json::NUM) return false;
        out.push_back((int64_t)v.num);
    }
    return true;
}

int main(int argc, char **argv) {
    std::map<std::string, std::string> arg;
    for (int i = 1; i + 1 < argc; i += 2) arg[argv[i]] = argv[i + 1];
    const std::string dtype = arg["--dtype"], out_dir = arg["--out"];
    if (argc % 2 == 0 || arg["--model"].empty() || out_dir.empty() || (dtype != "bfloat16" && dtype != "float32")) {
        fprintf(stderr, "usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N\n");
        return 2;
    }
    mynn_engine_options opt{};
    opt.dtype = dtype == "float32" ? MYNN_F32 : MYNN_BF16;
    opt.max_tokens = arg["--max-tokens"].empty() ? 4096 : atoi(arg["--max-tokens"].c_str());
    mynn_engine *engine = mynn_engine_open(arg["--model"].c_str(), &opt);
    if (!engine) return die("cannot open the model");
    const size_t V = (size_t)mynn_engine_vocab(engine);

    std::map<std::string, mynn_llm *> live;
    std::vector<mynn_llm *> idle;  // ended requests' sessions, their cache rows given back
    std::string line;
    std::vector<int64_t> tokens, want;
    std::vector<float> logits, rows;
    while (std::getline(std::cin, line)) {
        if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
        Json step;
        const Json *num, *entries;
        if (!mynn::parse_json(line.data(), line.size(), step) || !(num = step.get("step")) || num->kind != Json::NUM ||
            !(entries = step.get("entries")) || entries->kind != Json::ARR) {
            fprintf(stderr, "trace_run: not a step: %.80s\n", line.c_str());
            return 1;
        }
        logits.clear();
        for (const Json &e : entries->arr) {
            const Json *id = e.get("id");
            if (!id || id->kind != Json::STR || !integers(e.get("tokens"), tokens) || !integers(e.get("want"), want)) {
                fprintf(stderr, "trace_run: not an entry in step %lld\n", (long long)num->num);
                return 1;
            }
            mynn_llm *&s = live[id->str];
            if (!s && !idle.empty()) {
                s = idle.back();
                idle.pop_back();
            }
            if (!s && !(s = mynn_engine_session(engine, -1))) return die("cannot start a session");
            // (the session takes the places in rising order; the answer keeps the order they were asked in)
            std::vector<int64_t> sorted = want;
            std::sort(sorted.begin(), sorted.end());
            sorted.erase(std::unique(sorted.begin(), sorted.end()), sorted.end());
            rows.resize(sorted.size() * V);
            if (mynn_llm_feed(s, tokens.data(), tokens.size(), sorted.data(), sorted.size(), rows.data())) return die("step failed");
            for (int64_t w : want) {
                const size_t at = (size_t)(std::lower_bound(sorted.begin(), sorted.end(), w) - sorted.begin()) * V;
                logits.insert(logits.end(), rows.begin() + at, rows.begin() + at + V);
            }
        }
        const std::string n = std::to_string((long long)num->num);
        if (!logits.empty()) {
            const std::string path = out_dir + "/" + n + ".f32";
            FILE *f = fopen(path.c_str(), "wb");
            const bool ok = f && fwrite(logits.data(), 4, logits.size(), f) == logits.size();
            if ((f && fclose(f)) || !ok) {
                fprintf(stderr, "trace_run: cannot write %s\n", path.c_str());
                return 1;
            }
        }
        if (const Json *end = step.get("end"))
            for (const Json &id : end->arr) {
                auto it = live.find(id.str);
                if (it == live.end()) continue;
                mynn_llm_reset(it->second);
                idle.push_back(it->second);
                live.erase(it);
            }
        printf("done %s\n", n.c_str());
        fflush(stdout);
    }
    for (auto &kv : live) idle.push_back(kv.second);
    for (mynn_llm *s : idle) mynn_llm_destroy(s);
    mynn_engine_close(engine);
    return 0;
}
