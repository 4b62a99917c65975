// trace_run.cpp -- replays a trace of forced tokens through a model, step by step, and writes the logits asked for.
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
// Steps come from standard input, one JSON object a line:
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
// A request's tokens continue where its last step left off; "end" names the requests that are finished.  The model holds one live
// sequence: requests follow one another.  After a step OUT/<step>.f32 holds the wanted logits (little-endian f32, in order) and
// "done <step>" is printed.
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <iostream>
#include <memory>
#include <string>
#include <vector>

#include "registry.hpp"

using namespace bitnet_host;

static int die(const std::string &what) {
    fprintf(stderr, "trace_run: %s\n", what.c_str());
    return 1;
}

static bool int_list(const Json *j, std::vector<int32_t> &out) {
    out.clear();
    if (!j || j->kind != Json::Array) return false;
    for (const Json &v : j->items) {
        if (v.kind != Json::Number || v.num != (double)(int32_t)v.num) return false;
        out.push_back((int32_t)v.num);
    }
    return true;
}

int main(int argc, char **argv) {
    std::string model_dir, dtype, out;
    long max_tokens = 4096;
    for (int i = 1; i + 1 < argc; i += 2) {
        const std::string a = argv[i];
        if (a == "--model")
            model_dir = argv[i + 1];
        else if (a == "--dtype")
            dtype = argv[i + 1];
        else if (a == "--out")
            out = argv[i + 1];
        else if (a == "--max-tokens")
            max_tokens = atol(argv[i + 1]);
        else
            return die("unknown option " + a);
    }
    if (model_dir.empty() || out.empty() || (dtype != "bfloat16" && dtype != "float32") || max_tokens < 1 || max_tokens > (1 << 21))
        return die("usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N");
    OpenOptions opt;
    opt.f32 = dtype == "float32";
    opt.max_pos = (int)max_tokens + 2;
    std::string err;
    std::unique_ptr<Sequence> seq(open_model(model_dir, opt, err));
    if (!seq) return die(err);
    std::string live, line;  // the request the model's sequence belongs to
    while (std::getline(std::cin, line)) {
        if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
        Json j;
        if (!Json::parse(line.data(), line.size(), j, err)) return die(err);
        const Json *step = j.find("step"), *entries = j.find("entries"), *end = j.find("end");
        if (!step || step->kind != Json::Number || !entries || entries->kind != Json::Array) return die("a step without number or entries");
        const std::string number = std::to_string((long long)step->num);
        std::vector<float> logits;
        for (const Json &e : entries->items) {
            const Json *id = e.find("id");
            std::vector<int32_t> tokens, want;
            if (!id || !int_list(e.find("tokens"), tokens) || !int_list(e.find("want"), want) || tokens.empty()) return die("step " + number + ": bad entry");
            if (live.empty()) {
                if (seq->reset() != 0) return die(seq->error());
                live = id->str;
            } else if (live != id->str) {
                return die("step " + number + ": request " + id->str + " while " + live + " is not finished");
            }
            const size_t at = logits.size();
            logits.resize(at + want.size() * (size_t)seq->vocab());
            if (seq->forward(tokens.data(), (int)tokens.size(), want.data(), (int)want.size(), logits.data() + at) != 0) return die(seq->error());
        }
        if (!logits.empty()) {
            const std::string path = out + "/" + number + ".f32";
            FILE *f = fopen(path.c_str(), "wb");
            if (!f || fwrite(logits.data(), 4, logits.size(), f) != logits.size() || fclose(f) != 0) return die(path + ": cannot be written");
        }
        if (end)
            for (const Json &e : end->items)
                if (e.str == live) live.clear();
        printf("done %s\n", number.c_str());
        fflush(stdout);
    }
    return 0;
}
