// trace_main.cpp — replays a trace: token ids read from standard input, step by step, go through sessions of a model; logits
// that a step asks for are written to files.  Nothing is sampled.
//
//   trace_run --model PATH [--dtype bfloat16|float32] --out DIR [--max-tokens N] [--device D]
//
// One JSON object a line:
//   {"step": 0, "entries": [{"id": "a", "tokens": [12, 7, 40, 9], "want": [1, 3]}], "end": []}
// An entry's tokens continue the session of its id; `want` lists the places among them whose logits go to DIR/<step>.f32
// (little-endian 32-bit floats, [wanted][vocab], entry by entry).  Sessions named in `end` are closed after the step.  A line
// "done <step>" follows every step.
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <exception>
#include <iostream>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "json.h"
#include "llava_context.h"
#include "llava_hip.h"
#include "llava_session.h"

namespace {

struct failure : std::runtime_error {
    using std::runtime_error::runtime_error;
};

class replay {
public:
    replay(llava_context &c, std::string dir) : ctx(c), out_dir(std::move(dir)), vocab(c.get_model()->vocab_size()) {}

    void run(const json::value &line)
    {
        const u64 number = line.at("step").integer();
        std::vector<float> rows;
        for (const json::value &entry : line.at("entries").items()) evaluate(entry, rows);
        if (!rows.empty()) write(out_dir + "/" + std::to_string(number) + ".f32", rows);
        if (const json::value *end = line.find("end"))
            for (const json::value &id : end->items()) sessions.erase(id.text());
        std::printf("done %llu\n", static_cast<unsigned long long>(number));
        std::fflush(stdout);
    }

private:
    void evaluate(const json::value &entry, std::vector<float> &rows)
    {
        std::vector<u32> tokens;
        for (const json::value &t : entry.at("tokens").items()) tokens.push_back(t.size_value());
        std::vector<u32> want;
        if (const json::value *w = entry.find("want"))
            for (const json::value &p : w->items()) want.push_back(p.size_value());
        for (u32 p : want)
            if (p >= tokens.size()) throw failure("a wanted place outside the step's tokens");
        if (tokens.empty()) return;
        std::unique_ptr<llava_session> &session = sessions[entry.at("id").text()];
        if (!session) session = std::make_unique<llava_session>(&ctx);
        if (!session->good()) throw failure("no session");
        session->keep_all_logits(!want.empty());
        if (!session->push_tokens(tokens.data(), tokens.size())) throw failure("tokens refused");
        if (!session->start_next_token_prediction() || !session->wait()) throw failure("step failed");
        for (u32 p : want) {
            rows.resize(rows.size() + vocab);
            if (!session->read_logits_row(p, rows.data() + rows.size() - vocab)) throw failure("logits not readable");
        }
    }

    static void write(const std::string &path, const std::vector<float> &rows)
    {
        std::FILE *f = std::fopen(path.c_str(), "wb");
        const bool ok = f && std::fwrite(rows.data(), sizeof(float), rows.size(), f) == rows.size();
        if ((f && std::fclose(f) != 0) || !ok) throw failure("cannot write " + path);
    }

    llava_context &ctx;
    const std::string out_dir;
    const std::size_t vocab;
    std::map<std::string, std::unique_ptr<llava_session>> sessions;
};

int usage(const char *argv0)
{
    std::cerr << "usage: " << argv0 << " --model PATH [--dtype bfloat16|float32] --out DIR [--max-tokens N] [--device D] < steps\n";
    return 2;
}

}  // namespace

int main(int argc, char **argv)
{
    std::string model, out, dtype = "bfloat16";
    int device = 0;
    for (int i = 1; i < argc; i += 2) {
        const std::string a = argv[i];
        if (i + 1 >= argc) return usage(argv[0]);
        const char *v = argv[i + 1];
        if (a == "--model") model = v;
        else if (a == "--out") out = v;
        else if (a == "--dtype") dtype = v;
        else if (a == "--device") device = std::atoi(v);
        else if (a == "--max-tokens") continue;      // a session's cache grows with its sequence
        else return usage(argv[0]);
    }
    if (model.empty() || out.empty() || (dtype != "bfloat16" && dtype != "float32")) return usage(argv[0]);
    try {
        llava_context ctx;
        if (!ctx.load_model(model, device, dtype == "float32" ? LV_F32 : LV_BF16)) {
            std::cerr << "cannot load " << model << ": " << ctx.last_error() << std::endl;
            return 1;
        }
        if (dtype == "float32" && ctx.get_model()->as_ggml()) {
            // its weights are quantised and its cache rows fp16: not a 32-bit model
            std::cerr << "float32: this model has no 32-bit form" << std::endl;
            return 3;
        }
        replay r(ctx, out);
        std::string line;
        while (std::getline(std::cin, line))
            if (line.find_first_not_of(" \t\r") != std::string::npos) r.run(json::parse(line));
    } catch (const std::exception &e) {
        std::cerr << "trace_run: " << e.what() << std::endl;
        return 1;
    }
    return 0;
}
