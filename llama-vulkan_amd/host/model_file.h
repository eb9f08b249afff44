// model_file.h — what a session, the command line and the server need to know of a model on disk, whatever its format.
// Two formats exist: a GGJT file (ggml_file, the reference's) and a folder with config.json and model.safetensors
// (block_model_file), whose design is looked up by the configuration's "architecture".
#pragma once

#include <memory>
#include <string>
#include <vector>

#include "types.h"

struct lv_ctx;
struct lv_model;

class model_file {
public:
    virtual ~model_file() = default;

    // the right kind of object for the path; never null, is_open() tells whether the model can be used
    static std::unique_ptr<model_file> open(const std::string &path);

    [[nodiscard]] virtual bool is_open() const = 0;
    [[nodiscard]] virtual const std::string &error() const = 0;      // why is_open() is false
    virtual void print_info() const = 0;

    [[nodiscard]] virtual u32 vocab_size() const = 0;
    [[nodiscard]] virtual u32 layer_count() const = 0;
    [[nodiscard]] virtual u32 width() const = 0;                      // floats of the residual stream
    [[nodiscard]] virtual u32 max_context() const = 0;                // most tokens a session may hold
    [[nodiscard]] virtual u32 end_token() const = 0;                  // generation ends behind it; ~0u: none
    [[nodiscard]] virtual u32 newline_token() const { return ~0u; }   // the token the sampler's repetition penalty applies to; ~0u: none
    // A step may start at any position that has been evaluated.  False: the per-sequence state only moves forward, and going
    // back means evaluating the sequence again.
    [[nodiscard]] virtual bool can_rewind() const = 0;
    // record-mode buffers (LV_TRACE_*) a step of this model fills: floats of one row, 0 = not recorded
    [[nodiscard]] virtual u32 trace_floats(int which, u32 backlog) const = 0;

    // false when the text cannot be expressed in this model's tokens
    virtual bool tokenize(std::vector<u32> &output, const std::string &text, bool bos) const = 0;
    [[nodiscard]] virtual std::string token_text(u32 token) const = 0;
    [[nodiscard]] virtual std::string tokens_to_text(const u32 *tokens, u32 count) const = 0;

    // weights to the device; an lv_status.  compute: LV_BF16 or LV_F32 where the format leaves a choice, else ignored
    virtual int upload(lv_ctx *ctx, int compute, lv_model **out) const = 0;

    [[nodiscard]] virtual const ggml_file *as_ggml() const { return nullptr; }
};
