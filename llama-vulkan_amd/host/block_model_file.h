// block_model_file.h — a model folder (config.json, model.safetensors) whose layers are block layers (llava_hip.h,
// lv_block_model_upload).  The configuration's "architecture" picks the design that describes its layers; designs are listed in
// block_designs.cpp.
#pragma once

#include <memory>

#include "json.h"
#include "llava_hip.h"
#include "model_file.h"
#include "safetensors.h"

// a configuration as the device library takes it
struct block_description {
    lv_block_hparams hparams{};
    std::vector<lv_block_spec> layers;
    // layers as a sequence runs through them
    [[nodiscard]] u32 passes() const { return hparams.layers + (hparams.loop_times ? (hparams.loop_times - 1) * (hparams.loop_stop - hparams.loop_start) : 0); }
};

struct block_design {
    const char *name;
    block_description (*describe)(const json::value &config);   // throws json::error
};
const block_design *find_block_design(const std::string &name);

class block_model_file : public model_file {
public:
    explicit block_model_file(const std::string &folder);

    [[nodiscard]] bool is_open() const override { return problem.empty(); }
    [[nodiscard]] const std::string &error() const override { return problem; }
    void print_info() const override;
    [[nodiscard]] u32 vocab_size() const override { return description.hparams.vocab; }
    [[nodiscard]] u32 layer_count() const override { return description.passes(); }
    [[nodiscard]] u32 width() const override { return description.hparams.dim; }
    [[nodiscard]] u32 max_context() const override { return 1u << 20; }
    [[nodiscard]] u32 end_token() const override { return ~0u; }
    [[nodiscard]] bool can_rewind() const override { return false; }
    [[nodiscard]] u32 trace_floats(int which, u32) const override { return which == LV_TRACE_POST_ATTN || which == LV_TRACE_OUT ? width() : 0; }
    // No vocabulary comes with such a folder: text is token ids in decimal, separated by blanks or commas.
    bool tokenize(std::vector<u32> &output, const std::string &text, bool bos) const override;
    [[nodiscard]] std::string token_text(u32 token) const override { return std::to_string(token) + " "; }
    [[nodiscard]] std::string tokens_to_text(const u32 *tokens, u32 count) const override;
    int upload(lv_ctx *ctx, int compute, lv_model **out) const override;

private:
    std::string architecture, problem;
    block_description description;
    std::unique_ptr<safetensors_file> weights;
};
