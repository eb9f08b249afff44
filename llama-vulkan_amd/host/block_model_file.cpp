#include "block_model_file.h"

#include <fstream>
#include <iostream>
#include <sstream>

block_model_file::block_model_file(const std::string &folder)
{
    try {
        std::ifstream in(folder + "/config.json");
        if (!in) throw json::error("cannot read config.json");
        std::stringstream text;
        text << in.rdbuf();
        const json::value config = json::parse(text.str());
        architecture = config.at("architecture").text();
        const block_design *design = find_block_design(architecture);
        if (!design) throw json::error("unknown architecture " + architecture);
        description = design->describe(config);
        weights = std::make_unique<safetensors_file>(folder + "/model.safetensors");
        if (!weights->is_open()) throw json::error(weights->error());
    } catch (const std::exception &e) {
        problem = folder + ": " + e.what();
        std::cerr << problem << std::endl;
    }
}

void block_model_file::print_info() const
{
    std::cout << "architecture: " << architecture << "\nvocab_size: " << vocab_size() << "\nwidth: " << width() << "\nlayers: " << layer_count()
              << "\ntensors: " << weights->entries().size() << std::endl;
}

bool block_model_file::tokenize(std::vector<u32> &output, const std::string &text, bool) const
{
    u64 id = 0;
    bool digits = false;
    for (std::size_t i = 0; i <= text.size(); ++i) {
        const char c = i < text.size() ? text[i] : ' ';
        if (c >= '0' && c <= '9') {
            id = id * 10 + static_cast<u64>(c - '0');
            digits = true;
            if (id >= vocab_size()) return false;
        } else if (c == ' ' || c == ',' || c == '\n' || c == '\t' || c == '\r') {
            if (digits) output.push_back(static_cast<u32>(id));
            id = 0;
            digits = false;
        } else {
            return false;
        }
    }
    return true;
}

std::string block_model_file::tokens_to_text(const u32 *tokens, u32 count) const
{
    std::string s;
    for (u32 i = 0; i < count; ++i) s += token_text(tokens[i]);
    return s;
}

int block_model_file::upload(lv_ctx *ctx, int compute, lv_model **out) const
{
    std::vector<lv_tensor_desc> table;
    for (const safetensors_entry &e : weights->entries()) {
        // a matrix is [rows][cols]; a vector has one column, a scalar one row; other ranks and types belong to no tensor the device library reads
        const u32 type = e.dtype == "BF16" ? u32{LV_BF16} : e.dtype == "F32" ? u32{LV_F32} : ~0u;
        if (type == ~0u || e.shape.size() > 2 || (e.shape.size() >= 1 && e.shape[0] > 0xffffffffu) || (e.shape.size() == 2 && e.shape[1] > 0xffffffffu)) continue;
        table.push_back({e.name.c_str(), type, e.offset, e.shape.empty() ? 1u : static_cast<u32>(e.shape[0]), e.shape.size() == 2 ? static_cast<u32>(e.shape[1]) : 1u, e.size});
    }
    return lv_block_model_upload(ctx, weights->data(), weights->data_size(), &description.hparams, description.layers.data(), table.data(),
                                 static_cast<u32>(table.size()), compute, out);
}
