// block_designs.cpp — the designs a model folder may name, each a reader of its configuration.

#include "block_model_file.h"

namespace {

// Somesun: every layer mixes chunked grouped-query attention ("left": the keys' projection is also the values, norms over whole
// projections, a sink per head) and a gated delta rule with a decay per key channel ("right"), side by side; the feed-forward
// is a mixture of experts or absent.
block_description describe_somesun(const json::value &config)
{
    block_description d;
    d.hparams.vocab = config.at("vocab").size_value();
    d.hparams.dim = config.at("width").size_value();
    d.hparams.eps = static_cast<float>(config.at("norm").at("eps").number());
    for (const json::value &layer : config.at("layers").items()) {
        if (layer.at("type").text() != "parallel") throw json::error("unknown layer type " + layer.at("type").text());
        lv_block_spec b{};
        const json::value &mix = layer.at("mixer"), &left = mix.at("left"), &right = mix.at("right");
        b.attn_scale = static_cast<float>(mix.at("left_scale").number());
        b.delta_scale = static_cast<float>(mix.at("right_scale").number());
        b.attn.heads = left.at("heads").size_value();
        b.attn.kv_heads = left.at("kv_heads").size_value();
        b.attn.dim = left.at("dim").size_value();
        b.attn.vdim = left.at("vdim").size_value();
        b.attn.scale = static_cast<float>(left.at("scale").number());
        b.attn.chunk = left.at("mask").at("size").size_value();
        b.attn.rot_dims = left.at("rot").at("dims").size_value();
        b.attn.rot_base = left.at("rot").at("base").number();
        b.attn.flags = LV_ATTN_NORM_FULL | LV_ATTN_KEYS_AS_VALUES | LV_ATTN_SINK;
        if (!b.attn.heads || !b.attn.chunk) throw json::error("attention without heads or chunk size");
        b.delta.heads = right.at("heads").size_value();
        b.delta.kv_heads = right.at("kv_heads").size_value();
        b.delta.dim = right.at("dim").size_value();
        b.delta.vdim = right.at("vdim").size_value();
        b.delta.conv = right.at("conv").size_value();
        if (!b.delta.heads) throw json::error("delta rule without heads");
        const json::value *mlp = layer.find("mlp");
        if (mlp && !mlp->is_null()) {
            if (mlp->at("kind").text() != "moe") throw json::error("unknown feed-forward " + mlp->at("kind").text());
            b.moe.experts = mlp->at("router").at("experts").size_value();
            b.moe.top = mlp->at("router").at("top").size_value();
            b.moe.ff = mlp->at("expert").at("ff").size_value();
            if (!b.moe.experts) throw json::error("mixture without experts");
        }
        d.layers.push_back(b);
    }
    d.hparams.layers = static_cast<u32>(d.layers.size());
    return d;
}

constexpr block_design kDesigns[] = {
    {"Somesun", describe_somesun},
};

}  // namespace

const block_design *find_block_design(const std::string &name)
{
    for (const block_design &d : kDesigns)
        if (name == d.name) return &d;
    return nullptr;
}
