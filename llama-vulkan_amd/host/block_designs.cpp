// block_designs.cpp — the designs a model folder may name, each a reader of its configuration.

#include "block_model_file.h"

namespace {

bool present(const json::value *v) { return v && !v->is_null(); }

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
        if (present(mlp)) {
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

// Zedenex: a residual of several streams, tanh norms, a bigram embedding, the table as output matrix; layers of latent attention
// with a sink per head or of a state-space recurrence, a dense feed-forward or none behind them, some of them run in a loop.
block_description describe_zedenex(const json::value &config)
{
    block_description d;
    d.hparams.vocab = config.at("vocab").size_value();
    d.hparams.dim = config.at("width").size_value();
    d.hparams.eps = static_cast<float>(config.at("norm").at("eps").number());
    d.hparams.norm = LV_NORM_TANH;
    d.hparams.streams = config.at("streams").size_value();
    if (!d.hparams.streams) throw json::error("a residual without streams");
    d.hparams.tied_head = 1;
    const json::value &embedding = config.at("embedding");
    d.hparams.embed_scale = static_cast<float>(embedding.at("scale").number());
    if (present(embedding.find("bigram"))) {
        const json::value &bigram = embedding.at("bigram");
        const u32 buckets = bigram.at("buckets").size_value();
        if (!buckets) throw json::error("bigram embedding without buckets");
        d.hparams.bigram_buckets = buckets;
        d.hparams.bigram_prev = static_cast<u32>(bigram.at("mul_prev").integer() % buckets);     // the sum counts modulo the buckets
        d.hparams.bigram_cur = static_cast<u32>(bigram.at("mul_cur").integer() % buckets);
    }
    for (const json::value &layer : config.at("layers").items()) {
        lv_block_spec b{};
        const std::string &type = layer.at("type").text();
        const json::value &mix = layer.at("mixer");
        if (type == "latent_attention") {
            b.latent.heads = mix.at("heads").size_value();
            b.latent.dim = mix.at("dim").size_value();
            b.latent.rot_dim = mix.at("rot_dim").size_value();
            b.latent.vdim = mix.at("vdim").size_value();
            b.latent.q_rank = mix.at("q_rank").size_value();
            b.latent.kv_rank = mix.at("kv_rank").size_value();
            b.latent.scale = static_cast<float>(mix.at("scale").number());
            b.latent.rot_dims = mix.at("rot").at("dims").size_value();
            b.latent.rot_base = mix.at("rot").at("base").number();
            b.latent.flags = LV_ATTN_SINK;
            if (!b.latent.heads) throw json::error("attention without heads");
        } else if (type == "mamba2") {
            b.ssm.heads = mix.at("heads").size_value();
            b.ssm.groups = mix.at("groups").size_value();
            b.ssm.state = mix.at("state").size_value();
            b.ssm.vdim = mix.at("vdim").size_value();
            b.ssm.conv = mix.at("conv").size_value();
            b.ssm.norm_groups = mix.at("norm_groups").size_value();
            if (!b.ssm.heads) throw json::error("recurrence without heads");
        } else {
            throw json::error("unknown layer type " + type);
        }
        const json::value *mlp = layer.find("mlp");
        if (present(mlp)) {
            if (mlp->at("kind").text() != "dense") throw json::error("unknown feed-forward " + mlp->at("kind").text());
            b.dense.ff = mlp->at("ff").size_value();
            b.dense.act = LV_ACT_RELU;
            if (!b.dense.ff) throw json::error("feed-forward without width");
        }
        d.layers.push_back(b);
    }
    d.hparams.layers = static_cast<u32>(d.layers.size());
    if (present(config.find("loop"))) {
        const json::value &loop = config.at("loop");
        d.hparams.loop_start = loop.at("start").size_value();
        d.hparams.loop_stop = loop.at("stop").size_value();
        d.hparams.loop_times = loop.at("times").size_value();
        if (d.hparams.loop_start > d.hparams.loop_stop || d.hparams.loop_stop > d.hparams.layers || !d.hparams.loop_times) throw json::error("a loop over layers that are not there");
    }
    return d;
}

constexpr block_design kDesigns[] = {
    {"Somesun", describe_somesun},
    {"Zedenex", describe_zedenex},
};

}  // namespace

const block_design *find_block_design(const std::string &name)
{
    for (const block_design &d : kDesigns)
        if (name == d.name) return &d;
    return nullptr;
}
