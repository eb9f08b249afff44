// lv_block.hip — block models: upload, per-sequence state, and the step as launches of the kernels in lv_bf16_gemm.h,
// lv_bf16_gemv.h, lv_streams.h, lv_gqa.h, lv_delta.h, lv_latent.h, lv_ssm.h and lv_block_kernels.h.
//
// Device layout.  Matrices bf16 row-major, columns padded with zeros to a multiple of 64, rows to a multiple of 128.  All
// projections that read a layer's normed input are one matrix (sections padded to 16 rows), the two branches' output
// projections are one matrix over the concatenated branch outputs, and a feed-forward's (an expert's) gate and up rows alternate
// in blocks of 16, so that both products and the activation between them are one launch.  Vectors are fp32.
//
// A layer of a loop is stored once; the model's `order` lists its passes, and a session keeps a state for each pass.
#include "lv_block.h"

#include <algorithm>
#include <cmath>
#include <cstring>
#include <functional>
#include <new>
#include <string>
#include <unordered_map>
#include <vector>

#include "lv_block_kernels.h"
#include "lv_gqa_tile.h"

namespace lv {

static uint32_t up(uint32_t v, uint32_t a) { return (v + a - 1) / a * a; }

struct BfMatrix {
    const uint16_t *w = nullptr;
    uint32_t rows = 0, kp = 0;
};

// where a sublayer's input is taken from the residual and its output goes back
struct NormSite {
    const float *w = nullptr, *b = nullptr, *alpha = nullptr;      // b, alpha: LV_NORM_TANH
    const float *post = nullptr;                                   // norm of the sublayer's output (no streams)
    const StreamCoef *coef = nullptr;                              // (streams)
};

struct BlockLayer {
    lv_block_spec spec{};
    bool attn = false, delta = false, latent = false, ssm = false, moe = false, dense = false;
    BfMatrix in, out, a2, g2, router, gate_up, down, uq, uk, uv;
    uint32_t q_off = 0, k_off = 0, v_off = 0, dq_off = 0, dk_off = 0, dv_off = 0, b_off = 0, a_off = 0, g_off = 0;   // rows of `in`
    uint32_t a_rank = 0, g_rank = 0;
    uint32_t left_kp = 0;              // where the recurrent part starts in the joint output projection's input
    uint32_t gu_rows = 0, down_rows = 0;   // rows from one expert to the next
    uint32_t dp = 64, r = 1, groups = 1;   // attention: padded head size, heads per group, groups per kv head
    uint32_t dk = 64, dv = 64;             // padded sizes of expanded keys and values of latent attention
    uint32_t kc = 0, width = 0;            // its cache row: start of the rotated part, elements
    NormSite site[2];                  // mixer, feed-forward
    const float *q_norm = nullptr, *k_norm = nullptr, *sink = nullptr;
    const double *freq = nullptr;
    uint32_t freq_at = 0;              // latent attention: where its frequencies start in the model's
    const float *conv = nullptr, *conv_bias = nullptr, *a_log = nullptr, *dt_bias = nullptr, *skip = nullptr, *onorm = nullptr;
    const uint16_t *uk_t = nullptr;    // W_uk transposed head by head
    bool ff() const { return moe || dense; }
    uint32_t dstride() const { return up(spec.delta.dim, 64); }
    uint32_t channels() const { return 2 * spec.delta.kv_heads * spec.delta.dim + spec.delta.heads * spec.delta.vdim; }
    uint32_t sstride() const { return spec.ssm.state <= 64 ? 64 : spec.ssm.state <= 128 ? 128 : 256; }
    uint32_t ssm_inner() const { return spec.ssm.heads * spec.ssm.vdim; }
    uint32_t ssm_channels() const { return ssm_inner() + 2 * spec.ssm.groups * spec.ssm.state; }
    uint32_t latent_size() const { return spec.latent.dim + spec.latent.rot_dim; }
    // a pass's recurrent state and convolution ring
    uint64_t state_bytes() const { return delta ? 4ull * spec.delta.heads * spec.delta.vdim * dstride() : ssm ? 4ull * ssm_inner() * sstride() : 0; }
    uint64_t ring_bytes() const { return delta ? 4ull * spec.delta.conv * channels() : ssm ? 4ull * spec.ssm.conv * ssm_channels() : 0; }
};

struct BlockModel {
    lv_block_hparams hp{};
    bool f32 = false;                  // activations of batches and cache rows are fp32
    uint32_t dp = 0;                   // hp.dim rounded up to 64
    uint32_t copies = 1;               // of the residual: its streams
    uint8_t *arena = nullptr;
    uint64_t arena_bytes = 0;
    const uint16_t *embed = nullptr;   // [vocab][embed_ld]
    uint32_t embed_ld = 0;
    const uint16_t *bigram = nullptr;  // [buckets + 1][dim]
    NormSite final;
    BfMatrix head;
    std::vector<BlockLayer> layers;
    std::vector<uint32_t> order;       // layer of every pass
    const double *freq = nullptr;      // frequencies of all layers of latent attention, layer after layer
    uint32_t n_freq = 0;
    uint32_t elem() const { return f32 ? 4 : 2; }
    const BlockLayer &pass(size_t i) const { return layers[order[i]]; }
};

// per pass of a layer and sequence
struct LayerState {
    uint32_t ring = 0;                 // cache rows
    uint8_t *kc = nullptr, *vc = nullptr;      // latent attention: one kind of row, in kc
    float *state = nullptr, *conv = nullptr;
};

struct Workspace {                     // of batches; sized for `cap` tokens
    uint32_t cap = 0;
    float *x = nullptr, *y1 = nullptr, *y = nullptr, *dq = nullptr, *dk = nullptr, *dv = nullptr, *dg = nullptr, *beta = nullptr, *qk = nullptr, *o = nullptr,
          *gate = nullptr, *z = nullptr, *scores = nullptr, *y2 = nullptr, *sdt = nullptr, *sdecay = nullptr;
    void *act = nullptr, *q = nullptr, *k = nullptr, *v = nullptr, *vt = nullptr, *a1 = nullptr, *g1 = nullptr, *cat = nullptr, *ff = nullptr, *cq = nullptr,
         *ek = nullptr, *ev = nullptr, *sx = nullptr, *sb = nullptr, *sc = nullptr, *sbt = nullptr;
    uint32_t *ids = nullptr, *slots = nullptr, *tiles = nullptr;
    uint64_t vt_elems = 0, ek_elems = 0, ev_elems = 0;
};

struct BlockSession {
    const BlockModel *m = nullptr;
    hipStream_t st = nullptr;
    uint32_t positions = 0, position = 0;
    bool valid = true;
    std::vector<LayerState> layers;
    // one token
    float *xa = nullptr, *xb = nullptr, *y1 = nullptr, *left = nullptr, *o = nullptr, *gate = nullptr, *yo = nullptr, *h2 = nullptr, *z = nullptr, *act = nullptr,
          *yd = nullptr, *scores = nullptr, *part = nullptr, *y2 = nullptr;
    void *ql = nullptr;                // latent attention: queries (latent_put)
    float2 *turn = nullptr;            // the model's frequencies as (cos, sin) at the token's position
    uint32_t *ids = nullptr, *counters = nullptr, *last = nullptr;      // last: the sequence's last token, at [position % 2]
    Workspace ws;
};

// ---------------------------------------------------------------------------------------------------------------------------
// model
// ---------------------------------------------------------------------------------------------------------------------------
namespace {

// one block of the arena: fill(dst) produces `bytes` bytes in host memory
struct Fill {
    uint64_t off, bytes;
    std::function<void(uint8_t *)> fill;
};

class Loader {
public:
    Loader(const void *base, uint64_t size, const lv_tensor_desc *table, uint32_t n) : base_(static_cast<const uint8_t *>(base)), size_(size)
    {
        for (uint32_t i = 0; i < n; i++)
            if (table[i].name) by_name_.emplace(table[i].name, &table[i]);
    }
    int error = LV_OK;
    uint64_t bytes = 0;
    std::vector<Fill> fills;

    // tensor `name` of rows x cols; null and error set when it is absent or has another shape.  rows 0: any number of rows
    const lv_tensor_desc *find(const std::string &name, uint32_t rows, uint32_t cols, bool vector)
    {
        if (error != LV_OK) return nullptr;
        const auto it = by_name_.find(name);
        if (it == by_name_.end()) {
            error = fail(LV_ERR_MISSING, "lv_block_model_upload: tensor %s is not in the table", name.c_str());
            return nullptr;
        }
        const lv_tensor_desc &d = *it->second;
        if ((rows && d.rows != rows) || (cols && d.cols != cols) || !d.rows || !d.cols) {
            error = fail(LV_ERR_ARG, "lv_block_model_upload: %s is %u x %u, expected %u x %u", d.name, d.rows, d.cols, rows, cols);
            return nullptr;
        }
        const uint64_t e = d.ftype == LV_BF16 ? 2 : d.ftype == LV_F32 && vector ? 4 : 0, raw = e * d.rows * d.cols;
        if (!e || d.size != raw || d.offset > size_ || raw > size_ - d.offset) {
            error = fail(LV_ERR_ARG, "lv_block_model_upload: %s has type %u / %llu bytes at %llu (file holds %llu)", d.name, d.ftype, (unsigned long long)d.size,
                         (unsigned long long)d.offset, (unsigned long long)size_);
            return nullptr;
        }
        return &d;
    }
    const uint8_t *data(const lv_tensor_desc *d) const { return base_ + d->offset; }

    uint64_t place(uint64_t n, std::function<void(uint8_t *)> fn)
    {
        const uint64_t off = bytes;
        fills.push_back({off, n, std::move(fn)});
        bytes += (n + 255) / 256 * 256;
        return off;
    }

    // fp32 vector of `padded` floats from n tensor elements (rows x cols flattened), zeros behind
    uint64_t vec(const std::string &name, uint32_t rows, uint32_t cols, uint32_t padded)
    {
        const lv_tensor_desc *d = find(name, rows, cols, true);
        if (!d) return 0;
        const uint8_t *src = data(d);
        const uint32_t n = d->rows * d->cols, type = d->ftype;
        return place((uint64_t)padded * 4, [=](uint8_t *dst) { widen(dst, src, n, type); });
    }
    static void widen(uint8_t *dst, const uint8_t *src, uint32_t n, uint32_t type)
    {
        if (type == LV_F32) {
            std::memcpy(dst, src, (size_t)n * 4);
            return;
        }
        for (uint32_t i = 0; i < n; i++) {
            uint16_t h;
            std::memcpy(&h, src + 2 * (size_t)i, 2);
            const uint32_t w = (uint32_t)h << 16;
            std::memcpy(dst + 4 * (size_t)i, &w, 4);
        }
    }

    // sections of one matrix: tensor rows to matrix rows from `row`, tensor columns to matrix columns from `col`
    struct Part {
        const lv_tensor_desc *d;
        uint32_t row, col;
    };
    uint64_t matrix(const std::vector<Part> &parts, uint32_t rows, uint32_t kp, BfMatrix *m)
    {
        if (error != LV_OK) return 0;
        m->rows = rows;
        m->kp = kp;
        std::vector<std::pair<const uint8_t *, Part>> src;
        for (const Part &p : parts) src.push_back({data(p.d), p});
        return place((uint64_t)up(rows, 128) * kp * 2, [=](uint8_t *dst) {
            for (const auto &s : src)
                for (uint32_t r = 0; r < s.second.d->rows; r++)
                    std::memcpy(dst + ((uint64_t)(s.second.row + r) * kp + s.second.col) * 2, s.first + (uint64_t)r * s.second.d->cols * 2, (size_t)s.second.d->cols * 2);
        });
    }

private:
    const uint8_t *base_;
    uint64_t size_;
    std::unordered_map<std::string, const lv_tensor_desc *> by_name_;
};

// of pair k, in full turns per position
double frequency(double base, uint32_t dims, uint32_t k) { return std::pow(base, -2.0 * k / dims) / 6.283185307179586476925; }

uint32_t latent_kc(const lv_latent_spec &l) { return up(l.kv_rank, 16); }
uint32_t latent_width(const lv_latent_spec &l) { return up(latent_kc(l) + l.rot_dim, 64); }

int check_hparams(const lv_block_hparams &hp)
{
    if (!hp.vocab || !hp.dim || !hp.layers || hp.dim > 32768) return fail(LV_ERR_ARG, "lv_block_model_upload: vocabulary %u, width %u, %u layers", hp.vocab, hp.dim, hp.layers);
    if (hp.streams > kMaxStreams) return fail(LV_ERR_ARG, "lv_block_model_upload: %u residual streams (%u are built)", hp.streams, kMaxStreams);
    if (hp.norm > LV_NORM_TANH || (hp.norm == LV_NORM_TANH && !hp.streams)) return fail(LV_ERR_ARG, "lv_block_model_upload: norm %u on %u streams", hp.norm, hp.streams);
    if (hp.loop_times && (hp.loop_start > hp.loop_stop || hp.loop_stop > hp.layers || (uint64_t)hp.loop_times * (hp.loop_stop - hp.loop_start) > 4096))
        return fail(LV_ERR_ARG, "lv_block_model_upload: layers %u to %u of %u, %u times", hp.loop_start, hp.loop_stop, hp.layers, hp.loop_times);
    return LV_OK;
}

int check_spec(const lv_block_spec &b, uint32_t layer)
{
    const lv_attn_spec &a = b.attn;
    if (a.heads) {
        if (!a.kv_heads || a.heads % a.kv_heads || !a.dim || !a.vdim || std::max(a.dim, a.vdim) > 256)
            return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: attention of %u / %u heads of %u and %u (head sizes to 256 are built)", layer, a.heads, a.kv_heads, a.dim, a.vdim);
        if (a.rot_dims % 2 || a.rot_dims > a.dim || (a.rot_dims && !(a.rot_base > 0)))
            return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: rotation of %u of %u dimensions, base %g", layer, a.rot_dims, a.dim, a.rot_base);
        if ((a.flags & LV_ATTN_KEYS_AS_VALUES) && a.vdim != a.dim)
            return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: values are keys but head sizes differ (%u, %u)", layer, a.dim, a.vdim);
    }
    const lv_delta_spec &d = b.delta;
    if (d.heads && (!d.kv_heads || d.heads % d.kv_heads || !d.dim || d.dim > kDeltaMaxDim || !d.vdim || !d.conv))
        return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: delta rule of %u / %u heads, %u x %u, %u taps (key sizes to %u are built)", layer, d.heads, d.kv_heads, d.dim, d.vdim, d.conv,
                    kDeltaMaxDim);
    const lv_latent_spec &l = b.latent;
    if (l.heads && (!l.dim || !l.vdim || !l.q_rank || !l.kv_rank || l.dim + l.rot_dim > kGqaMaxDim || l.vdim > kGqaMaxDim || latent_width(l) > kLatentMaxWidth || l.heads > kLatentMaxHeads))
        return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: latent attention of %u heads of %u + %u and %u, latents of %u and %u (head sizes to %u and cache rows to %u are built)", layer,
                    l.heads, l.dim, l.rot_dim, l.vdim, l.q_rank, l.kv_rank, kGqaMaxDim, kLatentMaxWidth);
    if (l.heads && (l.rot_dim % 2 || l.rot_dims % 2 || l.rot_dims > l.rot_dim || (l.rot_dims && !(l.rot_base > 0))))
        return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: rotation of %u of %u dimensions, base %g", layer, l.rot_dims, l.rot_dim, l.rot_base);
    const lv_ssm_spec &m = b.ssm;
    if (m.heads && (!m.groups || m.heads % m.groups || !m.state || m.state > kSsmMaxState || !m.vdim || !m.conv || !m.norm_groups || (m.heads * m.vdim) % m.norm_groups))
        return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: state space of %u heads in %u groups, %u x %u, %u taps, %u norm groups (states to %u are built)", layer, m.heads, m.groups,
                    m.state, m.vdim, m.conv, m.norm_groups, kSsmMaxState);
    const int mixers = (a.heads || d.heads) + (l.heads != 0) + (m.heads != 0);
    if (mixers != 1) return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u has %s mixer", layer, mixers ? "more than one" : "no");
    if (b.dense.ff && (b.moe.experts || b.dense.act > LV_ACT_RELU)) return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: dense feed-forward with activation %u and %u experts", layer, b.dense.act, b.moe.experts);
    const lv_moe_spec &e = b.moe;
    if (e.experts && (!e.top || e.top > e.experts || e.top > kMaxTop || e.experts > kMaxExperts || !e.ff))
        return fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: %u of %u experts of %u", layer, e.top, e.experts, e.ff);
    return LV_OK;
}

}  // namespace

int block_model_create(hipStream_t st, const void *base, uint64_t base_size, const lv_block_hparams *hp, const lv_block_spec *blocks, const lv_tensor_desc *table,
                       uint32_t n_tensors, int compute, BlockModel **out)
{
    *out = nullptr;
    LV_TRY(check_hparams(*hp));
    if (compute != LV_BF16 && compute != LV_F32) return fail(LV_ERR_ARG, "lv_block_model_upload: compute type %d", compute);
    for (uint32_t i = 0; i < hp->layers; i++) LV_TRY(check_spec(blocks[i], i));
    BlockModel *m = new (std::nothrow) BlockModel;
    if (!m) return fail(LV_ERR_OOM, "lv_block_model_upload: host allocation");
    m->hp = *hp;
    m->f32 = compute == LV_F32;
    const uint32_t D = hp->dim, V = hp->vocab, Dp = m->dp = up(D, 64);
    m->copies = std::max(1u, hp->streams);
    m->layers.resize(hp->layers);
    for (uint32_t i = 0; i < hp->layers; i++) {
        if (hp->loop_times && i == hp->loop_start)
            for (uint32_t t = 1; t < hp->loop_times; t++)
                for (uint32_t j = hp->loop_start; j < hp->loop_stop; j++) m->order.push_back(j);
        m->order.push_back(i);
    }

    // where everything goes; pointers are set once the arena exists
    Loader ld(base, base_size, table, n_tensors);
    struct Fix { void *at; uint64_t off; };       // a pointer member of the model and its place in the arena
    std::vector<Fix> fixes;
    auto at = [&](auto **p, uint64_t off) { fixes.push_back({static_cast<void *>(p), off}); };
    using Part = Loader::Part;
    auto matrix = [&](BfMatrix *dst, const std::vector<Part> &parts, uint32_t rows, uint32_t kp) {
        const uint64_t off = ld.matrix(parts, rows, kp, dst);
        at(&dst->w, off);
    };
    auto vec = [&](const float **dst, const std::string &name, uint32_t rows, uint32_t cols, uint32_t padded) { at(dst, ld.vec(name, rows, cols, padded)); };
    auto tensor = [&](const std::string &name, uint32_t rows, uint32_t cols) { return ld.find(name, rows, cols, false); };

    // a norm with its streams' coefficients; `hc` empty: the model's end, which reads the sum of the streams
    auto site = [&](NormSite *n, const std::string &name, const std::string &hc) {
        vec(&n->w, name, D, 1, Dp);
        if (hp->norm == LV_NORM_TANH) {
            vec(&n->b, name + ".b", D, 1, Dp);
            vec(&n->alpha, name + ".alpha", 1, 1, 1);
        }
        const uint32_t S = hp->streams;
        if (!S) {
            if (!hc.empty()) vec(&n->post, name + "b", D, 1, Dp);
            return;
        }
        auto put = [&](std::function<void(StreamCoef &)> fn) {
            at(&n->coef, ld.place(sizeof(StreamCoef), [=](uint8_t *dst) {
                StreamCoef c{};
                fn(c);
                std::memcpy(dst, &c, sizeof c);
            }));
        };
        if (hc.empty()) return put([=](StreamCoef &c) { std::fill(c.in, c.in + S, 1.f); });
        const lv_tensor_desc *di = ld.find(hc + "in", S, 1, true), *dn = ld.find(hc + "out", S, 1, true), *dm = ld.find(hc + "mix", S, S, true);
        if (!di || !dn || !dm) return;
        const uint8_t *si = ld.data(di), *so = ld.data(dn), *sm = ld.data(dm);
        const uint32_t ti = di->ftype, to = dn->ftype, tm = dm->ftype;
        put([=](StreamCoef &c) {
            float mix[kMaxStreams * kMaxStreams];
            Loader::widen(reinterpret_cast<uint8_t *>(c.in), si, S, ti);
            Loader::widen(reinterpret_cast<uint8_t *>(c.out), so, S, to);
            Loader::widen(reinterpret_cast<uint8_t *>(mix), sm, S * S, tm);
            for (uint32_t f = 0; f < S; f++) std::copy(mix + f * S, mix + f * S + S, c.mix + f * kMaxStreams);
        });
    };

    if (const lv_tensor_desc *d = tensor("embed", V, D)) {
        if (hp->tied_head) {           // one table for both ends, rows padded as the products want them
            const uint64_t off = ld.matrix({{d, 0, 0}}, V, Dp, &m->head);
            at(&m->head.w, off);
            at(&m->embed, off);
            m->embed_ld = Dp;
        } else {
            const uint8_t *src = ld.data(d);
            const uint64_t n = d->size;
            at(&m->embed, ld.place(n, [=](uint8_t *dst) { std::memcpy(dst, src, n); }));
            m->embed_ld = D;
        }
    }
    if (hp->bigram_buckets)
        if (const lv_tensor_desc *d = tensor("bigram", hp->bigram_buckets + 1, D)) {
            const uint8_t *src = ld.data(d);
            const uint64_t n = d->size;
            at(&m->bigram, ld.place(n, [=](uint8_t *dst) { std::memcpy(dst, src, n); }));
        }
    site(&m->final, "final.norm", "");
    if (!hp->tied_head)
        if (const lv_tensor_desc *d = tensor("head", V, D)) matrix(&m->head, {{d, 0, 0}}, V, Dp);
    std::vector<double> freqs;
    for (uint32_t i = 0; i < hp->layers && ld.error == LV_OK; i++) {
        BlockLayer &l = m->layers[i];
        l.spec = blocks[i];
        const lv_attn_spec &a = l.spec.attn;
        const lv_delta_spec &dl = l.spec.delta;
        const lv_moe_spec &e = l.spec.moe;
        l.attn = a.heads != 0;
        l.delta = dl.heads != 0;
        l.moe = e.experts != 0;
        const lv_latent_spec &lt = l.spec.latent;
        const lv_ssm_spec &sm = l.spec.ssm;
        const lv_dense_spec &dn = l.spec.dense;
        l.latent = lt.heads != 0;
        l.ssm = sm.heads != 0;
        l.dense = dn.ff != 0;
        const std::string p = "l" + std::to_string(i) + ".", pa = p + "mix.left.", pd = p + "mix.right.", px = p + "mix.", pm = p + "mlp.";
        site(&l.site[0], p + "norm1", p + "hc1.");
        if (l.ff()) site(&l.site[1], p + "norm2", p + "hc2.");
        std::vector<Part> in, outp;
        uint32_t row = 0;
        // convolution weights, [channel][tap] in the file, as [tap][channel]
        auto convolution = [&](std::vector<const lv_tensor_desc *> parts, uint32_t taps) {
            struct Src { const uint8_t *data; uint32_t rows, type; };
            std::vector<Src> src;
            size_t C = 0;
            for (const lv_tensor_desc *d : parts) {
                if (!d) return;
                src.push_back({ld.data(d), d->rows, d->ftype});
                C += d->rows;
            }
            at(&l.conv, ld.place((uint64_t)C * taps * 4, [=](uint8_t *dst) {
                std::vector<float> w(C * taps);
                size_t c0 = 0;
                for (const Src &q : src) {
                    Loader::widen(reinterpret_cast<uint8_t *>(w.data() + c0 * taps), q.data, q.rows * taps, q.type);
                    c0 += q.rows;
                }
                for (size_t c = 0; c < C; c++)
                    for (size_t j = 0; j < taps; j++) std::memcpy(dst + (j * C + c) * 4, &w[c * taps + j], 4);
            }));
        };
        auto section = [&](const std::string &name, uint32_t rows, uint32_t *off, uint32_t pad = 16) -> uint32_t {   // rows 0: the tensor's own
            const lv_tensor_desc *d = tensor(name, rows, D);
            if (!d) return 0;
            *off = row;
            in.push_back({d, row, 0});
            row += up(d->rows, pad);
            return d->rows;
        };
        if (l.attn) {
            section(pa + "q", a.heads * a.dim, &l.q_off);
            section(pa + "k", a.kv_heads * a.dim, &l.k_off);
            if (a.flags & LV_ATTN_KEYS_AS_VALUES) l.v_off = l.k_off;
            else section(pa + "v", a.kv_heads * a.vdim, &l.v_off);
            if (a.flags & LV_ATTN_NORM_FULL) {
                vec(&l.q_norm, pa + "q.norm", a.heads * a.dim, 1, a.heads * a.dim);
                vec(&l.k_norm, pa + "k.norm", a.kv_heads * a.dim, 1, a.kv_heads * a.dim);
            }
            if (a.flags & LV_ATTN_SINK) vec(&l.sink, pa + "sink", a.heads, 1, a.heads);
            if (a.rot_dims) {
                const uint32_t dims = a.rot_dims;
                const double rb = a.rot_base;
                at(&l.freq, ld.place((uint64_t)dims / 2 * 8, [=](uint8_t *dst) {
                    for (uint32_t k = 0; k < dims / 2; k++) {
                        const double f = frequency(rb, dims, k);
                        std::memcpy(dst + 8 * (size_t)k, &f, 8);
                    }
                }));
            }
            l.left_kp = up(a.heads * a.vdim, 64);
            if (const lv_tensor_desc *d = tensor(pa + "o", D, a.heads * a.vdim)) outp.push_back({d, 0, 0});
            l.dp = 64;
            while (l.dp < std::max(a.dim, a.vdim)) l.dp *= 2;
            const uint32_t per = a.heads / a.kv_heads;
            l.groups = (per + 7) / 8;
            const uint32_t rr = (per + l.groups - 1) / l.groups;
            l.r = rr == 1 ? 1 : rr <= 4 ? 4 : 8;
            l.groups = (per + l.r - 1) / l.r;
        }
        if (l.delta) {
            section(pd + "q", dl.kv_heads * dl.dim, &l.dq_off);
            section(pd + "k", dl.kv_heads * dl.dim, &l.dk_off);
            section(pd + "v", dl.heads * dl.vdim, &l.dv_off);
            section(pd + "b", dl.heads, &l.b_off);
            l.a_rank = section(pd + "a1", 0, &l.a_off);
            l.g_rank = section(pd + "g1", 0, &l.g_off);
            if (l.a_rank > kDeltaMaxRank || l.g_rank > kDeltaMaxRank) ld.error = fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: ranks %u and %u", i, l.a_rank, l.g_rank);
            if (const lv_tensor_desc *d = tensor(pd + "a2", dl.heads * dl.dim, l.a_rank)) matrix(&l.a2, {{d, 0, 0}}, d->rows, up(l.a_rank, 64));
            if (const lv_tensor_desc *d = tensor(pd + "g2", dl.heads * dl.vdim, l.g_rank)) matrix(&l.g2, {{d, 0, 0}}, d->rows, up(l.g_rank, 64));
            if (const lv_tensor_desc *d = tensor(pd + "o", D, dl.heads * dl.vdim)) outp.push_back({d, 0, l.left_kp});
            const uint32_t nq = dl.kv_heads * dl.dim, nv = dl.heads * dl.vdim, taps = dl.conv;
            convolution({ld.find(pd + "q.conv", nq, taps, true), ld.find(pd + "k.conv", nq, taps, true), ld.find(pd + "v.conv", nv, taps, true)}, taps);
            vec(&l.a_log, pd + "A_log", dl.heads, 1, dl.heads);
            vec(&l.dt_bias, pd + "dt_bias", dl.heads * dl.dim, 1, dl.heads * dl.dim);
            vec(&l.onorm, pd + "norm", dl.vdim, 1, dl.vdim);
        }
        if (l.latent) {
            const uint32_t size = lt.dim + lt.rot_dim, kv_p = up(lt.kv_rank, 64), dim_p = up(lt.dim, 64);
            section(px + "dq", lt.q_rank, &l.q_off, 64);       // its rows are the columns of the next product: zero to the next 64
            section(px + "dkv", lt.kv_rank + lt.rot_dim, &l.k_off);
            vec(&l.q_norm, px + "dq.norm", lt.q_rank, 1, up(lt.q_rank, 64));
            vec(&l.k_norm, px + "dkv.norm", lt.kv_rank, 1, kv_p);
            if (lt.flags & LV_ATTN_SINK) vec(&l.sink, px + "sink", lt.heads, 1, lt.heads);
            l.freq_at = (uint32_t)freqs.size();
            for (uint32_t k = 0; k < lt.rot_dims / 2; k++) freqs.push_back(frequency(lt.rot_base, lt.rot_dims, k));
            if (const lv_tensor_desc *d = tensor(px + "uq", lt.heads * size, lt.q_rank)) matrix(&l.uq, {{d, 0, 0}}, d->rows, up(lt.q_rank, 64));
            if (const lv_tensor_desc *d = tensor(px + "uk", lt.heads * lt.dim, lt.kv_rank)) {
                matrix(&l.uk, {{d, 0, 0}}, d->rows, kv_p);
                const uint8_t *src = ld.data(d);
                const uint32_t heads = lt.heads, dim = lt.dim, rank = lt.kv_rank;
                at(&l.uk_t, ld.place((uint64_t)heads * kv_p * dim_p * 2, [=](uint8_t *dst) {
                    for (uint64_t h = 0; h < heads; h++)
                        for (uint64_t c = 0; c < dim; c++)
                            for (uint64_t r = 0; r < rank; r++) std::memcpy(dst + ((h * kv_p + r) * dim_p + c) * 2, src + ((h * dim + c) * rank + r) * 2, 2);
                }));
            }
            if (const lv_tensor_desc *d = tensor(px + "uv", lt.heads * lt.vdim, lt.kv_rank)) matrix(&l.uv, {{d, 0, 0}}, d->rows, kv_p);
            if (const lv_tensor_desc *d = tensor(px + "o", D, lt.heads * lt.vdim)) outp.push_back({d, 0, 0});
            l.left_kp = up(lt.heads * lt.vdim, 64);
            l.kc = latent_kc(lt);
            l.width = latent_width(lt);
            l.dp = 64;
            while (l.dp < std::max(size, lt.vdim)) l.dp *= 2;
            if (m->f32) {
                l.dk = l.dv = l.dp;
            } else {
                constexpr uint32_t built[][2] = {{64, 64}, {128, 64}, {128, 128}, {192, 128}, {256, 256}};
                for (const auto &t : built) {
                    l.dk = t[0];
                    l.dv = t[1];
                    if (l.dk >= size && l.dv >= lt.vdim) break;
                }
            }
        }
        if (l.ssm) {
            const uint32_t inner = l.ssm_inner(), C = l.ssm_channels();
            section(px + "in", inner + C + sm.heads, &l.q_off);
            convolution({ld.find(px + "conv", C, sm.conv, true)}, sm.conv);
            vec(&l.conv_bias, px + "conv.b", C, 1, C);
            vec(&l.dt_bias, px + "dt_bias", sm.heads, 1, sm.heads);
            vec(&l.a_log, px + "A_log", sm.heads, 1, sm.heads);
            vec(&l.skip, px + "D", sm.heads, 1, sm.heads);
            vec(&l.onorm, px + "norm", inner, 1, inner);
            if (const lv_tensor_desc *d = tensor(px + "o", D, inner)) outp.push_back({d, 0, 0});
            l.left_kp = up(inner, 64);
        }
        matrix(&l.in, in, row, Dp);
        matrix(&l.out, outp, D, up(l.left_kp + dl.heads * dl.vdim, 64));
        // gate and up rows in alternating blocks of 16
        const uint32_t ffn = l.dense ? dn.ff : e.ff;
        auto pairs = [&](const std::string &name) -> uint64_t {
            const lv_tensor_desc *g = tensor(name + "gate", ffn, D), *u = tensor(name + "up", ffn, D);
            if (!g || !u) return 0;
            const uint8_t *sg = ld.data(g), *su = ld.data(u);
            return ld.place((uint64_t)l.gu_rows * Dp * 2, [=](uint8_t *dst) {
                for (uint32_t f = 0; f < ffn; f++) {
                    const uint64_t r = (uint64_t)(f / 16) * 32 + f % 16;
                    std::memcpy(dst + r * Dp * 2, sg + (uint64_t)f * D * 2, (size_t)D * 2);
                    std::memcpy(dst + (r + 16) * Dp * 2, su + (uint64_t)f * D * 2, (size_t)D * 2);
                }
            });
        };
        if (l.ff()) {
            l.gu_rows = up(up(ffn, 16) * 2, 128);
            l.down_rows = up(D, 128);
            l.gate_up.rows = l.gu_rows;
            l.gate_up.kp = Dp;
            l.down.rows = D;
            l.down.kp = l.gu_rows / 2;
        }
        if (l.dense) {
            at(&l.gate_up.w, pairs(pm));
            if (const lv_tensor_desc *d = tensor(pm + "down", D, ffn)) matrix(&l.down, {{d, 0, 0}}, D, l.gu_rows / 2);
        }
        if (l.moe) {
            if (const lv_tensor_desc *d = tensor(pm + "router", e.experts, D)) matrix(&l.router, {{d, 0, 0}}, e.experts, Dp);
            for (uint32_t x = 0; x < e.experts && ld.error == LV_OK; x++) {
                const uint64_t off = pairs(pm + "e" + std::to_string(x) + ".");
                if (x == 0) at(&l.gate_up.w, off);      // expert after expert: every block is a multiple of 256 bytes
            }
            for (uint32_t x = 0; x < e.experts && ld.error == LV_OK; x++) {
                const lv_tensor_desc *d = tensor(pm + "e" + std::to_string(x) + ".down", D, e.ff);
                if (!d) break;
                BfMatrix tmp;
                const uint64_t off = ld.matrix({{d, 0, 0}}, D, l.down.kp, &tmp);
                if (x == 0) at(&l.down.w, off);
            }
        }
        const uint32_t widest = std::max(std::max(l.out.kp + sm.norm_groups + 8, Dp + (l.moe ? e.experts : 0)), std::max(l.moe ? e.top * l.down.kp : l.down.kp, l.uq.kp));
        if (widest > 36864) ld.error = fail(LV_ERR_ARG, "lv_block_model_upload: layer %u: a product over %u columns (36864 are built)", i, widest);
    }
    if (ld.error != LV_OK) {
        delete m;
        return ld.error;
    }
    m->n_freq = (uint32_t)freqs.size();
    at(&m->freq, ld.place(freqs.size() * 8 + 8, [freqs](uint8_t *dst) { std::memcpy(dst, freqs.data(), freqs.size() * 8); }));
    // a GEMM tile of 256 rows may read up to 128 rows behind a matrix: of the next one, or of this margin
    uint32_t widest = Dp;
    for (const BlockLayer &l : m->layers) widest = std::max(widest, std::max({l.out.kp, l.down.kp, l.a2.kp, l.g2.kp, l.uq.kp, l.uk.kp}));
    ld.bytes += 256ull * widest;
    hipError_t er = hipMalloc(reinterpret_cast<void **>(&m->arena), ld.bytes);
    if (er != hipSuccess) {
        (void)hipGetLastError();
        delete m;
        return fail(er == hipErrorOutOfMemory ? LV_ERR_OOM : LV_ERR_HIP, "lv_block_model_upload: arena of %llu bytes: %s", (unsigned long long)ld.bytes, hipGetErrorString(er));
    }
    m->arena_bytes = ld.bytes;
    std::vector<uint8_t> staging;
    for (const Fill &f : ld.fills) {
        staging.assign(f.bytes, 0);
        f.fill(staging.data());
        er = hipMemcpyAsync(m->arena + f.off, staging.data(), f.bytes, hipMemcpyHostToDevice, st);
        if (er == hipSuccess) er = hipStreamSynchronize(st);
        if (er != hipSuccess) {
            (void)hipFree(m->arena);
            delete m;
            return fail(LV_ERR_HIP, "lv_block_model_upload: %s", hipGetErrorString(er));
        }
    }
    for (const Fix &f : fixes) {
        const uint8_t *p = m->arena + f.off;
        std::memcpy(f.at, &p, sizeof p);
    }
    *out = m;
    return LV_OK;
}

void block_model_destroy(BlockModel *m)
{
    if (!m) return;
    (void)hipFree(m->arena);
    delete m;
}

uint64_t block_model_bytes(const BlockModel *m) { return m->arena_bytes; }
uint32_t block_model_passes(const BlockModel *m) { return (uint32_t)m->order.size(); }

// ---------------------------------------------------------------------------------------------------------------------------
// session
// ---------------------------------------------------------------------------------------------------------------------------
template <class T> static int dev_alloc(T **p, uint64_t bytes)
{
    const hipError_t e = hipMalloc(reinterpret_cast<void **>(p), std::max<uint64_t>(bytes, 256));
    if (e == hipSuccess) return LV_OK;
    (void)hipGetLastError();
    *p = nullptr;
    return fail(e == hipErrorOutOfMemory ? LV_ERR_OOM : LV_ERR_HIP, "session: %llu bytes: %s", (unsigned long long)bytes, hipGetErrorString(e));
}
// zeroed, so that padding columns that no kernel writes are finite
template <class T> static int dev_zeroed(hipStream_t st, T **p, uint64_t bytes)
{
    bytes = (bytes + 255) / 256 * 256;
    LV_TRY(dev_alloc(p, bytes));
    return zero_async(*p, bytes, st);
}
template <class T> static void drop(T *&p)
{
    (void)hipFree((void *)p);
    p = nullptr;
}

template <class F> static uint32_t layer_max(const BlockModel *m, F f)
{
    uint32_t v = 0;
    for (const BlockLayer &l : m->layers) v = std::max<uint32_t>(v, f(l));
    return v;
}

int block_session_create(const BlockModel *m, hipStream_t st, BlockSession **out)
{
    *out = nullptr;
    BlockSession *s = new (std::nothrow) BlockSession;
    if (!s) return fail(LV_ERR_OOM, "session: host allocation");
    s->m = m;
    s->st = st;
    s->layers.resize(m->order.size());
    auto make = [&]() -> int {
        const uint32_t Dp = m->dp;
        LV_TRY(dev_zeroed(st, &s->xa, m->copies * Dp * 4ull));
        LV_TRY(dev_zeroed(st, &s->xb, m->copies * Dp * 4ull));
        LV_TRY(dev_zeroed(st, &s->last, 8));
        LV_TRY(dev_zeroed(st, &s->turn, 8ull * m->n_freq));
        LV_TRY(dev_zeroed(st, &s->yo, Dp * 4ull));
        LV_TRY(dev_zeroed(st, &s->yd, Dp * 4ull));
        LV_TRY(dev_zeroed(st, &s->h2, Dp * 4ull));
        LV_TRY(dev_zeroed(st, &s->y1, 4ull * layer_max(m, [](const BlockLayer &l) { return l.in.rows; })));
        LV_TRY(dev_zeroed(st, &s->left, 4ull * layer_max(m, [](const BlockLayer &l) { return l.left_kp; })));
        LV_TRY(dev_zeroed(st, &s->y2, 4ull * layer_max(m, [](const BlockLayer &l) { return l.uq.rows; })));
        LV_TRY(dev_zeroed(st, &s->ql, (m->f32 ? 4ull : 6ull) * layer_max(m, [](const BlockLayer &l) { return l.spec.latent.heads * l.width; })));
        const uint64_t hv = 4ull * layer_max(m, [](const BlockLayer &l) { return std::max(l.spec.delta.heads * l.spec.delta.vdim, l.ssm_inner()); });
        LV_TRY(dev_zeroed(st, &s->o, hv));
        LV_TRY(dev_zeroed(st, &s->gate, hv));
        LV_TRY(dev_zeroed(st, &s->z, 4ull * layer_max(m, [](const BlockLayer &l) { return l.spec.moe.experts; })));
        LV_TRY(dev_zeroed(st, &s->act, 4ull * layer_max(m, [](const BlockLayer &l) { return std::max(1u, l.spec.moe.top) * l.down.kp; })));
        LV_TRY(dev_zeroed(st, &s->scores, 4ull * kMaxTop));
        LV_TRY(dev_zeroed(st, &s->ids, 4ull * kMaxTop));
        LV_TRY(dev_zeroed(st, &s->counters, 4ull * layer_max(m, [](const BlockLayer &l) { return l.spec.attn.kv_heads * l.groups; })));
        for (size_t i = 0; i < m->order.size(); i++) {
            const BlockLayer &l = m->pass(i);
            if (!l.delta && !l.ssm) continue;
            LV_TRY(dev_zeroed(st, &s->layers[i].state, l.state_bytes()));
            LV_TRY(dev_zeroed(st, &s->layers[i].conv, l.ring_bytes()));
        }
        HIP_TRY(hipStreamSynchronize(st));
        return LV_OK;
    };
    const int rc = make();
    if (rc != LV_OK) {
        block_session_destroy(s);
        return rc;
    }
    *out = s;
    return LV_OK;
}

static void workspace_free(Workspace &w)
{
    for (float **p : {&w.x, &w.y1, &w.y, &w.dq, &w.dk, &w.dv, &w.dg, &w.beta, &w.qk, &w.o, &w.gate, &w.z, &w.scores, &w.y2, &w.sdt, &w.sdecay}) drop(*p);
    for (void **p : {&w.act, &w.q, &w.k, &w.v, &w.vt, &w.a1, &w.g1, &w.cat, &w.ff, &w.cq, &w.ek, &w.ev, &w.sx, &w.sb, &w.sc, &w.sbt}) drop(*p);
    for (uint32_t **p : {&w.ids, &w.slots, &w.tiles}) drop(*p);
    w.cap = 0;
    w.vt_elems = w.ek_elems = w.ev_elems = 0;
}

void block_session_destroy(BlockSession *s)
{
    if (!s) return;
    for (LayerState &l : s->layers) {
        drop(l.kc);
        drop(l.vc);
        drop(l.state);
        drop(l.conv);
    }
    for (float **p : {&s->xa, &s->xb, &s->y1, &s->left, &s->o, &s->gate, &s->yo, &s->h2, &s->z, &s->act, &s->yd, &s->scores, &s->part, &s->y2}) drop(*p);
    drop(s->ql);
    drop(s->ids);
    drop(s->last);
    drop(s->turn);
    drop(s->counters);
    workspace_free(s->ws);
    delete s;
}

uint32_t block_session_position(const BlockSession *s) { return s->valid ? s->position : 0; }
void block_session_invalidate(BlockSession *s)
{
    s->valid = false;
    s->position = 0;
}
void block_session_advance(BlockSession *s, uint32_t pos)
{
    s->valid = true;
    s->position = pos;
}

int block_session_reserve(BlockSession *s, uint32_t positions)
{
    const BlockModel *m = s->m;
    uint64_t part = 0;
    for (size_t i = 0; i < m->order.size(); i++) {
        const BlockLayer &l = m->pass(i);
        if (!l.attn && !l.latent) continue;
        LayerState &ls = s->layers[i];
        const uint32_t ring = l.attn && l.spec.attn.chunk ? std::min(l.spec.attn.chunk, positions) : positions;
        if (l.attn) {
            const uint64_t splits = (ring + gqa_split(l.dp) - 1) / gqa_split(l.dp);
            part = std::max<uint64_t>(part, l.spec.attn.kv_heads * l.groups * splits * l.r * (l.dp + 2));
        } else {
            part = std::max<uint64_t>(part, ((uint64_t)l.spec.latent.heads * latent_part_stride(l.kc)) << latent_split_bits(l.spec.latent.heads, positions));
        }
        if (ring == ls.ring) continue;
        // A ring that grows has not wrapped yet (it held every position so far), and one that shrinks keeps the rows that
        // the smaller number of positions can have: row = position in both.  Latent rows are read by tiles of 128.
        const uint64_t row = (l.attn ? (uint64_t)l.spec.attn.kv_heads * l.dp : l.width) * m->elem(), keep = std::min(ring, ls.ring), rows = l.attn ? ring : up(ring, 128);
        uint8_t *fresh[2] = {nullptr, nullptr};
        for (int w = 0; w < (l.attn ? 2 : 1); w++) {
            int rc = dev_zeroed(s->st, &fresh[w], rows * row);
            if (rc == LV_OK && keep && hipMemcpyAsync(fresh[w], w ? ls.vc : ls.kc, keep * row, hipMemcpyDeviceToDevice, s->st) != hipSuccess)
                rc = fail(LV_ERR_HIP, "session: cache copy");
            if (rc != LV_OK) {
                (void)hipStreamSynchronize(s->st);
                drop(fresh[0]);
                drop(fresh[1]);
                return rc;
            }
        }
        HIP_TRY(hipStreamSynchronize(s->st));
        drop(ls.kc);
        drop(ls.vc);
        ls.kc = fresh[0];
        ls.vc = fresh[1];
        ls.ring = ring;
    }
    HIP_TRY(hipStreamSynchronize(s->st));
    drop(s->part);
    LV_TRY(dev_alloc(&s->part, part * 4));
    s->positions = positions;
    return LV_OK;
}

// ---------------------------------------------------------------------------------------------------------------------------
// launches
// ---------------------------------------------------------------------------------------------------------------------------
template <class K> static int allow_lds(K kernel, size_t bytes)
{
    if (bytes > 65536) HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes));
    return LV_OK;
}

template <int MODE, int INPUT, int R, int DEPTH> static int launch_gemv(hipStream_t st, const BfGemvArgs &a, uint32_t units, size_t lds)
{
    const uint32_t per_wg = kBfGemvWaves * R, wgs = std::min((units + per_wg - 1) / per_wg, 512u);
    auto *k = &bf16_gemv_kernel<MODE, INPUT, R, DEPTH>;
    LV_TRY(allow_lds(k, lds));
    k<<<dim3(wgs), dim3(kBfGemvThreads), lds, st>>>(a);
    HIP_TRY(hipGetLastError());
    return LV_OK;
}

// Rows a wave walks together: as many as still give every wave of the chip work, fewer where the last round of waves would then be
// far from full.
static uint32_t gemv_rows_together(uint32_t units, uint32_t most)
{
    constexpr uint32_t kWaves = 512 * kBfGemvWaves;
    auto rows_in_turn = [&](uint32_t r) { return ((units + r - 1) / r + kWaves - 1) / kWaves * r; };      // of the busiest wave
    uint32_t best = most;
    for (uint32_t r = most / 2; r; r /= 2)
        if (rows_in_turn(r) < rows_in_turn(best)) best = r;
    return best;
}

template <int MODE, int INPUT> static int gemv(hipStream_t st, const BfGemvArgs &a)
{
    const size_t lds = (size_t)a.kp * (MODE == kGemvDown ? a.top : 1) * 4 + (MODE == kGemvExperts ? a.experts * 4ull : 0) +
                       (INPUT == kInGroups ? group_sums(a.group.groups, kBfGemvWaves) * 4ull : 0);
    if constexpr (MODE == kGemvExperts || MODE == kGemvGlu) {
        const uint32_t units = MODE == kGemvExperts ? a.top * (a.expert_rows / 2) : a.rows / 2, r = gemv_rows_together(units, units >= 8192 ? 2 : 1);
        return r == 2 ? launch_gemv<MODE, INPUT, 2, 2>(st, a, units, lds) : launch_gemv<MODE, INPUT, 1, 4>(st, a, units, lds);
    } else {
        const uint32_t r = gemv_rows_together(a.rows, a.rows >= 16384 ? 4 : a.rows >= 8192 ? 2 : 1);
        return r == 4 ? launch_gemv<MODE, INPUT, 4, 2>(st, a, a.rows, lds) : r == 2 ? launch_gemv<MODE, INPUT, 2, 4>(st, a, a.rows, lds)
                                                                                    : launch_gemv<MODE, INPUT, 1, 8>(st, a, a.rows, lds);
    }
}

template <int EP, bool GROUPED, int NW> static int launch_bf_gemm(hipStream_t st, BfGemmArgs a)
{
    auto *k = &gemm_bf16_kernel<EP, GROUPED, NW>;
    a.row_tiles = (a.rows + bf_tile_rows(NW) - 1) / bf_tile_rows(NW);
    LV_TRY(allow_lds(k, bf_lds_bytes(NW)));
    k<<<dim3(bf_grid(a), 1, a.k_slice ? (a.kp + a.k_slice - 1) / a.k_slice : 1), dim3(NW * 64), bf_lds_bytes(NW), st>>>(a);
    HIP_TRY(hipGetLastError());
    return LV_OK;
}

template <int EP, bool GROUPED> static int gemm(hipStream_t st, bool f32, BfGemmArgs a, const BfMatrix &w, uint32_t n, uint32_t experts = 1)
{
    const uint32_t tile = f32 ? kF32Tile : kBfTile, token_tiles = (n + tile - 1) / tile;
    a.w = w.w;
    a.kp = w.kp;
    a.rows = w.rows;
    a.n = n;
    a.token_tiles = GROUPED ? std::min(token_tiles + experts, n) : token_tiles;
    if (f32) {
        a.row_tiles = (w.rows + tile - 1) / tile;
        gemm_f32_kernel<EP, GROUPED><<<dim3(bf_grid(a)), dim3(256), 0, st>>>(a);
        HIP_TRY(hipGetLastError());
        return LV_OK;
    }
    if constexpr (EP != kEpDecay && EP != kEpSigmoid) {      // those two have a few K steps only
        const uint64_t big_tiles = (uint64_t)((w.rows + 255) / 256) * std::max(token_tiles, GROUPED ? experts : 1u);
        if (big_tiles >= 256) return launch_bf_gemm<EP, GROUPED, 8>(st, a);
    }
    return launch_bf_gemm<EP, GROUPED, 4>(st, a);
}

// calls fn(element, integral constant DP, integral constant R) for a layer's attention
template <class Fn> static int gqa_dispatch(bool f32, const BlockLayer &l, Fn &&fn)
{
    auto with_r = [&](auto elem, auto dp) -> int {
        switch (l.r) {
        case 1: return fn(elem, dp, std::integral_constant<int, 1>{});
        case 4: return fn(elem, dp, std::integral_constant<int, 4>{});
        default: return fn(elem, dp, std::integral_constant<int, 8>{});
        }
    };
    auto with_dp = [&](auto elem) -> int {
        switch (l.dp) {
        case 64: return with_r(elem, std::integral_constant<int, 64>{});
        case 128: return with_r(elem, std::integral_constant<int, 128>{});
        default: return with_r(elem, std::integral_constant<int, 256>{});
        }
    };
    return f32 ? with_dp(float{}) : with_dp(uint16_t{});
}

// calls fn(integral constant J) for a delta rule's key channels in units of 64
template <class Fn> static int with_j(uint32_t j, Fn &&fn)
{
    switch (j) {
    case 1: return fn(std::integral_constant<int, 1>{});
    case 2: return fn(std::integral_constant<int, 2>{});
    case 3: return fn(std::integral_constant<int, 3>{});
    default: return fn(std::integral_constant<int, 4>{});
    }
}

// the same for a state-space recurrence's entries
template <class Fn> static int with_state(uint32_t j, Fn &&fn)
{
    switch (j) {
    case 1: return fn(std::integral_constant<int, 1>{});
    case 2: return fn(std::integral_constant<int, 2>{});
    default: return fn(std::integral_constant<int, 4>{});
    }
}

static GqaSpec gqa_spec(const BlockSession *s, size_t i)
{
    const BlockLayer &l = s->m->pass(i);
    const lv_attn_spec &a = l.spec.attn;
    GqaSpec g{};
    if (!l.attn) return g;
    g.heads = a.heads; g.kv_heads = a.kv_heads; g.dim = a.dim; g.vdim = a.vdim;
    g.q_off = l.q_off; g.k_off = l.k_off; g.v_off = l.v_off;
    g.q_norm = l.q_norm; g.k_norm = l.k_norm; g.sink = l.sink; g.freq = l.freq;
    g.rot_dims = a.rot_dims; g.chunk = a.chunk; g.scale = a.scale; g.eps = s->m->hp.eps;
    g.kc = s->layers[i].kc; g.vc = s->layers[i].vc;
    return g;
}

static DeltaSpec delta_spec(const BlockSession *s, size_t i)
{
    const BlockLayer &l = s->m->pass(i);
    const lv_delta_spec &d = l.spec.delta;
    DeltaSpec g{};
    if (!l.delta) return g;
    g.heads = d.heads; g.kv_heads = d.kv_heads; g.dim = d.dim; g.vdim = d.vdim; g.taps = d.conv;
    g.q_off = l.dq_off; g.k_off = l.dk_off; g.v_off = l.dv_off; g.b_off = l.b_off; g.a_off = l.a_off; g.g_off = l.g_off;
    g.a_rank = l.a_rank; g.g_rank = l.g_rank; g.a_kp = l.a2.kp; g.g_kp = l.g2.kp;
    g.conv = l.conv; g.a_log = l.a_log; g.dt_bias = l.dt_bias; g.norm = l.onorm;
    g.a2 = l.a2.w; g.g2 = l.g2.w; g.eps = s->m->hp.eps;
    g.state = s->layers[i].state; g.ring = s->layers[i].conv; g.dstride = l.dstride();
    return g;
}

static LatentSpec latent_spec(const BlockSession *s, size_t i)
{
    const BlockLayer &l = s->m->pass(i);
    const lv_latent_spec &a = l.spec.latent;
    LatentSpec g{};
    g.heads = a.heads; g.dim = a.dim; g.rot_dim = a.rot_dim; g.rot_dims = a.rot_dims; g.vdim = a.vdim; g.q_rank = a.q_rank; g.kv_rank = a.kv_rank;
    g.q_off = l.q_off; g.kv_off = l.k_off; g.kc = l.kc; g.width = l.width; g.dim_p = up(a.dim, 64); g.kv_p = l.uv.kp;
    g.q_norm = l.q_norm; g.kv_norm = l.k_norm; g.sink = l.sink; g.freq = s->m->freq + l.freq_at; g.turn = s->turn + l.freq_at;
    g.uk_t = l.uk_t; g.uv = l.uv.w; g.scale = a.scale; g.eps = s->m->hp.eps; g.cache = s->layers[i].kc;
    return g;
}

static SsmSpec ssm_spec(const BlockSession *s, size_t i)
{
    const BlockLayer &l = s->m->pass(i);
    const lv_ssm_spec &a = l.spec.ssm;
    SsmSpec g{};
    g.heads = a.heads; g.groups = a.groups; g.n = a.state; g.vdim = a.vdim; g.taps = a.conv; g.norm_groups = a.norm_groups;
    g.z_off = l.q_off; g.x_off = l.q_off + l.ssm_inner(); g.dt_off = g.x_off + l.ssm_channels();
    g.conv = l.conv; g.bias = l.conv_bias; g.a_log = l.a_log; g.dt_bias = l.dt_bias; g.skip = l.skip; g.norm = l.onorm;
    g.eps = s->m->hp.eps; g.state = s->layers[i].state; g.ring = s->layers[i].conv; g.nstride = l.sstride();
    return g;
}

static GroupInput group_in(const SsmSpec &m, const float *o, const float *y) { return {o, y + m.z_off, m.norm, m.inner(), m.norm_groups, m.eps}; }

static NormInput norm_in(const BlockModel *m, const float *x, const NormSite &to)
{
    NormInput n{};
    n.x = x; n.wpre = to.w; n.dim = m->hp.dim; n.dp = m->dp; n.parts = 1; n.part_stride = m->dp; n.eps = m->hp.eps;
    return n;
}
static StreamInput stream_in(const BlockModel *m, const float *x, const NormSite &to)
{
    StreamInput n{};
    n.x = x; n.gather = to.coef; n.w = to.w; n.b = to.b; n.alpha = to.alpha; n.dim = m->hp.dim; n.dp = m->dp; n.streams = m->hp.streams; n.eps = m->hp.eps;
    return n;
}

// a product of one token whose input is the norm of the residual, formed in the launch's head
template <int MODE> static int gemv_residual(const BlockModel *m, hipStream_t st, const BfGemvArgs &g)
{
    const uint32_t n = m->hp.streams;
    if (!n) return gemv<MODE, kInNorm>(st, g);
    return n <= 2 ? gemv<MODE, kInStreams2>(st, g) : n <= 4 ? gemv<MODE, kInStreams4>(st, g) : gemv<MODE, kInStreams8>(st, g);
}

// The residual of one token: a sublayer's output waits until the next launch that reads the residual takes it in.
class TokenResidual {
public:
    TokenResidual(const BlockModel *m, float *a, float *b) : cur(a), m_(m), other_(b) {}
    float *cur;
    void add(const float *y, const NormSite &from)
    {
        y_ = y;
        from_ = &from;
    }
    // g's input: the norm of the residual at `to`.  keep: the residual is read again afterwards
    void feed(BfGemvArgs &g, const NormSite &to, float *h_out = nullptr, bool keep = true)
    {
        if (m_->hp.streams) {
            g.streams = stream_in(m_, cur, to);
            g.streams.h_out = h_out;
            if (y_) {
                g.streams.y = y_;
                g.streams.spread = from_->coef;
                if (keep) g.streams.x_out = other_;
            }
        } else {
            g.norm = norm_in(m_, cur, to);
            g.norm.h_out = h_out;
            if (y_) {
                g.norm.y = y_;
                g.norm.wpost = from_->post;
                if (keep) g.norm.x_out = other_;
            }
        }
        if (y_ && keep) {
            std::swap(cur, other_);
            y_ = nullptr;
        }
    }

private:
    const BlockModel *m_;
    float *other_;
    const float *y_ = nullptr;
    const NormSite *from_ = nullptr;
};

static int embed(BlockSession *s, float *x, const uint32_t *cfg, uint32_t idx, uint32_t n)
{
    const BlockModel *m = s->m;
    EmbedArgs e{};
    e.x = x; e.table = m->embed; e.ld = m->embed_ld; e.dim = m->hp.dim; e.dp = m->dp; e.streams = m->copies; e.scale = m->hp.embed_scale ? m->hp.embed_scale : 1.f;
    e.cfg = cfg; e.idx = idx; e.bigram = m->bigram; e.buckets = m->hp.bigram_buckets; e.prev = m->hp.bigram_prev; e.cur = m->hp.bigram_cur; e.last = s->last;
    if (n == 1) {
        e.freq = m->freq;
        e.turn = s->turn;
        e.n_freq = m->n_freq;
    }
    embed_bf16_kernel<<<dim3((std::max(m->dp / 4, e.n_freq) + 255) / 256, n), dim3(256), 0, s->st>>>(e);
    HIP_TRY(hipGetLastError());
    return LV_OK;
}

// copies the residual of rows `row` .. row + n - 1 of a step (the sum of its streams) to the trace
static int trace_residual(const BlockModel *m, hipStream_t st, const BlockTrace *t, uint32_t layer, int which, uint32_t row, uint32_t n, const float *x)
{
    if (!t) return LV_OK;
    if (m->hp.streams) {
        stream_sum_kernel<<<dim3((m->hp.dim + 255) / 256, n), dim3(256), 0, st>>>(t->slot(layer, which, row), t->stride, x, m->hp.streams, m->hp.dim, m->dp);
        HIP_TRY(hipGetLastError());
    } else {
        HIP_TRY(hipMemcpy2DAsync(t->slot(layer, which, row), t->stride * 4ull, x, m->dp * 4ull, m->hp.dim * 4ull, n, hipMemcpyDeviceToDevice, st));
    }
    return LV_OK;
}

template <class T> static int stream_rows(hipStream_t st, const StreamRowsArgs &a, uint32_t n)
{
    auto run = [&](auto ns) -> int {
        auto *k = &stream_rows_kernel<T, decltype(ns)::value>;
        const size_t lds = a.in.dp * (a.in.y && a.parts > 1 ? 8ull : 4ull);
        LV_TRY(allow_lds(k, lds));
        k<<<dim3(n), dim3(256), lds, st>>>(a);
        HIP_TRY(hipGetLastError());
        return LV_OK;
    };
    using std::integral_constant;
    return a.in.streams <= 2 ? run(integral_constant<int, 2>{}) : a.in.streams <= 4 ? run(integral_constant<int, 4>{}) : run(integral_constant<int, 8>{});
}

template <class T> static int norm_rows(hipStream_t st, const NormRowsArgs &a, uint32_t n)
{
    const size_t lds = a.in.dp * 4ull;
    LV_TRY(allow_lds(&norm_rows_kernel<T>, lds));
    norm_rows_kernel<T><<<dim3(n), dim3(256), lds, st>>>(a);
    HIP_TRY(hipGetLastError());
    return LV_OK;
}

// ---- mixers of one token: from the joint projection in s->y1 to the arguments of the output projection ----------------------
static int token_branches(BlockSession *s, size_t i, const uint32_t *cfg, uint32_t idx, BfGemvArgs &o)
{
    const BlockModel *m = s->m;
    const BlockLayer &l = m->pass(i);
    MixStepArgs mx{};
    mx.delta.s = delta_spec(s, i);
    mx.delta.y = s->y1; mx.delta.pos_ptr = cfg; mx.delta.pos_add = idx;
    mx.delta.blocks = l.delta ? (l.spec.delta.vdim + kDeltaCols - 1) / kDeltaCols : 1;
    mx.delta.o = s->o; mx.delta.gate = s->gate;
    mx.delta_wgs = l.spec.delta.heads * mx.delta.blocks;
    mx.attn.s = gqa_spec(s, i);
    mx.attn.y = s->y1; mx.attn.pos_ptr = cfg; mx.attn.pos_add = idx;
    mx.attn.groups = l.groups;
    mx.attn.splits = l.attn ? (s->layers[i].ring + gqa_split(l.dp) - 1) / gqa_split(l.dp) : 1;
    mx.attn.part = s->part; mx.attn.counters = s->counters; mx.attn.out = s->left;
    const uint32_t wgs = mx.delta_wgs + (l.attn ? l.spec.attn.kv_heads * l.groups * mx.attn.splits : 0);
    LV_TRY(gqa_dispatch(m->f32, l, [&](auto elem, auto dp, auto r) -> int {
        constexpr int DP = decltype(dp)::value, R = decltype(r)::value;
        const size_t lds = 4ull * std::max<uint32_t>(l.attn ? gqa_lds_floats<DP, R, kGqaStepThreads>() : 0, l.delta ? delta_step_lds_floats(l.a2.kp, l.g2.kp) : 0);
        auto *k = &mix_step_kernel<decltype(elem), DP, R>;
        LV_TRY(allow_lds(k, lds));
        k<<<dim3(wgs), dim3(kGqaStepThreads), lds, s->st>>>(mx);
        HIP_TRY(hipGetLastError());
        return LV_OK;
    }));
    o.branch = {s->left, s->o, s->gate, l.onorm, l.spec.attn.heads * l.spec.attn.vdim, l.left_kp, l.spec.delta.heads, l.spec.delta.vdim,
                l.spec.attn_scale, l.spec.delta_scale, m->hp.eps};
    return gemv<kGemvRows, kInBranch>(s->st, o);
}

template <class CT> static int token_latent(BlockSession *s, size_t i, const uint32_t *cfg, uint32_t idx, BfGemvArgs &o)
{
    const BlockLayer &l = s->m->pass(i);
    const LatentSpec sp = latent_spec(s, i);
    BfGemvArgs q{};
    q.w = l.uq.w; q.rows = l.uq.rows; q.kp = l.uq.kp; q.out = s->y2;
    q.norm = {s->y1 + l.q_off, nullptr, nullptr, l.q_norm, nullptr, nullptr, sp.q_rank, l.uq.kp, 1, 0, sp.eps};
    LV_TRY((gemv<kGemvRows, kInNorm>(s->st, q)));
    latent_absorb_kernel<CT><<<dim3(sp.heads * (sp.kv_p / kAbsorbRows) + 1), dim3(256), 0, s->st>>>(LatentAbsorbArgs{sp, s->y1, s->y2, cfg, idx, s->ql});
    HIP_TRY(hipGetLastError());
    LatentStepArgs a{};
    a.s = sp; a.q = s->ql; a.pos_ptr = cfg; a.pos_add = idx; a.split_bits = latent_split_bits(sp.heads, s->positions); a.part = s->part; a.out = s->left;
    auto attend = [&](auto nq, auto nb) -> int {
        auto *k = &latent_attn_kernel<CT, decltype(nq)::value, decltype(nb)::value>;
        const size_t lds = latent_attn_lds<CT>(sp.width);
        LV_TRY(allow_lds(k, lds));
        k<<<dim3(latent_groups(sp.heads), 1u << a.split_bits), dim3(kLatentStepThreads), lds, s->st>>>(a);
        HIP_TRY(hipGetLastError());
        return LV_OK;
    };
    static_assert(kLatentMaxWidth <= 6 * 128, "pieces of a cache row");
    using std::integral_constant;
    using One = integral_constant<int, 1>;
    LV_TRY(sp.width <= 256                   ? attend(integral_constant<int, 2>{}, One{})
           : sp.width <= 640 && sp.kc <= 512 ? attend(integral_constant<int, 5>{}, One{})
                                             : attend(integral_constant<int, 6>{}, integral_constant<int, 2>{}));
    latent_value_kernel<<<dim3(sp.heads, (sp.vdim + kLatentValueRows - 1) / kLatentValueRows), dim3(kLatentStepThreads), 0, s->st>>>(a);
    HIP_TRY(hipGetLastError());
    o.x = s->left;
    return gemv<kGemvRows, kInPlain>(s->st, o);
}

static int token_ssm(BlockSession *s, size_t i, const uint32_t *cfg, uint32_t idx, BfGemvArgs &o)
{
    const SsmSpec sp = ssm_spec(s, i);
    SsmStepArgs a{sp, s->y1, cfg, idx, (sp.vdim + kSsmCols - 1) / kSsmCols, s->o};
    ssm_step_kernel<<<dim3(sp.heads * a.blocks), dim3(kSsmStepThreads), 0, s->st>>>(a);
    HIP_TRY(hipGetLastError());
    o.group = group_in(sp, s->o, s->y1);
    return gemv<kGemvRows, kInGroups>(s->st, o);
}

int block_step_token(BlockSession *s, const uint32_t *cfg, uint32_t idx, float *logits, const BlockTrace *trace)
{
    const BlockModel *m = s->m;
    hipStream_t st = s->st;
    const uint32_t D = m->hp.dim, Dp = m->dp;
    LV_TRY(embed(s, s->xa, cfg, idx, 1));
    TokenResidual res(m, s->xa, s->xb);
    auto keep = [&](uint32_t pass, int which) { return trace_residual(m, st, trace, pass, which, idx, 1, res.cur); };
    auto keep_end = [&](uint32_t pass) -> int {      // the residual behind a pass
        if (!m->pass(pass).ff()) LV_TRY(keep(pass, LV_TRACE_POST_ATTN));
        return keep(pass, LV_TRACE_OUT);
    };
    for (size_t i = 0; i < m->order.size(); i++) {
        const BlockLayer &l = m->pass(i);
        BfGemvArgs g{};
        g.w = l.in.w; g.rows = l.in.rows; g.kp = Dp; g.out = s->y1;
        res.feed(g, l.site[0]);
        LV_TRY(gemv_residual<kGemvRows>(m, st, g));
        if (i) LV_TRY(keep_end((uint32_t)i - 1));

        BfGemvArgs o{};
        o.w = l.out.w; o.rows = D; o.kp = l.out.kp; o.out = s->yo;
        if (l.latent) LV_TRY(m->f32 ? token_latent<float>(s, i, cfg, idx, o) : token_latent<uint16_t>(s, i, cfg, idx, o));
        else if (l.ssm) LV_TRY(token_ssm(s, i, cfg, idx, o));
        else LV_TRY(token_branches(s, i, cfg, idx, o));
        res.add(s->yo, l.site[0]);
        if (!l.ff()) continue;

        BfGemvArgs dn{};
        dn.w = l.down.w; dn.rows = D; dn.kp = l.down.kp; dn.out = s->yd; dn.x = s->act;
        if (l.dense) {
            BfGemvArgs gu{};
            gu.w = l.gate_up.w; gu.rows = l.gu_rows; gu.kp = Dp; gu.out = s->act; gu.act = l.spec.dense.act;
            res.feed(gu, l.site[1]);
            LV_TRY(gemv_residual<kGemvGlu>(m, st, gu));
            LV_TRY(keep((uint32_t)i, LV_TRACE_POST_ATTN));
            LV_TRY((gemv<kGemvRows, kInPlain>(st, dn)));
        } else {
            BfGemvArgs rt{};
            rt.w = l.router.w; rt.rows = l.spec.moe.experts; rt.kp = Dp; rt.out = s->z;
            res.feed(rt, l.site[1], s->h2);
            LV_TRY(gemv_residual<kGemvRows>(m, st, rt));
            LV_TRY(keep((uint32_t)i, LV_TRACE_POST_ATTN));
            BfGemvArgs gu{};
            gu.w = l.gate_up.w; gu.rows = l.gu_rows; gu.kp = Dp; gu.out = s->act; gu.x = s->h2;
            gu.z = s->z; gu.experts = l.spec.moe.experts; gu.top = l.spec.moe.top; gu.expert_rows = l.gu_rows; gu.ids = s->ids; gu.scores = s->scores;
            LV_TRY((gemv<kGemvExperts, kInPlain>(st, gu)));
            dn.top = l.spec.moe.top; dn.expert_rows = l.down_rows; dn.ids = s->ids;
            LV_TRY((gemv<kGemvDown, kInPlain>(st, dn)));
        }
        res.add(s->yd, l.site[1]);
    }
    if (trace) {      // the residual behind the last layer, which otherwise only the head's input holds
        BfGemvArgs g{};
        res.feed(g, m->final);
        if (m->hp.streams) {
            StreamRowsArgs a{};
            a.in = g.streams;
            a.parts = 1;
            LV_TRY(stream_rows<float>(st, a, 1));
        } else {
            NormRowsArgs a{};
            a.in = g.norm;
            LV_TRY(norm_rows<float>(st, a, 1));
        }
        LV_TRY(keep_end((uint32_t)m->order.size() - 1));
    }
    if (logits) {
        BfGemvArgs h{};
        h.w = m->head.w; h.rows = m->hp.vocab; h.kp = Dp; h.out = logits;
        res.feed(h, m->final, nullptr, false);
        LV_TRY(gemv_residual<kGemvRows>(m, st, h));
    }
    return LV_OK;
}

// router logits of a batch: K in at most so many slices, each a multiple of so many columns
constexpr uint32_t kRouterParts = 8, kRouterSlice = 128;

// ---- batches ---------------------------------------------------------------------------------------------------------------
static int workspace_reserve(BlockSession *s, uint32_t n)
{
    const BlockModel *m = s->m;
    Workspace &w = s->ws;
    const uint32_t cap = up(n, 128);
    if (cap <= w.cap) return LV_OK;
    HIP_TRY(hipStreamSynchronize(s->st));
    workspace_free(w);
    const uint64_t T = cap, E = m->elem();
    auto mx = [&](auto f) -> uint64_t { return layer_max(m, f); };
    hipStream_t st = s->st;
    LV_TRY(dev_zeroed(st, &w.x, T * m->copies * m->dp * 4));
    LV_TRY(dev_zeroed(st, &w.act, T * m->dp * E));
    LV_TRY(dev_zeroed(st, &w.y1, T * mx([](const BlockLayer &l) { return l.in.rows; }) * 4));
    LV_TRY(dev_zeroed(st, &w.y, T * m->dp * 4 * mx([](const BlockLayer &l) { return std::max(1u, l.spec.moe.top); })));
    LV_TRY(dev_zeroed(st, &w.q, T * E * mx([](const BlockLayer &l) { return std::max(l.spec.attn.heads * l.dp, l.spec.latent.heads * l.dk); })));
    const uint64_t kv = mx([](const BlockLayer &l) { return l.spec.attn.kv_heads * l.dp; });
    LV_TRY(dev_zeroed(st, &w.k, T * E * kv));
    LV_TRY(dev_zeroed(st, &w.v, T * E * kv));
    const uint64_t dk = mx([](const BlockLayer &l) { return l.delta ? l.spec.delta.kv_heads * l.dstride() : 0u; });
    LV_TRY(dev_zeroed(st, &w.dq, T * 4 * dk));
    LV_TRY(dev_zeroed(st, &w.dk, T * 4 * dk));
    LV_TRY(dev_zeroed(st, &w.dg, T * 4 * mx([](const BlockLayer &l) { return l.delta ? l.spec.delta.heads * l.dstride() : 0u; })));
    const uint64_t hv = mx([](const BlockLayer &l) { return l.spec.delta.heads * l.spec.delta.vdim; });
    LV_TRY(dev_zeroed(st, &w.dv, T * 4 * hv));
    LV_TRY(dev_zeroed(st, &w.o, T * 4 * std::max<uint64_t>(hv, mx([](const BlockLayer &l) { return l.ssm_inner(); }))));
    LV_TRY(dev_zeroed(st, &w.y2, T * 4 * mx([](const BlockLayer &l) { return l.uq.rows; })));
    LV_TRY(dev_zeroed(st, &w.cq, T * E * mx([](const BlockLayer &l) { return l.uq.kp; })));
    LV_TRY(dev_zeroed(st, &w.sx, T * E * mx([](const BlockLayer &l) { return l.ssm_inner(); })));
    const uint64_t bc = mx([](const BlockLayer &l) { return l.spec.ssm.groups * l.sstride(); }), sh = mx([](const BlockLayer &l) { return l.spec.ssm.heads; });
    LV_TRY(dev_zeroed(st, &w.sb, T * E * bc));
    LV_TRY(dev_zeroed(st, &w.sc, T * E * bc));
    LV_TRY(dev_zeroed(st, &w.sbt, m->f32 ? 0 : T * E * bc));
    LV_TRY(dev_zeroed(st, &w.sdt, T * 4 * sh));
    LV_TRY(dev_zeroed(st, &w.sdecay, m->f32 ? T * 4 * sh : 0));
    LV_TRY(dev_zeroed(st, &w.gate, T * 4 * hv));
    const uint64_t heads = mx([](const BlockLayer &l) { return l.spec.delta.heads; });
    LV_TRY(dev_zeroed(st, &w.beta, T * 4 * heads));
    LV_TRY(dev_zeroed(st, &w.qk, T * 4 * heads));
    LV_TRY(dev_zeroed(st, &w.a1, T * E * mx([](const BlockLayer &l) { return l.a2.kp; })));
    LV_TRY(dev_zeroed(st, &w.g1, T * E * mx([](const BlockLayer &l) { return l.g2.kp; })));
    LV_TRY(dev_zeroed(st, &w.cat, T * E * mx([](const BlockLayer &l) { return l.out.kp; })));
    const uint64_t experts = mx([](const BlockLayer &l) { return l.spec.moe.experts; }), top = mx([](const BlockLayer &l) { return l.spec.moe.top; });
    LV_TRY(dev_zeroed(st, &w.z, T * 4 * up((uint32_t)experts, 4) * kRouterParts));
    LV_TRY(dev_zeroed(st, &w.scores, T * 4 * top));
    LV_TRY(dev_zeroed(st, &w.ids, T * 4 * top));
    LV_TRY(dev_zeroed(st, &w.slots, T * 4 * top));
    LV_TRY(dev_zeroed(st, &w.tiles, 4 * (1 + 3 * (T * top / kF32Tile + experts + 1))));
    // a tile of 128 positions may start at any of the T * top
    LV_TRY(dev_zeroed(st, &w.ff, E * mx([&](const BlockLayer &l) { return (cap * std::max(1u, l.spec.moe.top) + 128) * l.down.kp; })));
    w.cap = cap;
    return LV_OK;
}

// device scratch that follows the number of keys: grown by halves, so that a sequence that gets longer does not allocate every time
static int scratch_reserve(BlockSession *s, void **p, uint64_t *elems, uint64_t need, uint32_t elem)
{
    if (need <= *elems) return LV_OK;
    HIP_TRY(hipStreamSynchronize(s->st));
    drop(*p);
    *elems = 0;
    need += need / 2;
    LV_TRY(dev_alloc(p, need * elem));
    *elems = need;
    return LV_OK;
}

// attention of a batch on the matrix cores: the transposed values, then the tiles.  dk, dv: padded sizes
static int gqa_tiles(BlockSession *s, uint32_t dk, uint32_t dv, const GqaBatchArgs &b)
{
    GqaTileArgs a{};
    a.b = b;
    a.base = b.s.chunk ? b.pos0 / b.s.chunk * b.s.chunk : 0;
    a.keys = b.pos0 + b.n - a.base;
    a.vt_ld = up(a.keys, kTileKeys);
    Workspace &w = s->ws;
    LV_TRY(scratch_reserve(s, &w.vt, &w.vt_elems, (uint64_t)b.s.kv_heads * dv * a.vt_ld, 2));
    a.vt = static_cast<uint16_t *>(w.vt);
    auto run = [&](auto k_size, auto v_size, auto qt) -> int {
        constexpr int DK = decltype(k_size)::value, DV = decltype(v_size)::value, QT = decltype(qt)::value;
        gqa_values_kernel<DV><<<dim3(b.s.kv_heads, a.vt_ld / kTileKeys), dim3(256), 0, s->st>>>(a);
        HIP_TRY(hipGetLastError());
        auto *k = &gqa_tile_kernel<DK, DV, QT>;
        LV_TRY(allow_lds(k, gqa_tile_lds<DK, DV>()));
        k<<<dim3(b.s.heads, (b.n + 64 * QT - 1) / (64 * QT)), dim3(256), gqa_tile_lds<DK, DV>(), s->st>>>(a);
        HIP_TRY(hipGetLastError());
        return LV_OK;
    };
    using std::integral_constant;
    using I64 = integral_constant<int, 64>;
    using I128 = integral_constant<int, 128>;
    using I192 = integral_constant<int, 192>;
    using I256 = integral_constant<int, 256>;
    // two query tiles a wave halve the LDS reads per product; few queries are better spread over more workgroups
    auto both = [&](auto k_size, auto v_size) -> int {
        return (uint64_t)b.n * b.s.heads >= 128 * 256 ? run(k_size, v_size, integral_constant<int, 2>{}) : run(k_size, v_size, integral_constant<int, 1>{});
    };
    if (dk == 64) return both(I64{}, I64{});
    if (dk == 128) return dv == 64 ? both(I128{}, I64{}) : both(I128{}, I128{});
    if (dk == 192) return both(I192{}, I128{});
    return run(I256{}, I256{}, integral_constant<int, 1>{});
}

// every query of a batch for itself, fp32 throughout
static int gqa_rows(BlockSession *s, const BlockLayer &l, const GqaBatchArgs &a)
{
    return gqa_dispatch(true, l, [&](auto elem, auto dp, auto r) -> int {
        constexpr int DP = decltype(dp)::value, R = decltype(r)::value;
        if constexpr (std::is_same_v<decltype(elem), float>) {
            auto *k = &gqa_rows_kernel<float, DP, R>;
            const size_t lds = 4 * gqa_lds_floats<DP, R, kGqaRowThreads>();
            LV_TRY(allow_lds(k, lds));
            k<<<dim3(a.s.kv_heads * a.groups, a.n), dim3(kGqaRowThreads), lds, s->st>>>(a);
            HIP_TRY(hipGetLastError());
        }
        return LV_OK;
    });
}

// ---- mixers of a batch: from the joint projection in w.y1 to the output projection's input in w.cat -------------------------
template <class T> static int batch_branches(BlockSession *s, size_t i, uint32_t pos, uint32_t n)
{
    constexpr bool f32 = sizeof(T) == 4;
    const BlockModel *m = s->m;
    const BlockLayer &l = m->pass(i);
    Workspace &w = s->ws;
    hipStream_t st = s->st;
    PrepareArgs p{};
    p.y = w.y1; p.ldy = l.in.rows; p.pos0 = pos; p.dp = l.dp;
    p.attn = gqa_spec(s, i); p.q = w.q; p.k = w.k; p.v = w.v;
    p.delta = delta_spec(s, i); p.dq = w.dq; p.dk = w.dk; p.dv = w.dv; p.beta = w.beta; p.qk = w.qk; p.a1 = w.a1; p.g1 = w.g1;
    LV_TRY(with_j(l.delta ? l.dstride() / 64 : 1, [&](auto j) -> int {
        prepare_kernel<T, decltype(j)::value><<<dim3(prepare_grid(p, n)), dim3(256), 0, st>>>(p, n);
        HIP_TRY(hipGetLastError());
        return LV_OK;
    }));
    if (l.attn) {
        GqaBatchArgs a{};
        a.s = p.attn; a.pos0 = a.own0 = pos; a.n = n; a.q = w.q; a.k = w.k; a.v = w.v; a.out = w.cat; a.ldo = l.out.kp; a.groups = l.groups;
        a.out_scale = l.spec.attn_scale;
        LV_TRY(f32 ? gqa_rows(s, l, a) : gqa_tiles(s, l.dp, l.dp, a));
    }
    if (l.delta) {
        const lv_delta_spec &d = l.spec.delta;
        BfGemmArgs dg{};
        dg.x = w.a1; dg.ldx = l.a2.kp; dg.out = w.dg; dg.ldo = d.heads * l.dstride(); dg.a_log = l.a_log; dg.bias = l.dt_bias; dg.head_dim = d.dim; dg.head_stride = l.dstride();
        LV_TRY((gemm<kEpDecay, false>(st, f32, dg, l.a2, n)));
        BfGemmArgs gg{};
        gg.x = w.g1; gg.ldx = l.g2.kp; gg.out = w.gate; gg.ldo = d.heads * d.vdim;
        LV_TRY((gemm<kEpSigmoid, false>(st, f32, gg, l.g2, n)));
        DeltaScanArgs sc{};
        sc.s = p.delta; sc.n = n; sc.fresh = pos == 0; sc.q = w.dq; sc.k = w.dk; sc.v = w.dv; sc.g = w.dg; sc.beta = w.beta; sc.qk = w.qk; sc.o = w.o;
        LV_TRY(with_j(l.dstride() / 64, [&](auto j) -> int {
            constexpr int J = decltype(j)::value;
            const size_t lds = 2 * 4ull * scan_stage_floats<J>();
            LV_TRY(allow_lds(&delta_scan_kernel<J>, lds));
            delta_scan_kernel<J><<<dim3(d.heads, (d.vdim + 15) / 16), dim3(kScanThreads), lds, st>>>(sc);
            HIP_TRY(hipGetLastError());
            return LV_OK;
        }));
        gated_rows_kernel<T><<<dim3(n), dim3(256), 0, st>>>(static_cast<T *>(w.cat) + l.left_kp, l.out.kp, w.o, w.gate, l.onorm, d.heads, d.vdim, m->hp.eps, l.spec.delta_scale);
        HIP_TRY(hipGetLastError());
    }
    const uint32_t tail = std::min(n, std::max(l.attn ? s->layers[i].ring : 0u, l.delta ? p.delta.taps : 0u));
    append_kernel<T><<<dim3(tail), dim3(256), 0, st>>>(p, n);
    HIP_TRY(hipGetLastError());
    return LV_OK;
}

template <class T> static int batch_latent(BlockSession *s, size_t i, uint32_t pos, uint32_t n)
{
    constexpr bool f32 = sizeof(T) == 4;
    const BlockLayer &l = s->m->pass(i);
    const LatentSpec sp = latent_spec(s, i);
    Workspace &w = s->ws;
    hipStream_t st = s->st;
    const uint32_t keys = pos + n, H = sp.heads;
    LV_TRY(scratch_reserve(s, &w.ek, &w.ek_elems, (uint64_t)keys * H * l.dk, sizeof(T)));
    LV_TRY(scratch_reserve(s, &w.ev, &w.ev_elems, (uint64_t)keys * H * l.dv, sizeof(T)));
    T *ek = static_cast<T *>(w.ek), *ev = static_cast<T *>(w.ev);
    latent_prepare_kernel<T><<<dim3(n), dim3(256), 0, st>>>(sp, w.y1, l.in.rows, pos, static_cast<T *>(w.cq), l.uq.kp);
    HIP_TRY(hipGetLastError());
    BfGemmArgs q{};
    q.x = w.cq; q.ldx = l.uq.kp; q.out = w.y2; q.ldo = l.uq.rows;
    LV_TRY((gemm<kEpStore, false>(st, f32, q, l.uq, n)));
    latent_queries_kernel<T><<<dim3(n), dim3(256), 0, st>>>(sp, w.y2, l.uq.rows, pos, static_cast<T *>(w.q), l.dk);
    HIP_TRY(hipGetLastError());
    // keys and values of every position, from the cache rows; columns behind the latent meet zero weights
    BfGemmArgs k{};
    k.x = sp.cache; k.ldx = sp.width; k.act = ek; k.lda = H * l.dk; k.head_dim = sp.dim; k.head_stride = l.dk;
    LV_TRY((gemm<kEpHeads, false>(st, f32, k, l.uk, keys)));
    BfGemmArgs v{};
    v.x = sp.cache; v.ldx = sp.width; v.act = ev; v.lda = H * l.dv; v.head_dim = sp.vdim; v.head_stride = l.dv;
    LV_TRY((gemm<kEpHeads, false>(st, f32, v, l.uv, keys)));
    if (l.dk > sp.dim) latent_keys_kernel<T><<<dim3(keys), dim3(256), 0, st>>>(sp, ek, l.dk);
    HIP_TRY(hipGetLastError());
    if (l.dv > sp.vdim) latent_value_pads_kernel<T><<<dim3(keys), dim3(256), 0, st>>>(ev, H, sp.vdim, l.dv);
    HIP_TRY(hipGetLastError());
    GqaBatchArgs a{};
    a.s.heads = a.s.kv_heads = H; a.s.dim = sp.dim + sp.rot_dim; a.s.vdim = sp.vdim; a.s.sink = sp.sink;
    a.pos0 = pos; a.own0 = 0; a.n = n; a.q = w.q; a.k = ek; a.v = ev; a.out = w.cat; a.ldo = l.out.kp; a.groups = 1; a.out_scale = 1.f;
    return f32 ? gqa_rows(s, l, a) : gqa_tiles(s, l.dk, l.dv, a);
}

template <class T> static int batch_ssm(BlockSession *s, size_t i, uint32_t pos, uint32_t n)
{
    const BlockLayer &l = s->m->pass(i);
    Workspace &w = s->ws;
    hipStream_t st = s->st;
    const SsmSpec sp = ssm_spec(s, i);
    SsmBatchArgs a{};
    a.s = sp; a.y = w.y1; a.ldy = l.in.rows; a.pos0 = pos; a.n = n; a.o = w.o;
    if constexpr (sizeof(T) == 4) {
        a.x = static_cast<float *>(w.sx); a.b = static_cast<float *>(w.sb); a.c = static_cast<float *>(w.sc); a.dt = w.sdt; a.decay = w.sdecay;
        ssm_prepare_kernel<<<dim3(ssm_prepare_columns(sp), (n + kSsmPrepareTokens - 1) / kSsmPrepareTokens), dim3(256), 0, st>>>(a);
        HIP_TRY(hipGetLastError());
        LV_TRY(with_state(l.sstride() / 64, [&](auto j) -> int {
            constexpr int J = decltype(j)::value;
            const size_t lds = 2 * 4ull * ssm_stage_floats<J>();
            LV_TRY(allow_lds(&ssm_scan_kernel<J>, lds));
            ssm_scan_kernel<J><<<dim3(sp.heads, (sp.vdim + 15) / 16), dim3(kSsmScanThreads), lds, st>>>(a);
            HIP_TRY(hipGetLastError());
            return LV_OK;
        }));
    } else {
        SsmChunkArgs c{};
        c.s = sp; c.y = w.y1; c.ldy = l.in.rows; c.pos0 = pos; c.n = n; c.ldt = up(n, kSsmChunk); c.o = w.o; c.dt = w.sdt;
        c.xt = static_cast<uint16_t *>(w.sx); c.b = static_cast<uint16_t *>(w.sb); c.c = static_cast<uint16_t *>(w.sc); c.bt = static_cast<uint16_t *>(w.sbt);
        ssm_operands_kernel<<<dim3(ssm_prepare_columns(sp), c.ldt / 8), dim3(256), 0, st>>>(c);
        HIP_TRY(hipGetLastError());
        LV_TRY(with_state(l.sstride() / 64, [&](auto j) -> int {
            constexpr int J = decltype(j)::value;
            LV_TRY(allow_lds(&ssm_chunk_kernel<J>, ssm_chunk_lds<J>()));
            ssm_chunk_kernel<J><<<dim3(sp.heads, (sp.vdim + 63) / 64), dim3(kSsmChunkThreads), ssm_chunk_lds<J>(), st>>>(c);
            HIP_TRY(hipGetLastError());
            return LV_OK;
        }));
    }
    ssm_append_kernel<<<dim3(std::min(n, sp.taps), (sp.channels() + 255) / 256), dim3(256), 0, st>>>(a);
    HIP_TRY(hipGetLastError());
    const GroupInput g = group_in(sp, w.o, w.y1);
    const size_t lds = 4ull * (g.n + group_sums(g.groups, 4) + 4);
    LV_TRY(allow_lds(&ssm_gate_kernel<T>, lds));
    ssm_gate_kernel<T><<<dim3(n), dim3(256), lds, st>>>(g, l.in.rows, static_cast<T *>(w.cat), l.out.kp);
    HIP_TRY(hipGetLastError());
    return LV_OK;
}

template <class T>
static int step_batch(BlockSession *s, const uint32_t *cfg, uint32_t pos, uint32_t idx0, uint32_t n, float *logits_last, float *logits_all, const BlockTrace *trace)
{
    constexpr bool f32 = sizeof(T) == 4;
    const BlockModel *m = s->m;
    hipStream_t st = s->st;
    const uint32_t Dp = m->dp;
    LV_TRY(workspace_reserve(s, n));
    Workspace &w = s->ws;
    LV_TRY(embed(s, w.x, cfg, idx0, n));
    if (m->bigram && n > 1) HIP_TRY(hipMemcpyAsync(s->last + ((pos + n - 1) & 1), cfg + idx0 + n, 4, hipMemcpyDeviceToDevice, st));
    const NormSite *from = nullptr;    // of the sublayer whose output waits to be added to the residual
    uint32_t parts = 0;                // vectors per token in w.y that make it up
    auto norm = [&](const NormSite &to, bool act) -> int {
        const bool pending = parts != 0;
        int rc;
        if (m->hp.streams) {
            StreamRowsArgs a{};
            a.in = stream_in(m, w.x, to);
            a.parts = parts;
            if (pending) {
                a.in.y = w.y;
                a.in.spread = from->coef;
                a.in.x_out = w.x;
            }
            a.act = act ? w.act : nullptr;
            rc = stream_rows<T>(st, a, n);
        } else {
            NormRowsArgs a{};
            a.in = norm_in(m, w.x, to);
            if (pending) {
                a.in.y = w.y;
                a.in.parts = parts;
                a.in.wpost = from->post;
                a.in.x_out = w.x;
            }
            a.act = act ? w.act : nullptr;
            rc = norm_rows<T>(st, a, n);
        }
        parts = 0;
        return rc;
    };
    auto keep = [&](uint32_t pass, int which) { return trace_residual(m, st, trace, pass, which, idx0, n, w.x); };
    auto keep_end = [&](uint32_t pass) -> int {
        if (!m->pass(pass).ff()) LV_TRY(keep(pass, LV_TRACE_POST_ATTN));
        return keep(pass, LV_TRACE_OUT);
    };
    for (size_t i = 0; i < m->order.size(); i++) {
        const BlockLayer &l = m->pass(i);
        LV_TRY(norm(l.site[0], true));
        if (i) LV_TRY(keep_end((uint32_t)i - 1));
        BfGemmArgs g{};
        g.x = w.act; g.ldx = Dp; g.out = w.y1; g.ldo = l.in.rows;
        LV_TRY((gemm<kEpStore, false>(st, f32, g, l.in, n)));
        LV_TRY(l.latent ? batch_latent<T>(s, i, pos, n) : l.ssm ? batch_ssm<T>(s, i, pos, n) : batch_branches<T>(s, i, pos, n));
        BfGemmArgs o{};
        o.x = w.cat; o.ldx = l.out.kp; o.out = w.y; o.ldo = Dp;
        LV_TRY((gemm<kEpStore, false>(st, f32, o, l.out, n)));
        parts = 1;
        from = &l.site[0];
        if (!l.ff()) continue;

        LV_TRY(norm(l.site[1], true));
        LV_TRY(keep((uint32_t)i, LV_TRACE_POST_ATTN));
        from = &l.site[1];
        if (l.dense) {
            BfGemmArgs gu{};
            gu.x = w.act; gu.ldx = Dp; gu.act = w.ff; gu.lda = l.down.kp; gu.activation = l.spec.dense.act;
            LV_TRY((gemm<kEpDense, false>(st, f32, gu, l.gate_up, n)));
            BfGemmArgs dn{};
            dn.x = w.ff; dn.ldx = l.down.kp; dn.out = w.y; dn.ldo = Dp;
            LV_TRY((gemm<kEpStore, false>(st, f32, dn, l.down, n)));
            parts = 1;
            continue;
        }
        const lv_moe_spec &e = l.spec.moe;
        const uint32_t ldz = up(e.experts, 4), total = n * e.top;
        BfGemmArgs rt{};
        rt.x = w.act; rt.ldx = Dp; rt.out = w.z; rt.ldo = ldz;
        uint32_t z_parts = 1;
        if (!f32 && Dp >= 2 * kRouterSlice) {       // few rows: slices of K fill the chip
            rt.k_slice = up((Dp + kRouterParts - 1) / kRouterParts, kRouterSlice);
            rt.slice_floats = (uint64_t)w.cap * ldz;
            z_parts = (Dp + rt.k_slice - 1) / rt.k_slice;
        }
        LV_TRY((gemm<kEpStore, false>(st, f32, rt, l.router, n)));
        route_rows_kernel<<<dim3(n), dim3(64), e.experts * 4ull, st>>>(w.z, ldz, z_parts, rt.slice_floats, e.experts, e.top, w.ids, w.scores);
        HIP_TRY(hipGetLastError());
        sort_experts_kernel<<<dim3(1), dim3(1024), e.experts * 8ull, st>>>(w.ids, total, e.experts, f32 ? kF32Tile : kBfTile, w.slots, w.tiles);
        HIP_TRY(hipGetLastError());
        BfGemmArgs gu{};
        gu.x = w.act; gu.ldx = Dp; gu.tiles = w.tiles; gu.slots = w.slots; gu.weights = w.scores; gu.top = e.top; gu.expert_rows = l.gu_rows; gu.gather = true;
        gu.act = w.ff; gu.lda = l.down.kp;
        LV_TRY((gemm<kEpGlu, true>(st, f32, gu, l.gate_up, total, e.experts)));
        BfGemmArgs dn{};
        dn.x = w.ff; dn.ldx = l.down.kp; dn.tiles = w.tiles; dn.slots = w.slots; dn.top = e.top; dn.expert_rows = l.down_rows; dn.out = w.y; dn.ldo = Dp;
        LV_TRY((gemm<kEpScatter, true>(st, f32, dn, l.down, total, e.experts)));
        parts = e.top;
    }
    if (trace || logits_all) {
        LV_TRY(norm(m->final, logits_all != nullptr));
        LV_TRY(keep_end((uint32_t)m->order.size() - 1));
    }
    if (logits_all) {
        BfGemmArgs h{};
        h.x = w.act; h.ldx = Dp; h.out = logits_all; h.ldo = m->hp.vocab;
        LV_TRY((gemm<kEpStore, false>(st, f32, h, m->head, n)));
        if (logits_last) HIP_TRY(hipMemcpyAsync(logits_last, logits_all + (size_t)(n - 1) * m->hp.vocab, m->hp.vocab * 4ull, hipMemcpyDeviceToDevice, st));
    } else if (logits_last) {
        BfGemvArgs h{};
        h.w = m->head.w; h.rows = m->hp.vocab; h.kp = Dp; h.out = logits_last;
        const float *x = w.x + (size_t)(n - 1) * m->copies * Dp;
        if (m->hp.streams) {
            if (parts > 1) {       // the launch's head takes one vector
                LV_TRY(norm(m->final, false));
            }
            h.streams = stream_in(m, x, m->final);
            if (parts) {
                h.streams.y = w.y + (size_t)(n - 1) * Dp;
                h.streams.spread = from->coef;
            }
        } else {
            h.norm = norm_in(m, x, m->final);
            if (parts) {
                h.norm.y = w.y + (size_t)(n - 1) * parts * Dp;
                h.norm.parts = parts;
                h.norm.wpost = from->post;
            }
        }
        LV_TRY(gemv_residual<kGemvRows>(m, st, h));
    }
    return LV_OK;
}

int block_step_batch(BlockSession *s, const uint32_t *cfg, uint32_t pos, uint32_t idx0, uint32_t n, float *logits_last, float *logits_all, const BlockTrace *trace)
{
    return s->m->f32 ? step_batch<float>(s, cfg, pos, idx0, n, logits_last, logits_all, trace)
                     : step_batch<uint16_t>(s, cfg, pos, idx0, n, logits_last, logits_all, trace);
}

// ---------------------------------------------------------------------------------------------------------------------------
// state of a pass as bytes: K (or latent) rows, V rows, convolution ring, recurrent state; the first one also holds the last token
// ---------------------------------------------------------------------------------------------------------------------------
namespace {
struct StatePiece {
    void *p;
    uint64_t bytes;
};
void state_pieces(const BlockSession *s, uint32_t pass, uint32_t n_tokens, StatePiece (&out)[5])
{
    const BlockLayer &l = s->m->pass(pass);
    const LayerState &ls = s->layers[pass];
    const uint64_t rows = l.attn && l.spec.attn.chunk ? std::min(n_tokens, l.spec.attn.chunk) : n_tokens;
    const uint64_t kv = l.attn ? rows * l.spec.attn.kv_heads * l.dp * s->m->elem() : 0;
    out[0] = {ls.kc, l.latent ? rows * l.width * s->m->elem() : kv};
    out[1] = {ls.vc, kv};
    out[2] = {ls.conv, n_tokens ? l.ring_bytes() : 0};
    out[3] = {ls.state, n_tokens ? l.state_bytes() : 0};
    out[4] = {s->last, pass == 0 && n_tokens && s->m->bigram ? 8u : 0u};
}
}  // namespace

uint64_t block_state_bytes(const BlockSession *s, uint32_t layer, uint32_t n_tokens)
{
    StatePiece p[5];
    state_pieces(s, layer, n_tokens, p);
    return p[0].bytes + p[1].bytes + p[2].bytes + p[3].bytes + p[4].bytes;
}

int block_state_copy(BlockSession *s, uint32_t layer, uint32_t n_tokens, void *host, bool write)
{
    StatePiece p[5];
    state_pieces(s, layer, n_tokens, p);
    uint8_t *h = static_cast<uint8_t *>(host);
    for (const StatePiece &q : p) {
        if (!q.bytes) continue;
        HIP_TRY(hipMemcpyAsync(write ? q.p : (void *)h, write ? (const void *)h : q.p, q.bytes, write ? hipMemcpyHostToDevice : hipMemcpyDeviceToHost, s->st));
        h += q.bytes;
    }
    HIP_TRY(hipStreamSynchronize(s->st));
    return LV_OK;
}

}  // namespace lv
