// lv_block_kernels.h — what a layer of a block model (lv_block.h) needs besides its products and mixers: embedding rows, row
// norms with a pending sublayer output, the step that turns the joint projection into mixer operands, cache appends, and the
// routing of a batch to experts.
#pragma once

#include "lv_delta.h"
#include "lv_latent.h"
#include "lv_ssm.h"

namespace lv {

// x[z][0 .. dp) = table[token] * scale (+ a row of the bigram table), fp32, zero beyond dim, in every stream
struct EmbedArgs {
    float *x;                    // [token][stream][dp]
    const uint16_t *table;       // rows of `ld` elements
    uint32_t ld, dim, dp, streams;
    float scale;
    const uint32_t *cfg;         // position of the step's first token, then the step's tokens
    uint32_t idx;                // the launch's first token in the step
    const uint16_t *bigram;      // [buckets + 1][dim]; null: none
    uint32_t buckets, prev, cur;
    uint32_t *last;              // a sequence's last token, at [position % 2]
    const double *freq;          // one token: the model's rotation frequencies, to `turn` as (cos, sin) at its position
    float2 *turn;
    uint32_t n_freq;
};
__device__ __forceinline__ void quad(float (&f)[4], const uint16_t *p)
{
    const uint2 u = *reinterpret_cast<const uint2 *>(p);
    f[0] = __uint_as_float(u.x << 16); f[1] = __uint_as_float(u.x & 0xffff0000u);
    f[2] = __uint_as_float(u.y << 16); f[3] = __uint_as_float(u.y & 0xffff0000u);
}
// a thread takes four elements
static __global__ __launch_bounds__(256) void embed_bf16_kernel(EmbedArgs a)
{
    const uint32_t i = blockIdx.x * 256 + threadIdx.x, z = blockIdx.y, at = a.idx + z, pos = a.cfg[0] + at, token = a.cfg[1 + at];
    const uint16_t *row = a.bigram;
    if (a.bigram) {
        uint32_t r = a.buckets;
        if (pos) r = (uint32_t)(((uint64_t)(at ? a.cfg[at] : a.last[(pos - 1) & 1]) * a.prev + (uint64_t)token * a.cur) % a.buckets);
        row += (size_t)r * a.dim;
        // a launch of one token leaves it for the next; one of several is followed by a copy, since its first row may read the slot
        if (gridDim.y == 1 && i == 0) a.last[pos & 1] = token;
    }
    if (i < a.n_freq) a.turn[i] = rotation(a.freq[i], pos);
    const uint32_t d = i * 4;
    if (d >= a.dp) return;
    const uint16_t *table = a.table + (size_t)token * a.ld;
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    if (a.dim % 4 == 0 && a.ld % 4 == 0) {
        if (d < a.dim) {
            quad(v, table + d);
            float w[4] = {0.f, 0.f, 0.f, 0.f};
            if (row) quad(w, row + d);
#pragma unroll
            for (uint32_t e = 0; e < 4; e++) v[e] = row ? v[e] * a.scale + w[e] : v[e] * a.scale;
        }
    } else {
#pragma unroll
        for (uint32_t e = 0; e < 4; e++)
            if (d + e < a.dim) {
                v[e] = bf16_to_float(table[d + e]) * a.scale;
                if (row) v[e] += bf16_to_float(row[d + e]);
            }
    }
    for (uint32_t t = 0; t < a.streams; t++) *reinterpret_cast<float4 *>(a.x + ((size_t)z * a.streams + t) * a.dp + d) = make_float4(v[0], v[1], v[2], v[3]);
}

// NormInput for a batch: one workgroup per row; x in place, h as activations
struct NormRowsArgs {
    NormInput in;            // x, y, x_out: first row; h_out unused
    void *act;               // [row][dp], null: only the residual is wanted
    float *h32;              // the same in fp32, null: not wanted
};
template <class T>
__global__ __launch_bounds__(256) void norm_rows_kernel(NormRowsArgs a)
{
    extern __shared__ float xs[];
    __shared__ float scratch[4];
    NormInput in = a.in;
    const uint32_t row = blockIdx.x, dp = in.dp;
    in.x += (size_t)row * dp;
    if (in.y) in.y += (size_t)row * in.parts * in.part_stride;
    float *x_out = in.x_out ? in.x_out + (size_t)row * dp : nullptr;
    float ypost = 1.f;
    if (in.y) {
        float s = 0.f;
        for (uint32_t i = threadIdx.x * 4; i < dp; i += 1024) {
            float4 v = *reinterpret_cast<const float4 *>(in.y + i);
            for (uint32_t p = 1; p < in.parts; p++) {
                const float4 u = *reinterpret_cast<const float4 *>(in.y + (size_t)p * in.part_stride + i);
                v.x += u.x; v.y += u.y; v.z += u.z; v.w += u.w;
            }
            s = fmaf(v.x, v.x, s); s = fmaf(v.y, v.y, s); s = fmaf(v.z, v.z, s); s = fmaf(v.w, v.w, s);
            *reinterpret_cast<float4 *>(xs + i) = v;
        }
        if (in.wpost) ypost = rsqrtf(block_sum_256(s, scratch) / (float)in.dim + in.eps);
    }
    float s = 0.f;
    for (uint32_t i = threadIdx.x * 4; i < dp; i += 1024) {
        float4 v = *reinterpret_cast<const float4 *>(in.x + i);
        if (in.y) {
            const float4 y = *reinterpret_cast<const float4 *>(xs + i);
            const float4 w = in.wpost ? *reinterpret_cast<const float4 *>(in.wpost + i) : make_float4(1.f, 1.f, 1.f, 1.f);
            v.x += y.x * ypost * w.x; v.y += y.y * ypost * w.y; v.z += y.z * ypost * w.z; v.w += y.w * ypost * w.w;
            if (x_out) *reinterpret_cast<float4 *>(x_out + i) = v;
        }
        s = fmaf(v.x, v.x, s); s = fmaf(v.y, v.y, s); s = fmaf(v.z, v.z, s); s = fmaf(v.w, v.w, s);
        *reinterpret_cast<float4 *>(xs + i) = v;
    }
    if (!a.act) return;
    const float inv = rsqrtf(block_sum_256(s, scratch) / (float)in.dim + in.eps);
    for (uint32_t i = threadIdx.x * 4; i < dp; i += 1024) {
        const float4 v = *reinterpret_cast<const float4 *>(xs + i), w = *reinterpret_cast<const float4 *>(in.wpre + i);
        const float h[4] = {v.x * inv * w.x, v.y * inv * w.y, v.z * inv * w.z, v.w * inv * w.w};
        T *o = static_cast<T *>(a.act) + (size_t)row * dp + i;
        if constexpr (sizeof(T) == 2)
            *reinterpret_cast<uint2 *>(o) = make_uint2((uint32_t)float_to_bf16(h[0]) | ((uint32_t)float_to_bf16(h[1]) << 16),
                                                       (uint32_t)float_to_bf16(h[2]) | ((uint32_t)float_to_bf16(h[3]) << 16));
        else *reinterpret_cast<float4 *>(o) = make_float4(h[0], h[1], h[2], h[3]);
        if (a.h32) *reinterpret_cast<float4 *>(a.h32 + (size_t)row * dp + i) = make_float4(h[0], h[1], h[2], h[3]);
    }
}

static_assert(kDeltaStepThreads == kGqaStepThreads, "one launch for both");

// Both mixers of one token in one launch: recurrent head blocks first (they take longest), then the attention groups.
struct MixStepArgs {
    DeltaStepArgs delta;
    GqaStepArgs attn;
    uint32_t delta_wgs;
};
template <class CT, int DP, int R>
__global__ __launch_bounds__(kGqaStepThreads) void mix_step_kernel(MixStepArgs a)
{
    extern __shared__ float lds[];
    if (blockIdx.x < a.delta_wgs) delta_step(a.delta, blockIdx.x, lds);
    else gqa_step<CT, DP, R>(a.attn, blockIdx.x - a.delta_wgs, lds);
}

// ---- batches: joint projection -> mixer operands ---------------------------------------------------------------------------
struct PrepareArgs {
    const float *y;              // [n][ldy]
    uint32_t ldy, pos0, dp;      // dp: padded head size of q, k, v (a power of two)
    GqaSpec attn;                // heads 0: none
    void *q, *k, *v;
    DeltaSpec delta;             // heads 0: none
    float *dq, *dk, *dv, *beta, *qk;
    void *a1, *g1;               // low-rank activations [n][a_kp], [n][g_kp]
};
constexpr uint32_t kPrepareTokens = 8;     // per workgroup of the recurrent branch
// workgroups: one per token (attention, and what is small), then per 8 tokens one for each key head and each 256 value channels
inline uint32_t prepare_columns(const DeltaSpec &s) { return s.heads ? s.kv_heads + (s.heads * s.vdim + 255) / 256 : 0; }
inline uint32_t prepare_grid(const PrepareArgs &a, uint32_t n) { return n + (n + kPrepareTokens - 1) / kPrepareTokens * prepare_columns(a.delta); }

template <class T> __device__ __forceinline__ void store_pair(T *o, float u, float v)
{
    if constexpr (sizeof(T) == 2) *reinterpret_cast<uint32_t *>(o) = (uint32_t)float_to_bf16(u) | ((uint32_t)float_to_bf16(v) << 16);
    else *reinterpret_cast<float2 *>(o) = make_float2(u, v);
}

template <class T>
__device__ __forceinline__ void prepare_token(const PrepareArgs &a, uint32_t t, float2 *turn, float *scratch)
{
    const uint32_t pos = a.pos0 + t;
    const float *y = a.y + (size_t)t * a.ldy;
    if (a.attn.heads) {
        const GqaSpec &s = a.attn;
        const uint32_t sh = 31 - __clz(a.dp / 2);
        for (uint32_t i = threadIdx.x; i < s.rot_dims / 2; i += 256) turn[i] = rotation(s.freq[i], pos);
        float sq[2] = {0.f, 0.f};
        if (s.q_norm) {
            for (uint32_t i = threadIdx.x; i < s.heads * s.dim; i += 256) sq[0] = fmaf(y[s.q_off + i], y[s.q_off + i], sq[0]);
            for (uint32_t i = threadIdx.x; i < s.kv_heads * s.dim; i += 256) sq[1] = fmaf(y[s.k_off + i], y[s.k_off + i], sq[1]);
        }
        block_sums_waves<2>(sq, scratch, 4);
        const float inv_q = s.q_norm ? rsqrtf(sq[0] / (float)(s.heads * s.dim) + s.eps) : 1.f;
        const float inv_k = s.q_norm ? rsqrtf(sq[1] / (float)(s.kv_heads * s.dim) + s.eps) : 1.f;
        for (uint32_t i = threadIdx.x; i < s.heads << sh; i += 256) {
            const uint32_t h = i >> sh, p = i & ((1u << sh) - 1);
            float u, v;
            head_pair(u, v, y + s.q_off, s.q_norm, h * s.dim, p, s.dim, inv_q, s, turn);
            store_pair(static_cast<T *>(a.q) + ((size_t)t * s.heads + h) * a.dp + 2 * p, u * s.scale, v * s.scale);
        }
        for (uint32_t i = threadIdx.x; i < s.kv_heads << sh; i += 256) {
            const uint32_t h = i >> sh, p = i & ((1u << sh) - 1);
            float u, v;
            head_pair(u, v, y + s.k_off, s.k_norm, h * s.dim, p, s.dim, inv_k, s, turn);
            const size_t o = ((size_t)t * s.kv_heads + h) * a.dp + 2 * p;
            store_pair(static_cast<T *>(a.k) + o, u, v);
            const float *yv = y + s.v_off + h * s.vdim + 2 * p;
            store_pair(static_cast<T *>(a.v) + o, 2 * p < s.vdim ? yv[0] : 0.f, 2 * p + 1 < s.vdim ? yv[1] : 0.f);
        }
    }
    if (a.delta.heads) {
        const DeltaSpec &s = a.delta;
        for (uint32_t h = threadIdx.x; h < s.heads; h += 256) a.beta[(size_t)t * s.heads + h] = sigmoid_f(y[s.b_off + h]);
        for (uint32_t i = threadIdx.x; i < s.a_kp; i += 256) static_cast<T *>(a.a1)[(size_t)t * s.a_kp + i] = float_to_elem<T>(i < s.a_rank ? y[s.a_off + i] : 0.f);
        for (uint32_t i = threadIdx.x; i < s.g_kp; i += 256) static_cast<T *>(a.g1)[(size_t)t * s.g_kp + i] = float_to_elem<T>(i < s.g_rank ? y[s.g_off + i] : 0.f);
    }
}

// J = delta.dstride / 64
template <class T, int J>
__global__ __launch_bounds__(256) void prepare_kernel(PrepareArgs a, uint32_t n)
{
    __shared__ float scratch[8];
    __shared__ float2 turn[kGqaMaxDim / 2];
    if (blockIdx.x < n) return prepare_token<T>(a, blockIdx.x, turn, scratch);
    const DeltaSpec &s = a.delta;
    const uint32_t nq = s.kv_heads * s.dim, nv = s.heads * s.vdim, cols = s.kv_heads + (nv + 255) / 256;
    const uint32_t idx = blockIdx.x - n, col = idx % cols, first = idx / cols * kPrepareTokens, last = min(first + kPrepareTokens, n);
    if (col >= s.kv_heads) {
        const uint32_t c = (col - s.kv_heads) * 256 + threadIdx.x;
        if (c >= nv) return;
        for (uint32_t t = first; t < last; t++)
            a.dv[(size_t)t * nv + c] = short_conv(s, a.y + (size_t)t * a.ldy, a.ldy, t, 2 * nq + c, a.pos0 + t, (a.pos0 + t) % s.taps);
        return;
    }
    const uint32_t lane = threadIdx.x & 63, h = col;
    for (uint32_t t = first + (threadIdx.x >> 6); t < last; t += 4) {
        const uint32_t pos = a.pos0 + t, slot = pos % s.taps;
        const float *y = a.y + (size_t)t * a.ldy;
        float q[J], k[J], sq = 0.f, sk = 0.f, sqk = 0.f;
#pragma unroll
        for (int j = 0; j < J; j++) {
            const uint32_t d = j * 64 + lane;
            q[j] = k[j] = 0.f;
            if (d < s.dim) {
                q[j] = short_conv(s, y, a.ldy, t, h * s.dim + d, pos, slot);
                k[j] = short_conv(s, y, a.ldy, t, nq + h * s.dim + d, pos, slot);
            }
            sq = fmaf(q[j], q[j], sq);
            sk = fmaf(k[j], k[j], sk);
        }
        const float fq = rsqrtf(wave_sum(sq) + 1e-6f) * rsqrtf((float)s.dim), fk = rsqrtf(wave_sum(sk) + 1e-6f);
#pragma unroll
        for (int j = 0; j < J; j++) {
            const uint32_t d = j * 64 + lane;
            q[j] *= fq;
            k[j] *= fk;
            sqk = fmaf(q[j], k[j], sqk);
            a.dq[((size_t)t * s.kv_heads + h) * s.dstride + d] = q[j];
            a.dk[((size_t)t * s.kv_heads + h) * s.dstride + d] = k[j];
        }
        sqk = wave_sum(sqk);
        if (lane == 0) a.qk[(size_t)t * s.kv_heads + h] = sqk;
    }
}

// The batch's last rows into the rings, after everything that reads older rows has run.  blockIdx.x = token counted from the
// end (0 = last).
template <class T>
__global__ __launch_bounds__(256) void append_kernel(PrepareArgs a, uint32_t n)
{
    const uint32_t t = n - 1 - blockIdx.x, pos = a.pos0 + t;
    // cache rows: what the next position's chunk may still need of this batch
    const uint32_t c0 = a.attn.heads ? gqa_chunk_start(a.attn, a.pos0 + n - 1) : 0;
    if (a.attn.heads && pos >= c0) {
        const uint32_t w = a.attn.kv_heads * a.dp / 8;      // 8 elements at a time
        const size_t dst = (size_t)(pos - c0) * w, src = (size_t)t * w;
        struct alignas(16) Eight { T e[8]; };
        for (uint32_t i = threadIdx.x; i < w; i += 256) {
            static_cast<Eight *>(a.attn.kc)[dst + i] = static_cast<const Eight *>(a.k)[src + i];
            static_cast<Eight *>(a.attn.vc)[dst + i] = static_cast<const Eight *>(a.v)[src + i];
        }
    }
    if (a.delta.heads && blockIdx.x < a.delta.taps) {
        const uint32_t C = a.delta.channels();
        for (uint32_t c = threadIdx.x; c < C; c += 256) a.delta.ring[(size_t)(pos % a.delta.taps) * C + c] = a.y[(size_t)t * a.ldy + a.delta.channel_at(c)];
    }
}

// recurrent read-outs of a batch -> the columns of the joint output projection's input behind the attention part
template <class T>
__global__ __launch_bounds__(256) void gated_rows_kernel(T *__restrict__ act, uint32_t ld, const float *__restrict__ o, const float *__restrict__ gate,
                                                         const float *__restrict__ w, uint32_t heads, uint32_t vdim, float eps, float scale)
{
    const size_t row = blockIdx.x, base = row * heads * vdim;
    for (uint32_t h = threadIdx.x >> 6; h < heads; h += 4)
        gated_head(o + base + h * vdim, gate + base + h * vdim, w, vdim, eps, scale, [&](uint32_t c, float v) { act[row * ld + h * vdim + c] = float_to_elem<T>(v); });
}

// ---- routing of a batch ----------------------------------------------------------------------------------------------------
// one wave per token; z: the K slices of the router logits, added here
__global__ __launch_bounds__(64) void route_rows_kernel(const float *__restrict__ z, uint32_t ldz, uint32_t parts, uint64_t part_floats, uint32_t experts, uint32_t top,
                                                        uint32_t *__restrict__ ids, float *__restrict__ scores)
{
    extern __shared__ float zs[];
    const size_t t = blockIdx.x;
    for (uint32_t e = threadIdx.x; e < experts; e += 64) {
        float v = z[t * ldz + e];
        for (uint32_t p = 1; p < parts; p++) v += z[p * part_floats + t * ldz + e];
        zs[e] = v;
    }
    __syncthreads();
    top_experts(zs, experts, top, ids + t * top, scores + t * top);
}

// Positions in expert order and the table of token tiles (BfGemmArgs::tiles).  One workgroup; LDS: 2 * experts words.  Where
// a token lands inside its expert's run does not matter to its result.
__global__ __launch_bounds__(1024) void sort_experts_kernel(const uint32_t *__restrict__ ids, uint32_t total, uint32_t experts, uint32_t tile, uint32_t *__restrict__ slots,
                                                            uint32_t *__restrict__ tiles)
{
    extern __shared__ uint32_t cnt[];
    uint32_t *at = cnt + experts;
    for (uint32_t e = threadIdx.x; e < experts; e += 1024) cnt[e] = 0;
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < total; i += 1024) atomicAdd(&cnt[ids[i]], 1u);
    __syncthreads();
    if (threadIdx.x == 0) {
        uint32_t pos = 0, nt = 0;
        for (uint32_t e = 0; e < experts; e++) {
            const uint32_t c = cnt[e];
            at[e] = pos;
            for (uint32_t f = 0; f < c; f += tile, nt++) {
                tiles[1 + 3 * nt] = e;
                tiles[2 + 3 * nt] = pos + f;
                tiles[3 + 3 * nt] = min(tile, c - f);
            }
            pos += c;
        }
        tiles[0] = nt;
    }
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < total; i += 1024) slots[atomicAdd(&at[ids[i]], 1u)] = i;
}

}  // namespace lv
