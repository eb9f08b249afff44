// lv_latent.h — attention over a low-rank latent that all heads share.
//
//   c_q    = rms(W_dq h) * w;  q = W_uq c_q: per head `dim` unrotated and then `rot_dim` rotated dimensions
//   c, k_r = W_dkv h: a latent of kv_rank, normed as c_q is, and one rotated key part for all heads
//   k      = W_uk c, v = W_uv c per head;  s = (q . k + turn(q_r) . turn(k_r)) * scale, over the keys j <= i
//   out    = sum_j exp(s_j) v_j / (sum_j exp(s_j) + exp(sink))
//
// Cache: one row of `width` elements per position and layer, [c, zeros to kc, turned k_r, zeros to width]; nothing per head.
//
// One token never forms keys or values of past positions: q . (W_uk c) = (W_uk^T q) . c, so a head's query is taken to the latent
// once (latent_absorb_kernel), scores and sums are over cache rows (latent_attn_kernel: all heads of a tile share the rows it has
// in LDS), and W_uv is applied to the summed latent (latent_value_kernel).  A batch expands keys and values of every position it
// can see with one product each and goes through the tile kernels of grouped-query attention.
//
// Queries of one token enter the products with bf16 rows as three bf16 pieces (24 bits), with fp32 rows as they are; weights
// of the softmax and their sums are fp32.
#pragma once

#include "lv_gqa.h"

namespace lv {

struct LatentSpec {
    uint32_t heads, dim, rot_dim, rot_dims, vdim, q_rank, kv_rank;
    uint32_t q_off, kv_off;             // where a token's latents start in its row of the joint projection
    uint32_t kc, width;                 // cache row: start of the rotated part, elements
    uint32_t dim_p, kv_p;               // dim and kv_rank rounded up to 64
    const float *q_norm, *kv_norm;
    const float *sink;                  // null: none
    const double *freq;                 // rot_dims / 2 angles per position, in full turns
    const float2 *turn;                 // the same as (cos, sin) at the position of a one-token step
    const uint16_t *uk_t;               // [head][kv_p][dim_p]: W_uk transposed head by head
    const uint16_t *uv;                 // [heads * vdim][kv_p]
    float scale, eps;
    void *cache;
};

constexpr uint32_t kLatentMaxWidth = 768;
constexpr uint32_t kLatentMaxHeads = 512;
constexpr int kLatentKeys = 32;         // keys of a block
constexpr int kLatentTile = 16;         // heads of a workgroup
constexpr uint32_t kLatentMaxSplits = 128;
constexpr int kLatentStepThreads = 512;
inline uint32_t latent_groups(uint32_t heads) { return (heads + kLatentTile - 1) / kLatentTile; }
// key ranges the grid of a one-token step provides, for a cache of `positions` rows: 2^this
inline uint32_t latent_split_bits(uint32_t heads, uint32_t positions)
{
    const uint32_t blocks = (positions + kLatentKeys - 1) / kLatentKeys, want = 256 / latent_groups(heads);
    const uint32_t most = want < 8 ? 8 : want > kLatentMaxSplits ? kLatentMaxSplits : want;
    uint32_t bits = 0;
    while (1u << bits < blocks && 2u << bits <= most) bits++;
    return bits;
}
__host__ __device__ constexpr uint32_t latent_part_stride(uint32_t kc) { return kc + 4; }     // sums, then maximum and sum of weights

// pair of a rotated part of rot_dim entries, turned by turn(pair); pairs behind rot_dims pass, and there are zeros behind rot_dim
template <class Turn>
__device__ __forceinline__ float2 latent_turn(const float *v, uint32_t pair, const LatentSpec &s, Turn turn)
{
    float a = 0.f, b = 0.f;
    if (2 * pair < s.rot_dim) {
        a = v[2 * pair];
        b = v[2 * pair + 1];
        if (2 * pair < s.rot_dims) turn_pair(a, b, turn(pair));
    }
    return make_float2(a, b);
}

// latent, rotated key part -> cache row; `scratch` a float per wave
template <class CT, class Turn>
__device__ __forceinline__ void latent_append(const LatentSpec &s, const float *y, uint32_t pos, float *scratch, Turn turn)
{
    const float *c = y + s.kv_off;
    CT *row = static_cast<CT *>(s.cache) + (size_t)pos * s.width;
    float sum = 0.f;
    for (uint32_t i = threadIdx.x; i < s.kv_rank; i += blockDim.x) sum = fmaf(c[i], c[i], sum);
    const float inv = rsqrtf(block_sum_waves(sum, scratch, blockDim.x >> 6) / (float)s.kv_rank + s.eps);
#pragma unroll 1
    for (uint32_t i = threadIdx.x; i < s.kc; i += blockDim.x) row[i] = float_to_elem<CT>(i < s.kv_rank ? c[i] * inv * s.kv_norm[i] : 0.f);
#pragma unroll 1
    for (uint32_t i = threadIdx.x; i < (s.width - s.kc) / 2; i += blockDim.x) {
        const float2 t = latent_turn(c + s.kv_rank, i, s, turn);
        row[s.kc + 2 * i] = float_to_elem<CT>(t.x);
        row[s.kc + 2 * i + 1] = float_to_elem<CT>(t.y);
    }
}

// A query as the attention kernel wants it: with bf16 rows three planes of bf16 pieces (largest first, 24 bits together), else fp32.
// `plane` = elements of a plane
__device__ __forceinline__ void latent_put(uint16_t *q, size_t plane, size_t i, float v)
{
#pragma unroll
    for (int p = 0; p < 3; p++) {
        const uint16_t h = float_to_bf16(v);
        q[p * plane + i] = h;
        v -= bf16_to_float(h);
    }
}
__device__ __forceinline__ void latent_put(float *q, size_t, size_t i, float v) { q[i] = v; }

// ---- one token -------------------------------------------------------------------------------------------------------------
struct LatentAbsorbArgs {
    LatentSpec s;
    const float *y;                     // the token's joint projection
    const float *q;                     // [heads][dim + rot_dim]
    const uint32_t *pos_ptr;
    uint32_t pos_add;
    void *out;                          // [heads][width], scaled (latent_put)
};
constexpr int kAbsorbRows = 64;         // latent dimensions per workgroup

// workgroups: heads * kv_p / 64, and one more for the cache row
template <class CT>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentAbsorbArgs a)
{
    __shared__ __attribute__((aligned(16))) float q[kGqaMaxDim];
    __shared__ float scratch[4];
    const LatentSpec &s = a.s;
    const uint32_t pos = *a.pos_ptr + a.pos_add, blocks = s.kv_p / kAbsorbRows, head = blockIdx.x / blocks, r0 = blockIdx.x % blocks * kAbsorbRows;
    if (head >= s.heads) return latent_append<CT>(s, a.y, pos, scratch, [&](uint32_t i) { return s.turn[i]; });
    const int sub = threadIdx.x & 7, r8 = threadIdx.x >> 3;
    const uint16_t *w = s.uk_t + ((size_t)head * s.kv_p + r0 + r8) * s.dim_p + sub * 8;
    uint4 v[2][4];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int k = 0; k < 4; k++)
            v[i][k] = k * 64 < (int)s.dim_p ? load_once(w + (size_t)i * 32 * s.dim_p + k * 64) : make_uint4(0, 0, 0, 0);
    const float *mine = a.q + (size_t)head * (s.dim + s.rot_dim);
    for (uint32_t i = threadIdx.x; i < s.dim_p; i += 256) q[i] = i < s.dim ? mine[i] * s.scale : 0.f;
    CT *out = static_cast<CT *>(a.out);
    const size_t plane = (size_t)s.heads * s.width, at = (size_t)head * s.width;
    if (r0 == 0)
#pragma unroll 1
        for (uint32_t i = threadIdx.x; i < (s.width - s.kc) / 2; i += 256) {
            const float2 t = latent_turn(mine + s.dim, i, s, [&](uint32_t k) { return s.turn[k]; });
            latent_put(out, plane, at + s.kc + 2 * i, t.x * s.scale);
            latent_put(out, plane, at + s.kc + 2 * i + 1, t.y * s.scale);
        }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 2; i++) {
        float t = 0.f;
#pragma unroll
        for (int k = 0; k < 4; k++) {
            if (k * 64 >= (int)s.dim_p) break;
            const float *x = q + k * 64 + sub * 8;
            const uint32_t u[4] = {v[i][k].x, v[i][k].y, v[i][k].z, v[i][k].w};
#pragma unroll
            for (int e = 0; e < 4; e++) {
                t = fmaf(__uint_as_float(u[e] << 16), x[2 * e], t);
                t = fmaf(__uint_as_float(u[e] & 0xffff0000u), x[2 * e + 1], t);
            }
        }
        t = group8_sum(t);
        const uint32_t r = r0 + i * 32 + r8;
        if (sub == 0 && r < s.kc) latent_put(out, plane, at + r, t);
    }
}

struct LatentStepArgs {
    LatentSpec s;
    const void *q;                      // [heads][width] (latent_put)
    const uint32_t *pos_ptr;
    uint32_t pos_add;
    uint32_t split_bits;                // the grid provides 2^this key ranges
    float *part;                        // [split][head][latent_part_stride(kc)]
    float *out;                         // latent_value_kernel: [heads * vdim]
};

// key blocks a query at pos sees, and how many of them a range takes; range i has keys if i * per < blocks
__device__ __forceinline__ void latent_ranges(const LatentStepArgs &a, uint32_t pos, uint32_t &blocks, uint32_t &per)
{
    blocks = pos / kLatentKeys + 1;
    per = (blocks + (1u << a.split_bits) - 1) >> a.split_bits;
}

template <class CT> constexpr uint32_t latent_key_stride(uint32_t width) { return width + 16 / sizeof(CT); }
template <class CT> inline size_t latent_attn_lds(uint32_t width)
{
    return (size_t)kLatentKeys * latent_key_stride<CT>(width) * sizeof(CT) + 4ull * (4 * kLatentKeys * 17 + kLatentTile * 36 + 3 * kLatentTile);
}

// One head's query as a lane's part of an operand: eight columns
template <class CT> struct LatentQuery;
template <> struct LatentQuery<uint16_t> {
    lv_bf8 p[3];
    __device__ __forceinline__ void load(const uint16_t *q, size_t plane, bool there)
    {
#pragma unroll
        for (int i = 0; i < 3; i++) p[i] = there ? *reinterpret_cast<const lv_bf8 *>(q + i * plane) : lv_bf8(0.f);
    }
    __device__ __forceinline__ lv_f4 times(const GqaRaw<uint16_t> &k, lv_f4 acc) const
    {
        const lv_bf8 f = __builtin_bit_cast(lv_bf8, k.v);
#pragma unroll
        for (int i = 2; i >= 0; i--) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f, p[i], acc, 0, 0, 0);
        return acc;
    }
};
template <> struct LatentQuery<float> {
    float q[8];
    __device__ __forceinline__ void load(const float *p, size_t, bool there)
    {
#pragma unroll
        for (int e = 0; e < 8; e++) q[e] = 0.f;
        if (there) load8(q, p);
    }
    __device__ __forceinline__ lv_f4 times(const GqaRaw<float> &k, lv_f4 acc) const
    {
        float f[8];
        k.get(f);
#pragma unroll
        for (int e = 0; e < 8; e++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(f[e], q[e], acc, 0, 0, 0);
        return acc;
    }
};
__device__ __forceinline__ void raw_to(uint16_t *p, const GqaRaw<uint16_t> &r) { *reinterpret_cast<uint4 *>(p) = r.v; }
__device__ __forceinline__ void raw_to(float *p, const GqaRaw<float> &r)
{
    reinterpret_cast<float4 *>(p)[0] = r.a;
    reinterpret_cast<float4 *>(p)[1] = r.b;
}

// grid (tiles of 16 heads, splits), 8 waves.  A wave brings its part of a block of 32 cache rows (16 rows, a quarter of their
// columns) straight into the registers of a matrix operand, multiplies it by the queries it holds, S^T = K Q^T, and leaves it in
// LDS for the sums; the next block is on its way meanwhile.  Sums: P [16 heads][4 keys] x rows [4 keys][16 latent dimensions] in
// fp32; a wave takes 64 latent dimensions, of which a lane's four neighbours belong to four products.
// NQ = 128-wide pieces of a row, NB = 512-wide pieces of the latent.  Code is kept short: every line of it is fetched on the way.
template <class CT, int NQ, int NB>
__global__ __launch_bounds__(kLatentStepThreads, 2) void latent_attn_kernel(LatentStepArgs a)
{
    extern __shared__ __attribute__((aligned(16))) uint8_t lat_lds[];
    const LatentSpec &s = a.s;
    const uint32_t W = s.width, KS = latent_key_stride<CT>(W);
    CT *kb = reinterpret_cast<CT *>(lat_lds);
    float *ps = reinterpret_cast<float *>(lat_lds + (size_t)kLatentKeys * KS * sizeof(CT)), *p = ps + 4 * kLatentKeys * 17, *ml = p + kLatentTile * 36;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l16 = lane & 15, g4 = lane >> 4;
    const uint32_t h0 = blockIdx.x * kLatentTile;
    const int kt = wave & 1, kq = wave >> 1;
    // columns (j * 4 + kq) * 32 + g4 * 8 .. + 7; columns past the row meet zero queries
    LatentQuery<CT> q[NQ];
#pragma unroll
    for (int j = 0; j < NQ; j++) {
        const uint32_t k = (j * 4 + kq) * 32;
        q[j].load(static_cast<const CT *>(a.q) + (size_t)(h0 + l16) * W + k + g4 * 8, (size_t)s.heads * W, k < W && h0 + l16 < s.heads);
    }
    const uint32_t pos = *a.pos_ptr + a.pos_add;
    uint32_t blocks, per;
    latent_ranges(a, pos, blocks, per);
    const uint32_t b0 = blockIdx.y * per, b1 = min(b0 + per, blocks);
    if (b0 >= blocks) return;
    GqaRaw<CT> next[NQ];
    auto request = [&](uint32_t b) {
        const CT *row = static_cast<const CT *>(s.cache) + (size_t)min(b * kLatentKeys + kt * 16 + l16, pos) * W + g4 * 8;
#pragma unroll
        for (int j = 0; j < NQ; j++) next[j].load(row + min((j * 4 + kq) * 32u, W - 32));
    };
    request(b0);
    if (threadIdx.x < kLatentTile) {
        ml[threadIdx.x] = -INFINITY;
        ml[kLatentTile + threadIdx.x] = 0.f;
    }
    lv_f4 acc[NB][4];
#pragma unroll
    for (int n = 0; n < NB; n++)
#pragma unroll
        for (int e = 0; e < 4; e++) acc[n][e] = lv_f4{0.f, 0.f, 0.f, 0.f};

    for (uint32_t b = b0; b < b1; b++) {
        if (b != b0) __syncthreads();      // the block before has been read
        lv_f4 sc = lv_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < NQ; j++) {
            const uint32_t k = (j * 4 + kq) * 32;
            if (k < W) raw_to(kb + (size_t)(kt * 16 + l16) * KS + k + g4 * 8, next[j]);
            sc = q[j].times(next[j], sc);
        }
#pragma unroll
        for (int r = 0; r < 4; r++) ps[(kq * kLatentKeys + kt * 16 + g4 * 4 + r) * 17 + l16] = sc[r];
        if (b + 1 < b1) request(b + 1);
        __syncthreads();
        {
            const uint32_t key = threadIdx.x & 31, h = threadIdx.x >> 5;
            float v = 0.f;
#pragma unroll
            for (int k = 0; k < 4; k++) v += ps[(k * kLatentKeys + key) * 17 + h];
            if (b * kLatentKeys + key > pos) v = -INFINITY;
            const float old = ml[h];
            const float m = fmaxf(half_wave_max(v), old), w = __expf(v - m), l = half_wave_sum(w);
            p[h * 36 + key] = w;
            if (key == 0) {
                const float f = __expf(old - m);
                ml[h] = m;
                ml[kLatentTile + h] = ml[kLatentTile + h] * f + l;
                ml[2 * kLatentTile + h] = f;
            }
        }
        __syncthreads();
        float f[4];
#pragma unroll
        for (int r = 0; r < 4; r++) f[r] = ml[2 * kLatentTile + g4 * 4 + r];
#pragma unroll
        for (int n = 0; n < NB; n++) {
            const uint32_t d = (n * 8 + wave) * 64;
            if (d >= s.kc) break;
#pragma unroll
            for (int e = 0; e < 4; e++)
#pragma unroll
                for (int r = 0; r < 4; r++) acc[n][e][r] *= f[r];
#pragma unroll
            for (int kk = 0; kk < kLatentKeys / 4; kk++) {
                const float w = p[l16 * 36 + kk * 4 + g4];
                const CT *row = kb + (size_t)(kk * 4 + g4) * KS + d + l16 * 4;
                float c[4];
                if constexpr (sizeof(CT) == 2) {
                    const uint2 u = *reinterpret_cast<const uint2 *>(row);
                    c[0] = __uint_as_float(u.x << 16); c[1] = __uint_as_float(u.x & 0xffff0000u);
                    c[2] = __uint_as_float(u.y << 16); c[3] = __uint_as_float(u.y & 0xffff0000u);
                } else {
                    const float4 u = *reinterpret_cast<const float4 *>(row);
                    c[0] = u.x; c[1] = u.y; c[2] = u.z; c[3] = u.w;
                }
#pragma unroll
                for (int e = 0; e < 4; e++) acc[n][e] = __builtin_amdgcn_mfma_f32_16x16x4f32(w, c[e], acc[n][e], 0, 0, 0);
            }
        }
    }
    const uint32_t PS = latent_part_stride(s.kc);
    float *part = a.part + ((size_t)blockIdx.y * s.heads + h0) * PS;
#pragma unroll
    for (int n = 0; n < NB; n++) {
        const uint32_t d = (n * 8 + wave) * 64 + l16 * 4;
        if (d >= s.kc) break;
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (h0 + g4 * 4 + r < s.heads) *reinterpret_cast<float4 *>(part + (size_t)(g4 * 4 + r) * PS + d) = make_float4(acc[n][0][r], acc[n][1][r], acc[n][2][r], acc[n][3][r]);
    }
    if (threadIdx.x < kLatentTile && h0 + threadIdx.x < s.heads) {
        part[(size_t)threadIdx.x * PS + s.kc] = ml[threadIdx.x];
        part[(size_t)threadIdx.x * PS + s.kc + 1] = ml[kLatentTile + threadIdx.x];
    }
}

constexpr int kLatentValueRows = 64;
// grid (heads, vdim / 64 up): the ranges' sums of one head, then up to 64 rows of W_uv.  Four groups of 128 threads take 16 ranges
// each at a time, four columns a thread; weights and the first 64 ranges are requested before anything is used.
static __global__ __launch_bounds__(kLatentStepThreads, 2) void latent_value_kernel(LatentStepArgs a)
{
    constexpr int AHEAD = 8, COLS = 512, RANGES = 16;
    __shared__ __attribute__((aligned(16))) float o[kLatentMaxWidth], sums[4][COLS];
    __shared__ float weight[kLatentMaxSplits];
    const LatentSpec &s = a.s;
    const uint32_t head = blockIdx.x, row = blockIdx.y * kLatentValueRows + (threadIdx.x >> 3), sub = threadIdx.x & 7, steps = s.kv_p / 64;
    const uint16_t *w = s.uv + ((size_t)head * s.vdim + min(row, s.vdim - 1)) * s.kv_p + sub * 8;
    uint4 v[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; i++) v[i] = load_once(w + min((uint32_t)i, steps - 1) * 64);
    const uint32_t pos = *a.pos_ptr + a.pos_add, PS = latent_part_stride(s.kc);
    uint32_t blocks, per;
    latent_ranges(a, pos, blocks, per);
    const float *part = a.part + (size_t)head * PS;
    const size_t next = (size_t)s.heads * PS;
    const uint32_t grp = __builtin_amdgcn_readfirstlane(threadIdx.x >> 7), c4 = (threadIdx.x & 127) * 4;
#pragma unroll 1
    for (uint32_t c0 = 0; c0 < s.kv_p; c0 += COLS) {
        const uint32_t c = min(c0 + c4, s.kc - 4);
        float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 1
        for (uint32_t g0 = grp * RANGES; g0 < kLatentMaxSplits; g0 += 4 * RANGES) {
            float4 z[RANGES];
#pragma unroll
            for (int i = 0; i < RANGES; i++) z[i] = *reinterpret_cast<const float4 *>(part + ((g0 + i) * per < blocks ? g0 + i : 0) * next + c);      // range 0 stands in for one without keys
            if (c0 == 0 && g0 < 4 * RANGES) {
                if (threadIdx.x < 64) {
                    const float sink = s.sink ? s.sink[head] : -INFINITY;
                    float m[2], l[2];
#pragma unroll
                    for (uint32_t k = 0; k < 2; k++) {
                        const uint32_t i = threadIdx.x + k * 64;
                        const bool has = i * per < blocks;
                        m[k] = has ? part[i * next + s.kc] : -INFINITY;
                        l[k] = has ? part[i * next + s.kc + 1] : 0.f;
                    }
                    const float half = half_wave_max(fmaxf(m[0], m[1])), top = fmaxf(fmaxf(half, __shfl_xor(half, 32, 64)), sink);
                    const float e0 = __expf(m[0] - top), e1 = __expf(m[1] - top), inv = 1.f / (wave_sum(fmaf(e0, l[0], e1 * l[1])) + __expf(sink - top));
                    weight[threadIdx.x] = e0 * inv;
                    weight[threadIdx.x + 64] = e1 * inv;
                }
                __syncthreads();
            }
#pragma unroll
            for (int i = 0; i < RANGES; i++) {
                const float f = weight[g0 + i];          // 0 for a range without keys
                t.x = fmaf(z[i].x, f, t.x); t.y = fmaf(z[i].y, f, t.y); t.z = fmaf(z[i].z, f, t.z); t.w = fmaf(z[i].w, f, t.w);
            }
            if ((g0 + 4 * RANGES) * per >= blocks) break;
        }
        *reinterpret_cast<float4 *>(&sums[grp][c4]) = t;
        __syncthreads();
        if (c0 + threadIdx.x < s.kv_p) {
            const uint32_t i = threadIdx.x;
            o[c0 + i] = c0 + i < s.kc ? (sums[0][i] + sums[1][i]) + (sums[2][i] + sums[3][i]) : 0.f;
        }
        __syncthreads();
    }
    auto dot8 = [&](const uint4 &q, const float *x) {
        const uint32_t u[4] = {q.x, q.y, q.z, q.w};
        float t = 0.f;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            t = fmaf(__uint_as_float(u[e] << 16), x[2 * e], t);
            t = fmaf(__uint_as_float(u[e] & 0xffff0000u), x[2 * e + 1], t);
        }
        return t;
    };
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < AHEAD; i++)
        if (i < (int)steps) t += dot8(v[i], o + i * 64 + sub * 8);
#pragma unroll 1
    for (uint32_t i = AHEAD; i < steps; i++) t += dot8(*reinterpret_cast<const uint4 *>(w + i * 64), o + i * 64 + sub * 8);
    t = group8_sum(t);
    if (sub == 0 && row < s.vdim) a.out[(size_t)head * s.vdim + row] = t;
}

// ---- batches ---------------------------------------------------------------------------------------------------------------
// one workgroup per token: the query latent as activations, the cache row
template <class T>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentSpec s, const float *__restrict__ y, uint32_t ldy, uint32_t pos0, T *__restrict__ cq, uint32_t ldq)
{
    __shared__ float scratch[4];
    const uint32_t t = blockIdx.x;
    const float *row = y + (size_t)t * ldy, *q = row + s.q_off;
    float sum = 0.f;
    for (uint32_t i = threadIdx.x; i < s.q_rank; i += 256) sum = fmaf(q[i], q[i], sum);
    const float inv = rsqrtf(block_sum_waves(sum, scratch, 4) / (float)s.q_rank + s.eps);
    for (uint32_t i = threadIdx.x; i < ldq; i += 256) cq[(size_t)t * ldq + i] = float_to_elem<T>(i < s.q_rank ? q[i] * inv * s.q_norm[i] : 0.f);
    latent_append<T>(s, row, pos0 + t, scratch, [&](uint32_t i) { return rotation(s.freq[i], pos0 + t); });
}

// one workgroup per token: [heads][dim + rot_dim] -> rotated, scaled, heads padded to dk elements
template <class T>
__global__ __launch_bounds__(256) void latent_queries_kernel(LatentSpec s, const float *__restrict__ q, uint32_t ldq, uint32_t pos0, T *__restrict__ out, uint32_t dk)
{
    __shared__ float2 turn[kGqaMaxDim / 2];
    const uint32_t t = blockIdx.x, size = s.dim + s.rot_dim;
    for (uint32_t i = threadIdx.x; i < s.rot_dims / 2; i += 256) turn[i] = rotation(s.freq[i], pos0 + t);
    __syncthreads();
    const float *row = q + (size_t)t * ldq;
    T *o = out + (size_t)t * s.heads * dk;
    for (uint32_t i = threadIdx.x; i < s.heads * dk; i += 256) {
        const uint32_t h = i / dk, d = i % dk;
        float v = d < size ? row[h * size + d] : 0.f;
        if (d >= s.dim && d - s.dim < s.rot_dims) {
            const uint32_t r = d - s.dim;
            const float other = row[h * size + (r & 1 ? d - 1 : d + 1)];
            const float2 c = turn[r / 2];
            v = r & 1 ? v * c.x + other * c.y : v * c.x - other * c.y;
        }
        o[i] = float_to_elem<T>(v * s.scale);
    }
}

// one workgroup per position: the rotated part of the key behind every head's expanded one, zeros behind that
template <class T>
__global__ __launch_bounds__(256) void latent_keys_kernel(LatentSpec s, T *__restrict__ k, uint32_t dk)
{
    const uint32_t rest = dk - s.dim;
    const T *rot = static_cast<const T *>(s.cache) + (size_t)blockIdx.x * s.width + s.kc;
    T *row = k + (size_t)blockIdx.x * s.heads * dk + s.dim;
    for (uint32_t i = threadIdx.x; i < s.heads * rest; i += 256) {
        const uint32_t h = i / rest, d = i % rest;
        row[(size_t)h * dk + d] = d < s.rot_dim ? rot[d] : float_to_elem<T>(0.f);
    }
}
// the same for values: zeros behind vdim
template <class T>
__global__ __launch_bounds__(256) void latent_value_pads_kernel(T *__restrict__ v, uint32_t heads, uint32_t vdim, uint32_t dv)
{
    const uint32_t rest = dv - vdim;
    T *row = v + (size_t)blockIdx.x * heads * dv + vdim;
    for (uint32_t i = threadIdx.x; i < heads * rest; i += 256) row[(size_t)(i / rest) * dv + i % rest] = float_to_elem<T>(0.f);
}

}  // namespace lv
