// lv_bf16_gemv.h — one-token products with bfloat16 weights: out[row] = sum_k W[row][k] * x[k], x and the sums in fp32.
//
// A workgroup (8 waves) puts x into LDS once, then its waves walk groups of rows with a register queue of 16-byte weight
// loads that keeps running from one group to the next and is filled before x is ready.  What x is (the "input") is part of
// the kernel, so that a layer needs no launches for its norms:
//   kInNorm    x = norm(residual + postnorm(y)) with the sublayer output y still pending; workgroup 0 also leaves the new
//              residual and x in memory for later launches
//   kInPlain   a vector in memory
//   kInBranch  the concatenated outputs of two mixers: scaled attention heads, then gated and normalised recurrent heads
//   kInGroups  a read-out times silu of its gate, normalised in equal parts
//   kInStreams2 .. 8   the norm of a residual of up to 2, 4 or 8 streams (lv_streams.h)
// kGemvGlu multiplies interleaved gate and up rows (act(gate) * up).  kGemvExperts multiplies the rows of several experts (gate and up interleaved, SwiGLU), chosen from the router logits in the
// kernel's head; kGemvDown sums a row over the chosen experts' down projections.
#pragma once

#include "lv_bf16_gemm.h"
#include "lv_streams.h"

namespace lv {

// 16 bytes of weights: read once per step, so they are not to push anything out of the caches
__device__ __forceinline__ uint4 load_once(const uint16_t *p)
{
    typedef uint32_t u4v __attribute__((ext_vector_type(4)));
    const u4v v = __builtin_nontemporal_load(reinterpret_cast<const u4v *>(p));
    return make_uint4(v.x, v.y, v.z, v.w);
}

enum BfInput { kInNorm = 0, kInPlain = 1, kInBranch = 2, kInGroups = 3, kInStreams2 = 4, kInStreams4 = 5, kInStreams8 = 6 };
enum BfGemvMode { kGemvRows = 0, kGemvExperts = 1, kGemvDown = 2, kGemvGlu = 3 };

constexpr int kBfGemvThreads = 512;
constexpr int kBfGemvWaves = kBfGemvThreads / 64;
constexpr uint32_t kMaxTop = 64;          // experts a token may use
constexpr uint32_t kMaxExperts = 4096;

// x' = x + rms(y) * wpost (y summed over `parts` vectors; wpost null: plain sum; y null: nothing pending), h = rms(x') * wpre
struct NormInput {
    const float *x, *y, *wpost, *wpre;
    float *x_out, *h_out;    // either may be null
    uint32_t dim, dp;        // dp = dim rounded up to 64; every vector is zero from dim to dp
    uint32_t parts, part_stride;
    float eps;
};

struct BranchInput {
    const float *left, *o, *gate, *onorm;
    uint32_t left_n, left_kp;       // attention outputs, and where the recurrent part starts
    uint32_t heads, vdim;
    float left_scale, right_scale, eps;
};

// o * silu(z) in `groups` equal parts, each divided by its own root mean square, times w
struct GroupInput {
    const float *o, *z, *w;
    uint32_t n, groups;
    float eps;
};

struct BfGemvArgs {
    const uint16_t *w;
    uint32_t rows, kp;
    float *out;
    NormInput norm;
    const float *x;              // kInPlain
    BranchInput branch;
    GroupInput group;
    StreamInput streams;
    uint32_t act;                // kGemvGlu: LV_ACT_*
    // experts
    const float *z;              // router logits
    uint32_t experts, top, expert_rows;   // expert_rows: weight rows from one expert to the next
    uint32_t *ids;               // chosen experts and their scores: written by kGemvExperts, read by kGemvDown
    float *scores;
};

// x lies in LDS in two planes, elements 8c .. 8c+3 and 8c+4 .. 8c+7, so that a lane's two 16-byte reads are consecutive over
// the lanes
__device__ __forceinline__ uint32_t bf_xs(uint32_t i, uint32_t kp) { return ((i >> 2) & 1) * (kp / 2) + (i >> 3) * 4 + (i & 3); }

// NormInput into xs; every thread keeps to its own elements between the passes
__device__ __forceinline__ void norm_input(const NormInput &a, float *xs, float *scratch)
{
    const uint32_t dp = a.dp, step = blockDim.x * 4;
    const int nw = blockDim.x >> 6;
    const bool lead = blockIdx.x == 0;
    float ypost = 1.f;
    if (a.y) {
        float s = 0.f;
        for (uint32_t i = threadIdx.x * 4; i < dp; i += step) {
            float4 v = *reinterpret_cast<const float4 *>(a.y + i);
            for (uint32_t p = 1; p < a.parts; p++) {
                const float4 u = *reinterpret_cast<const float4 *>(a.y + (size_t)p * a.part_stride + i);
                v.x += u.x; v.y += u.y; v.z += u.z; v.w += u.w;
            }
            s = fmaf(v.x, v.x, s); s = fmaf(v.y, v.y, s); s = fmaf(v.z, v.z, s); s = fmaf(v.w, v.w, s);
            *reinterpret_cast<float4 *>(xs + bf_xs(i, dp)) = v;
        }
        if (a.wpost) ypost = rsqrtf(block_sum_waves(s, scratch, nw) / (float)a.dim + a.eps);
    }
    float s = 0.f;
    for (uint32_t i = threadIdx.x * 4; i < dp; i += step) {
        float4 v = *reinterpret_cast<const float4 *>(a.x + i);
        float4 *slot = reinterpret_cast<float4 *>(xs + bf_xs(i, dp));
        if (a.y) {
            const float4 y = *slot;
            const float4 w = a.wpost ? *reinterpret_cast<const float4 *>(a.wpost + i) : make_float4(1.f, 1.f, 1.f, 1.f);
            v.x += y.x * ypost * w.x; v.y += y.y * ypost * w.y; v.z += y.z * ypost * w.z; v.w += y.w * ypost * w.w;
        }
        s = fmaf(v.x, v.x, s); s = fmaf(v.y, v.y, s); s = fmaf(v.z, v.z, s); s = fmaf(v.w, v.w, s);
        *slot = v;
        if (lead && a.x_out) *reinterpret_cast<float4 *>(a.x_out + i) = v;
    }
    const float inv = rsqrtf(block_sum_waves(s, scratch, nw) / (float)a.dim + a.eps);
    for (uint32_t i = threadIdx.x * 4; i < dp; i += step) {
        float4 *slot = reinterpret_cast<float4 *>(xs + bf_xs(i, dp));
        const float4 w = *reinterpret_cast<const float4 *>(a.wpre + i);
        float4 v = *slot;
        v.x *= inv * w.x; v.y *= inv * w.y; v.z *= inv * w.z; v.w *= inv * w.w;
        *slot = v;
        if (lead && a.h_out) *reinterpret_cast<float4 *>(a.h_out + i) = v;
    }
}

// one recurrent head's read-out: divided by its root mean square, weighted, gated, scaled.  A wave per head; put(c, value).
template <class Put>
__device__ __forceinline__ void gated_head(const float *o, const float *gate, const float *w, uint32_t vdim, float eps, float scale, Put put)
{
    const uint32_t lane = threadIdx.x & 63;
    float s = 0.f;
    for (uint32_t c = lane; c < vdim; c += 64) s = fmaf(o[c], o[c], s);
    const float inv = rsqrtf(wave_sum(s) / (float)vdim + eps);
    for (uint32_t c = lane; c < vdim; c += 64) put(c, o[c] * inv * w[c] * gate[c] * scale);
}

__device__ __forceinline__ void branch_input(const BranchInput &a, float *xs, uint32_t kp)
{
    for (uint32_t i = threadIdx.x; i < a.left_kp; i += blockDim.x) xs[bf_xs(i, kp)] = i < a.left_n ? a.left[i] * a.left_scale : 0.f;
    for (uint32_t i = a.left_kp + a.heads * a.vdim + threadIdx.x; i < kp; i += blockDim.x) xs[bf_xs(i, kp)] = 0.f;
    const uint32_t nw = blockDim.x >> 6;
    for (uint32_t h = threadIdx.x >> 6; h < a.heads; h += nw) {
        const uint32_t base = h * a.vdim;
        gated_head(a.o + base, a.gate + base, a.onorm, a.vdim, a.eps, a.right_scale,
                   [&](uint32_t c, float v) { xs[bf_xs(a.left_kp + base + c, kp)] = v; });
    }
}

// GroupInput: put(i, value) for one element or, where parts are multiples of four, a float4 of them; get(i, value) the other way.
// Waves share a group where there are fewer groups than waves; `sums` holds group_sums() floats and every thread keeps to its own
// elements between the passes.
__host__ __device__ constexpr uint32_t group_parts(uint32_t groups, uint32_t waves) { return groups >= waves ? 1 : waves / groups; }
__host__ __device__ constexpr uint32_t group_sums(uint32_t groups, uint32_t waves) { return groups * group_parts(groups, waves); }
template <class V, class Put, class Get>
__device__ __forceinline__ void group_passes(const GroupInput &a, float *sums, Put put, Get get)
{
    constexpr uint32_t N = sizeof(V) / 4;
    const uint32_t lane = threadIdx.x & 63, waves = blockDim.x >> 6, parts = group_parts(a.groups, waves), tasks = a.groups * parts, size = a.n / a.groups;
    for (uint32_t k = threadIdx.x >> 6; k < tasks; k += waves) {
        const uint32_t base = k / parts * size;
        float s = 0.f;
        for (uint32_t c = (k % parts * 64 + lane) * N; c < size; c += parts * 64 * N) {
            V v = *reinterpret_cast<const V *>(a.o + base + c);
            const V z = *reinterpret_cast<const V *>(a.z + base + c);
            float *f = reinterpret_cast<float *>(&v);
            const float *g = reinterpret_cast<const float *>(&z);
#pragma unroll
            for (uint32_t e = 0; e < N; e++) {
                f[e] *= silu_f(g[e]);
                s = fmaf(f[e], f[e], s);
            }
            put(base + c, v);
        }
        s = wave_sum(s);
        if (lane == 0) sums[k] = s;
    }
    __syncthreads();
    for (uint32_t k = threadIdx.x >> 6; k < tasks; k += waves) {
        const uint32_t g = k / parts, base = g * size;
        float s = 0.f;
        for (uint32_t p = 0; p < parts; p++) s += sums[g * parts + p];
        const float inv = rsqrtf(s / (float)size + a.eps);
        for (uint32_t c = (k % parts * 64 + lane) * N; c < size; c += parts * 64 * N) {
            V v;
            get(base + c, v);
            const V w = *reinterpret_cast<const V *>(a.w + base + c);
            float *f = reinterpret_cast<float *>(&v);
            const float *h = reinterpret_cast<const float *>(&w);
#pragma unroll
            for (uint32_t e = 0; e < N; e++) f[e] *= inv * h[e];
            put(base + c, v);
        }
    }
}
template <class Put, class Get>
__device__ __forceinline__ void group_input(const GroupInput &a, float *sums, Put put, Get get)
{
    if (a.n / a.groups % 4 == 0) group_passes<float4>(a, sums, put, get);
    else group_passes<float>(a, sums, put, get);
}

// The `top` largest of n router logits, largest first, the lower index on equal values (one wave; zs is consumed).  Scores are
// the sigmoids of the chosen logits, not renormalised.
__device__ __forceinline__ void top_experts(float *zs, uint32_t n, uint32_t top, uint32_t *ids, float *scores)
{
    const uint32_t lane = threadIdx.x & 63;
    for (uint32_t k = 0; k < top; k++) {
        float best = -INFINITY;
        uint32_t at = 0xffffffffu;
        for (uint32_t e = lane; e < n; e += 64)
            if (zs[e] > best) { best = zs[e]; at = e; }
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float ov = __shfl_xor(best, off, 64);
            const uint32_t oi = __shfl_xor(at, off, 64);
            if (ov > best || (ov == best && oi < at)) { best = ov; at = oi; }
        }
        if (at == 0xffffffffu) at = 0;      // nothing but NaN left
        if (lane == 0) {
            ids[k] = at;
            scores[k] = sigmoid_f(best);
            zs[at] = -INFINITY;
        }
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_SEQ_CST, "wavefront");
    }
}

// feed-forward width of one expert, padded: its gate rows (the padding rows are zero and yield zero)
__device__ __forceinline__ uint32_t kp_units(const BfGemvArgs &a) { return a.expert_rows / 2; }

// R = rows (kGemvExperts: gate and up pairs) a wave works on at a time, DEPTH = queue slots of one 512-column step each
template <int MODE, int INPUT, int R, int DEPTH>
__global__ __launch_bounds__(kBfGemvThreads) void bf16_gemv_kernel(BfGemvArgs a)
{
    constexpr bool PAIRS = MODE == kGemvExperts || MODE == kGemvGlu;      // gate and up rows
    constexpr int NR = PAIRS ? 2 * R : R;
    extern __shared__ float xs[];          // kp floats (kGemvDown: top * kp), then kGemvExperts: router logits
    __shared__ float scratch[kBfGemvWaves];
    __shared__ uint32_t sel_id[kMaxTop];
    __shared__ float sel_score[kMaxTop];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t kp = a.kp;
    const uint32_t segs = MODE == kGemvDown ? a.top : 1;
    const uint32_t ksteps = (kp + 511) / 512, iters = ksteps * segs;
    const uint32_t units = MODE == kGemvExperts ? a.top * kp_units(a) : MODE == kGemvGlu ? a.rows / 2 : a.rows;
    const uint32_t tasks = (units + R - 1) / R, nwaves = gridDim.x * kBfGemvWaves;
    const uint32_t first_task = blockIdx.x * kBfGemvWaves + wave;

    if constexpr (MODE == kGemvDown) {
        if (threadIdx.x < a.top) sel_id[threadIdx.x] = a.ids[threadIdx.x];
        __syncthreads();
    }
    if constexpr (MODE == kGemvExperts) {
        float *zs = xs + kp;
        for (uint32_t e = threadIdx.x; e < a.experts; e += kBfGemvThreads) zs[e] = a.z[e];
        __syncthreads();
        if (wave == 0) top_experts(zs, a.experts, a.top, sel_id, sel_score);
        __syncthreads();
        if (blockIdx.x == 0 && threadIdx.x < a.top) {
            a.ids[threadIdx.x] = sel_id[threadIdx.x];
            a.scores[threadIdx.x] = sel_score[threadIdx.x];
        }
    }

    uint4 q[DEPTH][NR];
    uint32_t ftask = first_task, fit = 0, fseg = 0;
    auto fetch = [&](uint4 (&slot)[NR]) {
        const uint32_t kk = fit * 512 + lane * 8;
        const bool ok = ftask < tasks && kk < kp;
        const uint16_t *p = a.w + kk;
        if constexpr (MODE == kGemvExperts) {
            const uint32_t u = ftask * R, per = kp_units(a);
            const uint32_t s = ok ? u / per : 0, f = ok ? u % per : 0;
            p += ((size_t)sel_id[s] * a.expert_rows + (f >> 4) * 32 + (f & 15)) * kp;
        } else if constexpr (MODE == kGemvGlu) {
            const uint32_t f = ftask * R;
            p += ((size_t)(f >> 4) * 32 + (f & 15)) * kp;
        } else {
            p += (size_t)ftask * R * kp;
            if constexpr (MODE == kGemvDown) p += (size_t)sel_id[fseg] * a.expert_rows * kp;
        }
#pragma unroll
        for (int r = 0; r < NR; r++) {
            const size_t off = PAIRS ? (size_t)(r % R + (r / R) * 16) * kp : (size_t)r * kp;
            slot[r] = ok ? load_once(p + off) : make_uint4(0, 0, 0, 0);
        }
        if (++fit == ksteps) {
            fit = 0;
            if (MODE != kGemvDown || ++fseg == segs) {
                fseg = 0;
                ftask += nwaves;
            }
        }
    };
#pragma unroll
    for (int d = 0; d < DEPTH; d++) fetch(q[d]);

    if constexpr (INPUT == kInNorm) {
        norm_input(a.norm, xs, scratch);
    } else if constexpr (INPUT == kInBranch) {
        branch_input(a.branch, xs, kp);
    } else if constexpr (INPUT == kInGroups) {
        for (uint32_t i = a.group.n + threadIdx.x; i < kp; i += kBfGemvThreads) xs[bf_xs(i, kp)] = 0.f;
        group_input(a.group, xs + kp, [&](uint32_t i, auto v) { *reinterpret_cast<decltype(v) *>(xs + bf_xs(i, kp)) = v; },
                    [&](uint32_t i, auto &v) { v = *reinterpret_cast<std::decay_t<decltype(v)> *>(xs + bf_xs(i, kp)); });
    } else if constexpr (INPUT >= kInStreams2) {
        stream_input<2 << (INPUT - kInStreams2)>(a.streams, blockIdx.x == 0, scratch, [&](uint32_t i, const float4 h) { *reinterpret_cast<float4 *>(xs + bf_xs(i, kp)) = h; },
                                                 [&](uint32_t i) { return *reinterpret_cast<const float4 *>(xs + bf_xs(i, kp)); });
    } else {
        for (uint32_t i = threadIdx.x * 4; i < kp * segs; i += kBfGemvThreads * 4) {
            const uint32_t sg = i / kp, k = i % kp;
            *reinterpret_cast<float4 *>(xs + sg * kp + bf_xs(k, kp)) = *reinterpret_cast<const float4 *>(a.x + i);
        }
    }
    __syncthreads();

    float acc[NR];
#pragma unroll
    for (int r = 0; r < NR; r++) acc[r] = 0.f;
    uint32_t task = first_task, it = 0, k = 0, seg = 0;
    const uint32_t my_tasks = first_task < tasks ? (tasks - first_task + nwaves - 1) / nwaves : 0;
    const uint32_t total = my_tasks * iters;
    for (uint32_t t0 = 0; t0 < total; t0 += DEPTH) {
#pragma unroll
        for (int d = 0; d < DEPTH; d++) {
            if (t0 + d < total) {
                const uint32_t c = k * 64 + lane;               // 8-element chunk
                const float *src = xs + seg * kp + (c * 8 < kp ? c * 4 : 0);
                const float4 x0 = *reinterpret_cast<const float4 *>(src), x1 = *reinterpret_cast<const float4 *>(src + kp / 2);
#pragma unroll
                for (int r = 0; r < NR; r++) {
                    const uint4 v = q[d][r];
                    float s = acc[r];
                    s = fmaf(__uint_as_float(v.x << 16), x0.x, s); s = fmaf(__uint_as_float(v.x & 0xffff0000u), x0.y, s);
                    s = fmaf(__uint_as_float(v.y << 16), x0.z, s); s = fmaf(__uint_as_float(v.y & 0xffff0000u), x0.w, s);
                    s = fmaf(__uint_as_float(v.z << 16), x1.x, s); s = fmaf(__uint_as_float(v.z & 0xffff0000u), x1.y, s);
                    s = fmaf(__uint_as_float(v.w << 16), x1.z, s); s = fmaf(__uint_as_float(v.w & 0xffff0000u), x1.w, s);
                    acc[r] = s;
                }
                fetch(q[d]);
                if (++k == ksteps) { k = 0; seg++; }
                if (++it == iters) {
                    float tot[NR];
#pragma unroll
                    for (int r = 0; r < NR; r++) { tot[r] = wave_sum(acc[r]); acc[r] = 0.f; }
                    if (lane < R) {
                        const uint32_t u = task * R + lane;
                        float v0 = tot[0], v1 = tot[NR - R];
#pragma unroll
                        for (int r = 1; r < R; r++)
                            if (lane == r) { v0 = tot[r]; v1 = tot[NR - R + r]; }
                        if (u < units) {
                            if constexpr (MODE == kGemvExperts) {
                                const float wt = sel_score[u / kp_units(a)];
                                a.out[u] = silu_f(wt * v0) * (wt * v1);
                            } else if constexpr (MODE == kGemvGlu) {
                                a.out[u] = glu_f(a.act, v0) * v1;
                            } else {
                                a.out[u] = v0;
                            }
                        }
                    }
                    it = 0; seg = 0;
                    task += nwaves;
                }
            }
        }
    }
}

}  // namespace lv
