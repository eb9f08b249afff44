// lv_gqa.h — grouped-query softmax attention over a ring of cache rows, with optional normalised projections, interleaved
// rotary positions, chunked visibility, values taken from the keys' projection, and a sink.
//
//   q, k   projections; RMS norm over the whole projection (weights), then rotation of the first rot_dims dimensions of a
//          head: pair (2i, 2i+1) by the angle p * f_i
//   s      = (q . k) * scale, over the keys j <= i with j / chunk == i / chunk (chunk 0: every j <= i)
//   out    = sum_j exp(s_j) v_j / (sum_j exp(s_j) + exp(sink))
//
// Cache: per layer two rings of rows, [row][kv head][DP] each, DP = head size rounded up to a power of two; a position lives in
// the row that counts it from its chunk's start, so a chunked layer needs chunk rows whatever the length of the sequence, and
// a new chunk overwrites the one before.  A batch of tokens keeps its own rows in scratch while it is evaluated (keys from the
// batch's first position on come from there, older ones from the ring); those of its last chunk are appended afterwards, so
// that a batch may run over any number of chunk borders.
//
// Everything but the MFMA path (gqa_tile_kernel: bf16 operands, weights as two bf16 pieces) is fp32 arithmetic on
// cache rows of either element type.
#pragma once

#include "lv_bf16_gemv.h"

namespace lv {

struct GqaSpec {
    uint32_t heads, kv_heads, dim, vdim;
    uint32_t q_off, k_off, v_off;       // where a token's projections start in its row of the joint projection
    const float *q_norm, *k_norm;       // null: not normalised
    const float *sink;                  // null: none
    const double *freq;                 // rot_dims / 2 angles per position, in full turns
    uint32_t rot_dims, chunk;
    float scale, eps;
    void *kc, *vc;
};

__device__ __forceinline__ uint32_t gqa_chunk_start(const GqaSpec &s, uint32_t pos) { return s.chunk ? pos - pos % s.chunk : 0; }

struct GqaStepArgs {
    GqaSpec s;
    const float *y;                     // the token's joint projection
    const uint32_t *pos_ptr;
    uint32_t pos_add;
    uint32_t groups;                    // head groups per kv head (R heads each, the last may hold fewer)
    uint32_t splits;                    // key splits the grid provides
    float *part;                        // [kv head][group][split][R][DP + 2]
    uint32_t *counters;                 // [kv head][group], zero before and after
    float *out;                         // [heads * vdim]
};

constexpr int kGqaSplit = 128;          // keys of a row kernel's block
// keys per workgroup of the one-token step: what 8 rounds of loads bring
__host__ __device__ constexpr uint32_t gqa_split(uint32_t dp) { return dp == 256 ? 64 : 128; }

constexpr uint32_t kGqaMaxDim = 256;

// (cos, sin) of a position's angle, freq in turns per position.  Reduced in double: positions far out lose nothing to the
// range reduction.
__device__ __forceinline__ float2 rotation(double freq, uint32_t pos)
{
    const double a = (double)pos * freq;
    float sn, cs;
    sincospif(2.f * (float)(a - rint(a)), &sn, &cs);
    return make_float2(cs, sn);
}
__device__ __forceinline__ void turn_pair(float &u, float &v, float2 t)
{
    const float r = u * t.x - v * t.y;
    v = v * t.x + u * t.y;
    u = r;
}

template <int LPK> __device__ __forceinline__ float lanes_sum(float v)
{
    if constexpr (LPK == 8) return group8_sum(v);
    v = group16_sum(v);
    if constexpr (LPK == 32) v += __shfl_xor(v, 16, 64);
    return v;
}

// A workgroup of NT threads works on keys a row at a time: DP / 8 lanes share a key, 8 elements each.
template <int DP, int NT>
struct GqaLanes {
    static constexpr int LPK = DP / 8;            // lanes per key
    static constexpr int KPR = NT / LPK;          // keys per round of the workgroup
};
constexpr int kGqaStepThreads = 512, kGqaRowThreads = 256;

// LDS, in floats: queries, own key and value, scores, sums of the waves, per-head scalars, scratch, rotation table
template <int DP, int R, int NT> constexpr int gqa_lds_floats() { return R * DP + 2 * DP + R * kGqaSplit + NT / 64 * R * DP + 4 * R + 16 + DP; }

// acc of all key groups -> red[0 .. R*DP), summed over the workgroup
template <int DP, int R, int NT>
__device__ __forceinline__ void gqa_reduce(float (&acc)[R][8], float *red)
{
    constexpr int LPK = DP / 8, NW = NT / 64;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    float *mine = red + wave * R * DP;
    if constexpr (LPK == 8) {       // two keys in a 16-lane row: rotate by 8
#pragma unroll
        for (int r = 0; r < R; r++)
#pragma unroll
            for (int e = 0; e < 8; e++) acc[r][e] += dpp_mov<0x128>(acc[r][e]);
    }
    if constexpr (LPK <= 16) {
        // four values at a time over the wave's four 16-lane rows; row j ends up with the total of value quad_partial_of_lane
        const int sub = lane % LPK, which = quad_partial_of_lane(lane);
#pragma unroll
        for (int r = 0; r < R; r++)
#pragma unroll
            for (int h = 0; h < 8; h += 4) {
                auto s01 = __builtin_amdgcn_permlane32_swap(__float_as_uint(acc[r][h]), __float_as_uint(acc[r][h + 1]), false, false);
                auto s23 = __builtin_amdgcn_permlane32_swap(__float_as_uint(acc[r][h + 2]), __float_as_uint(acc[r][h + 3]), false, false);
                const float x = __uint_as_float(s01[0]) + __uint_as_float(s01[1]), y = __uint_as_float(s23[0]) + __uint_as_float(s23[1]);
                auto t = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(y), false, false);
                if (LPK == 16 || (lane & 8) == 0) mine[r * DP + sub * 8 + h + which] = __uint_as_float(t[0]) + __uint_as_float(t[1]);
            }
    } else {
#pragma unroll
        for (int r = 0; r < R; r++)
#pragma unroll
            for (int h = 0; h < 8; h += 2) {
                auto s01 = __builtin_amdgcn_permlane32_swap(__float_as_uint(acc[r][h]), __float_as_uint(acc[r][h + 1]), false, false);
                mine[r * DP + (lane & 31) * 8 + h + (lane >> 5)] = __uint_as_float(s01[0]) + __uint_as_float(s01[1]);
            }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < R * DP; i += NT) {
        float t = red[i];
#pragma unroll
        for (int w = 1; w < NW; w++) t += red[w * R * DP + i];
        red[i] = t;
    }
    __syncthreads();
}

// elements 2i, 2i+1 of one head, normalised and rotated
__device__ __forceinline__ void head_pair(float &u, float &v, const float *y, const float *w, uint32_t base, uint32_t i, uint32_t dim, float inv, const GqaSpec &s,
                                          const float2 *turn)
{
    const uint32_t d = 2 * i;
    u = d < dim ? y[base + d] * inv * (w ? w[base + d] : 1.f) : 0.f;
    v = d + 1 < dim ? y[base + d + 1] * inv * (w ? w[base + d + 1] : 1.f) : 0.f;
    if (d < s.rot_dims) turn_pair(u, v, turn[i]);
}

// eight elements as they lie in memory
template <class CT> struct GqaRaw;
template <> struct GqaRaw<uint16_t> {
    uint4 v;
    __device__ __forceinline__ void load(const uint16_t *p) { v = *reinterpret_cast<const uint4 *>(p); }
    __device__ __forceinline__ void get(float (&f)[8]) const
    {
        const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int i = 0; i < 4; i++) {
            f[2 * i] = __uint_as_float(w[i] << 16);
            f[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
        }
    }
};
template <> struct GqaRaw<float> {
    float4 a, b;
    __device__ __forceinline__ void load(const float *p)
    {
        a = reinterpret_cast<const float4 *>(p)[0];
        b = reinterpret_cast<const float4 *>(p)[1];
    }
    __device__ __forceinline__ void get(float (&f)[8]) const { f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w; }
};

// One token, one group of R heads that share a kv head, one split of its keys: kGqaStepThreads threads.  The projections are
// requested first, then all cache rows of the split, so that norms and rotations go on while those are on their way (loads
// return in order).  The splits of a group meet in the last of them to arrive (see attention_kernel for what the hand-over
// relies on).  The split that holds the token's own position also appends its rows.
template <class CT, int DP, int R>
__device__ __forceinline__ void gqa_step(const GqaStepArgs &a, uint32_t idx, float *lds)
{
    constexpr int NT = kGqaStepThreads, NW = NT / 64;
    using L = GqaLanes<DP, NT>;
    constexpr int SPLIT = gqa_split(DP), ROUNDS = SPLIT / L::KPR, PAIRS = (R * DP / 2 + NT - 1) / NT, SUMS = 8;
    const GqaSpec &s = a.s;
    const uint32_t split = idx % a.splits, grp = idx / a.splits, hg = grp % a.groups, kvh = grp / a.groups;
    const uint32_t pos = *a.pos_ptr + a.pos_add;
    const uint32_t c0 = gqa_chunk_start(s, pos);
    const uint32_t active = (pos - c0) / SPLIT + 1;
    if (split >= active) return;
    const uint32_t k_begin = c0 + split * SPLIT, n = min((uint32_t)SPLIT, pos + 1 - k_begin);
    const bool own = split == active - 1;
    const uint32_t per_kv = s.heads / s.kv_heads, h0 = kvh * per_kv + hg * R, nh = min((uint32_t)R, per_kv - hg * R);
    const int sub = threadIdx.x % L::LPK, kg = threadIdx.x / L::LPK, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const float *yq = a.y + s.q_off, *yk = a.y + s.k_off, *yv = a.y + s.v_off;
    const uint32_t nq = s.heads * s.dim, nk = s.kv_heads * s.dim;

    float ys[SUMS], ks[2], pu[PAIRS], pv[PAIRS], wu[PAIRS], wv[PAIRS], ku = 0.f, kv = 0.f, kwu = 1.f, kwv = 1.f, vu = 0.f, vv = 0.f;
    if (s.q_norm) {
#pragma unroll
        for (int i = 0; i < SUMS; i++) ys[i] = threadIdx.x + i * NT < nq ? yq[threadIdx.x + i * NT] : 0.f;
#pragma unroll
        for (int i = 0; i < 2; i++) ks[i] = threadIdx.x + i * NT < nk ? yk[threadIdx.x + i * NT] : 0.f;
    }
    // the pair p of head r, and of the own key and value, that this thread turns
    const uint32_t own_d = 2 * threadIdx.x;
#pragma unroll
    for (int i = 0; i < PAIRS; i++) {
        const uint32_t e = threadIdx.x + i * NT, r = e / (DP / 2), d = e % (DP / 2) * 2;
        const uint32_t at = (h0 + r) * s.dim + d;
        const bool u = r < nh && d < s.dim, v = r < nh && d + 1 < s.dim;
        pu[i] = u ? yq[at] : 0.f;
        pv[i] = v ? yq[at + 1] : 0.f;
        wu[i] = u && s.q_norm ? s.q_norm[at] : 1.f;
        wv[i] = v && s.q_norm ? s.q_norm[at + 1] : 1.f;
    }
    if (own && own_d < DP) {
        const uint32_t at = kvh * s.dim + own_d, av = kvh * s.vdim + own_d;
        if (own_d < s.dim) ku = yk[at];
        if (own_d + 1 < s.dim) kv = yk[at + 1];
        if (s.k_norm && own_d < s.dim) kwu = s.k_norm[at];
        if (s.k_norm && own_d + 1 < s.dim) kwv = s.k_norm[at + 1];
        if (own_d < s.vdim) vu = yv[av];
        if (own_d + 1 < s.vdim) vv = yv[av + 1];
    }
    const double freq = threadIdx.x < s.rot_dims / 2 ? s.freq[threadIdx.x] : 0.0;

    CT *const kc = static_cast<CT *>(s.kc), *const vc = static_cast<CT *>(s.vc);
    GqaRaw<CT> kraw[ROUNDS], vraw[ROUNDS];
    {
        // row 0 of the split stands in for the rows it does not have
        const size_t step = (size_t)L::KPR * s.kv_heads * DP;
        const size_t at = ((size_t)(split * SPLIT) * s.kv_heads + kvh) * DP + sub * 8, mine = at + (size_t)kg * s.kv_heads * DP;
#pragma unroll
        for (int i = 0; i < ROUNDS; i++) kraw[i].load(kc + (i * L::KPR + kg < (int)n ? mine + i * step : at));
#pragma unroll
        for (int i = 0; i < ROUNDS; i++) vraw[i].load(vc + (i * L::KPR + kg < (int)n ? mine + i * step : at));
    }
    float *q = lds, *krow = q + R * DP, *vrow = krow + DP, *sc = vrow + DP, *red = sc + R * kGqaSplit, *ml = red + NW * R * DP, *scratch = ml + 4 * R;
    float2 *turn = reinterpret_cast<float2 *>(scratch + 16);

    float sq[2] = {0.f, 0.f};
    if (s.q_norm) {
#pragma unroll
        for (int i = 0; i < SUMS; i++) sq[0] = fmaf(ys[i], ys[i], sq[0]);
        sq[1] = fmaf(ks[0], ks[0], ks[1] * ks[1]);
        for (uint32_t i = threadIdx.x + SUMS * NT; i < nq; i += NT) sq[0] = fmaf(yq[i], yq[i], sq[0]);
        for (uint32_t i = threadIdx.x + 2 * NT; i < nk; i += NT) sq[1] = fmaf(yk[i], yk[i], sq[1]);
    }
    if (threadIdx.x < s.rot_dims / 2) turn[threadIdx.x] = rotation(freq, pos);
    block_sums_waves<2>(sq, scratch, NW);      // also publishes the rotation table
    const float inv_q = s.q_norm ? rsqrtf(sq[0] / (float)nq + s.eps) : 1.f;
    const float inv_k = s.q_norm ? rsqrtf(sq[1] / (float)nk + s.eps) : 1.f;
#pragma unroll
    for (int i = 0; i < PAIRS; i++) {
        const uint32_t e = threadIdx.x + i * NT, d = e % (DP / 2) * 2;
        float u = pu[i] * inv_q * wu[i] * s.scale, v = pv[i] * inv_q * wv[i] * s.scale;
        if (d < s.rot_dims) turn_pair(u, v, turn[d / 2]);
        if (PAIRS * NT == R * DP / 2 || e < R * DP / 2) *reinterpret_cast<float2 *>(q + 2 * e) = make_float2(u, v);
    }
    if (own && own_d < DP) {
        const size_t row = ((size_t)(pos - c0) * s.kv_heads + kvh) * DP + own_d;
        float u = ku * inv_k * kwu, v = kv * inv_k * kwv;
        if (own_d < s.rot_dims) turn_pair(u, v, turn[threadIdx.x]);
        const CT cu = float_to_elem<CT>(u), cv = float_to_elem<CT>(v), v0 = float_to_elem<CT>(vu), v1 = float_to_elem<CT>(vv);
        *reinterpret_cast<float2 *>(krow + own_d) = make_float2(elem_to_float(cu), elem_to_float(cv));
        *reinterpret_cast<float2 *>(vrow + own_d) = make_float2(elem_to_float(v0), elem_to_float(v1));
        if (hg == 0) {
            kc[row] = cu; kc[row + 1] = cv;
            vc[row] = v0; vc[row + 1] = v1;
        }
    }
    __syncthreads();
    {
        float qr[R][8];
#pragma unroll
        for (int r = 0; r < R; r++) load8(qr[r], q + r * DP + sub * 8);
#pragma unroll
        for (int i = 0; i < ROUNDS; i++) {
            const uint32_t j = i * L::KPR + kg;
            float f[8];
            kraw[i].get(f);
            if (k_begin + j == pos) load8(f, krow + sub * 8);
#pragma unroll
            for (int r = 0; r < R; r++) {
                float t = 0.f;
#pragma unroll
                for (int e = 0; e < 8; e++) t = fmaf(qr[r][e], f[e], t);
                t = lanes_sum<L::LPK>(t);
                if (sub == 0) sc[r * kGqaSplit + j] = j < n ? t : -INFINITY;
            }
        }
    }
    __syncthreads();
    for (int r = wave; r < R; r += NW) {
        float m = -INFINITY, l = 0.f;
        for (int j = lane; j < SPLIT; j += 64) m = fmaxf(m, sc[r * kGqaSplit + j]);
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
        for (int j = lane; j < SPLIT; j += 64) {
            const float p = __expf(sc[r * kGqaSplit + j] - m);      // 0 beyond the split's keys
            sc[r * kGqaSplit + j] = p;
            l += p;
        }
        l = wave_sum(l);
        if (lane == 0) { ml[2 * r] = m; ml[2 * r + 1] = l; }
    }
    __syncthreads();
    float acc[R][8];
#pragma unroll
    for (int r = 0; r < R; r++)
#pragma unroll
        for (int e = 0; e < 8; e++) acc[r][e] = 0.f;
#pragma unroll
    for (int i = 0; i < ROUNDS; i++) {
        const uint32_t j = i * L::KPR + kg;
        float f[8];
        vraw[i].get(f);
        if (k_begin + j == pos) load8(f, vrow + sub * 8);
#pragma unroll
        for (int r = 0; r < R; r++) {
            const float p = sc[r * kGqaSplit + j];
#pragma unroll
            for (int e = 0; e < 8; e++) acc[r][e] = fmaf(p, f[e], acc[r][e]);
        }
    }
    gqa_reduce<DP, R, NT>(acc, red);

    if (active == 1) {
        for (uint32_t i = threadIdx.x; i < nh * s.vdim; i += NT) {
            const uint32_t r = i / s.vdim, c = i % s.vdim;
            const float m = ml[2 * r], sk = s.sink ? s.sink[h0 + r] : -INFINITY, M = fmaxf(m, sk);
            a.out[(h0 + r) * s.vdim + c] = red[r * DP + c] * __expf(m - M) / (ml[2 * r + 1] * __expf(m - M) + __expf(sk - M));
        }
        return;
    }
    constexpr int PS = R * (DP + 2);
    uint32_t *part = reinterpret_cast<uint32_t *>(a.part + (size_t)grp * a.splits * PS);
    for (uint32_t i = threadIdx.x; i < PS; i += NT) {
        const uint32_t r = i / (DP + 2), c = i % (DP + 2);
        const float v = c < DP ? red[r * DP + c] : ml[2 * r + (c - DP)];
        __hip_atomic_store(part + (size_t)split * PS + i, __float_as_uint(v), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    uint32_t *arrived = reinterpret_cast<uint32_t *>(scratch);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (threadIdx.x == 0) *arrived = __hip_atomic_fetch_add(&a.counters[grp], 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (*arrived != active - 1) return;
    auto get = [&](uint32_t sp, uint32_t i) { return __uint_as_float(__hip_atomic_load(part + (size_t)sp * PS + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT)); };
    // every thread sums its element over the splits, in split order, with a running maximum of its own: one pass of loads
    for (uint32_t i = threadIdx.x; i < nh * s.vdim; i += NT) {
        const uint32_t r = i / s.vdim, c = i % s.vdim;
        float M = s.sink ? s.sink[h0 + r] : -INFINITY, l = s.sink ? 1.f : 0.f, t = 0.f;
        for (uint32_t s0 = 0; s0 < active; s0 += 16) {
            float v[16], w[16], z[16];
#pragma unroll
            for (int e = 0; e < 16; e++) {
                const uint32_t sp = min(s0 + e, active - 1);
                v[e] = get(sp, r * (DP + 2) + c);
                w[e] = get(sp, r * (DP + 2) + DP);
                z[e] = get(sp, r * (DP + 2) + DP + 1);
            }
            float top = M;
#pragma unroll
            for (int e = 0; e < 16; e++) top = fmaxf(top, w[e]);
            const float f = __expf(M - top);
            M = top;
            t *= f;
            l *= f;
#pragma unroll
            for (int e = 0; e < 16; e++) {
                const float p = s0 + e < active ? __expf(w[e] - top) : 0.f;
                t = fmaf(v[e], p, t);
                l = fmaf(z[e], p, l);
            }
        }
        a.out[(h0 + r) * s.vdim + c] = t / l;
    }
    if (threadIdx.x == 0) a.counters[grp] = 0u;
}

// ---- batches -------------------------------------------------------------------------------------------------------------
struct GqaBatchArgs {
    GqaSpec s;
    uint32_t pos0, n;            // the batch's first position and its tokens
    const void *q;               // [n][heads][DP], normalised, rotated, scaled
    const void *k, *v;           // [positions from own0][kv head][DP]: rows that are not in the ring, the batch's own among them
    uint32_t own0;
    void *out;                   // [n][ldo] activations, heads * vdim columns
    uint32_t ldo, groups;
    float out_scale;
};

// One token and head group per workgroup, fp32 arithmetic: the batch form for 32-bit models (and any head size).
template <class CT, int DP, int R>
__global__ __launch_bounds__(256) void gqa_rows_kernel(GqaBatchArgs a)
{
    constexpr int NT = kGqaRowThreads;
    using L = GqaLanes<DP, NT>;
    extern __shared__ float lds[];
    const GqaSpec &s = a.s;
    const uint32_t t = blockIdx.y, hg = blockIdx.x % a.groups, kvh = blockIdx.x / a.groups, pos = a.pos0 + t;
    const uint32_t per_kv = s.heads / s.kv_heads, h0 = kvh * per_kv + hg * R, nh = min((uint32_t)R, per_kv - hg * R);
    float *q = lds, *sc = q + R * DP + 2 * DP, *red = sc + R * kGqaSplit, *ml = red + NT / 64 * R * DP;
    const int sub = threadIdx.x % L::LPK, kg = threadIdx.x / L::LPK;
    for (uint32_t i = threadIdx.x; i < R * DP; i += 256) {
        const uint32_t r = i / DP;
        q[i] = r < nh ? elem_to_float(static_cast<const CT *>(a.q)[((size_t)t * s.heads + h0 + r) * DP + i % DP]) : 0.f;
    }
    if (threadIdx.x < R) {     // running maximum, running sum, factor for the sums so far
        const float sk = s.sink && threadIdx.x < nh ? s.sink[h0 + threadIdx.x] : -INFINITY;
        ml[4 * threadIdx.x] = sk;
        ml[4 * threadIdx.x + 1] = s.sink && threadIdx.x < nh ? 1.f : 0.f;
    }
    __syncthreads();
    float acc[R][8];
#pragma unroll
    for (int r = 0; r < R; r++)
#pragma unroll
        for (int e = 0; e < 8; e++) acc[r][e] = 0.f;
    const uint32_t c0 = gqa_chunk_start(s, pos);
    for (uint32_t k_begin = c0; k_begin <= pos; k_begin += kGqaSplit) {
        const uint32_t n = min((uint32_t)kGqaSplit, pos + 1 - k_begin);
        auto from = [&](const void *ring, const void *mine, uint32_t j, int d, float (&f)[8]) {
            const uint32_t p = k_begin + j;
            if (p >= a.own0) load8(f, static_cast<const CT *>(mine) + ((size_t)(p - a.own0) * s.kv_heads + kvh) * DP + d);
            else load8(f, static_cast<const CT *>(ring) + ((size_t)(p - c0) * s.kv_heads + kvh) * DP + d);
        };
        for (uint32_t j0 = 0; j0 < n; j0 += L::KPR) {
            const uint32_t j = j0 + kg;
            float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (j < n) from(s.kc, a.k, j, sub * 8, f);
#pragma unroll
            for (int r = 0; r < R; r++) {
                float qr[8], t = 0.f;
                load8(qr, q + r * DP + sub * 8);
#pragma unroll
                for (int e = 0; e < 8; e++) t = fmaf(qr[e], f[e], t);
                t = lanes_sum<L::LPK>(t);
                if (sub == 0 && j < n) sc[r * kGqaSplit + j] = t;
            }
        }
        __syncthreads();
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        for (int r = wave; r < R; r += 4) {
            float m = ml[4 * r];
            const float old = m;
            for (uint32_t j = lane; j < n; j += 64) m = fmaxf(m, sc[r * kGqaSplit + j]);
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
            float l = 0.f;
            for (uint32_t j = lane; j < n; j += 64) {
                const float p = __expf(sc[r * kGqaSplit + j] - m);
                sc[r * kGqaSplit + j] = p;
                l += p;
            }
            l = wave_sum(l);
            if (lane == 0) {
                const float f = __expf(old - m);
                ml[4 * r] = m;
                ml[4 * r + 1] = ml[4 * r + 1] * f + l;
                ml[4 * r + 2] = f;
            }
        }
        __syncthreads();
#pragma unroll
        for (int r = 0; r < R; r++) {
            const float f = ml[4 * r + 2];
#pragma unroll
            for (int e = 0; e < 8; e++) acc[r][e] *= f;
        }
        for (uint32_t j = kg; j < n; j += L::KPR) {
            float f[8];
            from(s.vc, a.v, j, sub * 8, f);
#pragma unroll
            for (int r = 0; r < R; r++) {
                const float p = sc[r * kGqaSplit + j];
#pragma unroll
                for (int e = 0; e < 8; e++) acc[r][e] = fmaf(p, f[e], acc[r][e]);
            }
        }
        __syncthreads();
    }
    gqa_reduce<DP, R, NT>(acc, red);
    for (uint32_t i = threadIdx.x; i < nh * s.vdim; i += 256) {
        const uint32_t r = i / s.vdim, c = i % s.vdim;
        static_cast<CT *>(a.out)[(size_t)t * a.ldo + (h0 + r) * s.vdim + c] = float_to_elem<CT>(red[r * DP + c] / ml[4 * r + 1] * a.out_scale);
    }
}

}  // namespace lv
