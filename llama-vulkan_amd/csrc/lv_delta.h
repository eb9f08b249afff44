// lv_delta.h — the gated delta rule with a decay per key channel: a recurrent mixer with one dim x vdim state per head.
//
//   q, k, v  projections, each through a causal convolution of `taps` steps per channel and silu; q and k (kv_heads of them,
//            shared by consecutive heads) are then unit vectors, q times dim^-1/2
//   beta     = sigmoid(b), one per head
//   g        = exp(-exp(A_log) softplus(a + dt_bias)), one per head and key channel
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//   out      = o / rms(o) * norm * gate, gate = sigmoid of a low-rank projection, vdim values per head
//
// All of it is fp32.  With S' = g S the read-out is o = S'^T q + (k . q) u, so the two reductions of a step, S'^T k and S'^T q,
// do not wait for each other.  Columns of S do not interact: 16 lanes (32 in a batch) share a column.
//
// State of a sequence and layer: S as [head][vdim][64 J] (a column contiguous, zero beyond dim) and a ring of the
// convolution's last `taps` inputs, [position % taps][channel], channels in the order q, k, v.  Nothing has to be cleared for
// a new sequence: positions before 0 and the state at position 0 are never read.
#pragma once

#include "lv_conv.h"

namespace lv {

struct DeltaSpec {
    uint32_t heads, kv_heads, dim, vdim, taps;
    uint32_t q_off, k_off, v_off, b_off, a_off, g_off;   // offsets in a token's joint projection
    uint32_t a_rank, g_rank, a_kp, g_kp;                 // low-rank widths of decay and gate, as stored (padded to 64)
    const float *conv;             // [taps][channels], last row = the current token
    const float *a_log, *dt_bias, *norm;
    const uint16_t *a2, *g2;       // [heads * dim][a_kp], [heads * vdim][g_kp]
    float eps;
    float *state, *ring;
    uint32_t dstride;              // 64 J
    __host__ __device__ uint32_t channels() const { return 2 * kv_heads * dim + heads * vdim; }
    // channel c (in q, k, v order) of the joint projection
    __device__ __forceinline__ uint32_t channel_at(uint32_t c) const
    {
        const uint32_t nq = kv_heads * dim;
        return c < nq ? q_off + c : c < 2 * nq ? k_off + (c - nq) : v_off + (c - 2 * nq);
    }
    __device__ __forceinline__ float conv_bias(uint32_t) const { return 0.f; }
};

struct DeltaStepArgs {
    DeltaSpec s;
    const float *y;
    const uint32_t *pos_ptr;
    uint32_t pos_add;
    uint32_t blocks;               // column blocks per head
    float *o, *gate;               // [heads * vdim]
};

constexpr int kDeltaCols = 32;     // columns per workgroup of the one-token step: 16 lanes to each
constexpr uint32_t kDeltaMaxDim = 256;
constexpr uint32_t kDeltaMaxRank = 4096;

constexpr int kDeltaStepThreads = 512;
constexpr int kLowRankRows = kDeltaStepThreads / 8;      // rows of a low-rank matrix a workgroup takes at a time

// Rows row0 + kLowRankRows * i (i < N) of a low-rank matrix against a vector in LDS, 8 consecutive lanes a row, every lane of the eight gets
// the sum.  fetch() requests the first 128 columns of all N rows, which is usually all there is; dot() does the rest.
template <int N>
struct LowRankRows {
    uint4 w[N][2];
    const uint16_t *at;
    uint32_t kp;
    uint32_t rows;      // of the N that exist

    __device__ __forceinline__ void fetch(const uint16_t *m, uint32_t row0, uint32_t end, uint32_t kp_)
    {
        kp = kp_;
        rows = row0 < end ? min((uint32_t)N, (end - row0 + kLowRankRows - 1) / kLowRankRows) : 0;
        at = m + (size_t)row0 * kp + (threadIdx.x & 7) * 8;
#pragma unroll
        for (int i = 0; i < N; i++)
#pragma unroll
            for (int k = 0; k < 2; k++)
                w[i][k] = i < (int)rows && k * 64 < (int)kp ? *reinterpret_cast<const uint4 *>(at + (size_t)i * kLowRankRows * kp + k * 64) : make_uint4(0, 0, 0, 0);
    }
    static __device__ __forceinline__ float dot8(const uint4 &v, const float *x)
    {
        const uint32_t u[4] = {v.x, v.y, v.z, v.w};
        float t = 0.f;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            t = fmaf(__uint_as_float(u[i] << 16), x[2 * i], t);
            t = fmaf(__uint_as_float(u[i] & 0xffff0000u), x[2 * i + 1], t);
        }
        return t;
    }
    __device__ __forceinline__ void dot(float (&out)[N], const float *x)
    {
        x += (threadIdx.x & 7) * 8;
#pragma unroll
        for (int i = 0; i < N; i++) {
            float t = dot8(w[i][0], x);
            if (kp > 64) t += dot8(w[i][1], x + 64);
            if (i < (int)rows)
                for (uint32_t k = 128; k < kp; k += 64) t += dot8(*reinterpret_cast<const uint4 *>(at + (size_t)i * kLowRankRows * kp + k), x + k);
            out[i] = group8_sum(t);
        }
    }
};

__host__ __device__ constexpr uint32_t delta_step_lds_floats(uint32_t a_kp, uint32_t g_kp) { return 3 * kDeltaMaxDim + kDeltaCols + a_kp + g_kp; }

// One token, one head, one block of kDeltaCols columns: kDeltaStepThreads threads.  Everything the block reads is requested
// first, the short-lived before the state (loads return in order).
__device__ __forceinline__ void delta_step(const DeltaStepArgs &a, uint32_t idx, float *lds)
{
    const DeltaSpec &s = a.s;
    const uint32_t head = idx / a.blocks, cb = idx % a.blocks, c_lo = cb * kDeltaCols, nc = min((uint32_t)kDeltaCols, s.vdim - c_lo);
    const uint32_t pos = *a.pos_ptr + a.pos_add, rep = s.heads / s.kv_heads, kvh = head / rep, nq = s.kv_heads * s.dim, C = s.channels();
    float *q = lds, *k = q + kDeltaMaxDim, *g = k + kDeltaMaxDim, *v = g + kDeltaMaxDim, *al = v + kDeltaCols, *gl = al + s.a_kp;
    const int lane = threadIdx.x & 63, l16 = threadIdx.x & 15, r8 = threadIdx.x >> 3, J = s.dstride / 64;
    const uint32_t rslot = pos % s.taps;

    // threads 0 .. 255: channel d of q, the others: of k; the first 32 also a column of v
    const uint32_t d = threadIdx.x & 255, half = threadIdx.x >> 8, cq = half * nq + kvh * s.dim + d, cv = 2 * nq + head * s.vdim + c_lo + threadIdx.x;
    ShortConv qk_in{}, v_in{};
    if (d < s.dim) qk_in.fetch(s, a.y, 0, 0, cq, pos, rslot);
    if (threadIdx.x < nc) v_in.fetch(s, a.y, 0, 0, cv, pos, rslot);
    const float beta_in = a.y[s.b_off + head], a_log = s.a_log[head];
    for (uint32_t i = threadIdx.x; i < s.a_kp; i += kDeltaStepThreads) al[i] = i < s.a_rank ? a.y[s.a_off + i] : 0.f;
    for (uint32_t i = threadIdx.x; i < s.g_kp; i += kDeltaStepThreads) gl[i] = i < s.g_rank ? a.y[s.g_off + i] : 0.f;
    LowRankRows<2> ra;
    LowRankRows<1> rg;
    ra.fetch(s.a2, head * s.dim + r8, (head + 1) * s.dim, s.a_kp);
    rg.fetch(s.g2, head * s.vdim + c_lo + r8, head * s.vdim + c_lo + nc, s.g_kp);
    const uint32_t c_own = threadIdx.x >> 4;      // this thread's column, 16 lanes to one
    float4 *const col = reinterpret_cast<float4 *>(s.state + ((size_t)head * s.vdim + c_lo + min(c_own, nc - 1)) * s.dstride) + l16;
    float4 st[4];
#pragma unroll
    for (int j = 0; j < 4; j++) st[j] = pos && j < J ? col[j * 16] : make_float4(0.f, 0.f, 0.f, 0.f);

    float x = 0.f;
    if (d < s.dim) {
        x = qk_in.value(s, a.y, 0, 0, pos, rslot);
        if (cb == 0 && head % rep == 0) s.ring[(size_t)rslot * C + cq] = qk_in.x[0];
    }
    (half ? k : q)[d] = x;
    if (threadIdx.x < nc) {
        v[threadIdx.x] = v_in.value(s, a.y, 0, 0, pos, rslot);
        s.ring[(size_t)rslot * C + cv] = v_in.x[0];
    }
    __syncthreads();
    // every wave sums over the head for itself; q and k stay as they are, their factors go into the products with them
    float sq = 0.f, sk = 0.f, sqk = 0.f;
    for (uint32_t e = lane; e < s.dstride; e += 64) {
        sq = fmaf(q[e], q[e], sq);
        sk = fmaf(k[e], k[e], sk);
        sqk = fmaf(q[e], k[e], sqk);
    }
    const float fq = rsqrtf(wave_sum(sq) + 1e-6f) * rsqrtf((float)s.dim), fk = rsqrtf(wave_sum(sk) + 1e-6f), qk = wave_sum(sqk) * fq * fk;
    const float beta = sigmoid_f(beta_in), ea = __expf(a_log);
    for (uint32_t r0 = 0; r0 < s.dstride; r0 += 2 * kLowRankRows) {
        if (r0) ra.fetch(s.a2, head * s.dim + r0 + r8, (head + 1) * s.dim, s.a_kp);
        float t[2];
        ra.dot(t, al);
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const uint32_t r = r0 + i * kLowRankRows + r8;
            if ((threadIdx.x & 7) == i && r < s.dstride) g[r] = r < s.dim ? decay_f(ea, t[i] + s.dt_bias[head * s.dim + r]) : 0.f;
        }
    }
    {
        float t[1];
        rg.dot(t, gl);
        if (r8 < (int)nc && (threadIdx.x & 7) == 0) a.gate[head * s.vdim + c_lo + r8] = sigmoid_f(t[0]);
    }
    __syncthreads();
    float pk = 0.f, pq = 0.f;
#pragma unroll
    for (int j = 0; j < 4; j++)
        if (j < J) {
            const int at = j * 64 + l16 * 4;
            float4 e = st[j];
            const float4 gg = *reinterpret_cast<const float4 *>(g + at), kk = *reinterpret_cast<const float4 *>(k + at), qq = *reinterpret_cast<const float4 *>(q + at);
            e.x *= gg.x; e.y *= gg.y; e.z *= gg.z; e.w *= gg.w;
            pk = fmaf(e.x, kk.x, pk); pk = fmaf(e.y, kk.y, pk); pk = fmaf(e.z, kk.z, pk); pk = fmaf(e.w, kk.w, pk);
            pq = fmaf(e.x, qq.x, pq); pq = fmaf(e.y, qq.y, pq); pq = fmaf(e.z, qq.z, pq); pq = fmaf(e.w, qq.w, pq);
            st[j] = e;
        }
    pk = group16_sum(pk) * fk;
    pq = group16_sum(pq) * fq;
    if (c_own >= nc) return;
    const float u = beta * (v[c_own] - pk), ku = fk * u;
#pragma unroll
    for (int j = 0; j < 4; j++)
        if (j < J) {
            const float4 kk = *reinterpret_cast<const float4 *>(k + j * 64 + l16 * 4);
            float4 e = st[j];
            e.x = fmaf(kk.x, ku, e.x); e.y = fmaf(kk.y, ku, e.y); e.z = fmaf(kk.z, ku, e.z); e.w = fmaf(kk.w, ku, e.w);
            col[j * 16] = e;
        }
    if (l16 == 0) a.o[head * s.vdim + c_lo + c_own] = fmaf(qk, u, pq);
}

// ---- batches -------------------------------------------------------------------------------------------------------------
struct DeltaScanArgs {
    DeltaSpec s;
    uint32_t n;
    bool fresh;               // the batch starts the sequence: the state is zero
    const float *q, *k;       // [n][kv_heads][dstride], unit vectors (q scaled), zero beyond dim
    const float *v;           // [n][heads * vdim]
    const float *g;           // [n][heads][dstride], finite beyond dim
    const float *beta, *qk;   // [n][heads], [n][kv_heads]
    float *o;                 // [n][heads * vdim]
};

constexpr int kScanTokens = 16;   // tokens staged in LDS at a time
template <int J> constexpr int scan_stage_floats() { return kScanTokens * (3 * 64 * J + 16) + 64; }

constexpr int kScanThreads = 512;

// All tokens of a batch for 16 columns of one head: 8 waves, two columns a wave, 32 lanes a column with 2 J of its entries each.
// grid (heads, vdim / 16 up).  The chain from token to token is what takes the time: the reductions of S'^T k and S'^T q share
// their steps, and two waves per SIMD fill each other's gaps.
template <int J>
__global__ __launch_bounds__(kScanThreads) void delta_scan_kernel(DeltaScanArgs a)
{
    constexpr int W = 64 * J, SF = scan_stage_floats<J>();
    constexpr int V = J % 2 ? 2 : 4, U = 2 * J / V;      // a lane's entries: U runs of V, the lanes' runs side by side
    typedef float vec __attribute__((ext_vector_type(V)));
    extern __shared__ float lds[];       // two stages
    const DeltaSpec &s = a.s;
    const uint32_t head = blockIdx.x, kvh = head / (s.heads / s.kv_heads), HV = s.heads * s.vdim;
    const int l32 = threadIdx.x & 31, ci = threadIdx.x >> 5, lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t col = blockIdx.y * 16 + ci;
    const bool live = col < s.vdim;
    vec *const colp = reinterpret_cast<vec *>(s.state + ((size_t)head * s.vdim + (live ? col : 0)) * W) + l32;
    vec S[U];
#pragma unroll
    for (int u = 0; u < U; u++) S[u] = a.fresh || !live ? vec(0.f) : colp[u * 32];

    // One stage in LDS: k, q, g [16][W] each, v [16][16], beta [16], k.q [16].  Direct loads, lane after lane in LDS order; tokens
    // past the end and columns past vdim bring some other value that nothing uses.
    auto issue = [&](uint32_t t0, int st) {
        float *b = lds + st * SF;
#pragma unroll
        for (int i = 0; i < (J + 1) / 2; i++) {
            const int e = i * kScanThreads + wave * 64;          // first float4 of the wave, of 256 J
            if (e >= 256 * J) break;
            const uint32_t t = min(t0 + (e + lane) / (W / 4), a.n - 1), d = (e + lane) % (W / 4) * 4;
            const size_t kq = ((size_t)t * s.kv_heads + kvh) * W + d;
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.k + kq), (lv_lds_any *)(b + e * 4), 16, 0, 0);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.q + kq), (lv_lds_any *)(b + kScanTokens * W + e * 4), 16, 0, 0);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.g + ((size_t)t * s.heads + head) * W + d), (lv_lds_any *)(b + 2 * kScanTokens * W + e * 4), 16, 0, 0);
        }
        if (wave < 4) {
            const uint32_t t = min(t0 + wave * 4 + lane / 16, a.n - 1), c = min(blockIdx.y * 16 + lane % 16, s.vdim - 1);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.v + (size_t)t * HV + head * s.vdim + c), (lv_lds_any *)(b + 3 * kScanTokens * W + wave * 64), 4, 0, 0);
        } else if (wave == 4) {
            const uint32_t t = min(t0 + (lane & 15), a.n - 1);
            const float *src = lane & 16 ? a.qk + (size_t)t * s.kv_heads + kvh : a.beta + (size_t)t * s.heads + head;
            __builtin_amdgcn_global_load_lds((lv_glb_any *)src, (lv_lds_any *)(b + 3 * kScanTokens * W + 256), 4, 0, 0);
        }
    };
    issue(0, 0);
    for (uint32_t t0 = 0, st = 0; t0 < a.n; t0 += kScanTokens, st ^= 1) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();      // this stage is in LDS for everyone, and everyone is done with the other one
        if (t0 + kScanTokens < a.n) issue(t0 + kScanTokens, st ^ 1);
        const float *b = lds + st * SF, *bk = b + l32 * V, *bq = bk + kScanTokens * W, *bg = bq + kScanTokens * W, *bv = b + 3 * kScanTokens * W;
        uint32_t keep = 0;
        const int nt = (int)min((uint32_t)kScanTokens, a.n - t0);
        auto token = [&](int t) __attribute__((always_inline)) {
            float pk = 0.f, pq = 0.f;
            vec kk[U];
#pragma unroll
            for (int u = 0; u < U; u++) {
                const int at = t * W + u * 32 * V;
                const vec gg = *reinterpret_cast<const vec *>(bg + at), qq = *reinterpret_cast<const vec *>(bq + at);
                kk[u] = *reinterpret_cast<const vec *>(bk + at);
#pragma unroll
                for (int e = 0; e < V; e++) {
                    S[u][e] *= gg[e];
                    pk = fmaf(S[u][e], kk[u][e], pk);
                    pq = fmaf(S[u][e], qq[e], pq);
                }
            }
            // over the column's two 16-lane rows: the first row takes pk, the second pq, then both go on in one go and are
            // handed to both rows again
            auto x = __builtin_amdgcn_permlane16_swap(__float_as_uint(pk), __float_as_uint(pq), false, false);
            const uint32_t both = __float_as_uint(group16_sum(__uint_as_float(x[0]) + __uint_as_float(x[1])));
            auto y = __builtin_amdgcn_permlane16_swap(both, both, false, false);
            const float sk = __uint_as_float(y[0]), sq = __uint_as_float(y[1]);
            const float up = bv[256 + t] * (bv[t * 16 + ci] - sk);
#pragma unroll
            for (int u = 0; u < U; u++)
#pragma unroll
                for (int e = 0; e < V; e++) S[u][e] = fmaf(kk[u][e], up, S[u][e]);
            // lane t of the column stores token t's read-out; picked by a mask, so that no branch parts the tokens
            keep |= __float_as_uint(fmaf(bv[272 + t], up, sq)) & (uint32_t)((int)((l32 ^ t) - 1) >> 31);
        };
        if (nt == kScanTokens) {
#pragma unroll
            for (int t = 0; t < kScanTokens; t++) token(t);
        } else {
            for (int t = 0; t < nt; t++) token(t);
        }
        if (live && l32 < nt) a.o[(size_t)(t0 + l32) * HV + head * s.vdim + col] = __uint_as_float(keep);
    }
    if (live) {
#pragma unroll
        for (int u = 0; u < U; u++) colp[u * 32] = S[u];
    }
}

}  // namespace lv
