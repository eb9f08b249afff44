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
// do not wait for each other.  Columns of S do not interact: 16 lanes share a column, each holding 4 J of its dim entries.
//
// State of a sequence and layer: S as [head][vdim][64 J] (a column contiguous, zero beyond dim) and a ring of the
// convolution's last `taps` inputs, [position % taps][channel], channels in the order q, k, v.  Nothing has to be cleared for
// a new sequence: positions before 0 and the state at position 0 are never read.
#pragma once

#include "lv_bf16_gemv.h"

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
};

struct DeltaStepArgs {
    DeltaSpec s;
    const float *y;
    const uint32_t *pos_ptr;
    uint32_t pos_add;
    uint32_t blocks;               // column blocks per head
    float *o, *gate;               // [heads * vdim]
};

constexpr int kDeltaCols = 32;     // columns per workgroup of the one-token step
constexpr uint32_t kDeltaMaxDim = 256;
constexpr uint32_t kDeltaMaxRank = 4096;

// channel c (in q, k, v order) of the joint projection
__device__ __forceinline__ uint32_t delta_channel_at(const DeltaSpec &s, uint32_t c)
{
    const uint32_t nq = s.kv_heads * s.dim;
    return c < nq ? s.q_off + c : c < 2 * nq ? s.k_off + (c - nq) : s.v_off + (c - 2 * nq);
}

// convolution and silu of channel c at position pos (slot = pos % taps).  y: the token's projection row; rows before it (in steps of ld floats)
// belong to positions pos - 1, pos - 2, .. as far as `behind` of them, older inputs are in the ring.
__device__ __forceinline__ float delta_conv(const DeltaSpec &s, const float *y, size_t ld, uint32_t behind, uint32_t c, uint32_t pos, uint32_t slot)
{
    const uint32_t at = delta_channel_at(s, c), C = s.channels();
    const float *w = s.conv + (size_t)(s.taps - 1) * C + c;
    float v = w[0] * y[at];
    for (uint32_t j0 = 1; j0 < s.taps && j0 <= pos; j0 += 3) {
        float x[3], f[3];      // three inputs on their way at once
#pragma unroll
        for (uint32_t e = 0; e < 3; e++) {
            const uint32_t j = j0 + e;
            const bool ok = j < s.taps && j <= pos;
            x[e] = !ok ? 0.f : j <= behind ? y[at - (ptrdiff_t)(j * ld)] : s.ring[(size_t)(slot >= j ? slot - j : slot + s.taps - j) * C + c];
            f[e] = ok ? w[-(ptrdiff_t)(j * (size_t)C)] : 0.f;
        }
#pragma unroll
        for (int e = 0; e < 3; e++) v = fmaf(f[e], x[e], v);
    }
    return silu_f(v);
}

// Rows row0 + 32 i (i < N) of a low-rank matrix against a vector in LDS, 8 consecutive lanes a row, every lane of the eight gets
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
        rows = row0 < end ? min((uint32_t)N, (end - row0 + 31) / 32) : 0;
        at = m + (size_t)row0 * kp + (threadIdx.x & 7) * 8;
#pragma unroll
        for (int i = 0; i < N; i++)
#pragma unroll
            for (int k = 0; k < 2; k++)
                w[i][k] = i < (int)rows && k * 64 < (int)kp ? *reinterpret_cast<const uint4 *>(at + (size_t)i * 32 * kp + k * 64) : make_uint4(0, 0, 0, 0);
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
                for (uint32_t k = 128; k < kp; k += 64) t += dot8(*reinterpret_cast<const uint4 *>(at + (size_t)i * 32 * kp + k), x + k);
            out[i] = group8_sum(t);
        }
    }
};

__host__ __device__ constexpr uint32_t delta_step_lds_floats(uint32_t a_kp, uint32_t g_kp) { return 3 * kDeltaMaxDim + kDeltaCols + 16 + a_kp + g_kp; }

// one token, one head, one block of kDeltaCols columns: 256 threads.  Everything the block reads is requested first.
__device__ __forceinline__ void delta_step(const DeltaStepArgs &a, uint32_t idx, float *lds)
{
    const DeltaSpec &s = a.s;
    const uint32_t head = idx / a.blocks, cb = idx % a.blocks, c_lo = cb * kDeltaCols, nc = min((uint32_t)kDeltaCols, s.vdim - c_lo);
    const uint32_t pos = *a.pos_ptr + a.pos_add, rep = s.heads / s.kv_heads, kvh = head / rep, nq = s.kv_heads * s.dim, C = s.channels();
    float *q = lds, *k = q + kDeltaMaxDim, *g = k + kDeltaMaxDim, *v = g + kDeltaMaxDim, *scratch = v + kDeltaCols, *al = scratch + 16, *gl = al + s.a_kp;
    const int l16 = threadIdx.x & 15, c_own = threadIdx.x >> 4, r8 = threadIdx.x >> 3;
    const int J = s.dstride / 64;

    float4 st[2][4];      // this thread's parts of columns c_own and c_own + 16
    float4 *col[2];
#pragma unroll
    for (int h = 0; h < 2; h++) {
        const uint32_t c = min((uint32_t)(c_own + 16 * h), nc - 1);
        col[h] = reinterpret_cast<float4 *>(s.state + ((size_t)head * s.vdim + c_lo + c) * s.dstride) + l16;
#pragma unroll
        for (int j = 0; j < 4; j++) st[h][j] = pos && j < J ? col[h][j * 16] : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    LowRankRows<4> ra;
    LowRankRows<1> rg;
    ra.fetch(s.a2, head * s.dim + r8, (head + 1) * s.dim, s.a_kp);
    rg.fetch(s.g2, head * s.vdim + c_lo + r8, head * s.vdim + c_lo + nc, s.g_kp);
    for (uint32_t i = threadIdx.x; i < s.a_kp; i += 256) al[i] = i < s.a_rank ? a.y[s.a_off + i] : 0.f;
    for (uint32_t i = threadIdx.x; i < s.g_kp; i += 256) gl[i] = i < s.g_rank ? a.y[s.g_off + i] : 0.f;
    const float beta = sigmoid_f(a.y[s.b_off + head]), ea = __expf(s.a_log[head]);

    float qv = 0.f, kv = 0.f;
    const uint32_t d = threadIdx.x, rslot = pos % s.taps;
    if (d < s.dim) {
        const uint32_t cq = kvh * s.dim + d, ck = nq + cq;
        qv = delta_conv(s, a.y, 0, 0, cq, pos, rslot);
        kv = delta_conv(s, a.y, 0, 0, ck, pos, rslot);
        if (cb == 0 && head % rep == 0) {
            s.ring[(size_t)rslot * C + cq] = a.y[s.q_off + cq];
            s.ring[(size_t)rslot * C + ck] = a.y[s.k_off + cq];
        }
    }
    if (threadIdx.x < nc) {
        const uint32_t c = head * s.vdim + c_lo + threadIdx.x;
        v[threadIdx.x] = delta_conv(s, a.y, 0, 0, 2 * nq + c, pos, rslot);
        s.ring[(size_t)rslot * C + 2 * nq + c] = a.y[s.v_off + c];
    }
    float sums[3] = {qv * qv, kv * kv, qv * kv};
    block_sums_waves<3>(sums, scratch, 4);      // also publishes al, gl and v
    const float fq = rsqrtf(sums[0] + 1e-6f) * rsqrtf((float)s.dim), fk = rsqrtf(sums[1] + 1e-6f), qk = sums[2] * fq * fk;
    q[threadIdx.x] = qv * fq;
    k[threadIdx.x] = kv * fk;
    for (uint32_t r0 = 0; r0 < s.dstride; r0 += 128) {
        if (r0) ra.fetch(s.a2, head * s.dim + r0 + r8, (head + 1) * s.dim, s.a_kp);
        float t[4];
        ra.dot(t, al);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t r = r0 + i * 32 + r8;
            if ((threadIdx.x & 7) == i && r < s.dstride)      // four lanes of the eight share the exponentials
                g[r] = r < s.dim ? decay_f(ea, t[i] + s.dt_bias[head * s.dim + r]) : 0.f;
        }
    }
    {
        float t[1];
        rg.dot(t, gl);
        if (r8 < (int)nc && (threadIdx.x & 7) == 0) a.gate[head * s.vdim + c_lo + r8] = sigmoid_f(t[0]);
    }
    __syncthreads();
#pragma unroll
    for (int h = 0; h < 2; h++) {
        const uint32_t c = c_own + 16 * h;
        float pk = 0.f, pq = 0.f;
#pragma unroll
        for (int j = 0; j < 4; j++)
            if (j < J) {
                const int at = j * 64 + l16 * 4;
                float4 x = st[h][j];
                const float4 gg = *reinterpret_cast<const float4 *>(g + at), kk = *reinterpret_cast<const float4 *>(k + at), qq = *reinterpret_cast<const float4 *>(q + at);
                x.x *= gg.x; x.y *= gg.y; x.z *= gg.z; x.w *= gg.w;
                pk = fmaf(x.x, kk.x, pk); pk = fmaf(x.y, kk.y, pk); pk = fmaf(x.z, kk.z, pk); pk = fmaf(x.w, kk.w, pk);
                pq = fmaf(x.x, qq.x, pq); pq = fmaf(x.y, qq.y, pq); pq = fmaf(x.z, qq.z, pq); pq = fmaf(x.w, qq.w, pq);
                st[h][j] = x;
            }
        pk = group16_sum(pk);
        pq = group16_sum(pq);
        if (c >= nc) continue;
        const float u = beta * (v[c] - pk);
#pragma unroll
        for (int j = 0; j < 4; j++)
            if (j < J) {
                const float4 kk = *reinterpret_cast<const float4 *>(k + j * 64 + l16 * 4);
                float4 x = st[h][j];
                x.x = fmaf(kk.x, u, x.x); x.y = fmaf(kk.y, u, x.y); x.z = fmaf(kk.z, u, x.z); x.w = fmaf(kk.w, u, x.w);
                col[h][j * 16] = x;
            }
        if (l16 == 0) a.o[head * s.vdim + c_lo + c] = fmaf(qk, u, pq);
    }
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

// All tokens of a batch for 16 columns of one head: a workgroup of 4 waves, 4 columns a wave.  grid (heads, vdim / 16 up).
template <int J>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaScanArgs a)
{
    constexpr int W = 64 * J, SF = scan_stage_floats<J>();
    extern __shared__ float lds[];       // two stages
    const DeltaSpec &s = a.s;
    const uint32_t head = blockIdx.x, kvh = head / (s.heads / s.kv_heads), HV = s.heads * s.vdim;
    const int l16 = threadIdx.x & 15, ci = threadIdx.x >> 4;
    const uint32_t col = blockIdx.y * 16 + ci;
    const bool live = col < s.vdim;
    float4 *const colp = reinterpret_cast<float4 *>(s.state + ((size_t)head * s.vdim + (live ? col : 0)) * W);
    float4 S[J];
#pragma unroll
    for (int j = 0; j < J; j++) S[j] = a.fresh || !live ? make_float4(0.f, 0.f, 0.f, 0.f) : colp[j * 16 + l16];

    // One stage in LDS: k, q, g [16][W] each, v [16][16], beta [16], k.q [16].  Direct loads, lane after lane in LDS order; tokens
    // past the end and columns past vdim bring some other value that nothing uses.
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    auto issue = [&](uint32_t t0, int st) {
        float *b = lds + st * SF;
#pragma unroll
        for (int i = 0; i < J; i++) {
            const int e = i * 256 + wave * 64;                   // first float4 of the wave
            const uint32_t t = min(t0 + (e + lane) / (W / 4), a.n - 1), d = (e + lane) % (W / 4) * 4;
            const size_t kq = ((size_t)t * s.kv_heads + kvh) * W + d;
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.k + kq), (lv_lds_any *)(b + e * 4), 16, 0, 0);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.q + kq), (lv_lds_any *)(b + kScanTokens * W + e * 4), 16, 0, 0);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.g + ((size_t)t * s.heads + head) * W + d), (lv_lds_any *)(b + 2 * kScanTokens * W + e * 4), 16, 0, 0);
        }
        {
            const uint32_t t = min(t0 + wave * 4 + lane / 16, a.n - 1), c = min(blockIdx.y * 16 + lane % 16, s.vdim - 1);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.v + (size_t)t * HV + head * s.vdim + c), (lv_lds_any *)(b + 3 * kScanTokens * W + wave * 64), 4, 0, 0);
        }
        if (wave == 0) {
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
        const float *b = lds + st * SF, *bk = b, *bq = b + kScanTokens * W, *bg = b + 2 * kScanTokens * W, *bv = b + 3 * kScanTokens * W;
        uint32_t keep = 0;
        const int nt = (int)min((uint32_t)kScanTokens, a.n - t0);
        auto token = [&](int t) __attribute__((always_inline)) {
            float pk = 0.f, pq = 0.f;
            float4 kk[J];
#pragma unroll
            for (int j = 0; j < J; j++) {
                const int at = t * W + j * 64 + l16 * 4;
                const float4 gg = *reinterpret_cast<const float4 *>(bg + at), qq = *reinterpret_cast<const float4 *>(bq + at);
                kk[j] = *reinterpret_cast<const float4 *>(bk + at);
                S[j].x *= gg.x; S[j].y *= gg.y; S[j].z *= gg.z; S[j].w *= gg.w;
                pk = fmaf(S[j].x, kk[j].x, pk); pk = fmaf(S[j].y, kk[j].y, pk); pk = fmaf(S[j].z, kk[j].z, pk); pk = fmaf(S[j].w, kk[j].w, pk);
                pq = fmaf(S[j].x, qq.x, pq); pq = fmaf(S[j].y, qq.y, pq); pq = fmaf(S[j].z, qq.z, pq); pq = fmaf(S[j].w, qq.w, pq);
            }
            pk = group16_sum(pk);
            pq = group16_sum(pq);
            const float u = bv[256 + t] * (bv[t * 16 + ci] - pk);
#pragma unroll
            for (int j = 0; j < J; j++) {
                S[j].x = fmaf(kk[j].x, u, S[j].x); S[j].y = fmaf(kk[j].y, u, S[j].y); S[j].z = fmaf(kk[j].z, u, S[j].z); S[j].w = fmaf(kk[j].w, u, S[j].w);
            }
            // lane t of the sixteen stores token t's read-out; picked by a mask, so that no branch parts the tokens
            keep |= __float_as_uint(fmaf(bv[272 + t], u, pq)) & (uint32_t)((int)((l16 ^ t) - 1) >> 31);
        };
        if (nt == kScanTokens) {
#pragma unroll
            for (int t = 0; t < kScanTokens; t++) token(t);
        } else {
            for (int t = 0; t < nt; t++) token(t);
        }
        if (live && l16 < nt) a.o[(size_t)(t0 + l16) * HV + head * s.vdim + col] = __uint_as_float(keep);
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < J; j++) colp[j * 16 + l16] = S[j];
    }
}

}  // namespace lv
