// lv_ssm.h — state-space recurrence with a scalar decay per head (Mamba-2), one state x vdim matrix per head.
//
//   z, x, B, C, dt   one projection; x, B and C together through a short causal convolution with bias and silu (lv_conv.h)
//   dt   <- softplus(dt + dt_bias), one per head;  a = exp(-exp(A_log) dt)
//   S    <- a S + dt B x^T   (B and C shared by the consecutive heads of a group);  y = S^T C + D x
//   out  = RMS norm of y silu(z) in equal parts, times weights (GroupInput)
//
// State, step sizes, decays and their products are fp32.  Columns of S do not interact and nothing is fed back from a read-out: from token to token a state entry goes
// through one multiply-add, and the sums of the read-outs are off that chain.
//
// Token by token (one-token steps, and batches of 32-bit models) a step is taken as it stands.  Batches with bf16 activations go
// in chunks of tokens on the matrix cores (ssm_chunk_kernel).
//
// State of a sequence and pass: S as [head][vdim][64 J] (a column contiguous, zero beyond the state size) and a ring of the
// convolution's last `taps` inputs.  Nothing has to be cleared for a new sequence: positions before 0 and the state at position 0
// are never read.
#pragma once

#include "lv_conv.h"

namespace lv {

struct SsmSpec {
    uint32_t heads, groups, n, vdim, taps, norm_groups;
    uint32_t z_off, x_off, dt_off;       // offsets in a token's projection; x, B and C follow one another
    const float *conv, *bias;            // [taps][channels] (last row = the current token), [channels]
    const float *a_log, *dt_bias, *skip, *norm;
    float eps;
    float *state, *ring;
    uint32_t nstride;                    // 64 J, J = 1, 2 or 4
    __host__ __device__ uint32_t inner() const { return heads * vdim; }
    __host__ __device__ uint32_t channels() const { return heads * vdim + 2 * groups * n; }
    __device__ __forceinline__ uint32_t channel_at(uint32_t c) const { return x_off + c; }
    __device__ __forceinline__ float conv_bias(uint32_t c) const { return bias[c]; }
};

constexpr uint32_t kSsmMaxState = 256;
constexpr int kSsmCols = 32;             // columns per workgroup of the one-token step: 16 lanes to each
constexpr int kSsmStepThreads = 512;

struct SsmStepArgs {
    SsmSpec s;
    const float *y;
    const uint32_t *pos_ptr;
    uint32_t pos_add;
    uint32_t blocks;                     // column blocks per head
    float *o;                            // [heads * vdim]
};

// One token, one head, one block of kSsmCols columns.  Everything is requested first, the short-lived before the state.
static __global__ __launch_bounds__(kSsmStepThreads) void ssm_step_kernel(SsmStepArgs a)
{
    __shared__ __attribute__((aligned(16))) float bc[2][kSsmMaxState];
    __shared__ float xs[kSsmCols];
    const SsmSpec &s = a.s;
    const uint32_t head = blockIdx.x / a.blocks, cb = blockIdx.x % a.blocks, c_lo = cb * kSsmCols, nc = min((uint32_t)kSsmCols, s.vdim - c_lo);
    const uint32_t pos = *a.pos_ptr + a.pos_add, rep = s.heads / s.groups, grp = head / rep, inner = s.inner(), C = s.channels(), slot = pos % s.taps, J = s.nstride / 64;
    // threads 0 .. 255: entry d of B, the others: of C; the first 32 also a column of x
    const uint32_t d = threadIdx.x & 255, half = threadIdx.x >> 8, cd = inner + (half * s.groups + grp) * s.n + d, cx = head * s.vdim + c_lo + threadIdx.x;
    ShortConv bc_in{}, x_in{};
    if (d < s.n) bc_in.fetch(s, a.y, 0, 0, cd, pos, slot);
    if (threadIdx.x < nc) x_in.fetch(s, a.y, 0, 0, cx, pos, slot);
    const float dt_in = a.y[s.dt_off + head] + s.dt_bias[head], a_log = s.a_log[head], skip = s.skip[head];
    const uint32_t c_own = threadIdx.x >> 4, l16 = threadIdx.x & 15;
    float4 *const col = reinterpret_cast<float4 *>(s.state + ((size_t)head * s.vdim + c_lo + min(c_own, nc - 1)) * s.nstride) + l16;
    float4 st[4];
#pragma unroll
    for (int j = 0; j < 4; j++) st[j] = pos && j < (int)J ? col[j * 16] : make_float4(0.f, 0.f, 0.f, 0.f);
    float v = 0.f;
    if (d < s.n) {
        v = bc_in.value(s, a.y, 0, 0, pos, slot);
        if (cb == 0 && head % rep == 0) s.ring[(size_t)slot * C + cd] = bc_in.x[0];
    }
    bc[half][d] = v;
    if (threadIdx.x < nc) {
        xs[threadIdx.x] = x_in.value(s, a.y, 0, 0, pos, slot);
        s.ring[(size_t)slot * C + cx] = x_in.x[0];
    }
    const float dt = softplus_f(dt_in), decay = __expf(-__expf(a_log) * dt);
    __syncthreads();
    if (c_own >= nc) return;
    const float x = xs[c_own], dx = dt * x;
    float y = 0.f;
#pragma unroll
    for (int j = 0; j < 4; j++)
        if (j < (int)J) {
            const float4 b = *reinterpret_cast<const float4 *>(&bc[0][j * 64 + l16 * 4]), c = *reinterpret_cast<const float4 *>(&bc[1][j * 64 + l16 * 4]);
            float4 e = st[j];
            e.x = fmaf(e.x, decay, dx * b.x); e.y = fmaf(e.y, decay, dx * b.y); e.z = fmaf(e.z, decay, dx * b.z); e.w = fmaf(e.w, decay, dx * b.w);
            y = fmaf(e.x, c.x, y); y = fmaf(e.y, c.y, y); y = fmaf(e.z, c.z, y); y = fmaf(e.w, c.w, y);
            col[j * 16] = e;
        }
    y = group16_sum(y);
    if (l16 == 0) a.o[head * s.vdim + c_lo + c_own] = fmaf(skip, x, y);
}

// ---- batches -------------------------------------------------------------------------------------------------------------
struct SsmBatchArgs {
    SsmSpec s;
    const float *y;                      // [n][ldy]: the projections
    uint32_t ldy, pos0, n;
    float *x;                            // [n][inner]
    float *b, *c;                        // [n][groups][nstride], zero beyond the state size
    float *dt, *decay;                   // [n][heads]
    float *o;                            // [n][inner]
};

constexpr uint32_t kSsmPrepareTokens = 8;
inline uint32_t ssm_prepare_columns(const SsmSpec &s) { return (s.heads * s.vdim + 2 * s.groups * s.nstride + s.heads + 255) / 256; }
// grid (ssm_prepare_columns, n / 8 up): a thread per channel (B and C padded) or head, eight tokens
static __global__ __launch_bounds__(256) void ssm_prepare_kernel(SsmBatchArgs a)
{
    const SsmSpec &s = a.s;
    const uint32_t inner = s.inner(), gn = s.groups * s.nstride, first = blockIdx.y * kSsmPrepareTokens, last = min(first + kSsmPrepareTokens, a.n);
    uint32_t c = blockIdx.x * 256 + threadIdx.x;
    if (c < inner + 2 * gn) {
        float *out = a.x + c;
        size_t ld = inner;
        uint32_t channel = c;
        bool pad = false;
        if (c >= inner) {
            c -= inner;
            out = c < gn ? a.b + c : a.c + (c - gn);
            ld = gn;
            const uint32_t which = c / gn, g = c % gn / s.nstride, d = c % s.nstride;
            pad = d >= s.n;
            channel = inner + (which * s.groups + g) * s.n + d;
        }
        float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (!pad) short_conv8(v, s, a.y, a.ldy, channel, a.pos0, first, a.n);
#pragma unroll
        for (uint32_t i = 0; i < kSsmPrepareTokens; i++)
            if (first + i < last) out[(first + i) * ld] = v[i];
        return;
    }
    c -= inner + 2 * gn;
    if (c >= s.heads) return;
    const float ea = __expf(s.a_log[c]), bias = s.dt_bias[c];
    for (uint32_t t = first; t < last; t++) {
        const float dt = softplus_f(a.y[(size_t)t * a.ldy + s.dt_off + c] + bias);
        a.dt[(size_t)t * s.heads + c] = dt;
        a.decay[(size_t)t * s.heads + c] = __expf(-ea * dt);
    }
}

// the batch's last convolution inputs into the ring; blockIdx.x = token counted from the end, blockIdx.y = 256 channels
static __global__ __launch_bounds__(256) void ssm_append_kernel(SsmBatchArgs a)
{
    const SsmSpec &s = a.s;
    const uint32_t t = a.n - 1 - blockIdx.x, C = s.channels(), c = blockIdx.y * 256 + threadIdx.x;
    if (c < C) s.ring[(size_t)((a.pos0 + t) % s.taps) * C + c] = a.y[(size_t)t * a.ldy + s.channel_at(c)];
}

constexpr int kSsmScanTokens = 16, kSsmScanThreads = 256;
template <int J> constexpr int ssm_stage_floats() { return kSsmScanTokens * (2 * 64 * J + 16) + 64; }

// All tokens of a batch for 16 columns of one head, in fp32 throughout: 4 waves, 16 lanes a column.  grid (heads, vdim / 16 up).
template <int J>
__global__ __launch_bounds__(kSsmScanThreads) void ssm_scan_kernel(SsmBatchArgs a)
{
    constexpr int W = 64 * J, SF = ssm_stage_floats<J>(), T = kSsmScanTokens;
    extern __shared__ __attribute__((aligned(16))) float lds[];       // two stages
    const SsmSpec &s = a.s;
    const uint32_t head = blockIdx.x, grp = head / (s.heads / s.groups), inner = s.inner();
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l16 = lane & 15, ci = threadIdx.x >> 4;
    const uint32_t col = blockIdx.y * 16 + ci;
    const bool live = col < s.vdim;
    float4 *const colp = reinterpret_cast<float4 *>(s.state + ((size_t)head * s.vdim + (live ? col : 0)) * W) + l16;
    float4 S[J];
#pragma unroll
    for (int j = 0; j < J; j++) S[j] = a.pos0 == 0 || !live ? make_float4(0.f, 0.f, 0.f, 0.f) : colp[j * 16];
    const float skip = s.skip[head];
    // One stage: B and C [16][W] each, x [16][16], dt [16], decay [16].  Direct loads, lane after lane in LDS order; tokens past
    // the end and columns past vdim bring some other value that nothing uses.
    auto issue = [&](uint32_t t0, int st) {
        float *b = lds + st * SF;
#pragma unroll
        for (int i = 0; i < J; i++) {
            const int e = (i * 4 + wave) * 64;             // first float4 of the wave, of 256 J
            const uint32_t t = min(t0 + (e + lane) / (W / 4), a.n - 1), d = (e + lane) % (W / 4) * 4;
            const size_t at = ((size_t)t * s.groups + grp) * W + d;
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.b + at), (lv_lds_any *)(b + e * 4), 16, 0, 0);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.c + at), (lv_lds_any *)(b + T * W + e * 4), 16, 0, 0);
        }
        {
            const uint32_t t = min(t0 + wave * 4 + lane / 16, a.n - 1), c = min(blockIdx.y * 16 + lane % 16, s.vdim - 1);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(a.x + (size_t)t * inner + head * s.vdim + c), (lv_lds_any *)(b + 2 * T * W + wave * 64), 4, 0, 0);
        }
        if (wave == 0) {
            const float *src = (lane & 16 ? a.decay : a.dt) + (size_t)min(t0 + (lane & 15), a.n - 1) * s.heads + head;
            __builtin_amdgcn_global_load_lds((lv_glb_any *)src, (lv_lds_any *)(b + 2 * T * W + 256), 4, 0, 0);
        }
    };
    issue(0, 0);
    for (uint32_t t0 = 0, st = 0; t0 < a.n; t0 += T, st ^= 1) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();      // this stage is in LDS for everyone, and everyone is done with the other one
        if (t0 + T < a.n) issue(t0 + T, st ^ 1);
        const float *b = lds + st * SF, *bb = b + l16 * 4, *bc = bb + T * W, *bx = b + 2 * T * W;
        float keep = 0.f;
        const int nt = (int)min((uint32_t)T, a.n - t0);
        auto token = [&](int t) __attribute__((always_inline)) {
            const float x = bx[t * 16 + ci], dx = bx[256 + t] * x, decay = bx[272 + t];
            float y = 0.f;
#pragma unroll
            for (int j = 0; j < J; j++) {
                const float4 vb = *reinterpret_cast<const float4 *>(bb + t * W + j * 64), vc = *reinterpret_cast<const float4 *>(bc + t * W + j * 64);
                S[j].x = fmaf(S[j].x, decay, dx * vb.x); S[j].y = fmaf(S[j].y, decay, dx * vb.y);
                S[j].z = fmaf(S[j].z, decay, dx * vb.z); S[j].w = fmaf(S[j].w, decay, dx * vb.w);
                y = fmaf(S[j].x, vc.x, y); y = fmaf(S[j].y, vc.y, y); y = fmaf(S[j].z, vc.z, y); y = fmaf(S[j].w, vc.w, y);
            }
            y = fmaf(skip, x, group16_sum(y));
            keep = l16 == t ? y : keep;      // lane t of the column stores token t's read-out
        };
        if (nt == T) {
#pragma unroll
            for (int t = 0; t < T; t++) token(t);
        } else {
            for (int t = 0; t < nt; t++) token(t);
        }
        if (live && l16 < nt) a.o[(size_t)(t0 + l16) * inner + head * s.vdim + col] = keep;
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < J; j++) colp[j * 16] = S[j];
    }
}

// ---- batches in chunks -------------------------------------------------------------------------------------------------------
// With l_t the running sum of -exp(A) dt inside a chunk of Q tokens, l its last one and S the state in front of it:
//   y_t = exp(l_t) S^T C_t + sum_{s <= t} (C_t . B_s) exp(l_t - l_s) dt_s x_s + D x_t
//   S  <- exp(l) S + sum_s B_s (exp(l - l_s) dt_s x_s)^T
// all products of matrices over the chunk; every exponent is a sum of decays of tokens in a row, so none of them overflows.  x, B
// and C are bf16 as a convolution's output; the state enters a product as three bf16 pieces (24 bits), weights and weighted x as
// two; sums are fp32.
struct SsmChunkArgs {
    SsmSpec s;
    const float *y;                      // [n][ldy]: the projections
    uint32_t ldy, pos0, n;
    uint32_t ldt;                        // n rounded up to kSsmChunk: tokens the operands below have, zeros past the end
    uint16_t *xt;                        // [ldt / 8][inner][8 tokens]
    uint16_t *b, *c;                     // [ldt][groups][nstride], zero beyond the state size, entries in ssm_place order
    uint16_t *bt;                        // [ldt / 8][groups][nstride][8 tokens]
    float *dt;                           // [heads][ldt]
    float *o;                            // [n][inner]
};
constexpr uint32_t kSsmChunk = 64;
// Where entry d of B or C lies in its row: the order in which a lane's state registers make up a matrix operand (place 8 g + 4 t + r
// of 32 holds entry 16 t + 4 g + r)
__host__ __device__ constexpr uint32_t ssm_place(uint32_t d) { return (d & ~31u) | ((d >> 2) & 3) << 3 | ((d >> 4) & 1) << 2 | (d & 3); }

// grid (ssm_prepare_columns, ldt / 8): a thread per channel (B and C padded) or head, eight tokens
static __global__ __launch_bounds__(256) void ssm_operands_kernel(SsmChunkArgs a)
{
    const SsmSpec &s = a.s;
    const uint32_t inner = s.inner(), gn = s.groups * s.nstride, t8 = blockIdx.y, t0 = t8 * 8;
    uint32_t c = blockIdx.x * 256 + threadIdx.x;
    if (c >= inner + 2 * gn) {
        c -= inner + 2 * gn;
        if (c >= s.heads) return;
        const float bias = s.dt_bias[c];
        float dt[8];
#pragma unroll
        for (uint32_t i = 0; i < 8; i++) dt[i] = t0 + i < a.n ? softplus_f(a.y[(size_t)(t0 + i) * a.ldy + s.dt_off + c] + bias) : 0.f;
        float4 *out = reinterpret_cast<float4 *>(a.dt + (size_t)c * a.ldt + t0);
        out[0] = make_float4(dt[0], dt[1], dt[2], dt[3]);
        out[1] = make_float4(dt[4], dt[5], dt[6], dt[7]);
        return;
    }
    uint32_t channel = c, place = 0, e = 0;
    bool pad = false;
    if (c >= inner) {
        e = c - inner;                   // of B, then of C
        const uint32_t d = e % s.nstride;
        pad = d >= s.n;
        channel = inner + e / s.nstride * s.n + d;
        place = e - d + ssm_place(d);
    }
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (!pad) short_conv8(v, s, a.y, a.ldy, channel, a.pos0, t0, a.n);
    uint16_t h[8];
#pragma unroll
    for (uint32_t i = 0; i < 8; i++) h[i] = float_to_bf16(v[i]);
    const uint4 eight = make_uint4(h[0] | (uint32_t)h[1] << 16, h[2] | (uint32_t)h[3] << 16, h[4] | (uint32_t)h[5] << 16, h[6] | (uint32_t)h[7] << 16);
    if (c < inner) {
        reinterpret_cast<uint4 *>(a.xt)[(size_t)t8 * inner + c] = eight;
        return;
    }
    uint16_t *rows = e < gn ? a.b + place : a.c + (place - gn);
#pragma unroll
    for (uint32_t i = 0; i < 8; i++) rows[(size_t)(t0 + i) * gn] = h[i];
    if (e < gn) reinterpret_cast<uint4 *>(a.bt)[(size_t)t8 * gn + e] = eight;
}

// the upper halves of two words, the first one's below
__device__ __forceinline__ uint32_t upper_halves(uint32_t a, uint32_t b) { return __builtin_amdgcn_perm(b, a, 0x07060302u); }
// The leading bf16 pieces of eight values, cut off them (not rounded: three in a row are all 24 bits); v keeps the rest
__device__ __forceinline__ lv_bf8 next_piece(float (&v)[8])
{
    uint4 p;
    uint32_t *w = reinterpret_cast<uint32_t *>(&p);
#pragma unroll
    for (int e = 0; e < 8; e += 2) {
        const uint32_t a = __float_as_uint(v[e]), b = __float_as_uint(v[e + 1]);
        w[e / 2] = upper_halves(a, b);
        v[e] -= __uint_as_float(a & 0xffff0000u);
        v[e + 1] -= __uint_as_float(b & 0xffff0000u);
    }
    return __builtin_bit_cast(lv_bf8, p);
}

constexpr int kSsmChunkThreads = 256;
template <int J> constexpr int ssm_chunk_stages() { return J <= 2 ? 2 : 1; }
template <int J> constexpr int ssm_chunk_stage_bytes() { return 3 * kSsmChunk * 64 * J * 2; }      // C and B rows, B by 8 tokens
constexpr int kSsmWeightLd = kSsmChunk + 8;
template <int J> constexpr int ssm_chunk_lds() { return ssm_chunk_stages<J>() * ssm_chunk_stage_bytes<J>() + 2 * kSsmChunk * kSsmWeightLd * 2 + 4 * 4 * kSsmChunk * 4; }

// All chunks of a batch, one after the other, for 64 columns of one head: 4 waves, 16 columns and all of their state each.  grid
// (heads, vdim / 64 up).  The weights (C_t . B_s) exp(l_t - l_s) dt_s of a chunk are shared out, 16 tokens a wave, and meet in LDS.
template <int J>
__global__ __launch_bounds__(kSsmChunkThreads) void ssm_chunk_kernel(SsmChunkArgs a)
{
    constexpr int W = 64 * J, ROW = W * 2, NST = ssm_chunk_stages<J>(), STAGE = ssm_chunk_stage_bytes<J>(), TILE = kSsmChunk * ROW;
    extern __shared__ __attribute__((aligned(128))) uint8_t chunk_lds[];
    const SsmSpec &s = a.s;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l16 = lane & 15, g4 = lane >> 4;
    uint16_t *const mh = reinterpret_cast<uint16_t *>(chunk_lds + NST * STAGE), *const ml = mh + kSsmChunk * kSsmWeightLd;
    // of this wave's own: l_t, dt_t, exp(l_t), exp(l - l_t) dt_t
    float *const lt = reinterpret_cast<float *>(ml + kSsmChunk * kSsmWeightLd) + wave * 4 * kSsmChunk, *const dts = lt + kSsmChunk, *const el = dts + kSsmChunk, *const wt = el + kSsmChunk;
    const uint32_t head = blockIdx.x, grp = head / (s.heads / s.groups), inner = s.inner(), p = blockIdx.y * 64 + wave * 16 + l16;
    const bool live = p < s.vdim;
    const uint32_t channel = head * s.vdim + min(p, s.vdim - 1);
    float4 *const state = reinterpret_cast<float4 *>(s.state + (size_t)channel * W);
    const float rate = -__expf(s.a_log[head]), skip = s.skip[head];

    // a stage: 256 threads bring 32 / J rows of C and of B at a time, and as many entries of B by 8 tokens
    const uint32_t gw = s.groups * W, row0 = threadIdx.x / (8 * J), ch0 = threadIdx.x % (8 * J);
    const size_t rows_at = ((size_t)row0 * s.groups + grp) * W + (ch0 ^ (row0 & 7)) * 8, by8_at = (((size_t)(threadIdx.x / W) * s.groups + grp) * W + threadIdx.x % W) * 8;
    const uint16_t *gc = a.c + rows_at, *gb = a.b + rows_at, *gt = a.bt + by8_at;      // of the next stage
    auto issue = [&](int st) {
        uint8_t *b = chunk_lds + st * STAGE + wave * 1024;
#pragma unroll
        for (int i = 0; i < 2 * J; i++) {
            const uint32_t on = i * (32 / J) * gw;       // both in steps of 256 threads' worth
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(gc + on), (lv_lds_any *)(b + i * 4096), 16, 0, 0);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(gb + on), (lv_lds_any *)(b + TILE + i * 4096), 16, 0, 0);
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(gt + on), (lv_lds_any *)(b + 2 * TILE + i * 4096), 16, 0, 0);
        }
        gc += kSsmChunk * gw;
        gb += kSsmChunk * gw;
        gt += kSsmChunk * gw;
    };
    uint4 xn[2];
    float dtn;
    auto request = [&](uint32_t t0) {
#pragma unroll
        for (int k = 0; k < 2; k++) xn[k] = reinterpret_cast<const uint4 *>(a.xt)[(size_t)(t0 / 8 + k * 4 + g4) * inner + channel];
        dtn = a.dt[(size_t)head * a.ldt + t0 + lane];
    };
    issue(0);
    request(0);
    lv_f4 S[4 * J];
#pragma unroll
    for (int i = 0; i < 4 * J; i++) {
        const float4 v = a.pos0 == 0 || !live ? make_float4(0.f, 0.f, 0.f, 0.f) : state[i * 4 + g4];
        S[i] = lv_f4{v.x, v.y, v.z, v.w};
    }

    for (uint32_t t0 = 0, st = 0; t0 < a.n; t0 += kSsmChunk, st = NST == 2 ? st ^ 1 : 0) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();      // this stage is in LDS for everyone, and everyone is done with the other one and with the weights
        const uint4 x[2] = {xn[0], xn[1]};
        const float dt = dtn;
        const bool more = t0 + kSsmChunk < a.n;
        if (more) {
            if (NST == 2) issue(st ^ 1);
            request(t0 + kSsmChunk);
        }
        const uint8_t *bc = chunk_lds + st * STAGE, *bb = bc + TILE, *bt = bb + TILE;
        auto frag = [&](const uint8_t *tile, int row, int k) { return *reinterpret_cast<const lv_bf8 *>(tile + row * ROW + ((k * 4 + g4) ^ (row & 7)) * 16); };

        const float l = wave_running_sum(rate * dt), end = __shfl(l, 63, 64);
        lt[lane] = l;
        dts[lane] = dt;
        el[lane] = __expf(l);
        wt[lane] = __expf(end - l) * dt;
        __builtin_amdgcn_fence(__ATOMIC_SEQ_CST, "wavefront");
        __builtin_amdgcn_wave_barrier();

        // weights: three tiles of 16 x 16 a wave, as (token tile, source tile); (0, 1) and (2, 3) are zeros
        const uint32_t mine = wave == 0 ? 0x302000u : wave == 1 ? 0x311110u : wave == 2 ? 0x232221u : 0x013332u;
#pragma unroll
        for (int q = 0; q < 3; q++) {
            const int ti = mine >> (8 * q + 4) & 15, si = mine >> (8 * q) & 15, t = ti * 16 + l16;
            lv_f4 g = lv_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < 2 * J; k++) g = __builtin_amdgcn_mfma_f32_16x16x32_bf16(frag(bb, si * 16 + l16, k), frag(bc, t, k), g, 0, 0, 0);
            const float4 ls = *reinterpret_cast<const float4 *>(lt + si * 16 + g4 * 4), ds = *reinterpret_cast<const float4 *>(dts + si * 16 + g4 * 4);
            const float lsv[4] = {ls.x, ls.y, ls.z, ls.w}, dsv[4] = {ds.x, ds.y, ds.z, ds.w}, to = lt[t];
            uint32_t m[4], r[4];
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int u = si * 16 + g4 * 4 + e;
                const float w = g[e] * dsv[e] * __expf(to - lsv[e]), v = u < t ? w : u == t ? w + skip : 0.f;
                m[e] = __float_as_uint(v);
                r[e] = __float_as_uint(v - __uint_as_float(m[e] & 0xffff0000u));
            }
            const int at = t * kSsmWeightLd + si * 16 + g4 * 4;
            *reinterpret_cast<uint2 *>(mh + at) = make_uint2(upper_halves(m[0], m[1]), upper_halves(m[2], m[3]));
            *reinterpret_cast<uint2 *>(ml + at) = make_uint2(upper_halves(r[0], r[1]), upper_halves(r[2], r[3]));
        }
        // read-outs: the state's part needs no weights and runs up to the barrier
        lv_f4 y[4];
#pragma unroll
        for (int i = 0; i < 4; i++) y[i] = lv_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < 2 * J; k++) {
            lv_bf8 q[3];
            {
                float v[8];
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = S[2 * k + e / 4][e % 4];
#pragma unroll
                for (int c = 0; c < 3; c++) q[c] = next_piece(v);
            }
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const lv_bf8 f = frag(bc, i * 16 + l16, k);
#pragma unroll
                for (int c = 2; c >= 0; c--) y[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f, q[c], y[i], 0, 0, 0);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float4 e = *reinterpret_cast<const float4 *>(el + i * 16 + g4 * 4);
            y[i][0] *= e.x; y[i][1] *= e.y; y[i][2] *= e.z; y[i][3] *= e.w;
        }
        const lv_bf8 fx[2] = {__builtin_bit_cast(lv_bf8, x[0]), __builtin_bit_cast(lv_bf8, x[1])};
        __syncthreads();      // the weights are there
#pragma unroll
        for (int i = 0; i < 4; i++)
#pragma unroll
            for (int k = 0; k <= i / 2; k++) {
                const int at = (i * 16 + l16) * kSsmWeightLd + k * 32 + g4 * 8;
                y[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const lv_bf8 *>(ml + at), fx[k], y[i], 0, 0, 0);
                y[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const lv_bf8 *>(mh + at), fx[k], y[i], 0, 0, 0);
            }
        // the state behind the chunk
        const float all = __expf(end);
#pragma unroll
        for (int i = 0; i < 4 * J; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) S[i][r] *= all;
#pragma unroll
        for (int k = 0; k < 2; k++) {
            float w[8];
            load8(w, wt + k * 32 + g4 * 8);
#pragma unroll
            for (int e = 0; e < 8; e++) w[e] *= (float)fx[k][e];
            const lv_bf8 xh = next_piece(w), xl = next_piece(w);
#pragma unroll
            for (int i = 0; i < 4 * J; i++) {
                const lv_bf8 f = *reinterpret_cast<const lv_bf8 *>(bt + ((k * 4 + g4) * W + i * 16 + l16) * 16);
                S[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f, xl, S[i], 0, 0, 0);
                S[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f, xh, S[i], 0, 0, 0);
            }
        }
        if (live) {
            float *out = a.o + (size_t)(t0 + g4 * 4) * inner + channel;
            const uint32_t left = a.n - t0;
            if (left >= kSsmChunk) {
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int r = 0; r < 4; r++) out[(i * 16 + r) * inner] = y[i][r];
            } else {
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        if ((uint32_t)(i * 16 + g4 * 4 + r) < left) out[(i * 16 + r) * inner] = y[i][r];
            }
        }
        if (NST == 1 && more) {
            __syncthreads();
            issue(0);
        }
    }
    if (live) {
#pragma unroll
        for (int i = 0; i < 4 * J; i++) state[i * 4 + g4] = make_float4(S[i][0], S[i][1], S[i][2], S[i][3]);
    }
}

// gated, normed read-outs of a batch as activations; LDS: inner + group_sums + 4 floats.  z: [row][ldz]
template <class T>
__global__ __launch_bounds__(256) void ssm_gate_kernel(GroupInput g, uint32_t ldz, T *__restrict__ act, uint32_t ld)
{
    extern __shared__ __attribute__((aligned(16))) float gs[];
    const size_t row = blockIdx.x;
    g.o += row * g.n;
    g.z += row * ldz;
    group_input(g, gs + g.n, [&](uint32_t i, auto v) { *reinterpret_cast<decltype(v) *>(gs + i) = v; },
                [&](uint32_t i, auto &v) { v = *reinterpret_cast<std::decay_t<decltype(v)> *>(gs + i); });
    __syncthreads();
    T *out = act + row * ld;          // ld is a multiple of 64; gs is readable to the next multiple of four
    for (uint32_t i = threadIdx.x * 4; i < ld; i += 1024) {
        const float4 v = *reinterpret_cast<const float4 *>(gs + min(i, g.n & ~3u));
        float f[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (uint32_t e = 0; e < 4; e++) f[e] = i + e < g.n ? f[e] : 0.f;
        if constexpr (sizeof(T) == 2)
            *reinterpret_cast<uint2 *>(out + i) = make_uint2((uint32_t)float_to_bf16(f[0]) | ((uint32_t)float_to_bf16(f[1]) << 16),
                                                             (uint32_t)float_to_bf16(f[2]) | ((uint32_t)float_to_bf16(f[3]) << 16));
        else *reinterpret_cast<float4 *>(out + i) = make_float4(f[0], f[1], f[2], f[3]);
    }
}

}  // namespace lv
