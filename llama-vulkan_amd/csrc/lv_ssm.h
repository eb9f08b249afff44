// lv_ssm.h — state-space recurrence with a scalar decay per head (Mamba-2), one state x vdim matrix per head.
//
//   z, x, B, C, dt   one projection; x, B and C together through a short causal convolution with bias and silu (lv_conv.h)
//   dt   <- softplus(dt + dt_bias), one per head;  a = exp(-exp(A_log) dt)
//   S    <- a S + dt B x^T   (B and C shared by the consecutive heads of a group);  y = S^T C + D x
//   out  = RMS norm of y silu(z) in equal parts, times weights (GroupInput)
//
// All of it is fp32.  Columns of S do not interact and nothing is fed back from a read-out: from token to token a state entry goes
// through one multiply-add, and the sums of the read-outs are off that chain.
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
    uint32_t nstride;                    // 64 J
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
        for (uint32_t t = first; t < last; t++) out[t * ld] = pad ? 0.f : short_conv(s, a.y + (size_t)t * a.ldy, a.ldy, t, channel, a.pos0 + t, (a.pos0 + t) % s.taps);
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

// the batch's last convolution inputs into the ring; blockIdx.x = token counted from the end
static __global__ __launch_bounds__(256) void ssm_append_kernel(SsmBatchArgs a)
{
    const SsmSpec &s = a.s;
    const uint32_t t = a.n - 1 - blockIdx.x, C = s.channels();
    for (uint32_t c = threadIdx.x; c < C; c += 256) s.ring[(size_t)((a.pos0 + t) % s.taps) * C + c] = a.y[(size_t)t * a.ldy + s.channel_at(c)];
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

// gated, normed read-outs of a batch as activations; LDS: inner + group_sums floats.  z: [row][ldz]
template <class T>
__global__ __launch_bounds__(256) void ssm_gate_kernel(GroupInput g, uint32_t ldz, T *__restrict__ act, uint32_t ld)
{
    extern __shared__ float gs[];
    const size_t row = blockIdx.x;
    g.o += row * g.n;
    g.z += row * ldz;
    group_input(g, gs + g.n, [&](uint32_t i, float v) { gs[i] = v; }, [&](uint32_t i) { return gs[i]; });
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < ld; i += 256) act[row * ld + i] = float_to_elem<T>(i < g.n ? gs[i] : 0.f);
}

}  // namespace lv
