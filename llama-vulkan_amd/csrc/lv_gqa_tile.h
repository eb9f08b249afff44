// lv_gqa_tile.h — grouped-query attention of a batch on the matrix cores (bf16 q, k, v rows; scores, softmax and sums fp32; the
// weights enter the value product as two bf16 pieces, 16 bits of each).
//
// A workgroup (4 waves) takes 64 or 128 queries of one head and walks the keys they can see in tiles of 64, double-buffered in
// LDS by direct loads.  Scores are computed transposed, S^T = K Q^T: a lane then holds 16 scores of ONE query (column l % 16),
// so the running maximum, the rescaling factor and the sum are per-lane scalars, and the registers of S^T are already the
// second operand of O^T = V^T P^T.  For that the values are transposed once per layer (gqa_values_kernel) with the keys of
// every 32 in the order the score registers have: place 8 g + 4 t + r holds key 16 t + 4 g + r.
#pragma once

#include "lv_gqa.h"

namespace lv {

struct GqaTileArgs {
    GqaBatchArgs b;
    uint32_t base;       // position of the first key any query of the batch can see: the start of its first token's chunk
    uint32_t keys;       // keys from there to the batch's last position
    uint32_t vt_ld;      // keys rounded up to 64
    uint16_t *vt;        // [kv head][DP][vt_ld]
};

constexpr int kTileKeys = 64;

// row of position p: the batch's (from own0 on) or the ring's
__device__ __forceinline__ const uint16_t *gqa_row(const GqaTileArgs &a, const void *mine, const void *ring, uint32_t p, uint32_t kvh, uint32_t dp)
{
    const GqaSpec &s = a.b.s;
    return p >= a.b.own0 ? static_cast<const uint16_t *>(mine) + ((size_t)(p - a.b.own0) * s.kv_heads + kvh) * dp
                         : static_cast<const uint16_t *>(ring) + ((size_t)(p - a.base) * s.kv_heads + kvh) * dp;
}

// grid (kv heads, vt_ld / 64): transposes 64 keys' values
template <int DP>
__global__ __launch_bounds__(256) void gqa_values_kernel(GqaTileArgs a)
{
    __shared__ uint16_t t[kTileKeys * (DP + 2)];
    const uint32_t kvh = blockIdx.x, k0 = blockIdx.y * kTileKeys;
    for (int i = threadIdx.x; i < kTileKeys * DP / 8; i += 256) {
        const uint32_t key = i / (DP / 8), d = i % (DP / 8) * 8, kk = k0 + key;
        uint4 v = make_uint4(0, 0, 0, 0);
        if (kk < a.keys) v = *reinterpret_cast<const uint4 *>(gqa_row(a, a.b.v, a.b.s.vc, a.base + kk, kvh, DP) + d);
        uint32_t *o = reinterpret_cast<uint32_t *>(t + key * (DP + 2) + d);
        o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < DP * 8; i += 256) {
        const int d = i / 8, c = i % 8;          // eight places c * 8 .. + 7 of row d
        uint32_t w[4];
#pragma unroll
        for (int e = 0; e < 4; e++) {
            uint32_t h[2];
#pragma unroll
            for (int u = 0; u < 2; u++) {
                const int j = 2 * e + u, key = (c / 4) * 32 + 16 * (j / 4) + 4 * (c % 4) + j % 4;
                h[u] = t[key * (DP + 2) + d];
            }
            w[e] = h[0] | (h[1] << 16);
        }
        *reinterpret_cast<uint4 *>(a.vt + ((size_t)kvh * DP + d) * a.vt_ld + k0 + c * 8) = make_uint4(w[0], w[1], w[2], w[3]);
    }
}

template <int DK, int DV> constexpr int gqa_tile_lds() { return 2 * kTileKeys * (DK + DV) * 2; }

// DK, DV = padded sizes of queries and keys, and of values.  QT = tiles of 16 queries per wave; a workgroup takes 64 * QT queries.  grid (heads, query tiles)
template <int DK, int DV, int QT>
__global__ __launch_bounds__(256) void gqa_tile_kernel(GqaTileArgs a)
{
    constexpr int KS = DK / 32, DT = DV / 16, ROW = DK * 2, STAGE = kTileKeys * (DK + DV) * 2, CH = DK / 8;
    extern __shared__ __attribute__((aligned(128))) uint8_t tile[];
    const GqaSpec &s = a.b.s;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l16 = lane & 15, g4 = lane >> 4;
    const uint32_t head = blockIdx.x, kvh = head / (s.heads / s.kv_heads);
    const uint32_t t0 = (gridDim.y - 1 - blockIdx.y) * 64 * QT;      // the tiles with the most keys start first
    const uint32_t last = min(t0 + 64 * QT, a.b.n) - 1;
    auto chunk_start = [&](uint32_t p) { return gqa_chunk_start(s, p); };

    // this lane's queries: one per 16-query tile
    lv_bf8 q[QT][KS];
    uint32_t lo[QT], hi[QT];     // the keys it sees, as positions
#pragma unroll
    for (int i = 0; i < QT; i++) {
        const uint32_t t = min(t0 + (wave * QT + i) * 16 + l16, a.b.n - 1);
        hi[i] = a.b.pos0 + t;
        lo[i] = chunk_start(hi[i]);
        const uint16_t *qr = static_cast<const uint16_t *>(a.b.q) + ((size_t)t * s.heads + head) * DK + g4 * 8;
#pragma unroll
        for (int k = 0; k < KS; k++) q[i][k] = *reinterpret_cast<const lv_bf8 *>(qr + k * 32);
    }
    const uint32_t wave_first = a.b.pos0 + min(t0 + wave * QT * 16, a.b.n - 1), wave_last = a.b.pos0 + min(t0 + (wave + 1) * QT * 16 - 1, a.b.n - 1);
    const uint32_t wave_lo = chunk_start(wave_first), inner_lo = chunk_start(wave_last);

    const uint32_t k_first = (chunk_start(a.b.pos0 + t0) - a.base) / kTileKeys * kTileKeys, k_end = a.b.pos0 + last - a.base + 1;
    const uint32_t p_max = a.base + a.keys - 1;
    auto issue = [&](int st, uint32_t k0) {
        uint8_t *kb = tile + st * STAGE, *vb = kb + kTileKeys * ROW;
        // 64 rows of DK key elements, then DV rows of 64 values: 1 KB (64 chunks of 16 bytes) per wave and instruction
#pragma unroll
        for (int i = 0; i < kTileKeys * CH / 256; i++) {
            const int c = (i * 4 + wave) * 64 + lane, row = c / CH, ch = c % CH;
            const uint16_t *src = gqa_row(a, a.b.k, s.kc, min(a.base + k0 + row, p_max), kvh, DK) + (ch ^ (row & 7)) * 8;
            __builtin_amdgcn_global_load_lds((lv_glb_any *)src, (lv_lds_any *)(kb + (i * 4 + wave) * 1024), 16, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < DV * 8 / 256; i++) {
            const int c = (i * 4 + wave) * 64 + lane, row = c / 8, ch = c % 8;
            const uint16_t *src = a.vt + ((size_t)kvh * DV + row) * a.vt_ld + k0 + (ch ^ (row & 7)) * 8;
            __builtin_amdgcn_global_load_lds((lv_glb_any *)src, (lv_lds_any *)(vb + (i * 4 + wave) * 1024), 16, 0, 0);
        }
    };

    lv_f4 o[DT][QT];
    float m[QT], l[QT];
    const float sink = s.sink ? s.sink[head] : -1e30f;
#pragma unroll
    for (int i = 0; i < QT; i++) {
        m[i] = sink;
        l[i] = s.sink && g4 == 0 ? 1.f : 0.f;      // the four lanes of a query hold parts of its sum
#pragma unroll
        for (int d = 0; d < DT; d++) o[d][i] = lv_f4{0.f, 0.f, 0.f, 0.f};
    }

    issue(0, k_first);
    int st = 0;
    for (uint32_t k0 = k_first; k0 < k_end; k0 += kTileKeys, st ^= 1) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (k0 + kTileKeys < k_end) issue(st ^ 1, k0 + kTileKeys);
        const uint32_t p0 = a.base + k0, p1 = p0 + kTileKeys - 1;
        if (p0 > wave_last || p1 < wave_lo) continue;      // nothing of this tile is visible to the wave's queries
        const uint8_t *kb = tile + st * STAGE, *vb = kb + kTileKeys * ROW;
        lv_f4 sc[4][QT];
#pragma unroll
        for (int kt = 0; kt < 4; kt++)
#pragma unroll
            for (int i = 0; i < QT; i++) sc[kt][i] = lv_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KS; k++)
#pragma unroll
            for (int kt = 0; kt < 4; kt++) {
                const int row = kt * 16 + l16;
                const lv_bf8 fk = *reinterpret_cast<const lv_bf8 *>(kb + row * ROW + ((k * 4 + g4) ^ (row & 7)) * 16);
#pragma unroll
                for (int i = 0; i < QT; i++) sc[kt][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fk, q[i][k], sc[kt][i], 0, 0, 0);
            }
        const bool edge = p1 > wave_first || p0 < inner_lo;   // some query of the wave does not see all of the tile
        lv_bf8 ph[2][QT], pl[2][QT];
#pragma unroll
        for (int i = 0; i < QT; i++) {
            if (edge) {
#pragma unroll
                for (int kt = 0; kt < 4; kt++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const uint32_t p = p0 + kt * 16 + g4 * 4 + r;
                        if (p < lo[i] || p > hi[i]) sc[kt][i][r] = -INFINITY;
                    }
            }
            float top = m[i];
#pragma unroll
            for (int kt = 0; kt < 4; kt++) top = fmaxf(fmaxf(fmaxf(sc[kt][i][0], sc[kt][i][1]), fmaxf(sc[kt][i][2], sc[kt][i][3])), top);
            top = fmaxf(top, __shfl_xor(top, 16, 64));
            top = fmaxf(top, __shfl_xor(top, 32, 64));
            const float f = __expf(m[i] - top);
            m[i] = top;
            float sum = 0.f;
#pragma unroll
            for (int kt = 0; kt < 4; kt++)
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    const float p = __expf(sc[kt][i][r] - top);
                    sum += p;
                    const __bf16 h = (__bf16)p;
                    ph[kt / 2][i][(kt & 1) * 4 + r] = h;
                    pl[kt / 2][i][(kt & 1) * 4 + r] = (__bf16)(p - (float)h);
                }
            l[i] = fmaf(l[i], f, sum);
#pragma unroll
            for (int d = 0; d < DT; d++)
#pragma unroll
                for (int r = 0; r < 4; r++) o[d][i][r] *= f;
        }
#pragma unroll
        for (int d = 0; d < DT; d++)
#pragma unroll
            for (int kh = 0; kh < 2; kh++) {
                const int row = d * 16 + l16;
                const lv_bf8 fv = *reinterpret_cast<const lv_bf8 *>(vb + row * 128 + ((kh * 4 + g4) ^ (row & 7)) * 16);
#pragma unroll
                for (int i = 0; i < QT; i++) {
                    o[d][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv, pl[kh][i], o[d][i], 0, 0, 0);
                    o[d][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv, ph[kh][i], o[d][i], 0, 0, 0);
                }
            }
    }
#pragma unroll
    for (int i = 0; i < QT; i++) {
        const uint32_t t = t0 + (wave * QT + i) * 16 + l16;
        float sum = l[i];
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        if (t >= a.b.n) continue;
        const float f = a.b.out_scale / sum;
        uint16_t *out = static_cast<uint16_t *>(a.b.out) + (size_t)t * a.b.ldo + head * s.vdim;
#pragma unroll
        for (int d = 0; d < DT; d++) {
            const uint32_t c = d * 16 + g4 * 4;
            uint16_t h[4];
#pragma unroll
            for (int r = 0; r < 4; r++) h[r] = float_to_bf16(o[d][i][r] * f);
            if (c + 3 < s.vdim && (s.vdim & 3) == 0) {
                *reinterpret_cast<uint2 *>(out + c) = make_uint2((uint32_t)h[0] | ((uint32_t)h[1] << 16), (uint32_t)h[2] | ((uint32_t)h[3] << 16));
            } else {
#pragma unroll
                for (int r = 0; r < 4; r++)
                    if (c + r < s.vdim) out[c + r] = h[r];
            }
        }
    }
}

}  // namespace lv
