// lv_bf16_gemm.h — matrix products of models whose weights are bfloat16: out[token][row] = sum_k x[token][k] * W[row][k].
//
// Two kernels with one set of epilogues:
//   gemm_bf16_kernel  bf16 activations, v_mfma_f32_16x16x32_bf16 (32-bit accumulation): the serving precision
//   gemm_f32_kernel   fp32 activations, v_mfma_f32_16x16x4_f32 on weights widened to fp32: true 32-bit products
// Both can be grouped (mixture of experts): a table of token tiles says which expert's rows a tile takes and which
// positions of the expert-sorted token list it covers.
//
// Weights are row-major [rows][kp], kp a multiple of 64 (zero columns), rows padded with zero rows to a multiple of 128 (a tile may read the rows behind those as well).
// In the MFMA a weight tile is operand A (M = weight row) and the tokens are operand B (N = token): lane l of the result
// holds token l % 16 and four consecutive weight rows 4 * (l / 16) .. + 3, i.e. one 16-byte store into the token's row.
//
// gemm_bf16_kernel<NW>: NW waves of 64 x 64 each, tile 32 NW weight rows x 128 tokens, K step 64.  Both operand tiles go to LDS
// by direct loads: two stages and two workgroups a CU with four waves, three stages and one workgroup with eight (fewer bytes
// into LDS per product, loads two steps ahead; for launches that fill the chip with it).  A row of a tile is 128 bytes; its
// eight 16-byte chunks are stored in the order chunk ^ (row % 8), so that the 16 rows an MFMA operand reads at one k spread over
// all banks.
#pragma once

#include "../../include/llava_hip.h"
#include "lv_device.h"

namespace lv {

typedef __bf16 lv_bf8 __attribute__((ext_vector_type(8)));
typedef float lv_f4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) void lv_lds_any;
typedef const __attribute__((address_space(1))) void lv_glb_any;

__device__ __forceinline__ float bf16_to_float(uint16_t h) { return __uint_as_float((uint32_t)h << 16); }
__device__ __forceinline__ uint16_t float_to_bf16(float f) { return __builtin_bit_cast(uint16_t, (__bf16)f); }   // round to nearest even
// activations and cache rows come in two element types: uint16_t (bf16 bits) and float
__device__ __forceinline__ float elem_to_float(uint16_t v) { return bf16_to_float(v); }
__device__ __forceinline__ float elem_to_float(float v) { return v; }
template <class T> __device__ __forceinline__ T float_to_elem(float f)
{
    if constexpr (sizeof(T) == 2) return float_to_bf16(f);
    else return f;
}
// eight consecutive elements (16-byte aligned) as floats
__device__ __forceinline__ void load8(float (&f)[8], const uint16_t *p)
{
    const uint4 v = *reinterpret_cast<const uint4 *>(p);
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int i = 0; i < 4; i++) {
        f[2 * i] = __uint_as_float(w[i] << 16);
        f[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
}
__device__ __forceinline__ void load8(float (&f)[8], const float *p)
{
    const float4 a = reinterpret_cast<const float4 *>(p)[0], b = reinterpret_cast<const float4 *>(p)[1];
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}

// fp32 to within a few units in the last place, in few instructions: decode kernels run once per launch, and every line of
// their code is fetched on the way
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.f + __expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }
// log(1 + e^z) to a few units in the last place also where it is small (a slow decay multiplies over thousands of tokens):
// max(z, 0) + log(1 + x) with x = e^-|z| <= 1, log(1 + x) = 2 artanh(t), t = x / (2 + x) <= 1/3, as its power series
__device__ __forceinline__ float softplus_f(float z)
{
    const float x = __expf(-fabsf(z)), t = x * __builtin_amdgcn_rcpf(2.f + x), tt = t * t;
    float p = 1.f / 15.f;
    p = fmaf(p, tt, 1.f / 13.f);
    p = fmaf(p, tt, 1.f / 11.f);
    p = fmaf(p, tt, 1.f / 9.f);
    p = fmaf(p, tt, 1.f / 7.f);
    p = fmaf(p, tt, 1.f / 5.f);
    p = fmaf(p, tt, 1.f / 3.f);
    p = fmaf(p, tt, 1.f);
    return fmaf(2.f * t, p, fmaxf(z, 0.f));
}
// tanh to a few units in the last place of its value, small arguments included: near 0 the odd power series (the first term left
// out is below 6e-8 of the value at 0.3), elsewhere 1 - 2 / (e^2|z| + 1)
__device__ __forceinline__ float tanh_f(float z)
{
    const float a = fabsf(z), q = z * z;
    float p = fmaf(q, 62.f / 2835.f, -17.f / 315.f);
    p = fmaf(p, q, 2.f / 15.f);
    p = fmaf(p, q, -1.f / 3.f);
    const float small = fmaf(a * q, p, a), large = fmaf(-2.f, __builtin_amdgcn_rcpf(__expf(2.f * a) + 1.f), 1.f);
    return __builtin_copysignf(a < 0.3f ? small : large, z);
}
// activation of a gated feed-forward, LV_ACT_*
__device__ __forceinline__ float glu_f(uint32_t act, float z) { return act == LV_ACT_RELU ? fmaxf(z, 0.f) : silu_f(z); }
// decay of one key channel: exp(-exp(A_log) softplus(z)), ea = exp(A_log)
__device__ __forceinline__ float decay_f(float ea, float z) { return __expf(-ea * softplus_f(z)); }

enum BfEpilogue {
    kEpStore = 0,    // out[token][row]
    kEpDecay = 1,    // out[token][head][lane-padded channel] = exp(-exp(A_log[head]) * softplus(v + bias[row]))
    kEpSigmoid = 2,  // out[token][row] = sigmoid(v)
    kEpGlu = 3,      // rows alternate 16 gate, 16 up: act[position][f] = silu(w g) * (w u), w = the expert's weight for the token
    kEpScatter = 4,  // grouped: out[slots[position]][row]
    kEpDense = 5,    // rows as for kEpGlu, one expert: act[token][f] = activation(g) * u
    kEpHeads = 6,    // activations instead of fp32, heads padded: act[token][head * head_stride + channel], row = head * head_dim + channel
};

struct BfGemmArgs {
    const void *x;           // activations (bf16 or fp32), rows readable up to the next multiple of the token tile
    const uint16_t *w;
    uint32_t ldx, kp;        // row stride of x in elements; padded K
    uint32_t rows;           // weight rows that exist
    uint32_t n;              // tokens (ungrouped)
    uint32_t row_tiles, token_tiles;
    float *out;
    uint32_t ldo;
    // K cut in slices (kEpStore): grid z = slice, its sum goes to out + slice * slice_floats; the reader adds them up
    uint32_t k_slice;        // columns per slice, a multiple of the K step; 0: one slice
    uint64_t slice_floats;
    // decay and head epilogues
    const float *a_log, *bias;
    uint32_t head_dim, head_stride;
    // grouped
    const uint32_t *tiles;   // [0] = number of tiles, then {expert, first position, positions} each
    const uint32_t *slots;   // position in expert order -> token * top + choice
    const float *weights;    // [token * top + choice]
    uint32_t top, expert_rows;   // weight rows from one expert to the next
    bool gather;             // x rows are tokens (slots[position] / top), otherwise positions
    void *act;               // kEpGlu, kEpDense, kEpHeads output [position][lda]
    uint32_t lda;
    uint32_t activation;     // kEpDense: LV_ACT_*
};

// four results of one token: weight rows row .. row + 3
template <int EP>
__device__ __forceinline__ void bf_store4(const BfGemmArgs &a, uint32_t orow, uint32_t row, const lv_f4 v)
{
    if (row >= a.rows) return;
    float r[4] = {v[0], v[1], v[2], v[3]};
    if constexpr (EP == kEpDecay) {
        if (a.head_dim % 4 == 0) {      // the four rows belong to one head
            const uint32_t h = row / a.head_dim, d = row - h * a.head_dim;
            const float ea = __expf(a.a_log[h]);
            const float4 b = *reinterpret_cast<const float4 *>(a.bias + row);
            *reinterpret_cast<float4 *>(a.out + (size_t)orow * a.ldo + h * a.head_stride + d) =
                make_float4(decay_f(ea, r[0] + b.x), decay_f(ea, r[1] + b.y), decay_f(ea, r[2] + b.z), decay_f(ea, r[3] + b.w));
            return;
        }
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (row + i < a.rows) {
                const uint32_t h = (row + i) / a.head_dim, d = (row + i) % a.head_dim;
                a.out[(size_t)orow * a.ldo + h * a.head_stride + d] = decay_f(__expf(a.a_log[h]), r[i] + a.bias[row + i]);
            }
        return;
    }
    if constexpr (EP == kEpSigmoid) {
#pragma unroll
        for (int i = 0; i < 4; i++) r[i] = sigmoid_f(r[i]);
    }
    float *o = a.out + (EP == kEpStore && a.k_slice ? blockIdx.z * a.slice_floats : 0) + (size_t)orow * a.ldo + row;
    if (row + 3 < a.rows && (a.ldo & 3) == 0) {
        *reinterpret_cast<float4 *>(o) = make_float4(r[0], r[1], r[2], r[3]);
    } else {
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (row + i < a.rows) o[i] = r[i];
    }
}

// four results of one token, rows row .. row + 3, into padded heads
template <class T>
__device__ __forceinline__ void bf_store_heads(const BfGemmArgs &a, uint32_t token, uint32_t row, const lv_f4 v)
{
    if (row >= a.rows) return;
    T *o = static_cast<T *>(a.act) + (size_t)token * a.lda;
    if (a.head_dim % 4 == 0) {
        const uint32_t h = row / a.head_dim;
        o += (size_t)h * a.head_stride + (row - h * a.head_dim);
        if constexpr (sizeof(T) == 2)
            *reinterpret_cast<uint2 *>(o) = make_uint2((uint32_t)float_to_bf16(v[0]) | ((uint32_t)float_to_bf16(v[1]) << 16),
                                                       (uint32_t)float_to_bf16(v[2]) | ((uint32_t)float_to_bf16(v[3]) << 16));
        else *reinterpret_cast<float4 *>(o) = make_float4(v[0], v[1], v[2], v[3]);
        return;
    }
#pragma unroll
    for (int i = 0; i < 4; i++)
        if (row + i < a.rows) o[(size_t)((row + i) / a.head_dim) * a.head_stride + (row + i) % a.head_dim] = float_to_elem<T>(v[i]);
}

template <class T>
__device__ __forceinline__ void bf_store_dense(const BfGemmArgs &a, uint32_t token, uint32_t f, const lv_f4 g, const lv_f4 u)
{
    T *o = static_cast<T *>(a.act) + (size_t)token * a.lda + f;
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = glu_f(a.activation, g[i]) * u[i];
    if constexpr (sizeof(T) == 2)
        *reinterpret_cast<uint2 *>(o) = make_uint2((uint32_t)float_to_bf16(v[0]) | ((uint32_t)float_to_bf16(v[1]) << 16),
                                                   (uint32_t)float_to_bf16(v[2]) | ((uint32_t)float_to_bf16(v[3]) << 16));
    else *reinterpret_cast<float4 *>(o) = make_float4(v[0], v[1], v[2], v[3]);
}

template <class T>
__device__ __forceinline__ void bf_store_glu(const BfGemmArgs &a, uint32_t position, uint32_t f, float wt, const lv_f4 g, const lv_f4 u)
{
    T *o = static_cast<T *>(a.act) + (size_t)position * a.lda + f;
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = silu_f(wt * g[i]) * (wt * u[i]);
    if constexpr (sizeof(T) == 2)
        *reinterpret_cast<uint2 *>(o) = make_uint2((uint32_t)float_to_bf16(v[0]) | ((uint32_t)float_to_bf16(v[1]) << 16),
                                                   (uint32_t)float_to_bf16(v[2]) | ((uint32_t)float_to_bf16(v[3]) << 16));
    else *reinterpret_cast<float4 *>(o) = make_float4(v[0], v[1], v[2], v[3]);
}

// Tile of this workgroup: workgroups are dealt to the 8 XCDs in turn; an XCD takes every eighth row tile and walks the token
// tiles of one row tile before the next, so that the weight tile is read into its L2 once.
template <bool GROUPED>
__device__ __forceinline__ bool bf_tile(const BfGemmArgs &a, uint32_t tile_tokens, uint32_t &rt, uint32_t &expert, uint32_t &first, uint32_t &count)
{
    const uint32_t pid = blockIdx.x, q = pid >> 3;
    rt = q / a.token_tiles * 8 + (pid & 7);
    const uint32_t tt = q % a.token_tiles;
    if (rt >= a.row_tiles) return false;
    if constexpr (GROUPED) {
        if (tt >= a.tiles[0]) return false;
        expert = a.tiles[1 + 3 * tt];
        first = a.tiles[2 + 3 * tt];
        count = a.tiles[3 + 3 * tt];
    } else {
        expert = 0;
        first = tt * tile_tokens;
        count = min(tile_tokens, a.n - first);
    }
    return true;
}
inline uint32_t bf_grid(const BfGemmArgs &a) { return (a.row_tiles + 7) / 8 * 8 * a.token_tiles; }

constexpr int kBfTile = 128;       // tokens per workgroup, bf16
constexpr int kBfStep = 64;
constexpr int bf_tile_rows(int nw) { return 32 * nw; }
constexpr int bf_stages(int nw) { return nw == 4 ? 2 : 3; }
constexpr int bf_stage_bytes(int nw) { return (bf_tile_rows(nw) + kBfTile) * kBfStep * 2; }
constexpr int bf_lds_bytes(int nw) { return bf_stages(nw) * bf_stage_bytes(nw); }

template <int EP, bool GROUPED, int NW>
__global__ __launch_bounds__(NW * 64, 2) void gemm_bf16_kernel(BfGemmArgs a)
{
    constexpr int RM = bf_tile_rows(NW), NST = bf_stages(NW), STAGE = bf_stage_bytes(NW);
    constexpr int LW = RM / NW / 8, LX = kBfTile / NW / 8, LPS = LW + LX;      // direct loads per wave and stage, 8 rows (1 KB) each
    extern __shared__ __attribute__((aligned(128))) uint8_t bf_lds[];
    uint32_t rt, expert, first, count;
    if (!bf_tile<GROUPED>(a, kBfTile, rt, expert, first, count)) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int l16 = lane & 15, g4 = lane >> 4;
    const uint32_t kp = a.kp;

    const uint16_t *gw, *gx[LX];
    {
        const int r8 = lane >> 3, c = (lane & 7) ^ r8;
        gw = a.w + ((size_t)expert * a.expert_rows + (size_t)rt * RM + wave * (RM / NW) + r8) * kp + c * 8;
#pragma unroll
        for (int i = 0; i < LX; i++) {
            const int row = wave * (kBfTile / NW) + i * 8 + r8;
            size_t xr = (size_t)first + row;
            if constexpr (GROUPED) {
                const uint32_t p = first + min((uint32_t)row, count - 1);
                xr = a.gather ? a.slots[p] / a.top : p;
            }
            gx[i] = static_cast<const uint16_t *>(a.x) + xr * a.ldx + c * 8;
        }
    }
    const uint32_t k_lo = EP == kEpStore && a.k_slice ? blockIdx.z * a.k_slice : 0;
    const uint32_t steps = (EP == kEpStore && a.k_slice ? min(a.k_slice, kp - k_lo) : kp) / kBfStep;
    // past the end a harmless repeat of the last step into a free buffer keeps the number of loads in flight the same
    auto issue = [&](uint32_t s, uint32_t slot) {
        uint8_t *buf = bf_lds + slot * STAGE;
        const uint32_t k0 = k_lo + min(s, steps - 1) * kBfStep;
#pragma unroll
        for (int i = 0; i < LW; i++)
            __builtin_amdgcn_global_load_lds((lv_glb_any *)(gw + (size_t)i * 8 * kp + k0), (lv_lds_any *)(buf + (wave * LW + i) * 1024), 16, 0, 0);
#pragma unroll
        for (int i = 0; i < LX; i++) __builtin_amdgcn_global_load_lds((lv_glb_any *)(gx[i] + k0), (lv_lds_any *)(buf + RM * 128 + (wave * LX + i) * 1024), 16, 0, 0);
    };

    const int wm = wave % (NW / 2), wn = wave / (NW / 2);
    lv_f4 acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) acc[i][j] = lv_f4{0.f, 0.f, 0.f, 0.f};

#pragma unroll
    for (int s = 0; s < NST - 1; s++) issue(s, s);
    uint32_t slot = 0, ahead = NST - 1;
    for (uint32_t s = 0; s < steps; s++) {
        // this wave's loads of stage s have landed; behind the barrier everyone's have, and everyone is done with stage s - 1
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"((NST - 2) * LPS) : "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        issue(s + NST - 1, ahead);
        const uint8_t *bw = bf_lds + slot * STAGE, *bx = bw + RM * 128;
#pragma unroll
        for (int kk = 0; kk < 2; kk++) {
            lv_bf8 fa[4], fb[4];
            const int ch = ((kk * 4 + g4) ^ (l16 & 7)) * 16;
#pragma unroll
            for (int i = 0; i < 4; i++) fa[i] = *reinterpret_cast<const lv_bf8 *>(bw + (wm * 64 + i * 16 + l16) * 128 + ch);
#pragma unroll
            for (int i = 0; i < 4; i++) fb[i] = *reinterpret_cast<const lv_bf8 *>(bx + (wn * 64 + i * 16 + l16) * 128 + ch);
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int j = 0; j < 4; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
        }
        slot = slot + 1 == NST ? 0 : slot + 1;
        ahead = ahead + 1 == NST ? 0 : ahead + 1;
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");      // the repeats have landed before the workgroup gives up its LDS
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const uint32_t t = wn * 64 + j * 16 + l16;
        if (t >= count) continue;
        const uint32_t p = first + t;
        if constexpr (EP == kEpGlu) {
            const float wt = a.weights[a.slots[p]];
#pragma unroll
            for (int i = 0; i < 4; i += 2) {
                const uint32_t row = rt * RM + wm * 64 + i * 16;        // the pair's gate block
                if (row < a.rows) bf_store_glu<uint16_t>(a, p, row / 2 + g4 * 4, wt, acc[i][j], acc[i + 1][j]);
            }
        } else if constexpr (EP == kEpDense) {
#pragma unroll
            for (int i = 0; i < 4; i += 2) {
                const uint32_t row = rt * RM + wm * 64 + i * 16;
                if (row < a.rows) bf_store_dense<uint16_t>(a, p, row / 2 + g4 * 4, acc[i][j], acc[i + 1][j]);
            }
        } else if constexpr (EP == kEpHeads) {
#pragma unroll
            for (int i = 0; i < 4; i++) bf_store_heads<uint16_t>(a, p, rt * RM + wm * 64 + i * 16 + g4 * 4, acc[i][j]);
        } else {
            const uint32_t orow = EP == kEpScatter ? a.slots[p] : p;
#pragma unroll
            for (int i = 0; i < 4; i++) bf_store4<EP>(a, orow, rt * RM + wm * 64 + i * 16 + g4 * 4, acc[i][j]);
        }
    }
}

constexpr int kF32Tile = 64;
constexpr int kF32Step = 32;
constexpr int kF32Ld = kF32Step + 4;

template <int EP, bool GROUPED>
__global__ __launch_bounds__(256) void gemm_f32_kernel(BfGemmArgs a)
{
    __shared__ __attribute__((aligned(16))) float ws[kF32Tile * kF32Ld], xs[kF32Tile * kF32Ld];
    uint32_t rt, expert, first, count;
    if (!bf_tile<GROUPED>(a, kF32Tile, rt, expert, first, count)) return;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, g4 = lane >> 4;
    const int wm = wave & 1, wn = wave >> 1;
    const uint32_t kp = a.kp;
    const int lr = threadIdx.x >> 2, lc = (threadIdx.x & 3) * 8;     // this thread's row and 8 columns of the tiles it loads
    const uint16_t *gw = a.w + ((size_t)expert * a.expert_rows + (size_t)rt * kF32Tile + lr) * kp + lc;
    size_t xr = (size_t)first + lr;
    if constexpr (GROUPED) {
        const uint32_t p = first + min((uint32_t)lr, count - 1);
        xr = a.gather ? a.slots[p] / a.top : p;
    }
    const float *gx = static_cast<const float *>(a.x) + xr * a.ldx + lc;
    lv_f4 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++) acc[i][j] = lv_f4{0.f, 0.f, 0.f, 0.f};
    for (uint32_t k0 = 0; k0 < kp; k0 += kF32Step) {
        float fw[8], fx[8];
        load8(fw, gw + k0);
        load8(fx, gx + k0);
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 8; i += 4) {
            *reinterpret_cast<float4 *>(ws + lr * kF32Ld + lc + i) = make_float4(fw[i], fw[i + 1], fw[i + 2], fw[i + 3]);
            *reinterpret_cast<float4 *>(xs + lr * kF32Ld + lc + i) = make_float4(fx[i], fx[i + 1], fx[i + 2], fx[i + 3]);
        }
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < kF32Step / 4; kk++) {
            float fa[2], fb[2];
#pragma unroll
            for (int i = 0; i < 2; i++) {
                fa[i] = ws[(wm * 32 + i * 16 + l16) * kF32Ld + kk * 4 + g4];
                fb[i] = xs[(wn * 32 + i * 16 + l16) * kF32Ld + kk * 4 + g4];
            }
#pragma unroll
            for (int i = 0; i < 2; i++)
#pragma unroll
                for (int j = 0; j < 2; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(fa[i], fb[j], acc[i][j], 0, 0, 0);
        }
    }
#pragma unroll
    for (int j = 0; j < 2; j++) {
        const uint32_t t = wn * 32 + j * 16 + l16;
        if (t >= count) continue;
        const uint32_t p = first + t;
        if constexpr (EP == kEpGlu) {
            bf_store_glu<float>(a, p, (rt * kF32Tile + wm * 32) / 2 + g4 * 4, a.weights[a.slots[p]], acc[0][j], acc[1][j]);
        } else if constexpr (EP == kEpDense) {
            bf_store_dense<float>(a, p, (rt * kF32Tile + wm * 32) / 2 + g4 * 4, acc[0][j], acc[1][j]);
        } else if constexpr (EP == kEpHeads) {
#pragma unroll
            for (int i = 0; i < 2; i++) bf_store_heads<float>(a, p, rt * kF32Tile + wm * 32 + i * 16 + g4 * 4, acc[i][j]);
        } else {
            const uint32_t orow = EP == kEpScatter ? a.slots[p] : p;
#pragma unroll
            for (int i = 0; i < 2; i++) bf_store4<EP>(a, orow, rt * kF32Tile + wm * 32 + i * 16 + g4 * 4, acc[i][j]);
        }
    }
}

}  // namespace lv
