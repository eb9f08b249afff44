// lv_streams.h — a residual of several streams (hyper-connections) and the norms in front of its sublayers.
//
//   u   = sum_t in[t] x_t;   h = norm(u);   y = sublayer(h);   x_t <- sum_f mix[f][t] x_f + out[t] y
//
// y stays pending until the next launch that needs an input: that one forms the new streams, the next sublayer's u and its norm
// in one go, so the streams are read and written once per sublayer.  The norm is tanh(alpha u) w + b, element by element, or an
// RMS norm.  Streams are fp32, [stream][dp], zero from dim to dp.
#pragma once

#include "lv_bf16_gemm.h"

namespace lv {

constexpr uint32_t kMaxStreams = 8;

// coefficients of one sublayer, padded to kMaxStreams
struct StreamCoef {
    float in[kMaxStreams], out[kMaxStreams], mix[kMaxStreams * kMaxStreams];      // mix[from * kMaxStreams + to]
};

struct StreamInput {
    const float *x;              // [stream][dp]
    float *x_out;                // the new streams, null: not wanted
    const float *y;              // pending sublayer output, null: none
    const StreamCoef *spread;    // of the pending sublayer
    const StreamCoef *gather;    // of the next one
    const float *w, *b, *alpha;  // norm; alpha null: RMS norm
    float *h_out;                // null: not wanted
    uint32_t dim, dp, streams;
    float eps;
};

// elements i .. i + 3 of the streams and of the pending output.  NS: streams there is room for
template <int NS>
struct StreamQuad {
    float4 x[NS], y;

    __device__ __forceinline__ void load(const StreamInput &a, uint32_t i)
    {
#pragma unroll
        for (int t = 0; t < NS; t++)
            if (t < (int)a.streams) x[t] = *reinterpret_cast<const float4 *>(a.x + (size_t)t * a.dp + i);
        y = a.y ? *reinterpret_cast<const float4 *>(a.y + i) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    // takes in the pending output and returns u
    __device__ __forceinline__ float4 gather(const StreamInput &a, uint32_t i, bool store) const
    {
        float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int t = 0; t < NS; t++) {
            if (t >= (int)a.streams) break;
            float4 v = x[t];
            if (a.y) {
                const float o = a.spread->out[t];
                v = make_float4(o * y.x, o * y.y, o * y.z, o * y.w);
#pragma unroll
                for (int f = 0; f < NS; f++) {
                    if (f >= (int)a.streams) break;
                    const float c = a.spread->mix[f * kMaxStreams + t];
                    v.x = fmaf(c, x[f].x, v.x); v.y = fmaf(c, x[f].y, v.y); v.z = fmaf(c, x[f].z, v.z); v.w = fmaf(c, x[f].w, v.w);
                }
                if (store && a.x_out) *reinterpret_cast<float4 *>(a.x_out + (size_t)t * a.dp + i) = v;
            }
            const float g = a.gather->in[t];
            u.x = fmaf(g, v.x, u.x); u.y = fmaf(g, v.y, u.y); u.z = fmaf(g, v.z, u.z); u.w = fmaf(g, v.w, u.w);
        }
        return u;
    }
};

// u of all elements, four at a time: use(i, u).  The next four are on their way meanwhile.
template <int NS, class Use>
__device__ __forceinline__ void stream_each(const StreamInput &a, bool store, Use use)
{
    const uint32_t step = blockDim.x * 4;
    uint32_t i = threadIdx.x * 4;
    if (i >= a.dp) return;
    StreamQuad<NS> next;
    next.load(a, i);
#pragma unroll 1
    do {
        const StreamQuad<NS> q = next;
        const uint32_t at = i;
        i += step;
        if (i < a.dp) next.load(a, i);
        use(at, q.gather(a, at, store));
    } while (i < a.dp);
}

// The whole input: put(i, h) gets four elements at a time, get(i) returns what put left there.  scratch: a float per wave.
template <int NS, class Put, class Get>
__device__ __forceinline__ void stream_input(const StreamInput &a, bool lead, float *scratch, Put put, Get get)
{
    if (a.alpha) {
        const float al = *a.alpha;
        stream_each<NS>(a, lead, [&](uint32_t i, const float4 u) {
            const float4 w = *reinterpret_cast<const float4 *>(a.w + i), b = *reinterpret_cast<const float4 *>(a.b + i);
            const float4 h = make_float4(fmaf(tanh_f(al * u.x), w.x, b.x), fmaf(tanh_f(al * u.y), w.y, b.y), fmaf(tanh_f(al * u.z), w.z, b.z), fmaf(tanh_f(al * u.w), w.w, b.w));
            put(i, h);
            if (lead && a.h_out) *reinterpret_cast<float4 *>(a.h_out + i) = h;
        });
        return;
    }
    float s = 0.f;
    stream_each<NS>(a, lead, [&](uint32_t i, const float4 u) {
        s = fmaf(u.x, u.x, s); s = fmaf(u.y, u.y, s); s = fmaf(u.z, u.z, s); s = fmaf(u.w, u.w, s);
        put(i, u);
    });
    const float inv = rsqrtf(block_sum_waves(s, scratch, blockDim.x >> 6) / (float)a.dim + a.eps);
    for (uint32_t i = threadIdx.x * 4; i < a.dp; i += blockDim.x * 4) {
        const float4 u = get(i), w = *reinterpret_cast<const float4 *>(a.w + i);
        const float4 h = make_float4(u.x * inv * w.x, u.y * inv * w.y, u.z * inv * w.z, u.w * inv * w.w);
        put(i, h);
        if (lead && a.h_out) *reinterpret_cast<float4 *>(a.h_out + i) = h;
    }
}

// A batch: one workgroup per row.  x: [row][stream][dp], y: [row][dp] or, with several vectors per row to be added up,
// [row][parts][dp].
struct StreamRowsArgs {
    StreamInput in;
    uint32_t parts;
    void *act;                   // [row][dp], null: only the streams are wanted
};
template <class T, int NS>
__global__ __launch_bounds__(256) void stream_rows_kernel(StreamRowsArgs a)
{
    extern __shared__ float us[];      // dp floats, and dp more where parts are added up
    __shared__ float scratch[4];
    StreamInput in = a.in;
    const size_t row = blockIdx.x;
    in.x += row * in.streams * in.dp;
    if (in.x_out) in.x_out += row * in.streams * in.dp;
    if (in.y) {
        in.y += row * a.parts * in.dp;
        if (a.parts > 1) {
            float *sum = us + in.dp;
            for (uint32_t i = threadIdx.x * 4; i < in.dp; i += 1024) {
                float4 v = *reinterpret_cast<const float4 *>(in.y + i);
                for (uint32_t p = 1; p < a.parts; p++) {
                    const float4 u = *reinterpret_cast<const float4 *>(in.y + (size_t)p * in.dp + i);
                    v.x += u.x; v.y += u.y; v.z += u.z; v.w += u.w;
                }
                *reinterpret_cast<float4 *>(sum + i) = v;      // every thread reads its own elements again
            }
            in.y = sum;
        }
    }
    if (!a.act) {
        stream_each<NS>(in, true, [](uint32_t, const float4) {});
        return;
    }
    T *act = static_cast<T *>(a.act) + row * in.dp;
    auto store = [&](uint32_t i, const float4 h) {
        if constexpr (sizeof(T) == 2)
            *reinterpret_cast<uint2 *>(act + i) = make_uint2((uint32_t)float_to_bf16(h.x) | ((uint32_t)float_to_bf16(h.y) << 16),
                                                             (uint32_t)float_to_bf16(h.z) | ((uint32_t)float_to_bf16(h.w) << 16));
        else *reinterpret_cast<float4 *>(act + i) = h;
    };
    if (in.alpha) {
        stream_input<NS>(in, true, scratch, store, [](uint32_t) { return make_float4(0.f, 0.f, 0.f, 0.f); });
    } else {
        stream_input<NS>(in, true, scratch, [&](uint32_t i, const float4 h) { *reinterpret_cast<float4 *>(us + i) = h; },
                         [&](uint32_t i) { return *reinterpret_cast<const float4 *>(us + i); });
        for (uint32_t i = threadIdx.x * 4; i < in.dp; i += 1024) store(i, *reinterpret_cast<const float4 *>(us + i));
    }
}

// sum of the streams, for record mode: rows of `stride` floats
__global__ __launch_bounds__(256) void stream_sum_kernel(float *__restrict__ out, uint32_t stride, const float *__restrict__ x, uint32_t streams, uint32_t dim, uint32_t dp)
{
    const uint32_t i = blockIdx.x * 256 + threadIdx.x;
    const size_t row = blockIdx.y;
    if (i >= dim) return;
    float v = 0.f;
    for (uint32_t t = 0; t < streams; t++) v += x[(row * streams + t) * dp + i];
    out[row * stride + i] = v;
}

}  // namespace lv
