// lv_conv.h — short causal convolutions with silu in front of a recurrence, over a token's projection row, the rows of the batch
// before it, and a ring of the last `taps` inputs of a sequence ([position % taps][channel]).
//
// A recurrence's description (Spec) provides: taps, conv ([taps][channels], last row = the current token), ring, channels(),
// channel_at(c) = where channel c lies in a projection row, conv_bias(c).
#pragma once

#include "lv_bf16_gemv.h"

namespace lv {

// Convolution and silu of channel c at position pos (slot = pos % taps).  y: the token's projection row; rows before it (in
// steps of ld floats) belong to positions pos - 1, pos - 2, .. as far as `behind` of them, older inputs are in the ring.
// fetch() requests the first four taps, which is usually all there are; value() does the rest.
struct ShortConv {
    float x[4], w[4], b;
    uint32_t at, c;

    template <class Spec>
    static __device__ __forceinline__ float input(const Spec &s, const float *y, size_t ld, uint32_t behind, uint32_t at, uint32_t c, uint32_t slot, uint32_t j)
    {
        return j <= behind ? y[at - (ptrdiff_t)(j * ld)] : s.ring[(size_t)(slot >= j ? slot - j : slot + s.taps - j) * s.channels() + c];
    }
    template <class Spec>
    __device__ __forceinline__ void fetch(const Spec &s, const float *y, size_t ld, uint32_t behind, uint32_t c_, uint32_t pos, uint32_t slot)
    {
        c = c_;
        at = s.channel_at(c);
        b = s.conv_bias(c);
        const float *wp = s.conv + (size_t)(s.taps - 1) * s.channels() + c;
#pragma unroll
        for (uint32_t j = 0; j < 4; j++) {
            const bool ok = j < s.taps && j <= pos;
            x[j] = ok ? input(s, y, ld, behind, at, c, slot, j) : 0.f;
            w[j] = ok ? wp[-(ptrdiff_t)(j * (size_t)s.channels())] : 0.f;
        }
    }
    template <class Spec>
    __device__ __forceinline__ float value(const Spec &s, const float *y, size_t ld, uint32_t behind, uint32_t pos, uint32_t slot) const
    {
        float v = fmaf(x[0], w[0], b);
#pragma unroll
        for (int j = 1; j < 4; j++) v = fmaf(x[j], w[j], v);
        for (uint32_t j = 4; j < s.taps && j <= pos; j++)
            v = fmaf(input(s, y, ld, behind, at, c, slot, j), s.conv[(size_t)(s.taps - 1 - j) * s.channels() + c], v);
        return silu_f(v);
    }
};
template <class Spec>
__device__ __forceinline__ float short_conv(const Spec &s, const float *y, size_t ld, uint32_t behind, uint32_t c, uint32_t pos, uint32_t slot)
{
    ShortConv v;
    v.fetch(s, y, ld, behind, c, pos, slot);
    return v.value(s, y, ld, behind, pos, slot);
}

// Eight consecutive tokens t0 .. t0 + 7 (t0 a multiple of 8) of a batch of n, whose first row is y and first position pos0; 0 for
// tokens past the end.  Up to four taps every input is read once.
template <class Spec>
__device__ __forceinline__ void short_conv8(float (&out)[8], const Spec &s, const float *y, size_t ld, uint32_t c, uint32_t pos0, uint32_t t0, uint32_t n)
{
    if (s.taps > 4) {
#pragma unroll 1
        for (uint32_t i = 0; i < 8; i++) {
            const uint32_t t = t0 + i;
            const float v = t < n ? short_conv(s, y + t * ld, ld, t, c, pos0 + t, (pos0 + t) % s.taps) : 0.f;
#pragma unroll
            for (uint32_t e = 0; e < 8; e++) out[e] = e == i ? v : out[e];
        }
        return;
    }
    const uint32_t at = s.channel_at(c);
    const float b = s.conv_bias(c);
    float in[11], w[4];      // in[i]: token t0 + i - 3
#pragma unroll
    for (uint32_t j = 0; j < 4; j++) w[j] = j < s.taps ? s.conv[(size_t)(s.taps - 1 - j) * s.channels() + c] : 0.f;
#pragma unroll
    for (uint32_t i = 0; i < 11; i++) {
        const uint32_t back = i < 3 ? 3 - i : 0, t = t0 + i - 3;
        in[i] = 0.f;
        if (t0 || !back) {
            if (t < n) in[i] = y[(size_t)t * ld + at];
        } else if (back < s.taps && back <= pos0) {
            in[i] = s.ring[(size_t)((pos0 - back) % s.taps) * s.channels() + c];
        }
    }
#pragma unroll
    for (uint32_t i = 0; i < 8; i++) {
        float v = fmaf(in[i + 3], w[0], b);
#pragma unroll
        for (uint32_t j = 1; j < 4; j++) v = fmaf(in[i + 3 - j], w[j], v);
        out[i] = t0 + i < n ? silu_f(v) : 0.f;
    }
}

}  // namespace lv
