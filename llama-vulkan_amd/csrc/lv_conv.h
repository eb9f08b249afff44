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

}  // namespace lv
