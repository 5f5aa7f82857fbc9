// Device code of the delta rule that prompts and decoding share.
#pragma once
#include "stack.h"
#include "rows.h"

namespace lmhip {

// Channel ch (q | k | v order) of the convolution at row m: the inputs of this step from the product, older ones from
// the state's ring (the input of position p lies at p % taps), zeros before position 0.
__device__ __forceinline__ float conv_at(const DeltaRows &a, int m, int ch, int in_col)
{
    const int b = m / a.r.T, t = m % a.r.T, C = 2 * a.KV * a.dim + a.H * a.vdim;
    const float *f = a.filters + (size_t)ch * a.taps;
    float s = 0.f;
    for (int i = 0; i < a.taps; i++) {
        const int tt = t - (a.taps - 1) + i, p = a.r.pos + tt;
        if (p < 0) continue;
        const float x = tt >= 0 ? a.cin[(size_t)(b * a.r.T + tt) * a.ldc + in_col] : a.conv[((size_t)b * a.taps + p % a.taps) * C + ch];
        s = fmaf(x, f[i], s);
    }
    return s;
}

}  // namespace lmhip
