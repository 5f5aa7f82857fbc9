// Device code of the experts that prompts and decoding share: the router of one row, and products of one vector.
#pragma once
#include "rows.h"

namespace lmhip {

// One wave: softmax over all E <= 1024 experts, the `top` largest scores in order (of equals the lower index), not
// renormalised.  A lane holds experts lane, lane + 64, ...
__device__ __forceinline__ void route_row(const float *z, int E, int top, int lane, int *out_idx, float *out_w)
{
    float v[16], mx = -3.0e38f;
#pragma unroll
    for (int i = 0; i < 16; i++) {
        const int e = lane + 64 * i;
        v[i] = e < E ? z[e] : -3.0e38f;
        mx = fmaxf(mx, v[i]);
    }
    mx = wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < 16; i++) {
        const bool in = lane + 64 * i < E;
        v[i] = in ? expf(v[i] - mx) : -1.f;
        sum += in ? v[i] : 0.f;
    }
    sum = wave_sum(sum);
    for (int s = 0; s < top; s++) {
        float best = -2.f;
        int idx = 0x7fffffff;
#pragma unroll
        for (int i = 0; i < 16; i++) if (v[i] > best) { best = v[i]; idx = lane + 64 * i; }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ob = __shfl_xor(best, o, WAVE);
            const int oi = __shfl_xor(idx, o, WAVE);
            if (ob > best || (ob == best && oi < idx)) { best = ob; idx = oi; }
        }
        if (lane == 0) { out_idx[s] = min(idx, E - 1); out_w[s] = best / sum; }   // (scores that are not numbers choose the last)
#pragma unroll
        for (int i = 0; i < 16; i++) if (lane + 64 * i == idx) v[i] = -1.f;
    }
}

template <typename WT> struct Vec8;
template <> struct Vec8<half_t> {
    static __device__ __forceinline__ void load(const half_t *p, float (&w)[8])
    {
        const half8 v = *reinterpret_cast<const half8 *>(p);
#pragma unroll
        for (int e = 0; e < 8; e++) w[e] = (float)v[e];
    }
};
template <> struct Vec8<float> {
    static __device__ __forceinline__ void load(const float *p, float (&w)[8])
    {
        const float4 a = *reinterpret_cast<const float4 *>(p), b = *reinterpret_cast<const float4 *>(p + 4);
        w[0] = a.x; w[1] = a.y; w[2] = a.z; w[3] = a.w; w[4] = b.x; w[5] = b.y; w[6] = b.z; w[7] = b.w;
    }
};

// lane's part of W[row] . x over `cols` (a multiple of 8)
template <typename WT>
__device__ __forceinline__ float dot_part(const WT *w, const float *x, int cols, int lane)
{
    float s = 0.f;
    for (int c = lane * 8; c < cols; c += 512) {
        float wv[8];
        Vec8<WT>::load(w + c, wv);
        const float4 x0 = *reinterpret_cast<const float4 *>(x + c), x1 = *reinterpret_cast<const float4 *>(x + c + 4);
        s = fmaf(wv[0], x0.x, s); s = fmaf(wv[1], x0.y, s); s = fmaf(wv[2], x0.z, s); s = fmaf(wv[3], x0.w, s);
        s = fmaf(wv[4], x1.x, s); s = fmaf(wv[5], x1.y, s); s = fmaf(wv[6], x1.z, s); s = fmaf(wv[7], x1.w, s);
    }
    return s;
}

}  // namespace lmhip
