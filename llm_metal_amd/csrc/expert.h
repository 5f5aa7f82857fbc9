// Device code of the experts that prompts and decoding share: the router of one row, and products of one vector.
#pragma once
#include "rows.h"

namespace lmhip {

// One wave: softmax over all E experts, the `top` largest scores in order (of equals the lower index), not renormalised.
// A lane holds experts lane, lane + 64, ... (NI of them).
template <int NI>
__device__ __forceinline__ void route_experts(const float *z, int E, int top, int lane, int *out_idx, float *out_w)
{
    float v[NI], mx = -3.0e38f;
#pragma unroll
    for (int i = 0; i < NI; i++) {
        const int e = lane + 64 * i;
        v[i] = e < E ? z[e] : -3.0e38f;
        mx = fmaxf(mx, v[i]);
    }
    mx = wave_peak(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NI; i++) {
        const bool in = lane + 64 * i < E;
        v[i] = in ? expf(v[i] - mx) : -1.f;
        sum += in ? v[i] : 0.f;
    }
    sum = wave_total(sum);
    for (int s = 0; s < top; s++) {
        float best = v[0];
#pragma unroll
        for (int i = 1; i < NI; i++) best = fmaxf(best, v[i]);
        best = wave_peak(best);
        int idx = E - 1;                                  // (what scores that are not numbers choose)
#pragma unroll
        for (int i = NI - 1; i >= 0; i--) {
            const unsigned long long has = __ballot(v[i] == best);
            if (has) idx = 64 * i + __ffsll(has) - 1;
        }
        idx = min(idx, E - 1);
        if (lane == 0) { out_idx[s] = idx; out_w[s] = best / sum; }
#pragma unroll
        for (int i = 0; i < NI; i++) if (lane + 64 * i == idx) v[i] = -1.f;
    }
}
// E <= 1024
__device__ __forceinline__ void route_row(const float *z, int E, int top, int lane, int *out_idx, float *out_w)
{
    if (E <= 64) route_experts<1>(z, E, top, lane, out_idx, out_w);
    else if (E <= 256) route_experts<4>(z, E, top, lane, out_idx, out_w);
    else route_experts<16>(z, E, top, lane, out_idx, out_w);
}

template <typename WT> struct Vec8;
// eight consecutive weights of a row as fp32
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

// eight products of a piece added to s
__device__ __forceinline__ float dot8(const float (&w)[8], const float *x, float s)
{
    const float4 a = *reinterpret_cast<const float4 *>(x), b = *reinterpret_cast<const float4 *>(x + 4);
    s = fmaf(w[0], a.x, s); s = fmaf(w[1], a.y, s); s = fmaf(w[2], a.z, s); s = fmaf(w[3], a.w, s);
    s = fmaf(w[4], b.x, s); s = fmaf(w[5], b.y, s); s = fmaf(w[6], b.z, s); s = fmaf(w[7], b.w, s);
    return s;
}

// lane's part of N rows . x over `cols` (a multiple of 8), added to s[]; U pieces of every row in flight.  The loads past
// the end of a row ask for its last piece again and count nothing.
template <int N, int U, typename WT>
__device__ __forceinline__ void dot_rows(const WT *const (&w)[N], const float *x, int cols, int lane, float (&s)[N])
{
    for (int c0 = lane * 8; c0 - lane * 8 < cols; c0 += 512 * U) {
        float wv[N][U][8];
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int n = 0; n < N; n++) Vec8<WT>::load(w[n] + min(c0 + 512 * u, cols - 8), wv[n][u]);
#pragma unroll
        for (int u = 0; u < U; u++)
            if (c0 + 512 * u < cols)
#pragma unroll
                for (int n = 0; n < N; n++) s[n] = dot8(wv[n][u], x + c0 + 512 * u, s[n]);
    }
}
template <typename WT>
__device__ __forceinline__ float dot_part(const WT *w, const float *x, int cols, int lane)
{
    const WT *const rows[1] = {w};
    float s[1] = {0.f};
    dot_rows<1, 4>(rows, x, cols, lane, s);
    return s[0];
}

}  // namespace lmhip
