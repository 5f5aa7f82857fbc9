// Mixture of experts: softmax router with the largest scores chosen, squared-ReLU experts.
#include "stack.h"
#include "rows.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

// One wave per row: softmax over all experts, the `top` largest scores in order (of equals the lower index), not
// renormalised.  A lane holds experts lane, lane + 64, ...
__global__ __launch_bounds__(256) void k_route(MoeRows a)
{
    const int m = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (m >= a.rows) return;
    const float *z = a.z + (size_t)m * a.ldz;
    float v[16], mx = -3.0e38f;
#pragma unroll
    for (int i = 0; i < 16; i++) {
        const int e = lane + 64 * i;
        v[i] = e < a.E ? z[e] : -3.0e38f;
        mx = fmaxf(mx, v[i]);
    }
    mx = wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < 16; i++) {
        const bool in = lane + 64 * i < a.E;
        v[i] = in ? expf(v[i] - mx) : -1.f;
        sum += in ? v[i] : 0.f;
    }
    sum = wave_sum(sum);
    for (int s = 0; s < a.top; s++) {
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
        if (lane == 0) { a.idx[(size_t)m * a.top + s] = idx; a.w[(size_t)m * a.top + s] = best / sum; }
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

// act[m][s][i] = relu(up_e[i] . h[m])^2 for the s-th chosen expert e of row m; a wave per i.  grid (ceil(ffp / 4), top, rows)
template <typename WT>
__global__ __launch_bounds__(256) void k_expert_up(MoeRows a)
{
    const int lane = threadIdx.x & 63, i = blockIdx.x * 4 + (threadIdx.x >> 6), s = blockIdx.y, m = blockIdx.z;
    if (i >= a.ffp) return;
    const size_t slot = (size_t)m * a.top + s;
    float v = 0.f;
    if (i < a.ff) v = wave_sum(dot_part((const WT *)a.up + ((size_t)a.idx[slot] * a.ff + i) * a.Dp, a.h + (size_t)m * a.Dp, a.Dp, lane));
    if (lane == 0) a.act[slot * a.ffp + i] = relu2(v);   // the padding is written too: zero
}

// y[m][d] = sum over the chosen experts of w * (down_e[d] . act); a wave per d.  grid (ceil(Dp / 4), rows)
template <typename WT>
__global__ __launch_bounds__(256) void k_expert_down(MoeRows a)
{
    const int lane = threadIdx.x & 63, d = blockIdx.x * 4 + (threadIdx.x >> 6), m = blockIdx.y;
    if (d >= a.Dp) return;
    float y = 0.f;
    if (d < a.D)
        for (int s = 0; s < a.top; s++) {
            const size_t slot = (size_t)m * a.top + s;
            y = fmaf(a.w[slot], dot_part((const WT *)a.down + ((size_t)a.idx[slot] * a.D + d) * a.ffp, a.act + slot * a.ffp, a.ffp, lane), y);
        }
    y = wave_sum(y);
    if (lane == 0) a.y[(size_t)m * a.Dp + d] = y;
}

}  // namespace

void launch_route(const MoeRows &a) { LAUNCH(k_route, dim3((a.rows + 3) / 4), dim3(256), 0, a); }

void launch_experts_per_row(const MoeRows &a)
{
    const dim3 up((a.ffp + 3) / 4, a.top, a.rows), down((a.Dp + 3) / 4, a.rows);
    if (a.f32) { LAUNCH(k_expert_up<float>, up, dim3(256), 0, a); LAUNCH(k_expert_down<float>, down, dim3(256), 0, a); }
    else { LAUNCH(k_expert_up<half_t>, up, dim3(256), 0, a); LAUNCH(k_expert_down<half_t>, down, dim3(256), 0, a); }
}

}  // namespace lmhip
