// Device code of grouped attention that prompts and decoding share.
#pragma once
#include "stack.h"

namespace lmhip {

// element i of a projected head part x (bias b): entries i and i + dims / 2 of the first `dims` turn together, the rest passes
__device__ __forceinline__ float rotated_half(const float *x, const float *b, int i, int dims, const float2 *cs)
{
    const float v = x[i] + b[i];
    if (i >= dims) return v;
    const int n = dims >> 1, o = i < n ? i + n : i - n;
    const float w = x[o] + b[o];
    const float2 c = cs[i < n ? i : o];
    return i < n ? v * c.x - w * c.y : v * c.x + w * c.y;
}

__device__ __forceinline__ const float2 *group_angles(const GroupRows &a, int p) { return a.rope + (size_t)p * (a.rot_dims >> 1); }

// entry i of key head g's rotated key (value) of row m at position p; zero in the padding
__device__ __forceinline__ float group_key(const GroupRows &a, int m, int p, int g, int i)
{
    const int at = a.o_k + g * a.dim;
    return i < a.dim ? rotated_half(a.cin + (size_t)m * a.ldc + at, a.bias + at, i, a.rot_dims, group_angles(a, p)) : 0.f;
}
__device__ __forceinline__ float group_value(const GroupRows &a, int m, int g, int i)
{
    const int at = a.o_v + g * a.vdim + i;
    return i < a.vdim ? a.cin[(size_t)m * a.ldc + at] + a.bias[at] : 0.f;
}

}  // namespace lmhip
