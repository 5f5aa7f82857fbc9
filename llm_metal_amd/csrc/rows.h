// Device helpers of the kernels that finish one row per workgroup and hand it to a product.
#pragma once
#include "devutil.h"
#include "gemm.h"

namespace lmhip {

// A row held in LDS (`n` floats, n % 8 == 0) as row m of a tiled F16 operand of Kb K blocks, times the power of two
// `s`; columns n .. 64 Kb are zero.  Eight columns of a row are 16 contiguous bytes of the tile.
__device__ __forceinline__ void store_row_f16(const float *row, int n, half_t *a16, int m, int Kb, float s)
{
    for (int k = threadIdx.x * 8; k < Kb * 64; k += blockDim.x * 8) {
        half8 h;
#pragma unroll
        for (int e = 0; e < 8; e++) h[e] = (k < n) ? f2h(row[k + e] * s) : (half_t)0;
        *reinterpret_cast<half8 *>(&a16[tiled_a_index(m, k, Kb)]) = h;
    }
}

// overflow-free ln(1 + e^z)
__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float silu(float z) { return z / (1.f + expf(-z)); }
// tanh form of GELU; the tanh as a quotient of exponentials, or as the library has it
__device__ __forceinline__ float gelu_tanh(float z)
{
    const float in = 0.7978845608f * fmaf(0.044715f * z * z, z, z);
    return z * __builtin_amdgcn_rcpf(1.f + __expf(-2.f * in));
}
__device__ __forceinline__ float gelu_tanh_exact(float z)
{
    return 0.5f * z * (1.f + tanhf(0.79788456080286536f * (z + 0.044715f * z * z * z)));
}
__device__ __forceinline__ float relu2(float z) { const float r = fmaxf(z, 0.f); return r * r; }

// sum over the G lanes of an aligned group (G = 4, 8, 16 or 32), left in every one of them; cross-lane moves ride on
// the additions (DPP) up to 16 lanes
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v)
{
    return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
// v of this lane plus v of the lane 16 (32) away: the swaps exchange the rows of sixteen (halves) of two registers, here
// two copies of v
__device__ __forceinline__ float swap16_add(float v)
{
    const auto t = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return __uint_as_float(t[0]) + __uint_as_float(t[1]);
}
__device__ __forceinline__ float swap32_add(float v)
{
    const auto t = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return __uint_as_float(t[0]) + __uint_as_float(t[1]);
}
template <int G>
__device__ __forceinline__ float group_sum(float v)
{
    v = dpp_add<0xB1>(v);                                 // quad lanes 1 0 3 2
    v = dpp_add<0x4E>(v);                                 // quad lanes 2 3 0 1
    if (G >= 8) v = dpp_add<0x141>(v);                    // mirror of eight lanes
    if (G >= 16) v = dpp_add<0x140>(v);                   // mirror of sixteen lanes
    if (G >= 32) v = swap16_add(v);
    return v;
}

// sum over the wave, left in every lane
__device__ __forceinline__ float wave_total(float v)
{
    return swap32_add(group_sum<32>(v));
}

// largest over the wave, left in every lane
template <int CTRL>
__device__ __forceinline__ float dpp_max(float v)
{
    return fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true)));
}
__device__ __forceinline__ float wave_peak(float v)
{
    v = dpp_max<0xB1>(v); v = dpp_max<0x4E>(v); v = dpp_max<0x141>(v); v = dpp_max<0x140>(v);
    const auto t = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = fmaxf(__uint_as_float(t[0]), __uint_as_float(t[1]));
    const auto u = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return fmaxf(__uint_as_float(u[0]), __uint_as_float(u[1]));
}

}  // namespace lmhip
