// Device code of latent attention that prompts and decoding share: one row's cache entry and one head's absorbed query.
#pragma once
#include "stack.h"
#include "expert.h"

namespace lmhip {

// element i of a rotated vector: pairs (2p, 2p + 1) of the first `dims` turn, the rest passes
__device__ __forceinline__ float rotated(const float *x, int i, int dims, const float2 *cs)
{
    if (i >= dims) return x[i];
    const float2 c = cs[i >> 1];
    return (i & 1) ? x[i] * c.x + x[i - 1] * c.y : x[i] * c.x - x[i + 1] * c.y;
}

// widths of a ring row / an absorbed query: latent part and rotated part, each padded to 8 with zeros
__device__ __forceinline__ int rank_pad(const LatentRows &a) { return (a.rank + 7) & ~7; }
__device__ __forceinline__ int row_width(const LatentRows &a) { return rank_pad(a) + ((a.rot + 7) & ~7); }

// One workgroup of 256: row m's latent and key part into the ring.  sm: 16 floats
__device__ __forceinline__ void latent_cache_row(const LatentRows &a, int m, float *sm)
{
    const int b = m / a.r.T, p = a.r.pos + m % a.r.T, tid = threadIdx.x;
    const int rp = rank_pad(a), w = row_width(a);
    const float *c = a.cin + (size_t)m * a.ldc + a.o_dkv, *k = c + a.rank;
    float *dst = a.ring + ((size_t)b * a.ring_rows + p % a.ring_rows) * w;
    const float2 *cs = a.rope + (size_t)p * (a.rot_dims / 2);
    float ss = 0.f;
    for (int i = tid; i < a.rank; i += 256) ss += c[i] * c[i];
    const float inv = 1.f / sqrtf(block_sum(ss, sm) / (float)a.rank + a.eps);
    for (int i = tid; i < w; i += 256)
        dst[i] = i < rp ? (i < a.rank ? c[i] * inv * a.g_c[i] : 0.f) : (i - rp < a.rot ? rotated(k, i - rp, a.rot_dims, cs) : 0.f);
}

// One workgroup of 256: head h's query of row m moved into the latent space, W_uk^T q_u, and its rotated part behind it.
// A thread takes eight latent columns of a share of the head's dimensions.  lds: dim + shares * rp floats
// (latent_query_lds)
inline __host__ __device__ int latent_query_shares(int rp) { const int n = 256 / (rp / 8); return n < 1 ? 1 : n > 8 ? 8 : n; }
template <typename WT>
__device__ __forceinline__ void latent_query_row(const LatentRows &a, int m, int h, float *lds)
{
    const int p = a.r.pos + m % a.r.T, tid = threadIdx.x, rp = rank_pad(a), w = row_width(a), nc = rp / 8;
    const int shares = latent_query_shares(rp), part = tid / nc, c = (tid % nc) * 8;
    float *qs = lds, *red = lds + ((a.dim + 3) & ~3);
    const float *q = a.cin + (size_t)m * a.ldc + a.o_q + h * (a.dim + a.rot);
    for (int i = tid; i < a.dim; i += 256) qs[i] = q[i];
    __syncthreads();
    float *out = a.q + ((size_t)m * a.H + h) * w;
    if (part < shares) {
        const WT *uk = (const WT *)a.ukv + (size_t)h * a.dim * a.ldu + c;
        float s[8] = {};
#pragma unroll 8
        for (int d = part; d < a.dim; d += shares) {
            float wv[8];
            Vec8<WT>::load(uk + (size_t)d * a.ldu, wv);
#pragma unroll
            for (int e = 0; e < 8; e++) s[e] = fmaf(wv[e], qs[d], s[e]);
        }
#pragma unroll
        for (int e = 0; e < 8; e++) red[part * rp + c + e] = s[e];
    }
    __syncthreads();
    for (int i = tid; i < rp; i += 256) {                 // the weight's padding columns are zero
        float s = 0.f;
        for (int k = 0; k < shares; k++) s += red[k * rp + i];
        out[i] = s;
    }
    const float2 *cs = a.rope + (size_t)p * (a.rot_dims / 2);
    for (int i = tid; i < w - rp; i += 256) out[rp + i] = i < a.rot ? rotated(q + a.dim, i, a.rot_dims, cs) : 0.f;
}
inline size_t latent_query_lds(const LatentRows &a)
{
    const int rp = pad8(a.rank);
    return ((size_t)((a.dim + 3) & ~3) + (size_t)latent_query_shares(rp) * rp) * sizeof(float);
}

}  // namespace lmhip
