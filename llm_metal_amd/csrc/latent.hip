// Latent attention: what is cached per token is one latent row and one rotated key part, shared by all heads.  The key
// projection is moved to the query (q_u . W_uk c = (W_uk^T q_u) . c) and the value projection behind the weighted sum,
// so a key row is read once for several heads and never expanded.  Scores, weights and sums are fp32.
#include "stack.h"
#include "rows.h"
#include <algorithm>

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

constexpr int HG = 4;        // heads that share the reading of a key row
constexpr int SLK = 64;      // keys per workgroup

__global__ __launch_bounds__(256) void k_rope_interleaved(float2 *tab, int n, int pairs, int dims, double base)
{
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const double angle = (double)(i / pairs) * pow(base, -2.0 * (double)(i % pairs) / (double)dims);
    tab[i] = make_float2((float)cos(angle), (float)sin(angle));
}

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

// grid (rows): the row's latent and key part into the ring
__global__ __launch_bounds__(256) void k_latent_cache(LatentRows a)
{
    __shared__ float sm[16];
    const int m = blockIdx.x, b = m / a.r.T, p = a.r.pos + m % a.r.T, tid = threadIdx.x;
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

// grid (H, rows): the query moved into the latent space, and its rotated part behind it
template <typename WT>
__global__ __launch_bounds__(256) void k_latent_query(LatentRows a, int m0)
{
    extern __shared__ float qs[];                         // [dim]
    const int h = blockIdx.x, m = m0 + blockIdx.y, p = a.r.pos + m % a.r.T, tid = threadIdx.x;
    const int rp = rank_pad(a), w = row_width(a);
    const float *q = a.cin + (size_t)m * a.ldc + a.o_q + h * (a.dim + a.rot);
    for (int i = tid; i < a.dim; i += 256) qs[i] = q[i];
    __syncthreads();
    float *out = a.q + ((size_t)m * a.H + h) * w;
    const WT *uk = (const WT *)a.ukv + (size_t)h * a.dim * a.ldu;
    for (int c = tid; c < rp; c += 256) {                 // the weight's padding columns are zero
        float s = 0.f;
        for (int d = 0; d < a.dim; d++) s = fmaf((float)uk[(size_t)d * a.ldu + c], qs[d], s);
        out[c] = s;
    }
    const float2 *cs = a.rope + (size_t)p * (a.rot_dims / 2);
    for (int i = tid; i < w - rp; i += 256) out[rp + i] = i < a.rot ? rotated(q + a.dim, i, a.rot_dims, cs) : 0.f;
}

// grid (slices, ceil(H / HG), rows): softmax statistics and weighted latent sum of HG heads over one slice of the
// row's visible keys.  LDS: queries [HG][w], scores [HG][SLK], partial sums [parts][HG][rp]
__global__ __launch_bounds__(256) void k_latent_attend(LatentRows a, int m0, int nsplit)
{
    extern __shared__ float lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int rp = rank_pad(a), w = row_width(a);
    float *qs = lds, *sc = qs + HG * w, *red = sc + HG * SLK;
    const int m = m0 + blockIdx.z, b = m / a.r.T, p = a.r.pos + m % a.r.T, h0 = blockIdx.y * HG;
    const int first = max(0, p - a.window + 1), j0 = first + blockIdx.x * SLK, nj = min(SLK, p - j0 + 1);
    const size_t slot0 = ((size_t)(m - m0) * a.H + h0) * nsplit + blockIdx.x;
    if (nj <= 0) {
        if (tid < HG && h0 + tid < a.H) { float *ml = a.part_ml + (slot0 + (size_t)tid * nsplit) * 2; ml[0] = -3.0e38f; ml[1] = 0.f; }
        return;
    }
    for (int i = tid; i < HG * w; i += 256) qs[i] = a.q[((size_t)m * a.H + min(h0 + i / w, a.H - 1)) * w + i % w];
    __syncthreads();
    const float *ring = a.ring + (size_t)b * a.ring_rows * w;
    // scores: sixteen lanes per key
    for (int jj = tid >> 4; jj < SLK; jj += 16) {
        if (jj >= nj) break;                              // uniform over the sixteen lanes of the key
        const float *key = ring + (size_t)((j0 + jj) % a.ring_rows) * w;
        float s[HG] = {};
        for (int c = (tid & 15) * 4; c < w; c += 64) {
            const float4 k = *reinterpret_cast<const float4 *>(key + c);
#pragma unroll
            for (int u = 0; u < HG; u++) {
                const float4 q = *reinterpret_cast<const float4 *>(qs + u * w + c);
                s[u] = fmaf(q.x, k.x, s[u]); s[u] = fmaf(q.y, k.y, s[u]); s[u] = fmaf(q.z, k.z, s[u]); s[u] = fmaf(q.w, k.w, s[u]);
            }
        }
#pragma unroll
        for (int u = 0; u < HG; u++) {
            const float t = group_sum<16>(s[u]);
            if ((tid & 15) == 0) sc[u * SLK + jj] = t * a.scale;
        }
    }
    __syncthreads();
    if (wave < HG) {                                      // one wave per head
        const float s = lane < nj ? sc[wave * SLK + lane] : -3.0e38f, mx = wave_max(s), e = lane < nj ? expf(s - mx) : 0.f, l = wave_sum(e);
        sc[wave * SLK + lane] = e;
        if (lane == 0 && h0 + wave < a.H) { float *ml = a.part_ml + (slot0 + (size_t)wave * nsplit) * 2; ml[0] = mx; ml[1] = l; }
    }
    __syncthreads();
    const int nc = rp / 4, parts = max(1, 256 / nc), part = tid / nc, c = (tid % nc) * 4;
    if (part < parts) {
        float4 o[HG];
#pragma unroll
        for (int u = 0; u < HG; u++) o[u] = make_float4(0.f, 0.f, 0.f, 0.f);
        for (int jj = part; jj < nj; jj += parts) {
            const float4 v = *reinterpret_cast<const float4 *>(ring + (size_t)((j0 + jj) % a.ring_rows) * w + c);
#pragma unroll
            for (int u = 0; u < HG; u++) {
                const float e = sc[u * SLK + jj];
                o[u].x = fmaf(e, v.x, o[u].x); o[u].y = fmaf(e, v.y, o[u].y); o[u].z = fmaf(e, v.z, o[u].z); o[u].w = fmaf(e, v.w, o[u].w);
            }
        }
#pragma unroll
        for (int u = 0; u < HG; u++) *reinterpret_cast<float4 *>(red + ((size_t)part * HG + u) * rp + c) = o[u];
    }
    __syncthreads();
    for (int i = tid; i < HG * rp; i += 256) {
        const int u = i / rp;
        if (h0 + u >= a.H) break;
        float s = 0.f;
        for (int q = 0; q < parts; q++) s += red[(size_t)q * HG * rp + i];
        a.part_o[(slot0 + (size_t)u * nsplit) * rp + i % rp] = s;
    }
}

// grid (H, rows): the slices of one head merged, then the value projection
template <typename WT>
__global__ __launch_bounds__(256) void k_latent_values(LatentRows a, int m0, int nsplit)
{
    extern __shared__ float ctx[];                        // [rp]
    const int h = blockIdx.x, m = m0 + blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, rp = rank_pad(a);
    const size_t slot0 = ((size_t)(m - m0) * a.H + h) * nsplit;
    const float *ml = a.part_ml + slot0 * 2;
    float mx = -3.0e38f, l = 0.f;
    for (int s = 0; s < nsplit; s++) mx = fmaxf(mx, ml[2 * s]);
    for (int s = 0; s < nsplit; s++) l = fmaf(ml[2 * s + 1], expf(ml[2 * s] - mx), l);
    for (int c = tid; c < rp; c += 256) {
        float o = 0.f;
        for (int s = 0; s < nsplit; s++)
            if (ml[2 * s + 1] > 0.f) o = fmaf(a.part_o[(slot0 + s) * rp + c], expf(ml[2 * s] - mx), o);
        ctx[c] = o / l;
    }
    __syncthreads();
    for (int i = wave; i < a.vdim; i += 4) {
        const WT *uv = (const WT *)a.ukv + ((size_t)a.H * a.dim + (size_t)h * a.vdim + i) * a.ldu;
        float s = 0.f;
        for (int c = lane; c < rp; c += 64) s = fmaf((float)uv[c], ctx[c], s);
        s = wave_sum(s);
        if (lane == 0) a.o[((size_t)m * a.H + h) * a.vdim + i] = s;
    }
}

int slices_of(const LatentRows &a) { return (std::min(a.window, a.r.pos + a.r.T) + SLK - 1) / SLK; }
int rows_per_launch(const LatentRows &a)
{
    const size_t per_row = (size_t)a.H * slices_of(a) * (size_t)pad8(a.rank);
    return (int)std::max<size_t>(1, std::min<size_t>((size_t)a.r.n(), ((size_t)32 << 20) / per_row));
}

}  // namespace

void launch_rope_interleaved(float2 *tab, int max_seq, int dims, double base)
{
    const int n = max_seq * (dims / 2);
    if (n > 0) LAUNCH(k_rope_interleaved, dim3((n + 255) / 256), dim3(256), 0, tab, n, dims / 2, dims, base);
}

void launch_latent_cache(const LatentRows &a) { LAUNCH(k_latent_cache, dim3(a.r.n()), dim3(256), 0, a); }

void launch_latent_attend(const LatentRows &in)
{
    LatentRows a = in;
    const int nsplit = slices_of(a), step = rows_per_launch(a), rp = pad8(a.rank), w = rp + pad8(a.rot);
    const size_t po = (size_t)step * a.H * nsplit * rp, pml = (size_t)step * a.H * nsplit * 2;
    a.part_o = (float *)scratch(SCR_PARTIAL, (po + pml) * sizeof(float));
    a.part_ml = a.part_o + po;
    const int parts = std::max(1, 256 / (rp / 4));
    const size_t lds = ((size_t)HG * w + (size_t)HG * SLK + (size_t)parts * HG * rp) * sizeof(float);
    for (int m0 = 0; m0 < a.r.n(); m0 += step) {
        const int nr = std::min(step, a.r.n() - m0);
        if (a.f32) LAUNCH(k_latent_query<float>, dim3(a.H, nr), dim3(256), (size_t)a.dim * 4, a, m0);
        else LAUNCH(k_latent_query<half_t>, dim3(a.H, nr), dim3(256), (size_t)a.dim * 4, a, m0);
        LAUNCH(k_latent_attend, dim3(nsplit, (a.H + HG - 1) / HG, nr), dim3(256), lds, a, m0, nsplit);
        if (a.f32) LAUNCH(k_latent_values<float>, dim3(a.H, nr), dim3(256), (size_t)rp * 4, a, m0, nsplit);
        else LAUNCH(k_latent_values<half_t>, dim3(a.H, nr), dim3(256), (size_t)rp * 4, a, m0, nsplit);
    }
}

}  // namespace lmhip
