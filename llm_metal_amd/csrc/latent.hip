// Latent attention: what is cached per token is one latent row and one rotated key part, shared by all heads.  The key
// projection is moved to the query (q_u . W_uk c = (W_uk^T q_u) . c) and the value projection behind the weighted sum,
// so a key row is read once for several heads and never expanded.  Scores, weights and sums are fp32.
#include "stack.h"
#include "latent_rows.h"
#include <algorithm>

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

constexpr int HG = 4;        // heads that share the reading of a key row

// grid (rows)
__global__ __launch_bounds__(256) void k_latent_cache(LatentRows a)
{
    __shared__ float sm[16];
    latent_cache_row(a, blockIdx.x, sm);
}

// grid (H, rows)
template <typename WT>
__global__ __launch_bounds__(256) void k_latent_query(LatentRows a, int m0)
{
    extern __shared__ float lds[];
    latent_query_row<WT>(a, m0 + blockIdx.y, blockIdx.x, lds);
}

// SLK (up to 64): keys per workgroup.  grid (slices, ceil(H / HG), rows): softmax statistics and weighted latent sum of HG heads over one slice of the
// row's visible keys.  LDS: queries [HG][w], scores [HG][SLK], partial sums [parts][HG][rp]
template <int SLK>
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
    const int slot_j0 = j0 % a.ring_rows;                 // row of key j0; the slice wraps at most once
    auto key_row = [&](int jj) __attribute__((always_inline)) {
        const int r = slot_j0 + jj;
        return ring + (size_t)(r >= a.ring_rows ? r - a.ring_rows : r) * w;
    };
    // scores: sixteen lanes per key
    for (int jj = tid >> 4; jj < SLK; jj += 16) {
        if (jj >= nj) break;                              // uniform over the sixteen lanes of the key
        const float *key = key_row(jj);
        float s[HG] = {};
#pragma unroll 4
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
        if (lane < SLK) sc[wave * SLK + lane] = e;
        if (lane == 0 && h0 + wave < a.H) { float *ml = a.part_ml + (slot0 + (size_t)wave * nsplit) * 2; ml[0] = mx; ml[1] = l; }
    }
    __syncthreads();
    const int nc = rp / 4, parts = max(1, 256 / nc), part = tid / nc, c = (tid % nc) * 4;
    if (part < parts) {
        float4 o[HG];
#pragma unroll
        for (int u = 0; u < HG; u++) o[u] = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
        for (int jj = part; jj < nj; jj += parts) {
            const float4 v = *reinterpret_cast<const float4 *>(key_row(jj) + c);
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

// grid (H, rows, ceil(vdim / VR)): the slices of one head merged, then VR rows of the value projection
constexpr int VR = 16;
template <typename WT>
__global__ __launch_bounds__(256) void k_latent_values(LatentRows a, int m0, int nsplit)
{
    extern __shared__ float ctx[];                        // [rp], the slices' factors [nsplit], sums [shares][rp]
    const int h = blockIdx.x, m = m0 + blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, rp = rank_pad(a);
    float *fac = ctx + rp;
    const size_t slot0 = ((size_t)(m - m0) * a.H + h) * nsplit;
    const float *ml = a.part_ml + slot0 * 2;
    float mx = -3.0e38f;
    for (int s = lane; s < nsplit; s += 64) mx = fmaxf(mx, ml[2 * s]);
    mx = wave_max(mx);
    float l = 0.f;
    for (int s = lane; s < nsplit; s += 64) l += ml[2 * s + 1] > 0.f ? ml[2 * s + 1] * expf(ml[2 * s] - mx) : 0.f;
    l = wave_total(l);
    for (int s = tid; s < nsplit; s += 256) fac[s] = ml[2 * s + 1] > 0.f ? expf(ml[2 * s] - mx) / l : 0.f;
    __syncthreads();
    // four columns of a share of the slices per thread (a slice without keys holds nothing that counts)
    float *red = fac + ((nsplit + 3) & ~3);
    const int nc = rp / 4, shares = max(1, min(8, 256 / nc)), part = tid / nc, c = (tid % nc) * 4;
    if (part < shares) {
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
        for (int s = part; s < nsplit; s += shares) {
            const float f = fac[s];
            const float4 v = *reinterpret_cast<const float4 *>(a.part_o + (slot0 + s) * rp + c);
            if (f > 0.f) { o.x = fmaf(v.x, f, o.x); o.y = fmaf(v.y, f, o.y); o.z = fmaf(v.z, f, o.z); o.w = fmaf(v.w, f, o.w); }
        }
        *reinterpret_cast<float4 *>(red + part * rp + c) = o;
    }
    __syncthreads();
    for (int i = tid; i < rp; i += 256) {
        float o = 0.f;
        for (int k = 0; k < shares; k++) o += red[k * rp + i];
        ctx[i] = o;
    }
    __syncthreads();
    const int i0 = blockIdx.z * VR + wave * (VR / 4);
    const WT *uv[VR / 4];
    float y[VR / 4] = {};
#pragma unroll
    for (int k = 0; k < VR / 4; k++) uv[k] = (const WT *)a.ukv + ((size_t)a.H * a.dim + (size_t)h * a.vdim + min(i0 + k, a.vdim - 1)) * a.ldu;
    dot_rows<VR / 4, 1>(uv, ctx, rp, lane, y);
#pragma unroll
    for (int k = 0; k < VR / 4; k++) {
        const float t = wave_total(y[k]);
        if (lane == 0 && i0 + k < a.vdim) a.o[((size_t)m * a.H + h) * a.vdim + i0 + k] = t;
    }
}

}  // namespace

void launch_latent_cache(const LatentRows &a) { LAUNCH(k_latent_cache, dim3(a.r.n()), dim3(256), 0, a); }

LatentSlices latent_slices(const LatentRows &a)
{
    LatentSlices s;
    s.keys = a.r.T == 1 ? 32 : 64;                        // decoding: more workgroups on fewer keys each
    s.n = (std::min(a.window, a.r.pos + a.r.T) + s.keys - 1) / s.keys;
    const size_t per_row = (size_t)a.H * s.n * (size_t)pad8(a.rank);
    s.rows = (int)std::max<size_t>(1, std::min<size_t>((size_t)a.r.n(), ((size_t)32 << 20) / per_row));
    return s;
}

// what the slices of `rows` rows leave for the value kernel
void latent_partials(LatentRows &a, const LatentSlices &s)
{
    const size_t po = (size_t)s.rows * a.H * s.n * pad8(a.rank), pml = (size_t)s.rows * a.H * s.n * 2;
    a.part_o = (float *)scratch(SCR_PARTIAL, (po + pml) * sizeof(float));
    a.part_ml = a.part_o + po;
}

void launch_latent_slices(const LatentRows &a, const LatentSlices &s, int m0, int nr)
{
    const int rp = pad8(a.rank), w = rp + pad8(a.rot), parts = std::max(1, 256 / (rp / 4));
    const size_t lds = ((size_t)HG * w + (size_t)HG * s.keys + (size_t)parts * HG * rp) * sizeof(float);
    const size_t vlds = ((size_t)rp + ((s.n + 3) & ~3) + (size_t)std::max(1, std::min(8, 256 / (rp / 4))) * rp) * sizeof(float);
    const dim3 grid(s.n, (a.H + HG - 1) / HG, nr), vgrid(a.H, nr, (a.vdim + VR - 1) / VR);
    if (s.keys == 32) LAUNCH(k_latent_attend<32>, grid, dim3(256), lds, a, m0, s.n);
    else LAUNCH(k_latent_attend<64>, grid, dim3(256), lds, a, m0, s.n);
    if (a.f32) LAUNCH(k_latent_values<float>, vgrid, dim3(256), vlds, a, m0, s.n);
    else LAUNCH(k_latent_values<half_t>, vgrid, dim3(256), vlds, a, m0, s.n);
}

void launch_latent_attend(const LatentRows &in)
{
    LatentRows a = in;
    const LatentSlices s = latent_slices(a);
    latent_partials(a, s);
    for (int m0 = 0; m0 < a.r.n(); m0 += s.rows) {
        const int nr = std::min(s.rows, a.r.n() - m0);
        const size_t qlds = latent_query_lds(a);
        if (a.f32) LAUNCH(k_latent_query<float>, dim3(a.H, nr), dim3(256), qlds, a, m0);
        else LAUNCH(k_latent_query<half_t>, dim3(a.H, nr), dim3(256), qlds, a, m0);
        launch_latent_slices(a, s, m0, nr);
    }
}

}  // namespace lmhip
