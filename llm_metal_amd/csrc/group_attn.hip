// Grouped attention inside chunks of positions, fp32: position i sees the positions of its chunk up to itself, a head reads
// the keys and values of its group.  Rotated keys and values lie in rings per sequence and key head; a layer may read the
// rings of an earlier one.  Slices of the visible keys are read once for several heads and merged behind.
#include "group_rows.h"
#include "rows.h"
#include <algorithm>

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

constexpr int HG = 4;        // heads that share the reading of a key row

__device__ __forceinline__ int up4(int n) { return (n + 3) & ~3; }
__device__ __forceinline__ float *key_ring(const GroupRows &a, int b, int g) { return a.kring + (size_t)(b * a.G + g) * a.ring_rows * up4(a.dim); }
__device__ __forceinline__ float *value_ring(const GroupRows &a, int b, int g) { return a.vring + (size_t)(b * a.G + g) * a.ring_rows * up4(a.vdim); }

// a thread per four entries of a row's keys | values of all key heads.  grid (ceil(G * (dp + vp) / 1024), rows); vec: four
// entries lie on 16 bytes and turn with four others, or pass, together
__global__ __launch_bounds__(256) void k_group_cache(GroupRows a, int vec)
{
    const int m = blockIdx.y, b = m / a.r.T, p = a.r.pos + m % a.r.T, slot = p % a.ring_rows;
    const int dp = up4(a.dim), vp = up4(a.vdim), x = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (x >= a.G * (dp + vp)) return;
    const bool key = x < a.G * dp;
    const int y = key ? x : x - a.G * dp, g = y / (key ? dp : vp), i = y % (key ? dp : vp);
    float4 v;
    if (vec) {
        const int at = key ? a.o_k + g * a.dim : a.o_v + g * a.vdim, n = a.rot_dims >> 1;
        const float *c = a.cin + (size_t)m * a.ldc + at, *bias = a.bias + at;
        auto four = [&](int d) __attribute__((always_inline)) {
            const float4 s = *reinterpret_cast<const float4 *>(c + d), t = *reinterpret_cast<const float4 *>(bias + d);
            return make_float4(s.x + t.x, s.y + t.y, s.z + t.z, s.w + t.w);
        };
        v = four(i);
        if (key && i < a.rot_dims) {
            const int o = i < n ? i + n : i - n;
            const float4 w = four(o), *cs = reinterpret_cast<const float4 *>(group_angles(a, p) + (i < n ? i : o)), c0 = cs[0], c1 = cs[1];
            const float s = i < n ? -1.f : 1.f;
            v = make_float4(v.x * c0.x + s * w.x * c0.y, v.y * c0.z + s * w.y * c0.w, v.z * c1.x + s * w.z * c1.y, v.w * c1.z + s * w.w * c1.w);
        }
    } else
#pragma unroll
        for (int e = 0; e < 4; e++) (&v.x)[e] = key ? group_key(a, m, p, g, i + e) : group_value(a, m, g, i + e);
    float *to = key ? key_ring(a, b, g) + (size_t)slot * dp : value_ring(a, b, g) + (size_t)slot * vp;
    *reinterpret_cast<float4 *>(to + i) = v;
}

// SLK (up to 64): keys per workgroup.  grid (slices, G * ceil(H / G / HG), rows): softmax statistics and weighted value sum
// of HG heads over one slice of the row's visible keys.  A single slice finishes its rows.  A step of one token of a layer
// with keys of its own takes the newest key and value from the product, and one workgroup per key head writes the rings.
// LDS: queries [HG][dp], scores [HG][SLK], newest key [dp] and value [vp], partial sums [parts][HG][vp]
template <int SLK>
__global__ __launch_bounds__(256) void k_group_attend(GroupRows a, int m0, int nsplit)
{
    extern __shared__ float lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int dp = up4(a.dim), vp = up4(a.vdim), per = a.H / a.G, blocks = (per + HG - 1) / HG;
    float *qs = lds, *sc = qs + HG * dp, *nk = sc + HG * SLK, *nv = nk + dp, *red = nv + vp;
    const int m = m0 + blockIdx.z, b = m / a.r.T, p = a.r.pos + m % a.r.T, g = blockIdx.y / blocks, part0 = (blockIdx.y % blocks) * HG;
    const int h0 = g * per + part0, nh = min(HG, per - part0);
    const int first = p / a.chunk * a.chunk, j0 = first + blockIdx.x * SLK, nj = min(SLK, p - j0 + 1);
    const size_t slot0 = ((size_t)(m - m0) * a.H + h0) * nsplit + blockIdx.x;
    if (nj <= 0) {                                        // (never the only slice)
        if (tid < nh) { float *ml = a.part_ml + (slot0 + (size_t)tid * nsplit) * 2; ml[0] = -3.0e38f; ml[1] = 0.f; }
        return;
    }
    const bool fresh = a.own && a.r.T == 1 && j0 + nj - 1 == p;
    const int old = fresh ? nj - 1 : nj;                  // keys of the slice that lie in the ring
    float *kr = key_ring(a, b, g), *vr = value_ring(a, b, g);
    for (int i = tid; i < HG * dp; i += 256) {
        const int u = i / dp, d = i % dp, at = a.o_q + (h0 + min(u, nh - 1)) * a.dim;
        qs[i] = d < a.dim ? rotated_half(a.cin + (size_t)m * a.ldc + at, a.bias + at, d, a.rot_dims, group_angles(a, p)) * a.scale : 0.f;
    }
    if (fresh) {
        const bool keep = part0 == 0;
        const int slot = p % a.ring_rows;
        for (int i = tid; i < dp + vp; i += 256) {
            const float v = i < dp ? group_key(a, m, p, g, i) : group_value(a, m, g, i - dp);
            nk[i] = v;                                    // nv lies behind nk
            if (keep) { if (i < dp) kr[(size_t)slot * dp + i] = v; else vr[(size_t)slot * vp + i - dp] = v; }
        }
    }
    __syncthreads();
    const int slot_j0 = j0 % a.ring_rows;                 // row of key j0; the slice wraps at most once
    auto ring_row = [&](int jj) __attribute__((always_inline)) { const int r = slot_j0 + jj; return (size_t)(r >= a.ring_rows ? r - a.ring_rows : r); };
    // scores: sixteen lanes per key
    auto score = [&](const float *key, int jj) __attribute__((always_inline)) {
        float s[HG] = {};
#pragma unroll 4
        for (int c = (tid & 15) * 4; c < dp; c += 64) {
            const float4 k = *reinterpret_cast<const float4 *>(key + c);
#pragma unroll
            for (int u = 0; u < HG; u++) {
                const float4 q = *reinterpret_cast<const float4 *>(qs + u * dp + c);
                s[u] = fmaf(q.x, k.x, s[u]); s[u] = fmaf(q.y, k.y, s[u]); s[u] = fmaf(q.z, k.z, s[u]); s[u] = fmaf(q.w, k.w, s[u]);
            }
        }
#pragma unroll
        for (int u = 0; u < HG; u++) {
            const float t = group_sum<16>(s[u]);
            if ((tid & 15) == 0) sc[u * SLK + jj] = t;
        }
    };
#pragma unroll
    for (int i = 0; i < SLK / 16; i++) {
        const int jj = i * 16 + (tid >> 4);
        if (jj < old) score(kr + ring_row(jj) * dp, jj);  // uniform over the sixteen lanes of the key
    }
    if (fresh && tid < 16) score(nk, nj - 1);
    __syncthreads();
    __shared__ float total[HG];
    if (wave < HG) {                                      // one wave per head
        const float s = lane < nj ? sc[wave * SLK + lane] : -3.0e38f, mx = wave_peak(s), e = lane < nj ? expf(s - mx) : 0.f, l = wave_total(e);
        if (lane < SLK) sc[wave * SLK + lane] = e;
        if (lane == 0) {
            total[wave] = l;
            if (wave < nh && nsplit > 1) { float *ml = a.part_ml + (slot0 + (size_t)wave * nsplit) * 2; ml[0] = mx; ml[1] = l; }
        }
    }
    __syncthreads();
    const int nc = vp / 4, parts = max(1, 256 / nc), part = tid / nc, c = (tid % nc) * 4;
    if (part < parts) {
        float4 o[HG];
#pragma unroll
        for (int u = 0; u < HG; u++) o[u] = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
        for (int jj = part; jj < old; jj += parts) {
            const float4 v = *reinterpret_cast<const float4 *>(vr + ring_row(jj) * vp + c);
#pragma unroll
            for (int u = 0; u < HG; u++) {
                const float e = sc[u * SLK + jj];
                o[u].x = fmaf(e, v.x, o[u].x); o[u].y = fmaf(e, v.y, o[u].y); o[u].z = fmaf(e, v.z, o[u].z); o[u].w = fmaf(e, v.w, o[u].w);
            }
        }
#pragma unroll
        for (int u = 0; u < HG; u++) *reinterpret_cast<float4 *>(red + ((size_t)part * HG + u) * vp + c) = o[u];
    }
    __syncthreads();
    for (int i = tid; i < nh * vp; i += 256) {
        const int u = i / vp, d = i % vp;
        float s = fresh ? sc[u * SLK + nj - 1] * nv[d] : 0.f;
        for (int q = 0; q < parts; q++) s += red[(size_t)q * HG * vp + i];
        if (nsplit > 1) a.part_o[(slot0 + (size_t)u * nsplit) * vp + d] = s;
        else if (d < a.vdim) {
            const int at = (h0 + u) * a.vdim + d;
            s /= total[u];
            a.o[(size_t)m * a.H * a.vdim + at] = a.gated ? s * sigmoid(a.cin[(size_t)m * a.ldc + a.o_g + at]) : s;
        }
    }
}

// grid (H, rows): the slices of one head merged.  LDS: factors [nsplit], sums [shares][vp]
__global__ __launch_bounds__(256) void k_group_merge(GroupRows a, int m0, int nsplit)
{
    extern __shared__ float fac[];
    const int h = blockIdx.x, m = m0 + blockIdx.y, tid = threadIdx.x, lane = tid & 63, vp = up4(a.vdim);
    const size_t slot0 = ((size_t)(m - m0) * a.H + h) * nsplit;
    const float *ml = a.part_ml + slot0 * 2;
    float mx = -3.0e38f;
    for (int s = lane; s < nsplit; s += 64) mx = fmaxf(mx, ml[2 * s]);
    mx = wave_peak(mx);
    float l = 0.f;
    for (int s = lane; s < nsplit; s += 64) l += ml[2 * s + 1] > 0.f ? ml[2 * s + 1] * expf(ml[2 * s] - mx) : 0.f;
    l = wave_total(l);
    for (int s = tid; s < nsplit; s += 256) fac[s] = ml[2 * s + 1] > 0.f ? expf(ml[2 * s] - mx) / l : 0.f;
    __syncthreads();
    float *red = fac + up4(nsplit);
    const int nc = vp / 4, shares = max(1, min(8, 256 / nc)), part = tid / nc, c = (tid % nc) * 4;
    if (part < shares) {
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
        for (int s = part; s < nsplit; s += shares) {
            const float f = fac[s];
            const float4 v = *reinterpret_cast<const float4 *>(a.part_o + (slot0 + s) * vp + c);
            if (f > 0.f) { o.x = fmaf(v.x, f, o.x); o.y = fmaf(v.y, f, o.y); o.z = fmaf(v.z, f, o.z); o.w = fmaf(v.w, f, o.w); }
        }
        *reinterpret_cast<float4 *>(red + part * vp + c) = o;
    }
    __syncthreads();
    for (int i = tid; i < a.vdim; i += 256) {
        float o = 0.f;
        for (int k = 0; k < shares; k++) o += red[k * vp + i];
        const int at = h * a.vdim + i;
        a.o[(size_t)m * a.H * a.vdim + at] = a.gated ? o * sigmoid(a.cin[(size_t)m * a.ldc + a.o_g + at]) : o;
    }
}

}  // namespace

void launch_group_cache(const GroupRows &a)
{
    const int n = a.G * (pad4(a.dim) + pad4(a.vdim)), vec = a.dim % 4 == 0 && a.vdim % 4 == 0 && a.rot_dims % 8 == 0;
    LAUNCH(k_group_cache, dim3((n + 1023) / 1024, a.r.n()), dim3(256), 0, a, vec);
}

void launch_group_attend(const GroupRows &in)
{
    GroupRows a = in;
    const int keys = a.r.T == 1 ? 32 : 64, dp = pad4(a.dim), vp = pad4(a.vdim);      // decoding: more workgroups on fewer keys each
    // slices of the longest visible span among the step's rows: the whole chunk once a row starts a new one
    const int in_chunk = a.r.pos % a.chunk + a.r.T, most = in_chunk > a.chunk ? a.chunk : in_chunk, n = (most + keys - 1) / keys;
    const size_t per_row = (size_t)a.H * n * vp;
    const int rows = (int)std::max<size_t>(1, std::min<size_t>({(size_t)a.r.n(), (size_t)32768, ((size_t)32 << 20) / per_row}));
    const size_t po = rows * per_row;
    a.part_o = (float *)scratch(SCR_PARTIAL, (po + (size_t)rows * a.H * n * 2) * sizeof(float));
    a.part_ml = a.part_o + po;
    const int parts = std::max(1, 256 / (vp / 4));
    const size_t lds = ((size_t)HG * dp + HG * keys + dp + vp + (size_t)parts * HG * vp) * sizeof(float);
    const size_t mlds = (size_t)(pad4(n) + std::max(1, std::min(8, 256 / (vp / 4))) * vp) * sizeof(float);
    for (int m0 = 0; m0 < a.r.n(); m0 += rows) {
        const int nr = std::min(rows, a.r.n() - m0);
        const dim3 grid(n, a.G * ((a.H / a.G + HG - 1) / HG), nr);
        if (keys == 32) LAUNCH(k_group_attend<32>, grid, dim3(256), lds, a, m0, n);
        else LAUNCH(k_group_attend<64>, grid, dim3(256), lds, a, m0, n);
        if (n > 1) LAUNCH(k_group_merge, dim3(a.H, nr), dim3(256), mlds, a, m0, n);
    }
}

}  // namespace lmhip
