// Grouped attention inside chunks over a prompt's rows in 16-bit precision: the visible keys and values of every key head
// are laid out as matrix-core fragments once per step and met by 128 queries of a head per workgroup (prompt_attn.h).
// Scores, running maximum and sums are fp32; the operands of the two products are F16.
#include "group_rows.h"
#include "prompt_attn.h"
#include <algorithm>

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

struct PromptArgs {
    GroupRows a;
    int first, n_keys, blocks;                           // position of key 0; keys; blocks of 32 of them
    half_t *frags;                                       // [B][G][blocks][NJ + 2 NDB fragments][64 lanes][8]
};

// grid (blocks, G, B): fragments of 32 keys of one key head
template <int NJ, int NDB>
__global__ __launch_bounds__(256) void k_group_frags(PromptArgs p)
{
    const GroupRows &a = p.a;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l31 = lane & 31, hh = lane >> 5;
    const int kb = blockIdx.x, g = blockIdx.y, b = blockIdx.z, dp = (a.dim + 3) & ~3, vp = (a.vdim + 3) & ~3;
    half_t *out = p.frags + (((size_t)b * a.G + g) * p.blocks + kb) * (NJ + 2 * NDB) * 512;
    const float *kr = a.kring + (size_t)(b * a.G + g) * a.ring_rows * dp, *vr = a.vring + (size_t)(b * a.G + g) * a.ring_rows * vp;
    for (int f = wave; f < NJ + 2 * NDB; f += 4) {
        half8 v;
        if (f < NJ) {
            const int kk = kb * 32 + l31, d0 = 16 * f + 8 * hh;
            const bool in = kk < p.n_keys;
            const float *key = kr + (size_t)((p.first + (in ? kk : 0)) % a.ring_rows) * dp;
            float4 x[2];
#pragma unroll
            for (int e = 0; e < 2; e++) x[e] = in && d0 + 4 * e < dp ? *reinterpret_cast<const float4 *>(key + d0 + 4 * e) : make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = (half_t)(&x[e >> 2].x)[e & 3];
        } else {
            const int db = (f - NJ) >> 1, u = (f - NJ) & 1, c = 32 * db + l31;
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const int kk = kb * 32 + 16 * u + 8 * (e >> 2) + 4 * hh + (e & 3);
                v[e] = (half_t)(kk < p.n_keys && c < a.vdim ? vr[(size_t)((p.first + kk) % a.ring_rows) * vp + c] : 0.f);
            }
        }
        *reinterpret_cast<half8 *>(out + ((size_t)f * 64 + lane) * 8) = v;
    }
}

// eight consecutive values with their biases (both on 16 bytes)
__device__ __forceinline__ void biased8(const float *x, const float *b, float (&y)[8])
{
#pragma unroll
    for (int i = 0; i < 8; i += 4) {
        const float4 v = *reinterpret_cast<const float4 *>(x + i), w = *reinterpret_cast<const float4 *>(b + i);
        y[i] = v.x + w.x; y[i + 1] = v.y + w.y; y[i + 2] = v.z + w.z; y[i + 3] = v.w + w.w;
    }
}

// grid (blocks of 128 queries, H, B), block 256
template <int NJ, int NDB>
__global__ __launch_bounds__(256) void k_group_prompt(PromptArgs p)
{
    constexpr int NF = NJ + 2 * NDB;
    __shared__ uint4 buf0[NF * 64], buf1[NF * 64];
    const GroupRows &a = p.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l31 = lane & 31, hh = lane >> 5;
    const int q0 = (gridDim.x - 1 - blockIdx.x) * 128, h = blockIdx.y, b = blockIdx.z, T = a.r.T;
    const int qw = q0 + 32 * wave, qi = min(qw + l31, T - 1);
    const int off = a.r.pos - p.first;                    // key index of the step's first token
    auto start = [&](int t) __attribute__((always_inline)) { return (a.r.pos + t) / a.chunk * a.chunk - p.first; };   // first key that token t sees
    PromptSpan sp;
    sp.live = qw < T;
    sp.last = off + qi; sp.lo = start(qi);
    sp.w_hi = off + min(qw + 31, T - 1); sp.w_lo = start(min(qw, T - 1));
    sp.all_hi = off + qw; sp.all_lo = start(min(qw + 31, T - 1));
    sp.kb0 = start(q0) >> 5; sp.kb1 = (off + min(q0 + 127, T - 1)) >> 5;
    const size_t m = (size_t)b * T + qi;
    half8 qf[NJ];
    {
        const int at = a.o_q + h * a.dim;
        const float *q = a.cin + m * a.ldc + at, *bias = a.bias + at;
        const float2 *cs = group_angles(a, a.r.pos + qi);
        const float f = a.scale * 1.44269504f;
        if (a.dim % 8 == 0 && a.rot_dims % 16 == 0) {     // eight dimensions turn with eight others, or pass, together
            const int n = a.rot_dims >> 1;
#pragma unroll
            for (int j = 0; j < NJ; j++) {
                const int d = 16 * j + 8 * hh;
                if (d >= a.dim) {
#pragma unroll
                    for (int e = 0; e < 8; e++) qf[j][e] = (half_t)0.f;
                    continue;
                }
                float x[8], w[8];
                biased8(q + d, bias + d, x);
                if (d < a.rot_dims) {
                    const int o = d < n ? d + n : d - n;
                    const float4 *c4 = reinterpret_cast<const float4 *>(cs + (d < n ? d : o));
                    biased8(q + o, bias + o, w);
#pragma unroll
                    for (int e = 0; e < 8; e += 2) {
                        const float4 c = c4[e >> 1];
                        x[e] = x[e] * c.x + (d < n ? -w[e] : w[e]) * c.y;
                        x[e + 1] = x[e + 1] * c.z + (d < n ? -w[e + 1] : w[e + 1]) * c.w;
                    }
                }
#pragma unroll
                for (int e = 0; e < 8; e++) qf[j][e] = (half_t)(x[e] * f);
            }
        } else
#pragma unroll
            for (int j = 0; j < NJ; j++)
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const int d = 16 * j + 8 * hh + e;
                    qf[j][e] = (half_t)(d < a.dim ? rotated_half(q, bias, d, a.rot_dims, cs) * f : 0.f);
                }
    }
    const uint4 *src = reinterpret_cast<const uint4 *>(p.frags) + ((size_t)b * a.G + h / (a.H / a.G)) * p.blocks * NF * 64 + lane;
    float16v O[NDB];
    float l_run;
    prompt_attend<NJ, NDB>(qf, src, sp, buf0, buf1, O, l_run);
    if (qw + l31 >= T) return;
    prompt_store<NDB>(O, l_run, a.o + (m * a.H + h) * a.vdim, a.vdim);
}

int nj_of(const GroupRows &a)
{
    for (int s : {2, 4, 8, 16}) if (a.dim <= 16 * s) return s;
    return 0;
}
int ndb_of(const GroupRows &a)
{
    for (int s : {1, 2, 4, 8}) if (a.vdim <= 32 * s) return s;
    return 0;
}

template <int NJ, int NDB>
void run(const PromptArgs &p)
{
    LAUNCH((k_group_frags<NJ, NDB>), dim3(p.blocks, p.a.G, p.a.r.B), dim3(256), 0, p);
    LAUNCH((k_group_prompt<NJ, NDB>), dim3((p.a.r.T + 127) / 128, p.a.H, p.a.r.B), dim3(256), 0, p);
}
template <int NJ>
void run_nj(const PromptArgs &p, int ndb) { if (ndb == 1) run<NJ, 1>(p); else if (ndb == 2) run<NJ, 2>(p); else if (ndb == 4) run<NJ, 4>(p); else run<NJ, 8>(p); }

}  // namespace

bool group_prompt_fits(const GroupRows &a) { return a.r.T >= 16 && nj_of(a) && ndb_of(a); }

size_t group_prompt_frag_halfs(const GroupRows &a, int B, int n_keys)
{
    return (size_t)B * a.G * ((n_keys + 31) / 32) * (nj_of(a) + 2 * ndb_of(a)) * 512;
}

void launch_group_prompt(const GroupRows &a, half_t *frags)
{
    PromptArgs p{};
    p.a = a; p.frags = frags; p.first = group_prompt_first(a);
    p.n_keys = a.r.pos + a.r.T - p.first; p.blocks = (p.n_keys + 31) / 32;
    const int ndb = ndb_of(a);
    switch (nj_of(a)) {
    case 2: run_nj<2>(p, ndb); break;
    case 4: run_nj<4>(p, ndb); break;
    case 8: run_nj<8>(p, ndb); break;
    default: run_nj<16>(p, ndb); break;
    }
}

}  // namespace lmhip
