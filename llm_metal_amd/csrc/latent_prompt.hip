// Latent attention over a prompt's rows in 16-bit precision: keys and values of the visible positions are expanded once
// per step (one product of the latents with both projections), laid out as matrix-core fragments, and met by 128 queries
// of a head per workgroup.  Scores, running maximum and sums are fp32; the operands of the two products are F16.
#include "stack.h"
#include "latent_rows.h"
#include "prompt_attn.h"
#include <algorithm>

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

struct PromptArgs {
    LatentRows a;
    int first, n_keys, blocks;                           // position of key 0; keys; blocks of 32 of them
    const float *kv;
    half_t *frags;                                       // [B][H][blocks][NJ + 2 NDB fragments][64 lanes][8]
};

// grid (n_keys, B): the latent of one visible position as a row of the expansion's operand
__global__ __launch_bounds__(256) void k_latent_operand(PromptArgs p, half_t *a16, float *inv)
{
    extern __shared__ float row[];                       // [rank padded to 8]
    __shared__ float sm[16];
    const LatentRows &a = p.a;
    const int rp = (a.rank + 7) & ~7, w = rp + ((a.rot + 7) & ~7), kk = blockIdx.x, b = blockIdx.y, m = b * p.n_keys + kk;
    const float *c = a.ring + ((size_t)b * a.ring_rows + (p.first + kk) % a.ring_rows) * w;
    float mx = 0.f;
    for (int i = threadIdx.x; i < rp; i += 256) { const float v = c[i]; row[i] = v; mx = fmaxf(mx, fabsf(v)); }
    const float s = row_scale_for(block_max(mx, sm));
    store_row_f16(row, rp, a16, m, tiled_kb(rp), s);
    if (threadIdx.x == 0) inv[m] = 1.f / s;
}

// grid (blocks, H, B): fragments of 32 keys of one head (prompt_attn.h)
template <int NJ, int NDB>
__global__ __launch_bounds__(256) void k_latent_frags(PromptArgs p)
{
    const LatentRows &a = p.a;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l31 = lane & 31, hh = lane >> 5;
    const int kb = blockIdx.x, h = blockIdx.y, b = blockIdx.z, ld = a.H * (a.dim + a.vdim);
    const int rp = (a.rank + 7) & ~7, w = rp + ((a.rot + 7) & ~7);
    half_t *out = p.frags + (((size_t)b * a.H + h) * p.blocks + kb) * (NJ + 2 * NDB) * 512;
    const float *kv = p.kv + (size_t)b * p.n_keys * ld;
    for (int f = wave; f < NJ + 2 * NDB; f += 4) {
        half8 v;
        if (f < NJ) {
            const int kk = kb * 32 + l31;
            const bool in = kk < p.n_keys;
            const float *key = kv + (size_t)(in ? kk : 0) * ld + h * a.dim;
            const float *rot = a.ring + ((size_t)b * a.ring_rows + (p.first + (in ? kk : 0)) % a.ring_rows) * w + rp;
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const int d = 16 * f + 8 * hh + e;
                v[e] = (half_t)(!in ? 0.f : d < a.dim ? key[d] : d < a.dim + a.rot ? rot[d - a.dim] : 0.f);
            }
        } else {
            const int db = (f - NJ) >> 1, u = (f - NJ) & 1, c = 32 * db + l31;
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const int kk = kb * 32 + 16 * u + 8 * (e >> 2) + 4 * hh + (e & 3);
                v[e] = (half_t)(kk < p.n_keys && c < a.vdim ? kv[(size_t)kk * ld + a.H * a.dim + h * a.vdim + c] : 0.f);
            }
        }
        *reinterpret_cast<half8 *>(out + ((size_t)f * 64 + lane) * 8) = v;
    }
}

// grid (blocks of 128 queries, H, B), block 256
template <int NJ, int NDB>
__global__ __launch_bounds__(256) void k_latent_prompt(PromptArgs p)
{
    constexpr int NF = NJ + 2 * NDB;
    __shared__ uint4 buf0[NF * 64], buf1[NF * 64];
    const LatentRows &a = p.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l31 = lane & 31, hh = lane >> 5;
    const int q0 = (gridDim.x - 1 - blockIdx.x) * 128, h = blockIdx.y, b = blockIdx.z, T = a.r.T;
    const int qw = q0 + 32 * wave, qi = min(qw + l31, T - 1);
    const int off = a.r.pos - p.first;                    // key index of the step's first token
    PromptSpan sp;
    sp.live = qw < T;
    sp.last = off + qi; sp.lo = sp.last - a.window + 1;
    sp.w_hi = off + min(qw + 31, T - 1); sp.w_lo = off + min(qw, T - 1) - a.window + 1;
    sp.all_hi = off + qw; sp.all_lo = off + qw + 31 - a.window + 1;
    sp.kb0 = max(0, off + q0 - a.window + 1) >> 5; sp.kb1 = (off + min(q0 + 127, T - 1)) >> 5;
    const size_t m = (size_t)b * T + qi;
    half8 qf[NJ];
    {
        const float *q = a.cin + m * a.ldc + a.o_q + h * (a.dim + a.rot);
        const float2 *cs = a.rope + (size_t)(a.r.pos + qi) * (a.rot_dims / 2);
        const float f = a.scale * 1.44269504f;
#pragma unroll
        for (int j = 0; j < NJ; j++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const int d = 16 * j + 8 * hh + e;
                qf[j][e] = (half_t)(d < a.dim ? q[d] * f : d < a.dim + a.rot ? rotated(q + a.dim, d - a.dim, a.rot_dims, cs) * f : 0.f);
            }
    }
    const uint4 *src = reinterpret_cast<const uint4 *>(p.frags) + ((size_t)b * a.H + h) * p.blocks * NF * 64 + lane;
    float16v O[NDB];
    float l_run;
    prompt_attend<NJ, NDB>(qf, src, sp, buf0, buf1, O, l_run);
    if (qw + l31 >= T) return;
    prompt_store<NDB>(O, l_run, a.o + (m * a.H + h) * a.vdim, a.vdim);
}

int nj_of(const LatentRows &a)
{
    const int n = (a.dim + a.rot + 15) / 16;
    for (int s : {2, 4, 6, 8, 12, 16}) if (n <= s) return s;
    return 0;
}
int ndb_of(const LatentRows &a)
{
    const int n = (a.vdim + 31) / 32;
    for (int s : {1, 2, 4}) if (n <= s) return s;
    return 0;
}

PromptArgs prompt_args(const LatentRows &a)
{
    PromptArgs p{};
    p.a = a; p.first = latent_prompt_first(a); p.n_keys = latent_prompt_keys(a); p.blocks = (p.n_keys + 31) / 32;
    return p;
}

template <int NJ, int NDB>
void run(const PromptArgs &p)
{
    LAUNCH((k_latent_frags<NJ, NDB>), dim3(p.blocks, p.a.H, p.a.r.B), dim3(256), 0, p);
    LAUNCH((k_latent_prompt<NJ, NDB>), dim3((p.a.r.T + 127) / 128, p.a.H, p.a.r.B), dim3(256), 0, p);
}
template <int NJ>
void run_nj(const PromptArgs &p, int ndb) { if (ndb == 1) run<NJ, 1>(p); else if (ndb == 2) run<NJ, 2>(p); else run<NJ, 4>(p); }

}  // namespace

bool latent_prompt_fits(const LatentRows &a) { return !a.f32 && a.r.T >= 16 && nj_of(a) && ndb_of(a); }
int latent_prompt_first(const LatentRows &a) { return std::max(0, a.r.pos - a.window + 1); }

size_t latent_prompt_frag_halfs(const LatentRows &a, int B, int n_keys)
{
    return (size_t)B * a.H * ((n_keys + 31) / 32) * (nj_of(a) + 2 * ndb_of(a)) * 512;
}

void launch_latent_operand(const LatentRows &a, half_t *a16, float *inv)
{
    const PromptArgs p = prompt_args(a);
    LAUNCH(k_latent_operand, dim3(p.n_keys, a.r.B), dim3(256), (size_t)pad8(a.rank) * 4, p, a16, inv);
}

void launch_latent_prompt(const LatentRows &a, const float *kv, half_t *frags)
{
    PromptArgs p = prompt_args(a);
    p.kv = kv; p.frags = frags;
    const int ndb = ndb_of(a);
    switch (nj_of(a)) {
    case 2: run_nj<2>(p, ndb); break;
    case 4: run_nj<4>(p, ndb); break;
    case 6: run_nj<6>(p, ndb); break;
    case 8: run_nj<8>(p, ndb); break;
    case 12: run_nj<12>(p, ndb); break;
    default: run_nj<16>(p, ndb); break;
    }
}

}  // namespace lmhip
