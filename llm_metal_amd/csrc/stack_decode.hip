// One token of one sequence through a layer: the steps of a layer-by-layer model fused for decoding with F16 weights and
// fp32 vectors.  Three launches for a delta layer, five for latent attention:
//   1  everything that reads the normed vector, as one product that forms the norm itself (matvec_layernorm)
//   2  the mixer -- convolutions, decays and the state's update, or cache row and absorbed queries -- and, in further
//      workgroups of the same launch, the chosen experts' up products
//  (3, 4  attention over the latents in slices, value projection)
//   5  residual += output projection and shared expert, and the experts' down products, with the head norm and gate or
//      the squared ReLU applied to the vectors on their way into LDS
#include "latent_rows.h"
#include "delta_rows.h"
#include "stack_decode.h"
#include <algorithm>

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

constexpr int UP_ROWS = 16;  // expert rows per workgroup, four per wave

// One workgroup of 256: rows UP_ROWS blk .. of the chosen experts' up products, over the normed vector it forms for
// itself.  lds: [Dp]
__device__ __forceinline__ void experts_up(const DecodeMoe &a, int blk, float *lds)
{
    __shared__ float red[16], w[32];
    __shared__ int idx[32];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    float sum = 0.f;
    for (int i = tid * 4; i < a.Dp; i += 1024) {
        const float4 v = *reinterpret_cast<const float4 *>(a.x + i);
        *reinterpret_cast<float4 *>(lds + i) = v;
        sum += (v.x + v.y) + (v.z + v.w);
    }
    if (wave == 0) route_row(a.z, a.E, a.top, lane, idx, w);
    const float mean = block_sum(sum, red) / (float)a.D;
    float ss = 0.f;
    for (int i = tid * 4; i < a.Dp; i += 1024)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const float d = i + e < a.D ? lds[i + e] - mean : 0.f;
            ss += d * d;
            lds[i + e] = d * a.g[i + e];
        }
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
    if (blk == 0 && tid < a.top) { a.idx[tid] = idx[tid]; a.w[tid] = w[tid]; }
    const int n = a.top * a.ffp;
    constexpr int PER = UP_ROWS / 4;
    const int r0 = blk * UP_ROWS + wave * PER;
    const half_t *rows[PER];
    float y[PER];
#pragma unroll
    for (int k = 0; k < PER; k++) {
        const int r = min(r0 + k, n - 1), s = r / a.ffp, i = min(r % a.ffp, a.ff - 1);
        rows[k] = a.up + ((size_t)idx[s] * a.up_rows + i) * a.Dp;
        y[k] = 0.f;
    }
    dot_rows<PER, 2>(rows, lds, a.Dp, lane, y);
#pragma unroll
    for (int k = 0; k < PER; k++) {
        const float v = wave_total(y[k]) * inv;
        if (lane == 0 && r0 + k < n) a.act[r0 + k] = (r0 + k) % a.ffp < a.ff ? relu2(v) : 0.f;   // the padding is written too
    }
}

// grid: H * nb workgroups for the mixer (nb column blocks of 256 / G per head), then those of the experts
template <int G, int R, int PC>
__global__ __launch_bounds__(256) void k_delta_decode(DecodeDelta s, DecodeMoe e, int nb)
{
    extern __shared__ float lds[];
    const DeltaRows &a = s.a;
    if ((int)blockIdx.x >= a.H * nb) { experts_up(e, blockIdx.x - a.H * nb, lds); return; }
    constexpr int DP = G * R, COLS = 256 / G, RB = R / 4;
    __shared__ float ks[DP], qs[DP], gs[PC ? DP : 1], red[32];
    const int tid = threadIdx.x, l = tid % G, col = tid / G, lane = tid & 63;
    const int h = blockIdx.x / nb, j0 = (blockIdx.x % nb) * COLS, j = j0 + col, jc = min(j, a.vdim - 1), kvh = h / (a.H / a.KV);
    const int qd = a.KV * a.dim, C = 2 * qd + a.H * a.vdim;
    float *ring = a.conv + (size_t)(a.r.pos % a.taps) * C;
    float *Sg = a.S + ((size_t)h * a.vdim + jc) * a.dim;
    float S[R];
#pragma unroll
    for (int x = 0; x < R; x++) {                         // asked for first: nothing below needs it for a while
        const int d = (x >> 2) * 4 * G + 4 * l + (x & 3);
        S[x] = (a.r.pos > 0 && d < a.dim) ? Sg[d] : 0.f;
    }
    // q, k and the decays of this head: a thread per channel (dim <= 256)
    float qv = 0.f, kv = 0.f, gv = 1.f;
    if (tid < a.dim) {
        const int ch = kvh * a.dim + tid;
        qv = silu(conv_at(a, 0, ch, a.o_q + ch));
        kv = silu(conv_at(a, 0, qd + ch, a.o_k + ch));
        if (h % (a.H / a.KV) == 0 && j0 == 0) { ring[ch] = a.cin[a.o_q + ch]; ring[qd + ch] = a.cin[a.o_k + ch]; }
        if (PC) {
            float t = 0.f;
            const half_t *w = s.a2 + ((size_t)h * a.dim + tid) * s.lda2;
#pragma unroll 8
            for (int c = 0; c < s.lda2; c += 8) {
                float wv[8];
                Vec8<half_t>::load(w + c, wv);
#pragma unroll
                for (int x = 0; x < 8; x++) t = fmaf(wv[x], a.cin[a.o_a + c + x], t);
            }
            gv = expf(-a.a_exp[h] * softplus(t + a.dt_bias[h * a.dim + tid]));
        }
    }
    // this column's value and gate
    const int vch = h * a.vdim + jc;
    const float v = silu(conv_at(a, 0, 2 * qd + vch, a.o_v + vch));
    if (l == 0 && j < a.vdim) ring[2 * qd + vch] = a.cin[a.o_v + vch];
    float gate;
    if (PC) {
        float t = 0.f;
        const half_t *w = s.g2 + (size_t)vch * s.ldg2;
        for (int c = l * 8; c < s.ldg2; c += G * 8) {
            float wv[8];
            Vec8<half_t>::load(w + c, wv);
#pragma unroll
            for (int x = 0; x < 8; x++) t = fmaf(wv[x], a.cin[s.o_g + c + x], t);
        }
        gate = sigmoid(group_sum<G>(t));
    } else gate = silu(a.cin[s.o_g + vch]);
    const float beta = sigmoid(a.cin[a.o_b + h]);
    const float gh = PC ? 1.f : expf(-a.a_exp[h] * softplus(a.cin[a.o_a + h] + a.dt_bias[h]));
    float sq = qv * qv, sk = kv * kv;
    block_sum2(sq, sk, red);
    const float dot = block_sum(qv * kv, red);
    const float iq = 1.f / (sqrtf(sq + 1e-6f) * sqrtf((float)a.dim)), ik = 1.f / sqrtf(sk + 1e-6f), kq = dot * iq * ik;
    if (tid < DP) { qs[tid] = qv * iq; ks[tid] = kv * ik; if (PC) gs[tid] = gv; }   // zeros beyond dim
    __syncthreads();
    float p = 0.f, w = 0.f, kk[R];
#pragma unroll
    for (int i = 0; i < RB; i++) {
        const int d = i * 4 * G + 4 * l;
#pragma unroll
        for (int x = 0; x < 4; x++) {
            kk[4 * i + x] = ks[d + x];
            S[4 * i + x] *= PC ? gs[PC ? d + x : 0] : gh;
            p = fmaf(S[4 * i + x], kk[4 * i + x], p); w = fmaf(S[4 * i + x], qs[d + x], w);
        }
    }
    p = group_sum<G>(p); w = group_sum<G>(w);
    const float u = beta * (v - p);
    if (j < a.vdim) {
#pragma unroll
        for (int x = 0; x < R; x++) {
            const int d = (x >> 2) * 4 * G + 4 * l + (x & 3);
            if (d < a.dim) Sg[d] = fmaf(kk[x], u, S[x]);
        }
        if (l == 0) { a.o[vch] = fmaf(u, kq, w); s.gate[vch] = gate; }
    }
    (void)lane;
}

// grid: H workgroups for the queries, one for the cache row, then those of the experts
__global__ __launch_bounds__(256) void k_latent_decode(LatentRows a, DecodeMoe e)
{
    extern __shared__ float lds[];
    __shared__ float sm[16];
    if ((int)blockIdx.x < a.H) latent_query_row<half_t>(a, 0, blockIdx.x, lds);
    else if ((int)blockIdx.x == a.H) latent_cache_row(a, 0, sm);
    else experts_up(e, blockIdx.x - a.H - 1, lds);
}

// x[d] += out[d] . (mixer output | shared activation) + sum over the chosen experts of w * down_e[d] . act_e (or y[d] = the
// sum, when a norm lies behind it); a wave takes PER values of d.  lds: [ldk] then [top * ffp]
template <int TPB, int PER>
__global__ __launch_bounds__(TPB) void k_out_decode(DecodeOut a, DecodeMoe e)
{
    extern __shared__ float lds[];
    constexpr int NW = TPB / 64;
    float *cat = lds, *act = lds + a.cat.ldk;
    const CatRows &c = a.cat;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int na = e.top * e.ffp;
    for (int i = tid * 4; i < na; i += TPB * 4) *reinterpret_cast<float4 *>(act + i) = *reinterpret_cast<const float4 *>(e.act + i);
    if (c.g_out) {
        for (int h = wave; h < c.H; h += NW) {
            const float *o = c.o + (size_t)h * c.vdim, *gt = c.gate + (size_t)h * c.vdim;      // the gate is already a factor
            float ss = 0.f;
            for (int d = lane; d < c.vdim; d += 64) ss += o[d] * o[d];
            const float inv = 1.f / sqrtf(wave_total(ss) / (float)c.vdim + c.eps);
            for (int d = lane; d < c.vdim; d += 64) cat[h * c.vdim + d] = o[d] * inv * c.g_out[h * c.g_stride + d] * gt[d];
        }
    } else
        for (int i = tid; i < c.H * c.vdim; i += TPB) cat[i] = c.o[i];
    for (int i = c.H * c.vdim + tid; i < c.ldk; i += TPB) {
        const int s = i - c.o_sh;
        cat[i] = s >= 0 && s < c.shared_ff ? relu2(c.shared[s]) : 0.f;
    }
    __syncthreads();
    // PER rows of one wave at a time, the pieces of four experts (or of the dense row) in flight together
    const int d0 = (blockIdx.x * NW + wave) * PER;
    if (d0 >= a.D) return;
    float y[PER] = {};
    const half_t *rows[PER];
#pragma unroll
    for (int k = 0; k < PER; k++) rows[k] = a.out + (size_t)min(d0 + k, a.D - 1) * c.ldk;
    dot_rows<PER, 8 / PER>(rows, cat, c.ldk, lane, y);
    for (int s0 = 0; s0 < e.top; s0 += 4) {
        const half_t *base[4];
        float wt[4];
#pragma unroll
        for (int u = 0; u < 4; u++) {
            const int s = min(s0 + u, e.top - 1);
            base[u] = e.down + ((size_t)e.idx[s] * e.down_rows) * e.ffp;
            wt[u] = s0 + u < e.top ? e.w[s] : 0.f;
        }
        for (int cc = lane * 8; cc < e.ffp; cc += 512) {
            float wv[PER][4][8];
#pragma unroll
            for (int k = 0; k < PER; k++)
#pragma unroll
                for (int u = 0; u < 4; u++) Vec8<half_t>::load(base[u] + (size_t)min(d0 + k, a.D - 1) * e.ffp + cc, wv[k][u]);
#pragma unroll
            for (int u = 0; u < 4; u++)
#pragma unroll
                for (int k = 0; k < PER; k++) y[k] = fmaf(wt[u], dot8(wv[k][u], act + min(s0 + u, e.top - 1) * e.ffp + cc, 0.f), y[k]);
        }
    }
#pragma unroll
    for (int k = 0; k < PER; k++) {
        const float t = wave_total(y[k]);
        if (lane == 0 && d0 + k < a.D) { if (a.y) a.y[d0 + k] = t; else a.x[d0 + k] += t; }
    }
}

int up_blocks(const DecodeMoe &e) { return (e.top * e.ffp + UP_ROWS - 1) / UP_ROWS; }

}  // namespace

bool decode_fits(int ldk, int top, int ffp, int Dp)
{
    return ((size_t)ldk + (size_t)top * ffp) * sizeof(float) <= DECODE_LDS && (size_t)Dp * sizeof(float) <= 60 * 1024;
}

void launch_delta_decode(const DecodeDelta &s, const DecodeMoe &e)
{
    const DeltaRows &a = s.a;
    const int G = a.dim <= 32 ? 4 : a.dim <= 64 ? 8 : a.dim <= 128 ? 16 : 32, cols = 256 / G, nb = (a.vdim + cols - 1) / cols;
    const dim3 grid(a.H * nb + up_blocks(e));
    const size_t lds = (size_t)e.Dp * sizeof(float);
#define DELTA(G_) do { if (a.per_channel) LAUNCH((k_delta_decode<G_, 8, 1>), grid, dim3(256), lds, s, e, nb); \
                       else LAUNCH((k_delta_decode<G_, 8, 0>), grid, dim3(256), lds, s, e, nb); } while (0)
    if (G == 4) DELTA(4); else if (G == 8) DELTA(8); else if (G == 16) DELTA(16); else DELTA(32);
#undef DELTA
}

void launch_latent_decode(const LatentRows &in, const DecodeMoe &e)
{
    LatentRows a = in;
    const LatentSlices s = latent_slices(a);
    latent_partials(a, s);
    LAUNCH(k_latent_decode, dim3(a.H + 1 + up_blocks(e)), dim3(256), std::max(latent_query_lds(a), (size_t)e.Dp * sizeof(float)), a, e);
    launch_latent_slices(a, s, 0, 1);
}

void launch_out_decode(const DecodeOut &a, const DecodeMoe &e)
{
    const size_t lds = ((size_t)a.cat.ldk + (size_t)e.top * e.ffp) * sizeof(float);
    static bool set = false;
    if (!set) {                                           // more than the default 64 KB
        for (const void *k : {reinterpret_cast<const void *>(&k_out_decode<512, 2>), reinterpret_cast<const void *>(&k_out_decode<512, 1>), reinterpret_cast<const void *>(&k_out_decode<256, 1>)})
            HIP_CHECK(hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)DECODE_LDS));
        set = true;
    }
    // as many rows per workgroup as still give every CU one: each stages both vectors
    const int cus = num_cus() > 0 ? num_cus() : 256;
    if (a.D >= 16 * cus) LAUNCH((k_out_decode<512, 2>), dim3((a.D + 15) / 16), dim3(512), lds, a, e);
    else if (a.D >= 8 * cus) LAUNCH((k_out_decode<512, 1>), dim3((a.D + 7) / 8), dim3(512), lds, a, e);
    else LAUNCH((k_out_decode<256, 1>), dim3((a.D + 3) / 4), dim3(256), lds, a, e);
}

}  // namespace lmhip
