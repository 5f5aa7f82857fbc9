// Gated delta rule: short causal convolutions, unit norms, decays, the recurrence over tokens, the gated head norm.
// Everything here is fp32, the matrix instructions of the recurrence included.
#include "stack.h"
#include "delta_rows.h"
#include "planes.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

// silu of the convolutions at NE channels for the tokens t0 .. t0 + TW - 1 of sequence b: y[token][channel], zeros past the
// end.  Up to four taps the inputs slide through registers, each read once; more taps are gathered token by token.
constexpr int TW = 8;        // tokens per wave
template <int NE>
__device__ __forceinline__ void conv_tokens(const DeltaRows &a, int b, int t0, const int (&ch)[NE], const int (&col)[NE], const bool (&in)[NE],
                                            float (&y)[TW][NE])
{
    const int T = a.r.T, nt = min(TW, T - t0), C = 2 * a.KV * a.dim + a.H * a.vdim;
    if (a.taps <= 4) {
        float f[NE][4], x[NE][TW + 3];
#pragma unroll
        for (int i = 0; i < TW + 3; i++) {
            const int tt = t0 - 3 + i, p = a.r.pos + tt;
#pragma unroll
            for (int e = 0; e < NE; e++) {
                float v = 0.f;
                if (in[e] && tt < T && p >= 0) {
                    if (tt >= 0) v = a.cin[(size_t)(b * T + tt) * a.ldc + col[e]];
                    else if (-tt < a.taps) v = a.conv[((size_t)b * a.taps + p % a.taps) * C + ch[e]];
                }
                x[e][i] = v;
            }
        }
#pragma unroll
        for (int e = 0; e < NE; e++)
#pragma unroll
            for (int i = 0; i < 4; i++) f[e][i] = in[e] && i >= 4 - a.taps ? a.filters[(size_t)ch[e] * a.taps + i - (4 - a.taps)] : 0.f;
#pragma unroll
        for (int i = 0; i < TW; i++)
#pragma unroll
            for (int e = 0; e < NE; e++)
                y[i][e] = silu(fmaf(f[e][3], x[e][i + 3], fmaf(f[e][2], x[e][i + 2], fmaf(f[e][1], x[e][i + 1], f[e][0] * x[e][i]))));
    } else {
#pragma unroll
        for (int i = 0; i < TW; i++)
#pragma unroll
            for (int e = 0; e < NE; e++) y[i][e] = in[e] && i < nt ? silu(conv_at(a, b * T + t0 + i, ch[e], col[e])) : 0.f;
    }
}

// One wave per (unit, TW tokens): units 0 .. KV-1 finish q and k of a key head, the others 64 channels of the values.  A
// lane holds channels lane, lane + 64, ... (E of them).  grid (ceil(units / 4), ceil(T / TW), B)
template <int E>
__global__ __launch_bounds__(256) void k_delta_inputs(DeltaRows a)
{
    const int lane = threadIdx.x & 63, u = blockIdx.x * 4 + (threadIdx.x >> 6), t0 = blockIdx.y * TW, b = blockIdx.z;
    const int qd = a.KV * a.dim, vd = a.H * a.vdim, m0 = b * a.r.T + t0, nt = min(TW, a.r.T - t0);
    if (u >= a.KV + (vd + 63) / 64) return;
    if (u < a.KV) {
        int ch[2 * E], col[2 * E];
        bool in[2 * E];
        float y[TW][2 * E];
#pragma unroll
        for (int e = 0; e < E; e++) {
            const int d = lane + 64 * e;
            in[e] = in[E + e] = d < a.dim;
            ch[e] = u * a.dim + d; col[e] = a.o_q + ch[e];
            ch[E + e] = qd + u * a.dim + d; col[E + e] = a.o_k + u * a.dim + d;
        }
        conv_tokens<2 * E>(a, b, t0, ch, col, in, y);
        float iq[TW], ik[TW];
#pragma unroll
        for (int i = 0; i < TW; i++) {
            float sq = 0.f, sk = 0.f;
#pragma unroll
            for (int e = 0; e < E; e++) { sq += y[i][e] * y[i][e]; sk += y[i][E + e] * y[i][E + e]; }
            iq[i] = wave_total(sq); ik[i] = wave_total(sk);
        }
#pragma unroll
        for (int i = 0; i < TW; i++) {
            if (i >= nt) break;
            const float fq = 1.f / (sqrtf(iq[i] + 1e-6f) * sqrtf((float)a.dim)), fk = 1.f / sqrtf(ik[i] + 1e-6f);
            const size_t o = ((size_t)(m0 + i) * a.KV + u) * a.dim + lane;
#pragma unroll
            for (int e = 0; e < E; e++)
                if (in[e]) { a.q[o + 64 * e] = y[i][e] * fq; a.k[o + 64 * e] = y[i][E + e] * fk; }
        }
        return;
    }
    const int c = (u - a.KV) * 64 + lane, ch[1] = {2 * qd + c}, col[1] = {a.o_v + c};
    const bool in[1] = {c < vd};
    float y[TW][1];
    conv_tokens<1>(a, b, t0, ch, col, in, y);
#pragma unroll
    for (int i = 0; i < TW; i++) if (i < nt && in[0]) a.v[(size_t)(m0 + i) * vd + c] = y[i][0];
}

// ---------------------------------------------------------------- tokens in chunks of sixteen
//
// Sixteen tokens are taken through the recurrence together.  With S the state ahead of them, d(j, i) the decay between
// writing token j and reading token i (the product of the decays of j + 1 .. i) and d(-, i) the one from S to i:
//     p_i = S^T (d(-, i) k_i)           w_i = S^T (d(-, i) q_i)
//     u_i = beta_i (v_i - p_i - sum_{j < i} A_ij u_j)      A_ij = k_i . d(j, i) k_j
//     o_i = w_i + sum_{j <= i} B_ij u_j                    B_ij = q_i . d(j, i) k_j
//     S  <- d(-, 15) S + sum_j d(j, 15) k_j u_j^T
// which is the token-by-token recurrence with the sums written out.  All decays enter as products of factors up to 1 --
// nothing is divided by a decay that may have vanished.  The u_i are U = M (V - P) with M = (I + diag(beta) A)^-1
// diag(beta), so a chunk is a few small matrix products.  What does not depend on the state (M, B, the decayed keys and
// queries) is made for all chunks at once by k_delta_prepare; k_delta_chunks then goes through them in order.
//
// Layouts, per (sequence, chunk, head), dimensions padded with zeros to DP (whole tiles of 16, the same number per wave):
//   kd, qd [tiles][lane][4]: lane -> token lane & 15, dimensions 4 (lane >> 4) + 0 .. 3 of the tile
//   ku     [tiles][lane][4]: lane -> dimension lane & 15 of the tile, tokens 4 (lane >> 4) + 0 .. 3
//   gc     [DP]: d(-, 15);  mb [2][16][16]: M, B
constexpr int CT = DELTA_CHUNK;
static_assert(CT == 16, "a chunk is one tile of the matrix instruction");

// grid (H, chunks, B), block 256.  LDS: k, q, g [16][DP + 4], A, B [16][17], beta [16]
__global__ __launch_bounds__(256) void k_delta_prepare(DeltaRows a, int DP)
{
    extern __shared__ float lds[];
    const int LD = DP + 4;
    float *ks = lds, *qs = ks + CT * LD, *gs = qs + CT * LD, *A = gs + CT * LD, *Bm = A + CT * 17, *beta = Bm + CT * 17;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = blockIdx.x, ck = blockIdx.y, b = blockIdx.z, T = a.r.T, kvh = h / (a.H / a.KV), t0 = ck * CT, nt = min(CT, T - t0);
    const size_t m0 = (size_t)b * T + t0, chunk = ((size_t)b * gridDim.y + ck) * a.H + h;
    const float ae = a.a_exp[h];
    // tokens past the end leave the state alone: no key, no step, decay 1
    const int n4 = DP / 4, step = 256 / n4, d = tid % n4 * 4;
    const bool vec = a.dim % 4 == 0;                      // the rows of k, q and a2 then start on 16 bytes
    for (int t = tid / n4; t < CT && tid < step * n4; t += step) {
        float4 k = make_float4(0.f, 0.f, 0.f, 0.f), q = k, z = k, g = make_float4(1.f, 1.f, 1.f, 1.f);
        if (t < nt && d < a.dim) {
            const float *kp = a.k + ((m0 + t) * a.KV + kvh) * a.dim + d, *qp = a.q + ((m0 + t) * a.KV + kvh) * a.dim + d;
            const float *zp = a.per_channel ? a.a2 + ((m0 + t) * a.H + h) * a.dim + d : nullptr;
            if (vec) {
                k = *reinterpret_cast<const float4 *>(kp); q = *reinterpret_cast<const float4 *>(qp);
                if (zp) z = *reinterpret_cast<const float4 *>(zp);
            } else
                for (int u = 0; u < 4 && d + u < a.dim; u++) { (&k.x)[u] = kp[u]; (&q.x)[u] = qp[u]; if (zp) (&z.x)[u] = zp[u]; }
            if (zp) {
                const float *bias = a.dt_bias + h * a.dim + d;
#pragma unroll
                for (int u = 0; u < 4; u++) if (d + u < a.dim) (&g.x)[u] = expf(-ae * softplus((&z.x)[u] + bias[u]));
            }
        }
        if (!a.per_channel && t < nt) g.x = g.y = g.z = g.w = expf(-ae * softplus(a.cin[(m0 + t) * a.ldc + a.o_a + h] + a.dt_bias[h]));
        *reinterpret_cast<float4 *>(&ks[t * LD + d]) = k;
        *reinterpret_cast<float4 *>(&qs[t * LD + d]) = q;
        *reinterpret_cast<float4 *>(&gs[t * LD + d]) = g;
    }
    if (tid < CT) beta[tid] = tid < nt ? sigmoid(a.cin[(m0 + tid) * a.ldc + a.o_b + h]) : 0.f;
    __syncthreads();
    {   // A and B: sixteen lanes share a row j of keys, each with every 16th piece of four dimensions, and walk the tokens i
        // from j on while the decay between builds up
        const int j = wave * 4 + (lane >> 4), part = lane & 15;
        float sa[CT], sb[CT];
#pragma unroll
        for (int i = 0; i < CT; i++) sa[i] = sb[i] = 0.f;
        for (int d = part * 4; d < DP; d += 64) {
            float4 c = *reinterpret_cast<const float4 *>(&ks[j * LD + d]);
#pragma unroll
            for (int i = 0; i < CT; i++) {
                if (i < wave * 4) continue;               // (the wave's first j; what lies below a lane's own j is not kept)
                const float4 k = *reinterpret_cast<const float4 *>(&ks[i * LD + d]), q = *reinterpret_cast<const float4 *>(&qs[i * LD + d]);
                const float4 g = *reinterpret_cast<const float4 *>(&gs[i * LD + d]);
                const bool later = i > j;
                c.x *= later ? g.x : 1.f; c.y *= later ? g.y : 1.f; c.z *= later ? g.z : 1.f; c.w *= later ? g.w : 1.f;
                sa[i] = fmaf(k.x, c.x, fmaf(k.y, c.y, fmaf(k.z, c.z, fmaf(k.w, c.w, sa[i]))));
                sb[i] = fmaf(q.x, c.x, fmaf(q.y, c.y, fmaf(q.z, c.z, fmaf(q.w, c.w, sb[i]))));
            }
        }
#pragma unroll
        for (int i = 0; i < CT; i++) {
            const float va = group_sum<16>(sa[i]), vb = group_sum<16>(sb[i]);
            if (part == 0) { A[i * 17 + j] = i > j ? va : 0.f; Bm[i * 17 + j] = i >= j ? vb : 0.f; }
        }
    }
    // decayed keys and queries: a thread per (token, four dimensions)
    for (int e = tid; e < CT * DP / 4; e += 256) {
        const int t = e % CT, d = (e / CT) * 4;           // (sixteen tokens side by side: their fragments are contiguous)
        float4 c = make_float4(1.f, 1.f, 1.f, 1.f);
        for (int x = 0; x <= t; x++) {
            const float4 g = *reinterpret_cast<const float4 *>(&gs[x * LD + d]);
            c.x *= g.x; c.y *= g.y; c.z *= g.z; c.w *= g.w;
        }
        const float4 k = *reinterpret_cast<const float4 *>(&ks[t * LD + d]), q = *reinterpret_cast<const float4 *>(&qs[t * LD + d]);
        const size_t o = chunk * DP * CT + ((size_t)(d / 16) * 64 + ((d % 16) / 4) * 16 + t) * 4;
        *reinterpret_cast<float4 *>(a.kd + o) = make_float4(k.x * c.x, k.y * c.y, k.z * c.z, k.w * c.w);
        *reinterpret_cast<float4 *>(a.qd + o) = make_float4(q.x * c.x, q.y * c.y, q.z * c.z, q.w * c.w);
        if (t == CT - 1) *reinterpret_cast<float4 *>(a.gc + chunk * DP + d) = c;
    }
    // keys as the state's update takes them: a thread per (dimension, four tokens)
    for (int e = tid; e < CT * DP / 4; e += 256) {
        const int d = e % DP, t4 = (e / DP) * 4;
        float r = 1.f, v[4];
        for (int x = CT - 1; x > t4 + 3; x--) r *= gs[x * LD + d];
#pragma unroll
        for (int x = 3; x >= 0; x--) { v[x] = ks[(t4 + x) * LD + d] * r; r *= gs[(t4 + x) * LD + d]; }
        const size_t o = chunk * DP * CT + ((size_t)(d / 16) * 64 + (t4 / 4) * 16 + d % 16) * 4;
        *reinterpret_cast<float4 *>(a.ku + o) = make_float4(v[0], v[1], v[2], v[3]);
    }
    __syncthreads();
    float *mb = a.mb + chunk * 2 * CT * CT;
    if (tid < CT) {                                       // column tid of M by forward substitution
        float x[CT];
#pragma unroll
        for (int i = 0; i < CT; i++) {
            float s = i == tid ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; j++) s = fmaf(-A[i * 17 + j], x[j], s);
            x[i] = beta[i] * s;
            mb[i * CT + tid] = x[i];
        }
    } else if (tid >= 64) {
        for (int e = tid - 64; e < CT * CT; e += 192) mb[CT * CT + e] = Bm[(e / CT) * 17 + e % CT];
    }
}

// grid (ceil(vdim / 16), H, B); a workgroup owns sixteen columns of a head's state, each of its waves TPW tiles of sixteen
// rows, held as the accumulators of v_mfma_f32_16x16x4_f32 (fp32 operands and sums).  The register order of an accumulator
// -- column lane & 15, rows 4 (lane >> 4) + 0 .. 3 -- is also a legal order of the reduction index of an operand, so S, U
// and V - P go from one product into the next as they are.  Per chunk the waves add their parts of P and W through LDS (one
// barrier); everything from memory is asked for SETS chunks ahead.
template <int TPW, int SETS, int NW>
__global__ __launch_bounds__(64 * NW) void k_delta_chunks(DeltaRows a, int DP, int chunks)
{
    __shared__ float4v red[2][NW][2][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, r4 = lane >> 4;
    const int h = blockIdx.y, b = blockIdx.z, T = a.r.T, j = blockIdx.x * 16 + c, jc = min(j, a.vdim - 1);
    const int vd = a.H * a.vdim;
    float *Sg = a.S + (((size_t)b * a.H + h) * a.vdim + jc) * a.dim;
    const int d0 = wave * TPW * 16 + 4 * r4;              // rows d0 + 16 tile + 0 .. 3
    float4v S[TPW];
#pragma unroll
    for (int i = 0; i < TPW; i++)
#pragma unroll
        for (int v = 0; v < 4; v++) {                     // position 0 starts from nothing, whatever the state held
            const int d = d0 + 16 * i + v;
            S[i][v] = (a.r.pos > 0 && d < a.dim) ? Sg[d] : 0.f;
        }
    auto at4 = [](const float *base, uint32_t i) __attribute__((always_inline)) {
        return *reinterpret_cast<const float4v *>(reinterpret_cast<const char *>(base) + 4u * i);
    };
    auto at1 = [](const float *base, uint32_t i) __attribute__((always_inline)) {
        return *reinterpret_cast<const float *>(reinterpret_cast<const char *>(base) + 4u * i);
    };
    const uint32_t out0 = (uint32_t)((b * T + 4 * r4) * vd + h * a.vdim + jc);
    struct Set { float4v k[TPW], q[TPW], u[TPW], g[TPW], m, b, v; };
    auto fetch = [&](Set &x, int ck) __attribute__((always_inline)) {
        const uint32_t chunk = (uint32_t)((b * chunks + min(ck, chunks - 1)) * a.H + h);
        const uint32_t f = chunk * (uint32_t)(DP * CT) + (uint32_t)(wave * TPW * 256 + lane * 4);
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            x.k[i] = at4(a.kd, f + 256 * i); x.q[i] = at4(a.qd, f + 256 * i); x.u[i] = at4(a.ku, f + 256 * i);
            x.g[i] = at4(a.gc, chunk * (uint32_t)DP + (uint32_t)(d0 + 16 * i));
        }
        const uint32_t mb = chunk * (uint32_t)(2 * CT * CT) + (uint32_t)(c * CT + 4 * r4);
        x.m = at4(a.mb, mb); x.b = at4(a.mb, mb + CT * CT);
#pragma unroll
        for (int v = 0; v < 4; v++)
            x.v[v] = at1(a.v, (uint32_t)(b * T + min(min(ck, chunks - 1) * CT + 4 * r4 + v, T - 1)) * (uint32_t)vd + (uint32_t)(h * a.vdim + jc));
    };
    auto take = [&](const Set &x, int ck) __attribute__((always_inline)) {
        float4v p = {0.f, 0.f, 0.f, 0.f}, w = p;
#pragma unroll
        for (int i = 0; i < TPW; i++)
#pragma unroll
            for (int v = 0; v < 4; v++) {
                p = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[i][v], S[i][v], p, 0, 0, 0);
                w = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[i][v], S[i][v], w, 0, 0, 0);
            }
        float4v(&rd)[NW][2][64] = red[ck & 1];
        rd[wave][0][lane] = p; rd[wave][1][lane] = w;
        __syncthreads();
        float4v pn[NW], wn[NW];
#pragma unroll
        for (int n = 0; n < NW; n++) pn[n] = rd[n][0][lane];
#pragma unroll
        for (int n = 0; n < NW; n++) wn[n] = rd[n][1][lane];
        p = pn[0]; w = wn[0];
#pragma unroll
        for (int n = 1; n < NW; n++) { p += pn[n]; w += wn[n]; }
        const float4v z = x.v - p;
        float4v u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int v = 0; v < 4; v++) u = __builtin_amdgcn_mfma_f32_16x16x4f32(x.m[v], z[v], u, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            S[i] *= x.g[i];
#pragma unroll
            for (int v = 0; v < 4; v++) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.u[i][v], u[v], S[i], 0, 0, 0);
        }
        if (ck % NW == wave) {                            // the waves take the outputs in turn
#pragma unroll
            for (int v = 0; v < 4; v++) w = __builtin_amdgcn_mfma_f32_16x16x4f32(x.b[v], u[v], w, 0, 0, 0);
            char *to = reinterpret_cast<char *>(a.o) + 4u * (out0 + (uint32_t)(ck * CT) * (uint32_t)vd);
            if (j < a.vdim) {
                if (ck * CT + CT <= T) {
#pragma unroll
                    for (int v = 0; v < 4; v++) *reinterpret_cast<float *>(to + 4u * (uint32_t)(v * vd)) = w[v];
                } else
#pragma unroll
                    for (int v = 0; v < 4; v++) if (ck * CT + 4 * r4 + v < T) *reinterpret_cast<float *>(to + 4u * (uint32_t)(v * vd)) = w[v];
            }
        }
    };
    Set x[SETS];
#pragma unroll
    for (int n = 0; n < SETS - 1; n++) fetch(x[n], n);
    for (int ck = 0; ck < chunks; ck += SETS)
#pragma unroll
        for (int n = 0; n < SETS; n++) {
            if (ck + n >= chunks) break;                  // uniform
            fetch(x[(n + SETS - 1) % SETS], ck + n + SETS - 1);
            take(x[n], ck + n);
        }
    if (j < a.vdim)
#pragma unroll
        for (int i = 0; i < TPW; i++)
#pragma unroll
            for (int v = 0; v < 4; v++) {
                const int d = d0 + 16 * i + v;
                if (d < a.dim) Sg[d] = S[i][v];
            }
}

// The last `taps` inputs of this step's convolutions into the state's ring.  grid (ceil(channels / 256), taps, B)
__global__ __launch_bounds__(256) void k_conv_keep(DeltaRows a)
{
    const int ch = blockIdx.x * 256 + threadIdx.x, i = blockIdx.y, b = blockIdx.z, T = a.r.T;
    const int qd = a.KV * a.dim, C = 2 * qd + a.H * a.vdim, t = T - 1 - i;
    if (ch >= C || t < 0) return;
    const int col = ch < qd ? a.o_q + ch : ch < 2 * qd ? a.o_k + ch - qd : a.o_v + ch - 2 * qd;
    a.conv[((size_t)b * a.taps + (a.r.pos + t) % a.taps) * C + ch] = a.cin[(size_t)(b * T + t) * a.ldc + col];
}

// One workgroup per row: mixer output with its head norm and gate | squared ReLU of the shared expert's up product.
__global__ __launch_bounds__(256) void k_cat_rows(CatRows a)
{
    extern __shared__ float row[];                        // [ldk]
    __shared__ float sm[16];
    const int m = xcd_block_row(blockIdx.x, gridDim.x), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    for (int i = a.H * a.vdim + tid; i < a.ldk; i += 256) row[i] = 0.f;
    if (!a.g_out && a.gate) {
#pragma unroll 4
        for (int i = tid; i < a.H * a.vdim; i += 256) {
            const float g = a.gate[(size_t)m * a.ld_gate + i];
            row[i] = a.o[(size_t)m * a.H * a.vdim + i] * (a.gate_silu ? silu(g) : sigmoid(g));
        }
    } else if (a.g_out) {
        // two heads of a wave at a time, up to 128 values of each requested together (longer heads: a second trip)
        for (int h0 = wave * 2; h0 < a.H; h0 += 8) {
            const float *o[2], *gt[2];
            float ss[2] = {0.f, 0.f}, ov[2][2], gv[2][2], wv[2][2];
#pragma unroll
            for (int k = 0; k < 2; k++) {
                const int h = min(h0 + k, a.H - 1);
                o[k] = a.o + ((size_t)m * a.H + h) * a.vdim; gt[k] = a.gate + (size_t)m * a.ld_gate + h * a.vdim;
#pragma unroll
                for (int e = 0; e < 2; e++) {
                    const int d = min(lane + 64 * e, a.vdim - 1);
                    ov[k][e] = o[k][d]; gv[k][e] = gt[k][d]; wv[k][e] = a.g_out[h * a.g_stride + d];
                }
            }
#pragma unroll
            for (int k = 0; k < 2; k++) {
#pragma unroll
                for (int e = 0; e < 2; e++) if (lane + 64 * e < a.vdim) ss[k] += ov[k][e] * ov[k][e];
                for (int d = lane + 128; d < a.vdim; d += 64) ss[k] += o[k][d] * o[k][d];
            }
#pragma unroll
            for (int k = 0; k < 2; k++) {
                const float inv = 1.f / sqrtf(wave_total(ss[k]) / (float)a.vdim + a.eps);
                if (h0 + k >= a.H) break;
                float *out = row + (h0 + k) * a.vdim;
#pragma unroll
                for (int e = 0; e < 2; e++)
                    if (lane + 64 * e < a.vdim) out[lane + 64 * e] = ov[k][e] * inv * wv[k][e] * (a.gate_silu ? silu(gv[k][e]) : sigmoid(gv[k][e]));
                for (int d = lane + 128; d < a.vdim; d += 64) out[d] = o[k][d] * inv * a.g_out[(h0 + k) * a.g_stride + d] * (a.gate_silu ? silu(gt[k][d]) : sigmoid(gt[k][d]));
            }
        }
    } else
#pragma unroll 8
        for (int i = tid; i < a.H * a.vdim; i += 256) row[i] = a.o[(size_t)m * a.H * a.vdim + i];
    __syncthreads();                                      // the zeros are down before the shared part overwrites some
#pragma unroll 4
    for (int i = tid; i < a.shared_ff; i += 256) row[a.o_sh + i] = relu2(a.shared[(size_t)m * a.ld_shared + i]);
    __syncthreads();
    if (a.cat)
        for (int i = tid; i < a.ldk; i += 256) a.cat[(size_t)m * a.ldk + i] = row[i];
    if (a.a16) {
        float mx = 0.f;
        for (int i = tid; i < a.ldk; i += 256) mx = fmaxf(mx, fabsf(row[i]));
        const float s = row_scale_for(block_max(mx, sm));
        store_row_f16(row, a.ldk, a.a16, m, tiled_kb(a.ldk), s);
        if (tid == 0) a.inv[m] = 1.f / s;
    }
}

}  // namespace

// waves of a workgroup of k_delta_chunks and tiles of each
struct ChunkShape { int nw, tpw; int dp() const { return nw * tpw * 16; } };
static ChunkShape chunk_shape(int dim)
{
    const int tiles = (dim + 15) / 16, nw = tiles < 4 ? tiles : 4, per = (tiles + nw - 1) / nw;
    return ChunkShape{nw, per <= 1 ? 1 : per <= 2 ? 2 : 4};
}
int delta_chunks(int T) { return (T + CT - 1) / CT; }
int delta_padded_dim(int dim) { return chunk_shape(dim).dp(); }

void launch_delta_inputs(const DeltaRows &a)
{
    const dim3 grid((a.KV + (a.H * a.vdim + 63) / 64 + 3) / 4, (a.r.T + TW - 1) / TW, a.r.B);
    if (a.dim <= 64) LAUNCH(k_delta_inputs<1>, grid, dim3(256), 0, a);
    else if (a.dim <= 128) LAUNCH(k_delta_inputs<2>, grid, dim3(256), 0, a);
    else LAUNCH(k_delta_inputs<4>, grid, dim3(256), 0, a);
    const int DP = delta_padded_dim(a.dim);
    LAUNCH(k_delta_prepare, dim3(a.H, delta_chunks(a.r.T), a.r.B), dim3(256), (size_t)(3 * CT * (DP + 4) + 2 * CT * 17 + CT) * sizeof(float), a, DP);
}

void launch_delta_scan(const DeltaRows &a)
{
    const ChunkShape cs = chunk_shape(a.dim);
    const dim3 grid((a.vdim + 15) / 16, a.H, a.r.B), block(64 * cs.nw);
    const int chunks = delta_chunks(a.r.T);
#define CHUNKS(T_, S_, N_) LAUNCH((k_delta_chunks<T_, S_, N_>), grid, block, 0, a, cs.dp(), chunks)
    if (cs.tpw == 2) CHUNKS(2, 4, 4); else if (cs.tpw == 4) CHUNKS(4, 2, 4);
    else if (cs.nw == 1) CHUNKS(1, 4, 1); else if (cs.nw == 2) CHUNKS(1, 4, 2); else if (cs.nw == 3) CHUNKS(1, 4, 3); else CHUNKS(1, 4, 4);
#undef CHUNKS
    const int C = 2 * a.KV * a.dim + a.H * a.vdim;
    LAUNCH(k_conv_keep, dim3((C + 255) / 256, a.taps, a.r.B), dim3(256), 0, a);
}

void launch_cat_rows(const CatRows &a, int rows) { LAUNCH(k_cat_rows, dim3(rows), dim3(256), (size_t)a.ldk * 4, a); }

}  // namespace lmhip
