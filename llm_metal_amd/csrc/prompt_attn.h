// Device code of attention over many rows on the matrix cores, shared by the kinds of attention that lay their keys and
// values out as fragments: blocks of 32 keys of one head, [NJ + 2 NDB fragments][64 lanes][8 F16].
//   K fragment j: lane -> key lane & 31, dimensions 16 j + 8 (lane >> 5) .. + 7.  V fragment (db, u): lane -> value column
//   32 db + (lane & 31), the keys that lane half holds of the score tile's rows 8 u .. 8 u + 7.
// A workgroup of four waves takes 128 queries of a head, a wave 32 of them; key blocks pass through LDS, the next one on its
// way while one is multiplied.  S^T = K Q^T leaves a query's scores in one lane pair, the running softmax needs one
// exchange, and the weights are already the operand of O^T += V^T P^T.  Scores, running maximum and sums are fp32.
#pragma once
#include "devutil.h"
#include "lds_copy.h"

namespace lmhip {

// keys (by index) that the queries of one wave see
struct PromptSpan {
    bool live;                           // the wave has queries
    int lo, last;                        // of this lane's query
    int w_lo, w_hi;                      // lowest and highest key that any query of the wave sees
    int all_lo, all_hi;                  // keys all_lo .. all_hi are seen by all of them
    int kb0, kb1;                        // key blocks the workgroup goes through
};

// `src`: the head's fragments, this lane's place in them.  O: columns of the value sum of this lane's query, 32 i +
// 8 (v >> 2) + 4 (lane >> 5) + (v & 3); they are to be divided by l_run.
template <int NJ, int NDB>
__device__ __forceinline__ void prompt_attend(const half8 (&qf)[NJ], const uint4 *src, const PromptSpan &sp, uint4 *buf0, uint4 *buf1,
                                              float16v (&O)[NDB], float &l_run)
{
    constexpr int NF = NJ + 2 * NDB;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, hh = lane >> 5;
#pragma unroll
    for (int i = 0; i < NDB; i++)
#pragma unroll
        for (int v = 0; v < 16; v++) O[i][v] = 0.f;
    float m_run = -1e30f;
    l_run = 0.f;
    auto request = [&](int kb, uint4 *buf) __attribute__((always_inline)) {
#pragma unroll
        for (int f = 0; f < (NF + 3) / 4; f++)
            if (wave + 4 * f < NF) copy_to_lds_1k(src + ((size_t)kb * NF + wave + 4 * f) * 64, buf + (wave + 4 * f) * 64);
    };
    auto step = [&](int kb, const uint4 *cur) __attribute__((always_inline)) {
        const int k0 = kb * 32;
        if (!sp.live || k0 > sp.w_hi || k0 + 31 < sp.w_lo) return;
        float16v s;
#pragma unroll
        for (int v = 0; v < 16; v++) s[v] = 0.f;
#pragma unroll
        for (int j = 0; j < NJ; j++) s = __builtin_amdgcn_mfma_f32_32x32x16_f16(__builtin_bit_cast(half8, cur[j * 64 + lane]), qf[j], s, 0, 0, 0);
        if (k0 + 31 > sp.all_hi || k0 < sp.all_lo) {      // a key of the block is hidden from some query of the wave
#pragma unroll
            for (int v = 0; v < 16; v++) {
                const int k = k0 + 8 * (v >> 2) + 4 * hh + (v & 3);
                if (k > sp.last || k < sp.lo) s[v] = -INFINITY;
            }
        }
        float mx = s[0];
#pragma unroll
        for (int v = 1; v < 16; v++) mx = fmaxf(mx, s[v]);
        mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
        const float m_new = fmaxf(m_run, mx);
        if (__any(m_new > m_run)) {
            const float alpha = exp2f(m_run - m_new);
            l_run *= alpha;
#pragma unroll
            for (int i = 0; i < NDB; i++)
#pragma unroll
                for (int v = 0; v < 16; v++) O[i][v] *= alpha;
            m_run = m_new;
        }
        half8 pf[2];
#pragma unroll
        for (int v = 0; v < 16; v++) {
            const float e = __builtin_amdgcn_exp2f(s[v] - m_run);
            l_run += e;
            pf[v >> 3][v & 7] = (half_t)e;
        }
#pragma unroll
        for (int i = 0; i < NDB; i++)
#pragma unroll
            for (int u = 0; u < 2; u++)
                O[i] = __builtin_amdgcn_mfma_f32_32x32x16_f16(__builtin_bit_cast(half8, cur[(NJ + 2 * i + u) * 64 + lane]), pf[u], O[i], 0, 0, 0);
    };
    request(sp.kb0, buf0);
    FA_WAIT_AND_BARRIER();
    for (int kb = sp.kb0; kb <= sp.kb1; kb += 2) {
        if (kb + 1 <= sp.kb1) request(kb + 1, buf1);
        step(kb, buf0);
        FA_WAIT_AND_BARRIER();
        if (kb + 1 > sp.kb1) break;
        if (kb + 2 <= sp.kb1) request(kb + 2, buf0);
        step(kb + 1, buf1);
        FA_WAIT_AND_BARRIER();
    }
    l_run += __shfl_xor(l_run, 32, WAVE);
}

// a lane's query row divided by its weight sum, columns below vdim
template <int NDB>
__device__ __forceinline__ void prompt_store(const float16v (&O)[NDB], float l_run, float *out, int vdim)
{
    const float inv = 1.f / l_run;
    const int hh = (threadIdx.x & 63) >> 5;
    const bool vec = vdim % 4 == 0;                      // rows of a multiple of four columns start on 16 bytes
#pragma unroll
    for (int i = 0; i < NDB; i++)
#pragma unroll
        for (int v = 0; v < 16; v += 4) {
            const int d = 32 * i + 8 * (v >> 2) + 4 * hh;
            if (vec) { if (d < vdim) *reinterpret_cast<float4 *>(out + d) = make_float4(O[i][v] * inv, O[i][v + 1] * inv, O[i][v + 2] * inv, O[i][v + 3] * inv); }
            else
#pragma unroll
                for (int e = 0; e < 4; e++) if (d + e < vdim) out[d + e] = O[i][v + e] * inv;
        }
}

}  // namespace lmhip
