// Launches of stack_decode.hip: one token of one sequence through a layer of a model described layer by layer.
#pragma once
#include "stack.h"

namespace lmhip {

// the experts of a layer; top == 0: none
struct DecodeMoe {
    const float *x, *g; int D, Dp; float eps;            // residual and norm weight: the normed vector is formed again
    const float *z; int E, top;                          // router logits
    int *idx; float *w;
    const half_t *up, *down; int up_rows, down_rows, ff, ffp;
    float *act;                                          // [top][ffp]
};

struct DecodeDelta {
    DeltaRows a;                                         // r = {1, 1, pos}
    const half_t *a2, *g2; int lda2, ldg2, o_g;          // per channel: second low-rank products; o_g: gate (or its first product) in cin
    float *gate;                                         // [H * vdim]: the gate as a factor
};

struct DecodeOut {
    CatRows cat;                                         // gate: factors as k_delta_decode leaves them
    const half_t *out; float *x, *y; int D;               // y: the sum goes there instead of onto x
};

constexpr size_t DECODE_LDS = 152 * 1024;
bool decode_fits(int ldk, int top, int ffp, int Dp);
void launch_delta_decode(const DecodeDelta &s, const DecodeMoe &e);
void launch_latent_decode(const LatentRows &a, const DecodeMoe &e);
void launch_out_decode(const DecodeOut &a, const DecodeMoe &e);

}  // namespace lmhip
