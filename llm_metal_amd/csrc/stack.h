// A decoder described layer by layer: every layer names its mixer (gated delta rule with one decay per head or per key
// channel, latent attention, grouped attention inside chunks of positions, mLSTM) and its feed-forward (mixture of experts,
// dense, or none).  Either one norm feeds both and their sum joins the residual, or each sublayer has a norm ahead of it
// and another behind it.  This header is the configuration, the weights as the kernels read them, what a sequence keeps
// between steps, and the launches.
// The steps themselves are driven by the generation state (inference.hip) like those of the other models.
#pragma once
#include "backend.h"
#include "devutil.h"
#include "gemm.h"
#include "../../include/loader_hip.h"
#include <string>
#include <vector>

namespace lmhip {

// ---------------------------------------------------------------- configuration (config.json)

enum MixerKind { MIX_DELTA, MIX_CHANNEL_DELTA, MIX_LATENT, MIX_GROUPED, MIX_MLSTM };
// NORM_SHARED: one layer norm per layer, x += mixer(h) + ff(h).  NORMS_AROUND: RMS norms, x += m post(sublayer(pre(x))) twice.
enum NormPlace { NORM_SHARED, NORMS_AROUND };

// Rotary angles per position of `dims` / 2 pairs: base^(-2i / dims), with factor > 0 stretched for wavelengths above
// original / low, kept below original / high, mixed in between.
struct Rotation {
    int dims = 0;
    double base = 0.0, factor = 0.0, low = 0.0, high = 0.0, original = 0.0;
    bool operator==(const Rotation &o) const
    {
        return dims == o.dims && base == o.base && factor == o.factor && low == o.low && high == o.high && original == o.original;
    }
    std::vector<double> frequencies() const;
};

struct LayerConfig {
    int mixer = MIX_DELTA;
    int heads = 0, dim = 0, vdim = 0;
    int kv_heads = 0, taps = 0;                          // delta rule
    int rot_dim = 0, kv_rank = 0, window = 0;            // latent attention (rot.dims: how many of the rot_dim turn)
    Rotation rot;                                        // both attentions
    float scale = 0.f;
    int chunk = 0, kv_from = -1;                         // grouped attention: positions per chunk; layer whose keys and values are read (-1: own)
    float gate_cap = 0.f;                                // mLSTM
    int dense_ff = 0;                                    // dense feed-forward of this width
    int experts = 0, top = 0, ff = 0, shared_ff = 0;     // experts == 0: no feed-forward; shared_ff == 0: no shared expert
};

struct StackConfig {
    int vocab = 0, width = 0;
    float emb_scale = 1.f, eps = 0.f;
    NormPlace norms = NORM_SHARED;
    float residual_mult = 1.f, logit_scale = 1.f;        // NORMS_AROUND
    bool tied = false;                                   // the head is the embedding table
    std::vector<LayerConfig> layers;
};

// config.json inside `path` when that is a directory, else next to it
std::string config_path_of(const char *path);
// false, with the reason in `why`, when the text is not a description this build can run
bool read_stack_config(const std::string &json_text, ModelType type, StackConfig &out, std::string &why);

// ---------------------------------------------------------------- weights

// Row-major weight matrix, F16 or fp32 by the state's precision; columns padded with zeros to a multiple of 8, so that
// every row starts on 16 bytes and the padded entries of the vectors (zero too) add nothing.
struct StackMat {
    MetalBuf *buf = nullptr;
    int rows = 0, cols = 0;
};
inline int pad8(int n) { return (n + 7) & ~7; }

struct StackLayer {
    LayerConfig c;
    MetalBuf *g_norm = nullptr;                          // [width padded]
    // One product serves everything that reads the normed vector; each part starts at a multiple of four rows.
    //   delta: q | k | v | b | a (or a1) | g (or g1);  latent: q | dkv;  then router | shared up
    //   grouped: q | k | v (its own only) | g;  mLSTM: q | k | v | g | i | f
    StackMat in;
    int o_q = 0, o_k = 0, o_v = 0, o_b = 0, o_a = 0, o_g = 0, o_dkv = 0, o_router = 0, o_shared = 0, o_i = 0, o_f = 0;
    MetalBuf *b_in = nullptr, *b_out = nullptr;          // fp32 biases of both products by output row (zeros where there is none)
    // norms behind the sublayers and ahead of the feed-forward; those behind carry the residual's factor
    MetalBuf *g_post = nullptr, *g_ff = nullptr, *g_ff_post = nullptr;
    StackMat ff_up, ff_down;                             // dense feed-forward [pad8(ff), D], [Dp, ff]
    int rank_a = 0, rank_g = 0;                          // per-channel decay: widths of the two low-rank products
    // One product for everything added to the residual by the dense part: columns [mixer output | shared activation]
    StackMat out;
    int hv = 0, o_sh = 0;                                // width of the mixer output; column where the shared activation starts
    MetalBuf *conv = nullptr, *a_exp = nullptr, *dt_bias = nullptr, *g_out = nullptr;   // fp32: filters [channels][taps], exp(A_log), bias, head norm
    StackMat a2, g2;
    MetalBuf *g_c = nullptr, *rope = nullptr;            // latent norm weight; (cos, sin) [max_seq][rot_dims / 2]
    StackMat ukv;                                        // [heads * dim | heads * vdim, rank]: key and value projections
    StackMat up, down;                                   // experts one after the other: [E * up_rows, width], [E * down_rows, ff]
    int up_rows = 0, down_rows = 0;                      // ff and width padded to the 32 rows of a tile
    int channels() const { return 2 * c.kv_heads * c.dim + c.heads * c.vdim; }
    bool delta() const { return c.mixer == MIX_DELTA || c.mixer == MIX_CHANNEL_DELTA; }
};

struct LayerStack {
    StackConfig cfg;
    int f32 = 0;                                         // weights and products in 32-bit; else F16 weights
    int D = 0, Dp = 0, V = 0, max_seq = 0;
    std::vector<StackLayer> layers;
    StackMat head;
    MetalBuf *g_final = nullptr, *emb = nullptr;         // emb: fp32 [V][D]
    std::vector<MetalBuf *> ropes;                       // the distinct rotation tables
};

// NULL, with a message, when a tensor is missing or mis-shaped or the weights do not fit F16
LayerStack *stack_load(ModelFile *f, const StackConfig &cfg, int f32, int max_seq);
void stack_free(LayerStack *st);

// ---------------------------------------------------------------- what sequences keep, and a run's scratch

// The (row, choice) pairs sorted by expert, each expert's share padded to whole blocks of 128 rows, so that every expert's
// weights meet all their rows in one product.
struct MoeGroups {
    int tiles;                                           // blocks of 128 rows at most
    int *count;                                          // [E]
    int *of;                                             // [tiles]: expert of a block, -1: no rows; then how many have rows
    int *src;                                            // [tiles * 128]: row of the step, -1: padding
    int *pos;                                            // [rows][top]: where the pair's result lies
};
struct StackRun {
    int B = 0, rows = 0;                                 // sequences; token rows the scratch holds
    // per layer.  delta: state [B][heads][vdim][dim] and the last `taps` inputs of the convolutions [B][taps][channels];
    // latent: ring of (latent | rotated key) rows [B][ring][row width].  Row of position p: p % taps, p % ring.
    // Nothing is cleared between sequences: what lies before position 0 is never read.
    // grouped: rings of rotated keys [B][kv_heads][ring][dim padded to 4] and of values; a layer that reads another's has
    // none.  mLSTM: S [B][heads][vdim][dim padded to 4] and, in two slots that alternate with the parity of the position,
    // the normaliser [2][B][heads][dim padded] and the running maximum [2][B][heads].
    struct Layer { MetalBuf *S = nullptr, *conv = nullptr, *ring = nullptr, *vring = nullptr, *n = nullptr, *m = nullptr; int ring_rows = 0; };
    std::vector<Layer> layers;
    MetalBuf *x2 = nullptr;                              // the residual's other place (fused steps of NORMS_AROUND)
    float *xr = nullptr;                                 // where the fused steps left it
    const float *post_g = nullptr, *post_b = nullptr;    // NORMS_AROUND: norm weight and bias of the sum that waits in cout
    MetalBuf *tok = nullptr, *want = nullptr;
    int *tok_host = nullptr, *want_host = nullptr;       // pinned; tok_host [B * max_seq], each portion in its own place
    MetalBuf *x = nullptr, *h = nullptr, *cin = nullptr, *cat = nullptr, *cout = nullptr;
    MetalBuf *a16 = nullptr, *inv = nullptr;             // F16 operand of a product and its row factors: the normed rows
    MetalBuf *b16 = nullptr, *binv = nullptr;            // the same of every other product
    MetalBuf *aux = nullptr;                             // the mixer's intermediates
    MetalBuf *route_idx = nullptr, *route_w = nullptr, *act = nullptr, *ymoe = nullptr;
    MetalBuf *moe_tab = nullptr, *moe_a16 = nullptr, *moe_inv = nullptr, *moe_up = nullptr, *moe_act = nullptr, *moe_y = nullptr;   // grouped experts
    MetalBuf *lat_a16 = nullptr, *lat_inv = nullptr, *lat_kv = nullptr, *lat_frags = nullptr;   // prompt attention: expanded keys and values
    int tok_end = 0;                                     // end of the positions whose tokens have been put there
    int moe_rows = 0;                                    // rows those hold
    int T = 0, pending = 0;                              // tokens per sequence of the last step; its last layer's sum still waits in cout (1) and ymoe (2) or moe_y (4, by `groups`)
    bool fused = false, one = false;                     // single tokens take the fused steps; the last step was one
    MoeGroups groups{};
    int groups_top = 0;
};
StackRun *stack_run_create(const LayerStack *st, int B);
void stack_run_free(StackRun *r);
// most tokens per sequence that one call of stack_forward takes
int stack_portion(const StackRun *r);

// One step: T tokens of each of the run's sequences, tokens[b * T + t] entering sequence b at position pos + t (a host
// array).  A sequence begins at pos 0; any other pos continues where the run's steps before it ended.
void stack_forward(LayerStack *st, StackRun *r, const int *tokens, int T, int pos);
// Logits of rows of the last step (b * T + t) into logits [n][V] on the device: the rows listed in `want` (host array, at
// most STACK_WANT of them; the stream must be synchronised before the next call), or with NULL the last token of each
// sequence.
constexpr int STACK_WANT = 64;
void stack_logits(LayerStack *st, StackRun *r, const int *want, int n, float *logits);

// ---------------------------------------------------------------- launches (rows: B * T tokens, row m = b * T + t)

struct Rows { int B, T, pos; int n() const { return B * T; } };

// norm.hip: x[src] += cout[src] + ymoe[src] (either may be null), kept in x when `keep`; then layer norm with weight g,
// written as the tiled F16 operand a16 with its row factors inv (when a16) and / or as fp32 h [rows][Dp] (when h).
// src = want[m] when `want`, else m * step + first.
struct NormRows {
    float *x; const float *cout, *ymoe;
    const float *g; half_t *a16; float *inv, *h;
    const int *want;
    int step, first, D, Dp, keep; float eps;
    // grouped experts: instead of ymoe the sum over s of route_w[row][s] * moe_y[moe_pos[row][s]]
    const float *moe_y, *route_w; const int *moe_pos; int top;
};
void launch_norm_rows(const NormRows &a, int rows);
// The same where norms lie around the sublayers: y = cout + post_b, x += y / rms(y) * post_g (cout null: x as it is), kept
// in x when `keep`; then RMS norm with weight g.
struct AroundRows {
    float *x; const float *cout, *post_b, *post_g;
    const float *g; half_t *a16; float *inv, *h;
    const int *want;
    int step, first, D, Dp, keep; float eps;
};
void launch_norms_around(const AroundRows &a, int rows);
// tanh-GELU of up rows [rows][ld] (n columns, the rest of K zero) as the operand a16 with inv, or (exact) as fp32 h [rows][K]
struct ActRows { const float *up; int ld, n, K; half_t *a16; float *inv, *h; };
void launch_gelu_rows(const ActRows &a, int rows);
void launch_embed_rows(const float *emb, const int *tok, float scale, float *x, int D, int Dp, int rows);
constexpr int STACK_FEW = 32;
void launch_embed_few(const float *emb, const int *tok, float scale, float *x, int D, int Dp, int rows);   // tok: host array of at most STACK_FEW

// gemm_f32.hip: C[m][n] = sum_k A[m][k] W[n][k], fp32 throughout
void launch_gemm_f32(const float *A, int lda, const float *W, int ldw, float *C, int ldc, int M, int N, int K);

// delta.hip
struct DeltaRows {
    Rows r;
    int H, KV, dim, vdim, taps, per_channel;
    const float *cin; int ldc, o_q, o_k, o_v, o_b, o_a;  // the input product
    const float *filters, *a_exp, *dt_bias;
    float *conv, *S;                                     // state
    float *q, *k, *v;                                    // intermediates: [rows][KV][dim] x 2, [rows][H][vdim]
    float *kd, *qd, *ku, *gc, *mb;                       // per chunk of tokens and head (delta.hip)
    const float *a2;                                     // per channel: W_a2 (W_a1 h) [rows][H * dim]
    float *o;                                            // [rows][H][vdim]
};
int delta_chunks(int T);                                 // chunks of a sequence's T tokens
int delta_padded_dim(int dim);
constexpr int DELTA_CHUNK = 16;
void launch_delta_inputs(const DeltaRows &a);            // convolutions and unit norms, then what the chunks need ahead
void launch_delta_scan(const DeltaRows &a);              // the recurrence; also moves the convolution's last inputs into the state

// The operand of the output product: mixer output (head norm and gate applied when g_out) | squared-ReLU of the shared
// up product, as fp32 cat [rows][ldk] and / or as a16 with inv
struct CatRows {
    const float *o; int H, vdim;                         // mixer output [rows][H * vdim]
    const float *g_out, *gate; int ld_gate, gate_silu; float eps;   // head norm weight (either may be null), gate rows (silu or sigmoid)
    int g_stride;                                        // from one head's norm weight to the next (0: one for all)
    const float *shared; int ld_shared, shared_ff, o_sh; // shared up rows
    float *cat; half_t *a16; float *inv; int ldk;
};
void launch_cat_rows(const CatRows &a, int rows);

// latent.hip
struct LatentRows {
    Rows r;
    int H, dim, rot, vdim, rank, window, ring_rows, rot_dims;
    float scale, eps;
    const float *cin; int ldc, o_q, o_dkv;
    const float *g_c; const float2 *rope;
    float *ring;                                         // [B][ring_rows][w], w = both parts padded to 8
    float *q;                                            // absorbed query [rows][H][w]
    float *part_o, *part_ml;                             // slices (scratch of the launch)
    float *o;                                            // [rows][H * vdim]
    int f32; const void *ukv; int ldu;                   // projections (keys, then values) and their row stride
};
void launch_latent_cache(const LatentRows &a);           // latent norm and key rotation into the ring
void launch_latent_attend(const LatentRows &a);          // any number of rows, over the latents themselves
struct LatentSlices { int keys, n, rows; };              // keys per workgroup, slices of a row's keys, rows per launch
LatentSlices latent_slices(const LatentRows &a);
void latent_partials(LatentRows &a, const LatentSlices &s);
void launch_latent_slices(const LatentRows &a, const LatentSlices &s, int m0, int nr);   // behind the absorbed queries: attention and values

// latent_prompt.hip: many rows of 16-bit precision with keys and values expanded once per step.  The step's visible keys
// are positions first .. pos + T - 1; kv holds W_uk c | W_uv c of them, [B][n_keys][H * (dim + vdim)].
bool latent_prompt_fits(const LatentRows &a);            // head sizes that kernel is built for, rows enough to pay
int latent_prompt_first(const LatentRows &a);
inline int latent_prompt_keys(const LatentRows &a) { return a.r.pos + a.r.T - latent_prompt_first(a); }
size_t latent_prompt_frag_halfs(const LatentRows &a, int B, int n_keys);
void launch_latent_operand(const LatentRows &a, half_t *a16, float *inv);        // the visible latents as a product's operand
void launch_latent_prompt(const LatentRows &a, const float *kv, half_t *frags);

// group_attn.hip: queries of H heads over G heads of keys; position i sees the positions of its chunk up to itself
struct GroupRows {
    Rows r;
    int H, G, dim, vdim, chunk, ring_rows, rot_dims, own; // own: this layer writes the rings
    float scale;
    const float *cin, *bias; int ldc, o_q, o_k, o_v, o_g; // the input product and its biases
    const float2 *rope;
    float *kring, *vring;
    float *part_o, *part_ml;                             // slices (scratch of the launch)
    float *o;                                            // [rows][H * vdim]
    int gated;                                           // single-token steps: o times sigmoid of the gate
};
void launch_group_cache(const GroupRows &a);             // rotated keys and values into the rings
void launch_group_attend(const GroupRows &a);            // any number of rows in fp32; a step of one token also writes the rings
// group_prompt.hip: many rows in 16-bit precision on the matrix cores, over the rings
bool group_prompt_fits(const GroupRows &a);
inline int group_prompt_first(const GroupRows &a) { return a.r.pos / a.chunk * a.chunk; }
size_t group_prompt_frag_halfs(const GroupRows &a, int B, int n_keys);
void launch_group_prompt(const GroupRows &a, half_t *frags);

// mlstm.hip
constexpr int MLSTM_CHUNK = 64;
struct MlstmRows {
    Rows r;
    int H, dim, vdim; float cap;
    const float *cin, *bias; int ldc, o_q, o_k, o_v, o_g, o_i, o_f;
    float *S, *n, *m;                                    // state
    // prompts: per (sequence, head) and token the parts of the gates, per chunk its decay, the state and the
    // normaliser ahead of it and the pair products
    float2 *u, *w; float *cf, *wk, *em, *qf, *gk, *Sc, *P;
    float *o;                                            // [rows][H * vdim]
    float *gate;                                         // single-token steps: the output gate as a factor, when wanted
};
inline int mlstm_chunks(int T) { return (T + MLSTM_CHUNK - 1) / MLSTM_CHUNK; }
inline size_t mlstm_state_floats(int dim, int vdim) { return (size_t)((vdim + 15) / 16 * 256 + 64) * ((dim + 15) / 16); }   // of one head ahead of a chunk
inline int pad4(int n) { return (n + 3) & ~3; }
void launch_mlstm(const MlstmRows &a);

// norm.hip: (cos, sin) of position * frequency, [max_seq][frequencies]
void launch_rope_table(float2 *tab, int max_seq, const std::vector<double> &freqs);

// moe.hip
struct MoeRows {
    int rows, E, top, ff, ffp, D, Dp, f32;
    int up_rows, down_rows;                              // rows from one expert to the next
    const float *z; int ldz;                             // router logits
    int *idx; float *w;                                  // [rows][top]
    const float *h;                                      // [rows][Dp]
    const void *up, *down;
    float *act;                                          // [rows][top][ffp]
    float *y;                                            // [rows][Dp]
};
void launch_route(const MoeRows &a);
void launch_experts_per_row(const MoeRows &a);           // each row reads its own experts

int moe_group_tiles(int rows, int top, int E);
size_t moe_group_ints(int rows, int top, int E);
MoeGroups moe_groups_at(int *base, int rows, int top, int E);
void launch_moe_groups(const MoeRows &a, const MoeGroups &g);
// rows of the tiled operand a16 (K columns, factors inv) gathered into the groups' order
void launch_moe_gather(const MoeGroups &g, const half_t *a16, const float *inv, half_t *out16, float *out_inv, int K);
// squared ReLU of [tiles * 128][ld] as the next product's operand of K columns (n of them real)
void launch_moe_act(const MoeGroups &g, const float *up, int ld, int n, half_t *out16, float *out_inv, int K);

}  // namespace lmhip
