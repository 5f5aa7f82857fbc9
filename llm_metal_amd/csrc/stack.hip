// A layer-by-layer model on the device: weights from the checkpoint into the matrices of stack.h, what the sequences of
// a run keep, and one step over any number of tokens.  The generation state (inference.hip) owns both and drives them.
#include "stack.h"
#include "rows.h"
#include "stack_decode.h"

#include <algorithm>
#include <math.h>
#include <string.h>

namespace lmhip {

// loader.hip
bool model_file_place(ModelFile *f, const char *name, int rows, int cols, MetalBuf *dst, int f32, size_t elem_off, int ld, int *overflow);

namespace {

MetalBuf *fbuf(size_t n) { return metal_buf_create(n * sizeof(float)); }
MetalBuf *zeroed(size_t bytes)
{
    MetalBuf *b = metal_buf_create(bytes);
    HIP_CHECK(hipMemsetAsync(dptr(b), 0, bytes, stream()));
    return b;
}

// ---------------------------------------------------------------- loading

struct Loading {
    ModelFile *f;
    LayerStack *st;
    MetalBuf *overflow;                                   // set by a weight that F16 cannot hold
    bool ok = true;

    size_t esize() const { return st->f32 ? 4 : 2; }
    bool shape(const std::string &name, int *rows, int *cols)
    {
        if (model_file_matrix_shape(f, name.c_str(), rows, cols)) return true;
        fprintf(stderr, "[FastGen] tensor '%s' not found or not a matrix\n", name.c_str());
        return ok = false;
    }
    StackMat matrix(int rows, int cols)
    {
        StackMat m;
        m.rows = rows; m.cols = pad8(cols);
        m.buf = zeroed((size_t)m.rows * m.cols * esize());
        return m;
    }
    // tensor [rows, cols] into rows row0 .. of a matrix, its columns from col0 on
    void place(const std::string &name, int rows, int cols, StackMat &m, int row0 = 0, int col0 = 0)
    {
        if (!ok) return;
        ok = model_file_place(f, name.c_str(), rows, cols, m.buf, st->f32, (size_t)row0 * m.cols + col0, m.cols, dptr_as<int>(overflow));
    }
    // fp32 vector (a matrix is taken row by row) times `factor`, padded with zeros
    MetalBuf *vector(const std::string &name, size_t n, size_t padded = 0, float factor = 1.f)
    {
        size_t got = 0;
        float *v = ok ? model_file_load_f32(f, name.c_str(), &got) : nullptr;
        if (!v || got != n) {
            if (ok) fprintf(stderr, "[FastGen] tensor '%s': %zu elements, expected %zu\n", name.c_str(), got, n);
            free(v);
            ok = false;
            return nullptr;
        }
        std::vector<float> p(std::max(n, padded), 0.f);
        for (size_t i = 0; i < n; i++) p[i] = v[i] * factor;
        free(v);
        return metal_buf_from_data(p.data(), p.size() * sizeof(float));
    }
    // fp32 vector into a longer one
    void place_vector(const std::string &name, size_t n, MetalBuf *dst, size_t at)
    {
        MetalBuf *v = vector(name, n);
        if (!v) return;
        std::vector<float> p(n);
        metal_buf_read(v, 0, p.data(), n * sizeof(float));
        metal_buf_write(dst, at * sizeof(float), p.data(), n * sizeof(float));
        metal_buf_free(v);
    }
};

void load_delta(Loading &ld, StackLayer &L, const std::string &p)
{
    const LayerConfig &c = L.c;
    const int D = ld.st->D, qd = c.kv_heads * c.dim, vd = c.heads * c.vdim;
    const bool pc = c.mixer == MIX_CHANNEL_DELTA;
    ld.place(p + "q", qd, D, L.in, L.o_q); ld.place(p + "k", qd, D, L.in, L.o_k); ld.place(p + "v", vd, D, L.in, L.o_v);
    ld.place(p + "b", c.heads, D, L.in, L.o_b);
    ld.place(p + (pc ? "a1" : "a"), pc ? L.rank_a : c.heads, D, L.in, L.o_a);
    ld.place(p + (pc ? "g1" : "g"), pc ? L.rank_g : vd, D, L.in, L.o_g);
    if (pc) {
        L.a2 = ld.matrix(c.heads * c.dim, L.rank_a); ld.place(p + "a2", c.heads * c.dim, L.rank_a, L.a2);
        L.g2 = ld.matrix(vd, L.rank_g); ld.place(p + "g2", vd, L.rank_g, L.g2);
    }
    L.conv = fbuf((size_t)L.channels() * c.taps);
    int at = 0;
    const char *names[3] = {"q.conv", "k.conv", "v.conv"};
    const int chans[3] = {qd, qd, vd};
    for (int i = 0; i < 3 && ld.ok; i++) {
        size_t n = 0;
        float *w = model_file_load_f32(ld.f, (p + names[i]).c_str(), &n);
        if (!w || n != (size_t)chans[i] * c.taps) { fprintf(stderr, "[FastGen] tensor '%s%s' is missing or mis-shaped\n", p.c_str(), names[i]); ld.ok = false; }
        else metal_buf_write(L.conv, (size_t)at * c.taps * sizeof(float), w, n * sizeof(float));
        free(w);
        at += chans[i];
    }
    L.a_exp = ld.vector(p + "A_log", c.heads);
    if (L.a_exp) {
        std::vector<float> a(c.heads);
        metal_buf_read(L.a_exp, 0, a.data(), a.size() * sizeof(float));
        for (float &v : a) v = (float)exp((double)v);
        metal_buf_write(L.a_exp, 0, a.data(), a.size() * sizeof(float));
    }
    L.dt_bias = ld.vector(p + "dt_bias", pc ? (size_t)c.heads * c.dim : c.heads);
    L.g_out = ld.vector(p + "norm", c.vdim);
}

void load_latent(Loading &ld, StackLayer &L, const std::string &p)
{
    const LayerConfig &c = L.c;
    const int D = ld.st->D;
    ld.place(p + "q", c.heads * (c.dim + c.rot_dim), D, L.in, L.o_q);
    ld.place(p + "dkv", c.kv_rank + c.rot_dim, D, L.in, L.o_dkv);
    L.g_c = ld.vector(p + "dkv.norm", c.kv_rank);
    L.ukv = ld.matrix(c.heads * (c.dim + c.vdim), c.kv_rank);
    ld.place(p + "uk", c.heads * c.dim, c.kv_rank, L.ukv);
    ld.place(p + "uv", c.heads * c.vdim, c.kv_rank, L.ukv, c.heads * c.dim);
}

// projection `name` with its bias
void place_biased(Loading &ld, StackLayer &L, const std::string &name, int rows, int at)
{
    ld.place(name, rows, ld.st->D, L.in, at);
    ld.place_vector(name + ".b", rows, L.b_in, at);
}

void load_grouped(Loading &ld, StackLayer &L, const std::string &p)
{
    const LayerConfig &c = L.c;
    place_biased(ld, L, p + "q", c.heads * c.dim, L.o_q);
    if (c.kv_from < 0) {
        place_biased(ld, L, p + "k", c.kv_heads * c.dim, L.o_k);
        place_biased(ld, L, p + "v", c.kv_heads * c.vdim, L.o_v);
    }
    ld.place(p + "g", c.heads * c.vdim, ld.st->D, L.in, L.o_g);
    L.b_out = ld.vector(p + "o.b", ld.st->D, ld.st->Dp);
}

void load_mlstm(Loading &ld, StackLayer &L, const std::string &p)
{
    const LayerConfig &c = L.c;
    const int D = ld.st->D, qd = c.heads * c.dim, vd = c.heads * c.vdim;
    ld.place(p + "q", qd, D, L.in, L.o_q); ld.place(p + "k", qd, D, L.in, L.o_k); ld.place(p + "v", vd, D, L.in, L.o_v);
    ld.place(p + "g", vd, D, L.in, L.o_g);
    place_biased(ld, L, p + "i", c.heads, L.o_i);
    place_biased(ld, L, p + "f", c.heads, L.o_f);
    L.g_out = ld.vector(p + "norm", vd);
}

void load_layer(Loading &ld, StackLayer &L, int i)
{
    const LayerConfig &c = L.c;
    const int D = ld.st->D;
    const std::string p = "l" + std::to_string(i) + ".", mix = p + "mix.", mlp = p + "mlp.";
    L.g_norm = ld.vector(p + "norm1", D, ld.st->Dp);
    // the parts of the input product
    int at = 0, cols = 0;
    auto part = [&](int &o, int n) { o = at; at = pad4(at + n); };
    if (L.delta()) {
        const int qd = c.kv_heads * c.dim, vd = c.heads * c.vdim;
        const bool pc = c.mixer == MIX_CHANNEL_DELTA;
        if (pc && (!ld.shape(mix + "a1", &L.rank_a, &cols) || !ld.shape(mix + "g1", &L.rank_g, &cols))) return;
        part(L.o_q, qd); part(L.o_k, qd); part(L.o_v, vd); part(L.o_b, c.heads);
        part(L.o_a, pc ? pad8(L.rank_a) : c.heads);       // read as rows of pad8 columns by the second low-rank product
        part(L.o_g, pc ? pad8(L.rank_g) : vd);
    } else if (c.mixer == MIX_LATENT) {
        part(L.o_q, c.heads * (c.dim + c.rot_dim)); part(L.o_dkv, c.kv_rank + c.rot_dim);
    } else if (c.mixer == MIX_GROUPED) {
        part(L.o_q, c.heads * c.dim);
        if (c.kv_from < 0) { part(L.o_k, c.kv_heads * c.dim); part(L.o_v, c.kv_heads * c.vdim); }
        part(L.o_g, c.heads * c.vdim);
    } else {
        part(L.o_q, c.heads * c.dim); part(L.o_k, c.heads * c.dim); part(L.o_v, c.heads * c.vdim); part(L.o_g, c.heads * c.vdim);
        part(L.o_i, c.heads); part(L.o_f, c.heads);
    }
    if (c.experts) { part(L.o_router, c.experts); if (c.shared_ff) part(L.o_shared, c.shared_ff); }
    L.in = ld.matrix(at, D);
    L.hv = c.heads * c.vdim;
    L.o_sh = pad8(L.hv);
    L.out = ld.matrix(ld.st->Dp, L.o_sh + c.shared_ff);
    if (ld.st->cfg.norms == NORMS_AROUND) {
        const float m = ld.st->cfg.residual_mult;
        L.b_in = zeroed((size_t)at * sizeof(float));
        L.g_post = ld.vector(p + "norm1b", D, ld.st->Dp, m);
        if (c.dense_ff) {
            L.g_ff = ld.vector(p + "norm2", D, ld.st->Dp); L.g_ff_post = ld.vector(p + "norm2b", D, ld.st->Dp, m);
            L.ff_up = ld.matrix(pad8(c.dense_ff), D); ld.place(mlp + "up", c.dense_ff, D, L.ff_up);
            L.ff_down = ld.matrix(ld.st->Dp, c.dense_ff); ld.place(mlp + "down", D, c.dense_ff, L.ff_down);
        }
    }
    switch (c.mixer) {
    case MIX_LATENT: load_latent(ld, L, mix); break;
    case MIX_GROUPED: load_grouped(ld, L, mix); break;
    case MIX_MLSTM: load_mlstm(ld, L, mix); break;
    default: load_delta(ld, L, mix);
    }
    ld.place(mix + "o", D, L.hv, L.out);
    if (!c.experts) return;
    ld.place(mlp + "router", c.experts, D, L.in, L.o_router);
    if (c.shared_ff) {
        ld.place(mlp + "shared.up", c.shared_ff, D, L.in, L.o_shared);
        ld.place(mlp + "shared.down", D, c.shared_ff, L.out, 0, L.o_sh);
    }
    L.up_rows = (c.ff + 31) & ~31; L.down_rows = (ld.st->Dp + 31) & ~31;
    L.up = ld.matrix(c.experts * L.up_rows, D);
    L.down = ld.matrix(c.experts * L.down_rows, c.ff);
    for (int e = 0; e < c.experts && ld.ok; e++) {
        const std::string ex = mlp + "e" + std::to_string(e) + ".";
        ld.place(ex + "up", c.ff, D, L.up, e * L.up_rows);
        ld.place(ex + "down", D, c.ff, L.down, e * L.down_rows);
    }
}

}  // namespace

LayerStack *stack_load(ModelFile *f, const StackConfig &cfg, int f32, int max_seq)
{
    LayerStack *st = new LayerStack();
    st->cfg = cfg; st->f32 = f32; st->D = cfg.width; st->Dp = pad8(cfg.width); st->V = cfg.vocab; st->max_seq = max_seq;
    Loading ld{f, st, zeroed(sizeof(int))};
    std::vector<Rotation> tables;                         // of st->ropes
    st->layers.resize(cfg.layers.size());
    for (size_t i = 0; i < st->layers.size() && ld.ok; i++) {
        StackLayer &L = st->layers[i];
        L.c = cfg.layers[i];
        load_layer(ld, L, (int)i);
        if ((L.c.mixer != MIX_LATENT && L.c.mixer != MIX_GROUPED) || !ld.ok) continue;
        size_t k = 0;
        while (k < tables.size() && !(tables[k] == L.c.rot)) k++;
        if (k == tables.size()) {
            tables.push_back(L.c.rot);
            st->ropes.push_back(metal_buf_create(std::max<size_t>(8, (size_t)max_seq * (L.c.rot.dims / 2) * sizeof(float2))));
            launch_rope_table(dptr_as<float2>(st->ropes[k]), max_seq, L.c.rot.frequencies());
        }
        L.rope = st->ropes[k];
    }
    if (ld.ok) {
        st->g_final = ld.vector("final.norm", st->D, st->Dp, cfg.logit_scale);
        st->head = ld.matrix(st->V, st->D);
        ld.place(cfg.tied ? "embed" : "head", st->V, st->D, st->head);
        st->emb = fbuf((size_t)st->V * st->D);
        if (ld.ok) ld.ok = model_file_place(f, "embed", st->V, st->D, st->emb, 1, 0, st->D, nullptr);
    }
    int over = 0;
    if (ld.ok) metal_buf_read(ld.overflow, 0, &over, sizeof over);
    metal_buf_free(ld.overflow);
    if (over) { fprintf(stderr, "[FastGen] a weight lies outside the F16 range; load the model in 32-bit precision\n"); ld.ok = false; }
    if (!ld.ok) { stack_free(st); return nullptr; }
    return st;
}

void stack_free(LayerStack *st)
{
    if (!st) return;
    for (StackLayer &L : st->layers)
        for (MetalBuf *b : {L.g_norm, L.in.buf, L.out.buf, L.conv, L.a_exp, L.dt_bias, L.g_out, L.a2.buf, L.g2.buf, L.g_c, L.ukv.buf,
                            L.up.buf, L.down.buf, L.b_in, L.b_out, L.g_post, L.g_ff, L.g_ff_post, L.ff_up.buf, L.ff_down.buf}) metal_buf_free(b);
    for (MetalBuf *b : st->ropes) metal_buf_free(b);
    for (MetalBuf *b : {st->head.buf, st->g_final, st->emb}) metal_buf_free(b);
    delete st;
}

// ---------------------------------------------------------------- runs

namespace {

constexpr int PORTION_ROWS = 2048;

// floats of a layer's intermediates for `rows` rows, in the order the step hands them out (each piece a multiple of 4)
struct Aux {
    float *base = nullptr;
    size_t at = 0;
    float *take(size_t n) { float *p = base ? base + at : nullptr; at += (n + 3) & ~(size_t)3; return p; }
};

struct DeltaAux { float *q, *k, *v, *kd, *qd, *ku, *gc, *mb, *a2, *g2, *o; };
DeltaAux delta_aux(Aux &x, const LayerConfig &c, int B, int T)
{
    const size_t rows = (size_t)B * T;
    const bool pc = c.mixer == MIX_CHANNEL_DELTA;
    DeltaAux d{};
    d.q = x.take(rows * c.kv_heads * c.dim); d.k = x.take(rows * c.kv_heads * c.dim); d.v = x.take(rows * c.heads * c.vdim);
    const size_t parts = (size_t)B * delta_chunks(T) * c.heads, dp = delta_padded_dim(c.dim);
    d.kd = x.take(parts * dp * DELTA_CHUNK); d.qd = x.take(parts * dp * DELTA_CHUNK); d.ku = x.take(parts * dp * DELTA_CHUNK);
    d.gc = x.take(parts * dp); d.mb = x.take(parts * 2 * DELTA_CHUNK * DELTA_CHUNK);
    d.a2 = x.take(pc ? rows * c.heads * c.dim : 0); d.g2 = x.take(pc ? rows * c.heads * c.vdim : 0);
    d.o = x.take(rows * c.heads * c.vdim);
    return d;
}

struct LatentAux { float *q, *o; };
LatentAux latent_aux(Aux &x, const LayerConfig &c, size_t rows)
{
    LatentAux d{};
    d.q = x.take(rows * c.heads * (pad8(c.kv_rank) + pad8(c.rot_dim)));
    d.o = x.take(rows * c.heads * c.vdim);
    return d;
}

struct MlstmAux { float2 *u, *w; float *cf, *wk, *em, *qf, *gk, *Sc, *P, *o, *gate; };
MlstmAux mlstm_aux(Aux &x, const LayerConfig &c, int B, int T)
{
    const size_t rows = (size_t)B * T, parts = (size_t)B * c.heads * mlstm_chunks(T), at = parts * MLSTM_CHUNK;
    MlstmAux d{};
    d.o = x.take(rows * c.heads * c.vdim); d.gate = x.take((size_t)B * c.heads * c.vdim);
    if (T == 1) return d;
    d.u = (float2 *)x.take(2 * at); d.w = (float2 *)x.take(2 * at);
    d.cf = x.take(at); d.wk = x.take(at); d.em = x.take(at); d.qf = x.take(at); d.gk = x.take(parts);
    d.Sc = x.take(parts * mlstm_state_floats(c.dim, c.vdim)); d.P = x.take(at * MLSTM_CHUNK);
    return d;
}

// C [M][w.rows] = A x w^T; A as the run's F16 operand (a16, inv) or, in 32-bit, as fp32 rows
void product(const LayerStack *st, const StackMat &w, const half_t *a16, const float *inv, const float *A, int lda, float *C, int M)
{
    const int N = w.rows, K = w.cols;
    if (st->f32) { launch_gemm_f32(A, lda, dptr_as<float>(w.buf), K, C, N, M, N, K); return; }
    const WeightOp op = weight_f16(tiled_weight_of(w.buf, N, K));
    const size_t plane = (size_t)M * N;
    if (use_big_gemm(M, N, K, 0)) {
        const int chunks = big_gemm_chunks(M, N, K, 0);
        if (chunks == 1) { launch_gemm_big(a16, inv, op, C, N, M, N, K); return; }
        float *P = (float *)scratch(SCR_PARTIAL, plane * chunks * sizeof(float));
        const int S = launch_gemm_big(a16, nullptr, op, P, N, M, N, K, chunks, plane);
        launch_reduce_planes(P, S, plane, N, inv, C, M, N);
        return;
    }
    const GemmPlan p = plan_gemm(M, N, K);
    if (p.S == 1) { launch_gemm(a16, inv, op, C, N, 0, M, N, K, p); return; }
    float *P = (float *)scratch(SCR_PARTIAL, plane * p.S * sizeof(float));
    launch_gemm(a16, nullptr, op, P, N, plane, M, N, K, p);
    launch_reduce_planes(P, p.S, plane, N, inv, C, M, N);
}

}  // namespace

StackRun *stack_run_create(const LayerStack *st, int B)
{
    StackRun *r = new StackRun();
    r->B = B;
    r->fused = !st->f32 && B == 1 && st->Dp <= 15360;
    for (const StackLayer &L : st->layers) r->fused = r->fused && decode_fits(L.out.cols, L.c.top, L.down.cols, st->Dp);
    // a ring serves every layer that reads it
    std::vector<int> span(st->layers.size(), 0);
    for (size_t i = 0; i < span.size(); i++) {
        const LayerConfig &c = st->layers[i].c;
        int &s = span[c.kv_from < 0 ? i : c.kv_from];
        s = std::max(s, c.mixer == MIX_LATENT ? c.window : c.chunk);
    }
    r->rows = std::max(1, std::min(PORTION_ROWS / B, st->max_seq)) * B;
    const int portion = r->rows / B;
    size_t n_in = 0, ko = 0, aux = 0, act = 0, top = 0, tab = 0, dense = 0;
    int up_ld = 0, ffp = 0;
    int kmax = st->Dp;
    bool moe = false;
    for (const StackLayer &L : st->layers) {
        const LayerConfig &c = L.c;
        StackRun::Layer k;
        Aux a;
        if (L.delta()) {
            k.S = fbuf((size_t)B * c.heads * c.vdim * c.dim);
            k.conv = fbuf((size_t)B * c.taps * L.channels());
            delta_aux(a, c, B, portion);
            kmax = std::max({kmax, L.a2.cols, L.g2.cols});
        } else if (c.mixer == MIX_MLSTM) {
            k.S = fbuf((size_t)B * c.heads * c.vdim * pad4(c.dim));
            k.n = fbuf((size_t)2 * B * c.heads * pad4(c.dim));
            k.m = fbuf((size_t)2 * B * c.heads);
            mlstm_aux(a, c, B, portion);
        } else {
            k.ring_rows = (int)std::min<long>(st->max_seq, (long)span[c.kv_from < 0 ? r->layers.size() : c.kv_from] - 1 + portion);
            if (c.mixer == MIX_LATENT) {
                k.ring = fbuf((size_t)B * k.ring_rows * (pad8(c.kv_rank) + pad8(c.rot_dim)));
                latent_aux(a, c, r->rows);
            } else {
                if (c.kv_from < 0) {
                    k.ring = fbuf((size_t)B * k.ring_rows * c.kv_heads * pad4(c.dim));
                    k.vring = fbuf((size_t)B * k.ring_rows * c.kv_heads * pad4(c.vdim));
                }
                a.take((size_t)r->rows * c.heads * c.vdim);
            }
        }
        r->layers.push_back(k);
        if (c.dense_ff) {
            n_in = std::max<size_t>(n_in, L.ff_up.rows); kmax = std::max(kmax, L.ff_down.cols);
            ko = std::max<size_t>(ko, L.ff_down.cols); dense = std::max<size_t>(dense, L.ff_down.cols);
        }
        n_in = std::max<size_t>(n_in, L.in.rows); ko = std::max<size_t>(ko, L.out.cols); aux = std::max(aux, a.at);
        if (c.experts) {
            const int tiles = moe_group_tiles(r->rows, c.top, c.experts);
            r->moe_rows = std::max(r->moe_rows, tiles * 128);
            tab = std::max(tab, moe_group_ints(r->rows, c.top, c.experts));
            up_ld = std::max(up_ld, L.up_rows); ffp = std::max(ffp, L.down.cols);
        }
        if (c.experts) { moe = true; top = std::max<size_t>(top, c.top); act = std::max<size_t>(act, (size_t)c.top * pad8(c.ff)); }
    }
    kmax = std::max<int>(kmax, (int)ko);
    r->tok = metal_buf_create((size_t)r->rows * sizeof(int));
    r->want = metal_buf_create(STACK_WANT * sizeof(int));
    HIP_CHECK(hipHostMalloc((void **)&r->tok_host, (size_t)B * st->max_seq * sizeof(int), hipHostMallocDefault));
    HIP_CHECK(hipHostMalloc((void **)&r->want_host, STACK_WANT * sizeof(int), hipHostMallocDefault));
    r->x = fbuf((size_t)r->rows * st->Dp);
    if (st->cfg.norms == NORMS_AROUND) r->x2 = fbuf(st->Dp);
    r->cin = fbuf((size_t)r->rows * n_in);
    r->cout = fbuf((size_t)r->rows * st->Dp);
    r->aux = fbuf(aux);
    r->h = fbuf((size_t)std::max(r->rows, STACK_WANT) * st->Dp);
    if (st->f32) r->cat = fbuf((size_t)r->rows * ko);
    else {
        r->a16 = metal_buf_create(tiled_elems(std::max(r->rows, STACK_WANT), st->Dp) * sizeof(half_t));
        r->b16 = metal_buf_create(tiled_elems(r->rows, kmax) * sizeof(half_t));
        r->inv = fbuf(std::max(r->rows, STACK_WANT));
        r->binv = fbuf(r->rows);
    }
    if (dense) r->act = fbuf(dense);
    if (moe) {
        r->route_idx = metal_buf_create((size_t)r->rows * top * sizeof(int));
        r->route_w = fbuf((size_t)r->rows * top);
        r->act = fbuf((size_t)r->rows * act);
        r->ymoe = fbuf((size_t)r->rows * st->Dp);
        if (!st->f32) {
            r->moe_tab = metal_buf_create(tab * sizeof(int));
            r->moe_a16 = metal_buf_create(tiled_elems(r->moe_rows, st->Dp) * sizeof(half_t));
            r->moe_inv = fbuf((size_t)2 * r->moe_rows);   // of the gathered rows | of the activations
            r->moe_up = fbuf((size_t)r->moe_rows * up_ld);
            r->moe_act = metal_buf_create(tiled_elems(r->moe_rows, ffp) * sizeof(half_t));
            r->moe_y = fbuf((size_t)r->moe_rows * st->Dp);
        }
    }
    return r;
}

void stack_run_free(StackRun *r)
{
    if (!r) return;
    for (StackRun::Layer &k : r->layers) for (MetalBuf *b : {k.S, k.conv, k.ring, k.vring, k.n, k.m}) metal_buf_free(b);
    for (MetalBuf *b : {r->tok, r->want, r->x, r->x2, r->h, r->cin, r->cat, r->cout, r->a16, r->inv, r->b16, r->binv, r->aux, r->route_idx, r->route_w, r->act, r->ymoe,
                        r->moe_tab, r->moe_a16, r->moe_inv, r->moe_up, r->moe_act, r->moe_y, r->lat_a16, r->lat_inv, r->lat_kv, r->lat_frags})
        metal_buf_free(b);
    if (r->tok_host) hipHostFree(r->tok_host);
    if (r->want_host) hipHostFree(r->want_host);
    delete r;
}

int stack_portion(const StackRun *r) { return r->rows / r->B; }

// ---------------------------------------------------------------- the step

namespace {

template <typename T> T *ptr(MetalBuf *b) { return b ? dptr_as<T>(b) : nullptr; }

// the norm ahead of a product over all rows of the step (or, with want / step, some of them), the pending sum added first
void norm(LayerStack *st, StackRun *r, MetalBuf *g, int rows, int keep, bool need_h, const int *want = nullptr, int step = 1, int first = 0)
{
    if (st->cfg.norms == NORMS_AROUND) {
        AroundRows n{};
        n.x = ptr<float>(r->x);
        if (r->pending) { n.cout = ptr<float>(r->cout); n.post_g = r->post_g; n.post_b = r->post_b; }
        n.g = ptr<float>(g); n.a16 = ptr<half_t>(r->a16); n.inv = ptr<float>(r->inv); n.h = st->f32 ? ptr<float>(r->h) : nullptr;
        n.want = want; n.step = step; n.first = first; n.D = st->D; n.Dp = st->Dp; n.keep = keep; n.eps = st->cfg.eps;
        launch_norms_around(n, rows);
        return;
    }
    NormRows n{};
    n.x = ptr<float>(r->x);
    if (r->pending & 1) n.cout = ptr<float>(r->cout);
    if (r->pending & 2) n.ymoe = ptr<float>(r->ymoe);
    if (r->pending & 4) { n.moe_y = ptr<float>(r->moe_y); n.moe_pos = r->groups.pos; n.route_w = ptr<float>(r->route_w); n.top = r->groups_top; }
    n.g = ptr<float>(g); n.a16 = ptr<half_t>(r->a16); n.inv = ptr<float>(r->inv); n.h = need_h || st->f32 ? ptr<float>(r->h) : nullptr;
    n.want = want; n.step = step; n.first = first; n.D = st->D; n.Dp = st->Dp; n.keep = keep; n.eps = st->cfg.eps;
    launch_norm_rows(n, rows);
}

DeltaRows delta_rows(const LayerStack *st, const StackRun *r, const StackLayer &L, const StackRun::Layer &k, const Rows &rows, const DeltaAux &d)
{
    const LayerConfig &c = L.c;
    DeltaRows a{};
    a.r = rows; a.H = c.heads; a.KV = c.kv_heads; a.dim = c.dim; a.vdim = c.vdim; a.taps = c.taps; a.per_channel = c.mixer == MIX_CHANNEL_DELTA;
    a.cin = ptr<float>(r->cin); a.ldc = L.in.rows; a.o_q = L.o_q; a.o_k = L.o_k; a.o_v = L.o_v; a.o_b = L.o_b; a.o_a = L.o_a;
    a.filters = ptr<float>(L.conv); a.a_exp = ptr<float>(L.a_exp); a.dt_bias = ptr<float>(L.dt_bias);
    a.conv = ptr<float>(k.conv); a.S = ptr<float>(k.S);
    a.q = d.q; a.k = d.k; a.v = d.v; a.kd = d.kd; a.qd = d.qd; a.ku = d.ku; a.gc = d.gc; a.mb = d.mb; a.a2 = d.a2; a.o = d.o;
    return a;
}

LatentRows latent_rows(const LayerStack *st, const StackRun *r, const StackLayer &L, const StackRun::Layer &k, const Rows &rows, const LatentAux &d)
{
    const LayerConfig &c = L.c;
    LatentRows a{};
    a.r = rows; a.H = c.heads; a.dim = c.dim; a.rot = c.rot_dim; a.vdim = c.vdim; a.rank = c.kv_rank; a.window = c.window;
    a.ring_rows = k.ring_rows; a.rot_dims = c.rot.dims; a.scale = c.scale; a.eps = st->cfg.eps;
    a.cin = ptr<float>(r->cin); a.ldc = L.in.rows; a.o_q = L.o_q; a.o_dkv = L.o_dkv;
    a.g_c = ptr<float>(L.g_c); a.rope = ptr<float2>(L.rope); a.ring = ptr<float>(k.ring);
    a.q = d.q; a.o = d.o; a.f32 = st->f32; a.ukv = dptr(L.ukv.buf); a.ldu = L.ukv.cols;
    return a;
}

GroupRows group_rows(const LayerStack *st, const StackRun *r, const StackLayer &L, const Rows &rows, float *o)
{
    const LayerConfig &c = L.c;
    const StackRun::Layer &k = r->layers[c.kv_from < 0 ? (size_t)(&L - st->layers.data()) : (size_t)c.kv_from];
    GroupRows a{};
    a.r = rows; a.H = c.heads; a.G = c.kv_heads; a.dim = c.dim; a.vdim = c.vdim; a.chunk = c.chunk; a.ring_rows = k.ring_rows;
    a.rot_dims = c.rot.dims; a.own = c.kv_from < 0; a.scale = c.scale;
    a.cin = ptr<float>(r->cin); a.bias = ptr<float>(L.b_in); a.ldc = L.in.rows; a.o_q = L.o_q; a.o_k = L.o_k; a.o_v = L.o_v; a.o_g = L.o_g;
    a.rope = ptr<float2>(L.rope); a.kring = ptr<float>(k.ring); a.vring = ptr<float>(k.vring); a.o = o;
    return a;
}

MlstmRows mlstm_rows(const StackRun *r, const StackLayer &L, const StackRun::Layer &k, const Rows &rows, const MlstmAux &d)
{
    const LayerConfig &c = L.c;
    MlstmRows a{};
    a.r = rows; a.H = c.heads; a.dim = c.dim; a.vdim = c.vdim; a.cap = c.gate_cap;
    a.cin = ptr<float>(r->cin); a.bias = ptr<float>(L.b_in); a.ldc = L.in.rows;
    a.o_q = L.o_q; a.o_k = L.o_k; a.o_v = L.o_v; a.o_g = L.o_g; a.o_i = L.o_i; a.o_f = L.o_f;
    a.S = ptr<float>(k.S); a.n = ptr<float>(k.n); a.m = ptr<float>(k.m);
    a.u = d.u; a.w = d.w; a.cf = d.cf; a.wk = d.wk; a.em = d.em; a.qf = d.qf; a.gk = d.gk; a.Sc = d.Sc; a.P = d.P; a.o = d.o;
    return a;
}

// mixer output | shared activation of a layer, without the mixer's own part
CatRows cat_rows(const LayerStack *st, const StackRun *r, const StackLayer &L)
{
    const LayerConfig &c = L.c;
    CatRows cat{};
    cat.H = c.heads; cat.vdim = c.vdim; cat.eps = st->cfg.eps; cat.g_out = ptr<float>(L.g_out); cat.gate_silu = c.mixer == MIX_DELTA;
    cat.g_stride = c.mixer == MIX_MLSTM ? c.vdim : 0;
    cat.shared = ptr<float>(r->cin) + L.o_shared; cat.ld_shared = L.in.rows; cat.shared_ff = c.shared_ff; cat.o_sh = L.o_sh;
    cat.cat = ptr<float>(r->cat); cat.a16 = ptr<half_t>(r->b16); cat.inv = ptr<float>(r->binv); cat.ldk = L.out.cols;
    return cat;
}

float *mix_delta(LayerStack *st, StackRun *r, StackLayer &L, StackRun::Layer &k, const Rows &rows, CatRows &cat)
{
    const LayerConfig &c = L.c;
    const int n = rows.n(), ldc = L.in.rows;
    const bool pc = c.mixer == MIX_CHANNEL_DELTA;
    Aux ax{ptr<float>(r->aux)};
    const DeltaAux d = delta_aux(ax, c, rows.B, rows.T);
    const float *cin = ptr<float>(r->cin);
    if (pc) {                                             // the second halves of the two low-rank products
        auto low_rank = [&](const StackMat &w, int col, float *out) {
            if (!st->f32) launch_rows_to_f16(cin + col, ldc, ptr<half_t>(r->b16), ptr<float>(r->binv), n, w.cols);
            product(st, w, ptr<half_t>(r->b16), ptr<float>(r->binv), cin + col, ldc, out, n);
        };
        low_rank(L.a2, L.o_a, d.a2);
        low_rank(L.g2, L.o_g, d.g2);
    }
    const DeltaRows a = delta_rows(st, r, L, k, rows, d);
    launch_delta_inputs(a);
    launch_delta_scan(a);
    cat.gate = pc ? d.g2 : cin + L.o_g; cat.ld_gate = pc ? L.hv : ldc;
    return d.o;
}

float *mix_latent(LayerStack *st, StackRun *r, StackLayer &L, StackRun::Layer &k, const Rows &rows)
{
    const LayerConfig &c = L.c;
    Aux ax{ptr<float>(r->aux)};
    const LatentAux d = latent_aux(ax, c, rows.n());
    const LatentRows a = latent_rows(st, r, L, k, rows, d);
    launch_latent_cache(a);
    if (!latent_prompt_fits(a)) { launch_latent_attend(a); return d.o; }
    const int nk = latent_prompt_keys(a), most = k.ring_rows;            // grown to what any step of this layer needs
    auto room = [&](MetalBuf *&b, size_t bytes) { if (!b || b->size < bytes) { metal_buf_free(b); b = metal_buf_create(bytes); } };
    room(r->lat_a16, tiled_elems(r->B * most, c.kv_rank) * sizeof(half_t));
    room(r->lat_inv, (size_t)r->B * most * sizeof(float));
    room(r->lat_kv, (size_t)r->B * most * L.ukv.rows * sizeof(float));
    room(r->lat_frags, latent_prompt_frag_halfs(a, r->B, most) * sizeof(half_t));
    launch_latent_operand(a, ptr<half_t>(r->lat_a16), ptr<float>(r->lat_inv));
    product(st, L.ukv, ptr<half_t>(r->lat_a16), ptr<float>(r->lat_inv), nullptr, 0, ptr<float>(r->lat_kv), r->B * nk);
    launch_latent_prompt(a, ptr<float>(r->lat_kv), ptr<half_t>(r->lat_frags));
    return d.o;
}

float *mix_grouped(LayerStack *st, StackRun *r, StackLayer &L, const Rows &rows, CatRows &cat)
{
    Aux ax{ptr<float>(r->aux)};
    const GroupRows a = group_rows(st, r, L, rows, ax.take((size_t)rows.n() * L.hv));
    cat.gate = ptr<float>(r->cin) + L.o_g; cat.ld_gate = L.in.rows;
    if (rows.T > 1 && a.own) launch_group_cache(a);
    if (st->f32 || !group_prompt_fits(a)) { launch_group_attend(a); return a.o; }
    const size_t bytes = group_prompt_frag_halfs(a, r->B, a.ring_rows) * sizeof(half_t);
    if (!r->lat_frags || r->lat_frags->size < bytes) { metal_buf_free(r->lat_frags); r->lat_frags = metal_buf_create(bytes); }
    launch_group_prompt(a, ptr<half_t>(r->lat_frags));
    return a.o;
}

float *mix_mlstm(LayerStack *st, StackRun *r, StackLayer &L, StackRun::Layer &k, const Rows &rows, CatRows &cat)
{
    Aux ax{ptr<float>(r->aux)};
    const MlstmRows a = mlstm_rows(r, L, k, rows, mlstm_aux(ax, L.c, rows.B, rows.T));
    cat.gate = ptr<float>(r->cin) + L.o_g; cat.ld_gate = L.in.rows;
    launch_mlstm(a);
    return a.o;
}

// the dense feed-forward over all rows of the step, its sum left waiting
void feed_forward(LayerStack *st, StackRun *r, StackLayer &L, int n)
{
    norm(st, r, L.g_ff, n, 1, false);
    product(st, L.ff_up, ptr<half_t>(r->a16), ptr<float>(r->inv), ptr<float>(r->h), st->Dp, ptr<float>(r->cin), n);
    ActRows act{};
    act.up = ptr<float>(r->cin); act.ld = L.ff_up.rows; act.n = L.c.dense_ff; act.K = L.ff_down.cols;
    act.a16 = ptr<half_t>(r->b16); act.inv = ptr<float>(r->binv); act.h = ptr<float>(r->cat);
    launch_gelu_rows(act, n);
    product(st, L.ff_down, act.a16, act.inv, act.h, act.K, ptr<float>(r->cout), n);
    r->pending = 1; r->post_g = ptr<float>(L.g_ff_post); r->post_b = nullptr;
}

// decoding one sequence with F16 weights and norms around the sublayers: the vector of every product is the residual with
// the sum before it, both normed inside the product's launch; the residual goes back and forth between two places
void decode_layers_around(LayerStack *st, StackRun *r, int pos)
{
    const Rows rows{1, 1, pos};
    float *cin = ptr<float>(r->cin), *cout = ptr<float>(r->cout), *act = ptr<float>(r->act);
    float *at = ptr<float>(r->x), *next = ptr<float>(r->x2);
    NormIn in{};
    in.eps = st->cfg.eps; in.dim = st->D;
    auto product_of = [&](const StackMat &w, MetalBuf *g, float *y, int gelu) {
        in.xr = at; in.g = ptr<float>(g); in.x_out = in.br ? next : nullptr;
        matvec_norms_around(w.buf, in, y, w.rows, w.cols, gelu);
        if (in.br) std::swap(at, next);
    };
    auto leave = [&](MetalBuf *g, MetalBuf *b) { in.br = cout; in.g_br = ptr<float>(g); in.b_br = ptr<float>(b); };
    for (size_t i = 0; i < st->layers.size(); i++) {
        StackLayer &L = st->layers[i];
        product_of(L.in, L.g_norm, cin, 0);
        DecodeOut o{};
        o.cat = cat_rows(st, r, L);
        o.out = ptr<half_t>(L.out.buf); o.y = cout; o.D = st->D;
        Aux ax{ptr<float>(r->aux)};
        if (L.c.mixer == MIX_GROUPED) {
            GroupRows a = group_rows(st, r, L, rows, ax.take(L.hv));
            a.gated = 1;
            launch_group_attend(a);
            o.cat.o = a.o;
        } else {
            const MlstmAux d = mlstm_aux(ax, L.c, 1, 1);
            MlstmRows a = mlstm_rows(r, L, r->layers[i], rows, d);
            a.gate = d.gate;
            launch_mlstm(a);
            o.cat.o = d.o; o.cat.gate = d.gate;
        }
        launch_out_decode(o, DecodeMoe{});
        leave(L.g_post, L.b_out);
        if (!L.c.dense_ff) continue;
        product_of(L.ff_up, L.g_ff, act, 1);
        matvec_rows(L.ff_down.buf, act, cout, L.ff_down.rows, L.ff_down.cols);
        leave(L.g_ff_post, nullptr);
    }
    r->xr = at; r->post_g = in.g_br; r->post_b = in.b_br;
}

// decoding one sequence with F16 weights: the fused steps of stack_decode.hip
void decode_layers(LayerStack *st, StackRun *r, int pos)
{
    const Rows rows{1, 1, pos};
    float *x = ptr<float>(r->x), *cin = ptr<float>(r->cin);
    for (size_t i = 0; i < st->layers.size(); i++) {
        StackLayer &L = st->layers[i];
        StackRun::Layer &k = r->layers[i];
        const LayerConfig &c = L.c;
        matvec_layernorm(L.in.buf, x, ptr<float>(L.g_norm), st->D, st->cfg.eps, cin, L.in.rows, L.in.cols);
        DecodeMoe e{};
        e.x = x; e.g = ptr<float>(L.g_norm); e.D = st->D; e.Dp = st->Dp; e.eps = st->cfg.eps;
        if (c.experts) {
            e.z = cin + L.o_router; e.E = c.experts; e.top = c.top; e.idx = ptr<int>(r->route_idx); e.w = ptr<float>(r->route_w);
            e.up = ptr<half_t>(L.up.buf); e.down = ptr<half_t>(L.down.buf); e.up_rows = L.up_rows; e.down_rows = L.down_rows;
            e.ff = c.ff; e.ffp = L.down.cols; e.act = ptr<float>(r->act);
        }
        DecodeOut o{};
        o.cat = cat_rows(st, r, L);
        o.out = ptr<half_t>(L.out.buf); o.x = x; o.D = st->D;
        Aux ax{ptr<float>(r->aux)};
        if (L.delta()) {
            const DeltaAux d = delta_aux(ax, c, 1, 1);
            DecodeDelta s{};
            s.a = delta_rows(st, r, L, k, rows, d);
            s.a2 = ptr<half_t>(L.a2.buf); s.g2 = ptr<half_t>(L.g2.buf); s.lda2 = L.a2.cols; s.ldg2 = L.g2.cols; s.o_g = L.o_g;
            s.gate = d.v;                                 // (the values stay in registers here)
            launch_delta_decode(s, e);
            o.cat.o = d.o; o.cat.gate = s.gate;
        } else {
            const LatentAux d = latent_aux(ax, c, 1);
            launch_latent_decode(latent_rows(st, r, L, k, rows, d), e);
            o.cat.o = d.o;
        }
        launch_out_decode(o, e);
    }
}

}  // namespace

void stack_forward(LayerStack *st, StackRun *r, const int *tokens, int T, int pos)
{
    const Rows rows{r->B, T, pos};
    const int n = rows.n();
    if (n <= STACK_FEW) launch_embed_few(ptr<float>(st->emb), tokens, st->cfg.emb_scale, ptr<float>(r->x), st->D, st->Dp, n);
    else {
        // many tokens travel through pinned memory, every position in a place of its own: only a sequence that has gone back
        // writes a place again, and waits for the copies from it
        if (pos < r->tok_end) HIP_CHECK(hipStreamSynchronize(stream()));
        r->tok_end = pos + T;
        int *th = r->tok_host + (size_t)pos * r->B;
        memcpy(th, tokens, (size_t)n * sizeof(int));
        HIP_CHECK(hipMemcpyAsync(dptr(r->tok), th, (size_t)n * sizeof(int), hipMemcpyHostToDevice, stream()));
        launch_embed_rows(ptr<float>(st->emb), ptr<int>(r->tok), st->cfg.emb_scale, ptr<float>(r->x), st->D, st->Dp, n);
    }
    r->T = T; r->pending = 0;
    r->one = n == 1 && r->fused;
    if (r->one) { if (st->cfg.norms == NORMS_AROUND) decode_layers_around(st, r, pos); else decode_layers(st, r, pos); return; }
    for (size_t i = 0; i < st->layers.size(); i++) {
        StackLayer &L = st->layers[i];
        const LayerConfig &c = L.c;
        // from a few rows per expert on, each expert's weights are read once for all its rows
        const bool grouped = c.experts && !st->f32 && n >= 16 && n * c.top >= c.experts;
        norm(st, r, L.g_norm, n, 1, c.experts && !grouped);
        product(st, L.in, ptr<half_t>(r->a16), ptr<float>(r->inv), ptr<float>(r->h), st->Dp, ptr<float>(r->cin), n);
        CatRows cat = cat_rows(st, r, L);
        switch (c.mixer) {
        case MIX_LATENT: cat.o = mix_latent(st, r, L, r->layers[i], rows); break;
        case MIX_GROUPED: cat.o = mix_grouped(st, r, L, rows, cat); break;
        case MIX_MLSTM: cat.o = mix_mlstm(st, r, L, r->layers[i], rows, cat); break;
        default: cat.o = mix_delta(st, r, L, r->layers[i], rows, cat);
        }
        launch_cat_rows(cat, n);
        product(st, L.out, cat.a16, cat.inv, cat.cat, cat.ldk, ptr<float>(r->cout), n);
        r->pending = 1; r->post_g = ptr<float>(L.g_post); r->post_b = ptr<float>(L.b_out);
        if (c.dense_ff) feed_forward(st, r, L, n);
        if (!c.experts) continue;
        MoeRows m{};
        m.rows = n; m.E = c.experts; m.top = c.top; m.ff = c.ff; m.ffp = L.down.cols; m.D = st->D; m.Dp = st->Dp; m.f32 = st->f32;
        m.up_rows = L.up_rows; m.down_rows = L.down_rows;
        m.z = ptr<float>(r->cin) + L.o_router; m.ldz = L.in.rows; m.idx = ptr<int>(r->route_idx); m.w = ptr<float>(r->route_w);
        m.h = ptr<float>(r->h); m.up = dptr(L.up.buf); m.down = dptr(L.down.buf); m.act = ptr<float>(r->act); m.y = ptr<float>(r->ymoe);
        launch_route(m);
        if (!grouped) { launch_experts_per_row(m); r->pending = 3; continue; }
        const MoeGroups g = moe_groups_at(ptr<int>(r->moe_tab), n, c.top, c.experts);
        const int M = g.tiles * 128;
        float *up = ptr<float>(r->moe_up), *inv = ptr<float>(r->moe_inv), *inv_act = inv + r->moe_rows;
        half_t *rows16 = ptr<half_t>(r->moe_a16), *act16 = ptr<half_t>(r->moe_act);
        launch_moe_groups(m, g);
        launch_moe_gather(g, ptr<half_t>(r->a16), ptr<float>(r->inv), rows16, inv, st->Dp);
        launch_gemm_groups(rows16, inv, tiled_weight_of(L.up.buf, L.up.rows, L.up.cols), tiled_elems(L.up_rows, L.up.cols), g.of, up, L.up_rows,
                           M, c.ff, L.up.cols, c.experts);
        launch_moe_act(g, up, L.up_rows, c.ff, act16, inv_act, m.ffp);
        launch_gemm_groups(act16, inv_act, tiled_weight_of(L.down.buf, L.down.rows, L.down.cols), tiled_elems(L.down_rows, L.down.cols), g.of,
                           ptr<float>(r->moe_y), st->Dp, M, st->Dp, L.down.cols, c.experts);
        r->pending = 5; r->groups = g; r->groups_top = c.top;
    }
}

void stack_logits(LayerStack *st, StackRun *r, const int *want, int n, float *logits)
{
    if (n <= 0) return;
    if (r->one) {                                         // whatever `want` says, it is the one row
        if (st->cfg.norms == NORMS_AROUND)
            matvec_norms_around(st->head.buf, NormIn{r->xr, ptr<float>(r->cout), ptr<float>(st->g_final), nullptr, st->cfg.eps, st->D, r->post_g, r->post_b},
                                logits, st->head.rows, st->head.cols, 0);
        else matvec_layernorm(st->head.buf, ptr<float>(r->x), ptr<float>(st->g_final), st->D, st->cfg.eps, logits, st->head.rows, st->head.cols);
        return;
    }
    const int *list = nullptr;
    if (want) {
        memcpy(r->want_host, want, (size_t)n * sizeof(int));
        HIP_CHECK(hipMemcpyAsync(dptr(r->want), r->want_host, (size_t)n * sizeof(int), hipMemcpyHostToDevice, stream()));
        list = ptr<int>(r->want);
    }
    norm(st, r, st->g_final, n, 0, false, list, r->T, r->T - 1);
    product(st, st->head, ptr<half_t>(r->a16), ptr<float>(r->inv), ptr<float>(r->h), st->Dp, logits, n);
}

}  // namespace lmhip
