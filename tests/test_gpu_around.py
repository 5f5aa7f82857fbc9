"""What is special about grouped attention inside chunks and the mLSTM (Paposun), on the GPU through the generation API
against oracle/stack_oracle.py: chunk edges, shared keys, far keys, rings that wrap, gates at their extremes, memory over
hundreds of tokens, layers wide enough for the large products."""
import copy
import os

import numpy as np
import pytest

from llm_metal_amd.sft import InferenceState
from llm_metal_amd.synth import write_stack_checkpoint
from oracle import stack_oracle as so
from tests.stack_models import MODELS, Model, around, dense, grouped, logit_error, mlstm
from tests.test_gpu_stack import TOL, moving_model, run_portions, say, state

pytestmark = pytest.mark.gpu
FMT = pytest.mark.parametrize("fmt", ["f32", "f16"])


def ways(inf, toks, tail=4):
    """The last logits: as one prompt, in two portions, and with the last tokens decoded."""
    pos, out = len(toks) - 1, []
    inf.reset()
    out.append(inf.forward_tokens(toks, [pos])[0])
    inf.reset()
    cut = max(1, pos - 17)
    inf.forward_tokens(toks[:cut])
    out.append(inf.forward_tokens(toks[cut:], [pos - cut])[0])
    inf.reset()
    cut = max(1, pos + 1 - tail)
    inf.forward_tokens(toks[:cut])
    for t in toks[cut:-1]:
        inf.forward_token(t)
    out.append(inf.forward_token(toks[-1]))
    return out


def most_telling(cfg, m, toks, at):
    """The prompt with another token at place `at`: of a few, the one whose exchange shows most at the end."""
    ref = so.run(cfg, m.W, toks)[-1]
    swaps = [toks[:at] + [(toks[at] + k) % cfg["vocab"]] + toks[at + 1:] for k in (7, 31, 62, 90)]
    outs = [so.run(cfg, m.W, t)[-1] for t in swaps]
    best = int(np.argmax([np.abs(o - ref).max() for o in outs]))
    assert np.abs(outs[best] - ref).max() > 100 * TOL["f32"] * ref.std()
    return swaps[best], outs[best]


@FMT
@pytest.mark.parametrize("chunk,n", [(1, 40), (2, 41), (16, 80), (16, 81), (31, 63), (32, 97), (33, 67), (64, 128), (64, 129), (65, 140), (100, 260), (128, 300)])
def test_chunk_edges(chunk, n, fmt, tmp_path):
    """One attention layer: the last token of the chunk before must not matter at all, the first one of the query's chunk must,
    also when the query is that first token."""
    cfg = around([(grouped(4, 2, chunk=chunk, scale=0.5), None)])
    m = Model(cfg, tmp_path)
    toks = m.tokens(n, seed=3)
    first = (n - 1) // chunk * chunk
    with state(m, fmt, max_seq=n) as inf:
        ref, want = ways(inf, toks), so.run(cfg, m.W, toks)[-1]
        for g in ref:
            assert logit_error(g[None], want[None]) < TOL[fmt]
        if first:
            outside = list(toks)
            outside[first - 1] = (toks[first - 1] + 7) % cfg["vocab"]
            for r, g in zip(ref, ways(inf, outside)):
                assert np.array_equal(r, g)
        inside, o_in = most_telling(cfg, m, toks, first)
        for g in ways(inf, inside):
            assert logit_error(g[None], o_in[None]) < TOL[fmt]


@FMT
def test_a_reader_with_longer_chunks_than_the_keys_owner(fmt, tmp_path):
    """Keys that the layer which wrote them no longer sees are there for the layer that borrows them, in prompts longer than a
    step's portion would keep for the owner alone, and in decoding."""
    cfg = around([(grouped(4, 2, chunk=8), None), (grouped(4, 2, chunk=90, kv_from=0, scale=0.6), None)])
    m = Model(cfg, tmp_path)
    n = 179                                                    # position 178: chunk 90 .. 179 of the reader, 176 .. of the owner
    toks = m.tokens(n, seed=4)
    with state(m, fmt, max_seq=n) as inf:
        for at in (90, 130, 175):
            t, want = most_telling(cfg, m, toks, at)
            for g in ways(inf, t, tail=60):
                assert logit_error(g[None], want[None]) < TOL[fmt]
        outside = list(toks)
        outside[89] = (toks[89] + 7) % cfg["vocab"]
        for r, g in zip(ways(inf, toks), ways(inf, outside)):
            assert np.array_equal(r, g)


@FMT
def test_one_far_key_among_hundreds(fmt, tmp_path):
    """One token's key stands out for every query: it holds nearly all the weight wherever it lies in a chunk of many slices,
    and none once the chunk is over."""
    D, d, loud = 64, 32, 11
    cfg = around([(grouped(4, 2, dim=d, vdim=32, chunk=300, scale=0.6, dims=2, base=1e4), None)], width=D)
    seen = {}

    def edit(name, a):
        if name == "embed":
            seen["e"] = a[loud] / np.linalg.norm(a[loud])
        if name == "l0.mix.k":
            a[[5, d + 5]] = 3.0 * seen["e"]
        if name == "l0.mix.q.b":
            a[5::d] = 1.0
        return a
    m = Model(cfg, tmp_path, edit=edit)
    n = 620                                                    # position 619: chunk 600 ..; position 599: chunk 300 ..
    toks = [t if t != loud else 12 for t in m.tokens(n, seed=5)]
    with state(m, fmt, max_seq=n) as inf:
        for size, places in ((600, (299, 300, 301, 331, 332, 333, 450, 598)), (n, (599, 600, 601, 615))):
            t = toks[:size]
            without = so.run(cfg, m.W, t)[-1]
            for at in places:
                loudly = t[:at] + [loud] + t[at + 1:]
                want = so.run(cfg, m.W, loudly)[-1]
                assert (logit_error(want[None], without[None]) > 0.05) == (at not in (299, 599))
                for g in ways(inf, loudly):
                    assert logit_error(g[None], want[None]) < TOL[fmt]


@pytest.mark.parametrize("cut", ["low", "between", "high", "none"])
def test_scaled_frequencies(cut, tmp_path):
    """Every regime of the frequency scale decides positions of its own, far from the start of the sequence too."""
    scaling = {"low": (8.0, 50.0, 60.0, 40), "between": (8.0, 1e-3, 100.0, 64), "high": (8.0, 1e-4, 2e-4, 900), "none": None}[cut]
    cfg = around([(grouped(4, 2, chunk=400, scaling=scaling, base=50.0, scale=0.6), None)])
    m = Model(cfg, tmp_path)
    toks = m.tokens(330, seed=6)
    want = so.run(cfg, m.W, toks)
    plain = copy.deepcopy(cfg)
    plain["layers"][0]["mixer"]["rot"].pop("scaling", None)
    other = so.run(plain, m.W, toks)
    assert (logit_error(other, want) > 100 * TOL["f32"]) == (cut in ("low", "between"))
    with state(m, "f32", max_seq=330) as inf:
        assert logit_error(run_portions(inf, toks, [100, 7, 1, 1, 200, 1]), want) < TOL["f32"]


@FMT
def test_long_prompts_and_rings_that_wrap(fmt, tmp_path):
    """More tokens than one step takes and than a ring holds, then decoding on."""
    cfg = around([(grouped(2, 1, dim=8, vdim=8, chunk=150), None), (mlstm(2, 8, 12), dense(16)), (grouped(2, 1, dim=8, vdim=8, chunk=60, kv_from=0), None)],
                 width=32, vocab=64)
    m = Model(cfg, tmp_path)
    n = 4500
    toks = m.tokens(n, seed=6)
    want = so.run(cfg, m.W, toks)
    say("long prompt", fmt)
    with state(m, fmt, max_seq=n) as inf:
        head = n - 170
        at = sorted(set(list(range(0, head, 97)) + [2047, 2048, 2049, 2099, 2100, 4049, 4050, 4095, 4096, 4097, 4199, 4200]))
        assert logit_error(inf.forward_tokens(toks[:head], at), want[at]) < TOL[fmt]
        got = np.stack([inf.forward_token(t) for t in toks[head:]])
        assert logit_error(got, want[head:]) < TOL[fmt]


def gates(i_bias, f_bias):
    """Input and forget gates spread over the heads between the given pre-activations."""
    def edit(name, a):
        if name.endswith(".i.b"):
            return np.linspace(*i_bias, a.size).astype(np.float32)
        if name.endswith(".f.b"):
            return np.linspace(*f_bias, a.size).astype(np.float32)
        return a
    return edit


@FMT
@pytest.mark.parametrize("i_bias,f_bias", [((-40, 40), (5, 5)), ((-9, 0), (-40, 40)), ((-9, -9), (9, -3)), ((30, -25), (30, -30)), ((3, 8), (1, 3))])
def test_gates_at_their_extremes(i_bias, f_bias, fmt, tmp_path):
    """Inputs that are hardly written (the running maximum starts at 0 and decides the denominator), states that are wiped in
    one token beside ones that keep everything, writes that dwarf what is there."""
    cfg = around([(mlstm(6, 20, 24, 14.0), None), (mlstm(4, 72, 8, 6.0), None)], eps=1e-6)
    m = Model(cfg, tmp_path, edit=gates(i_bias, f_bias))
    toks = m.tokens(200, seed=4)
    want = so.run(cfg, m.W, toks)
    with state(m, fmt, max_seq=256) as inf:
        for sizes in ([200], [70, 2, 1, 64, 63], [1]):
            inf.reset()
            assert logit_error(run_portions(inf, toks, sizes), want) < TOL[fmt]


def test_far_memory_survives_decoding(tmp_path):
    """A forget gate that stays open carries the first token over hundreds of decoded ones, and over portions."""
    cfg = around([(mlstm(4, 16, 16, 20.0), None), (mlstm(2, 40, 8, 20.0), None)], width=48)
    m = Model(cfg, tmp_path, edit=gates((0, -2), (30, 30)))
    toks = m.tokens(400, seed=9)
    other = [(toks[0] + 11) % cfg["vocab"]] + toks[1:]
    want, moved = so.run(cfg, m.W, toks)[-1], so.run(cfg, m.W, other)[-1]
    assert logit_error(moved[None], want[None]) > 50 * TOL["f32"]       # the first token shows at the last
    with state(m, "f32", max_seq=400) as inf:
        for t, w in ((toks, want), (other, moved)):
            inf.reset()
            inf.forward_tokens(t[:5])
            for x in t[5:-1]:
                inf.forward_token_argmax(x)
            assert logit_error(inf.forward_token(t[-1])[None], w[None]) < TOL["f32"]
            inf.reset()
            assert logit_error(run_portions(inf, t, [2, 130, 1, 65])[-1:], w[None]) < TOL["f32"]


@FMT
def test_portions_at_every_cut(fmt, tmp_path):
    """Two portions, cut at every place around the edges of chunks of attention and of the mLSTM's sixty-four tokens."""
    cfg = around([(grouped(2, 1, 8, 12, 64), None), (mlstm(2, 12, 8), dense(8)), (grouped(2, 1, 8, 12, 24, kv_from=0), None)], width=40, vocab=64)
    m = Model(cfg, tmp_path)
    n = 140
    toks = m.tokens(n, seed=7)
    want = so.run(cfg, m.W, toks)
    with state(m, fmt, max_seq=n) as inf:
        for cut in (1, 2, 15, 16, 17, 23, 24, 25, 62, 63, 64, 65, 66, 127, 128, 129, 138, 139):
            inf.reset()
            assert logit_error(run_portions(inf, toks, [cut, n - cut]), want) < TOL[fmt]
            inf.reset()
            assert logit_error(run_portions(inf, toks, [cut, 1, 2, n]), want) < TOL[fmt]


@FMT
def test_generated_batches_equal_the_single_sequence(fmt, tmp_path):
    """A prompt longer than a batch's portion, generated in lock step and alone."""
    m = moving_model(tmp_path)
    prompt = m.tokens(330, seed=10)
    want = so.run(m.cfg, m.W, prompt)[-1]
    with state(m, fmt, max_seq=380) as inf:
        alone = list(inf.generate(prompt, 12))
        assert alone[0] == int(np.argmax(want))
        if fmt == "f32":
            for row in inf.generate_batch(prompt, 12, 16):
                assert list(row) == alone
        assert [r[0] for r in inf.generate_batch(prompt, 3, 7)] == [alone[0]] * 7


def test_wide_layers_on_the_large_products(tmp_path):
    """Sizes at which a long prompt takes the kernels for many rows: the 16-bit prompt, the 16-bit fused decoding and the
    32-bit state agree, whole and in portions."""
    cfg = around([(grouped(16, 4, 128, 128, 300, scale=0.07, dims=64, base=2e5), dense(4096)), (mlstm(4, 256, 192, 12.0), dense(3000)),
                  (grouped(16, 4, 128, 128, 512, scale=0.09, dims=64, base=2e5, kv_from=0), None), (mlstm(8, 128, 128, 12.0), None)], width=1024, vocab=512)
    m = Model.__new__(Model)
    m.cfg, m.path = cfg, str(tmp_path)
    write_stack_checkpoint(m.path, cfg, seed=3)
    n = 1150
    toks = [int(t) for t in np.random.default_rng(4).integers(0, 512, n)]
    at = [0, 1, 127, 128, 299, 300, 301, 511, 512, 1022, 1023, 1024, 1100, n - 1]
    with state(m, "f32", max_seq=n) as inf:
        want = inf.forward_tokens(toks, at)
    with state(m, "f16", max_seq=n) as inf:
        whole = inf.forward_tokens(toks, at)
        assert logit_error(whole, want) < TOL["f16"]
        inf.reset()
        rows = run_portions(inf, toks, [600, 15, 2, 1, 500])
        assert logit_error(rows[at], want) < TOL["f16"]
        inf.reset()
        inf.forward_tokens(toks[:n - 60])
        last = [inf.forward_token(t) for t in toks[n - 60:]][-1]
        assert logit_error(last[None], want[-1:]) < TOL["f16"]


def test_missing_tensors_are_refused(tmp_path):
    cfg, _, _ = MODELS["norms around, mixed"]
    for cut in ("l0.mix.q.b", "l0.mix.o.b", "l1.mix.f.b", "l2.norm2b", "l3.mix.norm", "embed"):
        m = Model(cfg, tmp_path / cut)
        raw = open(os.path.join(m.path, "model.safetensors"), "rb").read()
        with open(os.path.join(m.path, "model.safetensors"), "wb") as f:
            f.write(raw.replace(f'"{cut}"'.encode(), f'"{cut[:-1]}_"'.encode(), 1))
        with pytest.raises(RuntimeError):
            state(m, "f32")
    with pytest.raises(RuntimeError):
        InferenceState(path=Model(cfg, tmp_path / "q8").path, model_type=None, max_seq=16, weight_format="q8_0")
