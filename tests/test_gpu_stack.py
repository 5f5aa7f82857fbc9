"""Models described layer by layer (Nevurax, Paposun) on the GPU through the generation API, against the plain numpy restatement in
oracle/stack_oracle.py: every mechanism alone, prompts against decoding, portions, batches, reused states, window edges,
rings that wrap, greedy generation, the command line and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from llm_metal_amd.configs import C1
from llm_metal_amd.sft import InferenceState
from llm_metal_amd.synth import make_model, write_stack_checkpoint
from oracle import stack_oracle as so
from tests.stack_models import MODELS, Model, config, channel, delta, latent, logit_error, moe

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"f32": 2e-5, "f16": 4e-3}
MIXED = pytest.mark.parametrize("mixed", ["mixed", "norms around, mixed"])


def say(*a):
    print(*a, flush=True, file=sys.stderr)


def state(model, fmt, max_seq=128):
    return InferenceState(path=model.path, model_type=None, max_seq=max_seq, weight_format=fmt)


def run_portions(inf, tokens, sizes):
    """All logits, the tokens cut into portions of the given sizes (the last one repeats)."""
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(sizes[min(i, len(sizes) - 1)], len(tokens) - at)
        out.append(inf.forward_tokens(tokens[at:at + n], range(n)))
        at, i = at + n, i + 1
    return np.concatenate(out)


@pytest.mark.parametrize("fmt", ["f32", "f16"])
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt_and_decoding_match_the_oracle(name, fmt, tmp_path):
    say("stack", name, fmt)
    cfg, ra, rg = MODELS[name]
    m = Model(cfg, tmp_path, ra, rg)
    toks = m.tokens(75)
    want = so.run(cfg, m.W, toks)
    with state(m, fmt) as inf:
        whole = inf.forward_tokens(toks, range(len(toks)))
        assert inf.position() == len(toks)
        assert logit_error(whole, want) < TOL[fmt]
        inf.reset()
        single = np.stack([inf.forward_token(t) for t in toks])
        assert logit_error(single, want) < TOL[fmt]


@MIXED
@pytest.mark.parametrize("fmt", ["f32", "f16"])
@pytest.mark.parametrize("sizes", [[2], [3, 2, 5, 7, 2, 11], [40, 1, 1, 1, 20, 2], [1, 33, 16, 17], [64, 2, 1], [5, 70]])
def test_portions_of_any_size(sizes, fmt, mixed, tmp_path):
    say("portions", mixed, sizes, fmt)
    cfg, ra, rg = MODELS[mixed]
    m = Model(cfg, tmp_path, ra, rg)
    toks = m.tokens(90, seed=2)
    want = so.run(cfg, m.W, toks)
    with state(m, fmt) as inf:
        assert logit_error(run_portions(inf, toks, sizes), want) < TOL[fmt]


@MIXED
@pytest.mark.parametrize("fmt", ["f32", "f16"])
def test_first_tokens_and_a_sequence_of_one(fmt, mixed, tmp_path):
    cfg, ra, rg = MODELS[mixed]
    m = Model(cfg, tmp_path, ra, rg)
    with state(m, fmt) as inf:
        for n in (1, 2, 3, 4, 5):
            toks = m.tokens(n, seed=20 + n)
            inf.reset()
            assert logit_error(inf.forward_tokens(toks, range(n)), so.run(cfg, m.W, toks)) < TOL[fmt]


@MIXED
def test_states_are_used_again(mixed, tmp_path):
    """A second sequence in the same state sees nothing of the first, whatever its length: bit-identical to a fresh state."""
    cfg, ra, rg = MODELS[mixed]
    m = Model(cfg, tmp_path, ra, rg)
    prompts = [m.tokens(n, seed=n) for n in (60, 3, 1, 41, 2)]
    for fmt in ("f32", "f16"):
        with state(m, fmt) as used:
            for p in prompts:
                used.reset()
                got = run_portions(used, p, [17, 2, 1])
                with state(m, fmt) as fresh:
                    assert np.array_equal(got, run_portions(fresh, p, [17, 2, 1]))


@MIXED
@pytest.mark.parametrize("fmt", ["f32", "f16"])
def test_lock_step_batches_against_each_alone(fmt, mixed, tmp_path):
    cfg, ra, rg = MODELS[mixed]
    m = Model(cfg, tmp_path, ra, rg)
    seqs = np.array([m.tokens(45, seed=50 + b) for b in range(5)])
    want = np.stack([so.run(cfg, m.W, s) for s in seqs])
    with state(m, fmt) as inf:
        for _ in range(2):                                     # the second pass reuses the batch's states
            got = np.stack([inf.step_batch(seqs[:, t], t) for t in range(seqs.shape[1])], axis=1)
            assert logit_error(got.reshape(-1, got.shape[-1]), want.reshape(-1, want.shape[-1])) < TOL[fmt]
        # the single sequence has states of its own
        assert logit_error(inf.forward_tokens(list(seqs[0]), range(45)), want[0]) < TOL[fmt]


@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 63, 64, 65, 100])
def test_window_edges(window, tmp_path):
    """One attention layer: a token just outside the window must not matter at all, one just inside must, in a prompt and in
    decoding.  The token put inside is the one of a few that the oracle says shows most."""
    cfg = config([(latent(4, window=window, scale=0.3), None)])
    m = Model(cfg, tmp_path)
    n = 140
    base = m.tokens(n, seed=3)
    pos = n - 1
    with state(m, "f32", max_seq=n) as inf:
        def both(toks):
            inf.reset()
            a = inf.forward_tokens(toks, [pos])[0]
            inf.reset()
            inf.forward_tokens(toks[:pos - 4])
            b = inf.forward_tokens(toks[pos - 4:pos]) is not None and inf.forward_token(toks[pos])
            return a, b
        ref = both(base)
        outside = list(base)
        outside[pos - window] = (base[pos - window] + 7) % cfg["vocab"]
        for r, g in zip(ref, both(outside)):
            assert np.array_equal(r, g)
        o_ref = so.run(cfg, m.W, base)[pos]
        swaps = [base[:pos - window + 1] + [(base[pos - window + 1] + k) % cfg["vocab"]] + base[pos - window + 2:] for k in (7, 31, 62, 90)]
        outs = [so.run(cfg, m.W, t)[pos] for t in swaps]
        best = int(np.argmax([np.abs(o - o_ref).max() for o in outs]))
        inside, o_in = swaps[best], outs[best]
        assert np.abs(o_ref - o_in).max() > 100 * TOL["f32"] * o_ref.std()          # the edge shows
        for g in both(inside):
            assert logit_error(g[None], o_in[None]) < TOL["f32"]


def test_long_prompts_and_rings_that_wrap(tmp_path):
    """More tokens than one step takes and than the attention ring holds, then decoding past the wrap."""
    cfg = config([(latent(2, window=50), None), (channel(2, 1, 16, 8, 3), moe(4, 2, 8, 8))], width=32, vocab=64)
    m = Model(cfg, tmp_path)
    n = 4500
    toks = m.tokens(n, seed=6)
    want = so.run(cfg, m.W, toks)
    for fmt in ("f32", "f16"):
        say("long prompt", fmt)
        with state(m, fmt, max_seq=n) as inf:
            head = n - 130
            at = list(range(0, head, 97)) + [2047, 2048, 2049, 2097, 2098, 4095, 4096, 4097, 4145, 4146]
            at = sorted(set(at))
            got = inf.forward_tokens(toks[:head], at)
            assert logit_error(got, want[at]) < TOL[fmt]
            got = np.stack([inf.forward_token(t) for t in toks[head:]])
            assert logit_error(got, want[head:]) < TOL[fmt]


def test_far_memory_survives_decoding(tmp_path):
    """A state that hardly decays carries its first tokens over hundreds of decoded ones."""
    def slow(name, a):
        return a - 6.0 if name.endswith("A_log") else a
    cfg = config([(delta(4, 2, 16, 16, 2), None), (channel(2, 2, 16, 8, 2), None)], width=48)
    m = Model(cfg, tmp_path, edit=slow)
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


def test_strong_decays_and_large_gates(tmp_path):
    """Decays that wipe a state at once (exp of large negative numbers) beside ones that keep it."""
    def spread(name, a):
        if name.endswith("A_log"):
            return np.linspace(-8.0, 4.5, a.size).astype(np.float32).reshape(a.shape)
        if name.endswith("dt_bias"):
            return np.linspace(-12.0, 25.0, a.size).astype(np.float32).reshape(a.shape)
        return a
    cfg = config([(channel(4, 2, 40, 16, 3), None), (delta(6, 3, 16, 16, 2), None)])
    m = Model(cfg, tmp_path, edit=spread)
    toks = m.tokens(100, seed=4)
    want = so.run(cfg, m.W, toks)
    for fmt in ("f32", "f16"):
        with state(m, fmt) as inf:
            assert logit_error(run_portions(inf, toks, [70, 2, 1]), want) < TOL[fmt]


def moving_model(path):
    """A tied head repeats its token: alternating signs on the final norm and larger sublayers make the sequence move."""
    cfg = dict(MODELS["norms around, mixed"][0], residual_mult=1.7)
    return Model(cfg, path, edit=lambda n, a: a * np.where(np.arange(a.size) % 2, 1, -1).astype(np.float32) if n == "final.norm" else a)


@MIXED
def test_greedy_generation_everywhere(mixed, tmp_path):
    cfg, ra, rg = MODELS[mixed]
    if mixed == "mixed":
        m = Model(cfg, tmp_path, ra, rg)
    else:
        m = moving_model(tmp_path)
        cfg = m.cfg
    prompt = m.tokens(23, seed=8 if mixed == "mixed" else 10)
    want = so.generate(cfg, m.W, prompt, 40)
    assert len(set(want)) >= 10
    logits = np.sort(so.run(cfg, m.W, prompt + want[:-1])[len(prompt) - 1:], axis=1)
    assert (logits[:, -1] - logits[:, -2]).min() > 10 * TOL["f32"] * logits.std()     # no close call in this sequence
    with state(m, "f32") as inf:
        assert list(inf.generate(prompt, 40)) == want
        assert [list(r) for r in inf.generate_batch(prompt, 40, 3)] == [want] * 3
        inf.set_eos([want[5]])
        stop = want.index(want[5]) + 1
        assert list(inf.generate(prompt, 40)) == want[:stop]
        inf.reset()
        nxt, got = None, []
        for t in prompt:
            nxt = inf.forward_token_argmax(t)
        for _ in range(10):
            got.append(nxt)
            nxt = inf.forward_token_argmax(nxt)
        assert got == want[:10]
    exe = os.path.join(ROOT, "llm_metal_amd", "run_sft_hip")
    out = subprocess.run([exe, "--mode", "generate", "--model", m.path, "--prompt", ",".join(map(str, prompt)), "--max-gen", "40", "--f32"],
                         capture_output=True, text=True, timeout=100)
    assert out.returncode == 0, out.stderr
    line = [x for x in out.stdout.splitlines() if x.startswith("tokens:")][0]
    assert [int(x) for x in line.split(":")[1].split()] == want


@MIXED
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner(dtype, mixed, tmp_path):
    cfg, ra, rg = MODELS[mixed + ", odd"]
    m = Model(cfg, tmp_path / "model", ra, rg)
    reqs = {"a": m.tokens(37, seed=1), "b": m.tokens(5, seed=2)}
    steps = [("a", 0, 20, [0, 19]), ("a", 20, 22, []), ("a", 22, 23, [0]), ("a", 23, 37, [13, 2]), ("b", 0, 4, [3]), ("b", 4, 5, [0])]
    lines = [json.dumps({"step": i, "entries": [{"id": r, "tokens": reqs[r][lo:hi], "want": w}], "end": [r] if hi == len(reqs[r]) else []})
             for i, (r, lo, hi, w) in enumerate(steps)]
    out = tmp_path / "out"
    out.mkdir()
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", m.path, "--dtype", dtype, "--out", str(out), "--max-tokens", "40"],
                       input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(len(steps))]
    ref = {k: so.run(cfg, m.W, v) for k, v in reqs.items()}
    for i, (r, lo, hi, w) in enumerate(steps):
        f = out / f"{i}.f32"
        assert f.exists() == bool(w)
        if w:
            got = np.fromfile(f, "<f4").reshape(len(w), cfg["vocab"])
            assert logit_error(got, ref[r][[lo + k for k in w]]) < TOL["f32" if dtype == "float32" else "f16"]


def test_wide_layers_on_the_large_products(tmp_path):
    """Sizes at which the products of a long prompt take the kernels for many rows: the 16-bit prompt, the 16-bit fused
    decoding and the 32-bit state agree, whole and in portions.  (Every expert is chosen, so that no rounding decides.)"""
    mlp = moe(4, 4, 320, 1024)
    cfg = config([(channel(8, 8, 128, 128, 4), mlp), (latent(8, 128, 64, 128, 256, window=300, scale=0.07), mlp), (delta(8, 4, 128, 128, 4), mlp)],
                 width=1024, vocab=512)
    m = Model.__new__(Model)
    m.cfg, m.path = cfg, str(tmp_path)
    write_stack_checkpoint(m.path, cfg, seed=3, rank_a=64, rank_g=64)
    n = 1150
    toks = [int(t) for t in np.random.default_rng(4).integers(0, 512, n)]
    at = [0, 1, 127, 128, 299, 300, 301, 512, 1022, 1023, 1024, 1100, n - 1]
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


def test_what_is_refused(tmp_path):
    cfg, ra, rg = MODELS["mixed"]
    m = Model(cfg, tmp_path, ra, rg)
    with pytest.raises(RuntimeError):
        state(m, "q8_0")
    with state(m, "f32", max_seq=10) as inf:
        inf.forward_tokens(m.tokens(8))
        for bad in ([1, 2, 3], [cfg["vocab"]], [-1]):
            with pytest.raises(RuntimeError):
                inf.forward_tokens(bad)
        with pytest.raises(RuntimeError):
            inf.forward_tokens([1, 2], [1, 0])
        assert inf.position() == 8
        inf.forward_tokens([1, 2])
    for cut in ("l2.mix.dt_bias", "l0.mlp.e6.down", "head"):              # a missing tensor
        broken = Model(cfg, tmp_path / cut, ra, rg)
        raw = open(os.path.join(broken.path, "model.safetensors"), "rb").read()
        with open(os.path.join(broken.path, "model.safetensors"), "wb") as f:
            f.write(raw.replace(f'"{cut}"'.encode(), f'"{cut[:-1]}_"'.encode(), 1))
        with pytest.raises(RuntimeError):
            state(broken, "f32")
    huge = Model(cfg, tmp_path / "huge", ra, rg, edit=lambda n, a: a * np.float32(1e6) if n == "head" else a)
    with pytest.raises(RuntimeError):
        state(huge, "f16")
    state(huge, "f32").free()


def test_states_give_their_memory_back(tmp_path):
    import ctypes
    from llm_metal_amd import lib
    cfg, ra, rg = MODELS["mixed"]
    m = Model(cfg, tmp_path, ra, rg)
    prompt = m.tokens(40)
    free = []
    with state(m, "f32") as keep:                              # keeps the library's own scratch alive
        keep.forward_tokens(prompt)
        for _ in range(4):
            with state(m, "f16") as inf:
                inf.generate(prompt, 5)
                inf.generate_batch(prompt, 5, 3)
            f, t = ctypes.c_size_t(0), ctypes.c_size_t(0)
            lib.load().hip_mem_info(ctypes.byref(f), ctypes.byref(t))
            free.append(f.value)
    assert free[1] == free[2] == free[3]


def test_portions_of_the_other_models():
    """inference_forward_tokens on a model that takes one token per step: the same logits as token by token."""
    model = make_model(C1, seed=7)
    toks = [3, 70, 11, 500, 42, 7]
    with InferenceState(C1, model, max_seq=16) as inf:
        want = np.stack([inf.forward_token(t) for t in toks])
        inf.reset()
        got = np.concatenate([inf.forward_tokens(toks[:4], [0, 3]), inf.forward_tokens(toks[4:], [1])])
    assert np.array_equal(got, want[[0, 3, 5]])
