"""Small layer-by-layer models for the tests: configurations (odd sizes on purpose) and their checkpoints."""
import numpy as np

from llm_metal_amd.synth import write_stack_checkpoint
from oracle import stack_oracle as so


def delta(heads=6, kv_heads=2, dim=24, vdim=40, conv=2):
    return {"type": "delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)}


def channel(heads=4, kv_heads=2, dim=48, vdim=16, conv=5):
    return {"type": "channel_delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)}


def latent(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, window=17, base=5000.0, scale=0.3, dims=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim if dims is None else dims}}}


def moe(experts=7, top=3, ff=24, shared=40):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def grouped(heads=6, kv_heads=2, dim=24, vdim=20, chunk=17, base=700.0, dims=None, scale=0.3, scaling=(3.0, 0.7, 2.5, 90), kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": chunk},
         "rot": {"base": base, "dims": dim if dims is None else dims}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def mlstm(heads=3, dim=20, vdim=28, cap=9.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def around(layers, width=96, vocab=160, mult=0.45, logits=0.6, eps=1e-5):
    return {"architecture": "Paposun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "logit_scale": logits,
            "layers": [{**mix, "mlp": ff} for mix, ff in layers]}


def config(layers, width=96, vocab=160, scale=0.7, eps=1e-5):
    return {"architecture": "Nevurax", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "layers": [{**mix, "mlp": ff} for mix, ff in layers]}


# name -> (configuration, rank_a, rank_g)
MODELS = {
    "delta alone": (config([(delta(), None)]), 12, 20),
    "delta, one tap, one head": (config([(delta(1, 1, 8, 8, 1), None)]), 12, 20),
    "delta, wide heads": (config([(delta(2, 1, 160, 130, 4), None)], width=64), 12, 20),
    "delta, key heads of 128": (config([(delta(2, 2, 128, 72, 3), None)], width=64), 12, 20),
    "channel alone": (config([(channel(), None)]), 12, 20),
    "channel, odd": (config([(channel(3, 3, 10, 6, 3), None)], width=100, vocab=133), 5, 9),
    "channel, wide heads": (config([(channel(2, 1, 200, 64, 4), None)], width=64), 40, 7),
    "latent alone": (config([(latent(), None)]), 12, 20),
    "latent, five heads, odd": (config([(latent(5, 10, 6, 7, 9, window=11), None)], width=100, vocab=133), 12, 20),
    "latent, window of one": (config([(latent(2, window=1), None)]), 12, 20),
    "latent, window beyond": (config([(latent(2, window=5000), None)]), 12, 20),
    "latent, wide": (config([(latent(6, 128, 64, 128, 256, window=70, scale=0.07), None)], width=64), 12, 20),
    "latent, part of the rotation": (config([(latent(4, dim=12, rot_dim=16, dims=10), None)]), 12, 20),
    "experts": (config([(delta(2, 1, 8, 8, 2), moe())]), 12, 20),
    "experts, one of one": (config([(delta(2, 1, 8, 8, 2), moe(1, 1, 13, 0))]), 12, 20),
    "experts, all of them": (config([(delta(2, 1, 8, 8, 2), moe(5, 5, 16, 8))]), 12, 20),
    "experts, many": (config([(delta(2, 1, 8, 8, 2), moe(90, 6, 40, 33))], width=72), 12, 20),
    "mixed": (config([(latent(), moe()), (channel(), moe(16, 2, 32, 48)), (delta(), None), (latent(window=33), moe(4, 1, 20, 0)),
                      (delta(4, 4, 32, 16, 4), moe(9, 4, 17, 24))]), 12, 20),
    "mixed, odd": (config([(channel(3, 1, 10, 6, 3), moe(5, 2, 13, 9)), (latent(5, 10, 6, 7, 9, window=11), moe(5, 2, 13, 9)),
                           (delta(5, 5, 7, 9, 2), moe(3, 2, 11, 5))], width=100, vocab=133), 5, 9),
    **{name: (cfg, 0, 0) for name, cfg in {
        "chunks alone": around([(grouped(), None)]),
        "chunks, five heads, odd": around([(grouped(5, 5, 10, 7, 11, dims=6), dense(13))], width=100, vocab=133),
        "chunks, six heads on one": around([(grouped(6, 1, 16, 8, 33, dims=4), None)]),
        "chunks of one": around([(grouped(2, 1, chunk=1), None)]),
        "chunks beyond": around([(grouped(4, 4, chunk=5000, scaling=None), None)]),
        "chunks, wide": around([(grouped(4, 2, 128, 136, 70, scale=0.08, dims=64), None)], width=64),
        "chunks, wider": around([(grouped(2, 1, 200, 256, 40, scale=0.06, dims=2), None)], width=64),
        "chunks, beyond the matrix cores": around([(grouped(2, 2, 300, 264, 40, scale=0.05), None)], width=64),
        "chunks, shared keys": around([(grouped(chunk=20), None), (grouped(chunk=50, kv_from=0, scale=0.2), dense(24)),
                                       (grouped(4, 1, 8, 16, 9), None), (grouped(chunk=7, kv_from=0), None), (grouped(4, 1, 8, 16, 41, kv_from=2), None)]),
        "mLSTM alone": around([(mlstm(), None)]),
        "mLSTM, one head of one": around([(mlstm(1, 1, 1, 4.0), None)]),
        "mLSTM, odd": around([(mlstm(3, 10, 7, 20.0), dense(9))], width=100, vocab=133),
        "mLSTM, wide keys": around([(mlstm(2, 130, 40), None)], width=64),
        "mLSTM, wider keys": around([(mlstm(2, 264, 72), None)], width=64),
        "mLSTM, wide values": around([(mlstm(2, 64, 200), None)], width=64),
        "dense": around([(grouped(2, 1, 8, 8, 5), dense(300)), (mlstm(1, 8, 8), dense(20))]),
        "norms around, mixed": around([(grouped(), dense()), (mlstm(), None), (grouped(chunk=31, kv_from=0), dense(40)), (mlstm(5, 8, 64, 15.0), dense(30)),
                                       (grouped(3, 3, 16, 32, 64), None), (grouped(3, 3, 16, 32, 64, kv_from=4), None)]),
        "norms around, mixed, odd": around([(mlstm(3, 10, 7, 20.0), None), (grouped(5, 5, 10, 7, 11, dims=6), dense(13)),
                                            (grouped(5, 5, 10, 7, 23, dims=6, kv_from=1), dense(21))], width=100, vocab=133, mult=1.3, logits=2.0),
    }.items()},
}


class Model:
    def __init__(self, cfg, folder, rank_a=12, rank_g=20, seed=5, edit=None):
        self.cfg, self.path = cfg, str(folder)
        w = write_stack_checkpoint(self.path, cfg, seed=seed, rank_a=rank_a, rank_g=rank_g, keep=True, edit=edit)
        self.W = {k: v.astype(np.float64) for k, v in w.items()}

    def tokens(self, n, seed=1, gap=4e-3):
        """Random tokens, drawn again where a router would be close to choosing other experts: 16-bit rounding must not
        decide which ones run."""
        rng = np.random.default_rng(seed)
        if not any("router" in (L.get("mlp") or {}) for L in self.cfg["layers"]):
            return [int(t) for t in rng.integers(0, self.cfg["vocab"], n)]
        gaps = []

        def watched(scores, top):
            s = np.sort(scores)[::-1]
            gaps.append(1.0 if top == len(s) else (s[top - 1] - s[top]) / s[top - 1])
            return np.argsort(-scores, kind="stable")[:top]

        plain, so.choose = so.choose, watched
        try:
            out, state = [], so.new_state(self.cfg)
            for _ in range(n):
                for _ in range(50):
                    t, trial = int(rng.integers(0, self.cfg["vocab"])), so.copy_state(state)
                    gaps.clear()
                    so.step(self.cfg, self.W, trial, t)
                    if min(gaps) > gap:
                        break
                out.append(t)
                state = trial
        finally:
            so.choose = plain
        return out


def logit_error(got, want):
    """Largest over the rows of the root mean square difference (mean taken off), against the spread of the logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(axis=-1, keepdims=True)
    return float(np.sqrt((d * d).mean(axis=-1)).max() / want.std())
