"""Small layered models for the tests: configurations in the form of config.json, and a LanguageModel made from one
with random weights.  ("_ranks" in a mixer is this file's own key: the ranks only show in tensor shapes.)"""
import math

import numpy as np

from oracle import layered_np as ref


def attention(heads=6, kv_heads=2, dim=40, vdim=28, size=7, scale=0.21, rot=24, base=3000.0, scaling=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size}}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
        if scaling:
            m["rot"]["scaling"] = scaling
    return {"type": "attention", "mixer": m, "mlp": mlp}


def delta(heads=6, kv_heads=3, dim=48, vdim=40, conv=3, ranks=(10, 70), mlp=None):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv,
                                               "_ranks": ranks}, "mlp": mlp}


def dense(ff=90):
    return {"kind": "dense", "ff": ff}


def moe(experts=7, top=3, ff=33):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


SCALING = {"factor": 6.0, "low": 1.5, "high": 5.0, "original": 96}


def config(layers, width=104, vocab=71, eps=3e-5, mult=0.7, side=0):
    c = {"architecture": "Vudelix", "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps}, "residual_mult": mult}
    if side:
        c["token_side"] = {"dim": side}
    return c


CASES = {
    # one mechanism at a time
    "attention": config([attention()]),
    "attention_scaled_rotation": config([attention(rot=40, scaling=SCALING, size=50)]),
    "attention_no_rotation": config([attention(rot=0, size=11)]),
    "attention_odd_head": config([attention(heads=3, kv_heads=3, dim=33, vdim=19, rot=32)]),
    "attention_one_key": config([attention(size=1)]),
    "attention_12_heads_on_one": config([attention(heads=12, kv_heads=1, dim=50, vdim=20, size=40)]),
    "attention_long_window": config([attention(size=270, dim=64, vdim=64, rot=64)]),
    "attention_wide_heads": config([attention(heads=2, kv_heads=1, dim=128, vdim=256, size=30, rot=64)]),
    "delta": config([delta()]),
    "delta_equal_heads_4_taps": config([delta(heads=2, kv_heads=2, dim=64, vdim=64, conv=4, ranks=(24, 24))]),
    "delta_one_tap": config([delta(heads=4, kv_heads=1, dim=20, vdim=12, conv=1, ranks=(3, 5))]),
    "delta_wide": config([delta(heads=2, kv_heads=1, dim=160, vdim=96, conv=5, ranks=(64, 130))]),
    "delta_wider": config([delta(heads=1, kv_heads=1, dim=256, vdim=130, conv=2, ranks=(8, 8))]),
    "delta_128": config([delta(heads=3, kv_heads=3, dim=128, vdim=128, conv=4, ranks=(128, 128))]),
    "dense": config([attention(mlp=dense())]),
    "moe": config([attention(mlp=moe())]),
    "moe_all_experts": config([attention(mlp=moe(4, 4, 20))]),
    "moe_one_of_many": config([attention(mlp=moe(80, 1, 24))]),
    "side": config([attention(), attention(size=3)], side=5),
    # together
    "mixed": config([delta(mlp=dense()), attention(mlp=moe(), scaling=SCALING), delta(heads=4, kv_heads=4, conv=2, mlp=moe(9, 2, 64)),
                     attention(heads=4, kv_heads=4, dim=32, vdim=32, size=19, rot=16, mlp=None), delta(mlp=None)], side=9),
    "mixed_wide": config([attention(heads=8, kv_heads=2, dim=64, vdim=64, size=37, rot=64, mlp=dense(700)),
                          delta(heads=8, kv_heads=4, dim=64, vdim=64, conv=4, ranks=(32, 32), mlp=moe(16, 4, 96))], width=520, vocab=300,
                         side=64),
    # wide and long enough for the library's products and the tile images
    "large": config([delta(heads=10, kv_heads=5, dim=64, vdim=64, conv=4, ranks=(400, 390), mlp=moe(6, 2, 200)),
                     attention(heads=10, kv_heads=5, dim=96, vdim=80, size=70, rot=96, mlp=dense(600))], width=576, vocab=520, side=48),
}


def bits(a):
    """bf16 bit patterns of an array of bf16-representable values"""
    return (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype(np.uint16)


def settle_routers(c, t, seed):
    """Makes every choice of experts clear: the routers read features that the embedding sets to well-spaced levels, in an
    order of the token's own, and that no layer writes to."""
    rng = np.random.default_rng(seed)
    n = max([layer["mlp"]["router"]["experts"] for layer in c["layers"] if layer.get("mlp") and layer["mlp"]["kind"] == "moe"], default=0)
    if not n:
        return t
    t = {k: np.array(v) for k, v in t.items()}
    levels = np.linspace(-2.5, 2.5, n)
    for token in range(c["vocab"]):
        t["embed"][token, :n] = rng.permutation(levels)
    for name, a in t.items():
        if name.endswith((".o", ".down", ".proj")):
            a[:n] = 0.0
        if name.endswith(".router"):
            a[:] = 0.0
            a[np.arange(a.shape[0]), np.arange(a.shape[0])] = 1.5
        if name.endswith(".norm2"):
            a[:n] = 1.0
    return {k: ref.bf16(v) for k, v in t.items()}


def tensors(case, seed=0):
    return settle_routers(CASES[case], ref.random_tensors(CASES[case], seed + 1000), seed)


def language_model(pkg, c, t, seq_len=512, precision="float32"):
    from llama2_jl_amd import layered
    cfg = layered.vudelix_config(c, lambda n: t[n].shape, seq_len, precision)
    w = layered.vudelix_weights(cfg, lambda n: bits(t[n]))
    return pkg.LanguageModel(cfg, pkg.IdTokenizer(cfg.vocab_size), w)


def tokens(n, vocab, seed=5):
    return np.random.default_rng(seed).integers(0, vocab, n).astype(np.int32)


def error(got, want):
    """root mean square difference over that of the expected values, worst row (a common offset taken off)"""
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(np.asarray(want, np.float64))
    d = got - want
    d = d - d.mean(1, keepdims=True)
    w = want - want.mean(1, keepdims=True)
    return float(np.max(np.sqrt((d ** 2).mean(1))) / math.sqrt((w ** 2).mean()))


def needle(size, vocab=40, width=64, heads=4, kv_heads=2, dim=32, vdim=24, marked=3):
    """A model of one attention layer in which token `marked` has a key that every query singles out, so that one key more
    or less in the window changes the result by far more than rounding."""
    c = config([attention(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, size=size, scale=0.5, rot=0)], width=width, vocab=vocab,
               mult=1.0)
    t = {k: np.array(v) for k, v in ref.random_tensors(c, 77).items()}
    e = np.random.default_rng(1).standard_normal(dim)
    t["embed"][:, 0] = 2.0   # every token: the feature that queries are made of
    t["embed"][:, 1] = 0.0
    t["embed"][marked, 1] = 12.0  # the marked token alone: the feature its key is made of
    for n, feature in (("q", 0), ("k", 1)):
        w = t["l0.mix." + n]
        w *= 0.02 if n == "q" else 0.3
        w[:, feature] = np.tile(e, w.shape[0] // dim) * 4.0
    return c, {k: ref.bf16(v) for k, v in t.items()}
