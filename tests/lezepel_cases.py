"""Small Lezepel models for the tests: configurations in the form of config.json, and a LanguageModel made from one with
random weights."""
import numpy as np

from layered_cases import bits
from oracle import lezepel_np as ref


def layer(heads=3, dim=20, rot_dim=6, vdim=12, kv_rank=28, q_rank=36, scale=0.23, base=900.0, dims=None, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
                      "rot": {"base": base, "dims": rot_dim if dims is None else dims}}}


def dense(ff=90):
    return {"kind": "dense", "ff": ff}


def moe(experts=7, top=3, ff=33):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def config(layers, width=104, vocab=71, eps=3e-5, scale=2.5, loop=None):
    c = {"architecture": "Lezepel", "embedding": {"scale": scale}, "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps}}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CASES = {
    # one mechanism at a time
    "latent": config([layer()]),
    "latent_odd_sizes": config([layer(heads=5, dim=7, rot_dim=2, vdim=9, kv_rank=13, q_rank=11)], width=75),
    "latent_one_head": config([layer(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, q_rank=1)], width=33),
    "latent_17_heads": config([layer(heads=17, dim=24, rot_dim=8, vdim=40, kv_rank=64, q_rank=48)]),
    "latent_rotated_part_larger": config([layer(heads=4, dim=8, rot_dim=56, vdim=32, base=50.0)]),
    "latent_part_of_it_turned": config([layer(rot_dim=14, dims=8)]),
    "latent_192": config([layer(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=160, q_rank=96, scale=0.07)]),
    "latent_96_80": config([layer(heads=3, dim=60, rot_dim=36, vdim=80, kv_rank=66, q_rank=40, scale=0.1)]),
    "latent_beyond_tiles": config([layer(heads=2, dim=200, rot_dim=40, vdim=150, kv_rank=100, q_rank=130, scale=0.05)]),
    "latent_large_rank": config([layer(heads=2, dim=16, rot_dim=16, vdim=70, kv_rank=600, q_rank=300)]),
    "latent_rank_300": config([layer(heads=9, dim=16, rot_dim=18, vdim=33, kv_rank=300, q_rank=70)]),
    "dense": config([layer(mlp=dense())]),
    "dense_wide": config([layer(mlp=dense(333))]),
    "moe": config([layer(mlp=moe())]),
    "moe_all_experts": config([layer(mlp=moe(4, 4, 20))]),
    "moe_one_of_many": config([layer(mlp=moe(80, 1, 24))]),
    "loop": config([layer(), layer(heads=2)], loop=(0, 2, 2)),
    "loop_inside": config([layer(), layer(heads=2), layer(dim=10), layer()], loop=(1, 3, 3)),
    "loop_once": config([layer(), layer(heads=2)], loop=(1, 2, 1)),
    # together
    "mixed": config([layer(mlp=dense()), layer(heads=5, mlp=moe(9, 2, 64)), layer(kv_rank=40, mlp=moe()), layer(mlp=None)], loop=(0, 3, 2)),
    "mixed_wide": config([layer(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=128, q_rank=192, scale=0.1, mlp=dense(700)),
                          layer(heads=8, dim=64, rot_dim=32, vdim=48, kv_rank=128, q_rank=192, scale=0.1, mlp=moe(16, 4, 96))], width=520,
                         vocab=300, loop=(1, 2, 2)),
    # wide and long enough for the library's products and the tile images
    "large": config([layer(heads=10, dim=96, rot_dim=32, vdim=80, kv_rank=200, q_rank=300, scale=0.08, mlp=moe(6, 2, 200)),
                     layer(heads=10, dim=96, rot_dim=32, vdim=80, kv_rank=200, q_rank=300, scale=0.08, mlp=dense(600))], width=576, vocab=520),
}


def settle_routers(c, t, seed):
    """Makes every choice of experts clear: the routers read features that the embedding sets to well-spaced levels, in an
    order of the token's own, and that nothing else writes to; the bias sets the even experts before the odd ones."""
    rng = np.random.default_rng(seed)
    n = max([a["mlp"]["router"]["experts"] for a in c["layers"] if a.get("mlp") and a["mlp"]["kind"] == "moe"], default=0)
    if not n:
        return t
    t = {k: np.array(v) for k, v in t.items()}
    levels = np.linspace(-2.5, 2.5, n) / c["embedding"]["scale"]
    for token in range(c["vocab"]):
        t["embed"][token, :n] = rng.permutation(levels)
    for name, a in t.items():
        if name.endswith((".o", ".down")):
            a[:n] = 0.0
        if name.endswith(".router"):
            a[:] = 0.0
            a[np.arange(a.shape[0]), np.arange(a.shape[0])] = 0.7
        if name.endswith(".router.b"):
            a[:] = 4.0 * (np.arange(a.size) % 2 == 0) + 0.01 * rng.standard_normal(a.size)
        if name.endswith(".norm1"):
            a[:n] = 1.0
        if name == "loop.step":
            a[:, :n] = 0.0
    return {k: ref.bf16(v) for k, v in t.items()}


def tensors(case, seed=0):
    return settle_routers(CASES[case], ref.random_tensors(CASES[case], seed + 1000), seed)


def language_model(pkg, c, t, seq_len=512, precision="float32"):
    from llama2_jl_amd import layered
    cfg = layered.lezepel_config(c, seq_len, precision)
    w = layered.lezepel_weights(cfg, lambda n: bits(t[n]))
    return pkg.LanguageModel(cfg, pkg.IdTokenizer(cfg.vocab_size), w)


def needle(vocab=40, width=64, heads=4, dim=24, rot_dim=8, vdim=20, kv_rank=32, q_rank=20, marked=3):
    """A model of one layer in which token `marked` has a key that every query singles out (about as strong as two hundred
    others), so that one key more or less changes the result by far more than rounding."""
    c = config([layer(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale=0.4)], width=width, vocab=vocab, scale=1.0)
    t = {k: np.array(v) for k, v in ref.random_tensors(c, 77).items()}
    e = np.random.default_rng(1).standard_normal(dim)
    t["embed"][:, 0] = 2.0        # every token: the feature that queries are made of
    t["embed"][:, 1] = 0.0
    t["embed"][marked, 1] = 12.0  # the marked token alone: the feature its key is made of
    for n in ("dq.norm", "dkv.norm", "dq", "dkv", "uq", "uk"):
        t["l0.mix." + n] *= 1.0 if n.endswith("norm") else 0.2
    t["l0.mix.dq"][0, 0], t["l0.mix.dkv"][0, 1] = 3.0, 2.0
    t["l0.mix.dkv"][kv_rank:] *= 0.2
    for h in range(heads):
        t["l0.mix.uq"][h * (dim + rot_dim):h * (dim + rot_dim) + dim, 0] = e * 0.3
        t["l0.mix.uk"][h * dim:(h + 1) * dim, 0] = e * 0.3
    return c, {k: ref.bf16(v) for k, v in t.items()}
