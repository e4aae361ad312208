"""Layered models that mix the mechanisms of different designs: every mixer with one norm or two, gated feed-forwards or plain
ones, both kinds of router, either rotation, per-token input and loops, against oracle/combined_np.py."""
import numpy as np
import pytest

import layered_cases as lc
import lezepel_cases as zc
from oracle import combined_np as ref
from oracle import layered_np, lezepel_np

pytestmark = pytest.mark.gpu
TOL = {"float32": 2e-5, "bfloat16": 3e-2}


def _layer(of, parallel, gated=False, act="relu2", route="sigmoid_in", bias=False, rot_half=False):
    return dict(of, parallel=parallel, gated=gated, act=act, route=route, bias=bias, rot_half=rot_half)


def _case(layers, loop=None, side=0, mult=0.7):
    return {"layers": layers, "width": 104, "vocab": 61, "norm": {"eps": 2e-5}, "residual_mult": mult, "embed_scale": 1.5, "loop": loop,
            "side": side}


CASES = {
    "window_parallel_dense_gated": _case([_layer(lc.attention(mlp=lc.dense()), True, True, "silu", rot_half=True)]),
    "window_parallel_dense_plain": _case([_layer(lc.attention(dim=33, vdim=19, rot=32, mlp=lc.dense()), True, False, "gelu_tanh", rot_half=True)]),
    "delta_parallel_dense_gated": _case([_layer(lc.delta(mlp=lc.dense()), True, True, "gelu_erf")]),
    "delta_parallel_experts": _case([_layer(lc.delta(mlp=lc.moe()), True, True, "relu", "sigmoid_in", True)]),
    "window_two_norms_gated": _case([_layer(lc.attention(mlp=lc.dense()), False, True, "silu")]),
    "window_two_norms_experts": _case([_layer(lc.attention(mlp=lc.moe()), False, True, "silu", "softmax_out", True)]),
    "latent_two_norms": _case([_layer(zc.layer(mlp=zc.dense()), False, False, "relu2")]),
    "latent_parallel_plain": _case([_layer(zc.layer(mlp=zc.dense()), True, False, "gelu_erf")]),
    "latent_experts_plain": _case([_layer(zc.layer(mlp=zc.moe()), True, False, "relu2", "softmax_out")]),
    "latent_experts_weight_in": _case([_layer(zc.layer(mlp=zc.moe()), False, True, "silu", "sigmoid_in")]),
    "all": _case([_layer(lc.delta(mlp=lc.dense()), False), _layer(lc.attention(mlp=lc.moe()), True, True, "silu", "softmax_out", True, True),
                  _layer(zc.layer(mlp=zc.dense()), True, True, "relu"), _layer(lc.delta(heads=4, kv_heads=4, conv=2, mlp=None), True),
                  _layer(zc.layer(heads=2, mlp=zc.moe()), False, False, "relu2", "sigmoid_in")], loop=(1, 4, 2), side=7),
}


def _model(pkg, c, t, precision):
    from llama2_jl_amd import _lib as L
    from llama2_jl_amd import layered
    layers, names = [], {"embed": (L.TOK_EMB, 0), "final.norm": (L.RMS_FINAL, 0), "head": (L.OUTPUT, 0), "loop.step": (L.LOOP_STEP, 0),
                         "side.embed": (L.SIDE_EMB, 0)}
    for i, s in enumerate(c["layers"]):
        own = {"layers": [dict(s, mlp=None)], "width": c["width"], "vocab": c["vocab"], "norm": c["norm"], "residual_mult": 1.0,
               "embedding": {"scale": 1.0}}
        if s["type"] == "latent_attention":
            spec, mix = layered.lezepel_config(own).layers[0], layered._LATENT_NAMES
        else:
            spec = layered.vudelix_config(own, lambda n: t["l%d." % i + n[3:]].shape).layers[0]
            mix = layered._ATTENTION_NAMES if s["type"] == "attention" else layered._DELTA_NAMES
            spec.rot_half = s["rot_half"]
        spec.parallel, spec.ff_gated, spec.ff_act = s["parallel"], s["gated"], list(ref.ACTS).index(s["act"])
        spec.route, spec.router_bias, spec.ff = ["sigmoid_in", "softmax_out"].index(s["route"]), s["bias"], layered.FF_NONE
        p, f = "l%d." % i, s.get("mlp")
        names.update({p + "mix." + n: (role, i) for n, role in mix.items()})
        names.update({p + "norm1": (L.RMS_ATT, i), p + "norm2": (L.RMS_FFN, i), p + "mlp.router": (L.ROUTER, i),
                      p + "mlp.router.b": (L.ROUTER_BIAS, i), p + "mlp.down": (L.W2, i), p + "mlp.gate": (L.W1, i),
                      p + "mlp.up": (L.W3 if s["gated"] else L.W1, i)})
        names.update({p + "side." + n: (role, i) for n, role in layered._SIDE_NAMES.items()})
        if f and f["kind"] == "dense":
            spec.ff, spec.ff_dim = layered.FF_DENSE, f["ff"]
        if f and f["kind"] == "moe":
            spec.ff, spec.ff_dim, spec.n_experts, spec.top = layered.FF_EXPERTS, f["expert"]["ff"], f["router"]["experts"], f["router"]["top"]
            for e in range(spec.n_experts):
                for n, role in (("gate", L.EXPERT_GATE), ("up", L.EXPERT_UP), ("down", L.EXPERT_DOWN)):
                    names[p + "mlp.e%d.%s" % (e, n)] = (role, i, e)
        layers.append(spec)
    cfg = layered.LayeredConfig(width=c["width"], vocab_size=c["vocab"], layers=layers, norm_eps=c["norm"]["eps"],
                                residual_mult=c["residual_mult"], embed_scale=c["embed_scale"], side_dim=c["side"], loop=c["loop"],
                                seq_len=128, precision=precision)
    w = layered.LayeredWeights({names[n]: lc.bits(a) for n, a in t.items()})
    return pkg.LanguageModel(cfg, pkg.IdTokenizer(c["vocab"]), w)


def _tensors(c, seed):
    rng, out = np.random.default_rng(seed), {}
    one = layered_np.random_tensors(lc.config([lc.delta()]), seed)  # (for the ranges of the delta rule's own vectors)
    for name, shape in ref.tensor_shapes(c).items():
        last = name.split(".")[-1]
        if last in ("norm", "norm1", "norm2"):
            v = 1.0 + 0.3 * rng.standard_normal(shape)
        elif last in ("A_log", "dt_bias"):
            v = rng.choice(one["l0.mix." + last].reshape(-1), shape)
        elif last in ("conv", "step"):
            v = 0.6 * rng.standard_normal(shape)
        elif last in ("embed", "b"):
            v = rng.standard_normal(shape)
        else:
            v = (3.0 if last == "router" else 1.4) * rng.standard_normal(shape) / np.sqrt(shape[-1])
        out[name] = lezepel_np.bf16(v)
    return out


# (random routers have close calls, which bf16 rounding of their input may decide either way)
RUNS = [(case, precision) for case, c in sorted(CASES.items()) for precision in sorted(TOL)
        if precision == "float32" or not any(s.get("mlp") and s["mlp"]["kind"] == "moe" for s in c["layers"])]


@pytest.mark.parametrize("case,precision", RUNS)
def test_prompt_portions_and_decode(pkg, case, precision):
    c = CASES[case]
    t = _tensors(c, 5)
    tok = lc.tokens(60, c["vocab"])
    want = ref.Sequence(c, t).run(tok)
    dev = _model(pkg, c, t, precision).device()
    assert lc.error(dev.prefill_logits(tok, np.arange(60)), want) <= TOL[precision]
    got = [dev.prefill_logits(tok[a:b], np.arange(b - a), a) for a, b in ((0, 2), (2, 25), (25, 30), (30, 50))]
    got.append(np.array([dev.forward(int(k), 50 + i)[0] for i, k in enumerate(tok[50:])]))
    assert lc.error(np.concatenate(got), want) <= TOL[precision]
    dev.reset()
    assert lc.error([dev.forward(int(k), i)[0] for i, k in enumerate(tok)], want) <= TOL["float32"]
    dev.close()
