"""Lezepel on the GPU against its numpy restatement (oracle/lezepel_np.py): every mechanism alone and together, prompt
passes, decoding, portions, marked keys far away and at every border, reuse of the cache, generation and the trace replay.

Bars as in test_gpu_layered.py: fp32 runs differ from the float64 restatement by rounding only (relative rms 2e-5), runs with
bf16 activations by bf16 rounding (3e-2)."""
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import layered_cases as lc
import lezepel_cases as zc
from oracle import lezepel_np as ref
from test_layered_host import _folder

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": 2e-5, "bfloat16": 3e-2}


def _length(case):
    return 300 if case == "large" else 90 if case.startswith(("mixed", "latent_17")) else 45


def _decode(dev, toks, pos0=0):
    return np.array([dev.forward(int(t), pos0 + i)[0] for i, t in enumerate(toks)])


@pytest.fixture(scope="module")
def expected():
    cache = {}

    def get(case):
        if case not in cache:
            c = zc.CASES[case]
            t = zc.tensors(case)
            tok = lc.tokens(_length(case), c["vocab"])
            s, res, logits = ref.Sequence(c, t), [], []
            for a in tok:
                logits.append(s.step(int(a)))
                res.append(s.residuals)
            cache[case] = (c, t, tok, np.array(logits), np.array(res).transpose(1, 0, 2))
        return cache[case]
    return get


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", sorted(zc.CASES))
def test_prompt_and_decode_match(pkg, expected, case, precision):
    c, t, tok, want, residuals = expected(case)
    dev = zc.language_model(pkg, c, t, precision=precision).device()
    dev.keep_residuals()
    n = len(tok)
    got = dev.prefill_logits(tok, np.arange(n))
    e_prompt = lc.error(got, want)
    e_layer = [lc.error(dev.residuals(i, n), residuals[i]) for i in range(len(residuals))]
    dev.reset()
    e_decode = lc.error(_decode(dev, tok), want)
    print("\n[%s, %s] prompt %.3g (layers %s), decode %.3g" % (case, precision, e_prompt, ["%.2g" % e for e in e_layer], e_decode))
    assert e_prompt <= TOL[precision] and max(e_layer) <= TOL[precision]
    assert e_decode <= TOL["float32"]  # decode steps are fp32 in both
    dev.close()


@pytest.mark.parametrize("library,copy", [(True, True), (False, True), (True, False), (False, False)])
def test_forms_of_the_large_products(pkg, expected, library, copy):
    """through hipBLASLt or not, gated up projections from tile images or not: whole prompts and portions that are no
    multiple of anything"""
    c, t, tok, want, _ = expected("large")
    dev = zc.language_model(pkg, c, t, precision="bfloat16").device()
    dev.set_prefill_library(library)
    dev.set_prefill_copy(copy)
    n = len(tok)
    assert lc.error(dev.prefill_logits(tok, np.arange(n)), want) <= TOL["bfloat16"]
    first = dev.prefill_logits(tok[:137], np.arange(137))
    rest = dev.prefill_logits(tok[137:], np.arange(n - 137), 137)
    assert lc.error(np.concatenate([first, rest]), want) <= TOL["bfloat16"]
    assert lc.error(dev.prefill_logits(tok[:190], [188, 189]), want[188:190]) <= TOL["bfloat16"]
    dev.close()


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", ["mixed", "latent_17_heads", "latent_odd_sizes", "latent_beyond_tiles", "loop_inside", "mixed_wide"])
def test_portions_do_not_change_the_logits(pkg, expected, case, precision):
    c, t, tok, want, _ = expected(case)
    dev = zc.language_model(pkg, c, t, precision=precision).device()
    n = len(tok)
    for cuts in ([2] * n, [3, 2, 16, 1, 17, 1, 1, 31, 2], [1] * 5 + [64, 2], [15, 2, 33], [18] * n, [n - 3, 2, 1]):
        pos, got = 0, []
        while pos < n:
            k = min(cuts[len(got) % len(cuts)], n - pos)
            part = tok[pos:pos + k]
            got.append(dev.forward(int(part[0]), pos)[0][None] if k == 1 and pos else dev.prefill_logits(part, np.arange(k), pos))
            pos += k
        e = lc.error(np.concatenate(got), want)
        assert e <= TOL[precision], "portions %s: %g" % (cuts[:9], e)
    dev.close()


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
def test_marked_key_at_every_border(pkg, precision):
    """A marked key at the borders of tiles and of the runs of keys that workgroups take, near and far, read from a prompt,
    from portions on both paths, and in decoding."""
    c, t = zc.needle()
    n = 330
    base = lc.tokens(n, c["vocab"])
    base[base == 3] = 4
    dev = zc.language_model(pkg, c, t, precision=precision, seq_len=400).device()
    for p in (0, 1, 15, 16, 31, 32, 63, 64, 127, 128, 255, 256, 300):
        tok = base.copy()
        tok[p] = 3
        want = ref.Sequence(c, t).run(tok)
        rows = sorted({p, p + 1, min(p + 31, n - 1), n - 26, n - 25, n - 1})
        got = dev.prefill_logits(tok, rows)
        for g, q in zip(got, rows):
            assert lc.error(g, want[q]) <= 2 * TOL[precision], "key %d from %d" % (p, q)
        dev.prefill_logits(tok[:n - 30], [], 0)
        for at, k in ((n - 30, 20), (n - 10, 5)):  # more and fewer than sixteen tokens
            assert lc.error(dev.prefill_logits(tok[at:at + k], np.arange(k), at), want[at:at + k]) <= 1.5 * TOL[precision]
        assert lc.error(_decode(dev, tok[n - 5:], n - 5), want[n - 5:]) <= 1.5 * TOL[precision]
    dev.close()


def test_a_lost_key_would_be_noticed(pkg):
    c, t = zc.needle()
    tok = lc.tokens(250, c["vocab"])
    tok[tok == 3] = 4
    tok[0] = 3
    dev = zc.language_model(pkg, c, t, seq_len=256).device()
    got = dev.prefill_logits(tok, [249])
    assert lc.error(got[0], ref.Sequence(c, t, "loses_first").run(tok)[249]) > 0.1
    dev.close()


def test_passes_of_a_loop_keep_their_own_caches(pkg, expected):
    c, t, tok, want, _ = expected("loop_inside")
    dev = zc.language_model(pkg, c, t).device()
    dev.prefill_logits(tok[:20], [], 0)
    got = _decode(dev, tok[20:40], 20)
    assert lc.error(got, want[20:40]) <= TOL["float32"]
    assert lc.error(ref.Sequence(c, t, "shared_cache").run(tok)[20:40], want[20:40]) > 1e-2
    dev.close()


def test_first_tokens(pkg, expected):
    for case in ("mixed", "latent_17_heads"):
        c, t, tok, want, _ = expected(case)
        for precision in ("float32", "bfloat16"):
            dev = zc.language_model(pkg, c, t, precision=precision).device()
            for n in (1, 2, 3, 4):
                assert lc.error(dev.prefill_logits(tok[:n], np.arange(n)), want[:n]) <= TOL[precision]
                dev.reset()
                assert lc.error(_decode(dev, tok[:n]), want[:n]) <= TOL["float32"]
            dev.close()


def test_cache_is_used_again(pkg, expected):
    """Requests one after the other in the same cache, with and without a reset between them, give what each gives alone."""
    c, t, tok, want, _ = expected("mixed")
    for precision in ("float32", "bfloat16"):
        dev = zc.language_model(pkg, c, t, precision=precision).device()
        other = lc.tokens(130, c["vocab"], 9)
        for reset in (True, False, False):
            dev.prefill_logits(other, [], 0)
            for i in range(5):
                dev.forward(int(other[i]), 130 + i)
            if reset:
                dev.reset()
            assert lc.error(dev.prefill_logits(tok[:20], np.arange(20)), want[:20]) <= TOL[precision]
            assert lc.error(_decode(dev, tok[20:40], 20), want[20:40]) <= TOL[precision]
        dev.reset()
        assert lc.error(_decode(dev, tok[:30]), want[:30]) <= TOL["float32"]
        dev.close()


def test_long_decoding(pkg):
    c = zc.CASES["mixed"]
    t = zc.tensors("mixed", 3)
    tok = lc.tokens(420, c["vocab"], 6)
    want = ref.Sequence(c, t).run(tok)
    dev = zc.language_model(pkg, c, t).device()
    dev.prefill_logits(tok[:3], [], 0)
    assert lc.error(_decode(dev, tok[3:], 3), want[3:]) <= TOL["float32"]
    dev.close()


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
def test_prompt_longer_than_one_chunk(pkg, precision):
    """2048 positions go at a time, and so do the cached positions whose keys are made anew"""
    c = zc.config([zc.layer(heads=2, dim=12, rot_dim=4, vdim=16, kv_rank=20, q_rank=24)], width=32, vocab=50)
    t = ref.random_tensors(c, 8)
    tok = lc.tokens(2140, 50, 2)
    want = ref.Sequence(c, t).run(tok)
    dev = zc.language_model(pkg, c, t, seq_len=2200, precision=precision).device()
    rows = np.array([0, 1, 2047, 2048, 2049, 2050, 2099])
    logits, nxt = dev.prefill_logits(tok[:2100], rows, want_next=True)
    assert lc.error(logits, want[rows]) <= TOL[precision]
    assert precision == "bfloat16" or nxt == int(np.argmax(want[2099]))
    assert lc.error(dev.prefill_logits(tok[2100:2137], np.arange(37), 2100), want[2100:2137]) <= TOL[precision]
    assert lc.error(_decode(dev, tok[2137:], 2137), want[2137:]) <= TOL[precision]
    dev.close()


def test_greedy_generation(pkg):
    c, t = zc.CASES["mixed"], zc.tensors("mixed")
    prompt = lc.tokens(11, c["vocab"], 8)
    want = ref.greedy(c, t, prompt, 40)
    for precision in ("float32", "bfloat16"):
        m = zc.language_model(pkg, c, t, precision=precision)
        assert pkg.generate(m, prompt, 40).tolist() == want
        # the prompt through the prompt pass, then the token loop
        dev = m.device()
        dev.reset()
        _, nxt = dev.prefill(prompt)
        ids = dev.generate_greedy([nxt], 39, pos0=len(prompt))
        if precision == "float32":
            assert [nxt] + ids.tolist() == want
        dev.close()


def test_sample_through_the_text_entry_point(pkg):
    c, t = zc.CASES["mixed"], zc.tensors("mixed")
    m = zc.language_model(pkg, c, t)
    prompt = [int(a) for a in lc.tokens(5, c["vocab"], 8)]
    out = io.StringIO()
    pkg.sample(m, " ".join(map(str, prompt)), temperature=0.0, bos_token=False, max_seq_len=25, out=out)
    ids = [int(w) for w in out.getvalue().split("\n")[0].split()]
    assert ids == prompt + ref.greedy(c, t, prompt, 25 - len(prompt) + 1)
    m.device().close()


def test_argument_checks(pkg, expected):
    import copy
    c, t, tok, _, _ = expected("mixed")
    m = zc.language_model(pkg, c, t, seq_len=64)
    dev = m.device()
    E = pkg.L2HError
    dev.prefill_logits(tok[:10], [], 0)
    for call in (lambda: dev.forward(1, 9), lambda: dev.prefill_logits(tok[:3], [], 5), lambda: dev.prefill_logits(tok[:60], [], 10)):
        with pytest.raises(E):
            call()
    dev.forward(1, 10)  # still whole
    dev.close()
    for change, what in ((lambda f: setattr(f, "loop", (0, 9, 2)), "run"), (lambda f: setattr(f, "loop", (2, 2, 2)), "run"),
                         (lambda f: setattr(f.layers[0], "kv_rank", 5000), "ranks"), (lambda f: setattr(f.layers[0], "n_kv_heads", 1), "head"),
                         (lambda f: setattr(f.layers[0], "rot_dims", 99), "rotated"), (lambda f: setattr(f.layers[1], "top", 99), "experts"),
                         (lambda f: setattr(f.layers[1], "route", 7), "router")):
        bad = zc.language_model(pkg, c, t)
        bad.config = copy.deepcopy(bad.config)
        change(bad.config)
        with pytest.raises(E, match=what):
            bad.device()
    for name in ("l1.mlp.e3.gate", "l0.mlp.up", "loop.step", "l2.mlp.router.b", "l3.mix.dkv.norm"):
        from llama2_jl_amd import layered
        lost = zc.language_model(pkg, c, t)
        lost.weights.tensors.pop(layered.lezepel_names(lost.config)[name])
        with pytest.raises(E, match="missing"):
            lost.device()


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_replay(pkg, tmp_path, dtype):
    c, t = zc.CASES["mixed"], zc.tensors("mixed")
    d = _folder(tmp_path, c, t)
    a, b = lc.tokens(50, c["vocab"], 1), lc.tokens(30, c["vocab"], 2)
    steps, expect = [], []
    for name, tok, cuts in (("a", a, [20, 2, 1, 1, 26]), ("b", b, [1, 1, 28])):
        want, pos = ref.Sequence(c, t).run(tok), 0
        for k in cuts:
            w = [0, k - 1] if k > 1 else [0]
            steps.append({"step": len(steps), "entries": [{"id": name, "tokens": tok[pos:pos + k].tolist(), "want": w if pos != 20 else []}],
                          "end": [name] if pos + k == len(tok) else []})
            expect.append(want[[pos + i for i in w]] if pos != 20 else None)
            pos += k
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(d), "--dtype", dtype, "--out", str(out), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110,
                       env=dict(os.environ, PATH=os.path.dirname(sys.executable) + os.pathsep + os.environ["PATH"]))
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(len(steps))]
    for i, want in enumerate(expect):
        f = out / ("%d.f32" % i)
        assert f.exists() == (want is not None)
        if want is not None:
            assert lc.error(np.fromfile(f, "<f4").reshape(want.shape), want) <= TOL[dtype]
