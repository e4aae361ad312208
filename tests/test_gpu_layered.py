"""Layered models on the GPU against the numpy restatement (oracle/layered_np.py): every mechanism alone and together,
prompt passes, decoding, portions, window edges, reuse of the state, generation and the trace replay.

Bars: fp32 runs differ from the float64 restatement by rounding only (relative rms 2e-5); runs with bf16 activations by bf16
rounding (3e-2).  A close call of a router would be a difference in kind: the cases' weights leave none."""
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import layered_cases as lc
from oracle import layered_np as ref
from test_layered_host import _folder

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": 2e-5, "bfloat16": 3e-2}


def _length(case):
    return 300 if case in ("attention_long_window", "large") else 90 if "window" in case or case.startswith("mixed") else 45


def _decode(dev, toks, pos0=0):
    return np.array([dev.forward(int(t), pos0 + i)[0] for i, t in enumerate(toks)])


@pytest.fixture(scope="module")
def expected():
    cache = {}

    def get(case):
        if case not in cache:
            c = lc.CASES[case]
            t = lc.tensors(case)
            tok = lc.tokens(_length(case), c["vocab"])
            s, res, logits = ref.Sequence(c, t), [], []
            for a in tok:
                logits.append(s.step(int(a)))
                res.append(s.residuals)
            cache[case] = (c, t, tok, np.array(logits), np.array(res).transpose(1, 0, 2))
        return cache[case]
    return get


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", sorted(lc.CASES))
def test_prompt_and_decode_match(pkg, expected, case, precision):
    c, t, tok, want, residuals = expected(case)
    dev = lc.language_model(pkg, c, t, precision=precision).device()
    dev.keep_residuals()
    n = len(tok)
    got = dev.prefill_logits(tok, np.arange(n))
    e_prompt = lc.error(got, want)
    e_layer = [lc.error(dev.residuals(i, n), residuals[i]) for i in range(len(c["layers"]))]
    dev.reset()
    e_decode = lc.error(_decode(dev, tok), want)
    print("\n[%s, %s] prompt %.3g (layers %s), decode %.3g" % (case, precision, e_prompt, ["%.2g" % e for e in e_layer], e_decode))
    assert e_prompt <= TOL[precision] and max(e_layer) <= TOL[precision]
    assert e_decode <= TOL["float32"]  # decode steps are fp32 in both
    dev.close()


@pytest.mark.parametrize("library,copy", [(True, True), (False, True), (True, False), (False, False)])
def test_forms_of_the_large_products(pkg, expected, library, copy):
    """through hipBLASLt or not, experts and up projections from tile images or not: whole prompts and portions that are
    no multiple of anything"""
    c, t, tok, want, _ = expected("large")
    dev = lc.language_model(pkg, c, t, precision="bfloat16").device()
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
@pytest.mark.parametrize("case", ["mixed", "attention_long_window", "delta_wide", "delta_one_tap", "mixed_wide"])
def test_portions_do_not_change_the_logits(pkg, expected, case, precision):
    c, t, tok, want, _ = expected(case)
    dev = lc.language_model(pkg, c, t, precision=precision).device()
    n = len(tok)
    for cuts in ([2] * n, [3, 2, 16, 1, 17, 1, 1, 31, 2], [1] * 5 + [64, 2], [15, 2, 33], [n - 3, 2, 1]):
        pos, got = 0, []
        while pos < n:
            k = min(cuts[len(got) % len(cuts)] if cuts[0] != 2 else 2, n - pos)
            part = tok[pos:pos + k]
            got.append(dev.forward(int(part[0]), pos)[0][None] if k == 1 and pos else dev.prefill_logits(part, np.arange(k), pos))
            pos += k
        e = lc.error(np.concatenate(got), want)
        assert e <= TOL[precision], "portions %s: %g" % (cuts[:9], e)
    dev.close()


@pytest.mark.parametrize("size", [1, 2, 9, 32, 33, 65, 255, 257, 300])
def test_window_edges(pkg, size):
    """A marked key just inside and just outside the window, read from prompts, from portions and in decoding, the window
    starting anywhere in a tile of keys."""
    c, t = lc.needle(size)
    at = [0, 5, 31, 32, 40]
    n = max(at) + size + 4
    tok = lc.tokens(n, c["vocab"])
    tok[tok == 3] = 4
    for precision in ("float32", "bfloat16"):
        dev = lc.language_model(pkg, c, t, precision=precision, seq_len=400).device()
        for p in at:
            tk = tok.copy()
            tk[p] = 3
            want = ref.Sequence(c, t).run(tk)
            edge = [p + size - 1, p + size]
            got = dev.prefill_logits(tk, np.arange(n))
            assert lc.error(got, want) <= TOL[precision]
            for q in edge:
                assert lc.error(got[q], want[q]) <= 2 * TOL[precision]
            # a portion that begins at the last position inside, and decoding over the edge
            if edge[0] > 0:
                dev.prefill_logits(tk[:edge[0]], [], 0)
                got = dev.prefill_logits(tk[edge[0]:], np.arange(n - edge[0]), edge[0])
                assert lc.error(got[:2], want[edge[0]:edge[0] + 2]) <= TOL[precision]
                dev.prefill_logits(tk[:edge[0]], [], 0)
                got = _decode(dev, tk[edge[0]:], edge[0])
                assert lc.error(got, want[edge[0]:]) <= 1.5 * TOL[precision]
        dev.close()


def test_window_edges_would_be_noticed(pkg):
    c, t = lc.needle(33)
    tok = lc.tokens(60, c["vocab"])
    tok[tok == 3] = 4
    tok[10] = 3
    dev = lc.language_model(pkg, c, t, seq_len=64).device()
    got = dev.prefill_logits(tok, np.arange(60))
    for twist, q in (("window+1", 43), ("window-1", 42)):
        assert lc.error(got[q], ref.Sequence(c, t, twist).run(tok)[q]) > 0.3
    dev.close()


def test_first_tokens(pkg, expected):
    """sequences of 1, 2, 3 tokens: convolutions see zeros before the start, the state starts at zero"""
    for case in ("mixed", "delta_wide"):
        c, t, tok, want, _ = expected(case)
        dev = lc.language_model(pkg, c, t).device()
        for n in (1, 2, 3, 4):
            assert lc.error(dev.prefill_logits(tok[:n], np.arange(n)), want[:n]) <= TOL["float32"]
            dev.reset()
            assert lc.error(_decode(dev, tok[:n]), want[:n]) <= TOL["float32"]
        dev.close()


def test_state_is_used_again(pkg, expected):
    """Requests one after the other in the same cache and state, with and without a reset between them, give what each
    gives alone."""
    c, t, tok, want, _ = expected("mixed")
    dev = lc.language_model(pkg, c, t, precision="float32").device()
    other = lc.tokens(130, c["vocab"], 9)
    for reset in (True, False, False):
        dev.prefill_logits(other, [], 0)
        for i in range(5):
            dev.forward(int(other[i]), 130 + i)
        if reset:
            dev.reset()
        assert lc.error(dev.prefill_logits(tok[:20], np.arange(20)), want[:20]) <= TOL["float32"]
        assert lc.error(_decode(dev, tok[20:40], 20), want[20:40]) <= TOL["float32"]
    # and one that starts in decoding
    assert lc.error(_decode(dev, tok[:30]), want[:30]) <= TOL["float32"]
    dev.close()


def test_long_decoding(pkg):
    c = lc.CASES["mixed"]
    t = lc.tensors("mixed", 3)
    tok = lc.tokens(420, c["vocab"], 6)
    want = ref.Sequence(c, t).run(tok)
    dev = lc.language_model(pkg, c, t).device()
    dev.prefill_logits(tok[:3], [], 0)
    assert lc.error(_decode(dev, tok[3:], 3), want[3:]) <= TOL["float32"]
    dev.close()


def test_prompt_longer_than_one_chunk(pkg):
    """2048 positions go at a time: a longer prompt continues from the cache and state its first chunk left"""
    c = lc.config([lc.delta(heads=2, kv_heads=1, dim=16, vdim=16, conv=4, ranks=(4, 4)), lc.attention(heads=2, kv_heads=1, dim=16, vdim=16, size=40, rot=16)],
                  width=32, vocab=50)
    t = ref.random_tensors(c, 8)
    tok = lc.tokens(2100, 50, 2)
    want = ref.Sequence(c, t).run(tok)
    dev = lc.language_model(pkg, c, t, seq_len=2200).device()
    rows = np.array([0, 1, 2047, 2048, 2049, 2050, 2099])
    logits, nxt = dev.prefill_logits(tok, rows, want_next=True)
    assert lc.error(logits, want[rows]) <= TOL["float32"] and nxt == int(np.argmax(want[-1]))
    assert lc.error(dev.forward(7, 2100)[0], ref.Sequence(c, t).run(list(tok) + [7])[-1]) <= TOL["float32"]
    dev.close()


def test_strong_decay_and_saturated_steps(pkg):
    """decays that vanish within a token, decays of one, and steps near 0 and 1 all pass through the recurrence"""
    c = lc.config([lc.delta(heads=4, kv_heads=2, dim=32, vdim=32, conv=4, ranks=(16, 16))])
    t = {k: np.array(v) for k, v in ref.random_tensors(c, 4).items()}
    t["l0.mix.A_log"][:] = [6.0, 2.0, -9.0, 0.0]
    t["l0.mix.dt_bias"][:40] = 30.0
    t["l0.mix.dt_bias"][40:80] = -40.0
    t["l0.mix.b"] *= 8.0
    t = {k: ref.bf16(v) for k, v in t.items()}
    tok = lc.tokens(150, c["vocab"], 3)
    want = ref.Sequence(c, t).run(tok)
    assert np.isfinite(want).all()
    dev = lc.language_model(pkg, c, t).device()
    assert lc.error(dev.prefill_logits(tok, np.arange(150)), want) <= TOL["float32"]
    dev.reset()
    assert lc.error(_decode(dev, tok), want) <= TOL["float32"]
    dev.close()


def test_greedy_generation(pkg):
    c, t = lc.CASES["mixed"], lc.tensors("mixed")
    prompt = lc.tokens(11, c["vocab"], 8)
    want = ref.greedy(c, t, prompt, 40)
    for precision in ("float32", "bfloat16"):
        m = lc.language_model(pkg, c, t, precision=precision)
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
    c, t = lc.CASES["mixed"], lc.tensors("mixed")
    m = lc.language_model(pkg, c, t)
    prompt = [int(a) for a in lc.tokens(5, c["vocab"], 8)]
    out = io.StringIO()
    pkg.sample(m, " ".join(map(str, prompt)), temperature=0.0, bos_token=False, max_seq_len=25, out=out)
    ids = [int(w) for w in out.getvalue().split("\n")[0].split()]
    assert ids == prompt + ref.greedy(c, t, prompt, 25 - len(prompt) + 1)
    # temperature: the probabilities of the device are those of the restatement's logits
    dev = m.device()
    dev.reset()
    dev.prefill(np.array(prompt, np.int32))
    tok, p = dev.sample_token(0.8, 0.37, want_probs=True)
    z = ref.Sequence(c, t).run(prompt)[-1] / 0.8
    q = np.exp(z - z.max())
    q /= q.sum()
    assert np.abs(p - q).max() < 1e-5 and tok == int(np.searchsorted(np.cumsum(q), 0.37))
    dev.close()


def test_argument_checks(pkg, expected):
    c, t, tok, _, _ = expected("mixed")
    m = lc.language_model(pkg, c, t, seq_len=64)
    dev = m.device()
    E = pkg.L2HError
    dev.prefill_logits(tok[:10], [], 0)
    for call in (lambda: dev.forward(1, 9), lambda: dev.forward(1, 11), lambda: dev.prefill_logits(tok[:3], [], 5),
                 lambda: dev.prefill_logits(tok[:60], [], 10), lambda: dev.prefill_logits([c["vocab"]], [], 10),
                 lambda: dev.prefill_logits(tok[:4], [2, 1], 10), lambda: dev.prefill_logits(tok[:4], [4], 10),
                 lambda: dev.kv_read(0, 0, 1), lambda: dev.set_wait_limit(5), lambda: dev.profile_matvec(5), lambda: dev.get_tensor(5, 0, 4)):
        with pytest.raises((E, ValueError)):
            call()
    dev.forward(1, 10)  # still whole
    dev.close()
    with pytest.raises(E):
        m.device(path=3)
    broken = lc.language_model(pkg, c, t)
    broken.weights.tensors.pop(next(k for k in broken.weights.tensors if len(k) == 3))
    with pytest.raises(E, match="expert"):
        broken.device()
    bad = dict(t, **{"l0.mlp.up": t["l0.mlp.up"][:-1]})
    with pytest.raises(E, match="shape"):
        lc.language_model(pkg, c, bad).device()


def test_prefill_logits_of_a_llama_model(pkg):
    """the wanted-rows form of the prompt pass on a GGUF-style model: the last row is what the plain form returns"""
    from llama2_jl_amd import synth
    cfg = pkg.ModelConfig(dim=256, hidden_dim=512, n_layers=2, n_heads=4, n_kv_heads=2, vocab_size=320, seq_len=64)
    dev = synth.synthetic_model(cfg, synth.PLAN_Q4_K_S, seed=7).device()
    tok = synth.seeded_prompt(3, 20, 320)
    last, nxt = dev.prefill(tok)
    rows, nxt2 = dev.prefill_logits(tok, [4, 19], 0, want_next=True)
    four, _ = dev.prefill(tok[:5])
    assert np.array_equal(rows[1], last) and nxt == nxt2 and lc.error(rows[0], four) < 1e-2
    dev.close()


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_replay(pkg, tmp_path, dtype):
    c, t = lc.CASES["mixed"], lc.tensors("mixed")
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
