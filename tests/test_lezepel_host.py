"""Lezepel without a GPU: that every mistake planted in the restatement would show, the restatement's parts by hand, and the
reader of model folders."""
import json

import numpy as np
import pytest

import layered_cases as lc
import lezepel_cases as zc
from oracle import lezepel_np as ref
from test_layered_host import _folder


def test_every_planted_mistake_shows():
    c, t = zc.CASES["mixed"], zc.tensors("mixed")
    tok = lc.tokens(40, c["vocab"])
    good = ref.Sequence(c, t).run(tok)
    for twist in ref.TWISTS:
        err = lc.error(ref.Sequence(c, t, twist).run(tok), good)
        assert err > 1e-2, "%s changes the logits by %g only" % (twist, err)


def test_one_far_key_shows():
    """the first position's key, 250 positions back, when it is the marked one; not so without the mark"""
    c, t = zc.needle()
    tok = lc.tokens(250, c["vocab"])
    tok[tok == 3] = 4
    tok[0] = 3
    good, bad = ref.Sequence(c, t).run(tok), ref.Sequence(c, t, "loses_first").run(tok)
    assert lc.error(bad[-1], good[-1]) > 0.1


def test_rotation_by_hand():
    f = ref.rot_frequencies(4, 100.0)
    assert np.allclose(f, [1.0, 0.1])
    y = ref.rotate_half(np.array([1.0, 0.0, 0.0, 2.0, 7.0]), 3, f)
    assert np.allclose(y, [np.cos(3.0), -2.0 * np.sin(0.3), np.sin(3.0), 2.0 * np.cos(0.3), 7.0])
    # scores depend on the distance only
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((2, 4))
    assert np.isclose(ref.rotate_half(q, 9, f) @ ref.rotate_half(k, 4, f), ref.rotate_half(q, 105, f) @ ref.rotate_half(k, 100, f))


def test_route_by_hand():
    idx, w, _ = ref.route(np.array([1.0]), np.array([[0.0], [3.0], [1.0]]), np.array([2.5, 0.0, 0.5]), 2)
    assert list(idx) == [1, 0] and np.allclose(w, np.exp([3.0, 2.5]) / np.exp([3.0, 2.5]).sum())


def test_queries_through_k_up_give_the_same_scores():
    """what the cache of latents rests on: q . (U c) = (U^T q) . c, and the weighted sum of U c is U times the weighted sum"""
    rng = np.random.default_rng(4)
    q, U, c, p = rng.standard_normal(6), rng.standard_normal((6, 9)), rng.standard_normal((5, 9)), rng.random(5)
    assert np.allclose((c @ U.T) @ q, c @ (U.T @ q)) and np.allclose(p @ (c @ U.T), U @ (p @ c))


def test_order_of_layer_runs(pkg):
    from llama2_jl_amd import layered
    for name, want in (("loop_inside", [0, 1, 2, 1, 2, 1, 2, 3]), ("loop_once", [0, 1]), ("latent", [0]), ("mixed", [0, 1, 2, 0, 1, 2, 3])):
        assert layered.lezepel_config(zc.CASES[name]).runs == want == [i for i, _ in ref.layer_runs(zc.CASES[name])]


def test_shapes_agree(pkg):
    from llama2_jl_amd import layered
    for c in zc.CASES.values():
        assert layered.lezepel_shapes(layered.lezepel_config(c)) == ref.tensor_shapes(c)


def test_model_folder_reader(pkg, tmp_path):
    c, t = zc.CASES["mixed"], zc.tensors("mixed")
    d = _folder(tmp_path, c, t)
    m = pkg.load_model(str(d), seq_len=33, precision="float32")
    cfg = m.config
    assert (cfg.architecture, cfg.n_layers, cfg.seq_len, cfg.loop, cfg.embed_scale) == ("Lezepel", 4, 33, (0, 3, 2), 2.5)
    assert [s.ff for s in cfg.layers] == [1, 2, 2, 0] and [s.n_heads for s in cfg.layers] == [3, 5, 3, 3]
    assert all(s.parallel and s.rot_half and s.out_gate for s in cfg.layers)
    assert len(m.weights.tensors) == len(t)  # every tensor has a place
    raw = json.loads((d / "config.json").read_text())
    for change in (lambda r: r.pop("embedding"), lambda r: r["layers"][1].update(type="attention"), lambda r: r["loop"].pop("times"),
                   lambda r: r["layers"][1]["mixer"].pop("kv_rank"), lambda r: r["layers"][0]["mlp"].update(kind="odd"),
                   lambda r: r["layers"][0]["mixer"].pop("rot"), lambda r: r["layers"].append(r["layers"][0])):
        r = json.loads(json.dumps(raw))
        change(r)
        (d / "config.json").write_text(json.dumps(r))
        with pytest.raises(ValueError):
            pkg.load_model(str(d))
    # a model without a loop
    r = json.loads(json.dumps(raw))
    r["loop"] = None
    (d / "config.json").write_text(json.dumps(r))
    assert pkg.load_model(str(d)).config.runs == [0, 1, 2, 3]


def test_work_of_the_bench_models(pkg):
    from llama2_jl_amd import bench_layered, layered
    cfg, _ = bench_layered.config("lezepel-tiny")
    by, fl = bench_layered.work(cfg, 64)
    shapes = layered.lezepel_shapes(cfg)
    mats = np.prod(shapes["head"])
    for i in cfg.runs:  # a looped layer's weights are read in every pass
        for n, s in shapes.items():
            if n.startswith("l%d." % i) and len(s) == 2:
                mats += np.prod(s) / (4 if ".mlp.e" in n else 1)  # two experts of eight are read
    assert by == 2 * mats + 8 * 4 * 64 * (128 + 64) and fl > 2 * 64 * (mats - np.prod(shapes["head"]))
