"""Layered models without a GPU: readers, containers, the numpy restatement itself (that every planted mistake would
show), and the agreement of the ctypes structures with the C header."""
import json
import os
import subprocess

import numpy as np
import pytest

import layered_cases as lc
from oracle import layered_np as ref

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_every_planted_mistake_shows():
    c, t = lc.CASES["mixed"], lc.tensors("mixed")
    tok = lc.tokens(40, c["vocab"])
    good = ref.Sequence(c, t).run(tok)
    for twist in ref.TWISTS:
        err = lc.error(ref.Sequence(c, t, twist).run(tok), good)
        assert err > 1e-2, "%s changes the logits by %g only" % (twist, err)


def test_marked_key_shows_at_the_edge_of_the_window():
    size = 9
    c, t = lc.needle(size)
    tok = np.full(30, 7, np.int32)
    tok[:] = lc.tokens(30, c["vocab"])
    tok[tok == 3] = 4
    tok[5] = 3
    good = ref.Sequence(c, t).run(tok)
    inside, outside = 5 + size - 1, 5 + size
    more, less = ref.Sequence(c, t, "window+1").run(tok), ref.Sequence(c, t, "window-1").run(tok)
    assert lc.error(more[outside], good[outside]) > 0.3 and lc.error(less[inside], good[inside]) > 0.3


def test_delta_rule_by_hand():
    """one head, two tokens, from the closed form S2 = (g2 S1)(I - b2 k2 k2^T) + b2 k2 v2^T"""
    rng = np.random.default_rng(2)
    k, q, v = (rng.standard_normal((2, n)) for n in (5, 5, 3))
    g, b = rng.uniform(0.2, 1.0, (2, 5)), rng.uniform(0.1, 1.0, 2)
    S, o0 = ref.delta_step(np.zeros((5, 3)), q[0], k[0], v[0], g[0], b[0])
    assert np.allclose(S, b[0] * np.outer(k[0], v[0])) and np.allclose(o0, S.T @ q[0])
    S2, o1 = ref.delta_step(S, q[1], k[1], v[1], g[1], b[1])
    D = g[1][:, None] * S
    want = (np.eye(5) - b[1] * np.outer(k[1], k[1])) @ D + b[1] * np.outer(k[1], v[1])
    assert np.allclose(S2, want) and np.allclose(o1, want.T @ q[1])


def test_rotation_frequencies_in_three_bands():
    rot = {"dims": 64, "base": 1000.0, "scaling": lc.SCALING}
    plain, scaled = ref.rot_frequencies(rot, False), ref.rot_frequencies(rot)
    wl, sc = 2 * np.pi / plain, lc.SCALING
    short, long = wl < sc["original"] / sc["high"], wl > sc["original"] / sc["low"]
    assert short.any() and long.any() and (~short & ~long).any()
    assert np.array_equal(scaled[short], plain[short]) and np.allclose(scaled[long] * sc["factor"], plain[long])
    mid = ~short & ~long
    assert np.all(scaled[mid] <= plain[mid]) and np.all(scaled[mid] >= plain[mid] / sc["factor"])


def test_safetensors_round_trip_and_damage(pkg, tmp_path):
    from llama2_jl_amd import safetensors as st
    a = {"m": np.arange(6, dtype=np.uint16).reshape(2, 3), "v": np.linspace(0, 1, 5, dtype=np.float32), "t": np.array([3, -1], np.int32)}
    p = str(tmp_path / "x.safetensors")
    st.write_safetensors(p, a)
    back = st.read_safetensors(p)
    assert {k: v[0] for k, v in back.items()} == {"m": "BF16", "v": "F32", "t": "I32"}
    for k in a:
        assert np.array_equal(back[k][1], a[k])
    raw = open(p, "rb").read()
    for bad in (raw[:4], raw[:-1], b"\xff" * 8 + raw[8:], raw.replace(b'"BF16"', b'"F8_9"')):
        open(p, "wb").write(bad)
        with pytest.raises(ValueError):
            st.read_safetensors(p)


def _folder(tmp_path, c, t):
    from llama2_jl_amd import safetensors as st
    d = tmp_path / "model"
    d.mkdir(exist_ok=True)
    clean = json.loads(json.dumps(c))
    for layer in clean["layers"]:
        layer["mixer"].pop("_ranks", None)
    (d / "config.json").write_text(json.dumps(clean))
    st.write_safetensors(str(d / "model.safetensors"), {k: lc.bits(v) for k, v in t.items()})
    return d


def test_model_folder_reader(pkg, tmp_path):
    c, t = lc.CASES["mixed"], lc.tensors("mixed")
    d = _folder(tmp_path, c, t)
    m = pkg.load_model(str(d), seq_len=33, precision="float32")
    assert m.config.architecture == "Vudelix" and m.config.n_layers == 5 and m.config.seq_len == 33 and m.config.side_dim == 9
    kinds = [(s.mixer, s.ff) for s in m.config.layers]
    assert kinds == [(1, 1), (0, 2), (1, 2), (0, 0), (1, 0)]
    assert (m.config.layers[0].decay_rank, m.config.layers[0].gate_rank) == (10, 70)
    assert len(m.weights.tensors) == len(t)  # every tensor has a place
    raw = json.loads((d / "config.json").read_text())
    for change in (lambda r: r.update(architecture="Other"), lambda r: r.pop("width"), lambda r: r["layers"][1].update(type="ring"),
                   lambda r: r["layers"][1]["mixer"].pop("mask"), lambda r: r["layers"][0]["mlp"].update(kind="odd"),
                   lambda r: r["layers"][0].update(mixer={"heads": 2}), lambda r: r["layers"].append(r["layers"][0])):
        r = json.loads(json.dumps(raw))
        change(r)
        (d / "config.json").write_text(json.dumps(r))
        with pytest.raises(ValueError):
            pkg.load_model(str(d))


def test_id_tokenizer(pkg):
    tok = pkg.IdTokenizer(12)
    assert pkg.encode("3 11  0", tok) == [3, 11, 0] and tok.decode([3, 11]) == "3 11 "
    with pytest.raises(ValueError):
        pkg.encode("12", tok)


def test_ctypes_structures_match_the_header(pkg, tmp_path):
    from llama2_jl_amd import layered
    lines = []
    for struct, cls in (("l2h_layer", layered._Layer), ("l2h_layered_config", layered._Config)):
        lines.append('printf("%%zu\\n", sizeof(%s));' % struct)
        for name, _ in cls._fields_:
            lines.append('printf("%%zu\\n", offsetof(%s, %s));' % (struct, name))
    src = tmp_path / "s.c"
    src.write_text('#include <stddef.h>\n#include <stdio.h>\n#include "l2h.h"\nint main(void) { %s return 0; }\n' % " ".join(lines))
    exe = str(tmp_path / "s")
    subprocess.run(["gcc", "-I", os.path.join(ROOT, "include"), str(src), "-o", exe], check=True)
    got = [int(x) for x in subprocess.run([exe], capture_output=True, text=True, check=True).stdout.split()]
    import ctypes
    want = []
    for cls in (layered._Layer, layered._Config):
        want.append(ctypes.sizeof(cls))
        want += [getattr(cls, name).offset for name, _ in cls._fields_]
    assert got == want


def test_shapes_and_work_of_the_bench_models(pkg):
    from llama2_jl_amd import bench_layered, layered
    for c in lc.CASES.values():
        t = ref.tensor_shapes(c)
        assert layered.vudelix_shapes(layered.vudelix_config(c, lambda n: t[n])) == t
    cfg, _ = bench_layered.config("vudelix-tiny")
    by, fl = bench_layered.work(cfg, 64)
    shapes = layered.vudelix_shapes(cfg)
    experts = [n for n in shapes if ".mlp.e" in n]
    mats = sum(np.prod(s) for n, s in shapes.items() if len(s) == 2 and n not in experts + ["embed", "side.embed"] and "conv" not in n)
    mats += sum(np.prod(shapes[n]) for n in experts) * 2 // 8  # two experts of eight are read
    state = 6 * 2 * 4 * 4 * 128 * 128 + 2 * 4 * 64 * 2 * 256  # read and written; keys and values of 64 positions
    assert by == 2 * mats + state and fl > 2 * 64 * (mats - 512 * 32000)
