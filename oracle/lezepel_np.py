"""Plain numpy restatement of the layered design Lezepel: one function per mechanism, float64, token by token, no shared
code with the product path.  Test infrastructure only.

A model is (config, tensors) as in layered_np.py.  With x the residual stream and n(.) the rmsnorm, a layer is
    h = n1(x);  x <- x + mixer(h) + ff(h)
and the mixer is attention over a cached latent: keys and values of all heads are linear in one small vector per position,
beside one rotated key part that the heads share.  A stretch of layers runs several times over.

`twist` plants one mistake by name, so that a test can show that it would notice it (see TWISTS)."""
import math

import numpy as np

from .layered_np import bf16, rms, sigmoid, silu, softmax

TWISTS = {
    "no_embed_scale": "embedding not scaled",
    "no_embed_again": "a repeated pass does not add the embedding",
    "embed_every_pass": "the first pass adds the embedding, too",
    "no_step": "the pass vectors left out",
    "step_every_layer": "the pass vector added before every layer of a pass",
    "shared_cache": "the passes of a repeated layer share one cache",
    "sequential": "the feed-forward reads the stream after the mixer's update",
    "no_gate": "output gate left out",
    "gate_per_head": "one gate per head instead of one per element",
    "no_q_norm": "query latent not normed",
    "no_kv_norm": "key/value latent not normed",
    "norm_rotated_key": "the shared rotated key part normed with the latent's statistics",
    "no_rotation": "rotation left out",
    "interleaved": "interleaved instead of half-split rotation pairs",
    "rotated_first": "query heads read as [rotated, unrotated]",
    "loses_first": "the first key of the sequence is not seen",
    "no_router_bias": "router bias left out",
    "softmax_all": "expert weights from the softmax over all logits",
    "weight_on_input": "expert weight on the expert's input",
    "dense_silu": "dense activation silu",
    "expert_relu": "expert activation relu",
}


def rot_frequencies(dims, base):
    return base ** (-2.0 * np.arange(dims // 2) / dims)


def rotate_half(x, pos, freqs, interleaved=False):
    """elements i and i + n (n = len(freqs)) of the last axis turned by pos * freqs[i]; the rest passes"""
    y, n = np.array(x, np.float64), len(freqs)
    ia, ib = (2 * np.arange(n), 2 * np.arange(n) + 1) if interleaved else (np.arange(n), np.arange(n) + n)
    c, s = np.cos(pos * freqs), np.sin(pos * freqs)
    y[..., ia] = x[..., ia] * c - x[..., ib] * s
    y[..., ib] = x[..., ib] * c + x[..., ia] * s
    return y


def latent_scores(qn, qr, kn, kr, scale):
    """one head: unrotated query and keys [n][dim], rotated query and the shared rotated keys [n][rot]"""
    return (kn @ qn + kr @ qr) * scale


def route(h, router, bias, top):
    """indices of the chosen experts, best first, and the softmax over their logits"""
    z = router @ h + bias
    idx = np.argsort(-z, kind="stable")[:top]
    return idx, softmax(z[idx]), z


def gated(h, gate, up, down, act):
    return down @ (act(gate @ h) * (up @ h))


def relu(z):
    return np.maximum(z, 0.0)


def layer_runs(config):
    """(layer, pass or None) in the order of computation; the pass is given where a pass begins or goes on"""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


class Sequence:
    def __init__(self, config, tensors, twist=None):
        self.c = config
        self.t = {k: (v if v.dtype == np.int32 else np.asarray(v, np.float64)) for k, v in tensors.items()}
        assert twist is None or twist in TWISTS
        self.twist = twist
        self.pos = 0
        self.runs = layer_runs(config)
        self.mem = [dict() for _ in self.runs]
        self.residuals = []  # of the last step: the stream after every layer run

    def latent_attention(self, i, m, h, mem):
        t, p, eps, tw = self.t, "l%d.mix." % i, self.c["norm"]["eps"], self.twist
        H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        f = rot_frequencies(m["rot"]["dims"], m["rot"]["base"])
        cq = t[p + "dq"] @ h
        if tw != "no_q_norm":
            cq = rms(cq, eps) * t[p + "dq.norm"]
        q = (t[p + "uq"] @ cq).reshape(H, D + R)
        qn, qr = (q[:, R:], q[:, :R]) if tw == "rotated_first" else (q[:, :D], q[:, D:])
        d = t[p + "dkv"] @ h
        c, kr = d[:C], d[C:]
        if tw == "norm_rotated_key":
            kr = kr / np.sqrt(np.mean(c * c) + eps)
        if tw != "no_kv_norm":
            c = rms(c, eps) * t[p + "dkv.norm"]
        if tw != "no_rotation":
            qr, kr = (rotate_half(a, self.pos, f, tw == "interleaved") for a in (qr, kr))
        keep = [mem.setdefault(n, []) for n in ("k", "v", "r")]
        new = ((t[p + "uk"] @ c).reshape(H, D), (t[p + "uv"] @ c).reshape(H, V), kr)
        for a, b in zip(keep, new):
            a.append(b)
        k, v, r = (np.array(a) for a in keep)
        if tw == "loses_first" and len(k) > 1:
            k, v, r = k[1:], v[1:], r[1:]
        o = np.array([softmax(latent_scores(qn[a], qr[a], k[:, a], r, m["scale"])) @ v[:, a] for a in range(H)])
        g = sigmoid(t[p + "g"] @ h).reshape(H, V)
        if tw == "gate_per_head":
            g = g[:, :1]
        if tw != "no_gate":
            o = o * g
        return t[p + "o"] @ o.reshape(-1)

    def feed_forward(self, i, m, h):
        t, p, tw = self.t, "l%d.mlp." % i, self.twist
        if m["kind"] == "dense":
            return gated(h, t[p + "gate"], t[p + "up"], t[p + "down"], silu if tw == "dense_silu" else relu)
        assert m["kind"] == "moe"
        b = t[p + "router.b"] * (0.0 if tw == "no_router_bias" else 1.0)
        idx, w, z = route(h, t[p + "router"], b, m["router"]["top"])
        if tw == "softmax_all":
            w = softmax(z)[idx]
        y, act = 0.0, relu if tw == "expert_relu" else silu
        for e, we in zip(idx, w):
            mats = [t[p + "e%d.%s" % (e, n)] for n in ("gate", "up", "down")]
            y = y + (gated(we * h, *mats, act) if tw == "weight_on_input" else we * gated(h, *mats, act))
        return y

    def step(self, token):
        c, t, eps, tw = self.c, self.t, self.c["norm"]["eps"], self.twist
        x0 = t["embed"][token] * (1.0 if tw == "no_embed_scale" else c["embedding"]["scale"])
        x, self.residuals = x0, []
        for r, (i, p) in enumerate(self.runs):
            layer = c["layers"][i]
            if p is not None and i == c["loop"]["start"]:
                if (p > 0 and tw != "no_embed_again") or tw == "embed_every_pass":
                    x = x + x0
            if p is not None and tw != "no_step" and (i == c["loop"]["start"] or tw == "step_every_layer"):
                x = x + t["loop.step"][p]
            mem = self.mem[[j for j, _ in self.runs].index(i) if tw == "shared_cache" else r]
            h = rms(x, eps) * t["l%d.norm1" % i]
            y = self.latent_attention(i, layer["mixer"], h, mem)
            if layer.get("mlp"):
                hf = rms(x + y, eps) * t["l%d.norm1" % i] if tw == "sequential" else h
                y = y + self.feed_forward(i, layer["mlp"], hf)
            x = x + y
            self.residuals.append(x)
        self.pos += 1
        return t["head"] @ (rms(x, eps) * t["final.norm"])

    def run(self, tokens):
        return np.array([self.step(int(a)) for a in tokens])


def greedy(config, tensors, prompt, n_new, twist=None):
    s = Sequence(config, tensors, twist)
    logits = s.run(prompt)[-1]
    out = []
    for _ in range(n_new):
        out.append(int(np.argmax(logits)))
        logits = s.step(out[-1])
    return out


# ---- random models for tests -----------------------------------------------------------------------
def tensor_shapes(c):
    W, s = c["width"], {}
    s["embed"] = s["head"] = (c["vocab"], W)
    s["final.norm"] = (W,)
    if c.get("loop"):
        s["loop.step"] = (c["loop"]["times"], W)
    for i, layer in enumerate(c["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        H, D, R, V, C, Q = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
        s[p + "norm1"] = (W,)
        s.update({p + "mix.dq": (Q, W), p + "mix.dq.norm": (Q,), p + "mix.uq": (H * (D + R), Q), p + "mix.dkv": (C + R, W),
                  p + "mix.dkv.norm": (C,), p + "mix.uk": (H * D, C), p + "mix.uv": (H * V, C), p + "mix.g": (H * V, W),
                  p + "mix.o": (W, H * V)})
        f = layer.get("mlp")
        if not f:
            continue
        if f["kind"] == "moe":
            n = f["router"]["experts"]
            s[p + "mlp.router"], s[p + "mlp.router.b"] = (n, W), (n,)
        for e in [""] if f["kind"] == "dense" else ["e%d." % e for e in range(f["router"]["experts"])]:
            ff = f["ff"] if f["kind"] == "dense" else f["expert"]["ff"]
            s[p + "mlp.%sgate" % e] = s[p + "mlp.%sup" % e] = (ff, W)
            s[p + "mlp.%sdown" % e] = (W, ff)
    return s


def random_tensors(c, seed):
    """bf16-representable random tensors with every mechanism switched on at a visible strength"""
    rng, out = np.random.default_rng(seed), {}
    for name, shape in tensor_shapes(c).items():
        last = name.split(".")[-1]
        if last in ("norm", "norm1"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif last == "embed":
            a = rng.standard_normal(shape) / c["embedding"]["scale"]
        elif last in ("b", "step"):
            a = 0.8 * rng.standard_normal(shape)
        else:
            a = 1.4 * rng.standard_normal(shape) / math.sqrt(shape[-1])
        out[name] = bf16(a)
    return out
