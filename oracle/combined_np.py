"""Layers that combine the mechanisms of the layered designs freely, composed from the restatements of layered_np.py and
lezepel_np.py.  A layer is a dictionary: "mixer" names a method of one of the two Sequence classes, "parallel", "gated",
"act", "route", "bias" and "rot_half" switch the rest.  Test infrastructure only."""
import numpy as np

from . import layered_np as a
from . import lezepel_np as b

ACTS = {"gelu_erf": a.gelu_erf, "relu2": lambda z: np.maximum(z, 0.0) ** 2, "gelu_tanh": a.gelu_tanh, "relu": b.relu, "silu": a.silu}


class _Attention(a.Sequence):
    """window attention with either layout of rotated pairs"""

    def attention_as(self, i, m, h, half):
        self.twist = "half_split" if half else None
        try:
            return self.attention(i, m, h)
        finally:
            self.twist = None


class Sequence:
    """config: layers, width, norm eps, residual_mult, embed_scale, side (dim or 0), loop (start, stop, times) or None"""

    def __init__(self, c, tensors):
        self.c, self.pos = c, 0
        self.t = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        loop = c.get("loop")
        self.runs = b.layer_runs({"layers": c["layers"], "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None})
        inner = {"layers": c["layers"], "norm": c["norm"]}
        self.parts = []  # the mechanisms' own sequences, one for each layer run: each holds that run's memory
        for _ in self.runs:
            self.parts.append((_Attention(inner, tensors), b.Sequence(dict(inner, embedding={"scale": 1.0}), tensors), {}))

    def mixer(self, r, i, h):
        layer = self.c["layers"][i]
        one, two, mem = self.parts[r]
        one.pos = two.pos = self.pos
        if layer["type"] == "latent_attention":
            return two.latent_attention(i, layer["mixer"], h, mem)
        if layer["type"] == "channel_delta":
            return one.channel_delta(i, layer["mixer"], h)
        return one.attention_as(i, layer["mixer"], h, layer.get("rot_half"))

    def expert(self, p, layer, h):
        act = ACTS[layer["act"]]
        if layer["gated"]:
            return b.gated(h, self.t[p + "gate"], self.t[p + "up"], self.t[p + "down"], act)
        return self.t[p + "down"] @ act(self.t[p + "up"] @ h)

    def feed_forward(self, i, layer, h):
        p, f = "l%d.mlp." % i, layer["mlp"]
        if f["kind"] == "dense":
            return self.expert(p, layer, h)
        z = self.t[p + "router"] @ h + (self.t[p + "router.b"] if layer["bias"] else 0.0)
        idx = np.argsort(-z, kind="stable")[:f["router"]["top"]]
        if layer["route"] == "sigmoid_in":
            return sum(self.expert(p + "e%d." % e, layer, a.sigmoid(z[e]) * h) for e in idx)
        return sum(w * self.expert(p + "e%d." % e, layer, h) for e, w in zip(idx, a.softmax(z[idx])))

    def step(self, token):
        c, t, eps, m = self.c, self.t, self.c["norm"]["eps"], self.c["residual_mult"]
        x = x0 = c["embed_scale"] * t["embed"][token]
        for r, (i, p) in enumerate(self.runs):
            layer = c["layers"][i]
            if p is not None and i == c["loop"][0]:
                x = (x + x0 if p else x) + t["loop.step"][p]
            h = a.rms(x, eps) * t["l%d.norm1" % i]
            y = self.mixer(r, i, h)
            if layer.get("mlp"):
                if layer["parallel"]:
                    y = y + self.feed_forward(i, layer, h)
                else:
                    x = x + m * y
                    y = self.feed_forward(i, layer, a.rms(x, eps) * t["l%d.norm2" % i])
            x = x + m * y
            if c.get("side"):
                s = a.Sequence({"layers": c["layers"], "norm": c["norm"], "token_side": {"dim": c["side"]}}, t)
                x = x + m * s.side_input(i, token, x)
        self.pos += 1
        return t["head"] @ (a.rms(x, eps) * t["final.norm"])

    def run(self, tokens):
        return np.array([self.step(int(k)) for k in tokens])


def tensor_shapes(c):
    """name -> shape: the mixers' from the two designs, the rest from the switches"""
    W, s = c["width"], {"embed": (c["vocab"], c["width"]), "head": (c["vocab"], c["width"]), "final.norm": (c["width"],)}
    if c.get("loop"):
        s["loop.step"] = (c["loop"][2], W)
    if c.get("side"):
        s["side.embed"] = (c["vocab"], c["side"] * len(c["layers"]))
    for i, layer in enumerate(c["layers"]):
        p = "l%d." % i
        of = b if layer["type"] == "latent_attention" else a
        one = of.tensor_shapes({"layers": [dict(layer, mlp=None)], "width": W, "vocab": 1})
        s.update({p + k[3:]: v for k, v in one.items() if k.startswith("l0.")})
        f = layer.get("mlp")
        if f:
            if not layer["parallel"]:
                s[p + "norm2"] = (W,)
            if f["kind"] == "moe":
                n = f["router"]["experts"]
                s[p + "mlp.router"] = (n, W)
                if layer["bias"]:
                    s[p + "mlp.router.b"] = (n,)
            for e in [""] if f["kind"] == "dense" else ["e%d." % e for e in range(f["router"]["experts"])]:
                ff = f["ff"] if f["kind"] == "dense" else f["expert"]["ff"]
                for name in (["gate"] if layer["gated"] else []) + ["up"]:
                    s[p + "mlp." + e + name] = (ff, W)
                s[p + "mlp." + e + "down"] = (W, ff)
        if c.get("side"):
            s.update({p + "side.gate": (c["side"], W), p + "side.proj": (W, c["side"]), p + "side.norm": (W,)})
    return s
