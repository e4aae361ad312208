"""Plain numpy restatement of the layered design Vudelix: one function per mechanism, float64, token by token or
position by position, no shared code with the product path.  Test infrastructure only.

A model is (config, tensors): config is the dictionary of config.json, tensors maps names to numpy arrays of shape
[out, in].  `Sequence` holds what a sequence carries from token to token; `Sequence.step` runs one token.

`twist` plants one mistake by name, so that a test can show that it would notice it (see TWISTS)."""
import math

import numpy as np

TWISTS = {
    "window+1": "one key too many in the sliding window",
    "window-1": "one key too few in the sliding window",
    "no_gate": "attention output gate left out",
    "no_qk_norm": "query/key norm left out",
    "half_split": "half-split instead of interleaved rotation pairs",
    "no_rot_scaling": "frequency scaling left out",
    "no_conv_state": "short convolution sees zeros before the last token",
    "decay_first_channel": "one decay per head instead of one per key channel",
    "read_before_write": "delta rule reads the state before the token's own write",
    "weight_on_output": "router weight on the expert's output instead of its input",
    "no_side": "per-token layer input left out",
    "head_tile": "head h uses key/value head h mod G instead of floor(h / (H / G))",
}


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def silu(z):
    return z * sigmoid(z)


def gelu_erf(z):
    return 0.5 * z * (1.0 + np.vectorize(math.erf)(z / math.sqrt(2.0)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    """x divided by its root mean square over the last axis"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def rot_frequencies(rot, scaled=True):
    """one frequency per rotated pair"""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc and scaled:
            wl = 2.0 * math.pi / f
            if wl < sc["original"] / sc["high"]:
                pass
            elif wl > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            else:
                s = (sc["original"] / wl - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate(x, pos, freqs, half_split=False):
    """pairs (2i, 2i+1) of the first 2 len(freqs) elements of the last axis turned by pos * freqs"""
    y = np.array(x, dtype=np.float64)
    n = len(freqs)
    ia, ib = (np.arange(n), np.arange(n) + n) if half_split else (2 * np.arange(n), 2 * np.arange(n) + 1)
    c, s = np.cos(pos * freqs), np.sin(pos * freqs)
    a, b = x[..., ia], x[..., ib]
    y[..., ia] = a * c - b * s
    y[..., ib] = b * c + a * s
    return y


def softmax(z):
    e = np.exp(z - np.max(z))
    return e / np.sum(e)


def attend(q, keys, values, scale, group):
    """q [H][dim], keys [n][G][dim], values [n][G][vdim], already cut to what is visible -> [H][vdim]"""
    H, G = q.shape[0], keys.shape[1]
    out = np.empty((H, values.shape[2]))
    for h in range(H):
        g = group(h, H, G)
        w = softmax((keys[:, g] @ q[h]) * scale)
        out[h] = w @ values[:, g]
    return out


def short_conv(window, taps):
    """window [taps][channels], newest last; taps [channels][taps]"""
    return np.sum(window * taps.T, axis=0)


def delta_step(S, q, k, v, g, beta, read_first=False):
    """one token of the gated delta rule for one head: S [dim][vdim], q, k, g [dim], v [vdim]"""
    S = g[:, None] * S
    if read_first:
        o = S.T @ q
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, (o if read_first else S.T @ q)


def route(h, router, top):
    """indices of the chosen experts, best first, and their scores"""
    s = sigmoid(router @ h)
    idx = np.argsort(-s, kind="stable")[:top]
    return idx, s[idx]


class Sequence:
    def __init__(self, config, tensors, twist=None):
        self.c = config
        self.t = {k: (v if v.dtype == np.int32 else np.asarray(v, np.float64)) for k, v in tensors.items()}
        assert twist is None or twist in TWISTS
        self.twist = twist
        self.pos = 0
        self.mem = [dict() for _ in config["layers"]]
        self.residuals = []  # of the last step: the stream after every layer

    # ---- mechanisms bound to a layer -------------------------------------------------------------
    def _group(self, h, H, G):
        return h % G if self.twist == "head_tile" else h // (H // G)

    def attention(self, i, m, h):
        t, mem, p, eps = self.t, self.mem[i], "l%d.mix." % i, self.c["norm"]["eps"]
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q, k = (t[p + "q"] @ h).reshape(H, D), (t[p + "k"] @ h).reshape(G, D)
        v = (t[p + "v"] @ h).reshape(G, V)
        if m.get("rot"):
            f = rot_frequencies(m["rot"], self.twist != "no_rot_scaling")
            half = self.twist == "half_split"
            q, k = rotate(q, self.pos, f, half), rotate(k, self.pos, f, half)
        if self.twist != "no_qk_norm":
            q, k = rms(q, eps), rms(k, eps)
        mem.setdefault("k", []).append(k)
        mem.setdefault("v", []).append(v)
        size = m["mask"]["size"] + {"window+1": 1, "window-1": -1}.get(self.twist, 0)
        lo = max(0, self.pos - size + 1)
        o = attend(q, np.array(mem["k"][lo:]), np.array(mem["v"][lo:]), m["scale"], self._group)
        if self.twist != "no_gate":
            o = o * sigmoid(t[p + "g"] @ h)[:, None]
        return t[p + "o"] @ o.reshape(-1)

    def channel_delta(self, i, m, h):
        t, mem, p, eps = self.t, self.mem[i], "l%d.mix." % i, self.c["norm"]["eps"]
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        x = {}
        for n in "qkv":
            raw = t[p + n] @ h
            taps = t[p + n + ".conv"]
            past = mem.setdefault("conv_" + n, [np.zeros_like(raw) for _ in range(taps.shape[1] - 1)])
            if self.twist == "no_conv_state":
                past = [0.0 * a for a in past]
            window = past + [raw]
            mem["conv_" + n] = window[1:]
            x[n] = silu(short_conv(np.array(window), taps))
        q, k, v = unit(x["q"].reshape(G, D)) / math.sqrt(D), unit(x["k"].reshape(G, D)), x["v"].reshape(H, V)
        beta = sigmoid(t[p + "b"] @ h)
        rate = np.exp(t[p + "A_log"])[:, None] * softplus(t[p + "a2"] @ (t[p + "a1"] @ h) + t[p + "dt_bias"]).reshape(H, D)
        g = np.exp(-rate)
        if self.twist == "decay_first_channel":
            g = np.repeat(g[:, :1], D, axis=1)
        S = mem.setdefault("S", np.zeros((H, D, V)))
        o = np.empty((H, V))
        for hh in range(H):
            kv = self._group(hh, H, G)
            S[hh], o[hh] = delta_step(S[hh], q[kv], k[kv], v[hh], g[hh], beta[hh], self.twist == "read_before_write")
        o = rms(o, eps) * t[p + "norm"] * sigmoid(t[p + "g2"] @ (t[p + "g1"] @ h)).reshape(H, V)
        return t[p + "o"] @ o.reshape(-1)

    def feed_forward(self, i, m, h):
        t, p = self.t, "l%d.mlp." % i
        if m["kind"] == "dense":
            return t[p + "down"] @ gelu_erf(t[p + "up"] @ h)
        assert m["kind"] == "moe"
        idx, w = route(h, t[p + "router"], m["router"]["top"])
        y = 0.0
        for e, we in zip(idx, w):
            up, down = t[p + "e%d.up" % e], t[p + "e%d.down" % e]
            if self.twist == "weight_on_output":
                y = y + we * (down @ np.maximum(up @ h, 0.0) ** 2)
            else:
                y = y + down @ np.maximum(up @ (we * h), 0.0) ** 2
        return y

    def side_input(self, i, token, x):
        t, d, p = self.t, self.c["token_side"]["dim"], "l%d.side." % i
        e = t["side.embed"][token, i * d:(i + 1) * d]
        y = t[p + "proj"] @ (gelu_tanh(t[p + "gate"] @ x) * e)
        return rms(y, self.c["norm"]["eps"]) * t[p + "norm"]

    # ---- one token -------------------------------------------------------------------------------
    def step(self, token):
        c, t, eps, m = self.c, self.t, self.c["norm"]["eps"], self.c["residual_mult"]
        x = t["embed"][token]
        self.residuals = []
        for i, layer in enumerate(c["layers"]):
            mixer = {"attention": self.attention, "channel_delta": self.channel_delta}[layer["type"]]
            x = x + m * mixer(i, layer["mixer"], rms(x, eps) * t["l%d.norm1" % i])
            if layer.get("mlp"):
                x = x + m * self.feed_forward(i, layer["mlp"], rms(x, eps) * t["l%d.norm2" % i])
            if c.get("token_side") and self.twist != "no_side":
                x = x + m * self.side_input(i, token, x)
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
def bf16(a):
    """values rounded to bfloat16 (nearest even), kept as float32"""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000
    return u.astype(np.uint32).view(np.float32)


def tensor_shapes(c):
    """name -> shape for a config; ranks of the two-factor projections come from the mixer's "ranks" (tests only)"""
    W, s = c["width"], {}
    s["embed"] = s["head"] = (c["vocab"], W)
    s["final.norm"] = (W,)
    side = (c.get("token_side") or {}).get("dim", 0)
    if side:
        s["side.embed"] = (c["vocab"], side * len(c["layers"]))
    for i, layer in enumerate(c["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        s[p + "norm1"] = (W,)
        if layer["type"] == "attention":
            s.update({p + "mix.q": (H * D, W), p + "mix.k": (G * D, W), p + "mix.v": (G * V, W), p + "mix.g": (H, W),
                      p + "mix.o": (W, H * V)})
        else:
            ra, rg = m["_ranks"]
            s.update({p + "mix.q": (G * D, W), p + "mix.k": (G * D, W), p + "mix.v": (H * V, W), p + "mix.b": (H, W),
                      p + "mix.A_log": (H,), p + "mix.norm": (V,), p + "mix.a1": (ra, W), p + "mix.a2": (H * D, ra),
                      p + "mix.dt_bias": (H * D,), p + "mix.g1": (rg, W), p + "mix.g2": (H * V, rg), p + "mix.o": (W, H * V)})
            for n, ch in (("q", G * D), ("k", G * D), ("v", H * V)):
                s[p + "mix.%s.conv" % n] = (ch, m["conv"])
        f = layer.get("mlp")
        if f:
            s[p + "norm2"] = (W,)
            if f["kind"] == "dense":
                s[p + "mlp.up"], s[p + "mlp.down"] = (f["ff"], W), (W, f["ff"])
            else:
                s[p + "mlp.router"] = (f["router"]["experts"], W)
                for e in range(f["router"]["experts"]):
                    s[p + "mlp.e%d.up" % e], s[p + "mlp.e%d.down" % e] = (f["expert"]["ff"], W), (W, f["expert"]["ff"])
        if side:
            s.update({p + "side.gate": (side, W), p + "side.proj": (W, side), p + "side.norm": (W,)})
    return s


def random_tensors(c, seed):
    """bf16-representable random tensors with every mechanism switched on at a visible strength"""
    rng, out = np.random.default_rng(seed), {}
    for name, shape in tensor_shapes(c).items():
        last = name.split(".")[-1]
        if last in ("norm", "norm1", "norm2"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif last == "A_log":
            a = rng.uniform(-2.5, 0.5, shape)
        elif last == "dt_bias":
            a = rng.uniform(-5.0, 0.5, shape)
        elif last == "conv":
            a = 0.6 * rng.standard_normal(shape)
        elif last in ("embed",):
            a = rng.standard_normal(shape)
        elif last == "router":
            a = 3.0 * rng.standard_normal(shape) / math.sqrt(shape[-1])
        else:
            a = 1.4 * rng.standard_normal(shape) / math.sqrt(shape[-1])
        out[name] = bf16(a)
    return out
