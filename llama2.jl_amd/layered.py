"""Layered models: decoders whose layers are described one by one (l2h_layered_create in include/l2h.h).

`LayerSpec` and `LayeredConfig` say what a model is made of; `LayeredDevice` is its resident copy, with the step
functions of `DeviceModel`.  A design is a reader that turns its config.json and tensor names into these
(`vudelix_config`, `vudelix_weights`; `lezepel_config`, `lezepel_weights`), registered in registry.py."""
import ctypes as C
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

import numpy as np

from . import _lib
from .inference import DeviceModel

ATTENTION, CHANNEL_DELTA, LATENT = 0, 1, 2
FF_NONE, FF_DENSE, FF_EXPERTS = 0, 1, 2
GELU_ERF, RELU2, GELU_TANH, RELU, SILU = 0, 1, 2, 3, 4
ROUTE_SIGMOID_IN, ROUTE_SOFTMAX_OUT = 0, 1


@dataclass
class LayerSpec:
    mixer: int
    n_heads: int
    n_kv_heads: int
    dim: int
    vdim: int
    # attention
    window: int = 0
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: Optional[Dict[str, float]] = None  # factor, low, high, original
    qk_norm: bool = False
    head_gate: bool = False
    scale: float = 1.0
    rot_half: bool = False      # pairs i, i + rot_dims / 2 instead of 2i, 2i + 1
    # latent attention
    q_rank: int = 0
    kv_rank: int = 0
    rot_size: int = 0           # size of the rotated part of a key, beside `dim`
    out_gate: bool = False
    # channel delta
    taps: int = 1
    decay_rank: int = 1
    gate_rank: int = 1
    # feed-forward
    ff: int = FF_NONE
    ff_dim: int = 0
    ff_act: int = GELU_ERF
    ff_gated: bool = False
    n_experts: int = 0
    top: int = 0
    route: int = ROUTE_SIGMOID_IN
    router_bias: bool = False
    parallel: bool = False      # one norm, mixer and feed-forward side by side


@dataclass
class LayeredConfig:
    width: int
    vocab_size: int
    layers: List[LayerSpec]
    norm_eps: float
    residual_mult: float = 1.0
    embed_scale: float = 1.0
    side_dim: int = 0
    loop: Optional[Tuple[int, int, int]] = None  # start, stop, times
    seq_len: int = 4096         # positions a sequence may reach (sizes the key/value cache)
    precision: str = "bfloat16"  # prompt pass: "bfloat16" or "float32"
    architecture: str = ""

    @property
    def n_layers(self):
        return len(self.layers)

    @property
    def dim(self):
        return self.width

    @property
    def runs(self):
        """the layers in the order they are computed"""
        n = list(range(self.n_layers))
        if not self.loop:
            return n
        start, stop, times = self.loop
        return n[:start] + n[start:stop] * times + n[stop:]

    def __str__(self):
        rows = ["architecture", "width", "vocab_size", "n_layers", "side_dim", "seq_len", "precision"]
        return "LayeredConfig(\n" + "".join("  %-14s = %s,\n" % (r, getattr(self, r)) for r in rows) + ")"


@dataclass
class LayeredWeights:
    """(role, layer) -> array [out][in] (or a vector), experts under (role, layer, expert).  uint16 arrays are bf16 bit
    patterns, float32 arrays are accepted for vectors."""
    tensors: Dict[Any, np.ndarray] = field(default_factory=dict)


class _Layer(C.Structure):
    _fields_ = [(n, C.c_int32) for n in
                ("mixer", "n_heads", "n_kv_heads", "dim", "vdim", "window", "rot_dims", "qk_norm", "head_gate", "taps",
                 "decay_rank", "gate_rank", "q_rank", "kv_rank", "rot_size", "out_gate", "rot_half", "parallel", "ff", "ff_dim",
                 "ff_act", "ff_gated", "n_experts", "top", "route", "router_bias")] + \
               [("scale", C.c_float)] + \
               [(n, C.c_double) for n in ("rot_base", "rot_factor", "rot_low", "rot_high", "rot_original")]


class _Config(C.Structure):
    _fields_ = [(n, C.c_int32) for n in ("width", "vocab_size", "n_layers", "seq_len", "side_dim", "precision", "loop_start",
                                          "loop_stop", "loop_times")] + \
               [(n, C.c_float) for n in ("norm_eps", "residual_mult", "embed_scale")]


PRECISIONS = {"bfloat16": 0, "float32": 1}


class LayeredDevice(DeviceModel):
    """l2h_model of a layered model: the weights in HBM plus the state of one sequence (key/value rows of attention
    layers, latents and rotated key parts of latent attention layers, recurrent state and convolution inputs of delta-rule
    layers; a looped layer has them for each pass).  The inherited step functions (forward,
    generate_greedy, prefill, sample_token, reset) are the same C calls as for a Llama model."""

    def __init__(self, config, weights, ctx=None, path=0, kv_fp16=False):
        if kv_fp16:
            raise ValueError("a layered model keeps an fp32 cache")
        if config.precision not in PRECISIONS:
            raise ValueError("precision %r: one of %s" % (config.precision, sorted(PRECISIONS)))
        super().__init__(config, weights, ctx, path, kv_fp16)

    def _create(self):
        c = self.config
        layers = (_Layer * c.n_layers)()
        for d, s in zip(layers, c.layers):
            for name, kind in _Layer._fields_:
                if kind is C.c_int32:
                    setattr(d, name, int(getattr(s, name)))
            d.scale, d.rot_base = float(s.scale), float(s.rot_base)
            if s.rot_scaling:
                d.rot_factor, d.rot_low, d.rot_high, d.rot_original = (float(s.rot_scaling[k]) for k in ("factor", "low", "high", "original"))
        cfg = _Config(c.width, c.vocab_size, c.n_layers, c.seq_len, c.side_dim, PRECISIONS[c.precision], *(c.loop or (0, 0, 0)),
                      float(c.norm_eps), float(c.residual_mult), float(c.embed_scale))
        self.ctx.check(_lib.lib().l2h_layered_create(self.ctx.handle, C.byref(cfg), layers, C.byref(self.handle)))

    def _upload(self, weights):
        for key, a in weights.tensors.items():
            a = np.ascontiguousarray(a)
            typ = {np.dtype("<u2"): _lib.TYPE_BF16, np.dtype("<f4"): _lib.TYPE_F32}[a.dtype]
            ne0, ne1 = (a.size, 1) if a.ndim == 1 else (a.shape[1], a.shape[0])
            if len(key) == 3:
                self.ctx.check(_lib.lib().l2h_layered_set_expert(self.handle, key[0], key[1], key[2], typ, _lib.ptr(a), ne0, ne1))
            else:
                self.ctx.check(_lib.lib().l2h_model_set_tensor(self.handle, key[0], key[1], typ, _lib.ptr(a), ne0, ne1))

    def keep_residuals(self, on=True):
        """Prompt passes keep the residual stream after every layer (l2h_layered_keep)."""
        self.ctx.check(_lib.lib().l2h_layered_keep(self.handle, 1 if on else 0))

    def residuals(self, layer, n):
        """[n][width] after layer run `layer` (config.runs) for the n positions of the last prompt pass (at most 2048)."""
        out = np.empty((n, self.config.width), np.float32)
        self.ctx.check(_lib.lib().l2h_layered_kept(self.handle, layer, _lib.ptr(out), out.size))
        return out

    def kv_read(self, layer, pos0, n):
        raise ValueError("the rows of a layered model's cache are not exchanged with the host")

    def kv_write(self, layer, pos0, k, v):
        raise ValueError("the rows of a layered model's cache are not exchanged with the host")

    def state(self, name):
        n = {"x": self.config.width, "logits": self.config.vocab_size}[name]
        out = np.empty(n, np.float32)
        self.ctx.check(_lib.lib().l2h_state_read(self.handle, self._STATE[name], _lib.ptr(out), n))
        return out


# ---- Vudelix ---------------------------------------------------------------------------------------------------------
class ConfigError(ValueError):
    pass


def _take(d, key, where):
    if key not in d or d[key] is None:
        raise ConfigError("config.json: %s has no %r" % (where, key))
    return d[key]


def vudelix_config(c, shape, seq_len=4096, precision="bfloat16"):
    """config.json of a Vudelix model -> LayeredConfig.  shape(name) gives a tensor's shape: the ranks of the two-factor
    projections are only there."""
    layers = []
    for i, entry in enumerate(_take(c, "layers", "the model")):
        where, m = "layer %d" % i, _take(entry, "mixer", "layer %d" % i)
        s = LayerSpec(mixer=-1, n_heads=_take(m, "heads", where), n_kv_heads=_take(m, "kv_heads", where), dim=_take(m, "dim", where),
                      vdim=_take(m, "vdim", where))
        kind = _take(entry, "type", where)
        if kind == "attention":
            s.mixer, s.qk_norm, s.head_gate = ATTENTION, True, True
            s.scale = _take(m, "scale", where)
            s.window = _take(_take(m, "mask", where), "size", where)
            rot = m.get("rot")
            if rot:
                s.rot_dims, s.rot_base = _take(rot, "dims", where), _take(rot, "base", where)
                if rot.get("scaling"):
                    s.rot_scaling = {k: _take(rot["scaling"], k, where) for k in ("factor", "low", "high", "original")}
        elif kind == "channel_delta":
            s.mixer, s.taps = CHANNEL_DELTA, _take(m, "conv", where)
            s.decay_rank, s.gate_rank = shape("l%d.mix.a1" % i)[0], shape("l%d.mix.g1" % i)[0]
        else:
            raise ConfigError("config.json: layer %d has type %r" % (i, kind))
        f = entry.get("mlp")
        if f:
            kind = _take(f, "kind", where)
            if kind == "dense":
                s.ff, s.ff_dim, s.ff_act = FF_DENSE, _take(f, "ff", where), GELU_ERF
            elif kind == "moe":
                s.ff, s.ff_act = FF_EXPERTS, RELU2
                s.ff_dim = _take(_take(f, "expert", where), "ff", where)
                s.n_experts, s.top = _take(_take(f, "router", where), "experts", where), _take(f["router"], "top", where)
            else:
                raise ConfigError("config.json: layer %d has a feed-forward of kind %r" % (i, kind))
        layers.append(s)
    side = c.get("token_side")
    return LayeredConfig(width=_take(c, "width", "the model"), vocab_size=_take(c, "vocab", "the model"), layers=layers,
                         norm_eps=_take(_take(c, "norm", "the model"), "eps", "norm"),
                         residual_mult=_take(c, "residual_mult", "the model"),
                         side_dim=_take(side, "dim", "token_side") if side else 0, seq_len=seq_len, precision=precision,
                         architecture="Vudelix")


_L = _lib
_ATTENTION_NAMES = {"q": _L.WQ, "k": _L.WK, "v": _L.WV, "g": _L.HEAD_GATE, "o": _L.WO}
_DELTA_NAMES = {"q": _L.WQ, "k": _L.WK, "v": _L.WV, "o": _L.WO, "b": _L.BETA, "A_log": _L.DECAY_RATE, "dt_bias": _L.DECAY_BIAS,
                "a1": _L.DECAY_IN, "a2": _L.DECAY_OUT, "g1": _L.GATE_IN, "g2": _L.GATE_OUT, "norm": _L.MIX_NORM,
                "q.conv": _L.CONV_Q, "k.conv": _L.CONV_K, "v.conv": _L.CONV_V}
_SIDE_NAMES = {"gate": _L.SIDE_GATE, "proj": _L.SIDE_PROJ, "norm": _L.SIDE_NORM}


def vudelix_names(config):
    """tensor name -> key of LayeredWeights.tensors, every tensor such a model has"""
    out = {"embed": (_L.TOK_EMB, 0), "final.norm": (_L.RMS_FINAL, 0), "head": (_L.OUTPUT, 0)}
    if config.side_dim:
        out["side.embed"] = (_L.SIDE_EMB, 0)
    for i, s in enumerate(config.layers):
        p = "l%d." % i
        out[p + "norm1"] = (_L.RMS_ATT, i)
        for name, role in (_ATTENTION_NAMES if s.mixer == ATTENTION else _DELTA_NAMES).items():
            out[p + "mix." + name] = (role, i)
        if s.ff != FF_NONE:
            out[p + "norm2"] = (_L.RMS_FFN, i)
        if s.ff == FF_DENSE:
            out[p + "mlp.up"], out[p + "mlp.down"] = (_L.W1, i), (_L.W2, i)
        if s.ff == FF_EXPERTS:
            out[p + "mlp.router"] = (_L.ROUTER, i)
            for e in range(s.n_experts):
                out[p + "mlp.e%d.up" % e], out[p + "mlp.e%d.down" % e] = (_L.EXPERT_UP, i, e), (_L.EXPERT_DOWN, i, e)
        if config.side_dim:
            for name, role in _SIDE_NAMES.items():
                out[p + "side." + name] = (role, i)
    return out


def vudelix_weights(config, tensor):
    """tensor(name) -> array; LayeredWeights with every tensor of the model"""
    return LayeredWeights({key: tensor(name) for name, key in vudelix_names(config).items()})


def vudelix_shapes(config):
    """tensor name -> shape"""
    W, out = config.width, {}
    for name in vudelix_names(config):
        parts = name.split(".")
        if name in ("embed", "head"):
            out[name] = (config.vocab_size, W)
        elif name == "side.embed":
            out[name] = (config.vocab_size, config.side_dim * config.n_layers)
        elif parts[-1] in ("norm1", "norm2") or name == "final.norm" or parts[1:] == ["side", "norm"]:
            out[name] = (W,)
        elif parts[1] == "side":
            out[name] = (config.side_dim, W) if parts[2] == "gate" else (W, config.side_dim)
        elif parts[1] == "mlp":
            s = config.layers[int(parts[0][1:])]
            out[name] = (s.n_experts, W) if parts[-1] == "router" else (s.ff_dim, W) if parts[-1] == "up" else (W, s.ff_dim)
        else:
            s = config.layers[int(parts[0][1:])]
            H, G, D, V = s.n_heads, s.n_kv_heads, s.dim, s.vdim
            qk = G if s.mixer == CHANNEL_DELTA else H
            vh = H if s.mixer == CHANNEL_DELTA else G
            n = ".".join(parts[2:])
            out[name] = {"q": (qk * D, W), "k": (G * D, W), "v": (vh * V, W), "g": (H, W), "o": (W, H * V), "b": (H, W),
                         "A_log": (H,), "dt_bias": (H * D,), "norm": (V,), "a1": (s.decay_rank, W), "a2": (H * D, s.decay_rank),
                         "g1": (s.gate_rank, W), "g2": (H * V, s.gate_rank), "q.conv": (qk * D, s.taps), "k.conv": (G * D, s.taps),
                         "v.conv": (vh * V, s.taps)}[n]
    return out


# ---- Lezepel ---------------------------------------------------------------------------------------------------------
def lezepel_config(c, seq_len=4096, precision="bfloat16"):
    """config.json of a Lezepel model -> LayeredConfig"""
    layers = []
    for i, entry in enumerate(_take(c, "layers", "the model")):
        where, m = "layer %d" % i, _take(entry, "mixer", "layer %d" % i)
        kind = _take(entry, "type", where)
        if kind != "latent_attention":
            raise ConfigError("config.json: layer %d has type %r" % (i, kind))
        heads, rot = _take(m, "heads", where), _take(m, "rot", where)
        s = LayerSpec(mixer=LATENT, n_heads=heads, n_kv_heads=heads, dim=_take(m, "dim", where), vdim=_take(m, "vdim", where),
                      q_rank=_take(m, "q_rank", where), kv_rank=_take(m, "kv_rank", where), rot_size=_take(m, "rot_dim", where),
                      scale=_take(m, "scale", where), rot_dims=_take(rot, "dims", where), rot_base=_take(rot, "base", where),
                      rot_half=True, out_gate=True, parallel=True, ff_gated=True)
        f = entry.get("mlp")
        if f:
            kind = _take(f, "kind", where)
            if kind == "dense":
                s.ff, s.ff_dim, s.ff_act = FF_DENSE, _take(f, "ff", where), RELU
            elif kind == "moe":
                s.ff, s.ff_act, s.ff_dim = FF_EXPERTS, SILU, _take(_take(f, "expert", where), "ff", where)
                router = _take(f, "router", where)
                s.n_experts, s.top = _take(router, "experts", where), _take(router, "top", where)
                s.route, s.router_bias = ROUTE_SOFTMAX_OUT, True
            else:
                raise ConfigError("config.json: layer %d has a feed-forward of kind %r" % (i, kind))
        layers.append(s)
    loop = c.get("loop")
    return LayeredConfig(width=_take(c, "width", "the model"), vocab_size=_take(c, "vocab", "the model"), layers=layers,
                         norm_eps=_take(_take(c, "norm", "the model"), "eps", "norm"),
                         embed_scale=_take(_take(c, "embedding", "the model"), "scale", "embedding"),
                         loop=tuple(_take(loop, k, "loop") for k in ("start", "stop", "times")) if loop else None,
                         seq_len=seq_len, precision=precision, architecture="Lezepel")


_LATENT_NAMES = {"dq": _L.Q_DOWN, "dq.norm": _L.Q_NORM, "uq": _L.Q_UP, "dkv": _L.KV_DOWN, "dkv.norm": _L.KV_NORM, "uk": _L.K_UP,
                 "uv": _L.V_UP, "g": _L.OUT_GATE, "o": _L.WO}


def lezepel_names(config):
    """tensor name -> key of LayeredWeights.tensors, every tensor such a model has"""
    out = {"embed": (_L.TOK_EMB, 0), "final.norm": (_L.RMS_FINAL, 0), "head": (_L.OUTPUT, 0)}
    if config.loop:
        out["loop.step"] = (_L.LOOP_STEP, 0)
    for i, s in enumerate(config.layers):
        p = "l%d." % i
        out[p + "norm1"] = (_L.RMS_ATT, i)
        for name, role in _LATENT_NAMES.items():
            out[p + "mix." + name] = (role, i)
        if s.ff == FF_DENSE:
            out[p + "mlp.gate"], out[p + "mlp.up"], out[p + "mlp.down"] = (_L.W1, i), (_L.W3, i), (_L.W2, i)
        if s.ff == FF_EXPERTS:
            out[p + "mlp.router"], out[p + "mlp.router.b"] = (_L.ROUTER, i), (_L.ROUTER_BIAS, i)
            for e in range(s.n_experts):
                for name, role in (("gate", _L.EXPERT_GATE), ("up", _L.EXPERT_UP), ("down", _L.EXPERT_DOWN)):
                    out[p + "mlp.e%d.%s" % (e, name)] = (role, i, e)
    return out


def lezepel_weights(config, tensor):
    """tensor(name) -> array; LayeredWeights with every tensor of the model"""
    return LayeredWeights({key: tensor(name) for name, key in lezepel_names(config).items()})


def lezepel_shapes(config):
    """tensor name -> shape"""
    W, out = config.width, {}
    for name in lezepel_names(config):
        parts = name.split(".")
        if name in ("embed", "head"):
            out[name] = (config.vocab_size, W)
        elif name == "loop.step":
            out[name] = (config.loop[2], W)
        elif parts[-1] == "norm1" or name == "final.norm":
            out[name] = (W,)
        else:
            s = config.layers[int(parts[0][1:])]
            H, D, R, V, n = s.n_heads, s.dim, s.rot_size, s.vdim, ".".join(parts[2:])
            if parts[1] == "mix":
                out[name] = {"dq": (s.q_rank, W), "dq.norm": (s.q_rank,), "uq": (H * (D + R), s.q_rank), "dkv": (s.kv_rank + R, W),
                             "dkv.norm": (s.kv_rank,), "uk": (H * D, s.kv_rank), "uv": (H * V, s.kv_rank), "g": (H * V, W),
                             "o": (W, H * V)}[n]
            elif n == "router.b":
                out[name] = (s.n_experts,)
            elif n == "router":
                out[name] = (s.n_experts, W)
            else:
                out[name] = (W, s.ff_dim) if parts[-1] == "down" else (s.ff_dim, W)
    return out


# architecture -> (shapes, weights): a model of a given configuration from its tensors by name
DESIGNS = {"Vudelix": (vudelix_shapes, vudelix_weights), "Lezepel": (lezepel_shapes, lezepel_weights)}
