"""Layered models: decoders whose layers are described one by one (l2h_layered_create in include/l2h.h).

`LayerSpec` and `LayeredConfig` say what a model is made of; `LayeredDevice` is its resident copy, with the step
functions of `DeviceModel`.  A design is a reader that turns its config.json and tensor names into these
(`vudelix_config`, `vudelix_weights`), registered in registry.py."""
import ctypes as C
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

import numpy as np

from . import _lib
from .inference import DeviceModel

ATTENTION, CHANNEL_DELTA = 0, 1
FF_NONE, FF_DENSE, FF_EXPERTS = 0, 1, 2
GELU_ERF, RELU2, GELU_TANH = 0, 1, 2


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
    # channel delta
    taps: int = 1
    decay_rank: int = 1
    gate_rank: int = 1
    # feed-forward
    ff: int = FF_NONE
    ff_dim: int = 0
    ff_act: int = GELU_ERF
    n_experts: int = 0
    top: int = 0


@dataclass
class LayeredConfig:
    width: int
    vocab_size: int
    layers: List[LayerSpec]
    norm_eps: float
    residual_mult: float = 1.0
    side_dim: int = 0
    seq_len: int = 4096         # positions a sequence may reach (sizes the key/value cache)
    precision: str = "bfloat16"  # prompt pass: "bfloat16" or "float32"
    architecture: str = ""

    @property
    def n_layers(self):
        return len(self.layers)

    @property
    def dim(self):
        return self.width

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
                 "decay_rank", "gate_rank", "ff", "ff_dim", "ff_act", "n_experts", "top")] + \
               [("scale", C.c_float)] + \
               [(n, C.c_double) for n in ("rot_base", "rot_factor", "rot_low", "rot_high", "rot_original")]


class _Config(C.Structure):
    _fields_ = [(n, C.c_int32) for n in ("width", "vocab_size", "n_layers", "seq_len", "side_dim", "precision")] + \
               [("norm_eps", C.c_float), ("residual_mult", C.c_float)]


PRECISIONS = {"bfloat16": 0, "float32": 1}


class LayeredDevice(DeviceModel):
    """l2h_model of a layered model: the weights in HBM plus the state of one sequence (key/value rows of attention
    layers, recurrent state and convolution inputs of delta-rule layers).  The inherited step functions (forward,
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
            for name in ("mixer", "n_heads", "n_kv_heads", "dim", "vdim", "window", "rot_dims", "taps", "decay_rank", "gate_rank",
                         "ff", "ff_dim", "ff_act", "n_experts", "top"):
                setattr(d, name, int(getattr(s, name)))
            d.qk_norm, d.head_gate, d.scale, d.rot_base = int(s.qk_norm), int(s.head_gate), float(s.scale), float(s.rot_base)
            if s.rot_scaling:
                d.rot_factor, d.rot_low, d.rot_high, d.rot_original = (float(s.rot_scaling[k]) for k in ("factor", "low", "high", "original"))
        cfg = _Config(c.width, c.vocab_size, c.n_layers, c.seq_len, c.side_dim, PRECISIONS[c.precision], float(c.norm_eps),
                      float(c.residual_mult))
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
        """[n][width] after `layer` for the n positions of the last prompt pass (at most 2048)."""
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
