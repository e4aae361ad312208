"""Which loader a model on disk takes: a .gguf file (architectures of gguf.py), or a folder with config.json, whose
"architecture" names an entry of ARCHITECTURES, and model.safetensors."""
import json
import os

from . import layered
from .gguf import load_gguf_model
from .inference import LanguageModel
from .safetensors import read_safetensors
from .tokenizer import IdTokenizer


def _array(tensors):
    def array(name):
        if name not in tensors:
            raise layered.ConfigError("model.safetensors has no tensor %r" % name)
        return tensors[name][1]
    return array


def _vudelix(raw, tensors, seq_len, precision):
    array = _array(tensors)
    config = layered.vudelix_config(raw, lambda name: array(name).shape, seq_len, precision)
    return config, layered.vudelix_weights(config, array)


def _lezepel(raw, tensors, seq_len, precision):
    config = layered.lezepel_config(raw, seq_len, precision)
    return config, layered.lezepel_weights(config, _array(tensors))


# architecture -> (config.json, tensors, seq_len, precision) -> (config, weights)
ARCHITECTURES = {"Vudelix": _vudelix, "Lezepel": _lezepel}


def load_model(path, seq_len=4096, precision="bfloat16"):
    """LanguageModel from a GGUF file or a model folder.  seq_len: positions a sequence may reach (folders; a GGUF file
    names its own); precision: of a layered model's prompt pass."""
    if not os.path.isdir(path):
        return load_gguf_model(path)
    with open(os.path.join(path, "config.json")) as f:
        raw = json.load(f)
    arch = raw.get("architecture")
    if arch not in ARCHITECTURES:
        raise ValueError("config.json: architecture %r is not one of %s" % (arch, sorted(ARCHITECTURES)))
    tensors = read_safetensors(os.path.join(path, "model.safetensors"))
    config, weights = ARCHITECTURES[arch](raw, tensors, seq_len, precision)
    return LanguageModel(config, IdTokenizer(config.vocab_size), weights)
