"""Model registry: which configuration, tensors and engine a model file or folder needs.

  GGUF file                                -> `engine.DecodeEngine` (its header names the architecture)
  folder with config.json + model.safetensors -> by the configuration's "architecture": `ARCHITECTURES`

A new design that is a stack of mixers registers a configuration reader here and, if it brings a new kind of layer, a
class in `mixers.MIXERS`.
"""
import json
import os
from dataclasses import dataclass, field

from .mixers import MIXERS


@dataclass
class MixerLayer:
    mixer: object
    ff: int = 0                  # width of the gated feed-forward; 0: none


@dataclass
class MixerConfig:
    """A stack of mixer layers over one residual stream, grouped RMS norms, embedding and head untied."""
    arch: str = ""
    n_vocab: int = 0
    n_embd: int = 0
    norm_groups: int = 1
    norm_eps: float = 1e-6
    layers: list = field(default_factory=list)
    emb_scale: float = 1.0
    final_softcap: float = 0.0

    @property
    def n_layer(self):
        return len(self.layers)

    def tensors(self):
        """name -> shape (None: any size) of everything the model file must hold."""
        E = self.n_embd
        t = {"embed": (self.n_vocab, E), "head": (self.n_vocab, E), "final.norm": (E,)}
        for i, L in enumerate(self.layers):
            t[f"l{i}.norm1"] = (E,)
            t.update({f"l{i}.mix.{k}": s for k, s in L.mixer.tensors(E).items()})
            if L.ff:
                t[f"l{i}.norm2"] = (E,)
                t.update({f"l{i}.mlp.gate": (L.ff, E), f"l{i}.mlp.up": (L.ff, E), f"l{i}.mlp.down": (E, L.ff)})
        return t


def vomotar_config(d):
    """config.json of the Vomotar design (parsed) -> MixerConfig."""
    layers = []
    for i, L in enumerate(d["layers"]):
        if L["type"] not in MIXERS:
            raise ValueError(f"layer {i}: mixer '{L['type']}' is not known (known: {', '.join(sorted(MIXERS))})")
        mlp = L.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: feed-forward '{mlp['kind']}' is not known")
        layers.append(MixerLayer(MIXERS[L["type"]].from_config(L["mixer"]), int(mlp["ff"]) if mlp is not None else 0))
    c = MixerConfig(arch=d["architecture"], n_vocab=int(d["vocab"]), n_embd=int(d["width"]),
                    norm_groups=int(d["norm"]["groups"]), norm_eps=float(d["norm"]["eps"]), layers=layers)
    if c.n_embd % c.norm_groups:
        raise ValueError(f"width {c.n_embd} does not split into {c.norm_groups} norm groups")
    return c


ARCHITECTURES = {"Vomotar": vomotar_config}


def load_config(folder):
    with open(os.path.join(folder, "config.json")) as f:
        d = json.load(f)
    arch = d.get("architecture")
    if arch not in ARCHITECTURES:
        raise ValueError(f"{folder}: architecture '{arch}' is not known (known: {', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[arch](d)


def load_engine(gpu, path, **kw):
    """The engine for a GGUF file or a model folder; `kw` goes to its constructor."""
    if os.path.isdir(path):
        from .mixer_engine import MixerEngine
        from .safetensors_file import SafetensorsFile
        return MixerEngine(gpu, load_config(path), SafetensorsFile(os.path.join(path, "model.safetensors")), **kw)
    from . import gguf
    from .engine import DecodeEngine
    cfg, tensors = gguf.load_model(path)
    return DecodeEngine(gpu, cfg, tensors, **kw)
