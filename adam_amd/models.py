"""Model registry: which configuration, tensors and engine a model file or folder needs.

  GGUF file                                -> `engine.DecodeEngine` (its header names the architecture)
  folder with config.json + model.safetensors -> by the configuration's "architecture": `ARCHITECTURES`

A new design that is a stack of mixers registers a configuration reader here and, if it brings a new kind of layer, a
class in `mixers.MIXERS` or `feed_forward`.
"""
import json
import os
from dataclasses import dataclass, field

from .feed_forward import Dense, Experts
from .mixers import MIXERS


@dataclass
class MixerLayer:
    mixer: object
    ff: object = None            # feed-forward; None: the layer has none


@dataclass
class BigramTable:
    """Embedding rows per pair of neighbouring tokens: row (previous * mul_prev + current * mul_cur) mod buckets."""
    buckets: int
    mul_prev: int
    mul_cur: int

    def __post_init__(self):
        if not (1 <= self.buckets < 1 << 31 and 0 <= self.mul_prev < 1 << 32 and 0 <= self.mul_cur < 1 << 32):
            raise ValueError(f"bigram table: {self}")


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
    norm_add: float = 0.0        # norms multiply by norm_add + weight
    post_norm: bool = False      # a sublayer's output passes a norm of its own before it is added
    pairs: BigramTable = None
    loop: tuple = None           # (start, stop, times): layers start .. stop - 1 run `times` times in a row

    def __post_init__(self):
        if self.n_embd % self.norm_groups:
            raise ValueError(f"width {self.n_embd} does not split into {self.norm_groups} norm groups")
        if self.post_norm and self.norm_groups != 1:
            raise ValueError("norms behind a sublayer take the full width")
        if self.loop is not None and not (0 <= self.loop[0] <= self.loop[1] <= len(self.layers) and self.loop[2] >= 1):
            raise ValueError(f"loop {self.loop} over {len(self.layers)} layers")

    @property
    def n_layer(self):
        return len(self.layers)

    def runs(self):
        """The layers' indices in the order they run; a layer that runs again has a state of its own there."""
        n = range(len(self.layers))
        if self.loop is None:
            return list(n)
        start, stop, times = self.loop
        return [*n[:start], *list(n[start:stop]) * times, *n[stop:]]

    def norms(self, i):
        """Names of layer i's norms over the residual stream."""
        names = ["norm1"] + (["norm1b"] if self.post_norm else [])
        if self.layers[i].ff is not None:
            names += ["norm2"] + (["norm2b"] if self.post_norm else [])
        return [f"l{i}.{n}" for n in names]

    def tensors(self):
        """name -> shape (None: any size) of everything the model file must hold."""
        E = self.n_embd
        t = {"embed": (self.n_vocab, E), "head": (self.n_vocab, E), "final.norm": (E,)}
        if self.pairs is not None:
            t["bigram"] = (self.pairs.buckets + 1, E)
        for i, L in enumerate(self.layers):
            t.update({n: (E,) for n in self.norms(i)})
            t.update({f"l{i}.mix.{k}": s for k, s in L.mixer.tensors(E).items()})
            if L.ff is not None:
                t.update({f"l{i}.mlp.{k}": s for k, s in L.ff.tensors(E).items()})
        return t


def _layers(d):
    layers = []
    for i, L in enumerate(d["layers"]):
        if L["type"] not in MIXERS:
            raise ValueError(f"layer {i}: mixer '{L['type']}' is not known (known: {', '.join(sorted(MIXERS))})")
        mlp, ff = L.get("mlp"), None
        if mlp is not None:
            if mlp["kind"] not in ("dense", "moe"):
                raise ValueError(f"layer {i}: feed-forward '{mlp['kind']}' is not known")
            ff = Dense(int(mlp["ff"])) if mlp["kind"] == "dense" else Experts.from_config(mlp)
        layers.append(MixerLayer(MIXERS[L["type"]].from_config(L["mixer"]), ff))
    return layers


def vomotar_config(d):
    """config.json of the Vomotar design (parsed) -> MixerConfig."""
    return MixerConfig(arch=d["architecture"], n_vocab=int(d["vocab"]), n_embd=int(d["width"]), norm_groups=int(d["norm"]["groups"]),
                       norm_eps=float(d["norm"]["eps"]), layers=_layers(d))


def zaparax_config(d):
    """config.json of the Zaparax design (parsed) -> MixerConfig."""
    emb, loop = d["embedding"], d.get("loop")
    b = emb.get("bigram")
    return MixerConfig(arch=d["architecture"], n_vocab=int(d["vocab"]), n_embd=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                       layers=_layers(d), emb_scale=float(emb.get("scale", 1.0)), norm_add=1.0, post_norm=True,
                       pairs=BigramTable(int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"])) if b else None,
                       loop=(int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else None)


ARCHITECTURES = {"Vomotar": vomotar_config, "Zaparax": zaparax_config}


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
