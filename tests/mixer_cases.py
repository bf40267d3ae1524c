"""Small layered-mixer models for the tests: configurations as config.json dictionaries and random weights.

Weights are drawn so that mistakes show: queries and keys are strong enough that attention is sharp, decays spread from
none to a few tokens, and the distance penalty is large enough to matter.
"""
import copy

import numpy as np

from adam_amd.safetensors_file import bf16_to_f32, f32_to_bf16


def delta(heads=4, kv_heads=2, dim=24, vdim=20, conv=4):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def par(heads=4, kv_heads=2, dim=16, vdim=24, size=10, scale=0.3, r_heads=3, r_dim=20, r_vdim=12, rot=12, base=5000.0, decay=None):
    decay = decay or [1.0 - 2.0 ** -(2 + 2 * i) for i in range(r_heads)]
    return {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size}},
        "right": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "rot": {"base": base, "dims": rot}, "decay": decay}}}


def config(layers, width=60, vocab=97, groups=3, eps=1e-4, ff=52):
    out = []
    for i, L in enumerate(layers):
        L = copy.deepcopy(L)
        L["mlp"] = L.get("mlp", {"kind": "dense", "ff": ff})
        out.append(L)
    return {"architecture": "Vomotar", "width": width, "vocab": vocab, "norm": {"groups": groups, "eps": eps}, "layers": out}


CONFIGS = {
    # grouped heads everywhere, odd sizes, a layer without a feed-forward, rotation of a part of each head
    "odd": config([delta(), par(), {**delta(heads=3, kv_heads=3, dim=17, vdim=33, conv=3), "mlp": None}, par(size=7)],
                  width=60, vocab=97, groups=3),
    # one head, one group, no convolution to speak of, chunk of one token beside a large one
    "ones": config([par(heads=1, kv_heads=1, dim=8, vdim=8, size=1, r_heads=1, r_dim=8, r_vdim=5, rot=8, decay=[0.9]),
                    delta(heads=1, kv_heads=1, dim=9, vdim=7, conv=1), par(size=1000)], width=33, vocab=41, groups=1, ff=16),
    # as wide as heads get: 128 and more, many groups
    "wide": config([delta(heads=2, kv_heads=1, dim=128, vdim=144, conv=5),
                    par(heads=2, kv_heads=1, dim=136, vdim=128, size=70, scale=0.05, r_heads=2, r_dim=192, r_vdim=80, rot=64)],
                   width=192, vocab=300, groups=8, ff=200),
}


def tensor_shapes(cfg, rank=11):
    E, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, E), "head": (V, E), "final.norm": (E,)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        s[p + "norm1"] = (E,)
        if L["type"] == "channel_delta":
            H, K, D, U, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            for n, r in (("q", K * D), ("k", K * D), ("v", H * U)):
                s[p + "mix." + n] = (r, E)
                s[p + f"mix.{n}.conv"] = (r, T)
            s.update({p + "mix.b": (H, E), p + "mix.A_log": (H,), p + "mix.dt_bias": (H * D,), p + "mix.norm": (U,),
                      p + "mix.a1": (rank, E), p + "mix.a2": (H * D, rank), p + "mix.g1": (rank + 3, E),
                      p + "mix.g2": (H * U, rank + 3), p + "mix.o": (E, H * U)})
        else:
            a, r = m["left"], m["right"]
            q = p + "mix.left."
            s.update({q + "q": (a["heads"] * a["dim"], E), q + "k": (a["kv_heads"] * a["dim"], E),
                      q + "v": (a["kv_heads"] * a["vdim"], E), q + "o": (E, a["heads"] * a["vdim"]), q + "r1": (a["heads"],),
                      q + "r2": (a["heads"],), q + "out": (E,)})
            q = p + "mix.right."
            s.update({q + "q": (r["heads"] * r["dim"], E), q + "k": (r["heads"] * r["dim"], E), q + "v": (r["heads"] * r["vdim"], E),
                      q + "g": (r["heads"] * r["vdim"], E), q + "o": (E, r["heads"] * r["vdim"]), q + "out": (E,)})
        if L["mlp"] is not None:
            F = L["mlp"]["ff"]
            s.update({p + "norm2": (E,), p + "mlp.gate": (F, E), p + "mlp.up": (F, E), p + "mlp.down": (E, F)})
    return s


def weights(cfg, seed=0):
    """name -> uint16 bfloat16 patterns."""
    rng = np.random.default_rng(seed)
    out = {}
    for n, s in tensor_shapes(cfg).items():
        if n.endswith((".norm1", ".norm2", "final.norm", "mix.norm", ".out")):
            w = rng.uniform(0.5, 1.5, s)
        elif n.endswith("A_log"):
            w = np.linspace(-4.0, 1.0, s[0])[rng.permutation(s[0])]
        elif n.endswith("dt_bias"):
            w = rng.uniform(-4.0, 1.0, s)
        elif n.endswith("r1"):
            w = np.linspace(0.05, 2.0, s[0])
        elif n.endswith("r2"):
            w = rng.uniform(0.1, 0.6, s)
        elif n.endswith(".conv"):
            w = rng.standard_normal(s) * 0.7
        elif n == "embed":
            w = rng.standard_normal(s)
        else:
            w = rng.standard_normal(s) / np.sqrt(s[-1])
            if n.endswith(("left.q", "left.k")):
                w = w * 1.5
        out[n] = f32_to_bf16(w.astype(np.float32))
    return out


def floats(W):
    return {n: bf16_to_f32(w).astype(np.float64) for n, w in W.items()}


def write_model(folder, cfg, W):
    """config.json and model.safetensors of a test model."""
    import json
    import os
    import struct
    head, at = {}, 0
    for n, w in W.items():
        head[n] = {"dtype": "BF16", "shape": list(w.shape), "data_offsets": [at, at + w.nbytes]}
        at += w.nbytes
    js = json.dumps(head).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(js)) + js + b"".join(np.ascontiguousarray(w).tobytes() for w in W.values()))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)


def rel(a, b):
    """Largest root mean square difference of a row, over the root mean square of all of b."""
    a, b = np.asarray(a, np.float64), np.asarray(b, np.float64)
    return float(np.sqrt(np.mean((a - b) ** 2, axis=-1)).max() / np.sqrt(np.mean(b * b)))
