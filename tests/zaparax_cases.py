"""Small Zaparax models for the tests: configurations as config.json dictionaries and random weights.

Weights are drawn so that mistakes show: attention is sharp and sinks take a visible share, decays spread from none to a
few tokens, corrections change which experts are chosen.  `steady` weights let the corrections alone decide the choice, so
that a reduced-precision run cannot choose otherwise.
"""
import copy

import numpy as np

from adam_amd.safetensors_file import f32_to_bf16


def att(heads=4, kv_heads=2, dim=12, vdim=20, window=7, scale=0.4, softcap=4.0, coef=0.5, every=5):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window}}
    if softcap:
        m["softcap"] = softcap
    if coef:
        m["q_temp"] = {"coef": coef, "every": every}
    return {"type": "attention", "mixer": m}


def ssm(heads=6, groups=3, state=10, vdim=7, conv=3, norm_groups=2):
    return {"type": "mamba2", "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": norm_groups}}


def moe(experts=5, identity=2, top=3, ff=20, shared=28):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def config(layers, width=60, vocab=97, eps=1e-4, loop=None, scale=3.0, bigram=(37, 5, 11)):
    out = []
    for L in layers:
        L = copy.deepcopy(L)
        L.setdefault("mlp", moe())
        out.append(L)
    emb = {"scale": scale}
    if bigram:
        emb["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    c = {"architecture": "Zaparax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": emb, "layers": out}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CONFIGS = {
    # grouped heads everywhere, odd sizes, a looped pair, a layer without a feed-forward
    "odd": config([att(), ssm(), att(heads=3, kv_heads=3, dim=9, vdim=5, window=19), {**ssm(heads=2, groups=1, norm_groups=7), "mlp": None}],
                  loop=(1, 3, 2)),
    # one of everything: a window of one token beside one wider than the sequence, one expert, no convolution to speak of
    "ones": config([att(heads=1, kv_heads=1, dim=8, vdim=8, window=1, scale=1.0, softcap=None, coef=0),
                    {**ssm(heads=1, groups=1, state=1, vdim=1, conv=1, norm_groups=1), "mlp": moe(1, 0, 1, 16, 0)},
                    att(heads=2, kv_heads=1, dim=33, vdim=3, window=4000, every=1)],
                   width=33, vocab=41, loop=(0, 1, 1), scale=1.0, bigram=None),
    # as wide as heads get, many experts, several passes over the whole stack
    "wide": config([{**att(heads=10, kv_heads=2, dim=136, vdim=72, window=33, scale=0.09), "mlp": moe(70, 9, 11, 40, 72)},
                    {**ssm(heads=4, groups=2, state=144, vdim=48, conv=5, norm_groups=3), "mlp": moe(3, 1, 4, 130, 24)}],
                   width=192, vocab=300, loop=(0, 2, 3), bigram=(251, 4093, 65521)),
}


def tensor_shapes(cfg):
    E, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, E), "head": (V, E), "final.norm": (E,)}
    if "bigram" in cfg["embedding"]:
        s["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, E)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        s.update({p + "norm1": (E,), p + "norm1b": (E,)})
        H, V = m["heads"], m["vdim"]
        if L["type"] == "attention":
            for n, r in (("q", H * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * V)):
                s.update({p + "mix." + n: (r, E), p + f"mix.{n}.b": (r,)})
            s.update({p + "mix.sink": (H,), p + "mix.o": (E, H * V)})
        else:
            ch = H * V + 2 * m["groups"] * m["state"]
            s.update({p + "mix.in": (H * V + ch + H, E), p + "mix.conv": (ch, m["conv"]), p + "mix.conv.b": (ch,), p + "mix.dt_bias": (H,),
                      p + "mix.A_log": (H,), p + "mix.D": (H,), p + "mix.norm": (H * V,), p + "mix.o": (E, H * V)})
        mlp = L["mlp"]
        if mlp is None:
            continue
        s.update({p + "norm2": (E,), p + "norm2b": (E,)})
        r, F = mlp["router"], mlp["expert"]["ff"]
        for e in range(r["experts"]):
            s.update({p + f"mlp.e{e}.gate": (F, E), p + f"mlp.e{e}.up": (F, E), p + f"mlp.e{e}.down": (E, F)})
        n = r["experts"] + r["identity"]
        s.update({p + "mlp.router": (n, E), p + "mlp.correction": (n,)})
        if "shared" in mlp:
            F = mlp["shared"]["ff"]
            s.update({p + "mlp.shared.gate": (F, E), p + "mlp.shared.up": (F, E), p + "mlp.shared.down": (E, F), p + "mlp.shared.sg": (1, E)})
    return s


def weights(cfg, seed=0, steady=False):
    """name -> uint16 bfloat16 patterns."""
    rng = np.random.default_rng(seed)
    out = {}
    for n, s in tensor_shapes(cfg).items():
        last = n.split(".")[-1]
        if last in ("norm1", "norm1b", "norm2", "norm2b") or n == "final.norm":
            w = rng.uniform(-0.5, 0.5, s)
        elif n.endswith("mix.norm"):
            w = rng.uniform(0.5, 1.5, s)
        elif last == "A_log":
            w = np.linspace(-4.0, 1.0, s[0])[rng.permutation(s[0])]
        elif last == "dt_bias":
            w = rng.uniform(-4.0, 1.0, s)
        elif last in ("D", "b"):
            w = rng.standard_normal(s) * 0.5
        elif last == "sink":
            w = np.linspace(-1.0, 2.5, s[0])
        elif last == "correction":
            w = rng.permutation(s[0]) * 2.0 if steady else rng.uniform(-0.15, 0.15, s)
        elif last == "conv":
            w = rng.standard_normal(s) * 0.7
        elif n in ("embed", "bigram"):
            w = rng.standard_normal(s)
        else:
            w = rng.standard_normal(s) / np.sqrt(s[-1])
            if last == "router":
                w = w * 2.0
        out[n] = f32_to_bf16(w.astype(np.float32))
    return out
