"""Sequence mixers of the layered models: what tensors each has, what a sequence keeps of it, and the ops it issues.

A mixer names its input projections (they all read the layer's normed hidden row, so they are stacked into one
matrix), issues its core op over the rows those projections leave in the `x` rows, and its output projection.  The
engine (`mixer_engine.MixerEngine`) owns rows, weights, state and cache; a mixer only describes.  Sizes and constants
come from the model's configuration; the ranks of low-rank projections come from the tensors.

Another mixer is another class with these members:
  tensors(E)            name -> shape, None where the tensor decides
  inputs()              names of the stacked input projections, in order
  vectors()             names of the tensors kept as float32 in the workspace
  biases()              names of the stacked input projections' biases, in the inputs' order ([]: none)
  widths(shape)         row buffer -> width it needs
  state_size(), cache_size()   elements per sequence in the float32 state map / in the key-value cache map
  const_size()          float32 constants from the configuration (`e.const`)
  core(e, p, x)         issue the sequence op: x maps an input's name to its column in the `x` rows
  output(e, p, x, out, epi)    issue the output projection into the rows `out`
"""
from dataclasses import dataclass

import numpy as np


MAX_DIM, MAX_TAPS = 256, 16            # what the kernels hold of a head in registers and shared memory


def _fits(name, **dims):
    for n, v in dims.items():
        top = MAX_TAPS if n == "conv" else MAX_DIM
        if not 1 <= v <= top:
            raise ValueError(f"{name}: {n} = {v} is outside 1 .. {top}")


def _grouped(name, heads, kv_heads):
    if kv_heads < 1 or heads % kv_heads:
        raise ValueError(f"{name}: {heads} heads do not share {kv_heads} key heads evenly")


class Mixer:
    def biases(self):
        return []


@dataclass
class ChannelDelta(Mixer):
    """Gated delta rule: short convolutions on q, k, v, unit q and k, one decay per head and key channel (low-rank),
    per-head norm and a low-rank sigmoid gate on the way out."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    @classmethod
    def from_config(cls, d):
        return cls(*(int(d[n]) for n in ("heads", "kv_heads", "dim", "vdim", "conv")))

    def __post_init__(self):
        _fits("delta rule", dim=self.dim, vdim=self.vdim, conv=self.conv)
        _grouped("delta rule", self.heads, self.kv_heads)

    def tensors(self, E):
        H, KH, D, V, T = self.heads, self.kv_heads, self.dim, self.vdim, self.conv
        return {"q": (KH * D, E), "k": (KH * D, E), "v": (H * V, E), "b": (H, E), "a1": (None, E), "a2": (H * D, None),
                "g1": (None, E), "g2": (H * V, None), "o": (E, H * V), "q.conv": (KH * D, T), "k.conv": (KH * D, T),
                "v.conv": (H * V, T), "A_log": (H,), "dt_bias": (H * D,), "norm": (V,)}

    def inputs(self):
        return ["q", "k", "v", "b", "a1", "g1"]

    def vectors(self):
        return ["q.conv", "k.conv", "v.conv", "A_log", "dt_bias", "norm"]

    def widths(self, shape):
        return {"a": self.heads * self.dim, "g": self.heads * self.vdim, "o": self.heads * self.vdim}

    def _channels(self):
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    def state_size(self):
        return self.heads * self.dim * self.vdim + self.conv * self._channels()

    def cache_size(self):
        return 0

    def const_size(self):
        return 0

    def core(self, e, p, x):
        A = e.A
        decay = e.linear_spec([p + "a2"], src=e.at("x", x["a1"]), out=e.at("a"))
        gate = e.linear_spec([p + "g2"], src=e.at("x", x["g1"]), out=e.at("g"))
        s_off = e.take_state(self.state_size())
        xo, xs = e.at("x", x["q"])
        oo, os_ = e.at("o")
        spec = A.DeltaSpec(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, taps=self.conv, x=xo,
                           x_stride=xs, x_b=x["b"] - x["q"], cq=e.vec(p + "q.conv"), ck=e.vec(p + "k.conv"),
                           cv=e.vec(p + "v.conv"), a_log=e.vec(p + "A_log"), dt_bias=e.vec(p + "dt_bias"), out=oo,
                           out_stride=os_, state_map=e.STATE_MAP, s_off=s_off,
                           conv_off=s_off + self.heads * self.dim * self.vdim, seq_stride=e.state_per_seq)
        e.delta_rule(spec, decay, gate)

    def output(self, e, p, x, out, epi):
        go, gs = e.at("g")
        e.linear([p + "o"], src=e.at("o"), out=out, epi=epi,
                 norm=e.norm(self.heads, e.vec(p + "norm"), self.vdim, gate=(go, gs, e.A.GATE_SIGMOID)))


@dataclass
class ChunkAttention(Mixer):
    """Softmax attention over the keys of the query's own chunk, with r1 ln(1 + r2 distance) taken off the scores and
    values divided by their root mean square; grouped key / value heads, no rotation."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int
    rows: str = "o"

    @classmethod
    def from_config(cls, d, rows="o"):
        return cls(int(d["heads"]), int(d["kv_heads"]), int(d["dim"]), int(d["vdim"]), float(d["scale"]),
                   int(d["mask"]["size"]), rows)

    def __post_init__(self):
        _fits("chunk attention", dim=self.dim, vdim=self.vdim)
        _grouped("chunk attention", self.heads, self.kv_heads)
        if self.chunk < 1:
            raise ValueError(f"chunk attention: a chunk of {self.chunk} tokens")

    def tensors(self, E):
        H, G, D, V = self.heads, self.kv_heads, self.dim, self.vdim
        return {"q": (H * D, E), "k": (G * D, E), "v": (G * V, E), "o": (E, H * V), "r1": (H,), "r2": (H,)}

    def inputs(self):
        return ["q", "k", "v"]

    def vectors(self):
        return ["r1", "r2"]

    def widths(self, shape):
        return {self.rows: self.heads * self.vdim}

    def state_size(self):
        return 0

    def cache_size(self):
        r8 = lambda n: (n + 7) // 8 * 8
        return self.kv_heads * self.chunk * (r8(self.dim) + r8(self.vdim))

    def const_size(self):
        return 0

    def core(self, e, p, x):
        r8 = lambda n: (n + 7) // 8 * 8
        off = e.take_cache(self.cache_size())
        xo, xs = e.at("x")
        oo, os_ = e.at(self.rows)
        e.chunk_attention(e.A.ChunkAttnSpec(
            heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, chunk=self.chunk, x=xo, x_stride=xs,
            x_q=x["q"], x_k=x["k"], x_v=x["v"], r1=e.vec(p + "r1"), r2=e.vec(p + "r2"), scale=self.scale, eps=e.cfg.norm_eps,
            out=oo, out_stride=os_, cache_map=e.CACHE_MAP, k_off=off, v_off=off + self.kv_heads * self.chunk * r8(self.dim),
            seq_stride=e.cache_per_seq))

    def output(self, e, p, x, out, epi):
        e.linear([p + "o"], src=e.at(self.rows), out=out, epi=epi)


@dataclass
class Retention(Mixer):
    """Linear attention with one fixed decay per head; rotary q and k, per-head norm without weight, silu gate."""
    heads: int
    dim: int
    vdim: int
    decay: tuple
    rot_base: float
    rot_dims: int
    rows: str = "o"

    @classmethod
    def from_config(cls, d, rows="o"):
        return cls(int(d["heads"]), int(d["dim"]), int(d["vdim"]), tuple(float(v) for v in d["decay"]), float(d["rot"]["base"]),
                   int(d["rot"]["dims"]), rows)

    def __post_init__(self):
        _fits("retention", dim=self.dim, vdim=self.vdim)
        if len(self.decay) != self.heads:
            raise ValueError(f"retention: {len(self.decay)} decays for {self.heads} heads")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError(f"retention: {self.rot_dims} rotated dimensions of {self.dim}")

    def tensors(self, E):
        H, D, V = self.heads, self.dim, self.vdim
        return {"q": (H * D, E), "k": (H * D, E), "v": (H * V, E), "g": (H * V, E), "o": (E, H * V)}

    def inputs(self):
        return ["q", "k", "v", "g"]

    def vectors(self):
        return []

    def widths(self, shape):
        return {self.rows: self.heads * self.vdim}

    def state_size(self):
        return self.heads * self.dim * self.vdim

    def cache_size(self):
        return 0

    def const_size(self):
        return self.rot_dims // 2 + self.heads

    def core(self, e, p, x):
        half = self.rot_dims // 2
        freq = e.const(np.float64(self.rot_base) ** (-2.0 * np.arange(half) / max(self.rot_dims, 1)))
        xo, xs = e.at("x")
        oo, os_ = e.at(self.rows)
        e.retention(e.A.RetentionSpec(
            heads=self.heads, dim=self.dim, vdim=self.vdim, rot_dims=self.rot_dims, freq=freq, decay=e.const(self.decay),
            x=xo, x_stride=xs, x_q=x["q"], x_k=x["k"], x_v=x["v"], out=oo, out_stride=os_, state_map=e.STATE_MAP,
            s_off=e.take_state(self.state_size()), seq_stride=e.state_per_seq))

    def output(self, e, p, x, out, epi):
        xo, xs = e.at("x", x["g"])
        e.linear([p + "o"], src=e.at(self.rows), out=out, epi=epi, norm=e.norm(self.heads, gate=(xo, xs, e.A.GATE_SILU)))


@dataclass
class Parallel(Mixer):
    """Mean of two branches over the same input, each through a full-width RMS norm with a weight of its own."""
    left: object
    right: object

    @classmethod
    def from_config(cls, d):
        return cls(ChunkAttention.from_config(d["left"], "o"), Retention.from_config(d["right"], "o2"))

    def _both(self):
        return (("left.", self.left), ("right.", self.right))

    def tensors(self, E):
        t = {n + "out": (E,) for n, _ in self._both()}
        for n, m in self._both():
            t.update({n + k: v for k, v in m.tensors(E).items()})
        return t

    def inputs(self):
        return [n + k for n, m in self._both() for k in m.inputs()]

    def vectors(self):
        return [n + k for n, m in self._both() for k in m.vectors() + ["out"]]

    def widths(self, shape):
        w = {"y": None, "y2": None}                   # None: the model width
        for _, m in self._both():
            w.update(m.widths(shape))
        return w

    def state_size(self):
        return self.left.state_size() + self.right.state_size()

    def cache_size(self):
        return self.left.cache_size() + self.right.cache_size()

    def const_size(self):
        return self.left.const_size() + self.right.const_size()

    @staticmethod
    def _cols(x, n):
        return {k[len(n):]: v for k, v in x.items() if k.startswith(n)}

    def core(self, e, p, x):
        for n, m in self._both():
            m.core(e, p + n, self._cols(x, n))

    def output(self, e, p, x, out, epi):
        for (n, m), rows in zip(self._both(), ("y", "y2")):
            m.output(e, p + n, self._cols(x, n), e.at(rows), e.A.EPI_STORE)
        e.merge("y", "y2", e.vec(p + "left.out"), e.vec(p + "right.out"), out, 0.5, epi)


@dataclass
class WindowAttention(Mixer):
    """Softmax attention over a sliding window with a learned sink per head in the denominator: queries and keys divided by
    their root mean square, a query temperature that grows with the logarithm of the position, capped scores, a linear
    distance penalty per head; grouped key / value heads, biased projections, no rotation."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int
    softcap: float = 0.0
    temp_coef: float = 0.0
    temp_every: int = 1
    rows: str = "o"

    @classmethod
    def from_config(cls, d, rows="o"):
        t = d.get("q_temp") or {}
        return cls(int(d["heads"]), int(d["kv_heads"]), int(d["dim"]), int(d["vdim"]), float(d["scale"]), int(d["mask"]["size"]),
                   float(d.get("softcap") or 0.0), float(t.get("coef", 0.0)), int(t.get("every", 1)), rows)

    def __post_init__(self):
        _fits("window attention", dim=self.dim, vdim=self.vdim)
        _grouped("window attention", self.heads, self.kv_heads)
        if self.window < 1 or self.softcap < 0 or self.temp_every < 1:
            raise ValueError(f"window attention: window {self.window}, cap {self.softcap}, temperature every {self.temp_every}")

    def tensors(self, E):
        H, G, D, V = self.heads, self.kv_heads, self.dim, self.vdim
        return {"q": (H * D, E), "q.b": (H * D,), "k": (G * D, E), "k.b": (G * D,), "v": (G * V, E), "v.b": (G * V,), "sink": (H,),
                "o": (E, H * V)}

    def inputs(self):
        return ["q", "k", "v"]

    def biases(self):
        return ["q.b", "k.b", "v.b"]

    def vectors(self):
        return ["sink"]

    def widths(self, shape):
        return {self.rows: self.heads * self.vdim}

    def state_size(self):
        return 0

    def cache_size(self):
        r8 = lambda n: (n + 7) // 8 * 8
        return self.kv_heads * self.window * (r8(self.dim) + r8(self.vdim))

    def const_size(self):
        return self.heads

    def core(self, e, p, x):
        r8 = lambda n: (n + 7) // 8 * 8
        off = e.take_cache(self.cache_size())
        xo, xs = e.at("x")
        oo, os_ = e.at(self.rows)
        slope = e.const(2.0 ** (-8.0 * np.arange(1, self.heads + 1) / self.heads))
        e.window_attention(e.A.WindowAttnSpec(
            heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, window=self.window, x=xo, x_stride=xs,
            x_q=x["q"], x_k=x["k"], x_v=x["v"], slope=slope, sink=e.vec(p + "sink"), has_sink=1, qk_norm=1, scale=self.scale,
            eps=e.cfg.norm_eps, softcap=self.softcap, temp_coef=self.temp_coef, temp_every=self.temp_every, out=oo, out_stride=os_,
            cache_map=e.CACHE_MAP, k_off=off, v_off=off + self.kv_heads * self.window * r8(self.dim), seq_stride=e.cache_per_seq))

    def output(self, e, p, x, out, epi):
        e.linear([p + "o"], src=e.at(self.rows), out=out, epi=epi)


@dataclass
class StateSpace(Mixer):
    """Mamba-2: one projection for gate, inputs and step sizes, a short biased convolution, a state per head that decays by
    one factor per token, gate ahead of a norm in equal parts."""
    heads: int
    groups: int
    state: int
    vdim: int
    conv: int
    norm_groups: int

    @classmethod
    def from_config(cls, d):
        return cls(*(int(d[n]) for n in ("heads", "groups", "state", "vdim", "conv", "norm_groups")))

    def __post_init__(self):
        _fits("state space", state=self.state, vdim=self.vdim, conv=self.conv)
        if self.groups < 1 or self.heads % self.groups:
            raise ValueError(f"state space: {self.heads} heads do not share {self.groups} groups evenly")
        if self.norm_groups < 1 or self.inner % self.norm_groups:
            raise ValueError(f"state space: {self.inner} channels do not split into {self.norm_groups} norm groups")

    @property
    def inner(self):
        return self.heads * self.vdim

    @property
    def channels(self):
        return self.inner + 2 * self.groups * self.state

    def tensors(self, E):
        return {"in": (self.inner + self.channels + self.heads, E), "conv": (self.channels, self.conv), "conv.b": (self.channels,),
                "dt_bias": (self.heads,), "A_log": (self.heads,), "D": (self.heads,), "norm": (self.inner,), "o": (E, self.inner)}

    def inputs(self):
        return ["in"]

    def vectors(self):
        return ["conv", "conv.b", "dt_bias", "A_log", "D", "norm"]

    def widths(self, shape):
        return {"o": self.inner}

    def state_size(self):
        return self.heads * self.state * self.vdim + self.conv * self.channels

    def cache_size(self):
        return 0

    def const_size(self):
        return 0

    def core(self, e, p, x):
        xo, xs = e.at("x", x["in"])
        oo, os_ = e.at("o")
        s_off = e.take_state(self.state_size())
        e.state_space(e.A.StateSpaceSpec(
            heads=self.heads, groups=self.groups, state=self.state, vdim=self.vdim, taps=self.conv, x=xo, x_stride=xs, x_c=self.inner,
            x_dt=self.inner + self.channels, conv=e.vec(p + "conv"), conv_b=e.vec(p + "conv.b"), dt_bias=e.vec(p + "dt_bias"),
            a_log=e.vec(p + "A_log"), skip=e.vec(p + "D"), out=oo, out_stride=os_, state_map=e.STATE_MAP, s_off=s_off,
            conv_off=s_off + self.heads * self.state * self.vdim, seq_stride=e.state_per_seq))

    def output(self, e, p, x, out, epi):
        zo, zs = e.at("x", x["in"])
        e.linear([p + "o"], src=e.at("o"), out=out, epi=epi,
                 norm=e.norm(self.norm_groups, e.vec(p + "norm"), self.inner, gate=(zo, zs, e.A.GATE_SILU_AHEAD)))


MIXERS = {"channel_delta": ChannelDelta, "parallel": Parallel, "attention": WindowAttention, "mamba2": StateSpace}
