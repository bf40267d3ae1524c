"""Feed-forwards of the layered models: what tensors each has, how its matrices are stacked, and the ops it issues.

As with the mixers, the engine owns rows, weights and operands; a feed-forward only describes.  Its members:
  tensors(E)        name -> shape
  vectors()         names of the tensors kept as float32 in the workspace
  stacks(E)         stack name -> blocks of matrices that lie under each other; a block is a tensor's name, or a (gate, up)
                    pair whose rows alternate in runs of 16
  widths(E)         row buffer -> width of one row per token
  single(E)         row buffer -> elements, for what only one token's step needs
  operands()        key -> operand elements per token (`e.operand(key)` is the region's offset)
  issue(e, p, norm, out, epi)   issue the ops: `norm` is the input's norm, `out` the rows the result goes to
"""
from dataclasses import dataclass


def up_to(n, m):
    return (n + m - 1) // m * m


@dataclass
class Dense:
    """W_down (silu(W_gate h) * (W_up h))."""
    ff: int

    def tensors(self, E):
        return {"gate": (self.ff, E), "up": (self.ff, E), "down": (E, self.ff)}

    def vectors(self):
        return []

    def stacks(self, E):
        return {"in": [("gate", "up")], "out": ["down"]}

    def widths(self, E):
        return {}

    def single(self, E):
        return {"act": up_to(self.ff, 16)}

    def operands(self):
        return {("act", self.ff): up_to(self.ff, 64)}

    def issue(self, e, p, norm, out, epi):
        act = (e.operand(("act", self.ff)), up_to(self.ff, 64))
        e.linear([p + "in"], src=e.residual(), out=e.at("act"), norm=norm, epi=e.A.EPI_SWIGLU, out_opnd=act)
        e.linear([p + "out"], src=e.at("act"), out=out, epi=epi, opnd=act[0], ready=1)


MAX_CHOICES, MAX_TOP = 1024, 64          # outputs of a router, experts a token takes
MAX_STEP = 32768                         # activations one token's second product holds in shared memory


@dataclass
class Experts:
    """Gated experts of which a token takes the `top` with the largest corrected softmax scores, weighted by the scores as
    they are; the last `identity` router outputs give the input back; a shared expert behind a sigmoid of its own."""
    experts: int
    identity: int
    top: int
    ff: int
    shared_ff: int = 0

    @classmethod
    def from_config(cls, d):
        r, s = d["router"], d.get("shared")
        return cls(int(r["experts"]), int(r.get("identity", 0)), int(r["top"]), int(d["expert"]["ff"]), int(s["ff"]) if s else 0)

    def __post_init__(self):
        n = self.experts + self.identity
        if self.experts < 1 or self.identity < 0 or n > MAX_CHOICES or not 1 <= self.top <= min(n, MAX_TOP):
            raise ValueError(f"experts: top {self.top} of {self.experts} + {self.identity} (at most {MAX_TOP} of {MAX_CHOICES})")
        held = min(self.top, self.experts) * up_to(self.ff, 64) + (up_to(self.shared_ff, 64) if self.shared_ff else 0)
        if self.ff < 1 or held > MAX_STEP:
            raise ValueError(f"experts: {held} activations a token (at most {MAX_STEP})")

    def tensors(self, E):
        n = self.experts + self.identity
        t = {"router": (n, E), "correction": (n,)}
        for e in range(self.experts):
            t.update({f"e{e}.gate": (self.ff, E), f"e{e}.up": (self.ff, E), f"e{e}.down": (E, self.ff)})
        if self.shared_ff:
            t.update({"shared.gate": (self.shared_ff, E), "shared.up": (self.shared_ff, E), "shared.down": (E, self.shared_ff),
                      "shared.sg": (1, E)})
        return t

    def vectors(self):
        return ["correction"]

    def stacks(self, E):
        each = range(self.experts)
        t = {"route": ["router"], "experts.in": [(f"e{e}.gate", f"e{e}.up") for e in each], "experts.out": [f"e{e}.down" for e in each]}
        if self.shared_ff:
            t.update({"route": [("shared.gate", "shared.up"), "router", "shared.sg"], "shared.out": ["shared.down"]})
        return t

    def widths(self, E):
        w = {"h": E, "route": self.experts + self.identity + 1}
        return {**w, "shared": E} if self.shared_ff else w

    def single(self, E):
        return {"act": self.top * up_to(self.ff, 64), "shared_act": up_to(self.shared_ff, 16)}

    def operands(self):
        r = {("experts", self.ff): self.top * up_to(self.ff, 64)}
        return {**r, ("act", self.shared_ff): up_to(self.shared_ff, 64)} if self.shared_ff else r

    def issue(self, e, p, norm, out, epi):
        A, n, F = e.A, self.experts + self.identity, up_to(self.ff, 64)
        keep, route, src = e.at("h"), e.at("route"), e.residual()
        shared, sh = {}, 0
        if self.shared_ff:
            S = up_to(self.shared_ff, 64)
            act = (e.operand(("act", self.shared_ff)), S)
            e.linear([p + "route"], src=src, out=e.at("shared_act"), norm=norm, keep=keep, epi=A.EPI_SWIGLU, out_opnd=act, tail=(n + 1, route))
            mid, sh = e.linear_spec([p + "shared.out"], src=e.at("shared_act"), out=e.at("shared"), opnd=act[0], ready=1)
            shared = dict(shared_ff=self.shared_ff, shared_ff_stride=S, shared_down=e.stack([p + "shared.out"])[1], shared_act=e.at("shared_act")[0])
        else:
            e.linear([p + "route"], src=src, out=route, norm=norm, keep=keep)
        mid, up, _, _, ks = e.stack([p + "experts.in"])
        _, down, _, _, _ = e.stack([p + "experts.out"])
        e.experts(mid, A.ExpertsSpec(
            experts=self.experts, identity=self.identity, top=self.top, ff=self.ff, ff_stride=F, width=e.cfg.n_embd, k_stride=ks,
            gate_up=up, gate_up_step=2 * up_to(self.ff, 16) * ks, down=down, down_step=e.cfg.n_embd * F, logits=route[0],
            logits_stride=route[1], correction=e.vec(p + "correction"), x=keep[0], x_stride=keep[1], opnd=0, act=e.at("act")[0],
            act_opnd=e.operand(("experts", self.ff)), out=out[0], out_stride=out[1], epi=epi, **shared), sh)
