"""Layered mixer models on the GPU: every op against the NumPy op surface, whole models against the plain statement of
the mechanisms, in one piece, in portions, token by token, in lockstep, and through generation and trace replay."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import oracle
from adam_amd import adamah as A
from adam_amd.engine import GenerationConfig
from adam_amd.mixer_engine import MixerEngine
from adam_amd.models import load_engine, vomotar_config
from adam_amd.safetensors_file import f32_to_bf16
from gpu_util import note
from mixer_cases import CONFIGS, config, delta, floats, par, rel, weights, write_model
from mixer_pair import CA, OP, ST, WS, WT, Pair
from oracle import mixers_np as M

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": 2e-5, "bfloat16": 6e-2}      # bfloat16: the worst row; the NumPy surface with the same rounding reaches 3.3e-2


# ---- products --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rows,n,k,groups,epi", [
    (1, 70, 33, 3, 0), (1, 96, 640, 0, 2), (1, 51, 1100, 1, 1), (1, 33, 1536, 32, 0), (2, 70, 33, 3, 0), (5, 64, 200, 5, 2),
    (16, 129, 64, 1, 1), (17, 64, 320, 2, 2), (31, 45, 96, 0, 0), (33, 96, 130, 13, 2), (64, 200, 256, 4, 1), (65, 130, 72, 0, 0),
    (200, 1000, 192, 3, 0), (300, 8224, 64, 1, 2), (300, 8200, 128, 1, 1),
    (1, 10, 20000, 4, 0), (3, 37, 16000, 4, 0)])
def test_linear(hip, dtype, rows, n, k, groups, epi):
    note(f"linear {dtype} rows {rows} n {n} k {k} groups {groups} epi {epi}")
    rng = np.random.default_rng(rows * 1000 + n)
    ks, src_rows = (k + 63) // 64 * 64, rows + 3
    out_w = n // 2 if epi == 2 else n
    wt_len = 0 if not groups else (k if groups % 2 else k // groups)
    act = int(rng.integers(0, 3)) if groups else 0
    src, gate, wt, out = 5, 5 + src_rows * k, 5 + 2 * src_rows * k, 5 + 2 * src_rows * k + k
    total = out + rows * (out_w + 3)
    opnd, oo = 64, 64 + rows * ks
    p = Pair(hip, total + 64, wt=n * ks + 8, opnd=oo + rows * ((out_w + 63) // 64 * 64 + 64), dtype=dtype)
    W = np.zeros((n, ks), np.uint16)
    W[:, :k] = f32_to_bf16((rng.standard_normal((n, k)) / np.sqrt(k)).astype(np.float32))
    p.put(WT, 8, W)
    p.put(WS, 0, rng.standard_normal(total))
    spec = A.LinearSpec(w=8, n=n, k=k, k_stride=ks, src=src, src_stride=k, groups=groups, eps=1e-4, wt=wt, wt_len=wt_len, gate=gate,
                        gate_stride=k, gate_act=act, opnd=opnd, ready=0, out=out, out_stride=out_w + 3, epi=epi, out_opnd=oo,
                        out_opnd_stride=(out_w + 63) // 64 * 64)
    h = p.up(spec.words())
    pick = p.up(rng.integers(0, src_rows, rows))
    tol = 2e-5 if dtype == "float32" or rows == 1 else 4e-2        # bfloat16: an operand may round the other way
    p.call("linear_dev", WS, OP, WT, h, pick, rows)
    if epi == 2 and rows > 1:
        # the pairs went to the operand rows: a product with the identity brings them out, its operand ready
        w2 = (out_w + 63) // 64 * 64
        eye = np.zeros((out_w, w2), np.float32)
        eye[np.arange(out_w), np.arange(out_w)] = 1
        for g in p.g:
            g.map_create_typed(WT, A.DTYPE_BF16, 1, eye.size)
        p.put(WT, 0, f32_to_bf16(eye))
        s2 = A.LinearSpec(w=0, n=out_w, k=out_w, k_stride=w2, opnd=oo, ready=1, out=out, out_stride=out_w + 3)
        p.call("linear_dev", WS, OP, WT, p.up(s2.words()), 0, rows)
    p.same(WS, out, rows * (out_w + 3) - 3, tol, "out")


@pytest.mark.parametrize("rows", [1, 3])
def test_linear_argmax_takes_the_first_of_equals(hip, rows):
    note(f"linear argmax rows {rows}")
    n, k = 5003, 64
    rng = np.random.default_rng(2)
    p = Pair(hip, rows * k + rows * n + 64, wt=n * k, opnd=rows * k)
    W = f32_to_bf16(rng.standard_normal((n, k)).astype(np.float32))
    W[4001] = W[2003] = W[2002] = f32_to_bf16(np.full(k, 4.0, np.float32))
    p.put(WT, 0, W)
    x = np.abs(rng.standard_normal((rows, k)))
    p.put(WS, 0, x)
    spec = A.LinearSpec(w=0, n=n, k=k, k_stride=k, src=0, src_stride=k, out=rows * k, out_stride=n)
    p.call("linear_argmax_dev", WS, OP, WT, p.up(spec.words()), p.up(rows * (k + n) + np.arange(rows)), rows)
    a, b = p.read(WS, rows * (k + n), rows)
    assert a.tolist() == b.tolist() == [2002.0] * rows


def test_merge_norm(hip):
    note("merge norm")
    rows, dim, st = 5, 77, 80
    p = Pair(hip, 3 * rows * st + 2 * dim + 9)
    p.put(WS, 0, np.random.default_rng(0).standard_normal(p.n))
    spec = A.MergeSpec(a=0, b=rows * st, stride=st, wa=3 * rows * st, wb=3 * rows * st + dim, dst=2 * rows * st, dst_stride=st, dim=dim,
                       eps=1e-3, scale=0.5)
    p.call("merge_norm_dev", WS, p.up(spec.words()), rows)
    p.same(WS, 2 * rows * st, rows * st, 1e-5)


# ---- recurrences -----------------------------------------------------------------------------------------------------
def delta_pair(hip, H, KH, D, V, taps, rank, rows, seqs, strong, seed):
    rng = np.random.default_rng(seed)
    n_ch = 2 * KH * D + H * V
    xs = n_ch + H + 2 * rank + 1
    at, pos = {}, 3
    for n, sz in (("x", rows * xs), ("a", rows * H * D), ("g", rows * H * V), ("o", rows * H * V), ("conv", n_ch * taps), ("A", H), ("dt", H * D)):
        at[n] = pos
        pos += sz
    ks = (rank + 63) // 64 * 64
    state = H * D * V + taps * n_ch + 5
    p = Pair(hip, pos + 16, wt=(H * D + H * V) * ks, opnd=2 * rows * ks, state=seqs * state)
    W = np.zeros((H * D + H * V, ks), np.uint16)
    W[:, :rank] = f32_to_bf16((rng.standard_normal((H * D + H * V, rank)) / np.sqrt(rank)).astype(np.float32))
    p.put(WT, 0, W)
    p.put(WS, at["conv"], rng.standard_normal(n_ch * taps) * 0.7)
    p.put(WS, at["A"], np.linspace(-3.0, 3.0 if strong else 0.5, H))
    p.put(WS, at["dt"], rng.uniform(-4, 2 if strong else 0, H * D))
    p.put(ST, 0, np.full(seqs * state, 7.0))        # what another sequence left behind
    low = lambda w, n, col, out: p.up(A.LinearSpec(w=w, n=n, k=rank, k_stride=ks, src=at["x"] + n_ch + H + col, src_stride=xs, opnd=0,
                                                   out=at[out], out_stride=n).words())
    dec, gate = low(0, H * D, 0, "a"), low(H * D * ks, H * V, rank, "g")
    c = at["conv"]
    spec = p.up(A.DeltaSpec(heads=H, kv_heads=KH, dim=D, vdim=V, taps=taps, x=at["x"], x_stride=xs, x_b=n_ch, cq=c, ck=c + KH * D * taps,
                            cv=c + 2 * KH * D * taps, a_log=at["A"], dt_bias=at["dt"], out=at["o"], out_stride=H * V, state_map=ST,
                            s_off=1, conv_off=1 + H * D * V, seq_stride=state).words())
    fresh = lambda n: p.put(WS, at["x"], rng.standard_normal((n, xs)))

    def run(n_seq, m, seq0, pos0):
        fresh(n_seq * m)
        p.call("delta_rule_dev", WS, OP, WT, spec, dec, gate, n_seq, m, seq0, pos0)
        p.same(WS, at["o"], n_seq * m * H * V, 2e-5, f"outputs {n_seq}x{m} at {pos0}")
        p.same(WS, at["g"], n_seq * m * H * V, 2e-5, "gate")
        p.same(ST, seq0 * state + 1, H * D * V, 2e-5, f"state after {pos0 + m}")
    return run


@pytest.mark.parametrize("H,KH,D,V,taps,rank,strong", [
    (4, 2, 24, 20, 4, 11, False), (3, 3, 17, 33, 3, 5, True), (1, 1, 1, 1, 1, 1, False), (2, 1, 64, 16, 2, 70, True),
    (2, 2, 128, 144, 5, 16, False), (2, 1, 200, 40, 4, 128, True), (2, 1, 256, 64, 8, 30, False),
    (1, 1, 256, 250, 16, 20, False)])
def test_delta_rule(hip, H, KH, D, V, taps, rank, strong):
    note(f"delta rule H {H} KH {KH} D {D} V {V} taps {taps} rank {rank}")
    run = delta_pair(hip, H, KH, D, V, taps, rank, 40, 3, strong, seed=D)
    pos = 0
    for m in (2, 1, 17, 1, 1, 40, 16, 3):            # one sequence in slot 1, portions and single tokens in turn
        run(1, m, 1, pos)
        pos += m
    run(1, 33, 1, 0)                                 # the slot again, another sequence
    for i in range(3):
        run(1, 5, i, 0)
    for t in range(3):                               # one token of each of three sequences
        run(3, 1, 0, 5 + t)
    run(1, 1, 2, 0)                                  # a sequence that starts with a single token
    run(1, 2, 2, 1)


def test_delta_rule_keeps_a_key_over_a_long_gap(hip):
    """A channel that does not decay holds a value through 300 tokens beside channels that forget within one."""
    note("delta rule, long gap")
    H, D, V, taps = 1, 16, 8, 1
    n_ch, rank = 2 * D + V, 1
    xs = n_ch + 1 + 2
    N = 300
    p = Pair(hip, N * xs + N * (D + 2 * V) + n_ch + 1 + D + 8, wt=(D + V) * 64, opnd=N * 64, state=D * V + n_ch)
    ao, go, oo = N * xs, N * (xs + D), N * (xs + D + V)
    cv = N * (xs + D + 2 * V)
    p.put(WS, cv, np.ones(n_ch))
    p.put(WS, cv + n_ch, [0.0])
    p.put(WS, cv + n_ch + 1, np.where(np.arange(D) < 4, -40.0, 6.0))       # decay 1 - e^-40, and e^-6 per token
    x = np.zeros((N, xs), np.float32)
    x[:, D + 8] = 9.0                                # filler keys: one of the channels that forget
    x[:, 2 * D:2 * D + V] = np.random.default_rng(0).standard_normal((N, V))
    x[:, n_ch] = 6.0
    x[0, D:2 * D] = 0
    x[0, D + 1] = 9.0                                # token 0 writes under channel 1
    x[-1, 1] = 9.0                                   # the last token asks for it
    p.put(WS, 0, x)
    low = lambda w, n, out: p.up(A.LinearSpec(w=w, n=n, k=1, k_stride=64, src=n_ch + 1, src_stride=xs, out=out, out_stride=n).words())
    spec = p.up(A.DeltaSpec(heads=1, kv_heads=1, dim=D, vdim=V, taps=taps, x=0, x_stride=xs, x_b=n_ch, cq=cv, ck=cv + D, cv=cv + 2 * D,
                            a_log=cv + n_ch, dt_bias=cv + n_ch + 1, out=oo, out_stride=V, state_map=ST, s_off=0, conv_off=D * V,
                            seq_stride=D * V + n_ch).words())
    p.call("delta_rule_dev", WS, OP, WT, spec, low(0, D, ao), low(D * 64, V, go), 1, N, 0, 0)
    p.same(WS, oo, N * V, 2e-5)
    got = p.read(WS, oo + (N - 1) * V, V)[0]
    v0 = x[0, 2 * D:2 * D + V]
    want = M.silu(v0.astype(float)) * M.sigmoid(6.0) * D ** -0.5
    assert np.abs(got - want).max() < 2e-3 * np.abs(want).max() + 1e-4


@pytest.mark.parametrize("H,D,V,rot", [(3, 20, 12, 12), (1, 8, 5, 8), (2, 64, 64, 0), (2, 192, 80, 64), (4, 128, 130, 128), (1, 256, 16, 2)])
def test_retention(hip, H, D, V, rot):
    note(f"retention H {H} D {D} V {V} rot {rot}")
    rng = np.random.default_rng(D + V)
    rows, xs = 40, H * (2 * D + V) + 7
    state = H * D * V + 3
    xo, oo = 2, 2 + rows * xs
    fr = oo + rows * H * V
    p = Pair(hip, fr + rot // 2 + H + 4, state=3 * state)
    p.put(ST, 0, np.full(3 * state, -3.0))
    p.put(WS, fr, 3000.0 ** (-2.0 * np.arange(rot // 2) / max(rot, 1)))
    p.put(WS, fr + rot // 2, 1.0 - 2.0 ** -np.linspace(1, 10, H))
    spec = p.up(A.RetentionSpec(heads=H, dim=D, vdim=V, rot_dims=rot, freq=fr, decay=fr + rot // 2, x=xo, x_stride=xs, x_q=1, x_k=1 + H * D,
                                x_v=1 + 2 * H * D, out=oo, out_stride=H * V, state_map=ST, s_off=2, seq_stride=state).words())

    def run(n_seq, m, seq0, pos):
        p.put(WS, xo, rng.standard_normal((n_seq * m, xs)))
        p.call("retention_dev", WS, spec, n_seq, m, seq0, pos)
        p.same(WS, oo, n_seq * m * H * V, 5e-5, f"outputs {n_seq}x{m} at {pos}")
        p.same(ST, seq0 * state + 2, H * D * V, 5e-5, f"state after {pos + m}")
    pos = 0
    for m in (1, 2, 16, 1, 33, 15, 40):
        run(1, m, 1, pos)
        pos += m
    run(1, 7, 1, 0)
    for i in (0, 2):
        run(1, 7, i, 0)
    run(3, 1, 0, 7)


# ---- attention -------------------------------------------------------------------------------------------------------
def attention_pair(hip, H, G, D, V, C, dtype, rows, seqs, seed, scale=0.25):
    rng = np.random.default_rng(seed)
    r8 = lambda n: (n + 7) // 8 * 8
    xs = H * D + G * (D + V) + 3
    oo = 4 + rows * xs
    ro = oo + rows * H * V
    kc, vc = G * C * r8(D), G * C * r8(V)
    p = Pair(hip, ro + 2 * H + 4, cache=seqs * (kc + vc + 8), dtype=dtype)
    p.put(WS, ro, np.concatenate([np.linspace(0.02, 1.5, H), rng.uniform(0.05, 0.6, H)]))
    spec = p.up(A.ChunkAttnSpec(heads=H, kv_heads=G, dim=D, vdim=V, chunk=C, x=4, x_stride=xs, x_q=1, x_k=1 + H * D, x_v=1 + (H + G) * D,
                                r1=ro, r2=ro + H, scale=scale, eps=1e-4, out=oo, out_stride=H * V, cache_map=CA, k_off=0, v_off=kc,
                                seq_stride=kc + vc + 8).words())
    tol = 3e-5 if dtype == "float32" else 2e-2

    def run(n_seq, m, seq0, pos, x=None):
        x = rng.standard_normal((n_seq * m, xs)) if x is None else x
        p.put(WS, 4, x)
        p.call("chunk_attention_dev", WS, spec, n_seq, m, seq0, pos)
        p.same(WS, oo, n_seq * m * H * V, tol, f"{n_seq}x{m} at {pos}")
        return p.read(WS, oo, n_seq * m * H * V)[0].reshape(n_seq * m, H, V)
    return run, xs, rng


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,V,C", [(4, 2, 16, 24, 10), (3, 3, 33, 7, 16), (1, 1, 1, 1, 1), (4, 1, 64, 48, 37), (2, 1, 136, 128, 70),
                                       (2, 2, 160, 200, 5), (2, 1, 256, 256, 100), (6, 3, 8, 80, 1000)])
def test_chunk_attention(hip, H, G, D, V, C, dtype):
    note(f"chunk attention H {H} G {G} D {D} V {V} chunk {C} {dtype}")
    run, _, _ = attention_pair(hip, H, G, D, V, C, dtype, 100, 3, seed=D + C)
    pos = 0
    for m in (2, 1, 3, 64, 1, 1, 100, 7, 33, 1):      # through chunk edges in portions and alone
        run(1, m, 1, pos)
        pos += m
    run(1, 13, 1, 0)                                  # the slot again
    for i in (0, 2):
        run(1, 13, i, 0)
    for t in range(4):
        run(3, 1, 0, 13 + t)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_chunk_attention_over_several_spans_of_keys(hip, dtype):
    """A chunk of 1500 tokens: a decoded token reads its keys in three spans; the edge to the next chunk comes after."""
    note(f"chunk attention, long chunk {dtype}")
    C = 1500
    run, _, _ = attention_pair(hip, 4, 2, 32, 40, C, dtype, 300, 1, seed=5, scale=0.6)
    pos = 0
    while pos < 1491:
        m = min(300, 1491 - pos)
        run(1, m, 0, pos)
        pos += m
        if pos in (300, 600, 1200):
            run(1, 1, 0, pos)
            pos += 1
    for pos in range(1491, 1504):
        run(1, 1, 0, pos)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cut", ["whole", "pairs", "alone"])
def test_a_standing_out_key_is_seen_inside_its_chunk_only(hip, dtype, cut):
    """Token j's key and token i's query are made to match strongly: i takes j's value when both lie in one chunk, and
    nothing of it when j is the last token ahead of i's chunk."""
    C, H, D, V = 12, 2, 16, 8
    note(f"standing-out key {dtype} {cut}")
    for j, i, seen in ((0, 11, True), (12, 23, True), (12, 12, True), (11, 12, False), (23, 24, False), (24, 30, True), (22, 24, False)):
        run, xs, rng = attention_pair(hip, H, H, D, V, C, dtype, 36, 1, seed=9, scale=1.0)
        x = rng.standard_normal((36, xs)) * 0.1
        v = rng.standard_normal((36, H, V))
        x[:, 1 + 2 * H * D:1 + 2 * H * D + H * V] = v.reshape(36, -1)
        x[i, 1:1 + H * D] = x[j, 1 + H * D:1 + 2 * H * D] = np.tile(np.eye(D)[3] * 6.0, H)
        step = {"whole": 36, "pairs": 2, "alone": 1}[cut]
        out = np.concatenate([run(1, step, 0, lo, x[lo:lo + step]) for lo in range(0, 36, step)])
        vn = v[j] / np.sqrt(np.mean(v[j] ** 2, axis=-1, keepdims=True) + 1e-4)
        assert (np.abs(out[i] - vn).max() < 0.05) == seen, (j, i)


# ---- models ----------------------------------------------------------------------------------------------------------
def tokens(cfg, n, seed=1):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def engine(hip, cfg, W, dtype="float32", **kw):
    return MixerEngine(hip, vomotar_config(cfg), W, A=A, dtype=dtype, **kw)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_model_whole_in_portions_and_token_by_token(hip, name, dtype):
    cfg = CONFIGS[name]
    W, n = weights(cfg, seed=2), 90
    toks = tokens(cfg, n)
    want = M.forward(cfg, floats(W), toks)
    for chunk in (256, 17, 1):
        note(f"model {name} {dtype} portions of {chunk}")
        eng = engine(hip, cfg, W, dtype, prefill_chunk=chunk)
        assert rel(eng.score("a", toks, range(n)), want) < TOL[dtype], chunk
    note(f"model {name} {dtype} uneven portions, slots freed and used again")
    eng = engine(hip, cfg, W, dtype, prefill_chunk=64, batch=2)
    rng = np.random.default_rng(4)
    for r in range(3):
        seq = {f"{r}{s}": tokens(cfg, 60, seed=30 + 2 * r + s) for s in range(2)}
        ref = {s: M.forward(cfg, floats(W), t) for s, t in seq.items()}
        at = dict.fromkeys(seq, 0)
        while any(a < 60 for a in at.values()):
            s = rng.choice([s for s in seq if at[s] < 60])
            m = int(min(rng.choice([1, 2, 3, 16, 25]), 60 - at[s]))
            assert rel(eng.score(s, seq[s][at[s]:at[s] + m], range(m)), ref[s][at[s]:at[s] + m]) < TOL[dtype], (r, s, at)
            at[s] += m
        for s in seq:
            eng.release(s)


def test_residual_after_every_layer(hip):
    """Each prefix of the stack as a model of its own: the residual rows after its last layer."""
    cfg = CONFIGS["odd"]
    W, toks = weights(cfg, seed=8), tokens(CONFIGS["odd"], 30)
    per_layer = []
    M.forward(cfg, floats(W), toks, per_layer)
    for n in range(1, len(cfg["layers"]) + 1):
        note(f"residual after {n} layers")
        eng = engine(hip, {**cfg, "layers": cfg["layers"][:n]}, W, prefill_chunk=30)
        eng.score("a", toks)
        assert rel(eng.read_rows("hidden", 30, cfg["width"]), per_layer[n - 1]) < 1e-5


@pytest.mark.parametrize("plan", [True, False])
def test_long_decoding_across_many_chunk_edges(hip, plan):
    cfg = config([delta(), par(size=7), par(size=50)], width=40, groups=2, vocab=64)
    W, toks = weights(cfg, seed=12), tokens(config([delta()], vocab=64), 400)
    note(f"long decoding plan={plan}")
    want = M.forward(cfg, floats(W), toks)
    eng = engine(hip, cfg, W, prefill_chunk=64, decode_plan=plan)
    got = [eng.score("a", toks[:5], range(5))] + [eng.score("a", [t], [0]) for t in toks[5:]]
    assert rel(np.concatenate(got), want) < 5e-5


def test_generation(hip):
    """Greedy tokens of the framework's loop, one step ahead of the read-back, equal those of the plain model; so do
    lockstep sequences; a prefix the state holds is reused."""
    cfg = CONFIGS["odd"]
    W, prompt = weights(cfg, seed=4), tokens(CONFIGS["odd"], 11)
    toks = list(prompt)
    for _ in range(40):
        toks.append(int(np.argmax(M.forward(cfg, floats(W), toks)[-1])))
    note("greedy generation")
    for kw in (dict(), dict(lookahead=False), dict(decode_plan=False), dict(sampling_mode="gpu_argmax")):
        eng = engine(hip, cfg, W, prefill_chunk=8, **kw)
        out, stats = eng.generate(prompt, GenerationConfig(max_tokens=40))
        assert out == toks[11:], kw
    assert stats["sampling_mode"] == "gpu_argmax"
    eng = engine(hip, cfg, W, prefill_chunk=8)
    eng.generate(prompt, GenerationConfig(max_tokens=40))
    follow = toks + tokens(cfg, 4, seed=8)
    more, st = eng.generate(follow, GenerationConfig(max_tokens=5), reuse_prefix=51)
    assert st["n_prompt_reused"] == 51
    assert more == engine(hip, cfg, W, prefill_chunk=8).generate(follow, GenerationConfig(max_tokens=5))[0]
    note("stop token")
    out, _ = eng.generate(prompt, GenerationConfig(max_tokens=40, eos_token_ids=(toks[20],)))
    assert out == toks[11:11 + toks[11:].index(toks[20])]
    note("lockstep")
    prompts = [tokens(cfg, 9, seed=20 + i) for i in range(4)]
    alone = [engine(hip, cfg, W, prefill_chunk=8).generate(p, GenerationConfig(max_tokens=30))[0] for p in prompts]
    out, _ = engine(hip, cfg, W, prefill_chunk=8, batch=4).generate_batch(prompts, 30)
    assert out == alone
    note("sampling")
    for kw in (dict(temperature=0.8, top_k=8, top_p=0.9, repeat_penalty=1.2, seed=3), dict(temperature=0.7, top_k=0, seed=3)):
        ref = MixerEngine(oracle.init(), vomotar_config(cfg), W, A=A, dtype="float32", prefill_chunk=8)
        want, _ = ref.generate(prompt, GenerationConfig(max_tokens=12, **kw))
        assert engine(hip, cfg, W, prefill_chunk=8).generate(prompt, GenerationConfig(max_tokens=12, **kw))[0] == want


def test_trace_replay_and_command_line(hip, tmp_path):
    """The programs, each in a process of its own, on a model folder."""
    cfg = CONFIGS["odd"]
    W, toks = weights(cfg, seed=5), tokens(CONFIGS["odd"], 50)
    write_model(tmp_path, cfg, W)
    want = M.forward(cfg, floats(W), toks)
    steps = [([0, 33], [32, 4]), ([33, 35], []), ([35, 36], [0]), ([36, 50], [13])]
    lines = [json.dumps({"step": i, "entries": [{"id": "q", "tokens": toks[a:b], "want": w}], "end": ["q"] if b == 50 else []})
             for i, ((a, b), w) in enumerate(steps)]
    for dtype in ("bfloat16", "float32"):
        note(f"trace_run {dtype}")
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(tmp_path),
                            "--max-tokens", "64"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=90)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
        assert not os.path.exists(tmp_path / "1.f32")
        for i, ((a, b), w) in enumerate(steps):
            if w:
                got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(len(w), -1)
                assert rel(got, want[[a + k for k in w]]) < TOL[dtype]
    note("python -m adam_amd")
    r = subprocess.run([sys.executable, "-m", "adam_amd", str(tmp_path), "--tokens", ",".join(map(str, toks[:9])), "--max-tokens", "6",
                        "--dtype", "float32"], capture_output=True, text=True, timeout=90, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    seq = list(toks[:9])
    for _ in range(6):
        seq.append(int(np.argmax(M.forward(cfg, floats(W), seq)[-1])))
    assert json.loads(r.stdout.splitlines()[-1])["tokens"] == seq[9:]


def test_calls_with_impossible_operands_are_refused(hip):
    """Ranges and sizes are checked on the host before anything is launched."""
    note("refused calls")
    eng = engine(hip, CONFIGS["ones"], weights(CONFIGS["ones"]))
    up = lambda s: hip.upload_dev(s.words())[0]
    mid, off, n, k, stride = eng._stacks[('head',)]
    good = dict(w=off, n=n, k=k, k_stride=stride, src=0, src_stride=k, out=0, out_stride=n)
    for bad in (dict(w=1 << 30), dict(k_stride=stride + 8), dict(groups=2), dict(epi=2), dict(out=(1 << 32) - 2), dict(n=0)):
        with pytest.raises(RuntimeError, match="-3"):
            hip.linear_dev(0, 2, mid, up(A.LinearSpec(**{**good, **bad})), 0, 1)
    with pytest.raises(RuntimeError, match="-3"):
        hip.linear_dev(0, 2, mid, hip.upload_dev(np.zeros(4, np.uint32))[0], 0, 1)       # not a spec
    r = dict(heads=1, dim=8, vdim=8, rot_dims=8, freq=0, decay=0, x=0, x_stride=32, x_q=0, x_k=8, x_v=16, out=0, out_stride=8, state_map=3,
             s_off=0, seq_stride=64)
    for bad in (dict(dim=300), dict(rot_dims=9), dict(seq_stride=63), dict(x_v=30), dict(state_map=9)):
        with pytest.raises(RuntimeError, match="-3"):
            hip.retention_dev(0, up(A.RetentionSpec(**{**r, **bad})), 1, 1, 0, 0)
