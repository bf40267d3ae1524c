"""Zaparax models on the GPU: every op against the NumPy op surface, whole models against the plain statement of the
mechanisms, in one piece, in portions, token by token, in lockstep, and through generation and trace replay."""
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
from adam_amd.models import zaparax_config
from adam_amd.safetensors_file import f32_to_bf16
from gpu_util import note
from mixer_cases import floats, rel, write_model
from mixer_pair import CA, OP, ST, WS, WT, Pair
from oracle import zaparax_np as Z
from zaparax_cases import CONFIGS, att, config, moe, ssm, weights

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": 5e-5, "bfloat16": 6e-2}
r8 = lambda n: (n + 7) // 8 * 8
r64 = lambda n: (n + 63) // 64 * 64


# ---- products ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rows,n,k,tail", [(1, 65, 33, 1), (1, 64, 4100, 0), (1, 83, 9000, 19), (2, 64, 200, 0), (5, 101, 96, 37),
                                           (33, 97, 130, 33), (64, 192, 256, 64), (200, 331, 192, 11)])
def test_linear_with_a_branch_added_kept_rows_and_a_tail(hip, dtype, rows, n, k, tail):
    """Rows = src + norm(branch): their norm is the operand, the sum and the operand are stored; gate and up pairs, then a tail."""
    note(f"linear branched {dtype} rows {rows} n {n} k {k} tail {tail}")
    rng = np.random.default_rng(n + k)
    ks, pairs, src_rows = r64(k), (n - tail) // 2, rows + 2
    at, pos = {}, 3
    for name, sz in (("src", src_rows * k), ("br", src_rows * (k + 1)), ("wt", k), ("bw", k), ("res", src_rows * (k + 2)),
                     ("keep", src_rows * (k + 4)), ("out", rows * (pairs + 1)), ("tail", rows * (tail + 2))):
        at[name] = pos
        pos += sz
    oo = rows * ks
    p = Pair(hip, pos + 8, wt=n * ks + 8, opnd=oo + rows * r64(pairs), dtype=dtype)
    W = np.zeros((n, ks), np.uint16)
    W[:, :k] = f32_to_bf16((rng.standard_normal((n, k)) / np.sqrt(k)).astype(np.float32))
    p.put(WT, 8, W)
    p.put(WS, 0, rng.standard_normal(pos))
    spec = A.LinearSpec(w=8, n=n, k=k, k_stride=ks, src=at["src"], src_stride=k, groups=1, eps=1e-4, wt=at["wt"], wt_len=k, wt_add=1.0,
                        branch=at["br"], branch_stride=k + 1, branch_wt=at["bw"], branched=2, res_out=at["res"], res_stride=k + 2,
                        keep=at["keep"], keep_stride=k + 4, kept=1, out=at["out"], out_stride=pairs + 1, epi=2, out_opnd=oo,
                        out_opnd_stride=r64(pairs), tail=tail, tail_out=at["tail"], tail_stride=tail + 2)
    pick = p.up(rng.permutation(src_rows)[:rows])
    p.call("linear_dev", WS, OP, WT, p.up(spec.words()), pick, rows)
    tol = 3e-5 if dtype == "float32" or rows == 1 else 4e-2
    p.same(WS, at["res"], src_rows * (k + 2), 2e-5, "sum")
    p.same(WS, at["keep"], src_rows * (k + 4), 2e-5, "operand")
    p.same(WS, at["tail"], rows * (tail + 2), tol, "tail")
    if rows == 1:
        p.same(WS, at["out"], pairs, tol, "pairs")
    else:
        w2 = r64(pairs)
        eye = np.zeros((pairs, w2), np.float32)
        eye[np.arange(pairs), np.arange(pairs)] = 1
        for g in p.g:
            g.map_create_typed(WT, A.DTYPE_BF16, 1, eye.size)
        p.put(WT, 0, f32_to_bf16(eye))
        p.call("linear_dev", WS, OP, WT, p.up(A.LinearSpec(w=0, n=pairs, k=pairs, k_stride=w2, opnd=oo, ready=1, out=at["out"],
                                                           out_stride=pairs + 1).words()), 0, rows)
        p.same(WS, at["out"], rows * (pairs + 1) - 1, tol, "pairs")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rows,n,k,groups,epi", [(1, 51, 330, 3, 0), (1, 64, 1100, 10, 1), (3, 70, 64, 2, 0), (40, 129, 96, 1, 1),
                                                 (130, 200, 256, 16, 0)])
def test_linear_with_a_bias_and_a_gate_ahead_of_the_norm(hip, dtype, rows, n, k, groups, epi):
    note(f"linear gated ahead {dtype} rows {rows} n {n} k {k} groups {groups} epi {epi}")
    rng = np.random.default_rng(n)
    ks = r64(k)
    gate, wt, bias = rows * k, 2 * rows * k, 2 * rows * k + k
    out = bias + n
    p = Pair(hip, out + rows * (n + 1), wt=n * ks, opnd=rows * ks, dtype=dtype)
    W = np.zeros((n, ks), np.uint16)
    W[:, :k] = f32_to_bf16((rng.standard_normal((n, k)) / np.sqrt(k)).astype(np.float32))
    p.put(WT, 0, W)
    p.put(WS, 0, rng.standard_normal(p.n))
    spec = A.LinearSpec(w=0, n=n, k=k, k_stride=ks, src=0, src_stride=k, groups=groups, eps=1e-4, wt=wt, wt_len=k, gate=gate, gate_stride=k,
                        gate_act=A.GATE_SILU_AHEAD, bias=bias, biased=1, out=out, out_stride=n + 1, epi=epi)
    p.call("linear_dev", WS, OP, WT, p.up(spec.words()), 0, rows)
    p.same(WS, out, rows * (n + 1) - 1, 3e-5 if dtype == "float32" or rows == 1 else 4e-2, "out")


# ---- embedding -----------------------------------------------------------------------------------------------------------
def test_bigram_embedding_keeps_each_sequences_last_token(hip):
    note("bigram embedding")
    V, E, Bk, rows, seqs, stride = 50, 37, 23, 20, 3, 9
    rng = np.random.default_rng(0)
    p = Pair(hip, rows * E + rows + 4, wt=(V + Bk + 1) * E + 3, state=seqs * stride)
    p.put(WT, 0, f32_to_bf16(rng.standard_normal((V + Bk + 1) * E + 3).astype(np.float32)))
    p.put(ST, 0, np.full(seqs * stride, 77.0))
    spec = p.up(A.BigramSpec(table=3, vocab=V, width=E, dst=2, scale=2.5, pairs=3 + V * E, buckets=Bk, mul_prev=4000000007, mul_cur=3999999979,
                             state_map=ST, prev_off=4, seq_stride=stride).words())
    locs = p.up(2 + rows * E + np.arange(rows))

    def run(n_seq, m, seq0, pos):
        p.put(WS, 2 + rows * E, rng.integers(0, V, n_seq * m))
        p.call("embed_bigram_dev", WS, WT, spec, locs, n_seq, m, seq0, pos)
        p.same(WS, 2, n_seq * m * E, 1e-6, f"rows {n_seq}x{m} at {pos}")
        p.same(ST, 0, seqs * stride, 1e-9, "last tokens")
    pos = 0
    for m in (2, 1, 1, 20, 7, 1):
        run(1, m, 1, pos)
        pos += m
    run(1, 1, 1, 0)
    for i in (0, 2):
        run(1, 1, i, 0)
    for t in range(3):
        run(3, 1, 0, 1 + t)


# ---- state space ---------------------------------------------------------------------------------------------------------
def space_pair(hip, H, G, N, V, taps, rows, seqs, strong, seed):
    rng = np.random.default_rng(seed)
    ch = H * V + 2 * G * N
    xs = H * V + ch + H + 3
    at, pos = {}, 5
    for n, sz in (("x", rows * xs), ("o", rows * (H * V + 1)), ("w", ch * taps), ("b", ch), ("dt", H), ("A", H), ("D", H)):
        at[n] = pos
        pos += sz
    state = H * N * V + taps * ch + 3
    p = Pair(hip, pos + 8, state=seqs * state)
    p.put(WS, at["w"], rng.standard_normal(ch * taps) * 0.7)
    p.put(WS, at["b"], rng.standard_normal(ch) * 0.5)
    p.put(WS, at["dt"], rng.uniform(-4, 3 if strong else 0, H))
    p.put(WS, at["A"], np.linspace(-4, 6.0 if strong else 0.5, H))
    p.put(WS, at["D"], rng.standard_normal(H))
    p.put(ST, 0, np.full(seqs * state, 7.0))             # what another sequence left behind
    spec = p.up(A.StateSpaceSpec(heads=H, groups=G, state=N, vdim=V, taps=taps, x=at["x"], x_stride=xs, x_c=H * V, x_dt=H * V + ch,
                                 conv=at["w"], conv_b=at["b"], dt_bias=at["dt"], a_log=at["A"], skip=at["D"], out=at["o"],
                                 out_stride=H * V + 1, state_map=ST, s_off=1, conv_off=1 + H * N * V, seq_stride=state).words())

    def run(n_seq, m, seq0, pos, x=None):
        p.put(WS, at["x"], rng.standard_normal((n_seq * m, xs)) if x is None else x)
        p.call("state_space_dev", WS, spec, n_seq, m, seq0, pos)
        p.same(WS, at["o"], n_seq * m * (H * V + 1) - 1, 3e-5, f"outputs {n_seq}x{m} at {pos}")
        p.same(ST, seq0 * state + 1, H * N * V, 5e-5, f"state after {pos + m}")
        return p.read(WS, at["o"], n_seq * m * (H * V + 1))[0].reshape(n_seq * m, -1)[:, :H * V].reshape(n_seq * m, H, V)
    return run, xs


@pytest.mark.parametrize("H,G,N,V,taps,strong", [(6, 3, 10, 7, 3, False), (1, 1, 1, 1, 1, True), (4, 1, 64, 33, 4, True), (4, 4, 100, 64, 2, False),
                                                 (2, 1, 144, 48, 5, False), (3, 1, 200, 130, 16, True), (2, 2, 256, 256, 4, False)])
def test_state_space(hip, H, G, N, V, taps, strong):
    note(f"state space H {H} G {G} N {N} V {V} taps {taps}")
    run, _ = space_pair(hip, H, G, N, V, taps, 40, 3, strong, seed=N)
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


def test_state_space_keeps_an_input_over_a_long_gap(hip):
    """Steps close to zero leave the state alone: what the first token wrote is read 300 tokens later."""
    note("state space, long gap")
    H, N, V, m = 2, 8, 4, 301
    run, xs = space_pair(hip, H, 1, N, V, 1, m, 1, False, seed=1)
    x = np.zeros((m, xs))
    x[:, -(H + 3):-3] = -60.0
    x[0, -(H + 3):-3] = 3.0
    x[0, H * V:] += np.where(np.arange(xs - H * V) < H * V + 2 * N, 2.0, 0.0)
    x[-1, 2 * H * V + N:2 * H * V + 2 * N] = 2.0
    out = run(1, m, 0, 0, x)
    assert np.abs(out[-1]).max() > 0.1               # (values against the NumPy surface: inside run)


# ---- window attention ----------------------------------------------------------------------------------------------------
def window_pair(hip, H, G, D, V, R, dtype, rows, seqs, seed, scale=0.25, cap=4.0, coef=0.5, every=5, sink=True, norm=True, slope=None):
    rng = np.random.default_rng(seed)
    xs = H * D + G * (D + V) + 3
    oo = 4 + rows * xs
    so = oo + rows * H * V
    kc, vc = G * R * r8(D), G * R * r8(V)
    p = Pair(hip, so + 2 * H + 4, cache=seqs * (kc + vc + 8), dtype=dtype)
    p.put(WS, so, 2.0 ** (-8.0 * np.arange(1, H + 1) / H) if slope is None else np.full(H, slope))
    p.put(WS, so + H, np.linspace(-1.0, 2.5, H))
    spec = p.up(A.WindowAttnSpec(heads=H, kv_heads=G, dim=D, vdim=V, window=R, x=4, x_stride=xs, x_q=1, x_k=1 + H * D, x_v=1 + (H + G) * D,
                                 slope=so, sink=so + H, has_sink=int(sink), qk_norm=int(norm), scale=scale, eps=1e-4, softcap=cap,
                                 temp_coef=coef, temp_every=every, out=oo, out_stride=H * V, cache_map=CA, k_off=0, v_off=kc,
                                 seq_stride=kc + vc + 8).words())
    tol = 3e-5 if dtype == "float32" else 2e-2

    def run(n_seq, m, seq0, pos, x=None):
        p.put(WS, 4, rng.standard_normal((n_seq * m, xs)) if x is None else x)
        p.call("window_attention_dev", WS, spec, n_seq, m, seq0, pos)
        p.same(WS, oo, n_seq * m * H * V, tol, f"{n_seq}x{m} at {pos}")
        return p.read(WS, oo, n_seq * m * H * V)[0].reshape(n_seq * m, H, V)
    return run, xs, rng


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,V,R", [(4, 2, 16, 24, 10), (3, 3, 33, 7, 16), (1, 1, 1, 1, 1), (5, 1, 64, 48, 37), (10, 2, 136, 128, 70),
                                       (2, 2, 160, 200, 5), (2, 1, 256, 256, 100), (6, 3, 8, 80, 1000)])
def test_window_attention(hip, H, G, D, V, R, dtype):
    note(f"window attention H {H} G {G} D {D} V {V} window {R} {dtype}")
    run, _, _ = window_pair(hip, H, G, D, V, R, dtype, 100, 3, seed=D + R, scale=1.0)
    pos = 0
    for m in (2, 1, 3, 64, 1, 1, 100, 7, 33, 1):      # portions and single tokens in turn
        run(1, m, 1, pos)
        pos += m
    run(1, 13, 1, 0)                                  # the slot again
    for i in (0, 2):
        run(1, 13, i, 0)
    for t in range(4):
        run(3, 1, 0, 13 + t)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kw", [dict(cap=0.0), dict(sink=False), dict(norm=False), dict(coef=0.0), dict(cap=30.0, scale=3.0, coef=1.0, every=3),
                                dict(cap=0.0, sink=False, norm=False, coef=0.0)])
def test_window_attention_with_parts_left_out(hip, dtype, kw):
    note(f"window attention {kw} {dtype}")
    run, _, _ = window_pair(hip, 6, 2, 24, 40, 21, dtype, 50, 1, seed=3, **kw)
    pos = 0
    for m in (50, 1, 2, 1, 30):
        run(1, m, 0, pos)
        pos += m


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,V,R,total,ones", [(4, 2, 32, 40, 1500, 1900, (300, 1200, 1502)), (64, 64, 8, 8, 700, 950, (300, 601))])
def test_window_attention_over_several_spans_of_keys(hip, H, G, D, V, R, total, ones, dtype):
    """A wide window: a decoded token reads its keys in spans, the ring turns over inside one of them; with many key heads the
    spans grow past what a workgroup takes at once."""
    note(f"window attention, wide window, H {H} {dtype}")
    run, _, _ = window_pair(hip, H, G, D, V, R, dtype, 300, 1, seed=5, scale=0.6, slope=0.003)
    pos = 0
    while pos < total:
        m = min(300, total - pos)
        run(1, m, 0, pos)
        pos += m
        if pos in ones:
            run(1, 1, 0, pos)
            pos += 1
    for pos in range(pos, pos + 4):
        run(1, 1, 0, pos)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cut", ["whole", "pairs", "alone"])
def test_a_standing_out_key_is_seen_inside_the_window_only(hip, dtype, cut):
    """Token j's key and token i's query match strongly: i takes j's value when j is the oldest token of its window, and
    nothing of it when j is one token further back."""
    R, H, D, V = 12, 2, 16, 8
    note(f"standing-out key {dtype} {cut}")
    for j, i, seen in ((0, 11, True), (0, 12, False), (1, 12, True), (9, 20, True), (9, 21, False), (24, 35, True), (23, 35, False), (35, 35, True)):
        run, xs, rng = window_pair(hip, H, H, D, V, R, dtype, 36, 1, seed=9, scale=2.0, cap=60.0, coef=0.0, slope=0.01)
        x = rng.standard_normal((36, xs)) * 0.1
        x[:, 1:1 + 2 * H * D] = np.where(np.arange(2 * H * D) % D < 8, 1.0, 0.0) + 0.01 * rng.standard_normal((36, 2 * H * D))
        x[:, 1 + H * D:1 + 2 * H * D] *= -1.0                              # keys away from every query ...
        v = rng.standard_normal((36, H, V))
        x[:, 1 + 2 * H * D:1 + 2 * H * D + H * V] = v.reshape(36, -1)
        x[i, 1:1 + H * D] = x[j, 1 + H * D:1 + 2 * H * D] = np.tile(np.where(np.arange(D) >= 8, 1.0, 0.0), H)   # ... but these two
        step = {"whole": 36, "pairs": 2, "alone": 1}[cut]
        out = np.concatenate([run(1, step, 0, lo, x[lo:lo + step]) for lo in range(0, 36, step)])
        assert (np.abs(out[i] - v[j]).max() < 0.05) == seen, (j, i)


# ---- experts -------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("E,I,top,ff,shared,width,epi", [(5, 2, 3, 20, 28, 60, 0), (1, 0, 1, 16, 0, 33, 1), (70, 9, 11, 40, 72, 192, 0),
                                                         (3, 4, 7, 130, 24, 100, 1), (300, 20, 2, 33, 16, 64, 0), (6, 1, 2, 600, 900, 1040, 0)])
def test_experts(hip, E, I, top, ff, shared, width, epi, dtype):
    note(f"experts {E} + {I} top {top} ff {ff} shared {shared} width {width} {dtype}")
    rng = np.random.default_rng(E + ff)
    n, ks, F, F16, S, S16 = E + I, r64(width), r64(ff), (ff + 15) // 16 * 16, r64(shared), (shared + 15) // 16 * 16
    most = 300
    at, pos = {}, 3
    for name, sz in (("h", most * width), ("log", most * (n + 1)), ("corr", n), ("out", most * width), ("act", top * F), ("sact", max(S16, 1)),
                     ("sout", most * width)):
        at[name] = pos
        pos += sz
    op = {"h": 0, "act": most * ks, "sact": most * (ks + top * F)}
    gu, dn = 0, E * 2 * F16 * ks
    sd = dn + E * width * F
    p = Pair(hip, pos + 8, wt=sd + width * S + 8, opnd=op["sact"] + most * S + 8, dtype=dtype)
    W = np.zeros((E, 2 * F16, ks), np.float32)
    for e in range(E):
        w = W[e].reshape(-1, 2, 16, ks)
        for s in range(2):
            m = np.zeros((F16, ks), np.float32)
            m[:ff, :width] = rng.standard_normal((ff, width)) / np.sqrt(width)
            w[:, s] = m.reshape(-1, 16, ks)
    p.put(WT, gu, f32_to_bf16(W))
    W = np.zeros((E * width, F), np.float32)
    W[:, :ff] = rng.standard_normal((E * width, ff)) / np.sqrt(ff)
    p.put(WT, dn, f32_to_bf16(W))
    if shared:
        W = np.zeros((width, S), np.float32)
        W[:, :shared] = rng.standard_normal((width, shared)) / np.sqrt(shared)
        p.put(WT, sd, f32_to_bf16(W))
    p.put(WS, at["corr"], rng.uniform(-0.2, 0.2, n))
    spec = p.up(A.ExpertsSpec(experts=E, identity=I, top=top, ff=ff, ff_stride=F, width=width, k_stride=ks, gate_up=gu, gate_up_step=2 * F16 * ks,
                              down=dn, down_step=width * F, logits=at["log"], logits_stride=n + 1, correction=at["corr"], x=at["h"],
                              x_stride=width, opnd=op["h"], act=at["act"], act_opnd=op["act"], shared_ff=shared, shared_ff_stride=S,
                              shared_down=sd, shared_act=at["sact"], out=at["out"], out_stride=width, epi=epi).words())
    sh = p.up(A.LinearSpec(w=sd, n=width, k=max(shared, 1), k_stride=max(S, 64), src=at["sact"], src_stride=S16, opnd=op["sact"], ready=1,
                           out=at["sout"], out_stride=width).words()) if shared else 0
    for rows in (1, 2, 33, most, 1, 5):
        h = rng.standard_normal((rows, width))
        p.put(WS, at["h"], h)
        p.put(WS, at["log"], rng.standard_normal((rows, n + 1)) * 2.0)
        p.put(WS, at["sact"], rng.standard_normal(max(S16, 1)))
        p.put(WS, at["out"], rng.standard_normal((rows, width)))
        if rows > 1:
            to = f32_to_bf16 if dtype == "bfloat16" else (lambda v: v)
            p.put(OP, op["h"], to(np.pad(h, ((0, 0), (0, ks - width))).astype(np.float32)))
            if shared:
                p.put(OP, op["sact"], to(np.pad(rng.standard_normal((rows, shared)), ((0, 0), (0, S - shared))).astype(np.float32)))
        p.call("experts_dev", WS, OP, WT, spec, sh, rows)
        p.same(WS, at["out"], rows * width, 5e-5 if dtype == "float32" or rows == 1 else 4e-2, f"rows {rows}")


def test_experts_with_equal_scores_take_the_first(hip):
    note("experts, equal scores")
    E, w = 6, 32
    p = Pair(hip, 2000, wt=E * (32 * 64 + w * 64), opnd=4 * 64 + 4 * 3 * 64 + 64)
    rng = np.random.default_rng(0)
    W1, W2 = np.zeros((E * 32, 64), np.float32), np.zeros((E * w, 64), np.float32)
    W1[:, :w], W2[:, :16] = rng.standard_normal((E * 32, w)), rng.standard_normal((E * w, 16))
    p.put(WT, 0, f32_to_bf16(W1))
    p.put(WT, E * 32 * 64, f32_to_bf16(W2))
    spec = p.up(A.ExpertsSpec(experts=E, top=3, ff=16, ff_stride=64, width=w, k_stride=64, gate_up_step=32 * 64, down=E * 32 * 64,
                              down_step=w * 64, logits=0, logits_stride=8, correction=64, x=100, x_stride=w, act=400, act_opnd=256, out=800,
                              out_stride=w).words())
    p.put(WS, 64, [0.0, 0.5, 0.0, 0.5, 0.5, 0.5])
    for rows in (1, 4):
        h = rng.standard_normal((rows, w))
        p.put(WS, 100, h)
        p.put(OP, 0, np.pad(h, ((0, 0), (0, 32))))
        p.call("experts_dev", WS, OP, WT, spec, 0, rows)
        p.same(WS, 800, rows * w, 2e-5, f"rows {rows}")


# ---- models --------------------------------------------------------------------------------------------------------------
def tokens(cfg, n, seed=1):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def engine(hip, cfg, W, dtype="float32", **kw):
    return MixerEngine(hip, zaparax_config(cfg), W, A=A, dtype=dtype, **kw)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_model_whole_in_portions_and_token_by_token(hip, name, dtype):
    cfg = CONFIGS[name]
    W, n = weights(cfg, seed=2, steady=dtype == "bfloat16"), 90
    toks = tokens(cfg, n)
    want = Z.forward(cfg, floats(W), toks)
    for chunk in (256, 17, 2, 1):
        note(f"model {name} {dtype} portions of {chunk}")
        eng = engine(hip, cfg, W, dtype, prefill_chunk=chunk)
        assert rel(eng.score("a", toks, range(n)), want) < TOL[dtype], chunk
    note(f"model {name} {dtype} uneven portions, slots freed and used again")
    eng = engine(hip, cfg, W, dtype, prefill_chunk=64, batch=2)
    rng = np.random.default_rng(4)
    for r in range(3):
        seq = {f"{r}{s}": tokens(cfg, 60, seed=30 + 2 * r + s) for s in range(2)}
        ref = {s: Z.forward(cfg, floats(W), t) for s, t in seq.items()}
        at = dict.fromkeys(seq, 0)
        while any(a < 60 for a in at.values()):
            s = rng.choice([s for s in seq if at[s] < 60])
            m = int(min(rng.choice([1, 2, 3, 16, 25]), 60 - at[s]))
            assert rel(eng.score(s, seq[s][at[s]:at[s] + m], range(m)), ref[s][at[s]:at[s] + m]) < TOL[dtype], (r, s, at)
            at[s] += m
        for s in seq:
            eng.release(s)


def test_residual_after_every_layer(hip):
    """Each prefix of the stack as a model of its own: the residual rows with its last sublayer's output still to be added."""
    cfg = {**CONFIGS["odd"], "loop": None}
    W, toks = weights(cfg, seed=8), tokens(cfg, 30)
    per_layer = []
    Z.forward(cfg, floats(W), toks, per_layer)
    for n in range(1, len(cfg["layers"]) + 1):
        note(f"residual after {n} layers")
        eng = engine(hip, {**cfg, "layers": cfg["layers"][:n]}, W, prefill_chunk=30)
        eng.score("a", toks)
        x, y = eng.read_rows(eng._residual, 30, cfg["width"]), eng.read_rows("branch", 30, cfg["width"])
        w = floats(W)[f"l{n - 1}.norm2b" if cfg["layers"][n - 1]["mlp"] else f"l{n - 1}.norm1b"]
        assert rel(x + Z.norm(y.astype(float), w, cfg["norm"]["eps"]), per_layer[n - 1]) < 2e-5


@pytest.mark.parametrize("plan", [True, False])
def test_long_decoding_past_many_windows(hip, plan):
    cfg = config([att(window=7), ssm(), att(window=50, every=40)], width=40, vocab=64, loop=(1, 2, 3))
    W, toks = weights(cfg, seed=12), tokens(cfg, 400)
    note(f"long decoding plan={plan}")
    want = Z.forward(cfg, floats(W), toks)
    eng = engine(hip, cfg, W, prefill_chunk=64, decode_plan=plan)
    got = [eng.score("a", toks[:5], range(5))] + [eng.score("a", [t], [0]) for t in toks[5:]]
    assert rel(np.concatenate(got), want) < 1e-4


def test_passes_of_a_loop_keep_their_own_state(hip):
    """Two layers run twice are four layers with the same weights."""
    note("loop against unrolled layers")
    cfg = config([ssm(), att(window=5)], width=44, vocab=50, loop=(0, 2, 2))
    W, toks = weights(cfg, seed=3), tokens(cfg, 40)
    flat = {**cfg, "layers": cfg["layers"] * 2, "loop": None}
    W2 = dict(W, **{f"l{int(n[1]) + 2}{n[2:]}": w for n, w in W.items() if n[0] == "l" and n[1].isdigit()})
    got = []
    for c, w in ((cfg, W), (flat, W2)):
        eng = engine(hip, c, w, prefill_chunk=16)
        got.append(np.concatenate([eng.score("a", toks[lo:hi], range(hi - lo)) for lo, hi in ((0, 21), (21, 22), (22, 24), (24, 40))]))
    assert rel(got[0], got[1]) < 1e-6


def test_generation(hip):
    """Greedy tokens of the framework's loop, one step ahead of the read-back, equal those of the plain model; so do
    lockstep sequences; a prefix the state holds is reused."""
    cfg = CONFIGS["odd"]
    W, prompt = weights(cfg, seed=4), tokens(CONFIGS["odd"], 11)
    toks = list(prompt)
    for _ in range(40):
        toks.append(int(np.argmax(Z.forward(cfg, floats(W), toks)[-1])))
    note("greedy generation")
    for kw in (dict(), dict(lookahead=False), dict(decode_plan=False), dict(sampling_mode="gpu_argmax")):
        out, stats = engine(hip, cfg, W, prefill_chunk=8, **kw).generate(prompt, GenerationConfig(max_tokens=40))
        assert out == toks[11:], kw
    eng = engine(hip, cfg, W, prefill_chunk=8)
    eng.generate(prompt, GenerationConfig(max_tokens=40))
    follow = toks + tokens(cfg, 4, seed=8)
    more, st = eng.generate(follow, GenerationConfig(max_tokens=5), reuse_prefix=51)
    assert st["n_prompt_reused"] == 51
    assert more == engine(hip, cfg, W, prefill_chunk=8).generate(follow, GenerationConfig(max_tokens=5))[0]
    note("lockstep")
    prompts = [tokens(cfg, 9, seed=20 + i) for i in range(4)]
    alone = [engine(hip, cfg, W, prefill_chunk=8).generate(p, GenerationConfig(max_tokens=30))[0] for p in prompts]
    out, _ = engine(hip, cfg, W, prefill_chunk=8, batch=4).generate_batch(prompts, 30)
    assert out == alone
    note("sampling")
    for kw in (dict(temperature=0.8, top_k=8, top_p=0.9, repeat_penalty=1.2, seed=3), dict(temperature=0.7, top_k=0, seed=3)):
        ref = MixerEngine(oracle.init(), zaparax_config(cfg), W, A=A, dtype="float32", prefill_chunk=8)
        want, _ = ref.generate(prompt, GenerationConfig(max_tokens=12, **kw))
        assert engine(hip, cfg, W, prefill_chunk=8).generate(prompt, GenerationConfig(max_tokens=12, **kw))[0] == want


def test_trace_replay_and_command_line(hip, tmp_path):
    """The programs, each in a process of its own, on a model folder."""
    cfg = CONFIGS["odd"]
    W, toks = weights(cfg, seed=5, steady=True), tokens(CONFIGS["odd"], 50)
    write_model(tmp_path, cfg, W)
    want = Z.forward(cfg, floats(W), toks)
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
        seq.append(int(np.argmax(Z.forward(cfg, floats(W), seq)[-1])))
    assert json.loads(r.stdout.splitlines()[-1])["tokens"] == seq[9:]


def test_calls_with_impossible_operands_are_refused(hip):
    """Ranges and sizes are checked on the host before anything is launched."""
    note("refused calls")
    eng = engine(hip, CONFIGS["odd"], weights(CONFIGS["odd"]))
    up = lambda s: hip.upload_dev(s.words())[0]
    win = dict(heads=2, kv_heads=1, dim=8, vdim=8, window=4, x=0, x_stride=40, x_q=0, x_k=16, x_v=24, temp_every=1, out=0, out_stride=16, cache_map=14,
               v_off=32, seq_stride=64)
    for bad in (dict(dim=300), dict(temp_every=0), dict(seq_stride=56), dict(x_v=33), dict(cache_map=3, k_off=4), dict(kv_heads=0), dict(window=0)):
        with pytest.raises(RuntimeError, match="-3"):
            hip.window_attention_dev(0, up(A.WindowAttnSpec(**{**win, **bad})), 1, 1, 0, 0)
    ssp = dict(heads=2, groups=1, state=4, vdim=3, taps=2, x=0, x_stride=24, x_c=6, x_dt=20, out=0, out_stride=6, state_map=3, conv_off=24, seq_stride=52)
    for bad in (dict(groups=3), dict(taps=17), dict(seq_stride=51), dict(x_dt=23), dict(state=257), dict(state_map=1)):
        with pytest.raises(RuntimeError, match="-3"):
            hip.state_space_dev(0, up(A.StateSpaceSpec(**{**ssp, **bad})), 1, 1, 0, 0)
    mid = eng.stack(["l0.mlp.experts.in"])[0]
    ex = dict(experts=2, top=1, ff=16, ff_stride=64, width=16, k_stride=64, gate_up_step=2048, down_step=1024, logits_stride=2, x_stride=16, out_stride=16)
    for bad in (dict(top=3), dict(ff_stride=60), dict(gate_up_step=2040), dict(experts=2000), dict(down=1 << 31), dict(epi=2)):
        with pytest.raises(RuntimeError, match="-3"):
            hip.experts_dev(0, 2, mid, up(A.ExpertsSpec(**{**ex, **bad})), 0, 1)
    emb = dict(table=0, vocab=4, width=8, dst=0, pairs=0, buckets=3, state_map=3, prev_off=0, seq_stride=8)
    locs = hip.upload_dev(np.zeros(1, np.uint32))[0]
    for bad in (dict(buckets=0), dict(prev_off=8), dict(vocab=1 << 30), dict(state_map=1)):
        with pytest.raises(RuntimeError, match="-3"):
            hip.embed_bigram_dev(0, mid, up(A.BigramSpec(**{**emb, **bad})), locs, 1, 1, 0, 0)
    off, n, k, stride = eng.stack(["head"])[1:]
    good = dict(w=off, n=n, k=k, k_stride=stride, src=0, src_stride=k, groups=1, out=4000, out_stride=n, branch=2000, branch_stride=k, branched=1)
    for bad in (dict(branched=3), dict(branched=2, res_out=k - 1), dict(groups=2), dict(tail=3), dict(branch=(1 << 32) - 2), dict(kept=1, keep=(1 << 32) - 2)):
        with pytest.raises(RuntimeError, match="-3"):
            hip.linear_dev(0, 2, mid, up(A.LinearSpec(**{**good, **bad})), 0, 1)
