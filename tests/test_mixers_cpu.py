"""Layered mixer models without a GPU: the engine on the NumPy op surface against the plain statement of the mechanisms,
loading and registry, sequence slots, and that the plain statement notices planted mistakes."""
import io
import json
import os

import numpy as np
import pytest

import oracle
from adam_amd import adamah as A
from adam_amd.engine import GenerationConfig
from adam_amd.mixer_engine import MixerEngine, SequenceSlots
from adam_amd.models import load_config, load_engine, vomotar_config
from adam_amd.replay import replay
from adam_amd.safetensors_file import SafetensorsFile, bf16_to_f32, f32_to_bf16
from mixer_cases import CONFIGS, config, delta, floats, par, rel, weights, write_model
from oracle import mixers_np as M


def engine(cfg, W, dtype="float32", **kw):
    return MixerEngine(oracle.init(), vomotar_config(cfg), W, A=A, dtype=dtype, **kw)


def tokens(cfg, n, seed=1):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


@pytest.mark.parametrize("name", ["odd", "ones"])
@pytest.mark.parametrize("chunk", [1, 2, 5, 64])
def test_engine_on_the_numpy_surface_equals_the_plain_model(name, chunk):
    cfg = CONFIGS[name]
    W, toks = weights(cfg), tokens(CONFIGS[name], 26)
    want = M.forward(cfg, floats(W), toks)
    eng = engine(cfg, W, prefill_chunk=chunk)
    assert rel(eng.score("a", toks, range(26)), want) < 2e-5
    # the same slot again, another sequence
    eng.release("a")
    toks2 = tokens(cfg, 9, seed=5)
    assert rel(eng.score("b", toks2, range(9)), M.forward(cfg, floats(W), toks2)) < 2e-5


def test_cut_anywhere_and_interleaved_sequences():
    cfg = CONFIGS["odd"]
    W = weights(cfg, seed=3)
    seqs = {n: tokens(cfg, 24, seed=10 + i) for i, n in enumerate("abc")}
    eng = engine(cfg, W, prefill_chunk=8, batch=3)
    want = {n: M.forward(cfg, floats(W), t) for n, t in seqs.items()}
    at, rng = dict.fromkeys(seqs, 0), np.random.default_rng(0)
    while any(at[n] < 24 for n in seqs):
        n = rng.choice([n for n in seqs if at[n] < 24])
        m = int(min(rng.integers(1, 6), 24 - at[n]))
        got = eng.score(n, seqs[n][at[n]:at[n] + m], range(m))
        assert rel(got, want[n][at[n]:at[n] + m]) < 2e-5
        at[n] += m


def test_greedy_generation_equals_the_plain_model():
    cfg = CONFIGS["odd"]
    W, prompt = weights(cfg, seed=4), tokens(CONFIGS["odd"], 11)
    toks = list(prompt)
    for _ in range(14):
        toks.append(int(np.argmax(M.forward(cfg, floats(W), toks)[-1])))
    eng = engine(cfg, W, prefill_chunk=4)
    out, stats = eng.generate(prompt, GenerationConfig(max_tokens=14))
    assert out == toks[11:] and stats["sampling_mode"] == "gpu_matvec_argmax"
    # the state now holds the prompt and everything generated: a longer prompt continues from there, any other starts over
    follow = toks + tokens(cfg, 3, seed=8)
    more, st = eng.generate(follow, GenerationConfig(max_tokens=3), reuse_prefix=25)
    assert st["n_prompt_reused"] == 25
    fresh, st = engine(cfg, W, prefill_chunk=4).generate(follow, GenerationConfig(max_tokens=3))
    assert more == fresh and st["n_prompt_reused"] == 0
    again, st = eng.generate(follow, GenerationConfig(max_tokens=3), reuse_prefix=25)
    assert again == fresh and st["n_prompt_reused"] == 0


def test_lockstep_batch_equals_sequences_alone():
    cfg = CONFIGS["odd"]
    W = weights(cfg, seed=6)
    prompts = [tokens(cfg, 9, seed=20 + i) for i in range(3)]
    alone = [engine(cfg, W, prefill_chunk=4).generate(p, GenerationConfig(max_tokens=12))[0] for p in prompts]
    out, _ = engine(cfg, W, prefill_chunk=4, batch=3).generate_batch(prompts, 12)
    assert out == alone


@pytest.mark.parametrize("kw", [dict(temperature=0.8, top_k=5, top_p=0.9, repeat_penalty=1.2, seed=3),
                                dict(temperature=0.7, top_k=0, seed=3)])
def test_sampling_modes_take_the_models_logits(kw):
    cfg = CONFIGS["odd"]
    W, prompt = weights(cfg, seed=7), tokens(CONFIGS["odd"], 6)
    eng = engine(cfg, W, prefill_chunk=4)
    out, stats = eng.generate(prompt, GenerationConfig(max_tokens=8, **kw))
    assert stats["sampling_mode"] == ("gpu_topk" if kw["top_k"] else "cpu")
    toks = prompt + out
    if kw["top_k"]:
        for i, t in enumerate(out):                  # every token drawn is among the penalised top k
            lg = M.forward(cfg, floats(W), toks[:6 + i])[-1]
            for p in set(out[:i]):
                lg[p] = lg[p] / 1.2 if lg[p] > 0 else lg[p] * 1.2
            assert t in np.argsort(lg)[::-1][:5]
    assert len(out) == 8


def test_steps_must_follow_each_other_and_tokens_lie_in_the_vocabulary():
    cfg = CONFIGS["ones"]
    eng = engine(cfg, weights(cfg), prefill_chunk=4)
    eng.score("a", [1, 2, 3])
    with pytest.raises(RuntimeError, match="cannot follow"):
        eng._forward_chunk([1, 2], 7)
    with pytest.raises(RuntimeError, match="in use"):
        eng.score("b", [1])
    with pytest.raises(ValueError, match="token ids"):
        eng.score("a", [cfg["vocab"]])


def test_slots():
    s = SequenceSlots(2)
    assert (s.open("a"), s.open("b"), s.open("a")) == (0, 1, 0)
    s.pos[0] = 9
    s.close("a")
    s.close("never there")
    assert s.open("c") == 0 and s.pos[0] == 0


def test_model_folder_round_trip(tmp_path):
    cfg = CONFIGS["odd"]
    W = weights(cfg)
    write_model(tmp_path, cfg, W)
    f = SafetensorsFile(os.path.join(tmp_path, "model.safetensors"))
    assert sorted(f.names()) == sorted(W)
    assert all(np.array_equal(f.bf16(n), W[n]) and np.array_equal(f.f32(n), bf16_to_f32(W[n])) for n in W)
    eng = load_engine(oracle.init(), str(tmp_path), A=A, dtype="float32", prefill_chunk=3)
    toks = tokens(cfg, 7)
    want = M.forward(cfg, floats(W), toks)
    assert rel(eng.score("x", toks, [6, 2]), want[[6, 2]]) < 2e-5
    # replay: same logits through the step protocol, files only where something is wanted
    eng.release("x")
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:4], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[4:], "want": [2, 0]}], "end": ["q"]},
             {"step": 2, "entries": [{"id": "r", "tokens": toks[:2], "want": [1]}], "end": ["r"]}]
    done = []
    replay(eng, io.StringIO("\n".join(json.dumps(s) for s in steps)), str(tmp_path), done.append)
    assert done == [0, 1, 2] and not os.path.exists(tmp_path / "0.f32")
    got = np.fromfile(tmp_path / "1.f32", "<f4").reshape(2, -1)
    assert rel(got, want[[6, 4]]) < 2e-5
    assert rel(np.fromfile(tmp_path / "2.f32", "<f4").reshape(1, -1), want[[1]]) < 2e-5


def test_wrong_files_fail_by_name(tmp_path):
    cfg = CONFIGS["odd"]
    W = weights(cfg)
    for bad, msg in ((dict(W, **{"l0.mix.q": W["l0.mix.q"][:-1]}), "l0.mix.q"), ({n: w for n, w in W.items() if n != "l1.mix.left.r2"}, "r2")):
        with pytest.raises(ValueError, match=msg):
            engine(cfg, bad)
    inexact = dict(W, **{"head": bf16_to_f32(W["head"]) * np.float32(1.001)})
    with pytest.raises(ValueError, match="head"):
        engine(cfg, inexact)
    engine(cfg, inexact, dtype="bfloat16")
    for change in ({"architecture": "Other"}, {"layers": [{"type": "other", "mixer": {}, "mlp": None}]}):
        write_model(tmp_path, {**cfg, **change}, W)
        with pytest.raises(ValueError, match="not known"):
            load_config(str(tmp_path))


def test_sizes_the_kernels_do_not_hold_are_refused_at_load():
    bad = [delta(dim=300), delta(conv=17), delta(heads=4, kv_heads=3), par(size=0), par(rot=13), par(r_heads=2, decay=[0.5]), par(r_vdim=257)]
    for layer in bad:
        with pytest.raises(ValueError):
            vomotar_config(config([layer]))
    with pytest.raises(ValueError, match="groups"):
        vomotar_config(config([delta()], width=50, groups=4))


def test_specs_agree_with_the_header_and_the_numpy_surface():
    """The structs that travel in handles: same fields in the same order, in C, in the binding and in the oracle."""
    import re
    from oracle import mixer_ops_np as O
    src = re.sub(r"/\*.*?\*/", "", open(os.path.join(os.path.dirname(A.__file__), "..", "include", "adamah_hip.h")).read(), flags=re.S)
    for c_name, cls, fields in (("AdamahLinearSpec", A.LinearSpec, O._LINEAR), ("AdamahMergeSpec", A.MergeSpec, O._MERGE),
                                ("AdamahDeltaSpec", A.DeltaSpec, O._DELTA), ("AdamahRetentionSpec", A.RetentionSpec, O._RET),
                                ("AdamahChunkAttnSpec", A.ChunkAttnSpec, O._ATT)):
        body = re.search(r"typedef struct %s \{(.*?)\}" % c_name, src, flags=re.S).group(1)
        decl = [(t, n.strip()) for t, names in re.findall(r"(uint32_t|float)([^;]*);", body) for n in names.split(",")]
        ours = [("float" if t is A.f32c else "uint32_t", n) for n, t in cls._fields_]
        assert decl == ours and [n for _, n in ours] == fields.split(), c_name


def test_bfloat16_rounding():
    x = np.array([1.0, 1.00390625, 1.01171875, -3.1415927, 65504.0, 1e-30, np.inf], np.float32)
    r = bf16_to_f32(f32_to_bf16(x))
    assert r[1] == 1.0 and r[2] == 1.015625 and r[0] == 1.0 and np.isinf(r[6])       # ties go to even
    assert np.all(np.abs(r[:6] - x[:6]) <= np.abs(x[:6]) * 2.0 ** -8)


# ---- the oracle itself -------------------------------------------------------------------------------------------------
def test_plain_delta_rule_recalls_what_was_written():
    """With unit keys, a step size of one and no decay the rule is exact recall of the last value under a key."""
    D, V = 6, 4
    rng = np.random.default_rng(0)
    keys = np.linalg.qr(rng.standard_normal((D, D)))[0]
    order, vals = [0, 1, 2, 1, 0, 3], rng.standard_normal((6, V))
    k = keys[order][:, None, :]
    o, S = M.delta_rule(k, k, vals[:, None], np.ones((6, 1, D)), np.ones((6, 1)))
    assert np.allclose(o[:, 0], vals)                       # the read-out sees the token's own write
    assert np.allclose(keys[[0, 1, 2, 3]] @ S[0], vals[[4, 3, 2, 5]])


def test_plain_retention_is_a_decayed_sum():
    """All keys equal, no rotation: the state is the geometric sum of the values."""
    dec = 0.75
    W = {"q": np.ones((1, 1)), "k": np.ones((1, 1)), "v": np.ones((1, 1)), "g": np.ones((1, 1)), "o": np.ones((1, 1))}
    c = {"heads": 1, "dim": 1, "vdim": 1, "decay": [dec], "rot": {"base": 10.0, "dims": 0}}
    h = np.ones((5, 1))
    s = np.array([sum(dec ** j for j in range(t + 1)) for t in range(5)])[:, None]
    assert np.allclose(M.retention(h, W, c, 0.0), s / np.abs(s) * M.silu(1.0))


def test_plain_rotation_depends_on_distance_only():
    x = np.random.default_rng(1).standard_normal((1, 2, 12))
    dot = lambda p, q: np.sum(M.rotate_half(x, 100.0, 8, p)[0, 0] * M.rotate_half(x, 100.0, 8, q)[0, 1])
    assert np.isclose(dot(3, 9), dot(40, 46)) and not np.isclose(dot(3, 9), dot(3, 10))
    assert np.array_equal(M.rotate_half(x, 100.0, 8, 5)[..., 8:], x[..., 8:])


def test_a_chunk_edge_one_token_off_shows():
    cfg = config([par(size=9)], width=40, groups=2)
    W, toks = floats(weights(cfg)), tokens(config([par()]), 30)
    right, wrong = M.forward(cfg, W, toks), M.forward(cfg, W, toks, plant="edge")
    err = np.sqrt(np.mean((right - wrong) ** 2, axis=1)) / np.sqrt(np.mean(right ** 2))
    assert err[8] > 0.02 and err[18] > 0.02 and err[:8].max() < 1e-12
