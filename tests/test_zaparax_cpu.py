"""Zaparax models without a GPU: the engine on the NumPy op surface against the plain statement of the mechanisms, reading
of configurations, and that the plain statement is what it says and notices planted mistakes."""
import io
import json
import os
import re

import numpy as np
import pytest

import oracle
from adam_amd import adamah as A
from adam_amd.engine import GenerationConfig
from adam_amd.feed_forward import Experts
from adam_amd.mixer_engine import MixerEngine
from adam_amd.models import load_config, load_engine, zaparax_config
from adam_amd.replay import replay
from mixer_cases import floats, rel, write_model
from oracle import zaparax_np as Z
from zaparax_cases import CONFIGS, att, config, moe, ssm, weights


def engine(cfg, W, dtype="float32", **kw):
    return MixerEngine(oracle.init(), zaparax_config(cfg), W, A=A, dtype=dtype, **kw)


def tokens(cfg, n, seed=1):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


@pytest.mark.parametrize("name", ["odd", "ones"])
@pytest.mark.parametrize("chunk", [1, 2, 5, 64])
def test_engine_on_the_numpy_surface_equals_the_plain_model(name, chunk):
    cfg = CONFIGS[name]
    W, toks = weights(cfg), tokens(cfg, 26)
    eng = engine(cfg, W, prefill_chunk=chunk)
    assert rel(eng.score("a", toks, range(26)), Z.forward(cfg, floats(W), toks)) < 2e-5
    eng.release("a")                                   # the same slot again, another sequence
    toks2 = tokens(cfg, 9, seed=5)
    assert rel(eng.score("b", toks2, range(9)), Z.forward(cfg, floats(W), toks2)) < 2e-5


def test_wide_model_on_the_numpy_surface():
    cfg = CONFIGS["wide"]
    W, toks = weights(cfg), tokens(cfg, 6)
    assert rel(engine(cfg, W, prefill_chunk=4).score("a", toks, range(6)), Z.forward(cfg, floats(W), toks)) < 2e-5


def test_cut_anywhere_and_interleaved_sequences():
    cfg = CONFIGS["odd"]
    W = weights(cfg, seed=3)
    seqs = {n: tokens(cfg, 24, seed=10 + i) for i, n in enumerate("abc")}
    eng = engine(cfg, W, prefill_chunk=8, batch=3)
    want = {n: Z.forward(cfg, floats(W), t) for n, t in seqs.items()}
    at, rng = dict.fromkeys(seqs, 0), np.random.default_rng(0)
    while any(at[n] < 24 for n in seqs):
        n = rng.choice([n for n in seqs if at[n] < 24])
        m = int(min(rng.integers(1, 6), 24 - at[n]))
        assert rel(eng.score(n, seqs[n][at[n]:at[n] + m], range(m)), want[n][at[n]:at[n] + m]) < 2e-5
        at[n] += m


def test_greedy_generation_and_lockstep_equal_the_plain_model():
    cfg = CONFIGS["odd"]
    W = weights(cfg, seed=4)
    prompts, want = [tokens(cfg, 9, seed=20 + i) for i in range(3)], []
    for p in prompts:
        toks = list(p)
        for _ in range(8):
            toks.append(int(np.argmax(Z.forward(cfg, floats(W), toks)[-1])))
        want.append(toks[9:])
    out, _ = engine(cfg, W, prefill_chunk=4).generate(prompts[0], GenerationConfig(max_tokens=8))
    assert out == want[0]
    out, _ = engine(cfg, W, prefill_chunk=4, batch=3).generate_batch(prompts, 8)
    assert out == want


def test_a_prefix_the_slot_holds_is_continued_with_its_last_token():
    cfg = CONFIGS["odd"]
    W, prompt = weights(cfg, seed=4), tokens(CONFIGS["odd"], 11)
    eng = engine(cfg, W, prefill_chunk=4)
    out, _ = eng.generate(prompt, GenerationConfig(max_tokens=6))
    follow = prompt + out + tokens(cfg, 3, seed=8)
    more, st = eng.generate(follow, GenerationConfig(max_tokens=3), reuse_prefix=17)
    fresh, _ = engine(cfg, W, prefill_chunk=4).generate(follow, GenerationConfig(max_tokens=3))
    assert st["n_prompt_reused"] == 17 and more == fresh


def test_model_folder_and_replay(tmp_path):
    cfg = CONFIGS["odd"]
    W, toks = weights(cfg), tokens(CONFIGS["odd"], 7)
    write_model(tmp_path, cfg, W)
    eng = load_engine(oracle.init(), str(tmp_path), A=A, dtype="float32", prefill_chunk=3)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:4], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[4:], "want": [2, 0]}], "end": ["q"]}]
    done = []
    replay(eng, io.StringIO("\n".join(json.dumps(s) for s in steps)), str(tmp_path), done.append)
    assert done == [0, 1] and not os.path.exists(tmp_path / "0.f32")
    assert rel(np.fromfile(tmp_path / "1.f32", "<f4").reshape(2, -1), Z.forward(cfg, floats(W), toks)[[6, 4]]) < 2e-5


def test_configuration_is_read_from_the_file(tmp_path):
    cfg = CONFIGS["wide"]
    write_model(tmp_path, cfg, {n: w for n, w in weights(cfg).items() if n == "embed"})
    c = load_config(str(tmp_path))
    assert c.runs() == [0, 1, 0, 1, 0, 1] and c.pairs.mul_cur == 65521 and c.post_norm and c.norm_add == 1.0
    assert c.layers[0].ff == Experts(70, 9, 11, 40, 72) and c.layers[1].mixer.norm_groups == 3
    assert sorted(c.tensors()) == sorted(weights(cfg))
    assert zaparax_config(CONFIGS["odd"]).runs() == [0, 1, 2, 1, 2, 3]
    assert zaparax_config(config([att(), ssm()])).runs() == [0, 1]
    assert zaparax_config(CONFIGS["ones"]).pairs is None


def test_sizes_that_do_not_fit_are_refused_at_load():
    for layer in (att(dim=257), att(window=0), att(heads=4, kv_heads=3), att(every=0), ssm(conv=17), ssm(state=300), ssm(heads=5, groups=2),
                  ssm(norm_groups=4), {**att(), "mlp": moe(2, 1, 4)}, {**att(), "mlp": moe(900, 200, 4)}, {**att(), "mlp": moe(8, 0, 8, 5000)},
                  {**att(), "mlp": {"kind": "other"}}):
        with pytest.raises(ValueError):
            zaparax_config(config([layer]))
    for loop in ((0, 3, 1), (1, 0, 2), (0, 1, 0)):
        with pytest.raises(ValueError):
            zaparax_config(config([att(), ssm()], loop=loop))
    W = weights(CONFIGS["odd"])
    for name in ("bigram", "l0.norm1b", "l1.mix.conv.b", "l2.mlp.e4.up", "l0.mlp.shared.sg"):
        with pytest.raises(ValueError, match=re.escape(name)):
            engine(CONFIGS["odd"], {n: w for n, w in W.items() if n != name})


def test_specs_agree_with_the_header_and_the_numpy_surface():
    from oracle import mixer_ops_np as O
    src = re.sub(r"/\*.*?\*/", "", open(os.path.join(os.path.dirname(A.__file__), "..", "include", "adamah_hip.h")).read(), flags=re.S)
    for c_name, cls, fields in (("AdamahWindowAttnSpec", A.WindowAttnSpec, O._WIN), ("AdamahStateSpaceSpec", A.StateSpaceSpec, O._SSM),
                                ("AdamahExpertsSpec", A.ExpertsSpec, O._MOE), ("AdamahBigramSpec", A.BigramSpec, O._BIGRAM)):
        body = re.search(r"typedef struct %s \{(.*?)\}" % c_name, src, flags=re.S).group(1)
        decl = [(t, n.strip()) for t, names in re.findall(r"(uint32_t|float)([^;]*);", body) for n in names.split(",")]
        ours = [("float" if t is A.f32c else "uint32_t", n) for n, t in cls._fields_]
        assert decl == ours and [n for _, n in ours] == fields.split(), c_name


# ---- the oracle itself -------------------------------------------------------------------------------------------------
def test_plain_state_space_is_a_decayed_sum():
    """One head, one dimension: the state is the sum of dt B x, each decayed by the steps behind it."""
    dt, x = np.array([0.5, 1.0, 0.25]), np.array([2.0, -1.0, 3.0])
    one = np.ones((3, 1, 1))
    y, S = Z.state_space(x[:, None, None], one, 2.0 * one, dt[:, None], np.array([np.log(0.7)]), np.array([0.1]))
    s = [sum(dt[j] * x[j] * np.exp(-0.7 * dt[j + 1:t + 1].sum()) for j in range(t + 1)) for t in range(3)]
    assert np.allclose(y[:, 0, 0], 2.0 * np.array(s) + 0.1 * x) and np.isclose(S[0, 0, 0], s[2])


def test_plain_convolution_ends_at_the_current_token():
    x = np.zeros((6, 1))
    x[2] = 1.0
    y = Z.short_conv(x, np.array([[1.0, 2.0, 4.0]]), np.array([0.5]))
    assert np.allclose(y[:, 0], Z.silu(np.array([0.5, 0.5, 4.5, 2.5, 1.5, 0.5])))


def test_plain_window_and_sink():
    i, j = np.arange(6)[:, None], np.arange(6)[None, :]
    w = Z.window_weights(np.zeros((6, 6)), i, j, 3, 0.0, sink=np.log(2.0))
    assert np.allclose(w[5], [0, 0, 0, 0.2, 0.2, 0.2]) and np.allclose(w[0], [1 / 3, 0, 0, 0, 0, 0])
    w = Z.window_weights(np.full((6, 6), 50.0), i, j, 6, np.log(2.0), softcap=1.0)
    assert np.allclose(w[1], [1 / 3, 2 / 3, 0, 0, 0, 0])                       # the nearer key counts double, the cap cancels
    assert Z.temperature(np.array([0, 3, 4, 9]), 2.0, 5).tolist() == pytest.approx([1, 1, 1 + 2 * np.log(2), 1 + 2 * np.log(3)])


def test_plain_experts_weigh_by_uncorrected_scores():
    rng = np.random.default_rng(0)
    W = {"router": np.zeros((3, 4)), "correction": np.array([0.0, 1.0, 2.0])}
    for e in range(2):
        W.update({f"e{e}.{n}": rng.standard_normal(s) for n, s in (("gate", (5, 4)), ("up", (5, 4)), ("down", (4, 5)))})
    h = rng.standard_normal((2, 4))
    y = Z.experts(h, W, {"router": {"experts": 2, "identity": 1, "top": 2}})
    assert np.allclose(y, (h + Z.gated(h, Z.sub(W, "e1."))) / 3.0)


@pytest.mark.parametrize("plant,first", [("window", 7), ("sink", 0), ("prev", 1), ("conv", 0), ("pass", 0)])
def test_a_planted_mistake_shows(plant, first):
    cfg = CONFIGS["odd"]
    W, toks = floats(weights(cfg)), tokens(cfg, 24)
    right, wrong = Z.forward(cfg, W, toks), Z.forward(cfg, W, toks, plant=plant)
    err = np.sqrt(np.mean((right - wrong) ** 2, axis=1)) / np.sqrt(np.mean(right ** 2))
    assert err[:first].max(initial=0.0) < 1e-12 and err[first:].max() > 0.02
