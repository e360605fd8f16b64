"""The Gefudra design without a GPU: the configuration, the layout's tensors, run order and cache needs, and the plain
implementation's own consistency."""
from __future__ import annotations

import copy

import numpy as np
import pytest

import plain_gefudra as P
from gefudra_common import CONFIGS, config, differential, latent, layer, mixer_weights, plain_logits, random_weights, as_numpy, tokens_of, wkv

import llama_cu_amd  # noqa: F401
from llama_cu_amd.config import ConfigError, GefudraConfig, architecture_of
from llama_cu_amd.parts import DecoderModel, PagedKV, SlotState


def built(cfg):
    arch = architecture_of(cfg)
    typed = arch.config_from_dict(cfg)
    return typed, DecoderModel(arch.build_spec(typed))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_layout_names_exactly_the_tensors_of_the_design(name):
    _, model = built(CONFIGS[name])
    want = {k: tuple(v.shape) for k, v in random_weights(CONFIGS[name], 1).items()}
    have = {k: tuple(v.shape) for k, v in model.tensors().items() if not v.optional}
    assert have == want


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_configuration_reads_back_and_takes_a_rank_from_the_tensors_shape(name):
    typed, _ = built(CONFIGS[name])
    assert GefudraConfig.from_dict(typed.to_dict()) == typed
    bare = copy.deepcopy(CONFIGS[name])
    for entry in bare["layers"]:
        entry["mixer"].pop("rank", None)
    arch = architecture_of(bare)
    shapes = {k: tuple(v.shape) for k, v in random_weights(CONFIGS[name], 1).items()}
    assert arch.complete_config(arch.config_from_dict(bare), shapes) == typed


def test_a_rank_that_nothing_gives_is_an_error_that_says_so():
    cfg = copy.deepcopy(CONFIGS["D"])
    cfg["layers"][1]["mixer"].pop("rank")
    arch = architecture_of(cfg)
    with pytest.raises(ConfigError) as e:
        arch.build_spec(arch.config_from_dict(cfg))
    assert "rank" in str(e.value) and "l1.mix.w1" in str(e.value)


def test_run_order_and_cache_needs():
    """The loop's layers stand in the run order once for every run, each with a cache or state of its own, and every run's
    first layer names the mix of the stream with the embedding."""
    _, model = built(CONFIGS["A"])
    order = model.spec.run_order
    assert [e.layer for e in order] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [e.before for e in order] == [None, 0, None, 0, None, 0, None, None]
    assert all(e.cache_of is None for e in order) and len(model.layers) == 4 and len(model.streams) == 1
    needs = model.cache_needs()
    assert isinstance(needs[0], PagedKV) and (needs[0].kv_heads, needs[0].window) == (1, 19)
    assert isinstance(needs[7], PagedKV) and needs[7].window == 0
    for i in (1, 3, 5):
        assert isinstance(needs[i], SlotState) and needs[i].shape == (3 * 20 * 20 + 72,) and not needs[i].can_truncate
        assert isinstance(needs[i + 1], PagedKV) and needs[i + 1].kv_heads == 2 and needs[i + 1].head_dim == 24
    _, model = built(CONFIGS["E"])
    assert [e.layer for e in model.spec.run_order] == [0, 1] and not model.streams
    # the layers of a run order may name no stream part that is not there
    spec = model.spec
    spec.run_order[0] = type(spec.run_order[0])(0, before=0)
    with pytest.raises(ValueError):
        DecoderModel(spec)


@pytest.mark.parametrize("change,key", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["layers"][0].update(type="window"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][2]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=14), "dims"),
    (lambda c: c["layers"][2]["mixer"].pop("diff"), "diff"),
    (lambda c: c["layers"][2]["mixer"].update(mask={"size": 4}), "mask"),
    (lambda c: c["layers"][1]["mixer"].pop("dim"), "dim"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c["loop"].update(stop=5), "stop"),
    (lambda c: c["loop"].update(start=3), "start"),
    (lambda c: c["loop"].pop("times"), "times"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_errors_name_their_key(change, key):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError) as e:
        GefudraConfig.from_dict(cfg)
    assert key in str(e.value)


def test_the_plain_model_is_causal_and_every_run_of_the_loop_counts():
    cfg = CONFIGS["A"]
    w = random_weights(cfg, 3)
    toks = tokens_of(cfg["vocab"], 24, 1)
    whole = plain_logits(cfg, w, toks)
    other = plain_logits(cfg, w, toks[:16] + tokens_of(cfg["vocab"], 8, 2))
    assert np.allclose(whole[:16], other[:16], atol=1e-12) and not np.allclose(whole[16:], other[16:], atol=1e-3)
    fewer = copy.deepcopy(cfg)
    fewer["loop"]["times"] = 2
    assert not np.allclose(plain_logits(fewer, w, toks), whole, atol=1e-3)
    assert P.run_order(fewer) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    without = copy.deepcopy(cfg)
    del without["loop"]
    assert P.run_order(without) == [(i, False) for i in range(4)]
    # the factor on the logits is one on the logits
    scaled = dict(cfg, logit_scale=3.2)
    assert np.allclose(plain_logits(scaled, w, toks), 2.0 * whole)


def test_the_windows_exact_edge_and_a_sink_that_takes_weight_and_gives_nothing():
    rng = np.random.default_rng(1)
    T, size = 12, 5
    q, k, v = rng.standard_normal((T, 4)), rng.standard_normal((T, 4)), rng.standard_normal((T, 3))
    seen = P.visible(T, size)
    assert seen[8].tolist() == [False] * 4 + [True] * 5 + [False] * 3
    a = P.attend(q, k, v, 1.0, seen)
    moved = v.copy()
    moved[3] += 100.0                                     # just outside the window of token 8, just inside that of token 7
    b = P.attend(q, k, moved, 1.0, seen)
    assert np.allclose(a[8], b[8]) and not np.allclose(a[7], b[7])
    with_sink = P.attend(q, k, v, 1.0, seen, sink=0.5)
    p = np.where(seen, np.exp(q @ k.T), 0.0)
    assert np.allclose(with_sink, p @ v / (p.sum(-1, keepdims=True) + np.exp(0.5)))
    assert np.allclose(P.attend(q, k, v, 1.0, seen, sink=-60.0), a)
    # one key and a sink as large as its score: half of the value
    assert np.allclose(P.attend(q[:1], k[:1], v[:1], 1.0, seen[:1, :1], sink=float(q[0] @ k[0])), 0.5 * v[:1])


def test_the_folded_form_of_latent_attention_and_the_difference_of_equal_maps():
    d, m, eps = 24, latent(2, 8, 12, 16, 10, 0.3, 7), 1e-5
    cfg = config(16, d, [layer("latent_attention", m)], eps)
    W = as_numpy(mixer_weights(cfg, 4), "p.")
    h = np.random.default_rng(2).standard_normal((15, d))
    want = P.latent_attention(h, W, "p.", m, eps)
    c = P.rms_norm(h @ W["p.dkv"].T, W["p.dkv.norm"], eps)
    q = (P.rms_norm(h @ W["p.dq"].T, W["p.dq.norm"], eps) @ W["p.uq"].T).reshape(15, 2, 8)
    o = []
    for i in range(2):
        folded = q[:, i] @ W["p.uk"][8 * i:8 * i + 8]
        o.append(P.attend(folded, c, c, m["scale"], P.visible(15, 7), sink=W["p.sink"][i]) @ W["p.uv"][12 * i:12 * i + 12].T)
    assert np.allclose((np.concatenate(o, -1) * P.sigmoid(h @ W["p.g"].T)) @ W["p.o"].T, want)
    # two equal maps: o = (1 - lambda) a, whose norm is that of a up to the sign
    m = differential(1, 1, 4, 6, 0.4, 0.25)
    W = as_numpy(mixer_weights(config(16, d, [layer("attention", m)], eps), 5), "p.")
    for s in "qk":
        W["p." + s][4:] = W["p." + s][:4]
    a = P.attend(h @ W["p.q"][:4].T, h @ W["p.k"][:4].T, h @ W["p.v"].T, 0.4, P.visible(15))
    lam = P.difference_weight(W, "p.", 0.25)
    want = (np.sign(1 - lam) * P.rms_div(a, eps / (1 - lam) ** 2) * 0.75 * P.sigmoid(h @ W["p.g"].T)) @ W["p.o"].T
    assert np.allclose(P.differential_attention(h, W, "p.", m, eps), want)


def test_the_time_mixer_of_the_plain_model_against_a_sum_over_the_tokens_before():
    d, m, eps = 12, wkv(1, 4, 2), 1e-5
    W = as_numpy(mixer_weights(config(16, d, [layer("wkv", m)], eps), 6), "p.")
    h = np.random.default_rng(3).standard_normal((9, d))
    before = np.vstack([np.zeros(d), h[:-1]])
    x = {s: h + (before - h) * W["p.mu." + s] for s in "rkvgw"}
    r, k, v = (x[s] @ W["p." + s].T for s in "rkv")
    w = np.exp(-np.exp(np.tanh(x["w"] @ W["p.w1"].T) @ W["p.w2"].T + W["p.w0"]))
    o = np.zeros((9, 4))
    for t in range(9):
        for s in range(t + 1):
            decay = W["p.u"][0] if s == t else np.prod(w[s + 1:t], axis=0)     # (a token's own decay comes after its read-out)
            o[t] += (r[t] * decay * k[s]).sum() * v[s]
    z = x["g"] @ W["p.g"].T
    want = (P.rms_div(o, eps) * W["p.norm"] * z * P.sigmoid(z)) @ W["p.o"].T
    assert np.allclose(P.wkv(h, W, "p.", m, eps), want)


def test_the_limits_of_the_feed_forward():
    W = {"f.gate": np.array([[1.0]]), "f.up": np.array([[1.0]]), "f.down": np.array([[1.0]])}
    f = {"limit": 2.0}
    y = lambda z: P.feed_forward(np.array([[z]]), W, "f.", f)[0, 0]
    s = lambda z: 1 / (1 + np.exp(-1.702 * z))
    assert np.isclose(y(1.0), s(1.0) * 2.0)
    assert np.isclose(y(9.0), 2.0 * s(2.0) * 3.0)           # both held at the limit
    assert np.isclose(y(-9.0), -9.0 * s(-9.0) * (-1.0))     # the gate has no lower limit


def test_the_bench_configurations_of_the_design_build_and_have_the_dense_models_feed_forward():
    """``bench.py --workload designs``: at both sizes as many layer runs as the dense model has layers, all three mixers, a loop."""
    import importlib.util
    import os
    spec = importlib.util.spec_from_file_location("bench", os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bench.py"))
    bench = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(bench)
    for z in bench.DESIGN_SIZES.values():
        cfg = bench.gefudra_config(z, 4096)
        model = DecoderModel(architecture_of(cfg.to_dict()).build_spec(cfg))
        assert len(model.spec.run_order) == z["layers"] and model.tensors() and model.streams
        assert {l.type for l in cfg.layers} == {"latent_attention", "attention", "wkv"}
        assert {l.ff.ff for l in cfg.layers} == {bench.llama_like(z, 4096).intermediate_size}
