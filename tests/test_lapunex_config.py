"""The Lapunex design without a GPU: the configuration, the layout's tensors, run order and cache needs, the rotation's tables,
and the plain implementation's own consistency."""
from __future__ import annotations

import copy

import numpy as np
import pytest

import plain_lapunex as P
from lapunex_common import CONFIGS, TAGS, as_numpy, config, dense, light, lightning, plain_logits, random_weights, tokens_of

import llama_cu_amd  # noqa: F401
from llama_cu_amd.config import ConfigError, LapunexConfig, architecture_of
from llama_cu_amd.parts import DecoderModel, PagedKV, PartSpec, SlotState, make_part


def built(cfg):
    arch = architecture_of(cfg)
    typed = arch.config_from_dict(cfg)
    return typed, DecoderModel(arch.build_spec(typed))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_layout_names_exactly_the_tensors_of_the_design_and_the_configuration_reads_back(name):
    typed, model = built(CONFIGS[name])
    want = {k: tuple(v.shape) for k, v in random_weights(CONFIGS[name], 1).items()}
    assert {k: tuple(v.shape) for k, v in model.tensors().items() if not v.optional or k == "head"} == want
    assert LapunexConfig.from_dict(typed.to_dict()) == typed


def test_run_order_and_cache_needs():
    _, model = built(CONFIGS["A"])
    assert [e.layer for e in model.spec.run_order] == [0, 1, 2, 1, 2, 3]
    assert all(e.cache_of is None and e.before is None for e in model.spec.run_order) and len(model.layers) == 4
    needs = model.cache_needs()
    assert isinstance(needs[0], SlotState) and needs[0].shape == (3 * 20 * 12,) and not needs[0].can_truncate
    pages, memory = needs[1].needs
    assert isinstance(pages, PagedKV) and (pages.kv_heads, pages.window) == (2, 0)
    # matrices, normalisers and maxima in one flat slot
    assert isinstance(memory, SlotState) and memory.shape == (3 * 20 * 28 + 3 * 20 + 3,)
    assert model.graph_safe and {p.streams for p in model.layers + [model.embedding, model.final_norm]} == {3}
    _, model = built(CONFIGS["D"])
    assert [e.layer for e in model.spec.run_order] == [0, 1] * 3 and all(n.pool() is None for n in model.cache_needs())


def test_parts_that_keep_other_numbers_of_streams_do_not_go_together():
    typed, _ = built(CONFIGS["D"])
    spec = architecture_of(CONFIGS["D"]).build_spec(typed)
    spec.embedding.params["streams"] = 1
    with pytest.raises(ValueError):
        DecoderModel(spec)
    with pytest.raises(ValueError):
        make_part("norm", PartSpec("streams_rmsnorm", {"size": 8, "eps": 1e-5, "streams": 9}))


@pytest.mark.parametrize("change,key", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 0.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, -0.5, 0.5]), "decay"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(gate_cap=0.0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(mask={"size": 4}), "mask"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=14), "dims"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][1]["mlp"].update(kind="mixture"), "kind"),
    (lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "top"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=5), "groups"),
    (lambda c: c.update(loop={"start": 3, "stop": 3, "times": 2}), "loop"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.update(streams=0), "streams"),
])
def test_an_error_names_its_key(change, key):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError) as e:
        architecture_of(cfg).config_from_dict(cfg)
    assert key in str(e.value)


@pytest.mark.parametrize("dims,base,scaling", [
    (8, 700.0, {"factor": 5.0, "original": 48, "fast": 4.0, "slow": 0.25}), (64, 10000.0, {"factor": 8.0, "original": 2048, "fast": 32.0, "slow": 1.0}),
    (2, 50.0, {"factor": 2.0, "original": 16, "fast": 1.0, "slow": 0.5}), (16, 1e6, {"factor": 1.0, "original": 64, "fast": 8.0, "slow": 2.0}),
    (32, 100.0, {"factor": 40.0, "original": 100000, "fast": 1.0, "slow": 1.0})])
def test_the_tables_of_the_blended_frequencies(dims, base, scaling):
    """Against the plain ones; fast pairs keep their frequency and slow ones have it divided."""
    part = make_part("position", PartSpec("rotary", {"head_dim": dims, "theta": base, "max_positions": 300, "yarn": scaling}))
    cos, sin = part.host_tables()
    freq, factor = P.yarn(dims, base, scaling)
    x = np.random.default_rng(1).standard_normal((300, 2, dims))
    want = P.rotate_half_split(x, np.arange(300.0), freq, factor)
    u, v = x[..., :dims // 2], x[..., dims // 2:]
    got = np.concatenate([u * cos[:, None] - v * sin[:, None], v * cos[:, None] + u * sin[:, None]], -1)
    assert np.abs(got - want).max() < 1e-5
    assert abs(np.hypot(cos, sin) - (0.1 * np.log(scaling["factor"]) + 1)).max() < 1e-6
    plain_freq = base ** (-2.0 * np.arange(dims // 2) / dims)
    assert np.all(freq <= plain_freq * (1 + 1e-12)) and np.all(freq >= plain_freq / scaling["factor"] * (1 - 1e-12))
    if dims == 64:
        turns = 2048 * plain_freq / (2 * np.pi)
        assert np.allclose(freq[turns > 40], plain_freq[turns > 40]) and np.allclose(freq[turns < 0.7], plain_freq[turns < 0.7] / 8)
        assert np.any((freq < plain_freq * 0.99) & (freq > plain_freq / 8 * 1.01))
    for bad in (dict(scaling, factor=0.0), dict(scaling, original=-1)):
        with pytest.raises(ValueError):
            make_part("position", PartSpec("rotary", {"head_dim": dims, "theta": base, "max_positions": 4, "yarn": bad}))


def test_a_memory_with_running_maximum_is_the_one_without():
    """The plain scan against the sums it stands for, with gates small enough to be multiplied out."""
    rng = np.random.default_rng(2)
    T, d, dv = 30, 5, 4
    q, k, v = rng.standard_normal((T, d)), rng.standard_normal((T, d)), rng.standard_normal((T, dv))
    i, f = P.mlstm_gates(rng.standard_normal(T) * 2, rng.standard_normal(T) + 1, 3.0)
    got = P.mlstm_scan(q, k, v, i, f)
    for t in range(T):
        w = np.array([np.exp(i[s] + f[s + 1:t + 1].sum()) for s in range(t + 1)])
        S, n = np.einsum("s,sd,sv->dv", w, k[:t + 1], v[:t + 1]), (w[:, None] * k[:t + 1]).sum(0)
        m = 0.0
        for s in range(t + 1):
            m = max(f[s] + m, i[s])
        want = (q[t] @ S) * np.exp(-m) / (max(abs(n @ q[t]) * np.exp(-m), np.exp(-m)) + 1e-6)
        assert np.allclose(got[t], want, rtol=1e-10)


def test_the_chunked_form_is_the_recurrence():
    rng = np.random.default_rng(3)
    T, d, dv, decay = 41, 6, 3, 0.9
    q, k, v = rng.standard_normal((T, d)), rng.standard_normal((T, d)), rng.standard_normal((T, dv))
    S, out = np.zeros((d, dv)), []
    for c0 in range(0, T, 16):
        t = np.arange(c0, min(T, c0 + 16))
        L = np.log(decay) * np.arange(1, len(t) + 1)
        w = np.where(t[None] <= t[:, None], (q[t] @ k[t].T) * np.exp(L[:, None] - L[None]), 0.0)
        out.append(np.exp(L)[:, None] * (q[t] @ S) + w @ v[t])
        S = np.exp(L[-1]) * S + (k[t] * np.exp(L[-1] - L)[:, None]).T @ v[t]
    assert np.allclose(np.concatenate(out), P.decay_scan(q, k, v, decay), rtol=1e-10)


def test_choice_within_groups():
    z = np.log(np.array([0.30, 0.01, 0.02, 0.25, 0.24, 0.18]))          # groups of two: best 0.30, 0.25, 0.24
    chosen, s = P.route(z, 2, {"count": 3, "keep": 1})
    assert chosen.tolist() == [0, 1] and np.allclose(s, [0.30, 0.01])
    assert P.route(z, 2, {"count": 3, "keep": 2})[0].tolist() == [0, 3]
    assert P.route(z, 3)[0].tolist() == [0, 3, 4]
    assert P.route(np.zeros(6), 3, {"count": 3, "keep": 2})[0].tolist() == [0, 1, 2]


def test_one_plain_stream_is_the_residual_sum():
    """A stream read, written and kept with weights of one is the usual residual."""
    cfg = config(50, 24, [light(lightning([0.5, 0.9], 8, 8), dense(16))], 1e-5, 1)
    W = as_numpy(random_weights(cfg, 4))
    for q in (1, 2):
        W[f"l0.hc{q}.in"], W[f"l0.hc{q}.out"], W[f"l0.hc{q}.mix"] = np.ones(1), np.ones(1), np.ones((1, 1))
    toks = tokens_of(50, 9, 1)
    x = W["embed"][toks]
    x = x + P.lightning(P.rms_norm(x, 1 + W["l0.norm1"], 1e-5), W, "l0.mix.", cfg["layers"][0]["mixer"], 1e-5)
    x = x + P.dense(P.rms_norm(x, 1 + W["l0.norm2"], 1e-5), W, "l0.mlp.")
    assert np.allclose(P.forward(cfg, W, toks), P.rms_norm(x, 1 + W["final.norm"], 1e-5) @ W["head"].T)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_later_token_changes_no_earlier_logits(name):
    cfg = CONFIGS[name]
    w = random_weights(cfg, 5)
    toks = tokens_of(cfg["vocab"], 20, 2)
    a = plain_logits(cfg, w, toks)
    b = plain_logits(cfg, w, toks[:13] + [(t + 1) % cfg["vocab"] for t in toks[13:]])
    assert (a[:13] - b[:13]).abs().max() < 1e-9 and (a[13:] - b[13:]).abs().max() > 1e-3


def test_a_steady_router_chooses_by_the_tokens_tag():
    cfg = CONFIGS["B"]
    w = as_numpy(random_weights(cfg, 6, steady_router=True))
    seen, real = {}, P.experts

    def spy(h, W, pre, f):
        z = h @ W[pre + "router"].T
        top = np.sort(z, -1)[:, ::-1]
        assert (top[:, 0] - top[:, 1]).min() > 0.05
        for t, row in enumerate(h):
            seen.setdefault(int(np.argmax(row[:TAGS])), set()).add(tuple(P.route(z[t], f["router"]["top"], f["router"].get("groups"))[0]))
        return real(h, W, pre, f)

    P.experts = spy
    try:
        P.forward(cfg, w, tokens_of(cfg["vocab"], 40, 3))
    finally:
        P.experts = real
    assert len(seen) == TAGS and all(len(v) == 1 for v in seen.values()) and len(set.union(*seen.values())) > 1
