"""The Lapunex design on the GPU against the plain implementation of ``plain_lapunex.py``: every mechanism alone, then
whole models through the engine's own step function, cache manager and scheduler, cut and batched in every way that
must not change a token's logits."""
from __future__ import annotations

import copy
import random

import numpy as np
import pytest
import torch

import plain_lapunex as P
from lapunex_common import (CONFIGS, Feeder, as_numpy, assert_close, both, built, config, dense, hand_step, left, light, lightning,
                            make_folder, mixer_weights, moe, plain_logits, random_weights, right, sharpened, tokens_of, yarn)

pytestmark = pytest.mark.gpu
TYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
REL = {"float32": 3e-4, "bfloat16": 8e-2}         # of the largest expected value
SAME = {"float32": 4e-5, "bfloat16": 6e-2}        # between two runs of the engine that cut or batch the same tokens differently


def rnd(*shape, seed=0, std=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * std


def f64(t):
    return t.double().numpy()


# ------------------------------------------------------------------ mechanisms alone


# (at the widest, one number of streams that has a kernel of its own and one that has not)
STREAM_SIZES = [(s, n, d) for n, d in ((5, 72), (3, 18), (2, 3000), (300, 2048), (2, 8200), (1, 5001)) for s in (1, 2, 3, 4, 5, 8)
                if n * d <= 100000 or s in (3, 8)]


@pytest.mark.parametrize("streams,n,d", STREAM_SIZES)
def test_streams_are_read_written_and_mixed(streams, n, d):
    """Outputs in either type and planes of partial sums; without an output; without reading weights; without writing back."""
    from llama_cu_amd.kernels import ops
    eps = 1e-5
    X, w, mix = rnd(n, streams, d, seed=1), rnd(d, seed=2), rnd(streams, streams, seed=3)
    inn, out_w = rnd(streams, seed=4), rnd(streams, seed=5)
    cu = lambda t: t.contiguous().cuda()
    for dt, planes in ((None, 0), (torch.float32, 0), (torch.bfloat16, 0), (torch.float32, 5)):
        for T in (torch.float32, torch.bfloat16):
            if dt == torch.bfloat16 and T == torch.float32:
                continue
            y = None if dt is None else rnd(planes, n, d, seed=6) if planes else rnd(n, d, seed=6).to(dt)
            want = f64(X) if y is None else P.update_streams(f64(X), f64(mix), f64(out_w), f64(y.float().sum(0) if planes else y.float()))
            for read in (inn, None):
                x = cu(X.reshape(n, -1))
                kw = {} if y is None else dict(delta=cu(y), mix=cu(mix), out_weights=cu(out_w))
                h = ops.streams_norm(x, streams, cu(w), eps, T, read=None if read is None else cu(read), **kw)
                u = P.read_streams(want, np.ones(streams) if read is None else f64(read))
                assert_close(x, want.reshape(n, -1), 2e-6)
                assert_close(h, P.rms_norm(u, f64(w), eps), 1e-5 if T == torch.float32 else 5e-3)
    x = cu(X.reshape(n, -1))
    ops.streams_norm(x, streams, cu(w), eps, torch.float32, write_back=False, **kw)
    assert torch.equal(x.cpu(), X.reshape(n, -1))


def test_streams_refuse_what_does_not_fit():
    from llama_cu_amd.kernels import ops
    x, w = torch.zeros(2, 24).cuda(), torch.zeros(8).cuda()
    for bad in (dict(streams=5), dict(streams=0), dict(delta=torch.zeros(2, 8).cuda()),
                dict(delta=torch.zeros(2, 9).cuda(), mix=torch.zeros(3, 3).cuda(), out_weights=torch.zeros(3).cuda()),
                dict(delta=torch.zeros(2, 8).cuda(), mix=torch.zeros(2, 3).cuda(), out_weights=torch.zeros(3).cuda())):
        with pytest.raises(ops.KernelError):
            ops.streams_norm(x, bad.pop("streams", 3), w, 1e-5, torch.float32, **bad)


@pytest.mark.parametrize("rows,packed,waits", [(3, True, False), (16, False, True), (29, True, True), (32, False, False)])
@pytest.mark.parametrize("streams", [1, 3, 4, 7])
def test_a_product_that_ends_in_the_streams_and_the_next_norm(rows, packed, waits, streams):
    from llama_cu_amd.kernels import ops
    n, k, eps = 192, 256, 1e-5
    x, w = rnd(rows, k, seed=1).bfloat16(), rnd(n, k, seed=2, std=0.1).bfloat16()
    X, mix, inn, out_w, nw = rnd(rows, streams, n, seed=3), rnd(streams, streams, seed=4), rnd(streams, seed=5), rnd(streams, seed=6), rnd(n, seed=7)
    y = f64(x.float()) @ f64(w.float()).T
    kw = {}
    if waits:                                                # the rows' own norm is a factor that the product applies
        shares = (x.float() ** 2).reshape(rows, 8, k // 8).sum(-1).contiguous()
        kw = dict(row_sumsq=shares.cuda(), norm_width=k, eps=eps)
        y = P.rms_div(f64(x.float()), eps) @ f64(w.float()).T
    want = P.update_streams(f64(X), f64(mix), f64(out_w), y)
    wg = ops.pack_weight(w.cuda()) if packed else w.cuda()
    for read in (inn, None):
        xs = X.reshape(rows, -1).cuda()
        h, sumsq = ops.gemm_skinny_streams(x.cuda(), wg, xs, streams, mix.cuda(), out_w.cuda(), None if read is None else read.cuda(), nw.cuda(),
                                           packed=packed, **kw)
        u = P.read_streams(want, np.ones(streams) if read is None else f64(read))
        assert_close(xs, want.reshape(rows, -1), 5e-6)
        assert_close(h, u * f64(nw), 5e-3)
        assert_close(sumsq.sum(1), (u ** 2).sum(1), 2e-5)
    with pytest.raises(ops.KernelError):
        ops.gemm_skinny_streams(x.cuda(), wg, xs, streams + 1, mix.cuda(), out_w.cuda(), None, nw.cuda(), packed=packed)


def attention_part(m, dtype, page, d=64, eps=1e-5, seed=11):
    from llama_cu_amd.parts import PartSpec
    from llama_cu_amd.models.lapunex import ATTENTION_NAMES
    w = mixer_weights(config(16, d, [both(m, right(1, 4, 4, 1.0), 1.0, 1.0)], eps, 1), seed, "l0.mix.left.")
    w["k.norm"] *= 2.0                                        # peaked scores
    w = {k: v.bfloat16().float() for k, v in w.items()}
    rot = m.get("rot")
    position = None if rot is None else PartSpec("rotary", {"head_dim": m["dim"], "theta": rot["base"], "rot_dim": rot["dims"],
                                                            "max_positions": 512, "yarn": rot.get("scaling")})
    part = built("mixer", "attention", {"hidden_size": d, "heads": m["heads"], "kv_heads": m["kv_heads"], "head_dim": m["dim"],
                                        "value_dim": m["vdim"], "scale": m["scale"], "position": position, "projection_norm_eps": eps,
                                        "sink": True, "head_gate": True, "names": ATTENTION_NAMES}, w, TYPES[dtype], page, pack=True)
    wn = as_numpy(w, "p.")
    return part, lambda h: P.attention(h, wn, "p.", m, eps)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("m,page", [
    (left(6, 2, 12, 20, 0.6, 8, 700.0, yarn(5.0, 48, 4.0, 0.25)), 16),         # a part of a head turned, stored at 32
    (left(8, 2, 64, 64, 0.25, 64, 5000.0, yarn(4.0, 64, 8.0, 0.5)), 32),       # whole heads
    (left(4, 1, 96, 48, 0.2, 40, 5000.0), 16),                                 # no blending; 20 pairs, values half as wide
    (left(3, 3, 16, 32, 0.5), 16),                                             # no rotation
    (left(1, 1, 4, 8, 1.0, 2, 50.0, yarn(2.0, 16, 1.0, 0.5)), 8),              # one head, one pair
    (left(2, 2, 6, 5, 1.0, 6, 50.0), 16),                                      # sizes that no piece of four fits
    (left(4, 2, 136, 96, 0.2, 24, 300.0, yarn(3.0, 30, 3.0, 0.3)), 16),        # too wide for the matrix-core kernels
    (left(18, 1, 16, 16, 0.5, 16, 300.0), 16),                                 # groups of eighteen heads (the generic kernel)
])
def test_attention_with_a_norm_over_the_projection_a_rotation_a_sink_and_a_gate_per_head(dtype, m, page):
    """Over shuffled pages among pages of NaN, in portions beside single tokens and whole; its rows times a factor as columns of a
    wider operand."""
    part, plain = attention_part(m, dtype, page)
    lens, tol = [150, 61], 5e-5 if dtype == "float32" else 6e-2
    rows = [rnd(n, 64, seed=60 + r).to(TYPES[dtype]) for r, n in enumerate(lens)]
    for steps in (None, [[(0, 0, lens[0]), (1, 0, lens[1])]]):
        feeder = Feeder(lens, page, seed=4, steps=steps)
        cache = part.cache_need().allocate(0, feeder.n_pages, page, 4, TYPES[dtype], torch.device("cuda"))
        cache.pages.fill_(float("nan"))

        def forward(step, x):
            part.prepare(step)
            out = part.forward(x.cuda(), step, cache, out_dtype=torch.float32)
            wide = torch.zeros(x.shape[0], part.output_width + 16, dtype=TYPES[dtype]).cuda()
            part.forward_rows(x.cuda(), step, cache, wide[:, 8:8 + part.output_width], 2.0)
            again = wide[:, 8:-8].float() @ part.output_matrix.float().T
            assert_close(again, 2.0 * out, 1e-5 if dtype == "float32" else 3e-2)
            assert wide[:, :8].abs().max() == 0 and wide[:, -8:].abs().max() == 0
            return out

        got = feeder.run(forward, rows)
        for r in range(2):
            assert_close(got[r], plain(f64(rows[r].float())), tol, f"request {r}, {'portions' if steps is None else 'whole'}")


LIGHTNING_SHAPES = [([0.5, 0.93, 0.998], 20, 12), ([0.9, 0.99, 0.7, 1.0], 32, 64), ([0.0, 0.9995], 64, 128), ([0.8], 1, 1), ([0.97, 0.2], 128, 40),
                    ([0.95], 140, 72), ([0.6, 0.99], 96, 96), ([0.99], 256, 17), ([0.9], 48, 300)]


def lightning_part(decay, dim, vdim, d, dtype, seed=13, pack=False, eps=1e-5):
    m = lightning(decay, dim, vdim)
    w = mixer_weights(config(16, d, [light(m)], eps, 1), seed)
    part = built("mixer", "lightning", {"hidden_size": d, "heads": len(decay), "head_dim": dim, "value_dim": vdim, "decay": decay, "norm_eps": eps},
                 w, TYPES[dtype], pack=pack)
    wn = as_numpy(w, "p.")
    return part, lambda h: P.lightning(h, wn, "p.", m, eps), w


def memory_part(heads, dim, vdim, cap, d, dtype, seed=14, pack=False, eps=1e-5, change=None):
    m = right(heads, dim, vdim, cap)
    w = mixer_weights(config(16, d, [both(left(1, 1, 8, 8, 1.0), m, 1.0, 1.0)], eps, 1), seed, "l0.mix.right.")
    if change is not None:
        change(w)
    part = built("mixer", "matrix_memory", {"hidden_size": d, "heads": heads, "head_dim": dim, "value_dim": vdim, "gate_cap": cap, "norm_eps": eps},
                 w, TYPES[dtype], pack=pack)
    wn = as_numpy(w, "p.")
    return part, lambda h: P.mlstm(h, wn, "p.", m, eps), w


def state_of(part, slots=3):
    """The mixer's state, filled with what another request may have left."""
    cache = part.cache_need().allocate(-1, 0, 0, slots, torch.float32, torch.device("cuda"))
    cache.state.normal_(0.0, 7.0)
    return cache


def in_portions(part, plain, lens, d, dtype, tol, steps=None, seed=20):
    rows = [rnd(n, d, seed=seed + r).to(TYPES[dtype]) for r, n in enumerate(lens)]
    cache = state_of(part)
    got = Feeder(lens, steps=steps).run(lambda step, x: part.forward(x.cuda(), step, cache, out_dtype=torch.float32), rows)
    for r in range(len(lens)):
        assert_close(got[r], plain(f64(rows[r].float())), tol, f"request {r}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decay,dim,vdim", LIGHTNING_SHAPES)
def test_linear_attention_with_a_fixed_decay_against_its_recurrence(dtype, decay, dim, vdim):
    """In portions and single tokens beside another request's, and in portions of chunks and more, from slots that held other values."""
    d = 56
    part, plain, _ = lightning_part(decay, dim, vdim, d, dtype, pack=True)
    tol = 3e-5 if dtype == "float32" else 4e-2
    in_portions(part, plain, [50, 27], d, dtype, tol)
    in_portions(part, plain, [300, 131], d, dtype, tol, steps=[[(0, 0, 64)], [(0, 64, 65), (1, 0, 2)], [(1, 2, 128), (0, 129, 1)], [(0, 130, 170), (1, 130, 1)]])


MEMORY_SHAPES = [(3, 20, 12, 5.0), (2, 64, 64, 12.0), (4, 32, 128, 15.0), (1, 4, 9, 1.0), (2, 128, 127, 8.0), (1, 140, 72, 6.0), (2, 96, 48, 3.0),
                 (1, 256, 33, 10.0)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,dim,vdim,cap", MEMORY_SHAPES)
def test_the_matrix_memory_against_its_recurrence(dtype, heads, dim, vdim, cap):
    d = 56
    part, plain, _ = memory_part(heads, dim, vdim, cap, d, dtype, pack=True)
    tol = 5e-5 if dtype == "float32" else 6e-2
    in_portions(part, plain, [50, 27], d, dtype, tol)
    in_portions(part, plain, [300, 131], d, dtype, tol, steps=[[(0, 0, 64)], [(0, 64, 65), (1, 0, 2)], [(1, 2, 128), (0, 129, 1)], [(0, 130, 170), (1, 130, 1)]])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["lightning", "memory"])
def test_long_portions_are_walked_in_runs(dtype, kind):
    """Portions of 256 tokens and more are walked in runs side by side and chained: a long portion from the start beside a short
    request, a second long one that goes on from the first's state beside another that starts, then single tokens."""
    d = 40
    for shape in ([([0.99, 0.6], 32, 24), ([0.999], 130, 70)] if kind == "lightning" else [(2, 32, 24, 6.0), (1, 130, 70, 9.0)]):
        part, plain, _ = (lightning_part if kind == "lightning" else memory_part)(*shape, d, dtype)
        steps = [[(0, 0, 513), (1, 0, 3)], [(1, 3, 525), (0, 513, 1087)], [(0, 1600, 1), (1, 528, 1)], [(0, 1601, 2), (1, 529, 4)]]
        in_portions(part, plain, [1603, 533], d, dtype, 5e-5 if dtype == "float32" else 6e-2, steps=steps, seed=30)


@pytest.mark.parametrize("kind", ["lightning", "memory"])
def test_a_token_far_back_is_remembered(kind):
    """With decays of nearly one, a strong key hundreds of tokens back still carries the output of a query that asks for it, in one
    portion (walked in runs), in portions and token by token."""
    d = 32
    if kind == "lightning":
        part, plain, w = lightning_part([0.9995], 16, 16, d, "float32")
    else:
        def open_gates(w):
            w["f"].zero_(); w["f.b"].fill_(9.0); w["i"].zero_(); w["i.b"].zero_()
        part, plain, w = memory_part(1, 16, 16, 12.0, d, "float32", change=open_gates)
    x = rnd(640, d, seed=15, std=0.1)
    x[20] = 30.0 * w["k"][0] / w["k"][0].norm()             # a key that stands out
    x[639] = 30.0 * w["q"][0] / w["q"][0].norm()
    want = plain(f64(x))
    without = x.clone()
    without[20] = 0.0
    assert np.abs(plain(f64(without))[639] - want[639]).max() > 0.1 * np.abs(want[639]).max()
    cache = state_of(part)
    for slot, cuts in ((0, [640]), (1, [300, 1, 2, 337]), (2, [600] + [1] * 40)):
        got, at = [], 0
        for take in cuts:
            got.append(part.forward(x[at:at + take].cuda(), hand_step([take], [at + take], [slot]), cache, out_dtype=torch.float32).clone())
            at += take
        assert_close(torch.cat(got), want, 5e-5, f"cut {len(cuts)}")


def test_gates_far_apart_overflow_nothing():
    """Forget gates that forget everything, input gates at both ends of the cap in turn: weights from e^-24 to e^24 in one state, in
    portions and token by token; the running maximum is carried from step to step."""
    d, cap = 24, 12.0

    def wild(w):
        w["i"] *= 40.0
        w["f"] *= 40.0
    part, plain, _ = memory_part(2, 8, 8, cap, d, "float32", change=wild)
    in_portions(part, plain, [90, 60], d, "float32", 1e-4, seed=40)
    in_portions(part, plain, [90, 60], d, "float32", 1e-4, steps=[[(0, 0, 90), (1, 0, 60)]], seed=40)
    x = rnd(30, d, seed=41)
    want = plain(f64(x))
    cache = state_of(part)
    got = [part.forward(x[t:t + 1].cuda(), hand_step([1], [t + 1], [1]), cache, out_dtype=torch.float32).clone() for t in range(30)]
    assert_close(torch.cat(got), want, 1e-4)


def test_single_tokens_of_many_requests_and_rows_that_wait_for_their_norm():
    """A step of single tokens: forty requests at different lengths (the norm applied by a kernel) and eight of them (by the output
    product), each against the plain recurrence."""
    d = 128
    for count in (40, 8):
        part, plain, _ = lightning_part([0.9, 0.99], 64, 64, d, "bfloat16", pack=True)
        mem, plain_mem, _ = memory_part(2, 64, 64, 9.0, d, "bfloat16", pack=True)
        lens = [3 + r % 5 for r in range(count)]
        rows = [rnd(n + 1, d, seed=100 + r).bfloat16() for r, n in enumerate(lens)]
        for p, reference in ((part, plain), (mem, plain_mem)):
            cache = state_of(p, count)
            p.forward(torch.cat([x[:-1] for x in rows]).cuda(), hand_step(lens, lens, list(range(count))), cache)
            got = p.forward(torch.stack([x[-1] for x in rows]).cuda(), hand_step([1] * count, [n + 1 for n in lens], list(range(count))), cache)
            for r in range(0, count, 3):
                assert_close(got[r], reference(f64(rows[r].float()))[-1], 3e-2, f"{count} requests, {r}")


@pytest.mark.parametrize("dtype,n,d,ff,experts,top,groups", [
    ("float32", 70, 64, 32, 12, 3, (3, 2)), ("float32", 9, 72, 24, 6, 6, (2, 2)), ("float32", 200, 40, 16, 4, 1, (4, 1)), ("bfloat16", 33, 64, 48, 12, 3, (4, 2)),
    ("bfloat16", 300, 76, 20, 9, 2, (3, 1)), ("float32", 5, 38, 8, 1, 1, None), ("bfloat16", 600, 128, 64, 8, 2, (4, 1)), ("float32", 40, 64, 16, 160, 5, (8, 3))])
def test_experts_within_groups_with_limits(dtype, n, d, ff, experts, top, groups):
    """Few and many rows an expert, widths that no 16 bytes fill; inputs that many of the limits cut; most tokens' best experts lie in more
    groups than are kept."""
    f = moe(experts, top, ff, 0.9, 1.7, groups)
    prefix = "l0.mlp."
    w = {k[len(prefix):]: v for k, v in random_weights(config(16, d, [light(lightning([0.5], 4, 4), f)], 1e-5, 1), 21).items() if k.startswith(prefix)}
    g = groups or (1, 1)
    from llama_cu_amd.models.lapunex import EXPERT_NAMES
    part = built("ffn", "gated_moe", {"hidden_size": d, "expert_size": ff, "experts": experts, "top": top, "router_bias": False, "scoring": "softmax_all",
                                      "renormalize": False, "scale": 1.7, "groups": g[0], "keep_groups": g[1], "activation": "limited",
                                      "alpha": 1.702, "limit": 0.9, "names": EXPERT_NAMES}, w, TYPES[dtype])
    h = rnd(n, d, seed=50).to(TYPES[dtype])
    wn = as_numpy(w, "p.")
    z = f64(h.float()) @ wn["p.router"].T
    if groups and groups[1] < groups[0] and top > 1:
        free = [set(P.route(row, top)[0]) for row in z]
        held = [set(P.route(row, top, f["router"]["groups"])[0]) for row in z]
        assert np.mean([a != b for a, b in zip(free, held)]) > 0.1
    want = P.experts(f64(h.float()), wn, "p.", f)
    tol = 3e-5 if dtype == "float32" else 4e-2
    got = part.forward(h.cuda())
    assert got.dtype == torch.float32
    assert_close(got, want, tol)
    base = rnd(n, d, seed=51).cuda()
    assert_close(part.forward(h.cuda(), add_to=base.clone()), want + f64(base.cpu()), tol, "added to another branch")
    if dtype == "float32":
        assert torch.equal(part.forward(h[:3].cuda()), got[:3])


def test_ties_between_groups_go_to_the_lower_index_and_the_scores_are_the_weights():
    from llama_cu_amd.kernels import ops
    h, router = torch.zeros(4, 16).cuda(), rnd(6, 16, seed=1).cuda()          # equal logits: equal scores
    ids, wts = ops.moe_route(h, router, 3, softmax_all=True, groups=3, keep=2, renorm=False, scale=2.0)
    assert ids.tolist() == [[0, 1, 2]] * 4
    assert_close(wts, torch.full((4, 3), 2.0 / 6), 1e-6)
    for bad in (dict(groups=4), dict(groups=3, keep=1), dict(groups=3, keep=4)):
        with pytest.raises(ops.KernelError):
            ops.moe_route(h, router, 3, softmax_all=True, **bad)
    with pytest.raises(ops.KernelError):
        ops.moe_route(h, router, 3, groups=3, keep=2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,i", [("A", 1), ("B", 1), ("C", 0), ("E", 0)])
def test_the_two_mixers_side_by_side(dtype, name, i):
    """One output product for both; the factors differ in size and sign."""
    cfg = CONFIGS[name]
    from llama_cu_amd.config import architecture_of
    arch = architecture_of(cfg)
    spec = arch.build_spec(arch.config_from_dict(cfg)).layers[i].params["mixer"]
    w = mixer_weights(cfg, 31, f"l{i}.mix.")
    part = built("mixer", "side_by_side", spec.params, w, TYPES[dtype], 16, pack=True)
    assert part.joint and all(m.w_o is None for m in part.mixers)
    lens = [70, 33]
    rows = [rnd(n, cfg["width"], seed=70 + r).to(TYPES[dtype]) for r, n in enumerate(lens)]
    feeder = Feeder(lens, 16, seed=4)
    cache = part.cache_need().allocate(0, feeder.n_pages, 16, 4, TYPES[dtype], torch.device("cuda"))
    cache.pages.fill_(float("nan"))
    for s in cache.more.values():
        s.normal_(0.0, 5.0)

    def forward(step, x):
        part.prepare(step)
        return part.forward(x.cuda(), step, cache, out_dtype=torch.float32)

    got = feeder.run(forward, rows)
    wn = as_numpy(w, "p.")
    for r in range(2):
        assert_close(got[r], P.parallel(f64(rows[r].float()), wn, "p.", cfg["layers"][i]["mixer"], cfg["norm"]["eps"]),
                     1e-4 if dtype == "float32" else 6e-2, f"request {r}")


# ------------------------------------------------------------------ whole models

_made = {}
# (heads of one or a few values are nearly signs behind their norm: seeds with which no head of the first tokens hangs on a rounding)
SEEDS = {"A": 8, "B": 2, "C": 3, "D": 4, "E": 5}


def model(name, sharp=1.0, steady=False):
    """(configuration, weights, folder) of a test model, made once.  ``steady``: for runs in bfloat16."""
    key = (name, sharp, steady)
    if key not in _made:
        cfg = sharpened(CONFIGS[name], sharp) if sharp != 1.0 else CONFIGS[name]
        w = random_weights(cfg, SEEDS[name], steady_router=steady)
        _made[key] = (cfg, w, make_folder(cfg, w))
    return _made[key]


def runner_for(folder, dtype, **kw):
    from llama_cu_amd.engine.runner import ModelRunner
    args = dict(dtype=dtype, page_size=16, max_tokens=1024, max_seqs=4, max_batch_tokens=1024)
    args.update(kw)
    return ModelRunner.from_folder(folder, **args)


@pytest.mark.parametrize("name,dtype", [(n, t) for n in sorted(CONFIGS) for t in ("float32", "bfloat16")])
def test_a_whole_prompt_against_the_plain_model(name, dtype):
    cfg, w, folder = model(name, steady=dtype == "bfloat16")
    toks = tokens_of(cfg["vocab"], 100, 1)
    r = runner_for(folder, dtype, page_size={"A": 16, "B": 32, "C": 48, "D": 64, "E": 16}[name])
    got = r.step([0], [toks], [list(range(len(toks)))])
    want = plain_logits(cfg, w, toks)
    assert_close(got, want, REL[dtype], f"model {name} in {dtype}")
    r.end(0)
    some = r.step([1], [toks], [[0, 57, 99]])               # rows of all streams gathered before the final norm
    assert_close(some, want[[0, 57, 99]], REL[dtype])
    r.end(1)
    r.cache.check()


@pytest.mark.parametrize("name,dtype", [("D", "float32"), ("E", "float32"), ("E", "bfloat16"), ("C", "float32"), ("D", "bfloat16")])
def test_models_of_one_kind_of_layer_and_the_first_tokens_of_a_sequence(name, dtype):
    """Recurrent layers alone (no pages at all) and layers with pages: a prompt in portions, then tokens one by one, a second request
    beside the first that starts with portions of one and two tokens, pages and slots used again."""
    cfg, w, folder = model(name, steady=dtype == "bfloat16")
    a, b = tokens_of(cfg["vocab"], 40, 50), tokens_of(cfg["vocab"], 21, 51)
    r = runner_for(folder, dtype, max_seqs=2, max_tokens=128)
    wa, wb = plain_logits(cfg, w, a), plain_logits(cfg, w, b)
    got_a = [r.step([0], [a[:17]], [list(range(17))]).clone()]
    out = r.step([0, 1], [a[17:30], b[:1]], [list(range(13)), [0]]).clone()
    got_a.append(out[:13])
    got_b = [out[13:]]
    out = r.step([1, 0], [b[1:3], a[30:31]], [[0, 1], [0]]).clone()
    got_b.append(out[:2]); got_a.append(out[2:])
    got_b.append(r.step([1], [b[3:]], [list(range(18))]).clone())
    r.end(1)
    got_a += [r.step([0], [[t]], [[0]]).clone() for t in a[31:]]
    assert_close(torch.cat(got_a), wa, REL[dtype], "first request")
    assert_close(torch.cat(got_b), wb, REL[dtype], "second request")
    again = r.step([2], [b], [list(range(21))])          # in the slot and the pages that the second request held
    assert_close(again, wb, REL[dtype], "the slot and pages used again")
    r.cache.check()


@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("B", "bfloat16"), ("C", "float32"), ("B", "float32"), ("A", "bfloat16")])
def test_prefill_against_token_by_token_decoding_and_portions_down_to_two_tokens(name, dtype):
    cfg, w, folder = model(name, steady=dtype == "bfloat16")
    toks = tokens_of(cfg["vocab"], 90, 2)
    r = runner_for(folder, dtype)
    whole = r.step([0], [toks], [list(range(len(toks)))]).clone()
    assert_close(whole, plain_logits(cfg, w, toks), REL[dtype], "the whole prompt")
    # one token at a time from the first (long enough for captured graphs to replay)
    single = torch.cat([r.step([1], [[t]], [[0]]).clone() for t in toks])
    sizes, at, parts = [2, 3, 5, 1, 17, 2, 31, 4, 2, 1, 64], 0, []
    for k in range(100):
        if at >= len(toks):
            break
        take = toks[at:at + sizes[k % len(sizes)]]
        parts.append(r.step([2], [take], [list(range(len(take)))]).clone())
        at += len(take)
    assert_close(single, whole, SAME[dtype], "token by token against the whole prompt")
    assert_close(torch.cat(parts), whole, SAME[dtype], "portions against the whole prompt")
    assert r.use_graphs and sum(r.graph_replays.values()) > 50, "decoding was not replayed from captured graphs"
    for i in range(3):
        r.end(i)
    r.cache.check()


@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("B", "float32"), ("B", "bfloat16")])
def test_batches_of_unequal_requests_and_pages_and_slots_used_again(name, dtype):
    """Seven requests of unequal lengths through an engine with three slots and a pool that holds only what is live:
    portions of some beside single tokens of others; finished requests give their pages and slots to new ones (pages
    that change hands are filled with NaN first; a slot keeps what its last owner left).  Every request's logits equal
    those it gets alone."""
    cfg, w, folder = model(name, sharp=(10.0 if name == "A" else 3.0) if dtype == "float32" else 1.5, steady=dtype == "bfloat16")
    lens = [70, 33, 1, 48, 19, 90, 7]
    reqs = [tokens_of(cfg["vocab"], n, 10 + i) for i, n in enumerate(lens)]
    r = runner_for(folder, dtype, max_seqs=3, max_tokens=3 * 96, max_batch_tokens=256, poison_freed=True)
    if dtype == "float32":
        want = [plain_logits(cfg, w, t) for t in reqs]
    else:       # each alone through the engine: a bfloat16 run is compared with another of its own
        want = []
        for i, t in enumerate(reqs):
            want.append(r.step([100 + i], [t], [list(range(len(t)))]).clone())
            r.end(100 + i)
    rng = random.Random(3)
    waiting, live, done = list(range(len(reqs))), {}, {i: [] for i in range(len(reqs))}
    pages_seen = [dict() for _ in r.groups]
    slots_seen = {}
    while waiting or live:
        while waiting and len(live) < 3:
            live[waiting.pop(0)] = 0
        ids, toks = [], []
        for i, at in live.items():
            left_over = len(reqs[i]) - at
            take = 1 if (left_over <= 12 or rng.random() < 0.3) else min(left_over - 12, rng.choice([2, 3, 9, 16, 25]))
            ids.append(i); toks.append(reqs[i][at:at + take])
        ctx = r.prepare(ids, toks, [list(range(len(t))) for t in toks])
        for i, s in zip(ids, ctx.state_slots):
            slots_seen.setdefault(s, set()).add(i)
        out = r.run(ctx).clone()
        for i in ids:
            r.cache.commit(i)
        for g, seen in enumerate(pages_seen):
            for page, owner in enumerate(r.cache.page_owners(g)):
                if owner >= 0:
                    seen.setdefault(page, set()).add(owner)
        at = 0
        for i, t in zip(ids, toks):
            done[i].append(out[at:at + len(t)])
            at += len(t)
            live[i] += len(t)
            if live[i] == len(reqs[i]):
                del live[i]
                r.end(i)
        r.cache.check()
    assert len(r.groups) == 1
    for g, seen in enumerate(pages_seen):
        assert max(len(v) for v in seen.values()) >= 2, f"no page of pool {g} was used again"
    assert max(len(v) for v in slots_seen.values()) >= 2, "no state slot was used again"
    for i in range(len(reqs)):
        assert_close(torch.cat(done[i]), want[i], REL[dtype] if dtype == "float32" else SAME[dtype], f"request {i} of {lens[i]} tokens")


@pytest.mark.parametrize("name", ["A", "B", "E"])
def test_keys_far_back_and_at_the_borders_of_pages_and_chunks(name):
    """Peaked scores make single keys carry an output, so one that is lost or misplaced shows; 330 tokens over pages of 16 and chunks
    of 16 to 64, cut inside both, the last 70 decoded one by one: every position's logits against the plain model."""
    cfg, w, folder = model(name, sharp=14.0 if name == "A" else 4.0)
    toks = tokens_of(cfg["vocab"], 330, 7)
    want = plain_logits(cfg, w, toks)
    r = runner_for(folder, "float32")
    parts = [r.step([0], [toks[:127]], [list(range(127))]).clone(), r.step([0], [toks[127:260]], [list(range(133))]).clone()]
    parts += [r.step([0], [[t]], [[0]]).clone() for t in toks[260:]]
    assert_close(torch.cat(parts), want, 2 * REL["float32"], "far keys")
    r.end(0)
    r.cache.check()


def test_planted_faults_show():
    """The inputs above are sharp enough: the plain model with a fault planted in it differs by far more than the tolerance."""
    cfg, w, _ = model("A", sharp=14.0)
    toks = tokens_of(cfg["vocab"], 120, 7)
    want = plain_logits(cfg, w, toks)

    def off(changed_cfg=None, **changed):
        got = plain_logits(changed_cfg or cfg, {k: changed.get(k.replace(".", "_"), v) for k, v in w.items()}, toks)
        return ((got - want).abs().max() / want.abs().max()).item()

    def with_cfg(change):
        c = copy.deepcopy(cfg)
        change(c["layers"])
        return off(c)

    faults = {
        "a sink left out": off(l1_mix_left_sink=torch.full((6,), -50.0)),
        "frequencies not blended": with_cfg(lambda l: l[1]["mixer"]["left"]["rot"].pop("scaling")),
        "groups forgotten": with_cfg(lambda l: l[1]["mlp"]["router"].pop("groups")),
        "another factor on the router": with_cfg(lambda l: l[1]["mlp"]["router"].update(scale=1.6)),
        "a decay that forgets": with_cfg(lambda l: l[0]["mixer"].update(decay=[0.5, 0.93, 0.9])),
        "limits forgotten": with_cfg(lambda l: l[1]["mlp"]["expert"].update(limit=100.0)),
        "the matrix between the streams turned round": off(l1_hc1_mix=w["l1.hc1.mix"].T.contiguous()),
        "a memory that keeps everything": off(l1_mix_right_f_b=torch.full((3,), 30.0)),
    }
    assert all(v > 20 * REL["float32"] for v in faults.values()), faults


def test_long_decoding_in_bfloat16():
    cfg, w, folder = model("B", steady=True)
    toks = tokens_of(cfg["vocab"], 260, 8)
    r = runner_for(folder, "bfloat16")
    want = r.step([1], [toks], [list(range(260))]).clone()
    got = [r.step([0], [toks[:20]], [list(range(20))]).clone()] + [r.step([0], [[t]], [[0]]).clone() for t in toks[20:]]
    assert_close(torch.cat(got), want, SAME["bfloat16"], "long decoding against the whole prompt")
    assert_close(want, plain_logits(cfg, w, toks), REL["bfloat16"], "the whole prompt against the plain model")
    assert sum(r.graph_replays.values()) > 100, "decoding was not replayed from captured graphs"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_prompt_whose_portions_are_walked_in_runs(dtype):
    """A prompt of 1,200 tokens in one step, and the same in portions of 700 and 498 and two single tokens."""
    cfg, w, folder = model("B", steady=dtype == "bfloat16")
    toks = tokens_of(cfg["vocab"], 1200, 9)
    want = plain_logits(cfg, w, toks)
    r = runner_for(folder, dtype, max_tokens=2560, max_batch_tokens=1280)
    places = list(range(0, 1200, 7)) + [1199]
    whole = r.step([0], [toks], [places]).clone()
    assert_close(whole, want[places], REL[dtype], "the whole prompt")
    out = [r.step([1], [toks[:700]], [[699]]).clone(), r.step([1], [toks[700:1198]], [[497]]).clone()]
    out += [r.step([1], [[t]], [[0]]).clone() for t in toks[1198:]]
    assert_close(torch.cat(out), want[[699, 1197, 1198, 1199]], REL[dtype], "in portions")


def test_many_requests_decoding_together():
    """Forty requests in one step of single tokens (the products for tens of rows, planes of partial sums that enter the streams), against
    the same requests decoded a few at a time."""
    cfg = config(96, 512, [
        light(lightning([0.9, 0.99, 0.95, 0.7], 128, 128), dense(4096)),
        both(left(4, 2, 128, 128, 0.1, 64, 5000.0, yarn(4.0, 64, 8.0, 0.5)), right(4, 128, 128, 9.0), 0.7, 0.9, moe(8, 2, 128, 2.0, 1.5, (4, 2))),
        light(lightning([0.99] * 8, 64, 64), dense(4096))], eps=1e-6, streams=3, loop=(0, 2, 2))
    w = random_weights(cfg, 21, steady_router=True)
    r = runner_for(make_folder(cfg, w), "bfloat16", max_seqs=44, max_tokens=44 * 64)
    prompts = [tokens_of(96, 20 + i % 7, 100 + i) for i in range(40)]
    tails = [tokens_of(96, 4, 200 + i) for i in range(40)]
    for i in range(0, 40, 8):
        r.step(list(range(i, i + 8)), prompts[i:i + 8], [[]] * 8)
    together = [r.step(list(range(40)), [[t[k]] for t in tails], [[0]] * 40).clone() for k in range(4)]
    for i in range(40):
        r.end(i)
    for i in range(0, 40, 4):
        r.step(list(range(i, i + 4)), prompts[i:i + 4], [[]] * 4)
    for k in range(4):
        apart = torch.cat([r.step(list(range(i, i + 4)), [[t[k]] for t in tails[i:i + 4]], [[0]] * 4).clone() for i in range(0, 40, 4)])
        assert_close(together[k], apart, SAME["bfloat16"], f"token {k}")
    plain = plain_logits(cfg, w, prompts[3] + tails[3])[-4:]
    assert_close(torch.stack([t[3] for t in together]), plain, REL["bfloat16"], "against the plain model")


def test_few_rows_end_in_the_streams_within_their_products(monkeypatch):
    """Single tokens and a short portion of a model whose feed-forwards are dense: every sublayer but those in front of experts ends
    in the next norm, and the last one in the final norm."""
    from llama_cu_amd.kernels import ops
    cfg = config(96, 256, [
        light(lightning([0.9, 0.99], 64, 64), dense(256)),
        both(left(4, 2, 64, 64, 0.12, 64, 5000.0, yarn(4.0, 64, 8.0, 0.5)), right(2, 64, 64, 9.0), 0.7, 0.9, dense(512)),
        light(lightning([0.95, 0.6], 64, 64))], eps=1e-6, streams=3, loop=(0, 2, 2))
    w = random_weights(cfg, 22)
    r = runner_for(make_folder(cfg, w), "bfloat16")
    r.use_graphs = False
    toks = tokens_of(96, 40, 60)
    want = plain_logits(cfg, w, toks)
    calls, real = [], ops.gemm_skinny_streams

    def counted(*a, **kw):
        calls.append(kw.get("row_sumsq") is not None)
        return real(*a, **kw)

    monkeypatch.setattr(ops, "gemm_skinny_streams", counted)
    got = []
    for at in range(0, 30, 6):
        calls.clear()
        got.append(r.step([0], [toks[at:at + 6]], [list(range(6))]).clone())
        assert len(calls) == 9 and not any(calls)            # (a portion: the lightning layers' norm is made by their own kernel)
    for t in toks[30:]:
        calls.clear()
        got.append(r.step([0], [[t]], [[0]]).clone())
        assert len(calls) == 9 and sum(calls) == 3
    assert_close(torch.cat(got), want, REL["bfloat16"])


def test_logits_do_not_depend_on_the_cut_or_the_batch_in_32_bit():
    cfg, w, folder = model("A")
    a, b = tokens_of(cfg["vocab"], 60, 20), tokens_of(cfg["vocab"], 41, 21)
    r = runner_for(folder, "float32")
    alone = r.step([0], [a], [list(range(60))]).clone()
    r.step([1], [b[:30]], [[]])
    p1 = r.step([2, 1], [a[:17], b[30:31]], [list(range(17)), [0]]).clone()
    p2 = r.step([1, 2], [b[31:], a[17:]], [[], list(range(43))]).clone()
    assert_close(torch.cat([p1[:17], p2]), alone, 2e-5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine_and_its_scheduler(dtype):
    """The framework's entry point: prompts of unequal lengths, more than run at a time, prefilled in portions; the
    generated tokens equal the plain model's arg-max continuation."""
    from llama_cu_amd.engine.engine import Engine
    cfg, w, folder = model("B", steady=dtype == "bfloat16")
    prompts = [tokens_of(cfg["vocab"], n, 30 + i) for i, n in enumerate([21, 5, 40, 2, 13])]
    steps = 12
    engine = Engine.from_folder(folder, dtype=dtype, page_size=16, max_tokens=512, max_seqs=3, prefill_chunk=16)
    got = engine.generate(prompts, max_steps=steps, ignore_eos=True)
    for k, (p, g) in enumerate(zip(prompts, got)):
        assert len(g) == steps
        seq = list(p) + list(g)
        logits = plain_logits(cfg, w, seq)[list(range(len(p) - 1, len(seq) - 1))]
        if dtype == "float32":
            assert torch.argmax(logits, -1).tolist() == list(g), f"prompt {k}"
        else:               # a close call may fall the other way
            for j, tok in enumerate(g):
                assert logits[j].max() - logits[j, tok] <= 0.08 * logits[j].abs().max(), f"prompt {k}, token {j}: {tok} is not the best"
    engine.runner.cache.check()


def test_trace_replay_of_the_design():
    """The replay program's own path: steps as JSON objects, logits as arrays; a pool for what is live and four slots, so
    that pages and slots change hands."""
    from llama_cu_amd.engine.trace import TraceReplayer
    cfg, w, folder = model("A")
    seqs = {n: tokens_of(cfg["vocab"], k, 40 + i) for i, (n, k) in enumerate([("x", 50), ("y", 30), ("z", 64), ("u", 9), ("v", 40)])}
    rep = TraceReplayer.open(folder, "float32", 256, max_live=4)
    out0 = rep.step({"step": 0, "entries": [{"id": "x", "tokens": seqs["x"][:33], "want": [0, 32]}], "end": []})
    out1 = rep.step({"step": 1, "entries": [{"id": "x", "tokens": seqs["x"][33:], "want": [16]}, {"id": "y", "tokens": seqs["y"], "want": [29]},
                                            {"id": "z", "tokens": seqs["z"], "want": [63]}, {"id": "u", "tokens": seqs["u"][:2], "want": []}],
                     "end": ["x", "y"]})
    out2 = rep.step({"step": 2, "entries": [{"id": "u", "tokens": seqs["u"][2:], "want": [6]}, {"id": "v", "tokens": seqs["v"], "want": [0, 39]}],
                     "end": ["u", "v", "z"]})
    want = {n: plain_logits(cfg, w, t) for n, t in seqs.items()}
    assert_close(out0, want["x"][[0, 32]], REL["float32"])
    assert_close(out1, torch.stack([want["x"][49], want["y"][29], want["z"][63]]), REL["float32"])
    assert_close(out2, torch.stack([want["u"][8], want["v"][0], want["v"][39]]), REL["float32"])
    assert rep.pages_used_again(0) > 0


def test_the_command_line_writes_a_random_model_generates_from_it_and_replays_a_trace(tmp_path):
    """``random-model`` writes a folder of the design from a configuration; ``generate`` continues a prompt from it;
    ``bin/trace_run`` (the program itself, steps on its standard input) gives the plain model's logits for the folder's
    weights."""
    import json
    import os
    import subprocess

    from llama_cu_amd.weights import open_safetensors
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = config(288, 96, [
        light(lightning([0.9, 0.99, 0.5], 32, 32), moe(6, 2, 32, 2.0, 1.5, (3, 2))),
        both(left(4, 2, 24, 32, 0.2, 16, 2000.0, yarn(3.0, 64, 8.0, 0.5)), right(3, 16, 24, 7.0), 0.8, 1.1, dense(64))],
        eps=1e-5, streams=2, scale=1.5, loop=(0, 2, 2))
    cfg_path, folder, out = str(tmp_path / "c.json"), str(tmp_path / "m"), str(tmp_path / "out")
    with open(cfg_path, "w") as f:
        json.dump(cfg, f)
    tool = os.path.join(root, "bin", "llama.cu_amd")
    p = subprocess.run([tool, "random-model", cfg_path, folder, "--seed", "3", "--std", "0.1"], capture_output=True, timeout=300)
    assert p.returncode == 0, p.stderr.decode()[-2000:]
    p = subprocess.run([tool, "generate", folder, "--max-steps", "6", "-p", "Hi", "--dtype", "float32", "--max-tokens", "256",
                        "--max-seqs", "2"], capture_output=True, timeout=300)
    assert p.returncode == 0, p.stderr.decode()[-2000:]
    assert p.stdout.startswith(b"Hi") and b"n toks = 6" in p.stderr
    files = open_safetensors(folder)
    w = {n: f.tensor(n).float() for f in files for n in f.names()}
    a, b = tokens_of(288, 30, 60), tokens_of(288, 12, 61)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:19], "want": [18]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[19:], "want": [0, 10]}, {"id": "b", "tokens": b, "want": [11]}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": [5], "want": [0]}], "end": ["b"]}]
    p = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", out,
                        "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps).encode(), capture_output=True, timeout=300)
    assert p.returncode == 0, p.stderr.decode()[-2000:]
    assert [l for l in p.stdout.decode().splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = plain_logits(cfg, w, a), plain_logits(cfg, w, b + [5])
    got = [torch.from_numpy(np.fromfile(os.path.join(out, f"{k}.f32"), dtype="<f4").reshape(-1, 288)) for k in range(3)]
    assert_close(got[0], wa[[18]], REL["float32"])
    assert_close(got[1], torch.stack([wa[19], wa[29], wb[11]]), REL["float32"])
    assert_close(got[2], wb[[12]], REL["float32"])
