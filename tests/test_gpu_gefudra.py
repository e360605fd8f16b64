"""The Gefudra design on the GPU against the plain implementation of ``plain_gefudra.py``: every mechanism alone, then
whole models through the engine's own step function, cache manager and scheduler, cut and batched in every way that
must not change a token's logits."""
from __future__ import annotations

import random

import numpy as np
import pytest
import torch

import plain_gefudra as P
from gefudra_common import (CONFIGS, Feeder, as_numpy, assert_close, built, config, differential, hand_step, latent, layer, make_folder,
                            mixer_weights, plain_logits, random_weights, sharpened, tokens_of, wkv)

pytestmark = pytest.mark.gpu
TYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
REL = {"float32": 3e-4, "bfloat16": 7e-2}         # of the largest expected value
SAME = {"float32": 3e-5, "bfloat16": 5e-2}        # between two runs of the engine that cut or batch the same tokens differently


def rnd(*shape, seed=0, std=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * std


def f64(t):
    return t.double().numpy()


# ------------------------------------------------------------------ mechanisms alone


@pytest.mark.parametrize("d", [72, 128, 2048])
def test_a_factor_on_a_branchs_output_where_the_norm_adds_it(d):
    """Rows in either type and planes of partial sums enter the stream times the factor; 32-bit output beside a bfloat16
    branch."""
    from llama_cu_amd.kernels import ops
    n, scale, eps = 9, 0.7, 1e-5
    x, w = rnd(n, d, seed=1), rnd(d, seed=2)
    for dt, out_dt in ((torch.bfloat16, torch.float32), (torch.bfloat16, torch.bfloat16), (torch.float32, torch.float32)):
        delta = rnd(n, d, seed=3).to(dt)
        xs, out = x.clone().cuda(), torch.empty(n, d, dtype=out_dt).cuda()
        ops.rmsnorm(xs, w.cuda(), eps, out, delta=delta.cuda(), delta_scale=scale)
        want = f64(x) + scale * f64(delta.float())
        assert_close(xs, want, 1e-6)
        assert_close(out, P.rms_norm(want, f64(w), eps), 2e-6 if out_dt == torch.float32 else 5e-3)
    planes = rnd(5, n, d, seed=4)
    for out_dt in (torch.float32, torch.bfloat16):
        xs, out = x.clone().cuda(), torch.empty(n, d, dtype=out_dt).cuda()
        ops.rmsnorm(xs, w.cuda(), eps, out, delta=planes.cuda(), delta_scale=scale)
        want = f64(x) + scale * f64(planes).sum(0)
        assert_close(xs, want, 2e-6)
        assert_close(out, P.rms_norm(want, f64(w), eps), 2e-6 if out_dt == torch.float32 else 5e-3)
    xs = x.clone().cuda()
    ops.residual_add(xs, delta.cuda(), scale)
    assert_close(xs, f64(x) + scale * f64(delta), 1e-6)


@pytest.mark.parametrize("rows,packed", [(3, True), (16, False), (29, True)])
def test_a_factor_on_a_branchs_output_where_a_product_ends_in_the_norm(rows, packed):
    from llama_cu_amd.kernels import ops
    n, k, scale = 128, 256, 0.35
    x, w, nw, res = rnd(rows, k, seed=1).bfloat16(), rnd(n, k, seed=2, std=0.1).bfloat16(), rnd(n, seed=3), rnd(rows, n, seed=4)
    want = f64(res) + scale * (f64(x.float()) @ f64(w.float()).T)
    wg = ops.pack_weight(w.cuda()) if packed else w.cuda()
    for kernel in (ops.gemm_skinny_add_norm, ops.gemm_mid_add_norm):
        r = res.clone().cuda()
        h, sumsq = kernel(x.cuda(), wg, r, nw.cuda(), packed=packed, scale=scale)
        assert_close(r, want, 2e-6)
        assert_close(h, want * f64(nw), 5e-3)
        assert_close(sumsq.sum(1), (want ** 2).sum(1), 1e-5)


@pytest.mark.parametrize("dtype,planes", [("float32", 0), ("bfloat16", 0), ("bfloat16", 3), ("float32", 2), ("float32", None)])
@pytest.mark.parametrize("d,n", [(72, 5), (128, 40), (18, 3)])
def test_the_mix_of_the_stream_with_the_embeddings_output(dtype, planes, d, n):
    w = rnd(d, 2 * d, seed=1, std=0.1).bfloat16().float()
    part = built("stream", "remix", {"hidden_size": d, "tensor": "in", "delta_scale": 0.6}, {"in": w}, TYPES[dtype])
    x0, x = rnd(n, d, seed=2).bfloat16().float(), rnd(n, d, seed=3)
    both = part.begin(x0.cuda())
    for again in range(2):                                  # the right half serves every run
        if planes is None:
            delta, add = None, 0.0
        elif planes:
            delta = rnd(planes, n, d, seed=4 + again)
            add = f64(delta).sum(0)
        else:
            delta = rnd(n, d, seed=4 + again).to(TYPES[dtype])
            add = f64(delta.float())
        got = part.forward(x.clone().cuda(), None if delta is None else delta.cuda(), both)
        want = np.concatenate([f64(x) + 0.6 * add, f64(x0)], -1) @ f64(w).T
        assert got.dtype == torch.float32
        assert_close(got, want, 3e-6 if dtype == "float32" else 8e-3, f"run {again}")


@pytest.mark.parametrize("dtype,n,d,ff", [("float32", 9, 72, 40), ("float32", 70, 128, 256), ("bfloat16", 9, 72, 40), ("bfloat16", 3, 128, 256),
                                          ("bfloat16", 20, 128, 4096), ("bfloat16", 60, 128, 4096), ("bfloat16", 150, 128, 4096),
                                          ("bfloat16", 300, 128, 264)])
def test_the_limited_feed_forward(dtype, n, d, ff):
    """The activation kernel and the epilogues of both products for few and for tens of rows; inputs that many of the limits cut."""
    w = {"gate": rnd(ff, d, seed=1, std=0.3), "up": rnd(ff, d, seed=2, std=0.3), "down": rnd(d, ff, seed=3, std=ff ** -0.5)}
    w = {k: v.bfloat16().float() for k, v in w.items()}
    part = built("ffn", "swiglu", {"hidden_size": d, "intermediate_size": ff, "names": {k: k for k in w}, "activation": "limited",
                                   "alpha": 1.702, "limit": 1.9}, w, TYPES[dtype], pack=True)
    h = rnd(n, d, seed=4).to(TYPES[dtype])
    want = P.feed_forward(f64(h.float()), as_numpy(w, "f."), "f.", {"limit": 1.9})
    gate, up = f64(h.float()) @ f64(w["gate"]).T, f64(h.float()) @ f64(w["up"]).T
    assert (gate > 1.9).mean() > 0.05 and (abs(up) > 1.9).mean() > 0.1
    assert_close(part.forward(h.cuda()), want, 1e-5 if dtype == "float32" else 2e-2)


def test_the_limited_activation_needs_a_limit_and_rows_that_wait_for_their_norm_take_it():
    from llama_cu_amd.kernels import ops
    from llama_cu_amd.parts import PartSpec, ScaledRows, make_part
    with pytest.raises(ValueError):
        make_part("ffn", PartSpec("swiglu", {"hidden_size": 8, "intermediate_size": 8, "activation": "limited"}))
    d, ff, n = 128, 4096, 11
    w = {"gate": rnd(ff, d, seed=1, std=0.3).bfloat16().float(), "up": rnd(ff, d, seed=2, std=0.3).bfloat16().float(),
         "down": rnd(d, ff, seed=3, std=0.02).bfloat16().float()}
    part = built("ffn", "swiglu", {"hidden_size": d, "intermediate_size": ff, "names": {k: k for k in w}, "activation": "limited",
                                   "alpha": 1.702, "limit": 1.1}, w, torch.bfloat16, pack=True)
    for rows in (n, 30):                                       # the product for few rows, and the one that shares them
        x = rnd(rows, d, seed=5).bfloat16()
        sumsq = (x.float() ** 2).reshape(rows, 8, 16).sum(-1).contiguous()
        assert part.takes_scaled_rows(rows)
        got = part.forward(ScaledRows(x.cuda(), sumsq.cuda(), d, 1e-5))
        want = P.feed_forward(P.rms_div(f64(x.float()), 1e-5), as_numpy(w, "f."), "f.", {"limit": 1.1})
        assert_close(got, want, 2e-2)
    with pytest.raises(ops.KernelError):
        ops.swiglu(torch.zeros(2, 8).cuda(), activation="limited")


@pytest.mark.parametrize("dtype,groups,m,rows,k", [
    ("bfloat16", 4, 8, 64, 128), ("bfloat16", 3, 20, 48, 128), ("bfloat16", 4, 3, 32, 40), ("bfloat16", 2, 90, 64, 128), ("bfloat16", 3, 33, 20, 24),
    ("bfloat16", 5, 7, 20, 20), ("float32", 3, 9, 20, 28), ("float32", 2, 70, 64, 128), ("float32", 3, 5, 7, 9)])
@pytest.mark.parametrize("gated", [False, True])
def test_products_of_several_matrices_each_with_rows_of_its_own(dtype, groups, m, rows, k, gated):
    """Also from columns of wider rows (a head's part of every row); with the gate in the epilogue, or behind the product."""
    from llama_cu_amd.parts import BuildContext
    from llama_cu_amd.parts.linear import GroupWeight, linear_groups
    T = TYPES[dtype]
    w = rnd(groups, rows, k, seed=1, std=k ** -0.5).to(T)
    weight = GroupWeight(w.cuda(), BuildContext(T, torch.device("cuda"), 64, 16, True))
    wide = rnd(m, groups * (k + 8), seed=2).to(T)
    x = wide.view(m, groups, k + 8)[:, :, :k].permute(1, 0, 2)
    want = np.concatenate([f64(x[i].float()) @ f64(w[i].float()).T for i in range(groups)], -1)
    g = rnd(m, groups * rows + 16, seed=3, std=2.0).to(T)
    if gated:
        want = want * P.sigmoid(f64(g[:, 16:].float()))
    out = torch.empty(m, groups * rows, dtype=T).cuda()
    got = linear_groups(wide.cuda().view(m, groups, k + 8)[:, :, :k].permute(1, 0, 2), weight, out, gate=g.cuda()[:, 16:] if gated else None)
    assert_close(got, want, 3e-6 if dtype == "float32" else 8e-3)
    if not gated:
        planes = rnd(groups, m, k, seed=4).to(T)             # rows of each group one after the other
        want = np.concatenate([f64(planes[i].float()) @ f64(w[i].float()).T for i in range(groups)], -1)
        assert_close(linear_groups(planes.cuda(), weight, out), want, 3e-6 if dtype == "float32" else 8e-3)


def attention_alone(part, plain, lens, dtype, page, tol, d, seed):
    """A mixer with pages alone: shuffled pages among pages of NaN, in portions beside single tokens, then whole prompts."""
    rows = [rnd(n, d, seed=seed + r).to(TYPES[dtype]) for r, n in enumerate(lens)]
    whole = [[(0, 0, lens[0]), (1, 0, lens[1])]]
    for steps in (None, whole):
        feeder = Feeder(lens, page, seed=4, steps=steps)
        cache = part.cache_need().allocate(0, feeder.n_pages, page, 4, TYPES[dtype], torch.device("cuda"))
        cache.pages.fill_(float("nan"))

        def forward(step, x):
            part.prepare(step)
            return part.forward(x.cuda(), step, cache, out_dtype=torch.float32)

        got = feeder.run(forward, rows)
        for r in range(2):
            assert_close(got[r], plain(f64(rows[r].float())), tol, f"request {r}, {'portions' if steps is None else 'whole'}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("m,page,folded", [
    (latent(3, 20, 12, 28, 36, 2.0, 19), 16, True),        # a latent that is filled up with zeros; folded queries as one matrix
    (latent(2, 8, 20, 44, 24, 1.5), 16, False),            # folded head by head; no window
    (latent(4, 64, 64, 128, 48, 0.5, 33), 32, True),       # the largest latent of the matrix-core kernels
    (latent(4, 32, 48, 96, 80, 0.8, 50), 16, False),
    (latent(1, 4, 8, 8, 4, 3.0, 1), 8, True),              # one head, a window of one key
    (latent(20, 8, 8, 32, 16, 1.0, 16), 16, False),        # groups of twenty heads (the generic kernel)
    (latent(2, 16, 24, 200, 20, 0.7, 48), 16, False),      # a latent wider than any head of the matrix-core kernels
])
def test_latent_attention_without_positions(dtype, m, page, folded):
    """Peaked scores and sinks as large as a good key's score: a key that is lost, seen too early or kept too long, and a sink
    that is left out, shows."""
    d, eps = 64, 1e-5
    cfg = config(16, d, [layer("latent_attention", m)], eps)
    w = mixer_weights(cfg, 11)
    part = built("mixer", "latent_attention", {
        "hidden_size": d, "heads": m["heads"], "head_dim": m["dim"], "rot_dim": 0, "value_dim": m["vdim"], "kv_rank": m["kv_rank"],
        "q_rank": m["q_rank"], "scale": m["scale"], "norm_eps": eps, "window": m["mask"]["size"] if "mask" in m else 0, "sink": True,
        "gate": True}, w, TYPES[dtype], page, pack=True)
    assert (part.w_folded_q is not None) == folded or dtype == "bfloat16"      # (a stored latent filled up may turn the choice)
    wn = as_numpy(w, "p.")
    attention_alone(part, lambda h: P.latent_attention(h, wn, "p.", m, eps), [150, 61], dtype, page, 3e-5 if dtype == "float32" else 6e-2, d, 60)


def test_latent_attention_with_a_turned_part_takes_no_query_latent():
    from llama_cu_amd.parts import PartSpec, make_part
    with pytest.raises(ValueError):
        make_part("mixer", PartSpec("latent_attention", {"hidden_size": 8, "heads": 1, "head_dim": 4, "rot_dim": 4, "value_dim": 4, "kv_rank": 8,
                                                         "scale": 1.0, "theta": 10.0, "max_positions": 8, "norm_eps": 1e-5, "q_rank": 4}))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("m,page,joint", [
    (differential(6, 2, 12, 20, 1.5, 0.3, 8, 300.0, 9.0), 16, True),
    (differential(4, 2, 32, 64, 0.8, 0.45, 32, 300.0, 20.0), 16, True),
    (differential(4, 4, 64, 128, 0.5, 0.5, 48, 300.0, 15.0), 32, True),     # the largest joint key; a rotation of a part of a map
    (differential(4, 2, 80, 96, 0.4, 0.5, 16, 300.0, 12.0), 16, False),     # maps stored apart, each with a copy of the values
    (differential(6, 1, 96, 40, 0.4, 0.2, 96, 300.0), 16, False),           # no cap
    (differential(1, 1, 4, 8, 3.0, 0.2, 2, 300.0, 6.0), 16, True),          # one head, a rotation of a single pair
    (differential(3, 3, 8, 4, 2.0, 0.6, None, 0.0, 2.0), 16, True),         # no rotation, a cap that flattens most scores
    (differential(2, 2, 5, 7, 2.0, 0.4, 4, 300.0, 8.0), 16, True),          # odd sizes
    (differential(2, 1, 100, 140, 0.3, 0.4, 100, 300.0, 8.0), 16, True),    # values too wide for the matrix-core kernels
    (differential(18, 1, 16, 32, 0.8, 0.4, 16, 300.0, 8.0), 16, None),      # groups of thirty-six maps, of eighteen when stored apart
])
def test_differential_attention(dtype, m, page, joint):
    from llama_cu_amd.parts import PartSpec
    d, eps = 64, 1e-5
    w = mixer_weights(config(16, d, [layer("attention", m)], eps), 12)
    rot = m.get("rot")
    position = None if rot is None else PartSpec("rotary", {"head_dim": m["dim"], "theta": rot["base"], "rot_dim": rot["dims"],
                                                            "max_positions": 512, "interleaved": False})
    part = built("mixer", "differential_attention", {
        "hidden_size": d, "heads": m["heads"], "kv_heads": m["kv_heads"], "head_dim": m["dim"], "value_dim": m["vdim"], "scale": m["scale"],
        "diff": m["diff"], "norm_eps": eps, "softcap": m.get("softcap", 0.0), "position": position}, w, TYPES[dtype], page, pack=True)
    if joint is not None:
        assert part.joint == (joint or dtype == "float32")
    wn = as_numpy(w, "p.")
    assert abs(part.lam - P.difference_weight(wn, "p.", m["diff"])) < 1e-5
    attention_alone(part, lambda h: P.differential_attention(h, wn, "p.", m, eps), [150, 61], dtype, page, 5e-5 if dtype == "float32" else 8e-2, d, 70)


@pytest.mark.parametrize("window", [0, 37])
def test_a_cap_on_the_scores_in_the_matrix_core_kernels(window):
    """Against the generic kernel in 32-bit at the same rounded operands: raw scores from far below the cap to far beyond it, the
    prefill kernel, the decode kernel over keys in one part and in several with its merge."""
    from llama_cu_amd.kernels import ops
    nh, nkv, dh, page, cap, scale = 8, 2, 64, 16, 5.0, 0.6
    n = 1100
    kv = rnd(2, n, nkv, dh, seed=1).bfloat16()
    q = (rnd(n, nh, dh, seed=2) * torch.linspace(0.02, 3.0, n)[:, None, None]).bfloat16()
    pages = (n + page - 1) // page
    perm = torch.randperm(pages, generator=torch.Generator().manual_seed(3))
    cache = torch.full((pages, 2, nkv * dh * page), float("nan"))
    kpad = torch.zeros(2, pages * page, nkv, dh)
    kpad[:, :n] = kv.float()
    for p in range(pages):
        blk = kpad[:, p * page:(p + 1) * page]                    # [2, page, nkv, dh]
        cache[perm[p], 0] = blk[0].permute(1, 2, 0).reshape(nkv, dh // 8, 8, page).permute(0, 1, 3, 2).reshape(-1)
        cache[perm[p], 1] = blk[1].permute(1, 2, 0).reshape(-1)
    bt = perm.to(torch.int32)[None].cuda()

    def run(c, qq, step, **kw):
        out = torch.empty(qq.shape[0], nh * dh, dtype=qq.dtype).cuda()
        return ops.paged_attention(qq.reshape(qq.shape[0], -1).contiguous(), out, c, step, 0, nh, nkv, dh, page, scale, window, softcap=cap, **kw)

    b16, f32 = cache.bfloat16().cuda(), cache.cuda()
    step = hand_step([n], [n], [0], bt, None)
    want = run(f32, q.float().cuda(), step)
    s = scale * np.einsum("id,jd->ij", f64(q[:, 3].float()), f64(kv[0, :, 0].float()))
    seen = P.visible(n, window or None)
    exact = P.attend(f64(q[:, 3].float()), f64(kv[0, :, 0].float()), f64(kv[1, :, 0].float()), scale, seen, softcap=cap)
    assert np.abs(s[seen]).max() > 3 * cap
    assert_close(want.view(n, nh, dh)[:, 3], exact, 2e-5, "the generic kernel")
    assert_close(run(b16, q.cuda(), step), want, 1e-2, "prefill")
    one = hand_step([1], [n], [0], bt, None)
    for splits in (1, 3):
        one.attn_splits = splits
        assert_close(run(b16, q[-1:].cuda(), one), want[-1:], 1e-2, f"decode in {splits} parts")
    # with sinks beside a cap the generic kernel runs
    sinks = torch.full((nh,), 2.0).cuda()
    got = run(b16, q[-1:].cuda(), one, sinks=sinks)
    p = np.where(seen[-1:], np.exp(cap * np.tanh(s[-1:] / cap)), 0.0)
    assert_close(got.view(nh, dh)[3:4], p @ f64(kv[1, :, 0].float()) / (p.sum() + np.exp(2.0)), 1e-2, "sinks beside a cap")


WKV_SHAPES = [(3, 20, 5), (4, 32, 16), (2, 64, 8), (1, 4, 1), (2, 128, 24), (1, 130, 3), (5, 7, 2), (1, 96, 64)]


def wkv_part(heads, dim, rank, d, dtype, seed=13, pack=False):
    eps = 1e-5
    cfg = config(16, d, [layer("wkv", wkv(heads, dim, rank))], eps)
    w = mixer_weights(cfg, seed)
    part = built("mixer", "wkv", {"hidden_size": d, "heads": heads, "head_dim": dim, "decay_rank": rank, "norm_eps": eps}, w, TYPES[dtype], pack=pack)
    wn = as_numpy(w, "p.")
    return part, lambda h: P.wkv(h, wn, "p.", wkv(heads, dim, rank), eps)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,dim,rank", WKV_SHAPES)
def test_the_time_mixer_against_its_recurrence(dtype, heads, dim, rank):
    """In portions and single tokens beside another request's, from slots that held other values (the state and the last
    token's row)."""
    d = 56
    part, plain = wkv_part(heads, dim, rank, d, dtype, pack=True)
    lens = [50, 27]
    rows = [rnd(n, d, seed=20 + r) for r, n in enumerate(lens)]
    cache = part.cache_need().allocate(-1, 0, 0, 3, TYPES[dtype], torch.device("cuda"))
    cache.state.normal_(0.0, 7.0)
    got = Feeder(lens).run(lambda step, x: part.forward(x.cuda(), step, cache, out_dtype=torch.float32), rows)
    for r in range(2):
        assert_close(got[r], plain(f64(rows[r])), 2e-5 if dtype == "float32" else 4e-2, f"request {r}")


@pytest.mark.parametrize("heads,dim,rank", [(3, 20, 5), (2, 64, 8), (2, 128, 24), (1, 130, 3)])
def test_the_time_mixer_walks_long_portions_in_runs(heads, dim, rank):
    """Portions of 512 tokens and more are walked in runs side by side and chained: a long portion from the start beside a
    short request, a second long one that goes on from the first's state beside another that starts, then single tokens."""
    d = 40
    part, plain = wkv_part(heads, dim, rank, d, "float32")
    lens = [1303, 533]
    rows = [rnd(n, d, seed=30 + r) for r, n in enumerate(lens)]
    cache = part.cache_need().allocate(-1, 0, 0, 3, torch.float32, torch.device("cuda"))
    cache.state.normal_(0.0, 7.0)
    steps = [[(0, 0, 513), (1, 0, 3)], [(1, 3, 525), (0, 513, 787)], [(0, 1300, 1), (1, 528, 1)], [(0, 1301, 2), (1, 529, 4)]]
    got = Feeder(lens, steps=steps).run(lambda step, x: part.forward(x.cuda(), step, cache, out_dtype=torch.float32), rows)
    for r in range(2):
        assert_close(got[r], plain(f64(rows[r])), 3e-5, f"request {r}")


def test_the_time_mixer_remembers_a_token_far_back():
    """With decays of nearly one, a strong key hundreds of tokens back still carries the output of a query that asks for it,
    in one portion, in portions and token by token; with strong decays nothing of it is left (and nothing overflows)."""
    d, heads, dim = 32, 1, 16
    for w0, remembered in ((-9.0, True), (3.0, False)):
        cfg = config(16, d, [layer("wkv", wkv(heads, dim, 2))], 1e-5)
        w = mixer_weights(cfg, 14)
        w["w0"] = torch.full((dim,), w0)
        part = built("mixer", "wkv", {"hidden_size": d, "heads": heads, "head_dim": dim, "decay_rank": 2, "norm_eps": 1e-5}, w, torch.float32)
        wn = as_numpy(w, "p.")
        x = rnd(640, d, seed=15, std=0.2)
        x[20] = 30.0 * w["k"][0] / w["k"][0].norm()             # a key that stands out
        x[639] = 30.0 * w["r"][0] / w["r"][0].norm()
        want = P.wkv(f64(x), wn, "p.", wkv(heads, dim, 2), 1e-5)
        without = x.clone()
        without[20] = 0.0
        moved = np.abs(P.wkv(f64(without), wn, "p.", wkv(heads, dim, 2), 1e-5)[639] - want[639]).max() / np.abs(want[639]).max()
        assert (moved > 0.1) == remembered
        cache = part.cache_need().allocate(-1, 0, 0, 3, torch.float32, torch.device("cuda"))
        for slot, cuts in ((0, [640]), (1, [300, 1, 2, 337]), (2, [600] + [1] * 40)):
            got, at = [], 0
            for take in cuts:
                got.append(part.forward(x[at:at + take].cuda(), hand_step([take], [at + take], [slot]), cache, out_dtype=torch.float32).clone())
                at += take
            assert_close(torch.cat(got), want, 5e-5, f"w0 {w0}, cut {len(cuts)}")


# ------------------------------------------------------------------ whole models

_made = {}


def model(name, sharp=1.0):
    """(configuration, weights, folder) of a test model, made once."""
    key = (name, sharp)
    if key not in _made:
        cfg = sharpened(CONFIGS[name], sharp) if sharp != 1.0 else CONFIGS[name]
        w = random_weights(cfg, 1 + sorted(CONFIGS).index(name))
        _made[key] = (cfg, w, make_folder(cfg, w))
    return _made[key]


def runner_for(folder, dtype, **kw):
    from llama_cu_amd.engine.runner import ModelRunner
    args = dict(dtype=dtype, page_size=16, max_tokens=1024, max_seqs=4, max_batch_tokens=1024)
    args.update(kw)
    return ModelRunner.from_folder(folder, **args)


@pytest.mark.parametrize("name,dtype", [(n, t) for n in sorted(CONFIGS) for t in ("float32", "bfloat16")])
def test_a_whole_prompt_against_the_plain_model(name, dtype):
    cfg, w, folder = model(name)
    toks = tokens_of(cfg["vocab"], 100, 1)
    r = runner_for(folder, dtype, page_size={"A": 16, "B": 32, "C": 48, "D": 64, "E": 16}[name])
    got = r.step([0], [toks], [list(range(len(toks)))])
    assert_close(got, plain_logits(cfg, w, toks), REL[dtype], f"model {name} in {dtype}")
    r.end(0)
    r.cache.check()


@pytest.mark.parametrize("name,dtype", [("D", "float32"), ("E", "float32"), ("E", "bfloat16"), ("C", "float32"), ("D", "bfloat16")])
def test_models_of_one_kind_of_layer_and_the_first_tokens_of_a_sequence(name, dtype):
    """Recurrent layers alone (no pages at all) and layers with pages alone: a prompt in portions, then tokens one by one,
    a second request beside the first that starts with portions of one and two tokens, pages and slots used again."""
    cfg, w, folder = model(name)
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
    cfg, w, folder = model(name)
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
    cfg, w, folder = model(name, sharp=3.0 if dtype == "float32" else 1.5)
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
            left = len(reqs[i]) - at
            take = 1 if (left <= 12 or rng.random() < 0.3) else min(left - 12, rng.choice([2, 3, 9, 16, 25]))
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
    assert len(r.groups) == 2
    for g, seen in enumerate(pages_seen):
        assert max(len(v) for v in seen.values()) >= 2, f"no page of pool {g} was used again"
    assert max(len(v) for v in slots_seen.values()) >= 2, "no state slot was used again"
    for i in range(len(reqs)):
        assert_close(torch.cat(done[i]), want[i], REL[dtype] if dtype == "float32" else SAME[dtype], f"request {i} of {lens[i]} tokens")


@pytest.mark.parametrize("name", ["A", "B", "E"])
def test_keys_far_back_and_at_the_borders_of_pages_and_windows(name):
    """Peaked scores make single keys carry an output, so one that is lost, misplaced or seen beyond its window shows; 330
    tokens over pages of 16 and windows that are and are not whole pages, cut inside both, the last 70 decoded one by one:
    every position's logits against the plain model."""
    cfg, w, folder = model(name, sharp=5.0)
    toks = tokens_of(cfg["vocab"], 330, 7)
    want = plain_logits(cfg, w, toks)
    r = runner_for(folder, "float32")
    parts = [r.step([0], [toks[:127]], [list(range(127))]).clone(), r.step([0], [toks[127:260]], [list(range(133))]).clone()]
    parts += [r.step([0], [[t]], [[0]]).clone() for t in toks[260:]]
    assert_close(torch.cat(parts), want, 2 * REL["float32"], "far keys")
    r.end(0)
    r.cache.check()


def test_a_window_one_off_a_lost_sink_and_a_lost_state_show():
    """The inputs above are sharp enough: the plain model with each fault planted in it differs by far more than the tolerance."""
    cfg, w, _ = model("A", sharp=5.0)
    toks = tokens_of(cfg["vocab"], 120, 7)
    want = plain_logits(cfg, w, toks)

    def off(changed_cfg=None, changed_w=None):
        got = plain_logits(changed_cfg or cfg, changed_w or w, toks)
        return ((got - want).abs().max() / want.abs().max()).item()

    import copy
    for size in (18, 20):
        c = copy.deepcopy(cfg)
        c["layers"][0]["mixer"]["mask"]["size"] = size
        assert off(c) > 20 * REL["float32"]
    assert off(changed_w={k: (v - 50.0 if k == "l0.mix.sink" else v) for k, v in w.items()}) > 20 * REL["float32"]
    assert off(changed_w={k: (torch.full_like(v, 4.0) if k == "l1.mix.w0" else v) for k, v in w.items()}) > 20 * REL["float32"]
    assert off(changed_w={k: (torch.zeros_like(v) if k == "l1.mix.mu.k" else v) for k, v in w.items()}) > 20 * REL["float32"]


def test_long_decoding_in_bfloat16():
    cfg, w, folder = model("B")
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
    cfg, w, folder = model("B")
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
    """Forty requests in one step of single tokens (the products for tens of rows, planes of partial sums, the mix of the
    stream with such planes), against the same requests decoded a few at a time."""
    cfg = config(96, 512, [
        layer("latent_attention", latent(4, 64, 64, 64, 128, 0.125, 24), 4096, 3.0),
        layer("wkv", wkv(8, 64, 16)),
        layer("attention", differential(4, 2, 64, 128, 0.125, 0.4, 64, 5000.0, 20.0), 4096, 3.0)], eps=1e-6, mult=0.6, logit_scale=0.5, loop=(0, 3, 2))
    folder = make_folder(cfg, random_weights(cfg, 21))
    r = runner_for(folder, "bfloat16", max_seqs=44, max_tokens=44 * 64)
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
    plain = plain_logits(cfg, random_weights(cfg, 21), prompts[3] + tails[3])[-4:]
    assert_close(torch.stack([t[3] for t in together]), plain, REL["bfloat16"], "against the plain model")


def test_logits_do_not_depend_on_the_cut_or_the_batch_in_32_bit():
    cfg, w, folder = model("A")
    a, b = tokens_of(cfg["vocab"], 60, 20), tokens_of(cfg["vocab"], 41, 21)
    r = runner_for(folder, "float32")
    alone = r.step([0], [a], [list(range(60))]).clone()
    r.step([1], [b[:30]], [[]])
    p1 = r.step([2, 1], [a[:17], b[30:31]], [list(range(17)), [0]]).clone()
    p2 = r.step([1, 2], [b[31:], a[17:]], [[], list(range(43))]).clone()
    assert_close(torch.cat([p1[:17], p2]), alone, 5e-6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine_and_its_scheduler(dtype):
    """The framework's entry point: prompts of unequal lengths, more than run at a time, prefilled in portions; the
    generated tokens equal the plain model's arg-max continuation."""
    from llama_cu_amd.engine.engine import Engine
    cfg, w, folder = model("B")
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
                assert logits[j].max() - logits[j, tok] <= 0.07 * logits[j].abs().max(), f"prompt {k}, token {j}: {tok} is not the best"
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
        layer("wkv", wkv(3, 32, 12)),
        layer("latent_attention", latent(4, 32, 24, 64, 48, 0.2, 21), 64, 2.0),
        layer("attention", differential(4, 2, 16, 32, 0.3, 0.4, 16, 2000.0, 12.0), 80, 2.0)], eps=1e-5, mult=0.8, logit_scale=1.25, loop=(1, 3, 2))
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
