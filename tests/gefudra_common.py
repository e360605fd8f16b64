"""Shared by the Gefudra tests: small configurations that differ in every size and option, random weights from the tests'
own generator, model folders in temporary places, the plain implementation's logits, and steps made by hand."""
from __future__ import annotations

import copy
import json
import math
import os
import random
import tempfile
from typing import Dict, List, Optional

import numpy as np
import torch

import plain_gefudra as P


def latent(heads, dim, vdim, kv_rank, q_rank, scale, window=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    return m


def differential(heads, kv_heads, dim, vdim, scale, diff, rot=None, base=10000.0, softcap=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if rot:
        m["rot"] = {"base": base, "dims": rot}
    if softcap:
        m["softcap"] = softcap
    return m


def wkv(heads, dim, rank):
    """(``rank``: read from the shape of a file's tensor where config.json does not give it)"""
    return {"heads": heads, "dim": dim, "rank": rank}


def layer(kind, mixer, ff=None, limit=None):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def config(vocab, width, layers, eps, mult=1.0, logit_scale=1.0, loop=None):
    c = {"architecture": "Gefudra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "logit_scale": logit_scale,
         "layers": layers}
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# no size a power of two where it need not be: windows of 19 and none, latents of 28 and 36 (folded queries as one matrix) and of 44
# and 24 (folded head by head), groups of three heads with two maps of 12 dims of which 8 are turned over values of 20, a time mixer
# of three heads of 20 with a rank of 5; layers with and without a feed-forward; two layers in a loop of three runs, one behind it
CFG_A = config(131, 72, [
    layer("latent_attention", latent(3, 20, 12, 28, 36, 0.3, 19), 40, 1.5),
    layer("wkv", wkv(3, 20, 5)),
    layer("attention", differential(6, 2, 12, 20, 0.4, 0.3, 8, 700.0, 9.0), 56, 0.8),
    layer("latent_attention", latent(2, 8, 20, 44, 24, 0.25), 24, 2.5),
], eps=1e-4, mult=0.7, logit_scale=1.6, loop=(1, 3, 3))

# sizes that the bfloat16 kernels like (multiples of 16, head sizes of the matrix-core kernels); the loop starts with the first layer
CFG_B = config(208, 128, [
    layer("wkv", wkv(4, 32, 16), 256, 3.0),
    layer("latent_attention", latent(4, 64, 64, 64, 64, 0.125, 33), 256, 3.0),
    layer("attention", differential(4, 2, 32, 64, 0.18, 0.45, 32, 5000.0, 20.0), 128, 3.0),
    layer("wkv", wkv(2, 64, 8)),
], eps=1e-6, mult=0.5, logit_scale=0.75, loop=(0, 2, 2))

# values that are often equal or 1 and need not be: one head, a window of 1, a rotation of a single pair and none, no cap, a rank of
# one, a loop over the whole model that runs once, factors of 1
CFG_C = config(97, 40, [
    layer("latent_attention", latent(1, 4, 8, 8, 4, 0.5, 1), 16, 0.5),
    layer("attention", differential(1, 1, 4, 8, 0.5, 0.2, 2, 50.0), 8, 1.0),
    layer("wkv", wkv(1, 4, 1)),
    layer("attention", differential(3, 3, 8, 4, 0.4, 0.6, softcap=2.0)),
], eps=1e-5, loop=(0, 4, 1))

# one kind of layer only: no pages at all ...
CFG_D = config(64, 48, [layer("wkv", wkv(2, 16, 3), 32, 2.0), layer("wkv", wkv(3, 12, 7))], eps=1e-5, mult=0.6, logit_scale=2.0, loop=(0, 2, 3))
# ... and pages only, no loop: maps too wide for one head of the matrix-core kernels together (stored apart), a latent too wide for any
CFG_E = config(80, 64, [
    layer("attention", differential(4, 2, 80, 96, 0.1, 0.5, 16, 300.0, 12.0), 48, 2.0),
    layer("latent_attention", latent(3, 16, 24, 144, 20, 0.25, 40)),
], eps=1e-5, mult=1.3)

CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C, "D": CFG_D, "E": CFG_E}


def sharpened(cfg: dict, factor: float) -> dict:
    """``cfg`` with every attention's scale multiplied by ``factor`` (and its cap with it): the softmax becomes peaked, so that
    single keys, often far back, carry an output, and a key that is lost or wrongly seen shows."""
    out = copy.deepcopy(cfg)
    for entry in out["layers"]:
        if "scale" in entry["mixer"]:
            entry["mixer"]["scale"] *= factor
        if "softcap" in entry["mixer"]:
            entry["mixer"]["softcap"] *= factor
    return out


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """Every tensor of the design for ``cfg``, float32 values that bfloat16 holds exactly."""
    g = torch.Generator().manual_seed(seed)
    d = cfg["width"]

    def mat(out, inp, gain=1.0):
        return torch.randn(out, inp, generator=g) * (gain / math.sqrt(inp))

    def vec(n, mean=0.0, std=0.1):
        return mean + std * torch.randn(n, generator=g)

    w = {"embed": torch.randn(cfg["vocab"], d, generator=g), "final.norm": vec(d, 1.0)}
    if cfg.get("loop"):
        w["loop.in"] = mat(d, 2 * d, 1.2)
    for i, entry in enumerate(cfg["layers"]):
        m, pre = entry["mixer"], f"l{i}.mix."
        w[f"l{i}.norm1"] = vec(d, 1.0, 0.2)
        if entry["type"] == "latent_attention":
            h, r = m["heads"], m["kv_rank"]
            w[pre + "dq"], w[pre + "dq.norm"] = mat(m["q_rank"], d), vec(m["q_rank"], 1.0, 0.2)
            w[pre + "uq"] = mat(h * m["dim"], m["q_rank"], 2.0)
            w[pre + "dkv"], w[pre + "dkv.norm"] = mat(r, d), vec(r, 1.0, 0.2)
            w[pre + "uk"], w[pre + "uv"] = mat(h * m["dim"], r, 2.0), mat(h * m["vdim"], r, 1.5)
            w[pre + "sink"] = vec(h, 1.0, 1.5)
            w[pre + "g"], w[pre + "o"] = mat(h * m["vdim"], d, 2.0), mat(d, h * m["vdim"], 2.0)
        elif entry["type"] == "attention":
            h, kv, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            w[pre + "q"], w[pre + "k"], w[pre + "v"] = mat(h * 2 * dim, d, 1.5), mat(kv * 2 * dim, d, 1.5), mat(kv * vd, d)
            for name in ("lq1", "lk1", "lq2", "lk2"):
                w[pre + name] = vec(dim, 0.1 if name != "lk2" else -0.1, 0.2)
            w[pre + "g"], w[pre + "o"] = mat(h * vd, d, 2.0), mat(d, h * vd, 1.5)
        else:
            hd = m["heads"] * m["dim"]
            for s in "rkvgw":
                w[pre + "mu." + s] = torch.rand(d, generator=g)
            for s in "rkvg":
                w[pre + s] = mat(hd, d, 1.5)
            # decays from 0.5 to nearly 1: states that remember from a few to some hundreds of tokens
            w[pre + "w1"], w[pre + "w2"], w[pre + "w0"] = mat(m["rank"], d), mat(hd, m["rank"]), vec(hd, -2.5, 1.2)
            w[pre + "u"] = torch.randn(m["heads"], m["dim"], generator=g)
            w[pre + "norm"], w[pre + "o"] = vec(hd, 1.0, 0.2), mat(d, hd)
        f = entry.get("mlp")
        if f is not None:
            w[f"l{i}.norm2"] = vec(d, 1.0, 0.2)
            pre = f"l{i}.mlp."
            w[pre + "gate"], w[pre + "up"], w[pre + "down"] = mat(f["ff"], d, 2.0), mat(f["ff"], d, 1.5), mat(d, f["ff"])
    return {k: v.to(torch.bfloat16).float().contiguous() for k, v in w.items()}


def mixer_weights(cfg: dict, seed: int, i: int = 0) -> Dict[str, torch.Tensor]:
    pre = f"l{i}.mix."
    return {k[len(pre):]: v for k, v in random_weights(cfg, seed).items() if k.startswith(pre)}


def make_folder(cfg: dict, weights: Dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16, folder: Optional[str] = None,
                leave_ranks_out: bool = True) -> str:
    """``leave_ranks_out``: config.json does not give a time mixer's rank (the engine takes it from the tensor's shape)."""
    from llama_cu_amd.weights import write_safetensors
    folder = folder or tempfile.mkdtemp(prefix="lcu_gefudra_")
    cfg = copy.deepcopy(cfg)
    if leave_ranks_out:
        for entry in cfg["layers"]:
            entry["mixer"].pop("rank", None)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), {k: v.to(dtype) for k, v in weights.items()})
    return folder


def as_numpy(weights: Dict[str, torch.Tensor], prefix: str = "") -> Dict[str, np.ndarray]:
    return {prefix + k: v.double().numpy() for k, v in weights.items()}


def plain_logits(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int]) -> torch.Tensor:
    return torch.from_numpy(P.forward(cfg, as_numpy(weights), tokens))


def tokens_of(vocab: int, n: int, seed: int) -> List[int]:
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def assert_close(got, want, rel: float, what: str = "") -> None:
    """The largest difference, relative to the largest expected magnitude."""
    got, want = torch.as_tensor(got).detach().double().cpu(), torch.as_tensor(want).detach().double().cpu()
    assert got.shape == want.shape, f"{what}: shape {tuple(got.shape)} against {tuple(want.shape)}"
    assert torch.isfinite(got).all(), f"{what}: not finite"
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-30)
    assert err <= rel, f"{what}: relative error {err:.3e} exceeds {rel:.1e}"


# ------------------------------------------------------------------ steps made by hand (on the GPU)


def i32(v):
    return torch.tensor(v, dtype=torch.int32).cuda()


def hand_step(q_lens, ctx_lens, slots, block_table=None, slot_map=None):
    """A step of requests that feed ``q_lens`` tokens and then hold ``ctx_lens``, in state ``slots``."""
    from llama_cu_amd.engine.batch import StepContext
    n = sum(q_lens)
    starts = [0]
    for x in q_lens:
        starts.append(starts[-1] + x)
    pos = [c - q + k for q, c in zip(q_lens, ctx_lens) for k in range(q)]
    return StepContext(n=n, n_req=len(q_lens), tokens=i32([0] * n), positions=i32(pos),
                       req_of_token=i32([r for r, x in enumerate(q_lens) for _ in range(x)]), q_start=i32(starts),
                       ctx_len=i32(ctx_lens), state_slot=i32(slots), logit_rows=i32([]), n_logits=0,
                       block_tables=[block_table] if block_table is not None else [],
                       slot_maps=[slot_map] if slot_map is not None else [], q_lens=list(q_lens), ctx_lens=list(ctx_lens),
                       state_slots=list(slots))


def built(category, kind, params, tensors, dtype, page=16, pack=False):
    """A part alone: made by the registry, its weights bound."""
    from llama_cu_amd.parts import BuildContext, PartSpec, make_part
    part = make_part(category, PartSpec(kind, params))
    want = {k for k, v in part.tensors().items() if not v.optional}
    assert want == set(tensors), (sorted(want), sorted(tensors))
    part.load({k: v.to(dtype).cuda() for k, v in tensors.items()}, BuildContext(dtype, torch.device("cuda"), 2048, page, pack))
    return part


class Feeder:
    """Feeds two requests' rows through a mixer in steps: the first request in portions of changing size beside single
    tokens and portions of the second, which starts later; slots 2 and 0 of a state that holds other values; with pages,
    a block table of shuffled pages among pages that nobody owns."""

    def __init__(self, lens, page=16, seed=0, steps=None):
        """``steps``: the plan, if not the usual one: [[(request, first token, tokens taken), ...], ...]."""
        self.lens, self.page, self.steps = lens, page, steps
        rng = random.Random(seed)
        need = [(n + page - 1) // page for n in lens]
        order = list(range(sum(need) + 3))
        rng.shuffle(order)
        self.tables, at = [], 0
        for k in need:
            self.tables.append(order[at:at + k])
            at += k
        self.n_pages = len(order)
        bt = torch.zeros(len(lens), max(need), dtype=torch.int32)
        for r, t in enumerate(self.tables):
            bt[r, :len(t)] = torch.tensor(t, dtype=torch.int32)
        self.bt = bt.cuda()

    def plan(self):
        if self.steps is not None:
            return self.steps
        l0, l1 = self.lens
        steps, a, b, k = [], 0, 0, 0
        sizes0, sizes1 = [5, 1, 2, 7, 1, 1, 3, 16, 2, 1], [1, 2, 1, 4, 9, 1, 2]
        while a < l0 or b < l1:
            step = []
            if a < l0:
                take = min(sizes0[k % len(sizes0)], l0 - a)
                step.append((0, a, take)); a += take
            if b < l1 and k >= 2:
                take = min(sizes1[k % len(sizes1)], l1 - b)
                step.append((1, b, take)); b += take
            steps.append(step)
            k += 1
        return steps

    def run(self, forward, rows):
        outs = [[], []]
        for step in self.plan():
            q_lens = [t for _, _, t in step]
            ctx = [at + t for _, at, t in step]
            pos_req = [(r, at + k) for r, at, t in step for k in range(t)]
            slot_map = i32([self.tables[r][p // self.page] * self.page + p % self.page for r, p in pos_req])
            bt = self.bt[[r for r, _, _ in step]].contiguous()
            ctx_step = hand_step(q_lens, ctx, [2 if r == 0 else 0 for r, _, _ in step], bt, slot_map)
            out = forward(ctx_step, torch.cat([rows[r][at:at + t] for r, at, t in step]))
            o = 0
            for r, _, t in step:
                outs[r].append(out[o:o + t].clone())
                o += t
        return [torch.cat(x) for x in outs]
