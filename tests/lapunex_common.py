"""Shared by the Lapunex tests: small configurations that differ in every size and option, random weights from the tests'
own generator, model folders in temporary places, and the plain implementation's logits."""
from __future__ import annotations

import copy
import json
import math
import os
import tempfile
from typing import Dict, List, Optional

import torch

import plain_lapunex as P
from gefudra_common import Feeder, as_numpy, assert_close, built, hand_step, tokens_of  # noqa: F401  (steps and parts made by hand)


def yarn(factor, original, fast, slow):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def left(heads, kv_heads, dim, vdim, scale, rot=None, base=10000.0, scaling=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot:
        m["rot"] = {"base": base, "dims": rot}
        if scaling:
            m["rot"]["scaling"] = scaling
    return m


def right(heads, dim, vdim, cap):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def lightning(decay, dim, vdim):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, scale=1.0, groups=None):
    r = {"experts": experts, "top": top, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": r}


def light(m, mlp=None):
    return {"type": "lightning", "mixer": m, "mlp": mlp}


def both(a, b, left_scale, right_scale, mlp=None):
    return {"type": "parallel", "mixer": {"left": a, "right": b, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def config(vocab, width, layers, eps, streams, scale=1.0, loop=None):
    c = {"architecture": "Lapunex", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "embedding": {"scale": scale},
         "layers": layers}
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# no size a power of two where it need not be: a width that no 16 bytes fill, groups of three heads of 12 of which 8 dims are turned over
# values of 20 beside a memory of three heads of 20 over 12, experts of 20 in three groups of which two are kept; layers with and without
# a feed-forward; two layers in a loop of two runs, one behind it
CFG_A = config(131, 76, [
    light(lightning([0.5, 0.93, 0.998], 20, 12), dense(40)),
    both(left(6, 2, 12, 20, 0.1, 8, 700.0, yarn(5.0, 48, 4.0, 0.25)), right(3, 20, 28, 5.0), 0.8, -0.7, moe(12, 3, 20, 1.1, 0.9, (3, 2))),
    light(lightning([0.0, 0.97], 8, 28)),
    both(left(2, 2, 10, 6, 0.15), right(2, 7, 15, 9.0), 1.2, 0.4, dense(24)),
], eps=1e-4, streams=3, scale=1.7, loop=(1, 3, 2))

# sizes that the bfloat16 kernels like (multiples of 16, head sizes of the matrix-core kernels); the loop starts with the first layer
CFG_B = config(208, 128, [
    light(lightning([0.6, 0.9, 0.99, 0.9995], 32, 64), moe(8, 2, 64, 2.5, 1.5, (4, 2))),
    both(left(8, 2, 64, 64, 0.125, 32, 5000.0, yarn(4.0, 64, 8.0, 0.5)), right(2, 64, 64, 12.0), 0.6, 0.9, dense(256)),
    light(lightning([0.95, 0.7], 64, 128), dense(128)),
], eps=1e-6, streams=4, scale=0.9, loop=(0, 2, 2))

# values that are often equal or 1 and need not be: one stream, one head, a rotation of a single pair and none, one expert of one, one group,
# every group kept, a loop over the whole model that runs once, factors of 1
CFG_C = config(97, 40, [
    both(left(1, 1, 4, 8, 0.5, 2, 50.0, yarn(2.0, 16, 1.0, 0.5)), right(1, 4, 1, 1.0), 1.0, 1.0, moe(1, 1, 16, 0.5)),
    light(lightning([1.0], 1, 1), moe(6, 6, 8, 1.0, 1.0, (2, 2))),
    both(left(3, 3, 8, 4, 0.4, 8, 300.0), right(1, 1, 4, 3.0), 1.0, 1.0),
    light(lightning([0.8, 0.8], 4, 4), moe(4, 1, 8, 3.0, 0.5, (4, 1))),
], eps=1e-5, streams=1, loop=(0, 4, 1))

# one kind of layer only: no pages at all ...
CFG_D = config(64, 48, [light(lightning([0.99, 0.4], 16, 24), dense(32)), light(lightning([0.9, 0.999, 0.8], 12, 20))], eps=1e-5, streams=2,
               scale=2.0, loop=(0, 2, 3))
# ... and pages in every layer, no loop: heads too wide for the matrix-core attention, memories wider than 128
CFG_E = config(80, 64, [
    both(left(4, 2, 136, 96, 0.1, 24, 300.0, yarn(3.0, 30, 3.0, 0.3)), right(2, 140, 72, 6.0), 0.5, 1.5, dense(48)),
    both(left(3, 1, 80, 112, 0.15, 48, 900.0, yarn(16.0, 100, 32.0, 1.0)), right(1, 40, 140, 4.0), 1.0, 0.8, moe(9, 2, 24, 0.9, 2.2, (3, 1))),
], eps=1e-5, streams=5, scale=1.3)

CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C, "D": CFG_D, "E": CFG_E}


def sharpened(cfg: dict, factor: float) -> dict:
    """``cfg`` with every attention's scale multiplied by ``factor``: the softmax becomes peaked, so that single keys, often far back,
    carry an output, and a key that is lost or misplaced shows."""
    out = copy.deepcopy(cfg)
    for entry in out["layers"]:
        if "left" in entry["mixer"]:
            entry["mixer"]["left"]["scale"] *= factor
    return out


TAGS = 4        # channels of the streams that a steady router reads


def random_weights(cfg: dict, seed: int, steady_router: bool = False) -> Dict[str, torch.Tensor]:
    """Every tensor of the design for ``cfg``, float32 values that bfloat16 holds exactly.  ``steady_router``: for runs in bfloat16, whose
    streams differ from the plain model's by some hundredths, which would make close calls between experts fall the other way (a
    choice is discrete; such a flip moves the logits by their size and is no fault): every token has one of ``TAGS`` tags, a channel
    of its embedding that stands out; no sublayer writes into these channels, and the routers read them alone, with weights well
    apart, so that a choice differs from tag to tag and layer to layer and never hangs on a rounding."""
    g = torch.Generator().manual_seed(seed)
    d, s = cfg["width"], cfg["streams"]

    def mat(out, inp, gain=1.0):
        return torch.randn(out, inp, generator=g) * (gain / math.sqrt(inp))

    def vec(n, mean=0.0, std=0.1):
        return mean + std * torch.randn(n, generator=g)

    def writes(m):
        if steady_router:
            m[:TAGS] = 0.0
        return m

    def norm():
        w = vec(d, 0.0, 0.2)
        if steady_router:
            w[:TAGS] = 0.0
        return w

    w = {"embed": torch.randn(cfg["vocab"], d, generator=g), "final.norm": vec(d), "head": mat(cfg["vocab"], d)}
    if steady_router:
        w["embed"][:, :TAGS] = 6.0 * torch.nn.functional.one_hot(torch.randint(0, TAGS, (cfg["vocab"],), generator=g), TAGS)
    for i, entry in enumerate(cfg["layers"]):
        m, f = entry["mixer"], entry.get("mlp")
        for q in (1, 2)[:2 if f else 1]:
            w[f"l{i}.hc{q}.in"], w[f"l{i}.hc{q}.out"] = vec(s, 1.0 / s, 0.4 / s), vec(s, 0.8, 0.4)
            w[f"l{i}.hc{q}.mix"] = 0.8 * torch.eye(s) + 0.25 * torch.randn(s, s, generator=g)
            w[f"l{i}.norm{q}"] = norm()
        pre = f"l{i}.mix."
        if entry["type"] == "lightning":
            hk, hv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for name, rows in (("q", hk), ("k", hk), ("v", hv), ("g", hv)):
                w[pre + name] = mat(rows, d, 1.5)
            w[pre + "norm"], w[pre + "o"] = vec(hv, 1.0, 0.2), writes(mat(d, hv, 2.0))
        else:
            a, b = m["left"], m["right"]
            nq, nk = a["heads"] * a["dim"], a["kv_heads"] * a["dim"]
            w[pre + "left.q"], w[pre + "left.k"], w[pre + "left.v"] = mat(nq, d), mat(nk, d), mat(a["kv_heads"] * a["vdim"], d, 2.0)
            w[pre + "left.q.norm"], w[pre + "left.k.norm"] = vec(nq, 1.5, 0.5), vec(nk, 1.5, 0.5)
            w[pre + "left.sink"], w[pre + "left.g"] = vec(a["heads"], 1.0, 1.5), mat(a["heads"], d, 2.0)
            w[pre + "left.o"] = writes(mat(d, a["heads"] * a["vdim"], 2.0))
            hk, hv = b["heads"] * b["dim"], b["heads"] * b["vdim"]
            for name, rows in (("q", hk), ("k", hk), ("v", hv), ("g", hv)):
                w[pre + "right." + name] = mat(rows, d, 1.5)
            w[pre + "right.i"], w[pre + "right.i.b"] = mat(b["heads"], d, 1.5), vec(b["heads"], 0.0, 1.0)
            # forget gates from 0.5 to nearly 1: memories of a few to some hundreds of tokens
            w[pre + "right.f"], w[pre + "right.f.b"] = mat(b["heads"], d, 1.5), vec(b["heads"], 3.5, 2.0)
            w[pre + "right.norm"], w[pre + "right.o"] = vec(hv, 1.0, 0.2), writes(mat(d, hv))
        if f is None:
            continue
        pre = f"l{i}.mlp."
        if f["kind"] == "dense":
            w[pre + "gate"], w[pre + "up"], w[pre + "down"] = mat(f["ff"], d, 1.5), mat(f["ff"], d, 1.5), writes(mat(d, f["ff"]))
            continue
        ff, n = f["expert"]["ff"], f["router"]["experts"]
        for e in range(n):
            w[f"{pre}e{e}.gate"], w[f"{pre}e{e}.up"], w[f"{pre}e{e}.down"] = mat(ff, d, 1.5), mat(ff, d, 1.5), writes(mat(d, ff, 2.0))
        w[pre + "router"] = mat(n, d, 2.0)
        if steady_router:
            w[pre + "router"].zero_()
            for tag in range(TAGS):
                w[pre + "router"][:, tag] = torch.randperm(n, generator=g).float() * (1.2 / n)
    return {k: v.to(torch.bfloat16).float().contiguous() for k, v in w.items()}


def mixer_weights(cfg: dict, seed: int, prefix: str = "l0.mix.") -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in random_weights(cfg, seed).items() if k.startswith(prefix)}


def make_folder(cfg: dict, weights: Dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16, folder: Optional[str] = None) -> str:
    from llama_cu_amd.weights import write_safetensors
    folder = folder or tempfile.mkdtemp(prefix="lcu_lapunex_")
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), {k: v.to(dtype) for k, v in weights.items()})
    return folder


def plain_logits(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int]) -> torch.Tensor:
    return torch.from_numpy(P.forward(cfg, as_numpy(weights), tokens))
