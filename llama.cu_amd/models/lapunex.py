"""The Lapunex decoder laid out of parts.

Several residual streams: every sublayer (RMS norms, weights stored around zero) reads a weighted sum of them and writes back
through a matrix between the streams and a weight per stream.  Two mixers: linear attention with a fixed decay per head and
one norm over all heads; and two mixers side by side, softmax attention (a norm over the whole query and key projections, a
rotation with blended frequencies of the first dims of half-split pairs, a sink, a gate per head) beside a matrix memory with
exponential gates.  The feed-forward is the dense gated one, or a mixture of gated experts with limits, chosen within groups by
softmax scores, or missing.  Some layers in a row may run several times with the same weights, each run with caches and states
of its own.  Everything here is data: which parts, with which sizes and constants from the configuration, under which tensor
names, in which order.
"""
from __future__ import annotations

from ..config import register_architecture
from ..config.lapunex import Dense, LapunexConfig
from ..parts import ModelSpec, PartSpec, RunEntry

# the factor inside the experts' sigmoid, g sigmoid(1.702 g): the design fixes it
GATE_ALPHA = 1.702

ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink", "g": "g"}
GATED_NAMES = {"gate": "gate", "up": "up", "down": "down"}
EXPERT_NAMES = {"router": "router", "gate": "e{}.gate", "up": "e{}.up", "down": "e{}.down"}


def lapunex_spec(cfg: LapunexConfig) -> ModelSpec:
    d = cfg.width

    def norm(tensor: str) -> PartSpec:
        return PartSpec("streams_rmsnorm", {"size": d, "eps": cfg.norm_eps, "streams": cfg.streams, "tensor": tensor, "one_plus": True}, "")

    def rotary(rot, head_dim: int):
        if rot is None:
            return None
        s = rot.scaling
        yarn = None if s is None else {"factor": s.factor, "original": s.original, "fast": s.fast, "slow": s.slow}
        return PartSpec("rotary", {"head_dim": head_dim, "theta": rot.base, "max_positions": cfg.max_positions, "rot_dim": rot.dims, "yarn": yarn})

    layers = []
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        if layer.type == "lightning":
            mixer = PartSpec("lightning", {"hidden_size": d, "heads": m.heads, "head_dim": m.dim, "value_dim": m.vdim, "decay": list(m.decay),
                                           "norm_eps": cfg.norm_eps}, "mix")
        else:
            a, b = m.left, m.right
            left = PartSpec("attention", {"hidden_size": d, "heads": a.heads, "kv_heads": a.kv_heads, "head_dim": a.dim, "value_dim": a.vdim,
                                          "scale": a.scale, "position": rotary(a.rot, a.dim), "projection_norm_eps": cfg.norm_eps,
                                          "sink": True, "head_gate": True, "names": ATTENTION_NAMES}, "left")
            right = PartSpec("matrix_memory", {"hidden_size": d, "heads": b.heads, "head_dim": b.dim, "value_dim": b.vdim,
                                               "gate_cap": b.gate_cap, "norm_eps": cfg.norm_eps}, "right")
            mixer = PartSpec("side_by_side", {"mixers": [left, right], "scales": [m.left_scale, m.right_scale]}, "mix")
        params = {"streams": cfg.streams, "norm1": norm("norm1"), "mixer": mixer, "connections": ("hc1", "hc2")}
        f = layer.mlp
        if f is not None:
            if isinstance(f, Dense):
                ffn = PartSpec("swiglu", {"hidden_size": d, "intermediate_size": f.ff, "names": GATED_NAMES}, "mlp")
            else:
                ffn = PartSpec("gated_moe", {"hidden_size": d, "expert_size": f.ff, "experts": f.experts, "top": f.top, "router_bias": False,
                                             "scoring": "softmax_all", "renormalize": False, "scale": f.scale, "groups": f.groups,
                                             "keep_groups": f.keep, "activation": "limited", "alpha": GATE_ALPHA, "limit": f.limit,
                                             "names": EXPERT_NAMES}, "mlp")
            params.update(norm2=norm("norm2"), ffn=ffn)
        layers.append(PartSpec("streams", params, f"l{i}"))
    # the layers of the loop stand several times in the run order
    order = list(range(len(layers)))
    if cfg.loop is not None:
        start, stop = cfg.loop.start, cfg.loop.stop
        order = order[:start] + order[start:stop] * cfg.loop.times + order[stop:]
    return ModelSpec(
        hidden_size=d, vocab_size=cfg.vocab, max_positions=cfg.max_positions,
        embedding=PartSpec("tokens", {"vocab_size": cfg.vocab, "hidden_size": d, "scale": cfg.embedding_scale, "tensor": "embed",
                                      "streams": cfg.streams}, ""),
        layers=layers, run_order=[RunEntry(i) for i in order], final_norm=norm("final.norm"),
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": d, "tied": False, "tensor": "head"}, ""),
        eos_token_ids=cfg.eos_token_ids)


register_architecture("Lapunex", LapunexConfig.from_dict, lapunex_spec)
