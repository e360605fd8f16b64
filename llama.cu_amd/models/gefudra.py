"""The Gefudra decoder laid out of parts.

Every layer is a pre-norm block (RMS norms; the feed-forward, with its norm, may be missing), and both sublayers' outputs
enter the stream times one factor.  Three mixers: latent attention without positions (queries through a latent of
their own, a window, a sink, an output gate), differential attention (two maps per head over the same values, a rotation
in half-split pairs, a cap on the scores, an output gate), and a recurrent mixer with a decay per key channel whose
projections read a mix of the token and the one before.  The feed-forward is the gated one with a limited activation.  Some
layers in a row may run several times with the same weights, each run with caches and states of its own; in front of
each run a matrix mixes the stream with the embedding's output.  The output matrix is the embedding table, the logits
are multiplied by a factor.  Everything here is data: which parts, with which sizes and constants from the
configuration, under which tensor names, in which order.
"""
from __future__ import annotations

from ..config import ConfigError, register_architecture
from ..config.gefudra import GefudraConfig, complete_config
from ..parts import ModelSpec, PartSpec, RunEntry

# the factor inside the feed-forward's sigmoid, g sigmoid(1.702 g): the design fixes it
GATE_ALPHA = 1.702

DENSE_NAMES = {"gate": "gate", "up": "up", "down": "down"}


def gefudra_spec(cfg: GefudraConfig) -> ModelSpec:
    d = cfg.width

    def norm(tensor: str, factor: float = 1.0) -> PartSpec:
        return PartSpec("rmsnorm", {"size": d, "eps": cfg.norm_eps, "tensor": tensor, "delta_scale": cfg.residual_mult, "factor": factor}, "")

    layers = []
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        if layer.type == "latent_attention":
            mixer = PartSpec("latent_attention", {"hidden_size": d, "heads": m.heads, "head_dim": m.dim, "rot_dim": 0, "value_dim": m.vdim,
                                                  "kv_rank": m.kv_rank, "q_rank": m.q_rank, "scale": m.scale, "norm_eps": cfg.norm_eps,
                                                  "window": m.window, "sink": True, "gate": True}, "mix")
        elif layer.type == "attention":
            position = None if m.rot is None else PartSpec("rotary", {"head_dim": m.dim, "theta": m.rot.base, "rot_dim": m.rot.dims,
                                                                      "max_positions": cfg.max_positions, "interleaved": False})
            mixer = PartSpec("differential_attention", {"hidden_size": d, "heads": m.heads, "kv_heads": m.kv_heads, "head_dim": m.dim,
                                                        "value_dim": m.vdim, "scale": m.scale, "diff": m.diff, "norm_eps": cfg.norm_eps,
                                                        "softcap": m.softcap or 0.0, "position": position, "gate": True}, "mix")
        else:
            if m.rank is None:
                raise ConfigError(f"config.json: layers[{i}].mixer: the rank of the decay's projection is neither given as 'rank' nor known "
                                  f"from the shape of a tensor l{i}.mix.w1")
            mixer = PartSpec("wkv", {"hidden_size": d, "heads": m.heads, "head_dim": m.dim, "decay_rank": m.rank, "norm_eps": cfg.norm_eps}, "mix")
        params = {"norm1": norm("norm1"), "mixer": mixer}
        if layer.ff is not None:
            params.update(norm2=norm("norm2"), ffn=PartSpec("swiglu", {"hidden_size": d, "intermediate_size": layer.ff.ff, "names": DENSE_NAMES,
                                                                       "activation": "limited", "alpha": GATE_ALPHA,
                                                                       "limit": layer.ff.limit}, "mlp"))
        layers.append(PartSpec("prenorm", params, f"l{i}"))
    # the layers of the loop stand several times in the run order, every run's first one behind the mix with the embedding
    order, streams = [RunEntry(i) for i in range(len(layers))], []
    if cfg.loop is not None:
        start, stop = cfg.loop.start, cfg.loop.stop
        streams = [PartSpec("remix", {"hidden_size": d, "tensor": "in", "delta_scale": cfg.residual_mult}, "loop")]
        one_run = [RunEntry(i, before=0 if i == start else None) for i in range(start, stop)]
        order = order[:start] + one_run * cfg.loop.times + order[stop:]
    return ModelSpec(
        hidden_size=d, vocab_size=cfg.vocab, max_positions=cfg.max_positions,
        embedding=PartSpec("tokens", {"vocab_size": cfg.vocab, "hidden_size": d, "tensor": "embed"}, ""),
        layers=layers, run_order=order, final_norm=norm("final.norm", cfg.logit_scale),
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": d, "tied": True, "tensor": "head"}, ""),
        eos_token_ids=cfg.eos_token_ids, streams=streams)


register_architecture("Gefudra", GefudraConfig.from_dict, gefudra_spec, complete_config=complete_config)
