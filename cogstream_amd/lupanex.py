"""Lupanex: a small decoder-only language model whose layers are listed one by one in config.json ("layers"), each a mixer and an
optional feed-forward (exact gelu between two matrices), around hyper-connected residual streams.

    attention    softmax attention with grouped key / value heads, weightless RMS norms on queries and keys, a query temperature that
                 grows with the position, and a learned score bias per head and bucket of distances ("mix.rel": one row per bucket)
    delta        gated delta rule: a matrix of state per head behind short convolutions

The embedding is scaled and gets a learned vector per position; a run of layers may be looped ("loop"). This module only reads the
configuration."""
from __future__ import annotations

from typing import Dict, Tuple

from .decoder import DecoderForCausalLM
from .weights import DecoderConfig, DecoderLayerConfig, DeltaRule, DistanceBias, HeadAttention, Loop


def parse_config(c: dict, shapes: Dict[str, Tuple[int, ...]]) -> DecoderConfig:
    """config.json, with the shapes of the checkpoint's tensors (the number of distance buckets is a shape only) -> DecoderConfig"""
    cfg = DecoderConfig(width=int(c["width"]), vocab_size=int(c["vocab"]), eps=float(c["norm"]["eps"]),
                        embed_scale=float(c["embedding"]["scale"]), max_positions=int(c["max_positions"]), streams=int(c.get("streams") or 0))
    loop = c.get("loop")
    if loop is not None:
        cfg.loop = Loop(int(loop["start"]), int(loop["stop"]), int(loop["times"]))
        if not (0 <= cfg.loop.start < cfg.loop.stop <= len(c["layers"]) and cfg.loop.times >= 1):
            raise ValueError(f"loop {loop} over {len(c['layers'])} layers")
    for i, lay in enumerate(c["layers"]):
        m = lay["mixer"]
        sizes = dict(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]))
        if sizes["heads"] % sizes["kv_heads"]:
            raise ValueError(f"layer {i}: {sizes['heads']} heads in {sizes['kv_heads']} groups")
        if lay["type"] == "attention":
            temp = m.get("q_temp") or {"coef": 0.0, "every": 0.0}
            mixer = HeadAttention(scale=float(m["scale"]), qk_norm=True, temp_coef=float(temp["coef"]), temp_every=float(temp["every"]),
                                  bias=DistanceBias(int(shapes[f"l{i}.mix.rel"][0]), float(m["bias_max"])), **sizes)
        elif lay["type"] == "delta":
            mixer = DeltaRule(taps=int(m["conv"]), **sizes)
        else:
            raise ValueError(f"layer {i}: mixer type {lay['type']!r} (known: attention, delta)")
        mlp = lay.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: feed-forward kind {mlp['kind']!r} (known: dense)")
        cfg.layers.append(DecoderLayerConfig(mixer=mixer, ff=0 if mlp is None else int(mlp["ff"]), mlp_act="gelu", post_norm=False))
    return cfg


class LupanexForCausalLM(DecoderForCausalLM):
    parse_config = staticmethod(parse_config)


__all__ = ["LupanexForCausalLM", "parse_config"]
