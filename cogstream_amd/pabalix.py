"""Pabalix: a small decoder-only language model whose layers are listed one by one in config.json ("layers"), each a latent-
attention mixer of one of three kinds and an optional gated-SiLU feed-forward with biases, with RMS norms on the input and the
output of every sublayer.

    latent_attention     rotate-half pairs, YaRN scaling
    latent_attention_2   interleaved pairs; may read an earlier layer's cached latents ("kv_from")
    latent_attention_3   rotate-half pairs, YaRN scaling, a softmax sink and an output gate per head

This module only reads the configuration."""
from __future__ import annotations

from .decoder import DecoderForCausalLM
from .weights import DecoderConfig, DecoderLayerConfig, LatentAttention, Rotation, YarnScaling

KINDS = {"latent_attention": dict(interleaved=False, sink=False, gate=False),
         "latent_attention_2": dict(interleaved=True, sink=False, gate=False),
         "latent_attention_3": dict(interleaved=False, sink=True, gate=True)}


def parse_config(c: dict) -> DecoderConfig:
    """config.json -> weights.DecoderConfig"""
    cfg = DecoderConfig(width=int(c["width"]), vocab_size=int(c["vocab"]), eps=float(c["norm"]["eps"]))
    for i, lay in enumerate(c["layers"]):
        if lay["type"] not in KINDS:
            raise ValueError(f"layer {i}: mixer type {lay['type']!r} (known: {', '.join(KINDS)})")
        kind, m = KINDS[lay["type"]], lay["mixer"]
        s = m["rot"].get("scaling")
        rot = Rotation(dims=int(m["rot"]["dims"]), base=float(m["rot"]["base"]), interleaved=kind["interleaved"],
                       scaling=None if s is None else YarnScaling(float(s["factor"]), float(s["original"]), float(s["fast"]), float(s["slow"])))
        src = m.get("kv_from")
        if src is not None and not (0 <= src < i and cfg.layers[src].mixer.kv_from is None):
            raise ValueError(f"layer {i}: kv_from {src} is not an earlier layer with latents of its own")
        mixer = LatentAttention(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                                q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), rot=rot,
                                kv_from=src, sink=kind["sink"], gate=kind["gate"])
        mlp = lay.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: feed-forward kind {mlp['kind']!r} (known: dense)")
        cfg.layers.append(DecoderLayerConfig(mixer=mixer, ff=0 if mlp is None else int(mlp["ff"]), mlp_bias=True, post_norm=True))
    return cfg


class PabalixForCausalLM(DecoderForCausalLM):
    @staticmethod
    def parse_config(c, shapes):
        return parse_config(c)


__all__ = ["PabalixForCausalLM", "parse_config"]
