"""Pabalix: a small decoder-only language model whose layers are listed one by one in config.json ("layers"), each a latent-
attention mixer of one of three kinds and an optional gated-SiLU feed-forward with biases, with RMS norms on the input and the
output of every sublayer.

    latent_attention     rotate-half pairs, YaRN scaling
    latent_attention_2   interleaved pairs; may read an earlier layer's cached latents ("kv_from")
    latent_attention_3   rotate-half pairs, YaRN scaling, a softmax sink and an output gate per head

This module only reads the configuration: the mechanisms are weights.DecoderConfig's, the computation cogs_decoder_forward's,
generation and batching llm.CausalEngine's and llm.Sequences'."""
from __future__ import annotations

from typing import List, Optional, Sequence, Union

import torch

from . import checkpoint as ck
from .llm import DecoderEngine, Sequences
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


class PabalixForCausalLM:
    """the model object AutoModelForCausalLM.from_pretrained returns for architecture "Pabalix\""""

    def __init__(self, llm: DecoderEngine, generation_config: Optional[dict] = None):
        self.llm, self.config = llm, llm.cfg
        self.device, self.dtype = llm.device, llm.dtype
        self.generation_config = dict(generation_config or {})

    @classmethod
    def from_pretrained(cls, path: str, torch_dtype=None, device=None, **unused) -> "PabalixForCausalLM":
        cfg = parse_config(ck.read_config(path))
        dev = torch.device("cuda", torch.cuda.current_device()) if device is None else torch.device(device)
        if dev.type == "cuda" and dev.index is None:
            dev = torch.device("cuda", torch.cuda.current_device())
        state, reader = ck.open_decoder(path, cfg, dev)
        llm = DecoderEngine(state, cfg, dtype=torch_dtype or torch.bfloat16, device=dev)
        reader.check_consumed(extra_ok=[f"l{i}.{n}" for i, lay in enumerate(cfg.layers) if not lay.ff for n in ("norm2", "norm2b")])
        reader.close()
        model = cls(llm, ck.load_generation(path))
        model.name_or_path = path
        return model

    def to(self, device=None, *a, **k) -> "PabalixForCausalLM":
        if device is not None and not isinstance(device, torch.dtype):
            d = torch.device("cuda", device) if isinstance(device, int) else torch.device(device)
            if d.type != "cuda" or (d.index is not None and d.index != self.device.index):
                raise ValueError(f"model was loaded on {self.device}; load it with from_pretrained(device={d})")
        return self

    def eval(self) -> "PabalixForCausalLM":
        return self

    def sequences(self) -> Sequences:
        """an empty set of live requests for explicit steps"""
        return Sequences(self.llm)

    def generate(self, input_ids: Union[torch.Tensor, Sequence[int], Sequence[Sequence[int]]], *, max_new_tokens: int = 64,
                 **kw) -> List[List[int]]:
        """new token ids of every prompt. input_ids: one prompt (token ids or a 1-D tensor) or several of any lengths (a 2-D
        tensor: one per row). Options: CausalEngine.generate_batch's; the checkpoint's generation_config.json is the default."""
        if isinstance(input_ids, torch.Tensor):
            input_ids = input_ids.tolist()
        prompts = [list(p) for p in input_ids] if len(input_ids) and not isinstance(input_ids[0], int) else [list(input_ids)]
        opts = {k: v for k, v in self.generation_config.items() if k in ("do_sample", "temperature", "top_k", "top_p",
                                                                         "repetition_penalty", "eos_token_id")}
        opts.update(kw)
        if isinstance(opts.get("eos_token_id"), int):
            opts["eos_token_id"] = [opts["eos_token_id"]]
        return self.llm.generate_batch(prompts, max_new_tokens=max_new_tokens, **opts)


__all__ = ["PabalixForCausalLM", "parse_config"]
