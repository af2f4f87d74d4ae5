"""The model object of decoder-only language models described layer by layer: an architecture is a function that reads its
config.json into weights.DecoderConfig (pabalix.py, lupanex.py) and a subclass of DecoderForCausalLM that names it. Mechanisms are
weights.DecoderConfig's, the computation cogs_decoder_forward's, generation and batching llm.CausalEngine's and llm.Sequences'."""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple, Union

import torch

from . import checkpoint as ck
from .llm import DecoderEngine, Sequences
from .weights import DecoderConfig


class DecoderForCausalLM:
    """what AutoModelForCausalLM.from_pretrained returns for such an architecture"""

    @staticmethod
    def parse_config(c: dict, shapes: Dict[str, Tuple[int, ...]]) -> DecoderConfig:
        """config.json, and the shapes of the checkpoint's tensors for sizes that only these give"""
        raise NotImplementedError

    def __init__(self, llm: DecoderEngine, generation_config: Optional[dict] = None):
        self.llm, self.config = llm, llm.cfg
        self.device, self.dtype = llm.device, llm.dtype
        self.generation_config = dict(generation_config or {})

    @classmethod
    def from_pretrained(cls, path: str, torch_dtype=None, device=None, **unused) -> "DecoderForCausalLM":
        cfg = cls.parse_config(ck.read_config(path), ck.tensor_shapes(path))
        dev = torch.device("cuda", torch.cuda.current_device()) if device is None else torch.device(device)
        if dev.type == "cuda" and dev.index is None:
            dev = torch.device("cuda", torch.cuda.current_device())
        state, reader = ck.open_decoder(path, cfg, dev)
        llm = DecoderEngine(state, cfg, dtype=torch_dtype or torch.bfloat16, device=dev)
        reader.check_consumed(extra_ok=[f"l{i}.{n}" for i, lay in enumerate(cfg.layers) if not lay.ff
                                        for n in ("norm2", "norm2b", "hc2.in", "hc2.out", "hc2.mix")])
        reader.close()
        model = cls(llm, ck.load_generation(path))
        model.name_or_path = path
        return model

    def to(self, device=None, *a, **k) -> "DecoderForCausalLM":
        if device is not None and not isinstance(device, torch.dtype):
            d = torch.device("cuda", device) if isinstance(device, int) else torch.device(device)
            if d.type != "cuda" or (d.index is not None and d.index != self.device.index):
                raise ValueError(f"model was loaded on {self.device}; load it with from_pretrained(device={d})")
        return self

    def eval(self) -> "DecoderForCausalLM":
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


__all__ = ["DecoderForCausalLM"]
