"""Oracle: the Pabalix decoder (a small decoder-only language model of latent-attention layers), one plain function per
mechanism, whole sequences only, no cache, no batching, one loop iteration per head and per query. TEST INFRASTRUCTURE
ONLY -- see oracle/__init__.py. Nothing here is shared with the product path.

A model is a dict `cfg` (the parsed config.json) and a dict `w` of tensors under the checkpoint's names. Everything is
computed in the dtype the weights have (the tests use float64 or float32); angles are always formed in float64."""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch


def rms(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def frequencies(rot: dict) -> Tuple[List[float], float]:
    """(rotation frequency of each pair, factor on cos and sin)"""
    n, base = rot["dims"], rot["base"]
    freq = [base ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if sc is None:
        return freq, 1.0

    def turning_dim(turns: float) -> float:      # the (fractional) pair index that makes `turns` turns over `original` positions
        return n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(turning_dim(sc["fast"])), 0)
    hi = min(math.ceil(turning_dim(sc["slow"])), n - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1


def rotate(x: torch.Tensor, rot: dict, interleaved: bool) -> torch.Tensor:
    """x [positions, dims]: row p rotated to position p"""
    n = rot["dims"]
    assert x.shape[-1] == n
    freq, mag = frequencies(rot)
    out = torch.empty_like(x)
    for i in range(n // 2):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + n // 2)
        ang = torch.arange(x.shape[0], dtype=torch.float64) * freq[i]
        c, s = (torch.cos(ang) * mag).to(x.dtype), (torch.sin(ang) * mag).to(x.dtype)
        out[:, a] = x[:, a] * c - x[:, b] * s
        out[:, b] = x[:, b] * c + x[:, a] * s
    return out


def sink_softmax(s: torch.Tensor, sink: Optional[torch.Tensor]) -> torch.Tensor:
    """weights of one query's visible keys; `sink` (a scalar) takes part in the sum only"""
    m = s.max() if sink is None else torch.maximum(s.max(), sink)
    e = torch.exp(s - m)
    z = e.sum()
    if sink is not None:
        z = z + torch.exp(sink - m)
    return e / z


def latents(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, mx: dict, eps: float, interleaved: bool):
    """what a layer with a W_dkv of its own stores: (normed latents [T, kv_rank], rotated shared key part [T, rot_dim])"""
    d = h @ w[pre + "dkv"].T
    c = rms(d[:, :mx["kv_rank"]], w[pre + "dkv.norm"], eps)
    return c, rotate(d[:, mx["kv_rank"]:], mx["rot"], interleaved)


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, layer: dict, eps: float, stored) -> torch.Tensor:
    """`stored` = (latents, rotated key part) of this layer or of the layer it borrows from"""
    mx, kind = layer["mixer"], layer["type"]
    interleaved = kind == "latent_attention_2"
    H, dn, dr, dv = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    T = h.shape[0]
    c, kr = stored
    q = rms(h @ w[pre + "dq"].T, w[pre + "dq.norm"], eps) @ w[pre + "uq"].T
    heads = []
    for hd in range(H):
        qh = q[:, hd * (dn + dr):(hd + 1) * (dn + dr)]
        qn, qr = qh[:, :dn], rotate(qh[:, dn:], mx["rot"], interleaved)
        kn = c @ w[pre + "uk"][hd * dn:(hd + 1) * dn].T
        v = c @ w[pre + "uv"][hd * dv:(hd + 1) * dv].T
        s = (qn @ kn.T + qr @ kr.T) * mx["scale"]
        sink = w[pre + "sink"][hd] if kind == "latent_attention_3" else None
        o = torch.stack([sink_softmax(s[i, :i + 1], sink) @ v[:i + 1] for i in range(T)])
        if kind == "latent_attention_3":
            o = o * (1 / (1 + torch.exp(-(h @ w[pre + "g"][hd]))))[:, None]
        heads.append(o)
    return torch.cat(heads, dim=1) @ w[pre + "o"].T


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    g = h @ w[pre + "gate"].T + w[pre + "gate.b"]
    u = h @ w[pre + "up"].T + w[pre + "up.b"]
    return (silu(g) * u) @ w[pre + "down"].T + w[pre + "down.b"]


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int]) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """-> (logits [T, vocab], residual stream behind every layer)"""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    stored, streams = {}, []
    for i, layer in enumerate(cfg["layers"]):
        pre, mx = f"l{i}.", layer["mixer"]
        h = rms(x, w[pre + "norm1"], eps)
        src = mx.get("kv_from")
        if src is None:
            stored[i] = latents(h, w, pre + "mix.", mx, eps, layer["type"] == "latent_attention_2")
        a = latent_attention(h, w, pre + "mix.", layer, eps, stored[i if src is None else src])
        x = x + rms(a, w[pre + "norm1b"], eps)
        if layer.get("mlp") is not None:
            x = x + rms(feed_forward(rms(x, w[pre + "norm2"], eps), w, pre + "mlp."), w[pre + "norm2b"], eps)
        streams.append(x)
    return rms(x, w["final.norm"], eps) @ w["head"].T, streams


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(cfg, w, seq)[0][-1].argmax()))
    return seq[len(prompt):]
