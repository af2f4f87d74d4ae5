"""Oracle: the Lupanex decoder (attention layers with a distance bias, gated delta-rule layers, hyper-connected residual
streams, looped layers), one plain function per mechanism, whole sequences only, no cache, no batching, one token or query at
a time. TEST INFRASTRUCTURE ONLY -- see oracle/__init__.py. Nothing here is shared with the product path.

A model is a dict `cfg` (the parsed config.json) and a dict `w` of tensors under the checkpoint's names. Everything is
computed in the dtype the weights have (the tests use float64)."""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1 / (1 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def gelu(z: torch.Tensor) -> torch.Tensor:
    return z * (1 + torch.erf(z / math.sqrt(2))) / 2


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


# ------------------------------------------------------------------------------------------------ attention
def bucket(n: int, rows: int, far: float) -> int:
    """the bias row of distance n: one each below rows / 2, then logarithmic up to distance `far`, then the last"""
    half = rows // 2
    if n < half:
        return n
    r = math.log(n / half) / math.log(far / half) * (rows - half)
    k = round(r) if abs(r - round(r)) < 1e-9 else math.floor(r)
    return min(rows - 1, half + k)


def temperature(p: int, q_temp: Optional[dict]) -> float:
    if q_temp is None:
        return 1.0
    return 1 + q_temp["coef"] * math.log(math.floor((p + 1) / q_temp["every"]) + 1)


def softmax(s: torch.Tensor) -> torch.Tensor:
    e = torch.exp(s - s.max())
    return e / e.sum()


def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float) -> torch.Tensor:
    H, G, d, dv, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    rel = w[pre + "rel"]
    dist = torch.tensor([bucket(n, rel.shape[0], m["bias_max"]) for n in range(T)])
    temp = torch.tensor([temperature(p, m.get("q_temp")) for p in range(T)], dtype=h.dtype)
    heads = []
    for i in range(H):
        g = i // (H // G)
        q = rms(h @ w[pre + "q"][i * d:(i + 1) * d].T, eps) * temp[:, None]
        k = rms(h @ w[pre + "k"][g * d:(g + 1) * d].T, eps)
        v = h @ w[pre + "v"][g * dv:(g + 1) * dv].T
        out = []
        for p in range(T):
            s = (k[:p + 1] @ q[p]) * m["scale"] + rel[dist[:p + 1].flip(0), i]
            out.append(softmax(s) @ v[:p + 1])
        heads.append(torch.stack(out))
    return torch.cat(heads, dim=1) @ w[pre + "o"].T


# ------------------------------------------------------------------------------------------------ gated delta rule
def short_conv(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """x [T, channels], taps [channels, n]: y_t = sum_j taps[:, n - 1 - j] x_{t - j}, zeros before the start"""
    n, out = taps.shape[1], []
    for t in range(x.shape[0]):
        y = torch.zeros_like(x[0])
        for j in range(min(n, t + 1)):
            y = y + taps[:, n - 1 - j] * x[t - j]
        out.append(y)
    return torch.stack(out)


def delta_recurrence(q, k, v, beta, g) -> torch.Tensor:
    """one head: q, k [T, d], v [T, dv], beta, g [T] -> read-outs [T, dv]"""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype)
    out = []
    for t in range(q.shape[0]):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out.append(S.T @ q[t])
    return torch.stack(out)


def delta(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float) -> torch.Tensor:
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w[pre + n].T, w[pre + n + ".conv"])) for n in "qkv")
    beta = sigmoid(h @ w[pre + "b"].T)
    z = h @ w[pre + "a"].T + w[pre + "dt_bias"]
    softplus = torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))
    decay = torch.exp(-torch.exp(w[pre + "A_log"]) * softplus)
    gate = silu(h @ w[pre + "g"].T)
    heads = []
    for i in range(H):
        j = i // (H // G)
        qh, kh = unit(q[:, j * d:(j + 1) * d]) * d ** -0.5, unit(k[:, j * d:(j + 1) * d])
        o = delta_recurrence(qh, kh, v[:, i * dv:(i + 1) * dv], beta[:, i], decay[:, i])
        heads.append(rms(o, eps) * w[pre + "norm"] * gate[:, i * dv:(i + 1) * dv])
    return torch.cat(heads, dim=1) @ w[pre + "o"].T


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    return gelu(h @ w[pre + "up"].T) @ w[pre + "down"].T


# ------------------------------------------------------------------------------------------------ the model
MIXERS = {"attention": attention, "delta": delta}


def read(xs: List[torch.Tensor], w, pre: str) -> torch.Tensor:
    if pre + "in" not in w:                # one plain residual stream
        return xs[0]
    u = torch.zeros_like(xs[0])
    for s, x in enumerate(xs):
        u = u + w[pre + "in"][s] * x
    return u


def write(xs: List[torch.Tensor], y: torch.Tensor, w, pre: str) -> List[torch.Tensor]:
    if pre + "in" not in w:
        return [xs[0] + y]
    out = []
    for t in range(len(xs)):
        z = w[pre + "out"][t] * y
        for s in range(len(xs)):
            z = z + w[pre + "mix"][s, t] * xs[s]
        out.append(z)
    return out


def order(cfg: dict) -> List[int]:
    """the layer of every layer run"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int]) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """-> (logits [T, vocab], sum of the residual streams behind every layer run)"""
    eps = cfg["norm"]["eps"]
    T = len(tokens)
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"] + w["pos"][:T]
    xs, states = [x] * cfg.get("streams", 1), []
    for i in order(cfg):
        lay, p = cfg["layers"][i], f"l{i}."
        h = rms(read(xs, w, p + "hc1."), eps) * w[p + "norm1"]
        xs = write(xs, MIXERS[lay["type"]](h, w, p + "mix.", lay["mixer"], eps), w, p + "hc1.")
        if lay.get("mlp") is not None:
            h = rms(read(xs, w, p + "hc2."), eps) * w[p + "norm2"]
            xs = write(xs, feed_forward(h, w, p + "mlp."), w, p + "hc2.")
        states.append(sum(xs))
    return rms(sum(xs), eps) * w["final.norm"] @ w["head"].T, states


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(cfg, w, seq)[0][-1].argmax()))
    return seq[len(prompt):]
