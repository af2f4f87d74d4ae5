"""Weight containers and the one-off packing into the layouts the HIP kernels expect.

Names follow the reference checkpoint (model/model.safetensors.index.json; module tree
model/cogreasoner_chat.py:214-248,591-598): model.vision_encoder.*, model.mm_projector.readout.{0,2}.*,
model.embed_tokens, model.layers.N.*, model.norm, lm_head. Packing rules are documented in include/cogs.h:
  * q/k rows of every head interleaved as rotary pairs (d, d+hd/2) -> (2i, 2i+1);
  * q,k,v stacked into one [.., hidden] matrix; gate/up rows interleaved;
  * K dimensions zero-padded to the GEMM slab (64 bf16 / 32 fp32 elements).
torch is used here for tensor storage and the one-time reshuffles only."""
from __future__ import annotations

import ctypes as C
import math
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple, Union

import torch

from . import _lib as L
from .ops import k_slab, pad_cols


@dataclass
class VisionConfig:
    """model/config.json:35-42 (vision_encoder_config) + configuration_videollama3_encoder.py:22-49"""
    hidden_size: int = 1152
    intermediate_size: int = 4304
    num_hidden_layers: int = 27
    num_attention_heads: int = 16
    num_channels: int = 3
    patch_size: int = 14
    layer_norm_eps: float = 1e-6

    @property
    def patch_dim(self) -> int:
        return self.num_channels * self.patch_size * self.patch_size


@dataclass
class LlmConfig:
    """model/config.json:12-43"""
    hidden_size: int = 3584
    intermediate_size: int = 18944
    num_hidden_layers: int = 28
    num_attention_heads: int = 28
    num_key_value_heads: int = 4
    vocab_size: int = 152064
    rms_norm_eps: float = 1e-6
    rope_theta: float = 1e6
    image_token_index: int = 151665
    eos_token_id: int = 151645

    @property
    def head_dim(self) -> int:
        return self.hidden_size // self.num_attention_heads


@dataclass
class YarnScaling:
    """context extension by slowing the pairs that turn rarely: pairs making more than `fast` turns over `original`
    positions keep their frequency, pairs making fewer than `slow` are divided by `factor`, a ramp between"""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass
class Rotation:
    """rotary positions over `dims` dimensions: pair i is (2i, 2i+1) if interleaved, else (i, i + dims/2)"""
    dims: int
    base: float
    interleaved: bool = False
    scaling: Optional[YarnScaling] = None

    def frequencies(self) -> List[float]:
        """radians per position of every pair (float64)"""
        n, s = self.dims, self.scaling
        freq = [self.base ** (-2.0 * i / n) for i in range(n // 2)]
        if s is None:
            return freq
        index = lambda turns: n * math.log(s.original / (2 * math.pi * turns)) / (2 * math.log(self.base))
        lo, hi = max(math.floor(index(s.fast)), 0), min(math.ceil(index(s.slow)), n - 1)
        ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(n // 2)]
        return [f / s.factor * r + f * (1.0 - r) for f, r in zip(freq, ramp)]

    @property
    def magnitude(self) -> float:
        """factor on cos and sin"""
        return 1.0 if self.scaling is None else 0.1 * math.log(self.scaling.factor) + 1.0

    def pair_order(self) -> torch.Tensor:
        """the packed order of the rotated rows: pairs adjacent"""
        return torch.arange(self.dims) if self.interleaved else rope_perm(self.dims)


@dataclass
class LatentAttention:
    """multi-head latent attention (include/cogs.h, cogs_latent_mixer)"""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: Rotation
    kv_from: Optional[int] = None      # earlier layer whose cached latents this layer reads
    sink: bool = False                 # a learned logit per head in the softmax sum
    gate: bool = False                 # sigmoid gate per head on the output


@dataclass
class DistanceBias:
    """a learned score bias per head and bucket of distances: one bucket per distance below buckets / 2, logarithmically wider ones
    up to distance `far`, the last for everything from there on"""
    buckets: int
    far: float

    def bucket_of(self) -> List[int]:
        """the bucket of every distance 0, 1, .. up to the first whose bucket is the last (all later ones share it)"""
        half = self.buckets // 2
        if half < 1 or self.far <= half:
            raise ValueError(f"distance bias of {self.buckets} buckets up to distance {self.far}: no room for logarithmic buckets")
        out: List[int] = []
        while not out or out[-1] < self.buckets - 1:
            n = len(out)
            if n < half:
                out.append(n)
                continue
            r = math.log(n / half) / math.log(self.far / half) * (self.buckets - half)
            near = round(r)            # a quotient of logarithms that is a whole number may come out just below it
            out.append(min(self.buckets - 1, half + (near if abs(r - near) < 1e-9 else math.floor(r))))
        return out


@dataclass
class HeadAttention:
    """softmax attention with keys and values per (shared) head (include/cogs.h, cogs_attn_mixer)"""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    qk_norm: bool = False              # weightless RMS norm of every query and key head row
    temp_coef: float = 0.0             # queries times 1 + temp_coef ln(floor((p + 1) / temp_every) + 1); temp_every 0: none
    temp_every: float = 0.0
    bias: Optional[DistanceBias] = None


@dataclass
class DeltaRule:
    """gated delta rule behind short causal convolutions (include/cogs.h, cogs_delta_mixer)"""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int


@dataclass
class DecoderLayerConfig:
    mixer: Union[LatentAttention, HeadAttention, DeltaRule]
    ff: int = 0                        # MLP width, 0 = no feed-forward sublayer
    mlp_act: str = "swiglu"            # "swiglu" (gated) or "gelu" (exact, up and down only)
    mlp_bias: bool = False
    post_norm: bool = True             # norms on the sublayers' outputs


@dataclass
class Loop:
    """layers start .. stop - 1 run `times` times in a row"""
    start: int
    stop: int
    times: int


@dataclass
class DecoderConfig:
    """a decoder-only model described layer by layer"""
    width: int
    vocab_size: int
    eps: float
    layers: List[DecoderLayerConfig] = field(default_factory=list)
    embed_scale: float = 1.0
    max_positions: int = 0             # > 0: a learned vector per position joins the embedding
    streams: int = 0                   # > 0: hyper-connected residual streams
    loop: Optional[Loop] = None

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[int]:
        """the layer of every layer run, loop passes unrolled"""
        n, lp = len(self.layers), self.loop
        if lp is None:
            return list(range(n))
        return [*range(lp.start), *[i for _ in range(lp.times) for i in range(lp.start, lp.stop)], *range(lp.stop, n)]


def rope_perm(hd: int) -> torch.Tensor:
    """new row 2i <- old i, 2i+1 <- old i + hd/2"""
    return torch.arange(hd).view(2, hd // 2).t().reshape(-1)


def _perm_heads(w: torch.Tensor, heads: int, hd: int) -> torch.Tensor:
    p = rope_perm(hd).to(w.device)
    shp = w.shape
    return w.reshape(heads, hd, *shp[1:])[:, p].reshape(shp)


def _pad_rows(x: torch.Tensor, rows: int) -> torch.Tensor:
    if x.shape[0] == rows:
        return x.contiguous()
    out = x.new_zeros(rows, *x.shape[1:])
    out[: x.shape[0]] = x
    return out


def zero_sum_rows(wf: torch.Tensor) -> torch.Tensor:
    """Make every row of a bf16 matrix sum to (essentially) zero by moving a few of its entries ONE bf16 step.
    A centred row rounded to bf16 keeps a row sum s of about sqrt(K/12) steps; the folded-LayerNorm GEMM never evaluates
    the term rstd * mean * s (include/cogs.h, cogs_gemm_desc.ln_ab), so s is an error that grows with |mean / std| of an
    activation row. Greedy, exact in fp64: starting at the row's most populated binade (many candidates, small steps)
    and going down binade by binade, floor(|s| / step) entries of that binade move one step against the sign of s. What
    is left is smaller than one step of the row's smallest entries. A moved entry is still a correctly rounded bf16
    neighbour of its exact value (error < 1.5 steps instead of <= 0.5); about ten of 1152 entries move."""
    assert wf.dtype == torch.bfloat16 and wf.dim() == 2
    w = wf.double()
    mag = w.abs()
    tiny = 2.0 ** -126
    expo = torch.floor(torch.log2(mag.clamp_min(tiny)))
    # log2 of an exact power of two is exact in fp64, but guard the binade edges against a 1-ulp slip of log2
    expo = torch.where(torch.ldexp(torch.ones_like(mag), expo.int()) > mag, expo - 1, expo)
    expo = torch.where(torch.ldexp(torch.ones_like(mag), (expo + 1).int()) <= mag, expo + 1, expo)
    live = mag >= 2.0 ** -100                       # zeros (padding rows / columns) and denormal dust never move
    s = w.sum(dim=1)
    if not bool(live.any()):
        return wf
    e_hi = int(expo[live].max().item())
    e_lo = int(expo[live].min().item())
    # per row: the most populated binade
    levels = torch.arange(e_lo, e_hi + 1, device=w.device, dtype=torch.float64)
    counts = torch.stack([((expo == lv) & live).sum(dim=1) for lv in levels.tolist()], dim=1)       # [rows, levels]
    start = levels[counts.argmax(dim=1)]                                                              # [rows]
    start_max = float(start.max().item())
    for lv in reversed(levels.tolist()):
        if lv > start_max:
            continue
        step = 2.0 ** (lv - 7)                      # bf16: 8 significant bits
        want = torch.floor(s.abs() / step)
        if not bool((want > 0).any()):               # no row has a whole step of this binade left to shed
            continue
        cand = (expo == lv) & live & (start >= lv)[:, None]
        rank = torch.cumsum(cand.to(torch.int32), dim=1)
        take = cand & (rank.double() <= want[:, None])
        delta = -torch.sign(s)[:, None] * step * take.double()
        w = w + delta
        s = s + delta.sum(dim=1)
    out = w.to(torch.bfloat16)
    assert bool((out.double() == w).all()), "a moved weight is not a bf16 value"
    return out


def fold_layernorm(w: torch.Tensor, b: torch.Tensor, gamma: torch.Tensor, beta: torch.Tensor):
    """Linear(LayerNorm(x)) with the affine part folded into the linear layer (modeling_videollama3_encoder.py:382-391):
    LN(x) W^T + b = rstd (x - mean) (W diag(gamma))^T + (b + W beta). The rows of W' = W diag(gamma) are CENTRED (their
    mean over the input dimension subtracted; zero-padded input columns excluded): sum_k x_k W''[n][k] then equals
    sum_k (x_k - mean) W'[n][k] and the GEMM epilogue only evaluates rstd * acc + c (cogs_gemm_desc.ln_ab / col_c). In
    bf16 the ROUNDED rows are made zero-sum as well (zero_sum_rows), which is what the contract in include/cogs.h asks
    for. Returns (W'' in W's dtype, s = fp32 row sums of the stored W'' (~0; for tests), c = fp32 b + W beta)."""
    wd = w.double() * gamma.double()[None, :]
    wd = wd - wd.mean(dim=1, keepdim=True)
    wf = wd.to(w.dtype)
    if wf.dtype == torch.bfloat16:
        wf = zero_sum_rows(wf)
    s = wf.double().sum(dim=1).float().contiguous()
    c = (b.double() + w.double() @ beta.double()).float().contiguous()
    return wf.contiguous(), s, c


class PackedVit:
    def __init__(self, state: Dict[str, torch.Tensor], cfg: VisionConfig, dtype=torch.bfloat16, device="cuda",
                 fold_ln: Optional[bool] = None):
        """fold_ln (default: bf16 yes, fp32 no): fold layer_norm1 into the QKV projection and layer_norm2 into fc1"""
        self.cfg, self.dtype, self.device = cfg, dtype, torch.device(device)
        self.fold_ln = (dtype == torch.bfloat16 and cfg.hidden_size % 64 == 0) if fold_ln is None else bool(fold_ln)
        slab = k_slab(dtype)
        H, I, hd = cfg.hidden_size, cfg.intermediate_size, cfg.hidden_size // cfg.num_attention_heads
        self.inter_pad = (I + slab - 1) // slab * slab
        self.patch_pad = (cfg.patch_dim + slab - 1) // slab * slab
        cv = lambda t: t.to(device=self.device, dtype=dtype)
        self.keep: List[torch.Tensor] = []

        def hold(t):
            t = t.contiguous()
            self.keep.append(t)
            return t

        g = lambda k: cv(state[k])
        self.patch_w = hold(pad_cols(g("embeddings.patch_embedding.weight").reshape(H, -1), slab))
        self.patch_b = hold(g("embeddings.patch_embedding.bias"))
        self.post_g = hold(g("post_layernorm.weight"))
        self.post_b = hold(g("post_layernorm.bias"))
        self.layers = (L.VitLayer * cfg.num_hidden_layers)()
        for i in range(cfg.num_hidden_layers):
            p = f"encoder.layers.{i}."
            a = p + "self_attn."
            qw = _perm_heads(g(a + "q_proj.weight"), cfg.num_attention_heads, hd)
            kw = _perm_heads(g(a + "k_proj.weight"), cfg.num_attention_heads, hd)
            qb = _perm_heads(g(a + "q_proj.bias"), cfg.num_attention_heads, hd)
            kb = _perm_heads(g(a + "k_proj.bias"), cfg.num_attention_heads, hd)
            lay = self.layers[i]
            ln1_g, ln1_b = hold(g(p + "layer_norm1.weight")), hold(g(p + "layer_norm1.bias"))
            lay.ln1_g, lay.ln1_b = ln1_g.data_ptr(), ln1_b.data_ptr()
            qkv_w = torch.cat([qw, kw, g(a + "v_proj.weight")], 0)
            qkv_b = hold(torch.cat([qb, kb, g(a + "v_proj.bias")], 0))
            if self.fold_ln:
                qkv_w, _, c_ = fold_layernorm(qkv_w, qkv_b, ln1_g, ln1_b)
                lay.qkv_c = hold(c_).data_ptr()
            lay.qkv_w = hold(qkv_w).data_ptr()
            lay.qkv_b = qkv_b.data_ptr()
            lay.o_w = hold(g(a + "out_proj.weight")).data_ptr()
            lay.o_b = hold(g(a + "out_proj.bias")).data_ptr()
            ln2_g, ln2_b = hold(g(p + "layer_norm2.weight")), hold(g(p + "layer_norm2.bias"))
            lay.ln2_g, lay.ln2_b = ln2_g.data_ptr(), ln2_b.data_ptr()
            fc1_w = _pad_rows(g(p + "mlp.fc1.weight"), self.inter_pad)
            fc1_b = hold(_pad_rows(g(p + "mlp.fc1.bias"), self.inter_pad))
            if self.fold_ln:
                fc1_w, _, c_ = fold_layernorm(fc1_w, fc1_b, ln2_g, ln2_b)
                lay.fc1_c = hold(c_).data_ptr()
            lay.fc1_w = hold(fc1_w).data_ptr()
            lay.fc1_b = fc1_b.data_ptr()
            lay.fc2_w = hold(pad_cols(g(p + "mlp.fc2.weight"), slab)).data_ptr()
            lay.fc2_b = hold(g(p + "mlp.fc2.bias")).data_ptr()
        w = L.VitWeights()
        w.dtype = L.dtype_code(dtype)
        w.hidden, w.inter_pad, w.layers, w.heads = H, self.inter_pad, cfg.num_hidden_layers, cfg.num_attention_heads
        w.patch_dim, w.patch_pad, w.ln_eps = cfg.patch_dim, self.patch_pad, cfg.layer_norm_eps
        w.patch_w, w.patch_b = self.patch_w.data_ptr(), self.patch_b.data_ptr()
        w.post_ln_g, w.post_ln_b = self.post_g.data_ptr(), self.post_b.data_ptr()
        w.layer = C.cast(self.layers, C.POINTER(L.VitLayer))
        self.struct = w


class PackedProjector:
    def __init__(self, state: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cuda"):
        cv = lambda t: t.to(device=device, dtype=dtype).contiguous()
        self.w1, self.b1 = cv(state["readout.0.weight"]), cv(state["readout.0.bias"])
        self.w2, self.b2 = cv(state["readout.2.weight"]), cv(state["readout.2.bias"])
        w = L.ProjWeights()
        w.dtype = L.dtype_code(dtype)
        w.in_dim, w.out_dim = self.w1.shape[1], self.w1.shape[0]
        w.w1, w.b1, w.w2, w.b2 = self.w1.data_ptr(), self.b1.data_ptr(), self.w2.data_ptr(), self.b2.data_ptr()
        self.struct = w
        self.in_dim, self.out_dim = w.in_dim, w.out_dim


class PackedLlm:
    def __init__(self, state: Dict[str, torch.Tensor], cfg: LlmConfig, dtype=torch.bfloat16, device="cuda"):
        self.cfg, self.dtype, self.device = cfg, dtype, torch.device(device)
        hd, hq, hkv = cfg.head_dim, cfg.num_attention_heads, cfg.num_key_value_heads
        cv = lambda t: t.to(device=self.device, dtype=dtype)
        self.keep: List[torch.Tensor] = []

        def hold(t):
            t = t.contiguous()
            self.keep.append(t)
            return t

        g = lambda k: cv(state[k])
        self.embed = hold(g("embed_tokens.weight"))
        self.final_norm = hold(g("norm.weight"))
        self.lm_head = hold(g("lm_head.weight"))
        self.layers = (L.LlmLayer * cfg.num_hidden_layers)()
        for i in range(cfg.num_hidden_layers):
            p = f"layers.{i}."
            a = p + "self_attn."
            qw, qb = _perm_heads(g(a + "q_proj.weight"), hq, hd), _perm_heads(g(a + "q_proj.bias"), hq, hd)
            kw, kb = _perm_heads(g(a + "k_proj.weight"), hkv, hd), _perm_heads(g(a + "k_proj.bias"), hkv, hd)
            lay = self.layers[i]
            lay.in_ln = hold(g(p + "input_layernorm.weight")).data_ptr()
            lay.qkv_w = hold(torch.cat([qw, kw, g(a + "v_proj.weight")], 0)).data_ptr()
            lay.qkv_b = hold(torch.cat([qb, kb, g(a + "v_proj.bias")], 0)).data_ptr()
            lay.o_w = hold(g(a + "o_proj.weight")).data_ptr()
            lay.post_ln = hold(g(p + "post_attention_layernorm.weight")).data_ptr()
            gu = torch.stack([g(p + "mlp.gate_proj.weight"), g(p + "mlp.up_proj.weight")], dim=1)
            lay.gu_w = hold(gu.reshape(2 * cfg.intermediate_size, cfg.hidden_size)).data_ptr()
            lay.down_w = hold(g(p + "mlp.down_proj.weight")).data_ptr()
        w = L.LlmWeights()
        w.dtype = L.dtype_code(dtype)
        w.hidden, w.inter, w.layers = cfg.hidden_size, cfg.intermediate_size, cfg.num_hidden_layers
        w.heads, w.kv_heads, w.head_dim, w.vocab = hq, hkv, hd, cfg.vocab_size
        w.rms_eps, w.rope_theta = cfg.rms_norm_eps, cfg.rope_theta
        w.final_norm, w.lm_head = self.final_norm.data_ptr(), self.lm_head.data_ptr()
        w.layer = C.cast(self.layers, C.POINTER(L.LlmLayer))
        self.struct = w


def _up(v: int, m: int) -> int:
    return (v + m - 1) // m * m


def _pad_to(x: torch.Tensor, *shape: int) -> torch.Tensor:
    if tuple(x.shape) == shape:
        return x.contiguous()
    out = x.new_zeros(*shape)
    out[tuple(slice(0, n) for n in x.shape)] = x
    return out


def decoder_tensors(cfg: DecoderConfig) -> Dict[str, Tuple[int, ...]]:
    """name -> shape of every tensor of a decoder described layer by layer"""
    W = cfg.width
    out: Dict[str, Tuple[int, ...]] = {"embed": (cfg.vocab_size, W), "final.norm": (W,), "head": (cfg.vocab_size, W)}
    if cfg.max_positions:
        out["pos"] = (cfg.max_positions, W)
    for i, lay in enumerate(cfg.layers):
        p, m = f"l{i}.", lay.mixer
        for n in ("1", "2") if lay.ff else ("1",):
            out[p + "norm" + n] = (W,)
            if lay.post_norm:
                out[p + f"norm{n}b"] = (W,)
            if cfg.streams:
                s = cfg.streams
                out[p + f"hc{n}.in"], out[p + f"hc{n}.out"], out[p + f"hc{n}.mix"] = (s,), (s,), (s, s)
        if lay.ff:
            for n, shape in (("gate", (lay.ff, W)), ("up", (lay.ff, W)), ("down", (W, lay.ff))):
                if n == "gate" and lay.mlp_act != "swiglu":
                    continue
                out[p + "mlp." + n] = shape
                if lay.mlp_bias:
                    out[p + f"mlp.{n}.b"] = shape[:1]
        out[p + "mix.o"] = (W, m.heads * m.vdim)
        if not isinstance(m, LatentAttention):
            rows = {"q": m.heads * m.dim, "k": m.kv_heads * m.dim, "v": m.kv_heads * m.vdim}
            if isinstance(m, DeltaRule):
                rows = {"q": m.kv_heads * m.dim, "k": m.kv_heads * m.dim, "v": m.heads * m.vdim}
                for n in "qkv":
                    out[p + f"mix.{n}.conv"] = (rows[n], m.taps)
                out[p + "mix.A_log"] = out[p + "mix.dt_bias"] = (m.heads,)
                out[p + "mix.norm"] = (m.vdim,)
                rows.update(g=m.heads * m.vdim, b=m.heads, a=m.heads)
            elif m.bias is not None:
                out[p + "mix.rel"] = (m.bias.buckets, m.heads)
            for n, r in rows.items():
                out[p + "mix." + n] = (r, W)
            continue
        out[p + "mix.dq"], out[p + "mix.dq.norm"] = (m.q_rank, W), (m.q_rank,)
        out[p + "mix.uq"] = (m.heads * (m.dim + m.rot_dim), m.q_rank)
        if m.kv_from is None:
            out[p + "mix.dkv"], out[p + "mix.dkv.norm"] = (m.kv_rank + m.rot_dim, W), (m.kv_rank,)
        out[p + "mix.uk"], out[p + "mix.uv"] = (m.heads * m.dim, m.kv_rank), (m.heads * m.vdim, m.kv_rank)
        if m.sink:
            out[p + "mix.sink"] = (m.heads,)
        if m.gate:
            out[p + "mix.g"] = (m.heads, W)
    return out


class PackedDecoder:
    """decoder_tensors -> the layouts of include/cogs.h (cogs_decoder_*): padded sizes, projections of a mixer stacked, rotary pairs
    adjacent, gate / up rows interleaved, W_uk also transposed per head for the absorbed decode, bias tables by distance"""

    def __init__(self, state: Dict[str, torch.Tensor], cfg: DecoderConfig, dtype=torch.bfloat16, device="cuda"):
        self.cfg, self.dtype, self.device = cfg, dtype, torch.device(device)
        self.keep: List[object] = []
        self.state = state
        self.width_p, self.vocab_p = _up(cfg.width, 64), _up(cfg.vocab_size, 4)
        Wp = self.width_p
        self.embed = self._hold(_pad_to(self._get("embed"), cfg.vocab_size, Wp))
        self.head = self._hold(_pad_to(self._get("head"), self.vocab_p, Wp))
        self.layers = (L.DecoderLayer * len(cfg.layers))()
        widths: List[List[int]] = []          # per layer: columns of its blocks in a token's cache
        states: List[int] = []                # per layer: floats of recurrent state
        for i, lc in enumerate(cfg.layers):
            p, lay, m = f"l{i}.", self.layers[i], lc.mixer
            for n in ("1", "2") if lc.ff else ("1",):
                setattr(lay, "norm" + n, self._vec(p + "norm" + n, Wp))
                if lc.post_norm:
                    setattr(lay, f"norm{n}b", self._vec(p + f"norm{n}b", Wp))
                if cfg.streams:
                    s, hc = cfg.streams, getattr(lay, "hyper" + n)
                    hc.in_, hc.out = self._vec(p + f"hc{n}.in", s), self._vec(p + f"hc{n}.out", s)
                    hc.mix = self._vec(p + f"hc{n}.mix", s, s)
            if isinstance(m, LatentAttention):
                lay.mixer = L.MIX_LATENT
                blocks, floats = self._latent(lay.latent, p + "mix.", m, i)
            elif isinstance(m, HeadAttention):
                lay.mixer = L.MIX_ATTENTION
                blocks, floats = self._heads(lay.attn, p + "mix.", m)
            else:
                lay.mixer = L.MIX_DELTA
                blocks, floats = self._delta(lay.delta, p + "mix.", m)
            widths.append(blocks)
            states.append(floats)
            dv = _up(m.vdim, 16)
            o = _pad_to(self._get(p + "mix.o").view(cfg.width, m.heads, m.vdim), Wp, m.heads, dv).view(Wp, m.heads * dv)
            getattr(lay, ("latent", "attn", "delta")[lay.mixer]).o_w = self._hold(_pad_to(o, Wp, _up(m.heads * dv, 64))).data_ptr()
            if lc.ff:
                self._mlp(lay.mlp, p + "mlp.", lc)
        w = L.DecoderWeights()
        w.dtype, w.width, w.vocab, w.layers, w.eps = L.dtype_code(dtype), cfg.width, cfg.vocab_size, len(cfg.layers), cfg.eps
        w.embed_scale, w.max_positions, w.streams = cfg.embed_scale, cfg.max_positions, cfg.streams
        if cfg.max_positions:
            w.pos = self._hold(_pad_to(self._get("pos"), cfg.max_positions, Wp)).data_ptr()
        if cfg.loop is not None:
            w.loop_start, w.loop_stop, w.loop_times = cfg.loop.start, cfg.loop.stop, cfg.loop.times
        w.final_norm, w.head = self._vec("final.norm", Wp), self.head.data_ptr()
        w.layer = C.cast(self.layers, C.POINTER(L.DecoderLayer))
        self.struct = w
        del self.state
        # columns of every cached block in a token's cache, and floats of state, in the order of the layer runs
        self.cache_widths = [b for i in cfg.runs() for b in widths[i]]
        self.state_floats = sum(states[i] for i in cfg.runs())

    def _hold(self, t: torch.Tensor) -> torch.Tensor:
        t = t.contiguous()
        self.keep.append(t)
        return t

    def _get(self, k: str) -> torch.Tensor:
        return self.state[k].to(device=self.device, dtype=self.dtype)

    def _f32(self, k: str) -> torch.Tensor:
        return self.state[k].to(device=self.device, dtype=torch.float32)

    def _vec(self, k: str, *shape: int) -> int:
        return self._hold(_pad_to(self._f32(k), *shape)).data_ptr()

    def _head_rows(self, k: str, heads: int, n: int, padded: int) -> torch.Tensor:
        """[heads * n, width] -> [heads * padded, width_p]"""
        return _pad_to(self._get(k).view(heads, n, self.cfg.width), heads, padded, self.width_p).view(heads * padded, self.width_p)

    def _latent(self, x, a: str, m: LatentAttention, i: int):
        if m.rot.dims != m.rot_dim:
            raise ValueError(f"layer {i}: rotation over {m.rot.dims} dimensions, rotated part of {m.rot_dim}")
        g, hold, Wp = self._get, self._hold, self.width_p
        qrp, kvp, rotc, hp = _up(m.q_rank, 64), _up(m.kv_rank, 64), _up(m.rot_dim, 32), _up(m.heads, 4)
        dn, dk, dv = _up(m.dim, 8), _up(m.dim, 32), _up(m.vdim, 16)
        dq = dk + rotc
        order = m.rot.pair_order().to(self.device)
        x.heads, x.dim, x.rot_dim, x.vdim, x.q_rank, x.kv_rank = m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank
        x.kv_from, x.gated = -1 if m.kv_from is None else m.kv_from, int(m.gate)
        x.scale, x.rot_mag = m.scale, m.rot.magnitude
        freq = (C.c_double * (m.rot_dim // 2))(*m.rot.frequencies())
        self.keep.append(freq)
        x.rot_freq = C.cast(freq, C.POINTER(C.c_double))
        rows = [_pad_to(g(a + "dq"), qrp, Wp)]
        x.q_norm = self._vec(a + "dq.norm", qrp)
        if m.kv_from is None:
            d = g(a + "dkv")
            rows += [_pad_to(d[:m.kv_rank], kvp, Wp), _pad_to(d[m.kv_rank:][order], rotc, Wp)]
            x.kv_norm = self._vec(a + "dkv.norm", kvp)
        if m.gate:
            rows.append(_pad_to(g(a + "g"), hp, Wp))
        x.in_w = hold(torch.cat(rows, 0)).data_ptr()
        uq = g(a + "uq").view(m.heads, m.dim + m.rot_dim, m.q_rank)
        q = uq.new_zeros(m.heads, dq, qrp)
        q[:, :m.dim, :m.q_rank] = uq[:, :m.dim]
        q[:, dk:dk + m.rot_dim, :m.q_rank] = uq[:, m.dim:][:, order]
        x.q_w = hold(q.view(m.heads * dq, qrp)).data_ptr()
        uk = g(a + "uk").view(m.heads, m.dim, m.kv_rank)
        uv = g(a + "uv").view(m.heads, m.vdim, m.kv_rank)
        x.kv_w = hold(torch.cat([_pad_to(uk, m.heads, dn, kvp).view(-1, kvp), _pad_to(uv, m.heads, dv, kvp).view(-1, kvp)], 0)).data_ptr()
        x.k_abs = hold(_pad_to(uk.transpose(1, 2), m.heads, kvp, dk)).data_ptr()
        if m.sink:
            x.sink = hold(self._f32(a + "sink") * math.log2(math.e)).data_ptr()
        return [kvp + rotc] if m.kv_from is None else [], 0

    def _heads(self, x, a: str, m: HeadAttention):
        dk, dv = _up(m.dim, 32), _up(m.vdim, 16)
        x.heads, x.kv_heads, x.dim, x.vdim, x.scale = m.heads, m.kv_heads, m.dim, m.vdim, m.scale
        x.qk_norm, x.temp_coef, x.temp_every = int(m.qk_norm), m.temp_coef, m.temp_every
        x.in_w = self._hold(torch.cat([self._head_rows(a + "q", m.heads, m.dim, dk), self._head_rows(a + "k", m.kv_heads, m.dim, dk),
                                       self._head_rows(a + "v", m.kv_heads, m.vdim, dv)], 0)).data_ptr()
        if m.bias is not None:
            rows = torch.tensor(m.bias.bucket_of(), device=self.device)
            x.dist_bias, x.dist_n = self._hold(self._f32(a + "rel")[rows].t() * math.log2(math.e)).data_ptr(), len(rows)
        return [_up(dk + dv, 32)] * m.kv_heads, 0

    def _delta(self, x, a: str, m: DeltaRule):
        dk, dv, hp = _up(m.dim, 16), _up(m.vdim, 16), _up(m.heads, 4)
        x.heads, x.kv_heads, x.dim, x.vdim, x.taps = m.heads, m.kv_heads, m.dim, m.vdim, m.taps
        parts = (("q", m.kv_heads, m.dim, dk), ("k", m.kv_heads, m.dim, dk), ("v", m.heads, m.vdim, dv))
        x.in_w = self._hold(torch.cat([self._head_rows(a + n, *s) for n, *s in parts + (("g", m.heads, m.vdim, dv),)] +
                                      [_pad_to(self._get(a + n), hp, self.width_p) for n in "ba"], 0)).data_ptr()
        conv = [_pad_to(self._f32(a + n + ".conv").view(h, d, m.taps), h, dp, m.taps).view(h * dp, m.taps) for n, h, d, dp in parts]
        x.conv = self._hold(torch.cat(conv, 0).t()).data_ptr()
        x.neg_a, x.dt_bias = self._hold(-torch.exp(self._f32(a + "A_log"))).data_ptr(), self._vec(a + "dt_bias", m.heads)
        x.norm = self._vec(a + "norm", dv)
        channels = 2 * m.kv_heads * dk + m.heads * dv
        return [], m.heads * dk * dv + m.taps * channels

    def _mlp(self, x, f: str, lc: DecoderLayerConfig):
        g, hold, Wp, ffp = self._get, self._hold, self.width_p, _up(lc.ff, 64)
        pad = lambda n: _pad_to(g(f + n), ffp, Wp)
        bias = lambda n: _pad_to(g(f + n + ".b"), ffp)
        x.ff = lc.ff
        if lc.mlp_act == "swiglu":
            x.act = L.ACT_SWIGLU
            x.up_w = hold(torch.stack([pad("gate"), pad("up")], dim=1).view(2 * ffp, Wp)).data_ptr()
            if lc.mlp_bias:
                x.up_b = hold(torch.stack([bias("gate"), bias("up")], dim=1).view(2 * ffp)).data_ptr()
        else:
            x.act = {"gelu": L.ACT_GELU_ERF}[lc.mlp_act]
            x.up_w = hold(pad("up")).data_ptr()
            if lc.mlp_bias:
                x.up_b = hold(bias("up")).data_ptr()
        x.down_w = hold(_pad_to(g(f + "down"), Wp, ffp)).data_ptr()
        if lc.mlp_bias:
            x.down_b = hold(_pad_to(g(f + "down.b"), Wp)).data_ptr()


# ---- random initialisation at arbitrary dimensions (no checkpoints are reachable: README.md:56-58) ----

def random_vit_state(cfg: VisionConfig, seed: int = 0, device="cpu", dtype=torch.float32, std: float = 0.02):
    g = torch.Generator(device=device).manual_seed(seed)
    r = lambda *s: (torch.randn(*s, generator=g, device=device, dtype=torch.float32) * std).to(dtype)
    H, I = cfg.hidden_size, cfg.intermediate_size
    st = {
        "embeddings.patch_embedding.weight": r(H, cfg.num_channels, cfg.patch_size, cfg.patch_size),
        "embeddings.patch_embedding.bias": r(H),
        "post_layernorm.weight": 1 + r(H), "post_layernorm.bias": r(H),
    }
    for i in range(cfg.num_hidden_layers):
        p = f"encoder.layers.{i}."
        for n in ("q_proj", "k_proj", "v_proj", "out_proj"):
            st[p + f"self_attn.{n}.weight"] = r(H, H)
            st[p + f"self_attn.{n}.bias"] = r(H)
        for n in ("layer_norm1", "layer_norm2"):
            st[p + n + ".weight"] = 1 + r(H)
            st[p + n + ".bias"] = r(H)
        st[p + "mlp.fc1.weight"], st[p + "mlp.fc1.bias"] = r(I, H), r(I)
        st[p + "mlp.fc2.weight"], st[p + "mlp.fc2.bias"] = r(H, I), r(H)
    return st


def random_proj_state(in_dim: int, out_dim: int, seed: int = 1, device="cpu", dtype=torch.float32, std: float = 0.02):
    g = torch.Generator(device=device).manual_seed(seed)
    r = lambda *s: (torch.randn(*s, generator=g, device=device, dtype=torch.float32) * std).to(dtype)
    return {"readout.0.weight": r(out_dim, in_dim), "readout.0.bias": r(out_dim),
            "readout.2.weight": r(out_dim, out_dim), "readout.2.bias": r(out_dim)}


def random_llm_state(cfg: LlmConfig, seed: int = 2, device="cpu", dtype=torch.float32, std: float = 0.02):
    g = torch.Generator(device=device).manual_seed(seed)
    r = lambda *s: (torch.randn(*s, generator=g, device=device, dtype=torch.float32) * std).to(dtype)
    H, I, hd = cfg.hidden_size, cfg.intermediate_size, cfg.head_dim
    kvd = cfg.num_key_value_heads * hd
    st = {"embed_tokens.weight": r(cfg.vocab_size, H), "norm.weight": 1 + r(H), "lm_head.weight": r(cfg.vocab_size, H)}
    for i in range(cfg.num_hidden_layers):
        p = f"layers.{i}."
        st[p + "input_layernorm.weight"] = 1 + r(H)
        st[p + "post_attention_layernorm.weight"] = 1 + r(H)
        st[p + "self_attn.q_proj.weight"], st[p + "self_attn.q_proj.bias"] = r(H, H), r(H)
        st[p + "self_attn.k_proj.weight"], st[p + "self_attn.k_proj.bias"] = r(kvd, H), r(kvd)
        st[p + "self_attn.v_proj.weight"], st[p + "self_attn.v_proj.bias"] = r(kvd, H), r(kvd)
        st[p + "self_attn.o_proj.weight"] = r(H, H)
        st[p + "mlp.gate_proj.weight"], st[p + "mlp.up_proj.weight"] = r(I, H), r(I, H)
        st[p + "mlp.down_proj.weight"] = r(H, I)
    return st


def random_decoder_state(cfg: DecoderConfig, seed: int = 3, device="cpu", dtype=torch.float32, std: Optional[float] = None):
    """decoder_tensors with norms near one and matrices of standard deviation `std` (default 1 / sqrt(inputs)); embeddings and bias
    tables of deviation one, hyper-connections that keep the streams' size, decays of a few to a few hundred tokens"""
    g = torch.Generator(device=device).manual_seed(seed)
    st = {}
    for name, shape in decoder_tensors(cfg).items():
        t = torch.randn(*shape, generator=g, device=device, dtype=torch.float32)
        last = name.rsplit(".", 1)[-1]
        if "norm" in last:
            t = 1 + 0.1 * t
        elif name.split(".")[1:2] in (["hc1"], ["hc2"]):
            t = 0.2 * t + {"in": shape[-1] ** -0.5, "out": 1.0, "mix": torch.eye(shape[-1], device=device)}[last]
        elif last == "A_log":
            t = t - 2
        elif len(shape) == 2 and last not in ("embed", "pos", "rel"):
            t = t * (shape[1] ** -0.5 if std is None else std)
        elif name.endswith(".b"):
            t = t * 0.1
        st[name] = t.to(dtype)
    return st


# ---------------------------------------------------------------------------------------------------------
# LoRA adapters. evaluate/answer_generate.py:181-182 loads two peft adapters
# ("full_module" for generate, "language_module" for qa_selection; r = 8, alpha = 16 on q,k,v,o,gate,up,down of
# the 28 decoder layers, the second-stage one also on both projector linears: train/second_stage_training.py:
# 241-264, first_stage_training.py:447-465) and switches them with set_adapter (:71-73). Here every adapter gets
# its own MERGED copy of the targeted matrices (W + alpha/r * B.A, summed in fp32, rounded once): 288 GB of HBM
# hold several 15 GB weight sets, the kernels stay untouched and switching is a pointer-table swap.

LORA_LLM_TARGETS = ("self_attn.q_proj", "self_attn.k_proj", "self_attn.v_proj", "self_attn.o_proj",
                    "mlp.gate_proj", "mlp.up_proj", "mlp.down_proj")


def _lora_lookup(lora_state: Dict[str, torch.Tensor], module: str):
    """(A [r,in], B [out,r]) of `module` under any of the key spellings peft writes / the tests use"""
    for prefix in ("", "base_model.model.model.", "base_model.model.", "model."):
        for mid in ("", ".default"):
            a = lora_state.get(f"{prefix}{module}.lora_A{mid}.weight")
            b = lora_state.get(f"{prefix}{module}.lora_B{mid}.weight")
            if a is not None and b is not None:
                return a, b
    return None


def merge_lora(llm_state: Dict[str, torch.Tensor], proj_state: Optional[Dict[str, torch.Tensor]],
               lora_state: Dict[str, torch.Tensor], cfg: LlmConfig, lora_alpha: float = 16.0):
    """-> (llm_state', proj_state') with W' = W + (alpha / r) * B @ A for every targeted module; untouched
    tensors are shared with the inputs (no copy)."""
    def merged(w, ab):
        a, b = ab
        r = a.shape[0]
        d = (b.to(w.device, torch.float32) @ a.to(w.device, torch.float32)) * (lora_alpha / r)
        return (w.float() + d).to(w.dtype)

    out = dict(llm_state)
    for i in range(cfg.num_hidden_layers):
        for t in LORA_LLM_TARGETS:
            ab = _lora_lookup(lora_state, f"layers.{i}.{t}")
            if ab is not None:
                out[f"layers.{i}.{t}.weight"] = merged(llm_state[f"layers.{i}.{t}.weight"], ab)
    pout = None
    if proj_state is not None:
        pout = dict(proj_state)
        for t in ("readout.0", "readout.2"):
            ab = _lora_lookup(lora_state, f"mm_projector.{t}")
            if ab is not None:
                pout[t + ".weight"] = merged(proj_state[t + ".weight"], ab)
    return out, pout


def random_lora_state(cfg: LlmConfig, seed: int = 7, r: int = 8, proj_dims=None, device="cpu", dtype=torch.float32,
                      std: float = 0.05):
    """test adapter in peft's key layout (both A and B random, so the branch is not a no-op)"""
    g = torch.Generator(device=device).manual_seed(seed)
    rnd = lambda *s: (torch.randn(*s, generator=g, device=device, dtype=torch.float32) * std).to(dtype)
    H, I, hd = cfg.hidden_size, cfg.intermediate_size, cfg.head_dim
    kvd = cfg.num_key_value_heads * hd
    dims = {"self_attn.q_proj": (H, H), "self_attn.k_proj": (kvd, H), "self_attn.v_proj": (kvd, H),
            "self_attn.o_proj": (H, H), "mlp.gate_proj": (I, H), "mlp.up_proj": (I, H), "mlp.down_proj": (H, I)}
    st = {}
    for i in range(cfg.num_hidden_layers):
        for t, (o, n) in dims.items():
            k = f"base_model.model.model.layers.{i}.{t}"
            st[k + ".lora_A.weight"], st[k + ".lora_B.weight"] = rnd(r, n), rnd(o, r)
    if proj_dims is not None:
        din, dout = proj_dims
        for t, (o, n) in (("readout.0", (dout, din)), ("readout.2", (dout, dout))):
            k = f"base_model.model.model.mm_projector.{t}"
            st[k + ".lora_A.weight"], st[k + ".lora_B.weight"] = rnd(r, n), rnd(o, r)
    return st
