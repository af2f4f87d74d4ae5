"""Lupanex on the GPU against its oracle (oracle/lupanex.py): every mechanism alone, prompts against token-by-token decoding, prompts
in portions, unequal batches, caches and states that grow, are freed and used again, keys at every place of interest, the edges of
the distance buckets, memories over hundreds of tokens, first tokens, long decoding, other sizes, and generation through the
framework's entry points. float32 pins the arithmetic, bfloat16 the kernels."""
import json
import os
import subprocess
import sys

import pytest
import torch

from lupanex_models import CONFIGS, attention, config, delta, double, parse, public, rms_err, state, tokens
from oracle import lupanex as lo

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# largest row error of the logits. bfloat16: about twice what rounding the operands of the matrix products does to these models
TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2}
TINY = 2.5        # the eight-wide models have nothing to average rounding errors over
DTYPES = [torch.float32, torch.bfloat16]
LONG = {"wide": 100, "large": 100}
_cache = {}


def tol(name, dtype):
    return TOL[dtype] * (TINY if name.startswith("one") else 1)


def engine(cfg, st, dtype):
    from cogstream_amd.llm import DecoderEngine
    return DecoderEngine(st, parse(cfg), dtype=dtype, device="cuda:0")


def named(name, dtype, n=150):
    """(config, weights, engine, tokens, oracle logits, oracle streams) of a shared model, made once"""
    if (name, dtype) not in _cache:
        cfg = CONFIGS[name]
        st = state(cfg)
        _cache[(name, dtype)] = (cfg, st, engine(cfg, st, dtype))
    cfg, st, e = _cache[(name, dtype)]
    if (name, n) not in _cache:
        t = tokens(cfg, n)
        _cache[(name, n)] = (t,) + lo.forward(cfg, double(st), t)
    return (cfg, st, e) + _cache[(name, n)]


def sequences(e, reserve=64):
    from cogstream_amd.llm import Sequences
    return Sequences(e, reserve)


def run(e, toks, cuts=(), reserve=64):
    """logits of every token, the prompt cut at `cuts`"""
    s = sequences(e, reserve)
    edges = [0, *cuts, len(toks)]
    return torch.cat([s.step([("r", toks[a:b], list(range(b - a)))]) for a, b in zip(edges, edges[1:])])


def both_ways(cfg, st, dtype, n, seed=0, cuts=(37, 90), limit=None):
    """a model whole, in portions and token by token against its oracle"""
    toks = tokens(cfg, n, seed=seed)
    lg = lo.forward(cfg, double(st), toks)[0]
    e = engine(cfg, st, dtype)
    for c in ((), [x for x in cuts if x < n], range(1, n)):
        assert rms_err(run(e, toks, c), lg) < (limit or TOL[dtype]), c
    return e, toks, lg


# ------------------------------------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_against_the_oracle_layer_by_layer(dev, name, dtype):
    """logits and the residual stream behind every layer run, all sizes (also those above the matrix kernels' instances)"""
    n = LONG.get(name, 150)
    cfg, st, e, toks, lg, streams = named(name, dtype, n)
    W = cfg["width"]
    buf = torch.empty(len(streams), n, e.packed.width_p, device=dev)
    got = e.forward_batch(e.embed_tokens(torch.tensor(toks)), [n], [e.new_cache(n)], list(range(n)), streams=buf)
    assert got.shape == (n, cfg["vocab"])
    for i, want in enumerate(streams):
        assert rms_err(buf[i, :, :W], want) < tol(name, dtype), (name, i)
        assert not buf[i, :, W:].any()
    assert rms_err(got, lg) < tol(name, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_decoding_against_the_oracle(dev, name, dtype):
    """from the first token on"""
    n = LONG.get(name, 150)
    cfg, st, e, toks, lg, _ = named(name, dtype, n)
    assert rms_err(run(e, toks, range(1, n)), lg) < tol(name, dtype)


def alone(mech):
    """one layer in which one mechanism decides"""
    st = None
    if mech == "bias":                     # no content scores at all: the weights are the bias table's
        cfg = config([attention(heads=4, kv_heads=2, rows=10, far=80, temp=None, ff=None)], width=128)
        st = state(cfg)
        st["l0.mix.q"] *= 0
    elif mech == "temperature":            # every position its own temperature, and a steep one
        cfg = config([attention(heads=3, dim=32, rows=4, far=9, temp=(1.5, 1), ff=None)], width=128)
    elif mech == "temperature_fraction":   # a period that is no whole number of tokens
        cfg = config([attention(heads=2, temp=(0.7, 6.5), ff=None)], width=64)
    elif mech == "qk_norm":                # queries and keys of very unlike sizes
        cfg = config([attention(heads=2, dim=40, ff=None)], width=64, eps=1e-2)
        st = state(cfg)
        st["l0.mix.q"] *= 0.05
        st["l0.mix.k"] *= torch.logspace(-2, 1, st["l0.mix.k"].shape[0])[:, None]
    elif mech == "groups":
        cfg = config([attention(heads=12, kv_heads=3, dim=16, vdim=16, ff=None)], width=128)
    elif mech == "delta":
        cfg = config([delta(ff=None)], width=128)
    elif mech == "delta_fast":             # decays from nearly nothing kept to everything kept, heads unlike
        cfg = config([delta(heads=4, kv_heads=1, dim=32, vdim=16, ff=None)], width=128)
        st = state(cfg)
        st["l0.mix.A_log"], st["l0.mix.dt_bias"] = torch.tensor([4.0, 1.0, -3.0, -9.0]), torch.tensor([6.0, 0.0, -1.0, -8.0])
    elif mech == "delta_hard":             # beta near 0 and near 1, keys often alike
        cfg = config([delta(heads=4, kv_heads=2, dim=8, vdim=16, ff=None)], width=128, vocab=6)
        st = state(cfg)
        st["l0.mix.b"] *= 8
    elif mech == "delta_zero":             # unit vectors of nothing: the first query and key channels see silu(0)
        cfg = config([delta(heads=2, kv_heads=2, conv=4, ff=None)], width=64)
        st = state(cfg)
        st["l0.mix.q"][:20] *= 0
        st["l0.mix.k"][:20] *= 1e-4
    elif mech in ("conv1", "conv2", "conv7", "conv12"):
        cfg = config([delta(heads=2, conv=int(mech[4:]), ff=None)], width=64)
    elif mech == "hyper":                  # the sublayers do nothing: the streams only mix
        cfg = config([delta(heads=2, kv_heads=1), attention(heads=2)], width=64, streams=6, loop=(0, 2, 2))
        st = state(cfg)
        for k in st:
            if k.endswith(("mix.o", "mlp.down")):
                st[k] = st[k] * 0
    elif mech == "hyper1":                 # a single stream with weights of its own
        cfg = config([attention(heads=2), delta(heads=2, kv_heads=1)], width=64, streams=1)
    elif mech == "loop":
        cfg = config([delta(heads=2, kv_heads=2), attention(heads=2)], width=64, loop=(0, 1, 4))
    elif mech == "feed_forward":
        cfg = config([delta(heads=1, kv_heads=1, dim=4, vdim=4, ff=200)], width=64)
        st = state(cfg)
        st["l0.mix.o"] *= 0
        st["l0.mlp.up"] *= 2
    elif mech == "positions":              # one word over and over
        cfg = config([attention(heads=2, ff=None)], width=64)
        st = state(cfg)
        st["embed"][:] = st["embed"][0]
    st = state(cfg) if st is None else st
    return cfg, {k: v.to(torch.bfloat16).float() for k, v in st.items()}


@pytest.mark.parametrize("mech", ["bias", "temperature", "temperature_fraction", "qk_norm", "groups", "delta", "delta_fast", "delta_hard", "delta_zero", "conv1", "conv2",
                                  "conv7", "conv12", "hyper", "hyper1", "loop", "feed_forward", "positions"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_mechanism_alone(dev, mech, dtype):
    cfg, st = alone(mech)
    both_ways(cfg, st, dtype, 110)


@pytest.mark.parametrize("rows,far", [(2, 3), (6, 40), (16, 128), (32, 64), (8, 2000)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_edges_of_the_distance_buckets(dev, rows, far, dtype):
    """each head's table has one bucket far above the others, so the output is the mean of exactly that bucket's values: every
    first and last distance of every bucket, in prompts, portions and decoding"""
    n = 330
    cfg = config([attention(heads=rows, kv_heads=1, dim=8, vdim=32, rows=rows, far=far, temp=None, ff=None)], width=64, vocab=128)
    st = state(cfg, seed=rows)
    st["l0.mix.q"] *= 0
    st["l0.mix.rel"] = 16 * torch.eye(rows) - 3
    toks = tokens(cfg, n)
    lg = lo.forward(cfg, double(st), toks)[0]
    e = engine(cfg, st, dtype)
    assert rms_err(run(e, toks), lg) < TOL[dtype]
    assert rms_err(run(e, toks, [200, 203, *range(230, n)]), lg) < TOL[dtype]


# ------------------------------------------------------------------------------------------------ one key among many
def needle_model(heads=2, kv_heads=2, dim=32, scale=0.7, seed=7):
    """token 1 asks for token 2: one score is far above all others, so whether exactly that key is seen shows in the logits"""
    cfg = config([attention(heads=heads, kv_heads=kv_heads, dim=dim, vdim=32, rows=12, far=100, scale=scale, temp=(0.1, 50), ff=None)], width=64, vocab=64, streams=2)
    st = state(cfg, seed=seed)
    st["pos"] *= 0.02
    st["l0.mix.rel"] *= 0.3
    w = double(st)
    x = w["embed"] * cfg["embedding"]["scale"]
    h = lo.rms(sum(w["l0.hc1.in"][s] * x for s in range(2)), cfg["norm"]["eps"]) * w["l0.norm1"]
    for i in range(heads):
        g = i // (heads // kv_heads)
        q, k = w["l0.mix.q"][i * dim:(i + 1) * dim], w["l0.mix.k"][g * dim:(g + 1) * dim]
        st["l0.mix.q"][i * dim:(i + 1) * dim] = (q + torch.outer(k @ h[2] - q @ h[1], h[1]) / (h[1] @ h[1])).float()
    return cfg, {k: v.to(torch.bfloat16).float() for k, v in st.items()}


@pytest.mark.parametrize("heads,kv_heads", [(2, 2), (6, 2)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_single_key_at_every_place_of_interest(dev, heads, kv_heads, dtype):
    """the asked-for key first, last, at tile and split borders, itself, and one past the query (which must not be seen)"""
    cfg, st = needle_model(heads, kv_heads)
    e, w = engine(cfg, st, dtype), double(st)
    n = 330
    base = [t if t > 2 else 3 + t for t in tokens(cfg, n)]
    ask = n - 1
    without = None
    for at in (None, 0, 1, 15, 16, 31, 32, 63, 64, 65, 127, 128, 255, 256, 319, 320, n - 2):
        toks = list(base)
        toks[ask] = 1
        if at is not None:
            toks[at] = 2
        lg = lo.forward(cfg, w, toks)[0]
        if at is None:
            without = lg[ask]
        else:
            assert rms_err(lg[ask:], without[None]) > 0.3            # the oracle's answer depends on that key
        assert rms_err(run(e, toks)[ask:], lg[ask:]) < TOL[dtype], ("prompt", at)
        assert rms_err(run(e, toks, [ask])[ask:], lg[ask:]) < TOL[dtype], ("decoded", at)
        assert rms_err(run(e, toks, [ask - 70])[ask:], lg[ask:]) < TOL[dtype], ("second portion", at)
    # the key right behind the query: invisible, also when it shares the query's tile
    for ask in (0, 15, 62, 63, 64, 126, 127, 128, 200):
        toks = list(base)
        toks[ask], toks[ask + 1] = 1, 2
        lg = lo.forward(cfg, w, toks[:ask + 2])[0]
        assert rms_err(run(e, toks[:ask + 2]), lg) < TOL[dtype], ask


def memory_model(dim=48):
    """a delta layer that keeps everything and writes only on token 2, whose key token 1 reads back"""
    cfg = config([delta(heads=2, kv_heads=1, dim=dim, vdim=32, conv=2, ff=None)], width=64, vocab=40, streams=1)
    st = state(cfg, seed=4)
    st["pos"] *= 0
    w = double(st)
    h = lo.rms(w["l0.hc1.in"][0] * w["embed"] * cfg["embedding"]["scale"], cfg["norm"]["eps"]) * w["l0.norm1"]
    for n in "qkv":
        st[f"l0.mix.{n}.conv"] = torch.tensor([0.0, 1.0]).repeat(len(st[f"l0.mix.{n}.conv"]), 1)
    want = torch.full((40, 2), -12.0, dtype=torch.float64)
    want[2] = 6
    st["l0.mix.b"] = (torch.linalg.pinv(h) @ want).T.float()
    st["l0.mix.dt_bias"] = torch.full((2,), -20.0)
    q, k = w["l0.mix.q"], w["l0.mix.k"]
    st["l0.mix.q"] = (q + torch.outer(k @ h[2] - q @ h[1], h[1]) / (h[1] @ h[1])).float()
    return cfg, {k: v.to(torch.bfloat16).float() for k, v in st.items()}


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_write_is_read_back_from_any_distance(dev, dtype):
    """a single write at chunk borders, the first token, the query's neighbour, read hundreds of tokens later: in one prompt, decoded, and
    with portions of every kind between write and read"""
    cfg, st = memory_model()
    e, w = engine(cfg, st, dtype), double(st)
    n = 330
    base = [t if t > 2 else 3 + t for t in tokens(cfg, n)]
    ask, without = n - 1, None
    for at in (None, 0, 1, 15, 16, 30, 31, 32, 33, 63, 64, 160, 319, 320, n - 2):
        toks = list(base)
        toks[ask] = 1
        if at is not None:
            toks[at] = 2
        lg = lo.forward(cfg, w, toks)[0]
        if at is None:
            without = lg[ask]
        else:
            assert rms_err(lg[ask:], without[None]) > 0.2
        for cuts in ((), [ask], [32, 64, 97], [2, 3, ask - 2], [max(at or 1, 1), (at or 1) + 1] if (at or 1) + 1 < n else [at]):
            assert rms_err(run(e, toks, cuts)[ask:], lg[ask:]) < TOL[dtype], (at, cuts)


# ------------------------------------------------------------------------------------------------ schedules
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["peaked", "mixed"])
def test_portions_of_a_prompt(dev, name, dtype):
    cfg, st, e, toks, lg, _ = named(name, dtype)
    for cuts in ([2], [1, 3], [31], [32], [33], [64], [63, 65], [128], [149], [148], [50, 52, 54, 118], list(range(2, 150, 2)), list(range(3, 150, 3)), list(range(7, 150, 29))):
        assert rms_err(run(e, toks, cuts), lg) < TOL[dtype], cuts


@pytest.mark.parametrize("n", [1, 2, 3, 4, 5, 15, 16, 17, 31, 32, 33, 63, 64, 65, 129])
@pytest.mark.parametrize("dtype", DTYPES)
def test_short_sequences_and_first_tokens(dev, n, dtype):
    cfg, st, e, toks, lg, _ = named("peaked", dtype)
    assert rms_err(run(e, toks[:n]), lg[:n]) < TOL[dtype]
    assert rms_err(run(e, toks[:n] + toks[n:n + 2], [n, n + 1]), lg[:n + 2]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["peaked", "mixed"])
def test_unequal_batch_against_each_alone(dev, name, dtype):
    """prompts of 1 .. 140 tokens in one step, then decoded together, shorter requests ending earlier; and steps that mix whole
    prompts with single tokens"""
    cfg, st, e, _, _, _ = named(name, dtype)
    w = double(st)
    lens = [1, 140, 2, 65, 64, 33, 17, 90]
    full = [tokens(cfg, n + 3 + i, seed=i) for i, n in enumerate(lens)]
    want = [lo.forward(cfg, w, t)[0] for t in full]
    s = sequences(e, 16)
    out = s.step([(i, full[i][:n], list(range(n))) for i, n in enumerate(lens)])
    at = 0
    for i, n in enumerate(lens):
        assert rms_err(out[at:at + n], want[i][:n]) < TOL[dtype], i
        at += n
    pos = list(lens)
    while True:
        live = [i for i in range(len(lens)) if pos[i] < len(full[i])]
        if not live:
            break
        order = live[::-1] if len(live) % 2 else live          # the order in a batch is nothing a request sees
        out = s.step([(i, [full[i][pos[i]]], [0]) for i in order])
        for r, i in enumerate(order):
            assert rms_err(out[r:r + 1], want[i][pos[i]:pos[i] + 1]) < TOL[dtype], (i, pos[i])
            pos[i] += 1
        for i in live:
            if pos[i] == len(full[i]):
                s.release(i)
    assert not s.caches
    s = sequences(e)
    s.step([("a", full[1][:100], []), ("b", full[3][:1], [])])
    out = s.step([("b", full[3][1:2], [0]), ("c", full[7], [len(full[7]) - 1]), ("a", full[1][100:], [0, 40])])
    assert rms_err(out, torch.stack([want[3][1], want[7][-1], want[1][100], want[1][140]])) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_batch_decoding(dev, dtype):
    """more sequences than one MFMA column tile, and more rows than the few-row GEMM takes"""
    cfg, st, e, toks, lg, _ = named("peaked", dtype)
    for count in (2, 16, 17, 40, 70):
        s = sequences(e)
        s.step([(i, toks[:1 + i], []) for i in range(count)])
        out = s.step([(i, [toks[1 + i]], [0]) for i in range(count)])
        assert rms_err(out, lg[1:1 + count]) < TOL[dtype], count


@pytest.mark.parametrize("dtype", DTYPES)
def test_memory_that_is_freed_and_used_again(dev, dtype):
    """caches, states and workspaces that hold another request's rows, or NaN, change nothing"""
    cfg, st, e, toks, lg, _ = named("mixed", dtype)
    s = sequences(e, 16)
    for r in range(6):
        n = [90, 20, 130, 60, 7, 150][r]
        poison = [torch.full((sum(e.packed.cache_widths) * (-(-n // 16) * 16),), float("nan"), device=dev, dtype=dtype),
                  torch.full((e.packed.state_floats,), float("nan"), device=dev)]
        del poison
        e.handle._ws["decoder"].view(torch.int16).fill_(0x7fc0)          # NaN in either type
        other = [t ^ 1 if (t ^ 1) < cfg["vocab"] else t for t in toks]
        s.step([("junk", other[:n], [])])
        s.release("junk")
        out = s.step([("x", toks[:n - 2], list(range(n - 2)))])
        assert rms_err(out, lg[:n - 2]) < TOL[dtype], r
        for k in (n - 2, n - 1):
            assert rms_err(s.step([("x", [toks[k]], [0])]), lg[k:k + 1]) < TOL[dtype], r
        s.release("x")
    # a cache with everything NaN, from the first token on, by either kernel of the delta rule
    for cuts in ((), range(1, 12)):
        c = e.new_cache(64)
        c.k.fill_(float("nan"))
        c.state.fill_(float("nan"))
        edges = [0, *cuts, 12]
        for a, b in zip(edges, edges[1:]):
            out = e.forward_batch(e.embed_tokens(torch.tensor(toks[a:b])), [b - a], [c], [b - a - 1])
            assert rms_err(out, lg[b - 1:b]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_through_a_growing_cache(dev, dtype):
    cfg, st, e, toks, lg, _ = named("peaked", dtype, 400)
    assert rms_err(run(e, toks, range(5, 400), reserve=8), lg) < TOL[dtype]


def test_forms_and_kernels_agree(dev):
    """bfloat16: chunked against token-by-token delta rule, MFMA against row-wise attention, few-row against general GEMM, and any
    number of key splits: all inside the tolerance of the oracle"""
    from cogstream_amd import _lib as L
    cfg, st, e, toks, lg, _ = named("peaked", torch.bfloat16, 400)
    for name, value in (("delta_chunk", 0), ("mla_rowwise", 1), ("gemm_skinny", 0), ("mla_split_keys", 16), ("mla_split_keys", 100), ("mla_split_keys", 4096)):
        with L.debug_switch(name, value):
            assert rms_err(run(e, toks, [20, 380, *range(381, 400)]), lg) < TOL[torch.bfloat16], (name, value)


def test_unsupported_calls_are_refused(dev):
    from cogstream_amd import _lib as L
    cfg, st, e, toks, _, _ = named("peaked", torch.bfloat16)
    emb = e.embed_tokens(torch.tensor(toks[:4]))
    c = e.new_cache(8)
    for args in (([3], [e.new_cache(2)], []), ([1, 2], [c, c], []), ([3], [c], [3]), ([3], [c], [-1])):
        with pytest.raises(L.CogsError):
            e.forward_batch(emb[:3], *args)
    assert c.len == 0
    e.forward_batch(emb, [4], [c], [])
    c.reset(2)                                           # the state is that of four tokens
    with pytest.raises(L.CogsError):
        e.forward_batch(emb[:1], [1], [c], [])
    short = config([attention(heads=2), delta(heads=2)], width=64, positions=20)
    s = sequences(engine(short, state(short), torch.bfloat16))
    s.step([("r", tokens(short, 20), [])])
    with pytest.raises(L.CogsError):
        s.step([("r", [1], [0])])


# ------------------------------------------------------------------------------------------------ the framework's entry points
def _checkpoint(tmp_path, name):
    from cogstream_amd import checkpoint as ck
    cfg = CONFIGS[name]
    st = state(cfg)
    ck.save_decoder(str(tmp_path), public(cfg), st)
    return cfg, st


def test_greedy_generation_through_the_registry(dev, tmp_path):
    """AutoModelForCausalLM -> generate: one prompt, several unequal prompts in one batch, in groups, with an end token, and the
    single-sequence loop with its prefix cache, against the oracle's greedy continuation"""
    from cogstream_amd.auto import AutoModelForCausalLM
    from cogstream_amd.llm import PrefixKV
    cfg, st = _checkpoint(tmp_path, "peaked")
    m = AutoModelForCausalLM.from_pretrained(str(tmp_path), torch_dtype=torch.float32)
    assert type(m).__name__ == "LupanexForCausalLM"
    w = double(st)
    prompts = [tokens(cfg, n, seed=n) for n in (9, 1, 30, 66)]
    want = [lo.greedy(cfg, w, p, 8) for p in prompts]
    assert m.generate(prompts[0], max_new_tokens=8) == [want[0]]
    assert m.generate(torch.tensor(prompts[2]), max_new_tokens=8) == [want[2]]
    assert m.generate(prompts, max_new_tokens=8) == want
    assert m.generate(prompts, max_new_tokens=8, max_batch=3) == want
    stop = want[3][2]
    cut = [w[:w.index(stop) + 1] if stop in w else w for w in want]
    assert m.generate(prompts, max_new_tokens=8, eos_token_id=[stop]) == cut
    e = m.llm
    emb = e.embed_tokens(torch.tensor(prompts[3]))
    assert e.generate(emb, max_new_tokens=8) == want[3]
    # a state can stand behind the whole previous prompt, or start again
    pre = PrefixKV(e)
    assert e.generate(emb, max_new_tokens=8, prefix=pre) == want[3]
    longer = prompts[3] + tokens(cfg, 40, seed=5)
    assert e.generate(e.embed_tokens(torch.tensor(longer)), max_new_tokens=4, prefix=pre) == lo.greedy(cfg, w, longer, 4)
    assert pre.reused == 66
    other = longer[:80] + prompts[2]
    assert e.generate(e.embed_tokens(torch.tensor(other)), max_new_tokens=4, prefix=pre) == lo.greedy(cfg, w, other, 4)
    assert pre.reused == 66
    a = m.generate(prompts, max_new_tokens=6, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
    assert a == m.generate(prompts, max_new_tokens=6, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
    assert m.generate(prompts, max_new_tokens=8, do_sample=True, top_k=1) == want


def test_two_designs_share_a_handle(dev):
    """the handle keeps one decoder; engines of either design re-activate themselves, in turns and in either type"""
    import pabalix_models as pm
    from cogstream_amd.llm import DecoderEngine
    from cogstream_amd.pabalix import parse_config
    from oracle import pabalix as po
    a = named("peaked", torch.bfloat16)
    pc = pm.CONFIGS["plain"]
    pst = pm.state(pc)
    ptoks = pm.tokens(pc, 90)
    plg = po.forward(pc, double(pst), ptoks)[0]
    sa, sb = sequences(a[2]), sequences(DecoderEngine(pst, parse_config(pc), dtype=torch.float32, device="cuda:0"))
    for x, y in ((0, 60), (60, 61), (61, 90)):
        ra = sa.step([("r", a[3][x:y], list(range(y - x)))])
        rb = sb.step([("r", ptoks[x:y], list(range(y - x)))])
        assert rms_err(ra, a[4][x:y]) < TOL[torch.bfloat16] and rms_err(rb, plg[x:y]) < TOL[torch.float32]


def test_command_lines(dev, tmp_path):
    """python -m cogstream_amd.generate and bin/trace_run in processes of their own"""
    cfg, st = _checkpoint(tmp_path, "mixed")
    w = double(st)
    prompts = [tokens(cfg, n, seed=n) for n in (9, 30)]
    r = subprocess.run([sys.executable, "-m", "cogstream_amd.generate", "--model_path", str(tmp_path), "--dtype", "float32", "--max_new_tokens", "6",
                        "--greedy"] + [x for p in prompts for x in ("--prompt", ",".join(map(str, p)))], capture_output=True, text=True, cwd=ROOT, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [json.loads(x)["tokens"] for x in r.stdout.splitlines()] == [lo.greedy(cfg, w, p, 6) for p in prompts]
    out = tmp_path / "out"
    out.mkdir()
    a, b = tokens(cfg, 40, seed=1), tokens(cfg, 25, seed=2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:37], "want": [0, 36]}, {"id": "b", "tokens": b[:24], "want": [23]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[37:38], "want": []}, {"id": "b", "tokens": b[24:], "want": []}], "end": ["b"]},
             {"step": 7, "entries": [{"id": "a", "tokens": a[38:39], "want": [0]}], "end": ["a"]},
             {"step": 8, "entries": [{"id": "a", "tokens": b, "want": [24]}], "end": []}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, cwd=str(tmp_path), timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 7", "done 8"]
    la, lb = lo.forward(cfg, w, a)[0], lo.forward(cfg, w, b)[0]
    load = lambda n: torch.frombuffer(bytearray((out / f"{n}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"])
    assert rms_err(load(0), torch.stack([la[0], la[36], lb[23]])) < TOL[torch.float32]
    assert rms_err(load(7), la[38:39]) < TOL[torch.float32] and rms_err(load(8), lb[24:25]) < TOL[torch.float32]
