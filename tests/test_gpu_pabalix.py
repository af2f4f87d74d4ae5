"""Pabalix on the GPU against its oracle (oracle/pabalix.py): every mechanism, prompts against token-by-token decoding, prompts
in portions, unequal batches, caches that grow, are freed and used again, keys at every place of interest, first tokens, long
decoding, other sizes, and generation through the framework's entry points. float32 pins the arithmetic, bfloat16 the kernels."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import pabalix as po
from pabalix_models import A, B, CONFIGS, G, YARN, config, double, mixer, rms_err, state, tokens

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# largest row error of the logits. bfloat16: about twice what rounding the operands of the matrix products does to these models
TOL = {torch.float32: 2e-5, torch.bfloat16: 3e-2}
TINY = 2.5        # the eight-wide model has nothing to average rounding errors over
DTYPES = [torch.float32, torch.bfloat16]
_cache = {}


def engine(cfg, st, dtype):
    from cogstream_amd.llm import DecoderEngine
    from cogstream_amd.pabalix import parse_config
    return DecoderEngine(st, parse_config(cfg), dtype=dtype, device="cuda:0")


def named(name, dtype, dev, n=0):
    """(config, weights, engine, tokens, oracle logits, oracle streams) of a shared model, made once"""
    key = (name, dtype)
    if key not in _cache:
        cfg = CONFIGS[name]
        st = state(cfg)
        _cache[key] = (cfg, st, engine(cfg, st, dtype))
    cfg, st, e = _cache[key]
    if (name, n) not in _cache:
        t = tokens(cfg, n)
        _cache[(name, n)] = (t,) + po.forward(cfg, double(st), t)
    return (cfg, st, e) + _cache[(name, n)]


def sequences(e, reserve=64):
    from cogstream_amd.llm import Sequences
    return Sequences(e, reserve)


def run(e, toks, cuts=(), reserve=64):
    """logits of every token, the prompt cut at `cuts`"""
    s = sequences(e, reserve)
    edges = [0, *cuts, len(toks)]
    return torch.cat([s.step([("r", toks[a:b], list(range(b - a)))]) for a, b in zip(edges, edges[1:])])


# ------------------------------------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_against_the_oracle_layer_by_layer(dev, name, dtype):
    """logits and the residual stream behind every layer, all sizes (also ranks and heads above the MFMA kernels' instances)"""
    n = 70 if name in ("wide", "large_rank") else 150
    cfg, st, e, toks, lg, streams = named(name, dtype, dev, n)
    W, tol = cfg["width"], TOL[dtype] * (TINY if name == "one" else 1)
    buf = torch.empty(len(cfg["layers"]), n, e.packed.width_p, device=dev)
    got = e.forward_batch(e.embed_tokens(torch.tensor(toks)), [n], [e.new_cache(n)], list(range(n)), streams=buf)
    assert got.shape == (n, cfg["vocab"])
    for i, want in enumerate(streams):
        assert rms_err(buf[i, :, :W], want) < tol, (name, i)
        assert not buf[i, :, W:].any()
    assert rms_err(got, lg) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_decoding_against_the_oracle(dev, name, dtype):
    """the absorbed form, from the first token on"""
    n = 70 if name in ("wide", "large_rank") else 150
    cfg, st, e, toks, lg, _ = named(name, dtype, dev, n)
    got = run(e, toks, range(1, n))
    assert rms_err(got, lg) < TOL[dtype] * (TINY if name == "one" else 1)


@pytest.mark.parametrize("kind", [A, B, G])
@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_far_from_the_start(dev, kind, dtype):
    """one layer, peaked scores, positions in the thousands: prompt and decoded"""
    n = 2100
    cfg = config([dict(mixer(kind, heads=2, dim=8, rot=32, vdim=16, gain=2.0, base=30.0, scaling=None if kind == B else YARN), ff=None)], width=64, vocab=64)
    st = state(cfg, seed=5)
    toks, w = tokens(cfg, n), double(state(cfg, seed=5))
    lg = po.forward(cfg, w, toks)[0]
    e = engine(cfg, st, dtype)
    assert rms_err(run(e, toks), lg) < TOL[dtype]
    assert rms_err(run(e, toks, range(n - 40, n))[-40:], lg[-40:]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_and_gate_at_their_extremes(dev, dtype):
    """a sink far above every score, one far below, and saturated gates, for prompts and decoding"""
    cfg = config([mixer(G, heads=4, scaling=YARN)])
    st = state(cfg, seed=2)
    st["l0.mix.sink"] = torch.tensor([40.0, -40.0, 3.0, 0.0])
    st["l0.mix.g"] = st["l0.mix.g"] * torch.tensor([8.0, -8.0, 0.0, 1.0])[:, None]
    toks = tokens(cfg, 60)
    lg = po.forward(cfg, double(st), toks)[0]
    e = engine(cfg, st, dtype)
    assert rms_err(run(e, toks), lg) < TOL[dtype] and rms_err(run(e, toks, range(1, 60)), lg) < TOL[dtype]


# ------------------------------------------------------------------------------------------------ one key among many
def needle_model(kind, dtype_seed=7):
    """token 1 asks for token 2: one score is far above all others, so whether exactly that key is seen shows in the logits"""
    cfg = config([dict(mixer(kind, heads=2, dim=16, rot=4, vdim=32, q_rank=64, kv_rank=64, scale=1.0, base=1e6, scaling=None if kind == B else (1.0, 64, 32.0, 1.0)), ff=None)],
                 width=64, vocab=64)
    st = state(cfg, seed=dtype_seed)
    if kind == G:
        st["l0.mix.sink"] = torch.tensor([0.5, 1.0])
    w, eps = double(st), cfg["norm"]["eps"]
    h = po.rms(w["embed"], w["l0.norm1"], eps)
    cq = po.rms(h @ w["l0.mix.dq"].T, w["l0.mix.dq.norm"], eps)[1]
    c = po.rms((h @ w["l0.mix.dkv"].T)[:, :64], w["l0.mix.dkv.norm"], eps)[2]
    for hd in range(2):
        st["l0.mix.uq"][hd * 20] = (5 * cq / (cq @ cq)).float()
        st["l0.mix.uk"][hd * 16] = (5 * c / (c @ c)).float()
    st = {k: v.to(torch.bfloat16).float() for k, v in st.items()}
    return cfg, st


@pytest.mark.parametrize("kind", [A, B, G])
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_single_key_at_every_place_of_interest(dev, kind, dtype):
    """the asked-for key first, last, at tile and split borders, itself, and one past the query (which must not be seen)"""
    cfg, st = needle_model(kind)
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
        lg = po.forward(cfg, w, toks)[0]
        if at is None:
            without = lg[ask]
        else:
            assert rms_err(lg[ask:], without[None]) > 0.3            # the oracle's answer depends on that key
        got = run(e, toks)
        assert rms_err(got[ask:], lg[ask:]) < TOL[dtype], ("prompt", at)
        assert rms_err(run(e, toks, [ask])[ask:], lg[ask:]) < TOL[dtype], ("decoded", at)
        assert rms_err(run(e, toks, [ask - 70])[ask:], lg[ask:]) < TOL[dtype], ("second portion", at)
    # the key right behind the query: invisible, also when it shares the query's tile
    for ask in (0, 15, 62, 63, 64, 126, 127, 128, 200):
        toks = list(base)
        toks[ask], toks[ask + 1] = 1, 2
        lg = po.forward(cfg, w, toks[:ask + 2])[0]
        assert rms_err(run(e, toks[:ask + 2]), lg) < TOL[dtype], ask


# ------------------------------------------------------------------------------------------------ schedules
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["peaked", "mixed"])
def test_portions_of_a_prompt(dev, name, dtype):
    cfg, st, e, toks, lg, _ = named(name, dtype, dev, 150)
    for cuts in ([2], [1, 3], [64], [63, 65], [128], [149], [148], [50, 52, 54, 118], list(range(2, 150, 2)), list(range(7, 150, 29))):
        assert rms_err(run(e, toks, cuts), lg) < TOL[dtype], cuts


@pytest.mark.parametrize("n", [1, 2, 3, 15, 16, 17, 63, 64, 65, 129])
@pytest.mark.parametrize("dtype", DTYPES)
def test_short_sequences_and_first_tokens(dev, n, dtype):
    cfg, st, e, toks, lg, _ = named("peaked", dtype, dev, 150)
    assert rms_err(run(e, toks[:n]), lg[:n]) < TOL[dtype]
    assert rms_err(run(e, toks[:n] + toks[n:n + 2], [n, n + 1]), lg[:n + 2]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["peaked", "mixed"])
def test_unequal_batch_against_each_alone(dev, name, dtype):
    """prompts of 1 .. 140 tokens in one step, then decoded together, shorter requests ending earlier; and steps that mix whole
    prompts with single tokens"""
    cfg, st, e, _, _, _ = named(name, dtype, dev, 150)
    w = double(st)
    lens = [1, 140, 2, 65, 64, 33, 17, 90]
    full = [tokens(cfg, n + 3 + i, seed=i) for i, n in enumerate(lens)]
    want = [po.forward(cfg, w, t)[0] for t in full]
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
    cfg, st, e, toks, lg, _ = named("peaked", dtype, dev, 150)
    for count in (2, 16, 17, 40, 70):
        s = sequences(e)
        s.step([(i, toks[:1 + i], []) for i in range(count)])
        out = s.step([(i, [toks[1 + i]], [0]) for i in range(count)])
        assert rms_err(out, lg[1:1 + count]) < TOL[dtype], count


@pytest.mark.parametrize("dtype", DTYPES)
def test_memory_that_is_freed_and_used_again(dev, dtype):
    """caches and workspaces that hold another request's rows, or NaN, change nothing"""
    cfg, st, e, toks, lg, _ = named("mixed", dtype, dev, 150)
    s = sequences(e, 16)
    for r in range(6):
        n = [90, 20, 130, 60, 7, 150][r]
        size = sum(e.packed.cache_widths) * (-(-n // 16) * 16)
        poison = torch.full((size,), float("nan"), device=dev, dtype=dtype)
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


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_through_a_growing_cache(dev, dtype):
    cfg, st, e, toks, lg, _ = named("peaked", dtype, dev, 400)
    got = run(e, toks, range(5, 400), reserve=8)
    assert rms_err(got, lg) < TOL[dtype]


def test_forms_and_kernels_agree(dev):
    """bfloat16: absorbed against expanded single tokens, MFMA against row-wise attention, few-row against general GEMM, and any
    number of key splits: all inside the tolerance of the oracle"""
    from cogstream_amd import _lib as L
    cfg, st, e, toks, lg, _ = named("peaked", torch.bfloat16, dev, 400)
    for name, value in (("mla_absorb", 0), ("mla_rowwise", 1), ("gemm_skinny", 0), ("mla_split_keys", 16), ("mla_split_keys", 100), ("mla_split_keys", 4096)):
        with L.debug_switch(name, value):
            assert rms_err(run(e, toks, [20, 380, *range(381, 400)]), lg) < TOL[torch.bfloat16], (name, value)


def test_unsupported_calls_are_refused(dev):
    from cogstream_amd import _lib as L
    cfg, st, e, toks, _, _ = named("peaked", torch.bfloat16, dev, 150)
    emb = e.embed_tokens(torch.tensor(toks[:4]))
    c = e.new_cache(8)
    for args in (([3], [e.new_cache(2)], []), ([1, 2], [c, c], []), ([3], [c], [3]), ([3], [c], [-1])):
        with pytest.raises(L.CogsError):
            e.forward_batch(emb[:3], *args)
    assert c.len == 0


# ------------------------------------------------------------------------------------------------ fused GEMM epilogues
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 5, 200, 700, 2048])
def test_gemm_swiglu_with_bias_and_rotation_without(dev, dtype, M):
    """biases inside the gated activation (rows and biases interleaved) and rotary columns without a bias, in every GEMM body"""
    from cogstream_amd import _lib as L
    from cogstream_amd import ops
    g = torch.Generator().manual_seed(M)
    K, N = 320, 768
    a = torch.randn(M, K, generator=g).to(dtype)
    w = (torch.randn(N, K, generator=g) * K ** -0.5).to(dtype)
    b = torch.randn(N, generator=g).to(dtype)
    lin = a.double() @ w.double().T
    v = lin + b.double()
    want = torch.nn.functional.silu(v[:, 0::2]) * v[:, 1::2]
    got = ops.gemm(a.to(dev), w.to(dev), b.to(dev), act=L.ACT_SWIGLU)
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    assert float((got.cpu().double() - want).abs().max() / want.abs().max()) < tol
    for hd in (96, 192):
        ang = torch.rand(M, hd // 2, generator=g) * 6
        c, s = ang.cos(), ang.sin()
        x = lin.view(M, N // hd, hd // 2, 2)
        want = torch.stack([x[..., 0] * c[:, None] - x[..., 1] * s[:, None], x[..., 1] * c[:, None] + x[..., 0] * s[:, None]], -1).view(M, N)
        got = ops.gemm(a.to(dev), w.to(dev), rope_cos=torch.stack([c, s], -1).to(dev).contiguous(), rope_cols=N, head_dim=hd)
        assert float((got.cpu().double() - want).abs().max() / want.abs().max()) < tol


# ------------------------------------------------------------------------------------------------ the framework's entry points
def _checkpoint(tmp_path, name):
    from cogstream_amd import checkpoint as ck
    cfg = CONFIGS[name]
    st = state(cfg)
    ck.save_decoder(str(tmp_path), cfg, st)
    return cfg, st


def test_greedy_generation_through_the_registry(dev, tmp_path):
    """AutoModelForCausalLM -> generate: one prompt, several unequal prompts in one batch, in groups, with an end token, and the
    single-sequence loop with its prefix cache, against the oracle's greedy continuation"""
    from cogstream_amd.auto import AutoModelForCausalLM
    from cogstream_amd.llm import PrefixKV
    cfg, st = _checkpoint(tmp_path, "peaked")
    m = AutoModelForCausalLM.from_pretrained(str(tmp_path), torch_dtype=torch.float32)
    prompts = [tokens(cfg, n, seed=n) for n in (9, 1, 30, 66)]
    want = [po.greedy(cfg, double(st), p, 8) for p in prompts]
    assert m.generate(prompts[0], max_new_tokens=8) == [want[0]]
    assert m.generate(torch.tensor(prompts[2]), max_new_tokens=8) == [want[2]]
    assert m.generate(prompts, max_new_tokens=8) == want
    assert m.generate(prompts, max_new_tokens=8, max_batch=3) == want
    stop = want[3][2]
    cut = [w[:w.index(stop) + 1] if stop in w else w for w in want]
    assert m.generate(prompts, max_new_tokens=8, eos_token_id=[stop]) == cut
    assert m.generate(prompts, max_new_tokens=8, eos_token_id=stop) == cut
    e = m.llm
    emb = e.embed_tokens(torch.tensor(prompts[3]))
    assert e.generate(emb, max_new_tokens=8) == want[3]
    pre = PrefixKV(e)
    assert e.generate(emb, max_new_tokens=8, prefix=pre) == want[3]
    longer = prompts[3] + tokens(cfg, 40, seed=5)
    assert e.generate(e.embed_tokens(torch.tensor(longer)), max_new_tokens=4, prefix=pre) == po.greedy(cfg, double(st), longer, 4)
    assert pre.reused == 66
    # sampling: a request's draws do not depend on its batch; top_k = 1 is greedy
    a = m.generate(prompts, max_new_tokens=6, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
    assert a == m.generate(prompts, max_new_tokens=6, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
    assert a[0] == m.generate(prompts[0], max_new_tokens=6, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)[0]
    assert m.generate(prompts, max_new_tokens=8, do_sample=True, top_k=1) == want


def test_two_models_share_a_handle(dev):
    """the handle keeps one decoder; engines re-activate themselves, also in turns and in either type"""
    a, b = named("peaked", torch.float32, dev, 150), named("mixed", torch.bfloat16, dev, 150)
    sa, sb = sequences(a[2]), sequences(b[2])
    for lo, hi in ((0, 60), (60, 61), (61, 90)):
        ra = sa.step([("r", a[3][lo:hi], list(range(hi - lo)))])
        rb = sb.step([("r", b[3][lo:hi], list(range(hi - lo)))])
        assert rms_err(ra, a[4][lo:hi]) < TOL[torch.float32] and rms_err(rb, b[4][lo:hi]) < TOL[torch.bfloat16]


def test_command_lines(dev, tmp_path):
    """python -m cogstream_amd.generate and bin/trace_run in processes of their own"""
    cfg, st = _checkpoint(tmp_path, "peaked")
    w = double(st)
    prompts = [tokens(cfg, n, seed=n) for n in (9, 30)]
    r = subprocess.run([sys.executable, "-m", "cogstream_amd.generate", "--model_path", str(tmp_path), "--dtype", "float32", "--max_new_tokens", "6",
                        "--greedy"] + [x for p in prompts for x in ("--prompt", ",".join(map(str, p)))], capture_output=True, text=True, cwd=ROOT, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [json.loads(x)["tokens"] for x in r.stdout.splitlines()] == [po.greedy(cfg, w, p, 6) for p in prompts]
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
    assert sorted(os.listdir(out)) == ["0.f32", "7.f32", "8.f32"]
    la, lb = po.forward(cfg, w, a)[0], po.forward(cfg, w, b)[0]
    load = lambda n: torch.frombuffer(bytearray((out / f"{n}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"])
    assert rms_err(load(0), torch.stack([la[0], la[36], lb[23]])) < TOL[torch.float32]
    assert rms_err(load(7), la[38:39]) < TOL[torch.float32] and rms_err(load(8), lb[24:25]) < TOL[torch.float32]


def test_qwen2_engine_takes_the_same_batches(dev):
    """Sequences and generate_batch over the Qwen2 engine: its logits are its own single-sequence ones"""
    from cogstream_amd.llm import Qwen2Engine
    from cogstream_amd.weights import LlmConfig, random_llm_state
    cfg = LlmConfig(hidden_size=256, intermediate_size=512, num_hidden_layers=2, num_attention_heads=2, num_key_value_heads=1,
                    vocab_size=512, image_token_index=500, eos_token_id=499)
    e = Qwen2Engine(random_llm_state(cfg, seed=7, std=0.05), cfg, dtype=torch.float32, device=dev)
    prompts = [list(range(3, 40)), [5, 6, 7], [9]]
    s = sequences(e, 8)
    out = s.step([(i, p, [len(p) - 1]) for i, p in enumerate(prompts)])
    for i, p in enumerate(prompts):
        want = e.forward(e.embed_tokens(torch.tensor(p)), e.new_cache(64))["logits"]
        assert torch.equal(out[i], want)
    got = e.generate_batch(prompts, max_new_tokens=5)
    assert got == [e.generate(e.embed_tokens(torch.tensor(p)), max_new_tokens=5) for p in prompts]
