"""Lupanex without a GPU: the configuration and its tensor names, distance buckets, the packed layouts (recomputed from the packed
tensors with plain torch), the chunked form of the delta rule, caches with a state, the model registry, and that the oracle notices
what the GPU tests are meant to notice."""
import json
import math

import pytest
import torch

from lupanex_models import CONFIGS, attention, config, delta, double, parse, public, rms_err, shapes, state, tokens
from oracle import lupanex as lo


def _view(ptr, shape, packed):
    return next(t for t in packed.keep if isinstance(t, torch.Tensor) and t.data_ptr() == ptr).view(*shape)


def exact_bucket(n, rows, far):
    """in whole numbers: k logarithmic steps fit below n if (far / half)^k <= (n / half)^steps"""
    half, steps = rows // 2, rows - rows // 2
    if n < half:
        return n
    k = 0
    while k < steps and far ** (k + 1) * half ** steps <= n ** steps * half ** (k + 1):
        k += 1
    return min(rows - 1, half + k)


@pytest.mark.parametrize("rows,far", [(2, 3), (2, 64), (4, 9), (6, 90), (8, 1000), (12, 50), (16, 128), (32, 64), (32, 256), (32, 4096), (64, 33)])
def test_distance_buckets(rows, far):
    from cogstream_amd.weights import DistanceBias
    mine = DistanceBias(rows, float(far)).bucket_of()
    want = [exact_bucket(n, rows, far) for n in range(len(mine) + 50)]
    assert mine == want[:len(mine)] and mine[-1] == rows - 1 and (len(mine) == 1 or mine[-2] < rows - 1)
    assert set(want[len(mine):]) == {rows - 1} and [lo.bucket(n, rows, far) for n in range(len(want))] == want


def test_a_distance_bias_without_logarithmic_buckets_is_refused():
    from cogstream_amd.weights import DistanceBias
    for rows, far in ((1, 8.0), (8, 4.0), (8, 2.0)):
        with pytest.raises(ValueError):
            DistanceBias(rows, far).bucket_of()


def test_configuration():
    for name, cfg in CONFIGS.items():
        dc = parse(public(cfg) | {"layers": cfg["layers"]})
        assert dc.runs() == lo.order(cfg) and dc.streams == cfg.get("streams", 0) and dc.max_positions == cfg["max_positions"], name
        for lay, mine in zip(cfg["layers"], dc.layers):
            m = lay["mixer"]
            assert (mine.mixer.heads, mine.mixer.kv_heads, mine.mixer.dim, mine.mixer.vdim) == (m["heads"], m["kv_heads"], m["dim"], m["vdim"])
            assert mine.ff == (lay["mlp"] or {"ff": 0})["ff"] and not mine.post_norm and not mine.mlp_bias and mine.mlp_act == "gelu"
            if lay["type"] == "attention":
                t = m.get("q_temp") or dict(coef=0, every=0)
                assert (mine.mixer.bias.buckets, mine.mixer.bias.far, mine.mixer.scale) == (lay["rows"], m["bias_max"], m["scale"])
                assert (mine.mixer.temp_coef, mine.mixer.temp_every) == (t["coef"], t["every"]) and mine.mixer.qk_norm
            else:
                assert mine.mixer.taps == m["conv"]
    for lay in (dict(attention(), type="other"), attention(heads=4, kv_heads=3), delta(heads=5, kv_heads=2)):
        with pytest.raises(ValueError):
            parse(config([lay]))
    for loop in ((1, 1, 2), (0, 3, 2), (-1, 1, 2), (0, 1, 0)):
        with pytest.raises(ValueError):
            parse(config([delta(), delta()], loop=loop))
    bad = config([delta()])
    bad["layers"][0]["mlp"]["kind"] = "sparse"
    with pytest.raises(ValueError):
        parse(bad)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_packed_layouts_give_the_same_projections(name):
    from cogstream_amd.weights import PackedDecoder
    cfg = CONFIGS[name]
    st = state(cfg)
    pk = PackedDecoder(st, parse(cfg), torch.float32, "cpu")
    up = lambda v, m: -(-v // m) * m
    gen = torch.Generator().manual_seed(3)
    W, Wp = cfg["width"], up(cfg["width"], 64)
    hp = torch.zeros(5, Wp)
    hp[:, :W] = h = torch.randn(5, W, generator=gen)
    assert torch.equal(_view(pk.struct.pos, (cfg["max_positions"], Wp), pk)[:, :W], st["pos"])
    widths, floats = [], []
    for i, lay in enumerate(cfg["layers"]):
        m, pre, x = lay["mixer"], f"l{i}.mix.", pk.layers[i]
        H, G, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        dv = up(v, 16)
        if lay["type"] == "attention":
            x, dk = x.attn, up(d, 32)
            parts = (("q", H, d, dk), ("k", G, d, dk), ("v", G, v, dv))
            widths.append([up(dk + dv, 32)] * G)
            floats.append(0)
            rel = st[pre + "rel"]
            want = torch.stack([rel[lo.bucket(n, rel.shape[0], m["bias_max"])] for n in range(x.dist_n + 40)]) / math.log(2)
            table = _view(x.dist_bias, (H, x.dist_n), pk)
            assert torch.allclose(table.T, want[:x.dist_n], rtol=1e-6) and torch.allclose(table[:, -1].expand(40, H), want[x.dist_n:], rtol=1e-6)
        else:
            x, dk, hp4 = x.delta, up(d, 16), up(H, 4)
            parts = (("q", G, d, dk), ("k", G, d, dk), ("v", H, v, dv), ("g", H, v, dv), ("b", 1, H, hp4), ("a", 1, H, hp4))
            channels = 2 * G * dk + H * dv
            widths.append([])
            floats.append(H * dk * dv + m["conv"] * channels)
            conv, at = _view(x.conv, (m["conv"], channels), pk), 0
            for n, heads, size, padded in parts[:3]:
                c = conv[:, at:at + heads * padded].view(m["conv"], heads, padded)
                assert torch.equal(c[..., :size].reshape(m["conv"], -1).T, st[pre + n + ".conv"]) and not c[..., size:].any()
                at += heads * padded
            assert torch.allclose(_view(x.neg_a, (H,), pk), -st[pre + "A_log"].exp()) and torch.equal(_view(x.dt_bias, (H,), pk), st[pre + "dt_bias"])
            assert torch.equal(_view(x.norm, (dv,), pk)[:v], st[pre + "norm"])
        total = sum(heads * padded for _, heads, _, padded in parts)
        t, at = hp @ _view(x.in_w, (total, Wp), pk).T, 0
        for n, heads, size, padded in parts:
            p = t[:, at:at + heads * padded].view(5, heads, padded)
            assert torch.allclose(p[..., :size].reshape(5, -1), h @ st[pre + n].T, atol=1e-5) and not p[..., size:].any(), n
            at += heads * padded
        o, val = torch.zeros(5, up(H * dv, 64)), torch.randn(5, H, v, generator=gen)
        o[:, :H * dv].view(5, H, dv)[..., :v] = val
        y = o @ _view(x.o_w, (Wp, o.shape[1]), pk).T
        assert torch.allclose(y[:, :W], val.reshape(5, -1) @ st[pre + "o"].T, atol=1e-4) and not y[:, W:].any()
        s = cfg.get("streams", 0)
        for q, hc in (("1", pk.layers[i].hyper1), ("2", pk.layers[i].hyper2)):
            if not s or q == "2" and lay["mlp"] is None:
                continue
            assert torch.equal(_view(hc.in_, (s,), pk), st[f"l{i}.hc{q}.in"]) and torch.equal(_view(hc.out, (s,), pk), st[f"l{i}.hc{q}.out"])
            assert torch.equal(_view(hc.mix, (s, s), pk), st[f"l{i}.hc{q}.mix"])
        if lay["mlp"] is not None:
            ml, ffp = pk.layers[i].mlp, up(lay["mlp"]["ff"], 64)
            a = torch.nn.functional.gelu(hp @ _view(ml.up_w, (ffp, Wp), pk).T) @ _view(ml.down_w, (Wp, ffp), pk).T
            assert torch.allclose(a[:, :W], lo.feed_forward(h, st, f"l{i}.mlp."), atol=1e-4) and not a[:, W:].any()
            assert not ml.up_b and not ml.down_b
    assert pk.cache_widths == [w for i in lo.order(cfg) for w in widths[i]] and pk.state_floats == sum(floats[i] for i in lo.order(cfg))


def test_chunked_delta_rule_is_the_recurrence():
    """the algebra of the prompt kernels (csrc/delta.hip, head comment) in float64, with decays down to nothing"""
    g = torch.Generator().manual_seed(1)
    T, d, dv, CH = 75, 6, 5, 32
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    q, k, v = lo.unit(rnd(T, d)), lo.unit(rnd(T, d)), rnd(T, dv)
    beta, ln_g = torch.sigmoid(rnd(T)), -torch.exp(3 * rnd(T))
    want = lo.delta_recurrence(q, k, v, beta, ln_g.exp())
    S, out = torch.zeros(d, dv, dtype=torch.float64), []
    for a in range(0, T, CH):
        K, Q, V, b, G = k[a:a + CH], q[a:a + CH], v[a:a + CH], beta[a:a + CH], ln_g[a:a + CH].cumsum(0)
        e = torch.tril(torch.exp(torch.tril(G[:, None] - G[None])))
        inv = torch.linalg.inv(torch.eye(len(b), dtype=torch.float64) + torch.tril(b[:, None] * e * (K @ K.T), -1))
        U = inv @ (b[:, None] * (V - G.exp()[:, None] * (K @ S)))
        out.append(G.exp()[:, None] * (Q @ S) + (e * (Q @ K.T)) @ U)
        S = G[-1].exp() * S + K.T @ ((G[-1] - G).exp()[:, None] * U)
    assert torch.allclose(torch.cat(out), want, atol=1e-12)


def test_a_cache_whose_state_does_not_belong_to_its_length_is_marked():
    from cogstream_amd.llm import DecoderCache
    c = DecoderCache([4, 6], 10, 8, torch.float32, "cpu")
    c.reset(0)
    assert not c.stale and [b.shape for b in c._blocks()] == [(8, 4), (8, 6)]
    c.struct.len = 5
    c.reset(5)
    assert not c.stale
    c.reset(3)
    assert c.stale
    c.restore(3, torch.arange(10.0))
    assert not c.stale and c.len == 3 and c.state.tolist() == list(range(10))
    c.reset(2)
    c.reset(0)
    assert not c.stale
    plain = DecoderCache([4], 0, 8, torch.float32, "cpu")
    plain.struct.len = 5
    plain.reset(2)                                        # rows alone can be cut back
    assert not plain.stale and plain.len == 2 and plain.state is None


def test_registry_and_loader(tmp_path):
    from cogstream_amd import auto
    from cogstream_amd import checkpoint as ck
    from cogstream_amd.lupanex import LupanexForCausalLM, parse_config
    cfg = CONFIGS["mixed"]
    st = state(cfg)
    ck.save_decoder(str(tmp_path), public(cfg), st)
    assert auto._resolve(str(tmp_path), "config.json", "AutoModelForCausalLM", auto._DEFAULT_MODEL) is LupanexForCausalLM
    found = ck.tensor_shapes(str(tmp_path))
    dc = parse_config(ck.read_config(str(tmp_path)), found)
    assert dc == parse(cfg) and {k: tuple(v.shape) for k, v in st.items()} == found
    view, reader = ck.open_decoder(str(tmp_path), dc, "cpu")
    for k in st:
        assert torch.equal(view[k].float(), st[k])
    reader.check_consumed()
    ck.save_decoder(str(tmp_path / "s"), public(cfg), dict(st, **{"l0.hc1.mix": st["l0.hc1.mix"][:-1]}))
    with pytest.raises(RuntimeError, match="l0.hc1.mix"):
        ck.open_decoder(str(tmp_path / "s"), dc, "cpu")
    ck.save_decoder(str(tmp_path / "m"), public(cfg), {k: v for k, v in st.items() if k != "l1.mix.A_log"})
    with pytest.raises(RuntimeError, match="l1.mix.A_log"):
        ck.open_decoder(str(tmp_path / "m"), dc, "cpu")


FAULTS = ["far_key", "bias", "bias_far", "bias_head", "temperature", "qk_norm", "group", "conv_tap", "conv_side", "decay", "beta", "read_before_write", "unit", "head_norm",
          "delta_gate", "state_lost", "loop_shares_nothing", "mix_transposed", "hc_in", "hc_out", "position", "embed_scale", "gelu_form"]


@pytest.mark.parametrize("fault", FAULTS)
def test_faults_show_in_the_test_models(fault):
    """the weights the GPU tests use let a fault of each mechanism show far above their tolerance (mistakes planted here)"""
    cfg = json.loads(json.dumps(CONFIGS["peaked"]))
    st = state(cfg)
    w, toks = double(st), tokens(cfg, 90)
    good = lo.forward(cfg, w, toks)[0]
    names = ["softmax", "bucket", "temperature", "rms", "short_conv", "delta_recurrence", "unit", "sigmoid", "order", "gelu", "attention"]
    saved = {n: getattr(lo, n) for n in names}
    soft, rec = saved["softmax"], saved["delta_recurrence"]
    put = lambda name, fn: setattr(lo, name, fn)
    try:
        if fault == "far_key":
            put("softmax", lambda s: soft(torch.where(torch.arange(len(s)) < len(s) - 64, s - 1e9, s)))
        elif fault == "bias":
            put("bucket", lambda n, rows, far: saved["bucket"](n + 1, rows, far))
        elif fault == "bias_far":
            put("bucket", lambda n, rows, far: min(saved["bucket"](n, rows, far), rows - 2))
        elif fault == "bias_head":
            w["l1.mix.rel"] = w["l1.mix.rel"].roll(1, 1)
        elif fault == "temperature":
            put("temperature", lambda p, t: saved["temperature"](p - 1, t))
        elif fault == "qk_norm":
            cfg["layers"][1]["mixer"]["scale"] *= 1.1
        elif fault == "group":
            w["l1.mix.k"] = w["l1.mix.k"].view(2, 32, -1).flip(0).reshape(64, -1)
        elif fault == "conv_tap":
            put("short_conv", lambda x, t: saved["short_conv"](x, torch.cat([torch.zeros_like(t[:, :1]), t[:, 1:]], 1)))
        elif fault == "conv_side":
            put("short_conv", lambda x, t: saved["short_conv"](x, t.flip(1)))
        elif fault == "decay":
            put("delta_recurrence", lambda q, k, v, b, g: rec(q, k, v, b, g.roll(1)))
        elif fault == "beta":
            put("delta_recurrence", lambda q, k, v, b, g: rec(q, k, v, b.roll(1), g))
        elif fault == "read_before_write":
            put("delta_recurrence", lambda q, k, v, b, g: torch.cat([torch.zeros_like(v[:1]), rec(torch.cat([q[1:], q[:1]]), k, v, b, g)[:-1]]))
        elif fault == "unit":
            put("unit", lambda x: x)
        elif fault == "head_norm":
            w["l0.mix.norm"] = torch.ones_like(w["l0.mix.norm"])
        elif fault == "delta_gate":
            w["l0.mix.g"] = w["l0.mix.g"].roll(32, 0)
        elif fault == "state_lost":
            put("delta_recurrence", lambda q, k, v, b, g: rec(q, k, v, b, torch.where(torch.arange(len(g)) == 80, 0.0, g)))
        elif fault == "loop_shares_nothing":
            put("order", lambda c: [0, 0, 1, 1, 2])
        elif fault == "mix_transposed":
            w["l1.hc1.mix"] = w["l1.hc1.mix"].T
        elif fault == "hc_in":
            w["l0.hc2.in"] = w["l0.hc2.in"].flip(0)
        elif fault == "hc_out":
            w.update({k: torch.ones_like(v) for k, v in w.items() if k.endswith("hc2.out")})
        elif fault == "position":
            w["pos"] = w["pos"].roll(1, 0)
        elif fault == "embed_scale":
            w["embed"] = w["embed"] * 1.2
        elif fault == "gelu_form":
            put("gelu", lambda z: torch.nn.functional.silu(1.702 * z) / 1.702)
        bad = lo.forward(cfg, w, toks)[0]
    finally:
        for n in names:
            setattr(lo, n, saved[n])
    # (a state or key lost at one place is looked for right behind it; the last ones are small by nature and show in float32)
    assert rms_err(bad[80:], good[80:]) > (0.005 if fault in ("temperature", "gelu_form") else 0.035)


def test_shapes_helper_names_every_attention_table():
    assert set(shapes(CONFIGS["mixed"])) == {"l0.mix.rel", "l2.mix.rel"}
