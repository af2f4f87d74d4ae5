"""Pabalix without a GPU: the configuration and its tensor names, rotations, the packed layouts (recomputed from the packed
tensors with plain torch), the model registry, and that the oracle notices what the GPU tests are meant to notice."""
import ctypes as C
import json
import math
import os

import pytest
import torch

from oracle import pabalix as po
from pabalix_models import A, B, CONFIGS, G, YARN, config, double, mixer, rms_err, state, tokens


def _view(ptr, shape, packed):
    return next(t for t in packed.keep if isinstance(t, torch.Tensor) and t.data_ptr() == ptr).view(*shape)


def test_rotation_frequencies_match_the_oracle():
    from cogstream_amd.pabalix import parse_config
    for cfg in CONFIGS.values():
        for lay, mine in zip(cfg["layers"], parse_config(cfg).layers):
            f, mag = po.frequencies(lay["mixer"]["rot"])
            assert mine.mixer.rot.frequencies() == pytest.approx(f, rel=1e-14) and mine.mixer.rot.magnitude == pytest.approx(mag)
    # a pair inside the ramp, one on either side, and a ramp of no width
    f, mag = po.frequencies(dict(dims=20, base=5000.0, scaling=dict(factor=5.0, original=1000, fast=20.0, slow=1.5)))
    g = [5000.0 ** (-2 * i / 20) for i in range(10)]
    r = [a / b for a, b in zip(f, g)]
    assert r[0] == 1 and r[-1] == pytest.approx(0.2) and any(0.21 < x < 0.99 for x in r) and mag == pytest.approx(1 + 0.1 * math.log(5))
    f, _ = po.frequencies(dict(dims=8, base=10.0, scaling=dict(factor=2.0, original=100000, fast=1e-9, slow=1e-9)))
    assert f == [10.0 ** (-2 * i / 8) for i in range(4)]


def test_oracle_rotation_keeps_norms_and_relative_positions():
    g = torch.Generator().manual_seed(0)
    for inter in (False, True):
        rot = dict(dims=8, base=100.0)
        q, k = torch.randn(8, generator=g, dtype=torch.float64), torch.randn(8, generator=g, dtype=torch.float64)
        a, b = po.rotate(q.repeat(40, 1), rot, inter), po.rotate(k.repeat(40, 1), rot, inter)
        s = a @ b.T
        assert torch.allclose(s.diagonal(7), s[0, 7].expand(33)) and torch.allclose(a.norm(dim=1), q.norm())
    assert not torch.allclose(po.rotate(q[None].repeat(2, 1), rot, False), po.rotate(q[None].repeat(2, 1), rot, True))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_packed_layouts_give_the_same_projections(name):
    """latents, queries (rotated pairs adjacent), keys, values, the absorbed product and the MLP from the packed tensors"""
    from cogstream_amd.pabalix import parse_config
    from cogstream_amd.weights import PackedDecoder
    cfg = CONFIGS[name]
    dc, st = parse_config(cfg), state(cfg)
    pk = PackedDecoder(st, dc, torch.float32, "cpu")
    up = lambda v, m: -(-v // m) * m
    gen = torch.Generator().manual_seed(3)
    W, Wp = cfg["width"], up(cfg["width"], 64)
    assert pk.width_p == Wp and pk.embed.shape == (cfg["vocab"], Wp) and pk.vocab_p == up(cfg["vocab"], 4)
    h = torch.randn(5, W, generator=gen)
    hp = torch.zeros(5, Wp)
    hp[:, :W] = h
    for i, lay in enumerate(cfg["layers"]):
        m, x, pre = lay["mixer"], pk.layers[i].latent, f"l{i}.mix."
        qrp, kvp, rc = up(m["q_rank"], 64), up(m["kv_rank"], 64), up(m["rot_dim"], 32)
        dn, dk, dv = up(m["dim"], 8), up(m["dim"], 32), up(m["vdim"], 16)
        dq, H, own = dk + rc, m["heads"], m.get("kv_from") is None
        order = list(range(m["rot_dim"])) if lay["type"] == B else [j for i2 in range(m["rot_dim"] // 2) for j in (i2, i2 + m["rot_dim"] // 2)]
        rows = qrp + (kvp + rc if own else 0) + (up(H, 4) if lay["type"] == G else 0)
        t = hp @ _view(x.in_w, (rows, Wp), pk).T
        assert torch.allclose(t[:, :m["q_rank"]], h @ st[pre + "dq"].T, atol=1e-5) and not t[:, m["q_rank"]:qrp].any()
        if own:
            d = h @ st[pre + "dkv"].T
            assert torch.allclose(t[:, qrp:qrp + m["kv_rank"]], d[:, :m["kv_rank"]], atol=1e-5)
            assert torch.allclose(t[:, qrp + kvp:qrp + kvp + m["rot_dim"]], d[:, m["kv_rank"]:][:, order], atol=1e-5)
        if lay["type"] == G:
            at = qrp + (kvp + rc if own else 0)
            assert torch.allclose(t[:, at:at + H], h @ st[pre + "g"].T, atol=1e-5)
            assert torch.allclose(_view(x.sink, (H,), pk), st[pre + "sink"] / math.log(2))
        c, cq = torch.randn(5, m["kv_rank"], generator=gen), torch.randn(5, m["q_rank"], generator=gen)
        cp, cqp = torch.zeros(5, kvp), torch.zeros(5, qrp)
        cp[:, :m["kv_rank"]], cqp[:, :m["q_rank"]] = c, cq
        q = (cqp @ _view(x.q_w, (H * dq, qrp), pk).T).view(5, H, dq)
        want = (cq @ st[pre + "uq"].T).view(5, H, -1)
        assert torch.allclose(q[..., :m["dim"]], want[..., :m["dim"]], atol=1e-5)
        assert torch.allclose(q[..., dk:dk + m["rot_dim"]], want[..., m["dim"]:][..., order], atol=1e-5)
        assert not q[..., m["dim"]:dk].any() and not q[..., dk + m["rot_dim"]:].any()
        kv = cp @ _view(x.kv_w, (H * (dn + dv), kvp), pk).T
        k, v = (c @ st[pre + "uk"].T).view(5, H, -1), (c @ st[pre + "uv"].T).view(5, H, -1)
        assert torch.allclose(kv[:, :H * dn].view(5, H, dn)[..., :m["dim"]], k, atol=1e-5)
        assert torch.allclose(kv[:, H * dn:].view(5, H, dv)[..., :m["vdim"]], v, atol=1e-5)
        ab = torch.einsum("bhk,hnk->bhn", torch.nn.functional.pad(want[..., :m["dim"]], (0, dk - m["dim"])), _view(x.k_abs, (H, kvp, dk), pk))
        assert torch.allclose(torch.einsum("bhn,jn->bhj", ab, cp), torch.einsum("bhd,jhd->bhj", want[..., :m["dim"]], k), atol=1e-3)
        o = torch.zeros(5, up(H * dv, 64))
        o[:, :H * dv].view(5, H, dv)[..., :m["vdim"]] = v
        y = o @ _view(x.o_w, (Wp, o.shape[1]), pk).T
        assert torch.allclose(y[:, :W], v.reshape(5, -1) @ st[pre + "o"].T, atol=1e-4) and not y[:, W:].any()
        if lay["mlp"] is not None:
            ml, f = pk.layers[i].mlp, f"l{i}.mlp."
            ffp = up(ml.ff, 64)
            gu = hp @ _view(ml.up_w, (2 * ffp, Wp), pk).T + _view(ml.up_b, (2 * ffp,), pk)
            a = torch.nn.functional.silu(gu[:, 0::2]) * gu[:, 1::2]
            y = a @ _view(ml.down_w, (Wp, ffp), pk).T + _view(ml.down_b, (Wp,), pk)
            assert torch.allclose(y[:, :W], po.feed_forward(h, st, f), atol=1e-4) and not y[:, W:].any()
        else:
            assert pk.layers[i].mlp.ff == 0


def test_ctypes_structs_match_the_header(tmp_path):
    import shutil
    import subprocess
    from cogstream_amd import _lib as L
    if shutil.which("gcc") is None:
        pytest.skip("no gcc")
    names = {"cogs_latent_mixer": L.LatentMixer, "cogs_attn_mixer": L.AttnMixer, "cogs_delta_mixer": L.DeltaMixer, "cogs_hyper": L.Hyper,
             "cogs_decoder_mlp": L.DecoderMlp, "cogs_decoder_layer": L.DecoderLayer,
             "cogs_decoder_weights": L.DecoderWeights, "cogs_kv": L.KV}
    lines = [f'printf("{n} %zu", sizeof({n}));' + "".join(f'printf(" %zu", offsetof({n}, {f[0].rstrip("_")}));' for f in t._fields_) + 'printf("\\n");'
             for n, t in names.items()]
    src = tmp_path / "t.c"
    src.write_text('#include <stdio.h>\n#include <stddef.h>\n#include "cogs.h"\nint main(void) {' + "\n".join(lines) + "return 0; }\n")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    subprocess.check_call(["gcc", "-std=c99", "-I", os.path.join(root, "include"), str(src), "-o", str(tmp_path / "t")])
    for line in subprocess.check_output([str(tmp_path / "t")], text=True).splitlines():
        n, *v = line.split()
        t = names[n]
        assert [C.sizeof(t)] + [getattr(t, f[0]).offset for f in t._fields_] == [int(x) for x in v], n


def test_registry_and_loader(tmp_path):
    from cogstream_amd import auto
    from cogstream_amd import checkpoint as ck
    from cogstream_amd.pabalix import PabalixForCausalLM, parse_config
    cfg = CONFIGS["mixed"]
    dc = parse_config(cfg)
    st = state(cfg)
    ck.save_decoder(str(tmp_path), cfg, st)
    assert auto._resolve(str(tmp_path), "config.json", "AutoModelForCausalLM", auto._DEFAULT_MODEL) is PabalixForCausalLM
    view, reader = ck.open_decoder(str(tmp_path), dc, "cpu")
    for k in st:
        assert torch.equal(view[k].float(), st[k])
    reader.check_consumed()
    # a tensor of another shape, a tensor that is missing, an unknown architecture / mixer / feed-forward, a bad kv_from
    ck.save_decoder(str(tmp_path / "s"), cfg, dict(st, head=st["head"][:-1]))
    with pytest.raises(RuntimeError, match="head"):
        ck.open_decoder(str(tmp_path / "s"), dc, "cpu")
    ck.save_decoder(str(tmp_path / "m"), cfg, {k: v for k, v in st.items() if k != "l0.mix.sink"})
    with pytest.raises(RuntimeError, match="l0.mix.sink"):
        ck.open_decoder(str(tmp_path / "m"), dc, "cpu")
    with open(tmp_path / "config.json", "w") as f:
        json.dump(dict(cfg, architecture="Nothing"), f)
    with pytest.raises(ValueError, match="Nothing"):
        auto.AutoModelForCausalLM.from_pretrained(str(tmp_path))
    for bad in (dict(mixer(A), type="other"), mixer(B, kv_from=1), mixer(B, kv_from=4)):
        with pytest.raises(ValueError):
            parse_config(config([mixer(B), mixer(B, kv_from=0), bad]))
    lay = config([mixer(A)])
    lay["layers"][0]["mlp"]["kind"] = "sparse"
    with pytest.raises(ValueError):
        parse_config(lay)


def test_generation_loop_of_the_base_class_batches_any_engine():
    """Sequences over an engine without a batched step: one forward per sequence, wanted rows in order, caches grow by moving"""
    from cogstream_amd.llm import CausalEngine, KVCache, Sequences

    class Cache(KVCache):
        def __init__(self, n):
            self.k = self.v = torch.zeros(1, n, 1)
            self.struct = type("S", (), dict(len=0, max_len=n))()

    class Toy(CausalEngine):
        """logits of a row = running sum of the sequence's tokens, one-hot"""
        device, cfg = "cpu", type("Cfg", (), dict(vocab_size=50))()

        def new_cache(self, n):
            return Cache(n)

        def embed_tokens(self, ids):
            return ids.float()[:, None]

        def logits_of(self, hidden):
            return torch.nn.functional.one_hot(hidden[:, 0].long() % 50, 50).float()

        def forward(self, e, cache, want_logits=True, want_hidden=False):
            cache.k[0, cache.len:cache.len + len(e)] = e
            hid = cache.k[0].cumsum(0)[cache.len:cache.len + len(e)]
            cache.reset(cache.len + len(e))
            return {"logits": self.logits_of(hid[-1:])[0]} if want_logits else {"hidden": hid}

    s = Sequences(Toy(), reserve=2)
    out = s.step([("a", [1, 2, 3], [0, 2]), ("b", [7], [0]), ("c", [4, 4], [])])
    assert out.argmax(1).tolist() == [1, 6, 7]
    for i in range(5):
        out = s.step([("b", [1], [0]), ("a", [2], [0])])
        assert out.argmax(1).tolist() == [8 + i, 8 + 2 * i]
    s.release("a")
    assert s.step([("a", [9], [0])]).argmax(1).tolist() == [9] and s.step([("c", [1], [])]) is None
    for bad in ([("a", [], [])], [("a", [50], [])], [("a", [1], [1])], [("a", [1], []), ("a", [2], [])]):
        with pytest.raises(ValueError):
            s.step(bad)


@pytest.mark.parametrize("fault", ["far_key", "sink", "gate", "pairs", "yarn", "norm_b", "window"])
def test_faults_show_in_the_test_models(fault):
    """the weights the GPU tests use let a fault of each mechanism show far above their tolerance (mistakes planted here)"""
    cfg = CONFIGS["peaked"]
    w, toks = double(state(cfg)), tokens(cfg, 70)
    good = po.forward(cfg, w, toks)[0]
    saved = po.sink_softmax, po.rotate, po.frequencies
    try:
        if fault == "far_key":
            po.sink_softmax = lambda s, sink: saved[0](torch.where(torch.arange(len(s)) == 2, s - 1e9, s) if len(s) > 60 else s, sink)
        elif fault == "window":
            po.sink_softmax = lambda s, sink: saved[0](torch.where(torch.arange(len(s)) < len(s) - 64, s - 1e9, s), sink)
        elif fault == "sink":
            po.sink_softmax = lambda s, sink: saved[0](s, None)
        elif fault == "pairs":
            po.rotate = lambda x, rot, inter: saved[1](x, rot, not inter)
        elif fault == "yarn":
            po.frequencies = lambda rot: saved[2](dict(rot, scaling=None))
        elif fault == "gate":
            w = dict(w, **{"l0.mix.g": w["l0.mix.g"] * 0})
        elif fault == "norm_b":
            w = dict(w, **{"l3.norm2b": torch.ones_like(w["l3.norm2b"])})
        bad = po.forward(cfg, w, toks)[0]
    finally:
        po.sink_softmax, po.rotate, po.frequencies = saved
    assert rms_err(bad[-5:], good[-5:]) > 0.06
