"""Small Lupanex configurations and weights for the tests, made from seeds (no checkpoint)."""
import torch

from cogstream_amd.lupanex import parse_config
from cogstream_amd.weights import decoder_tensors, random_decoder_state
from pabalix_models import double, rms_err, tokens  # noqa: F401


def attention(heads=3, kv_heads=None, dim=24, vdim=40, rows=12, far=50, scale=None, temp=(0.4, 10), gain=1.0, **kw):
    m = dict(heads=heads, kv_heads=kv_heads or heads, dim=dim, vdim=vdim, bias_max=far, scale=gain * dim ** -0.5 if scale is None else scale)
    if temp is not None:
        m["q_temp"] = dict(coef=temp[0], every=temp[1])
    return dict(type="attention", mixer=m, rows=rows, **kw)


def delta(heads=4, kv_heads=2, dim=20, vdim=28, conv=3, **kw):
    return dict(type="delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), **kw)


def config(layers, width=136, vocab=211, ff=104, eps=1e-5, streams=3, loop=None, scale=1.7, positions=512):
    """rows of the bias tables (a size no key gives) travel in the tensors' shapes: shapes(cfg)"""
    out = []
    for lay in layers:
        lay = dict(lay)
        f = lay.pop("ff", ff)
        lay["mlp"] = None if f is None else dict(kind="dense", ff=f)
        out.append(lay)
    cfg = dict(architecture="Lupanex", layers=out, norm=dict(eps=eps), vocab=vocab, width=width, streams=streams,
               embedding=dict(scale=scale), max_positions=positions)
    if streams is None:                # a plain residual
        del cfg["streams"]
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def shapes(cfg):
    return {f"l{i}.mix.rel": (lay["rows"], lay["mixer"]["heads"]) for i, lay in enumerate(cfg["layers"]) if lay["type"] == "attention"}


def parse(cfg):
    return parse_config(cfg, shapes(cfg))


CONFIGS = {
    # every branch: grouped heads, layers without a feed-forward, a loop over unlike layers in the middle, odd sizes everywhere
    "mixed": config([attention(heads=6, kv_heads=2), delta(), dict(attention(heads=4, kv_heads=1, dim=10, vdim=18, rows=6, far=90, temp=None), ff=None),
                     dict(delta(heads=3, kv_heads=1, dim=36, vdim=12, conv=5), ff=72), delta(heads=2, kv_heads=2, conv=2)], loop=(1, 4, 2)),
    # scores and decays that let single keys and old tokens show
    "peaked": config([delta(heads=4, kv_heads=4, dim=32, vdim=32, conv=4), attention(heads=4, kv_heads=2, dim=32, vdim=32, gain=1.5, rows=16, far=70),
                      delta(heads=2, kv_heads=1, dim=32, vdim=48, conv=4)], width=192, ff=128, streams=2, loop=(0, 2, 2)),
    "one": config([attention(heads=1, dim=4, vdim=4, rows=2, far=3, temp=(0.3, 1))], width=8, vocab=5, ff=4, streams=1),
    "one_delta": config([delta(heads=1, kv_heads=1, dim=4, vdim=4, conv=1)], width=8, vocab=5, ff=4, streams=1, scale=1.0),
    # the whole model in a loop, every size alike, a loop of one pass
    "same": config([delta(heads=4, kv_heads=4, dim=32, vdim=32, conv=4), attention(heads=4, dim=32, vdim=32, rows=32, far=64)], width=64, vocab=128, ff=64,
                   streams=4, loop=(0, 2, 2)),
    "plain": config([delta(heads=2, kv_heads=1), attention(heads=2, kv_heads=1)], width=72, vocab=90, streams=None),
    "once": config([attention(heads=2), delta(heads=2, kv_heads=1)], width=64, vocab=96, streams=5, loop=(1, 2, 1)),
    "wide": config([delta(heads=8, kv_heads=4, dim=128, vdim=128, conv=4), attention(heads=20, kv_heads=1, dim=128, vdim=128, rows=32, far=64),
                    attention(heads=12, kv_heads=4, dim=64, vdim=64, rows=8, far=1000)], width=512, vocab=400, ff=320, streams=4),
    # above the matrix kernels' instances: row-wise attention, the token-by-token recurrence, a state that does not fit registers
    "large": config([attention(heads=2, dim=200, vdim=272), delta(heads=2, kv_heads=1, dim=300, vdim=200), delta(heads=1, kv_heads=1, dim=200, vdim=264, conv=6),
                     attention(heads=2, kv_heads=1, dim=160, vdim=176)], width=256, vocab=160, ff=192, streams=9),
}


def state(cfg, seed=2, bf16=True):
    """fp32 weights (values representable in bf16, so that both modes of the framework and the oracle see the same model)"""
    st = random_decoder_state(parse(cfg), seed=seed)
    assert set(st) == set(decoder_tensors(parse(cfg)))
    for k, v in st.items():
        if "norm" in k.rsplit(".", 1)[-1]:
            st[k] = (v - 1) * 3 + 1          # uneven enough that a missing or swapped norm shows
        elif k.endswith(".rel"):
            st[k] = v * 2
    return {k: v.to(torch.bfloat16).float() for k, v in st.items()} if bf16 else st


def public(cfg):
    """the configuration as a checkpoint has it"""
    return dict(cfg, layers=[{k: v for k, v in lay.items() if k != "rows"} for lay in cfg["layers"]])
