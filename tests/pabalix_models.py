"""Small Pabalix configurations and weights for the tests, made from seeds (no checkpoint)."""
import torch

from cogstream_amd.pabalix import parse_config
from cogstream_amd.weights import random_decoder_state


def mixer(kind, heads=3, dim=24, rot=16, vdim=40, q_rank=72, kv_rank=56, base=10000.0, scale=None, scaling=None, kv_from=None, gain=1.0):
    m = dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
             scale=(dim + rot) ** -0.5 * gain if scale is None else scale, rot=dict(base=base, dims=rot))
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type=kind, mixer=m)


def config(layers, width=136, vocab=211, ff=104, eps=1e-5):
    out = []
    for lay in layers:
        lay = dict(lay)
        f = lay.pop("ff", ff)
        lay["mlp"] = None if f is None else dict(kind="dense", ff=f)
        out.append(lay)
    return dict(architecture="Pabalix", layers=out, norm=dict(eps=eps), vocab=vocab, width=width)


A, B, G = "latent_attention", "latent_attention_2", "latent_attention_3"
YARN = (3.0, 64, 24.0, 1.5)          # the ramp lies inside the pairs of a 16-dimensional rotation

# sizes no two of which agree by accident; every branch of the design
CONFIGS = {
    "mixed": config([mixer(G, heads=5, scaling=YARN, base=500.0), mixer(A, heads=2, dim=40, rot=8, vdim=16, kv_rank=40, scaling=(2.0, 128, 16.0, 2.0)),
                     mixer(B, heads=3, dim=20, rot=12, vdim=28, kv_rank=44, q_rank=30), dict(mixer(B, heads=6, dim=32, rot=12, vdim=8, kv_rank=44, q_rank=50, kv_from=2), ff=None),
                     mixer(B, heads=1, dim=8, rot=12, vdim=70, kv_rank=44, q_rank=24, kv_from=2), mixer(G, heads=2, dim=16, rot=32, vdim=24, base=2000.0, scaling=YARN)]),
    "peaked": config([mixer(G, heads=4, gain=1.5, scaling=YARN), mixer(B, heads=4, gain=1.5), mixer(B, heads=4, gain=1.5, kv_from=1), mixer(A, heads=4, gain=1.5, scaling=YARN)],
                     width=192, ff=128),
    "plain": config([mixer(A, heads=2), mixer(G, heads=2), dict(mixer(B, heads=2), ff=None)], width=64, vocab=96),     # no YaRN anywhere
    "one": config([mixer(A, heads=1, dim=8, rot=2, vdim=8, q_rank=8, kv_rank=8, scaling=YARN)], width=8, vocab=5, ff=4),
    "same": config([mixer(k, heads=4, dim=32, rot=32, vdim=32, q_rank=64, kv_rank=64, scaling=None if k == B else (1.0, 900, 25.0, 2.0)) for k in (A, B, G)],
                   width=64, vocab=128, ff=64),                                                                         # everything alike, a factor of 1
    "wide": config([mixer(G, heads=20, dim=128, rot=64, vdim=128, q_rank=192, kv_rank=512, scaling=YARN), mixer(B, heads=17, dim=64, rot=32, vdim=64, kv_rank=256)],
                   width=512, vocab=400, ff=320),
    "large_rank": config([mixer(A, heads=3, dim=160, rot=64, vdim=192, kv_rank=640, scaling=YARN), mixer(G, heads=2, dim=200, rot=96, vdim=272, kv_rank=1000)],
                         width=256, vocab=160, ff=192),
}


def state(cfg, seed=0, bf16=True):
    """fp32 weights (values representable in bf16, so that both modes of the framework and the oracle see the same model)"""
    st = random_decoder_state(parse_config(cfg), seed=seed)
    for k, v in st.items():
        if k.endswith(".sink"):
            st[k] = v * 2 + 1
        elif "norm" in k.rsplit(".", 1)[-1]:
            st[k] = (v - 1) * 3 + 1          # uneven enough that a missing or swapped norm shows
    return {k: v.to(torch.bfloat16).float() for k, v in st.items()} if bf16 else st


def tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def double(st):
    return {k: v.double() for k, v in st.items()}


def rms_err(got, want):
    """per row: root mean square of the difference (mean taken off) over that of the reference; the largest row"""
    got, want = got.detach().double().cpu(), want.double()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt()).max())
