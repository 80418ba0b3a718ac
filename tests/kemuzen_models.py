"""Small random Kemuzen models for the tests: configurations, weights, and a directory to open them from."""
import math

import torch

from nvmai_amd.kemuzen import KemuzenConfig


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _mask(size, keep):
    return None if size is None else dict({"size": size}, **({} if keep is None else {"keep_first": keep}))


def attention(heads, kv_heads, dim, vdim, size, keep, softcap=12.0, scale=None, ff=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
         "softcap": softcap, "mask": _mask(size, keep)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return _layer("attention", m, ff)


def delta(heads, kv_heads, dim, vdim, conv, ff=None):
    return _layer("delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, ff)


def parallel(left, right, scales, ff=None):
    """left: heads, kv_heads, dim, vdim, window; right: heads, vdim, state, groups, conv, norm groups"""
    H, G, dim, vdim, size = left
    h, P, N, g, conv, parts = right
    return _layer("parallel", {"left": {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "scale": dim ** -0.5, "mask": _mask(size, None)},
                               "right": {"heads": h, "vdim": P, "state": N, "groups": g, "conv": conv, "norm_groups": parts},
                               "left_scale": scales[0], "right_scale": scales[1]}, ff)


def config(vocab, width, layers, side, eps=1e-5, scale=2.0, cap=11.0):
    out = {"architecture": "Kemuzen", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}
    if side:
        out["token_side"] = {"dim": side}
    if cap:
        out["logit_softcap"] = cap
    return out


MODELS = {
    # every kind of padding; sharers of one cache with wider, longer-kept and narrower masks; norm groups across heads
    "mixed": config(131, 72, [attention(6, 2, 20, 24, 17, 3, ff=90), delta(4, 2, 24, 40, 3, ff=70),
                              parallel((3, 1, 20, 12, 9), (6, 20, 20, 2, 5, 4), (0.7, 1.3), ff=33),
                              attention(6, 2, 20, 24, 50, 70, softcap=5.0, kv_from=0), delta(3, 3, 40, 12, 4),
                              attention(6, 2, 20, 24, 5, 1, scale=0.4, ff=40, kv_from=0)], side=12),
    "aligned": config(256, 128, [parallel((4, 4, 64, 64, 33), (4, 64, 64, 4, 4, 1), (1.0, 0.5), ff=256), attention(8, 2, 32, 64, 32, 64, ff=64),
                                 delta(2, 1, 64, 128, 4, ff=128), attention(4, 4, 128, 64, 64, 4)], side=64, scale=1.0),
    "wide": config(64, 96, [attention(34, 2, 160, 144, 100, 9, ff=64), parallel((17, 1, 40, 16, 21), (3, 48, 160, 1, 4, 3), (1.1, 0.6)),
                            delta(2, 2, 144, 160, 2)], side=8, cap=30.0),
    # the smallest of everything, filters of one tap, no kept tokens
    "ones": config(40, 2, [attention(1, 1, 1, 1, 1, 0, ff=1), delta(1, 1, 1, 1, 1), parallel((1, 1, 3, 1, 2), (1, 2, 1, 1, 1, 1), (1.0, 1.0), ff=3),
                           attention(2, 1, 3, 2, 4, 2)], side=1),
    # nothing hidden, no caps, no side input
    "open": config(97, 48, [attention(4, 2, 32, 48, None, None, softcap=None, ff=100), attention(4, 2, 32, 48, 300, 2, softcap=None, kv_from=0),
                            parallel((2, 2, 16, 16, 70), (2, 24, 32, 1, 4, 2), (1.0, 1.0))], side=0, cap=None, scale=6.0),
    # sizes that only the general forms take
    "large": config(61, 64, [attention(2, 1, 288, 272, 40, 5), delta(1, 1, 272, 272, 3, ff=20)], side=5),
}


def weights(cfg, seed, sharp=4.0, embed_std=1.0):
    """BF16 tensors.  sharp scales the queries' norm weights, so that single keys stand out wherever they are;
    decays spread from quick forgetting to near 1."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in KemuzenConfig(cfg).tensor_shapes().items():
        last = name.rsplit(".", 1)[-1]
        if last == "conv":
            v = torch.randn(shape, generator=gen) * (0.6 / math.sqrt(shape[1]))
            v[:, -1] += 0.7
        elif len(shape) == 2:
            v = torch.randn(shape, generator=gen) * shape[1] ** -0.5
            if name == "embed":
                v = torch.randn(shape, generator=gen) * embed_std
            elif name == "side.embed":
                v = torch.randn(shape, generator=gen)
        elif last == "A_log":
            v = torch.rand(shape, generator=gen) * 4.0 - 2.0
        elif last == "dt_bias":
            v = torch.rand(shape, generator=gen) * 6.0 - 4.0
        elif last in ("norm1", "norm2", "b") or name == "final.norm":
            v = torch.randn(shape, generator=gen) * 0.2
        else:
            v = 1.0 + torch.randn(shape, generator=gen) * 0.2
            if name.endswith("q.norm"):
                v = v * sharp
        out[name] = v.to(torch.bfloat16)
    return out
