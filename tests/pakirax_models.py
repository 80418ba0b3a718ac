"""Small random Pakirax models for the tests: configurations, weights, and a directory to open them from."""
import json
import os

import numpy as np
import torch

from nvmai_amd.pakirax import PakiraxConfig
from nvmai_amd.safetensors_file import write_safetensors


def gla(heads, dim, vdim, tau, ff=None):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, window, base=10000.0, scale=None, ff=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "mask": {"size": window},
                      "rot": {"base": base, "dims": rot_dim}},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(vocab, width, layers, eps=1e-5, residual_mult=0.5):
    return {"architecture": "Pakirax", "vocab": vocab, "width": width, "residual_mult": residual_mult, "norm": {"eps": eps},
            "layers": layers}


# sizes that need every kind of padding, layers of one type with different sizes, every feed-forward arrangement
MODELS = {
    "mixed": config(131, 72, [latent(3, 20, 12, 24, 40, 36, 17, ff=90), gla(2, 24, 40, 4.0, ff=70), latent(3, 20, 12, 24, 40, 36, 50),
                              gla(5, 8, 12, 16.0), latent(2, 16, 8, 16, 72, 20, 5, base=500.0, ff=33)]),
    "aligned": config(256, 128, [gla(2, 64, 128, 8.0), latent(4, 64, 64, 64, 64, 128, 33, scale=0.3, ff=256),
                                 gla(1, 128, 64, 16.0, ff=64)], residual_mult=0.25),
    "wide_heads": config(64, 64, [latent(17, 32, 16, 32, 192, 64, 100, ff=128), gla(17, 16, 16, 1.0)], residual_mult=1.0),
    "one_of_each": config(40, 16, [gla(1, 1, 1, 1.0), latent(1, 1, 2, 1, 1, 1, 1, ff=1), latent(1, 3, 2, 5, 2, 7, 9)]),
    "attention_only": config(97, 48, [latent(2, 32, 32, 48, 96, 64, 70, base=1e6, ff=100), latent(2, 16, 32, 16, 64, 32, 300)]),
    "gla_only": config(97, 48, [gla(3, 16, 32, 2.0, ff=50), gla(2, 40, 20, 16.0)]),
}


def weights(cfg, seed, sharp=3.0, decay_rank=6, embed_std=1.0):
    """BF16 tensors.  sharp scales the queries of latent attention, so that single keys stand out wherever they are;
    the decay biases spread from quick forgetting to near 1.
    A small embed_std leaves the residual to the layers (with a large one greedy generation repeats its last token)."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    ranks = lambda i: decay_rank + i
    for name, shape in PakiraxConfig(cfg).tensor_shapes(ranks).items():
        if len(shape) == 1:
            v = torch.randn(shape, generator=gen) * 0.2
            if name.endswith("a2.b"):
                v = torch.rand(shape, generator=gen) * 9.0 - 2.0
            elif not name.endswith(".b"):
                v = v + 1.0
        else:
            v = torch.randn(shape, generator=gen) * shape[1] ** -0.5
            if name.endswith(".uq"):
                v = v * sharp
            elif name == "embed":
                v = torch.randn(shape, generator=gen) * embed_std
        out[name] = v.to(torch.bfloat16)
    return out


def numpy64(tensors):
    return {k: v.float().numpy().astype(np.float64) for k, v in tensors.items()}


def write_model(path, cfg, tensors):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(path, "model.safetensors"), tensors)
    return str(path)


def tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def logit_error(got, want):
    """Per row: root mean square of the difference with its mean taken off, over the spread of the expected logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean())
