"""Model registry: which classes a model directory is opened with.  A directory names its design in config.json
("architecture") or is a .gturbo directory (manifest.json) of the hybrid mixture-of-experts model."""
import json
import os


class Family:
    """name; part: the part library (build.PARTS) its kernels are in, None: the whole library; activations: the context
    types it runs in, by name; open: (ctx, path, options) -> step driver."""

    def __init__(self, name, part, activations, open_):
        self.name, self.part, self.activations, self.open = name, part, activations, open_


def _open_pakirax(ctx, path, batch=1, max_context=32768, max_chunk=2048):
    from .pakirax import PakiraxDecoder, PakiraxWeights
    cfg, weights = PakiraxWeights.from_directory(ctx, path)
    return PakiraxDecoder(ctx, cfg, weights, batch, max_context, max_chunk)


def _open_kemuzen(ctx, path, batch=1, max_context=32768, max_chunk=2048):
    from .kemuzen import KemuzenDecoder, KemuzenWeights
    cfg, weights = KemuzenWeights.from_directory(ctx, path)
    return KemuzenDecoder(ctx, cfg, weights, batch, max_context, max_chunk)


def _open_hybrid(ctx, path, batch=1, max_context=32768, max_chunk=None):
    from . import gturbo
    from .decoder import HybridDecoder, HybridWeights
    cfg, weights = HybridWeights.from_gturbo(ctx, gturbo.GTurboModel(path))
    return HybridDecoder(ctx, cfg, weights, batch, max_context)


FAMILIES = {"Pakirax": Family("Pakirax", "dense", ("bfloat16", "float32"), _open_pakirax),
            "Kemuzen": Family("Kemuzen", "scan", ("bfloat16", "float32"), _open_kemuzen),
            "hybrid-moe": Family("hybrid-moe", None, ("bfloat16", "float16"), _open_hybrid)}


class UnknownModel(ValueError):
    pass


def family_of(path):
    """The family of a model directory.  Reads no weights and needs no library."""
    if os.path.exists(os.path.join(path, "manifest.json")):
        return FAMILIES["hybrid-moe"]
    try:
        with open(os.path.join(path, "config.json")) as f:
            name = json.load(f).get("architecture")
    except FileNotFoundError:
        raise UnknownModel("%s holds neither manifest.json nor config.json" % path)
    if name not in FAMILIES or name == "hybrid-moe":
        raise UnknownModel("architecture %r is not one of %s" % (name, ", ".join(sorted(set(FAMILIES) - {"hybrid-moe"}))))
    return FAMILIES[name]


def open_model(path, dtype="bfloat16", device=0, **options):
    """The step driver of a model directory in a context of its own."""
    from . import ops
    family = family_of(path)
    if dtype not in family.activations:
        raise UnknownModel("%s runs in %s, not in %s" % (family.name, " or ".join(family.activations), dtype))
    act = {"bfloat16": ops.ACT_BF16, "float16": ops.ACT_FP16, "float32": ops.ACT_FP32}[dtype]
    return family.open(ops.Context(device, act), path, **options)
