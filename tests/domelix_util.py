"""Helpers of the Domelix tests: small irregular configurations. Checkpoint
writing, engines and the step driver are the ones of vurizen_util. A left
mixer's 'rows' (of its bias table) is for the weight generator only: the package
reads it from the tensor."""

from vurizen_util import (  # noqa: F401
    close_in_bf16, describe, make_engine, rel_err, row_errs, run_schedule,
    same_as_whole, tokens, write_checkpoint,
)


def experts(n=6, top=2, ff=20, groups=(3, 2)):
    router = {"experts": n, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def _spec(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": experts() if mlp == "default" else mlp}


def decays(n):
    return [(0.97, 0.5, 0.999, 0.8, 1.0)[i % 5] for i in range(n)]


def left(heads=3, kv_heads=1, dim=12, vdim=20, scale=0.3, bias_max=50, rows=10):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
            "bias_max": bias_max, "rows": rows}


def right(heads=2, dim=10, vdim=14, decay=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay or decays(heads)}


def parallel_layer(lf=None, rt=None, mlp="default"):
    return _spec("parallel", {"left": lf or left(), "right": rt or right()}, mlp)


def delta_layer(heads=4, kv_heads=2, dim=12, vdim=9, conv=4, mlp="default"):
    return _spec("delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                           "conv": conv}, mlp)


def retention_layer(heads=3, dim=14, vdim=22, dims=8, base=300.0, decay=None, mlp="default"):
    mx = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay or decays(heads)}
    if dims:
        mx["rot"] = {"dims": dims, "base": base}
    return _spec("retention", mx, mlp)


def small_config(layers=None, width=40, vocab=83, eps=1e-5) -> dict:
    """Sizes away from powers of two and from each other, every mixer kind,
    grouped and ungrouped routers, a layer without feed-forward, two parallel
    layers of unlike geometry."""
    if layers is None:
        layers = [
            delta_layer(),
            parallel_layer(),
            retention_layer(mlp=experts(4, 3, 28, None)),
            parallel_layer(left(4, 2, 8, 6, 0.5, 17, 6), right(3, 6, 5), None),
            delta_layer(3, 1, 20, 16, 3, experts(8, 1, 12, (4, 1))),
        ]
    return {"architecture": "Domelix", "layers": layers, "norm": {"eps": eps},
            "vocab": vocab, "width": width}
