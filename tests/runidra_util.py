"""Helpers of the Runidra tests: small irregular configurations. Checkpoint
writing, engines and the step driver are the ones of vurizen_util."""

from vurizen_util import (  # noqa: F401
    close_in_bf16, describe, make_engine, rel_err, row_errs, run_schedule,
    same_as_whole, tokens, write_checkpoint,
)


def dense(ff=44):
    return {"kind": "dense", "ff": ff}


def experts(n=5, top=2, ff=24, shared=36):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def mlstm_layer(heads=3, dim=12, vdim=20, cap=6.0, mlp="default"):
    return {"type": "mlstm",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap},
            "mlp": dense() if mlp == "default" else mlp}


def latent_layer(heads=3, dim=20, rot_dim=12, vdim=28, rank=24, q_rank=36, window=9,
                 scale=0.25, base=500.0, mlp="default"):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
                      "kv_rank": rank, "q_rank": q_rank, "mask": {"size": window},
                      "scale": scale, "rot": {"dims": rot_dim, "base": base}},
            "mlp": dense() if mlp == "default" else mlp}


def small_config(layers=None, width=40, vocab=83, eps=1e-5, streams=3, loop=(1, 4, 2),
                 logit_scale=1.4, softcap=6.0) -> dict:
    """Sizes away from powers of two and from each other; three streams; a
    loop over the middle of the stack (both mixers and a layer without
    feed-forward inside it); two windows; dense feed-forwards, experts with
    and without a shared one."""
    if layers is None:
        layers = [
            mlstm_layer(),
            latent_layer(mlp=experts()),
            mlstm_layer(2, 20, 8, 15.0, None),
            latent_layer(4, 8, 4, 12, 40, 20, 33, 0.4, 10000.0, dense(28)),
            mlstm_layer(1, 16, 16, 2.0, experts(3, 1, 16, 0)),
        ]
    cfg = {"architecture": "Runidra", "layers": layers, "norm": {"eps": eps},
           "vocab": vocab, "width": width, "streams": streams,
           "logit_scale": logit_scale, "logit_softcap": softcap}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg
