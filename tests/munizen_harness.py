"""Shared pieces of the Munizen tests: small configurations of the design (sizes of the tests' own making: widths that are no
multiple of 32 or of 4, head sizes on and off the matrix cores' shapes, rotated parts shorter than a head, chunks of one
position and longer than a sequence, one to eight streams, one norm group and many, loops over a prefix, the middle or all of
the layers), random checkpoints written as a model directory.  The replay helper that feeds sequences to the engine's row-step
path in a given cut is the one of gazutar_harness (it is not specific to a model)."""
import json
import os
import tempfile

import torch

from gazutar_harness import F32_BAR, Replay, rel_err, row_errs, tokens_of  # noqa: F401 (re-exported)

BF16_ROW = 6e-2


def assert_close(got: torch.Tensor, want: torch.Tensor, dtype: str, what="") -> None:
    """Every row (rms of the difference / rms of the expected row) within F32_BAR in the float32 mode; in the bfloat16 mode
    (activations rounded on their way into the matrix cores) within BF16_ROW and the median row within a third of it."""
    e = row_errs(got, want)
    if dtype == "float32":
        assert float(e.max()) <= F32_BAR, (what, float(e.max()), int(e.argmax()))
    else:
        assert float(e.max()) <= BF16_ROW and float(e.median()) <= BF16_ROW / 3, (what, float(e.max()), int(e.argmax()), float(e.median()))


def attention(heads=6, kv_heads=3, dim=24, vdim=20, chunk=17, scale=0.3, diff=0.45, dims=16, base=10000.0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff,
         "rot": {"base": base, "dims": dims}}
    if chunk:
        m["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": m}


def delta(heads=3, dim=20):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def with_mlp(layer, mlp):
    return dict(layer, mlp=mlp)


def config(layers, width=84, vocab=97, streams=3, groups=2, loop=(0, 0, 0), eps=1e-5):
    cfg = {"architecture": "Munizen", "vocab": vocab, "width": width, "streams": streams,
           "norm": {"eps": eps, "groups": groups}, "layers": layers}
    if loop[2]:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


# the delta rule first and again inside the loop, a layer without feed-forward of either kind, grouped and ungrouped heads,
# a loop over the middle layers (three passes), head sizes on and off the matrix cores' shapes, chunks short and long
MIXED = config([
    with_mlp(delta(), dense()),
    with_mlp(attention(), dense(ff=24)),
    with_mlp(delta(heads=2, dim=33), None),
    with_mlp(attention(heads=4, kv_heads=4, dim=32, vdim=16, chunk=9, dims=32), None),
    with_mlp(attention(heads=2, kv_heads=1, dim=10, vdim=6, chunk=0, dims=4), dense()),
], loop=(1, 4, 3))
RANKS = {0: 6, 2: 5}


def write_model_dir(cfg: dict, weights: dict) -> str:
    from safetensors.torch import save_file

    d = tempfile.mkdtemp(prefix="munizen_")
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, os.path.join(d, "model.safetensors"))
    return d
