"""Shared pieces of the Sikevik tests: small configurations of the design (sizes of the tests' own making: widths that are
odd or no multiple of 32, head sizes on and off the matrix cores' shapes, grouped and ungrouped key/value heads, windows
shorter and longer than the kept first tokens, none kept at all, dense and sparse feed-forwards and none, routers that take
one expert or all, shared experts of other sizes than the experts and none, loops over a prefix, the middle or all of the
layers, one pass and three, no loop at all), random checkpoints written as a model directory.  The replay helper that feeds
sequences to the engine's row-step path in a given cut is the one of gazutar_harness (it is not specific to a model)."""
import json
import os
import tempfile

import torch

from gazutar_harness import F32_BAR, Replay, rel_err, row_errs, tokens_of  # noqa: F401 (re-exported)

BF16_MEDIAN, BF16_ROW = 2e-2, 6e-2


def assert_close(got: torch.Tensor, want: torch.Tensor, dtype: str, what="") -> None:
    """float32 mode: every row within F32_BAR (row-wise rms difference / rms of the expected row).  bfloat16 mode: the
    rounding of activations on their way into the matrix cores gives these stacks about 1e-2 per row, and a router's
    near-tie that falls the other way replaces an expert for that token: the median row within BF16_MEDIAN, at most a
    quarter of the rows over BF16_ROW.  Position-exact faults are the float32 runs' business."""
    e = row_errs(got, want)
    if dtype == "float32":
        assert float(e.max()) <= F32_BAR, (what, float(e.max()), int(e.argmax()))
    else:
        off = int((e > BF16_ROW).sum())
        assert float(e.median()) <= BF16_MEDIAN and off <= max(1, e.numel() // 4), (what, float(e.median()), off, e.numel())


def attention(heads=6, kv_heads=2, dim=24, vdim=20, window=17, kept=3, scale=0.25):
    mask = None if window is None else {"size": window, "keep_first": kept}
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": mask, "scale": scale}}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(ff=40, experts=7, top=3, scale=1.75, shared=24):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def with_mlp(layer, mlp):
    return dict(layer, mlp=mlp)


def config(layers, width=80, vocab=97, loop=(0, 0, 0), eps=1e-5, scale=3.0):
    cfg = {"architecture": "Sikevik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "layers": layers}
    if loop[2]:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


# sparse first, a layer without feed-forward, dense ones, unequal layers, a loop over the middle layers (three passes)
MIXED = config([
    with_mlp(attention(), moe()),
    with_mlp(attention(heads=4, kv_heads=4, dim=32, vdim=16, window=9, kept=1), moe(ff=16, experts=12, top=1, shared=0)),
    with_mlp(attention(heads=2, kv_heads=1, dim=64, vdim=48, window=13, kept=20, scale=0.15), None),
    with_mlp(attention(heads=5, kv_heads=1, dim=10, vdim=6, window=40, kept=0), dense()),
    with_mlp(attention(heads=4, kv_heads=2, dim=32, vdim=32, window=200, kept=5), moe(ff=24, experts=5, top=5, scale=1.0, shared=72)),
], loop=(1, 4, 3))


def write_model_dir(cfg: dict, weights: dict) -> str:
    from safetensors.torch import save_file

    d = tempfile.mkdtemp(prefix="sikevik_")
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, os.path.join(d, "model.safetensors"))
    return d
