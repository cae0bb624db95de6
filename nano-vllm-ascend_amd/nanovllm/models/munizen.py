"""Munizen: a pre-norm decoder with several residual streams per token (hyper-connections) whose configuration lists its
layers and may run a stretch of them several times with the same weights (every pass with caches and states of its own):

  streams          X_1 .. X_s, all the embedding row at the start; a sublayer f: y = f(norm(sum_i in_i X_i)),
                   X_j <- sum_i mix[i, j] X_i + out_j y; the model's output is the sum of the streams
  norm             RMS norm over `groups` equal parts of the channels, plain weight
  token shift      what a mixer reads is h + (h of the previous token - h) * shift
  attention        differential attention: two rotated softmax maps per head over the same values, within chunks of the sequence
  general_delta    generalised delta rule, a matrix state per head with a decay and a removal rate per key channel
  feed-forward     W_down (silu(W_gate h) * (W_up h)), or none

The mechanisms are the classes of layers/seqmix.py; this file reads the configuration, wires the layers, names the
checkpoint's tensors and says what cache and state a sequence needs:

  config.json   {"architecture": "Munizen", "vocab", "width", "streams", "norm": {"eps", "groups"},
                "loop": {"start", "stop", "times"} | absent,
                "layers": [{"type": "attention" | "general_delta", "mixer": {...}, "mlp": {"kind": "dense", "ff"} | null}]}
  checkpoint    embed, head, final.norm, l<i>.norm1 / norm2 / shift, l<i>.hc1 / hc2.in / out / mix, l<i>.mix.<name>(.b),
                l<i>.mlp.gate / up / down; the rank of the decay's low-rank projection is that of l<i>.mix.w1
  per sequence  pages: K rows of both maps and V rows of every attention, once per pass; a state slot: the last row of every
                layer's shifted input and the delta rule's fp32 matrix states, once per pass
"""
from __future__ import annotations

import json
import os

import torch
from torch import nn

from nanovllm import ops
from nanovllm.layers.seqmix import (DifferentialAttention, GatedDenseMLP, GeneralDeltaMixer, StreamCoefficients, StreamResidual,
                                    TokenShift, _vector)
from nanovllm.models.gazutar import safetensors_shapes
from nanovllm.models.looped import LoopedLayers


class MunizenConfig(LoopedLayers):
    """config.json of this design with the attribute names the engine reads from a configuration object."""
    architectures = ["Munizen"]
    model_type = "munizen"
    max_position_embeddings = None
    eos_token_id = None
    native = True                    # not a transformers configuration

    def __init__(self, raw: dict, tensor_shapes: dict | None = None, dtype: str = "bfloat16"):
        self.raw = raw
        self.vocab_size, self.hidden_size = int(raw["vocab"]), int(raw["width"])
        self.layers = raw["layers"]
        self.num_hidden_layers = len(self.layers)
        self.norm_eps, self.norm_groups = float(raw["norm"]["eps"]), int(raw["norm"].get("groups") or 1)
        assert self.hidden_size % self.norm_groups == 0
        self.streams = int(raw.get("streams") or 1)
        self.read_loop(raw.get("loop"), len(self.layers))
        self.tensor_shapes = tensor_shapes or {}
        self.torch_dtype = dtype

    @classmethod
    def from_dir(cls, path: str, dtype: str = "bfloat16") -> "MunizenConfig":
        with open(os.path.join(path, "config.json")) as f:
            raw = json.load(f)
        ckpt = os.path.join(path, "model.safetensors")
        return cls(raw, safetensors_shapes(ckpt) if os.path.exists(ckpt) else None, dtype)

    def rank_of(self, layer: int) -> int:
        shape = self.tensor_shapes.get(f"l{layer}.mix.w1")
        if shape is not None:
            return int(shape[0])
        return int(self.layers[layer]["mixer"].get("rank", max(8, self.hidden_size // 16)))  # synthetic weights only


class MunizenLayer(nn.Module):
    def __init__(self, cfg: MunizenConfig, index: int):
        super().__init__()
        spec, W, eps = cfg.layers[index], cfg.hidden_size, cfg.norm_eps
        m = spec["mixer"]
        self.kind, self.lanes = spec["type"], cfg.lanes_of(index)
        if self.kind == "attention":
            rot = m.get("rot") or {"dims": 0, "base": 1.0}
            self.mix = DifferentialAttention(W, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                                             int(m["mask"]["size"]) if m.get("mask") else 0, float(m["scale"]), float(m["diff"]),
                                             eps, int(rot["dims"]), float(rot["base"]))
        elif self.kind == "general_delta":
            self.mix = GeneralDeltaMixer(W, int(m["heads"]), int(m["dim"]), cfg.rank_of(index), eps)
        else:
            raise NotImplementedError(f"layer {index}: mixer type {self.kind!r}")
        self.norm1, self.shift, self.hc1 = _vector(W, 1.0), TokenShift(W), StreamCoefficients(cfg.streams)
        ml = spec.get("mlp")
        self.mlp = self.norm2 = self.hc2 = None
        if ml is not None:
            if ml.get("kind", "dense") != "dense":
                raise NotImplementedError(f"layer {index}: feed-forward kind {ml.get('kind')!r}")
            self.mlp = GatedDenseMLP(W, int(ml["ff"]), act="silu", bias=False)
            self.norm2, self.hc2 = _vector(W, 1.0), StreamCoefficients(cfg.streams)


class MunizenForCausalLM(nn.Module):
    hybrid_state = True   # sequences own state slots beside their pages: ModelRunner takes the row-step path
    fp32_residual = True

    def __init__(self, config: MunizenConfig):
        super().__init__()
        self.config = config
        W, V = config.hidden_size, config.vocab_size
        self.embed = nn.Parameter(torch.empty(V, W), requires_grad=False)
        self.head = nn.Parameter(torch.empty(V, W), requires_grad=False)
        self.layers = nn.ModuleList([MunizenLayer(config, i) for i in range(len(config.layers))])
        self.final_norm = _vector(W, 1.0)
        self.trace_layers: list | None = None  # bring-up hook: receives the sum of the streams after every layer run

    # ---- checkpoint names -> parameters (utils/loader.py) ------------------------------------------------------
    def map_checkpoint_name(self, name: str):
        """-> parameter path, (parameter path, shard) for tensors that land inside a merged parameter, or None for a tensor
        this configuration has no use for."""
        if name in ("embed", "head"):
            return name
        if name == "final.norm":
            return "final_norm"
        layer, rest = name.split(".", 1)
        i = int(layer[1:])
        pre, L = f"layers.{i}.", self.layers[i]
        if rest == "norm1":
            return pre + "norm1"
        if rest == "norm2":
            return pre + "norm2" if L.mlp is not None else None
        if rest == "shift":
            return pre + "shift.weight"
        part, leaf = rest.split(".", 1)
        if part in ("hc1", "hc2"):
            return pre + part + "." + {"in": "read", "out": "write", "mix": "mix"}[leaf] if getattr(L, part) is not None else None
        if part == "mlp":
            return pre + "mlp." + {"gate": "gate", "up": "up", "down": "down"}[leaf] if L.mlp is not None else None
        pre += "mix."
        if L.kind == "attention":
            if leaf in ("lq1", "lk1", "lq2", "lk2"):
                return pre + "lam", ("lq1", "lk1", "lq2", "lk2").index(leaf)
            if leaf in ("o", "o.b"):
                return pre + {"o": "o", "o.b": "o_b"}[leaf]
            return (pre + "qkvg.bias", leaf[:-2]) if leaf.endswith(".b") else (pre + "qkvg.weight", leaf)
        if leaf in ("w2", "w0", "norm", "o"):
            return pre + leaf
        return (pre + "proj.bias", leaf[:-2]) if leaf.endswith(".b") else (pre + "proj.weight", leaf)

    def synthetic_state(self, seed: int = 0):
        """Random tensors under the checkpoint's names (no-checkpoint mode: benchmarks)."""
        g = torch.Generator().manual_seed(seed)
        cfg, W, s = self.config, self.config.hidden_size, self.config.streams

        def mat(*shape, std=None):
            return torch.randn(*shape, generator=g) * (std if std is not None else shape[-1] ** -0.5)

        yield "embed", mat(cfg.vocab_size, W, std=W ** -0.5)
        yield "head", mat(cfg.vocab_size, W)
        yield "final.norm", 1 + mat(W, std=0.05)
        for i, layer in enumerate(self.layers):
            p, x = f"l{i}.", layer.mix
            yield p + "norm1", 1 + mat(W, std=0.05)
            yield p + "shift", torch.rand(W, generator=g)
            for q in ("hc1", "hc2") if layer.mlp is not None else ("hc1",):
                yield p + q + ".in", (1 + mat(s, std=0.2)) / s
                yield p + q + ".out", 1 + mat(s, std=0.2)
                yield p + q + ".mix", torch.eye(s) + mat(s, s, std=0.05)
            merged = x.qkvg if layer.kind == "attention" else x.proj
            for n, (_, rows) in merged.offsets.items():
                yield p + "mix." + n, mat(rows, W)
            if layer.kind == "attention":
                for n in ("q", "k", "v"):
                    yield p + f"mix.{n}.b", mat(merged.offsets[n][1], std=0.1)
                for n in ("lq1", "lk1", "lq2", "lk2"):
                    yield p + "mix." + n, mat(x.D, std=0.1)
                yield p + "mix.o", mat(W, x.H * x.Dv)
                yield p + "mix.o.b", mat(W, std=0.1)
            else:
                n = x.H * x.D
                yield p + "mix.a.b", mat(n, std=0.5)
                yield p + "mix.w2", mat(n, x.w2.shape[1])
                yield p + "mix.w0", mat(n, std=0.5)
                yield p + "mix.norm", 1 + mat(n, std=0.05)
                yield p + "mix.o", mat(W, n)
            if layer.mlp is not None:
                ff = layer.mlp.gate.shape[0]
                yield p + "norm2", 1 + mat(W, std=0.05)
                yield p + "mlp.gate", mat(ff, W)
                yield p + "mlp.up", mat(ff, W)
                yield p + "mlp.down", mat(W, ff)

    # ---- cache and state ------------------------------------------------------------------------------------------
    def cache_bytes_per_block(self, block_size: int, itemsize: int) -> int:
        return block_size * itemsize * sum(l.lanes * (2 * l.mix.G * l.mix.D + l.mix.G * l.mix.Dv)
                                           for l in self.layers if l.kind == "attention")

    def state_bytes_per_slot(self) -> int:
        return 4 * sum(l.lanes * (l.shift.state_shape(1)[1] + (l.mix.state_shape(1)[1] if l.kind == "general_delta" else 0))
                       for l in self.layers)

    def bind_cache(self, num_blocks: int, block_size: int, n_slots: int, dtype: torch.dtype, device) -> None:
        """Pages for the K / V rows (serving dtype), state slots for the shifted inputs and the delta rule's matrix states
        (fp32), one set per pass of a looped layer.  Nothing has to be cleared when a page or a slot changes hands: a
        sequence's first row starts every state from zero and no kernel reads a cache row its own sequence has not written."""
        def lanes(layer, shape, dt):
            return [torch.zeros(shape, dtype=dt, device=device) for _ in range(layer.lanes)]

        for l in self.layers:
            l.shift.state = lanes(l, l.shift.state_shape(n_slots), torch.float32)
            if l.kind == "attention":
                ks, vs = l.mix.cache_shapes(num_blocks, block_size)
                l.mix.k_cache, l.mix.v_cache = lanes(l, ks, dtype), lanes(l, vs, dtype)
            else:
                l.mix.state = lanes(l, l.mix.state_shape(n_slots), torch.float32)

    # ---- one step over the rows the context describes ----------------------------------------------------------------
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor | None = None) -> torch.Tensor:
        cfg = self.config
        x = StreamResidual(ops.embedding_f32(input_ids, self.embed), cfg.streams, cfg.norm_groups, cfg.norm_eps)
        for i, lane, _ in cfg.layer_runs:
            layer = self.layers[i]
            x.leave(layer.mix(x.read(layer.hc1, layer.norm1, layer.shift, lane), lane), layer.hc1)
            if layer.mlp is not None:
                x.leave(layer.mlp(x.read(layer.hc2, layer.norm2)), layer.hc2)
            if self.trace_layers is not None:
                self.trace_layers.append(x.total(store=True))
        return x.total()

    def compute_logits(self, hidden: torch.Tensor, rows: torch.Tensor | None = None) -> torch.Tensor:
        """fp32 logits of the given rows (default: all)."""
        if rows is not None:
            hidden = hidden.index_select(0, rows)
        h = ops.stream_mix(hidden.unsqueeze(1), None, None, None, None, None, self.final_norm, self.config.norm_groups,
                           self.config.norm_eps)
        return ops.gemm_any(h, self.head)
