"""Sikevik: a sandwich-normed decoder (x <- x + n(mixer(n(x; w_1)); w_1b), x <- x + n(ff(n(x; w_2)); w_2b), n an RMS norm with
a plain weight, fp32 residual) whose configuration lists its layers and may run a stretch of them several times with the
same weights:

  embedding    scaled table rows plus sinusoids of the positions - the only place where positions enter
  order        layers [0, start), then `times` passes over [start, stop), then [stop, n).  Every pass begins with a
               projection of the stream and the embedding output side by side, x <- W [x | e], and has K/V pages of its own
               ("lane")
  attention    normed query and key heads (one weight for all heads), no rotation; a sliding window beside the sequence's
               first tokens, which stay visible; one added to the softmax's denominator
  feed-forward dense (tanh-form GELU) or top-k experts (squared ReLU) with renormalised, scaled softmax weights and a
               shared expert; or none

The mechanisms are the classes of layers/seqmix.py; this file reads the configuration, wires the layers, names the
checkpoint's tensors and says what cache a sequence needs:

  config.json   {"architecture": "Sikevik", "vocab", "width", "norm": {"eps"}, "embedding": {"scale"},
                "loop": {"start", "stop", "times"} | absent, "layers": [{"type": "attention", "mixer": {"heads", "kv_heads",
                "dim", "vdim", "scale", "mask": {"size", "keep_first"}}, "mlp": {"kind": "dense", "ff"} | {"kind": "moe",
                "expert": {"ff"}, "router": {"experts", "top", "scale"}, "shared": {"ff"}} | null}]}
  checkpoint    embed (also the output projection), final.norm, loop.in, l<i>.norm1 / norm1b / norm2 / norm2b,
                l<i>.mix.q / k / v / o / q.norm / k.norm, l<i>.mlp.up / down, l<i>.mlp.router / e<k>.up / down / shared.up / down
  per sequence  pages: K / V rows of every attention, once per pass; no recurrent state
"""
from __future__ import annotations

import json
import os

import torch
from torch import nn

from nanovllm import ops
from nanovllm.layers.seqmix import (CAUSAL, DenseMLP, OutputNorm, PassInput, RotaryWindowAttention, SharedSparseMLP,
                                    SinkAttentionMixer, SinusoidEmbedding, _vector)
from nanovllm.models.looped import LoopedLayers


class SikevikConfig(LoopedLayers):
    """config.json of this design with the attribute names the engine reads from a configuration object."""
    architectures = ["Sikevik"]
    model_type = "sikevik"
    max_position_embeddings = None
    eos_token_id = None
    native = True                    # not a transformers configuration

    def __init__(self, raw: dict, dtype: str = "bfloat16"):
        self.raw = raw
        self.vocab_size, self.hidden_size = int(raw["vocab"]), int(raw["width"])
        self.layers = raw["layers"]
        self.num_hidden_layers = len(self.layers)
        self.norm_eps = float(raw["norm"]["eps"])
        self.embedding_scale = float((raw.get("embedding") or {}).get("scale", 1.0))
        self.read_loop(raw.get("loop"), len(self.layers))
        self.torch_dtype = dtype

    @classmethod
    def from_dir(cls, path: str, dtype: str = "bfloat16") -> "SikevikConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls(json.load(f), dtype)


class SikevikLayer(nn.Module):
    def __init__(self, cfg: SikevikConfig, index: int):
        super().__init__()
        spec, W, eps = cfg.layers[index], cfg.hidden_size, cfg.norm_eps
        if spec["type"] != "attention":
            raise NotImplementedError(f"layer {index}: mixer type {spec['type']!r}")
        m, self.lanes = spec["mixer"], cfg.lanes_of(index)
        mask = m.get("mask") or {}
        attn = RotaryWindowAttention(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                                     int(mask["size"]) if mask else CAUSAL, float(m["scale"]), eps, 0, 1.0, unit_norm=True,
                                     norm_weights=True, sink=0.0, keep_first=int(mask.get("keep_first") or 0))
        self.mix = SinkAttentionMixer(W, attn)
        self.norm1, self.out1 = _vector(W, 1.0), OutputNorm(W, eps)
        ml = spec.get("mlp")
        self.mlp = self.norm2 = self.out2 = None
        if ml is None:
            return
        if ml["kind"] == "dense":
            self.mlp = DenseMLP(W, int(ml["ff"]))
        elif ml["kind"] == "moe":
            r, shared = ml["router"], ml.get("shared")
            self.mlp = SharedSparseMLP(W, int(ml["expert"]["ff"]), int(r["experts"]), int(r["top"]),
                                       int(shared["ff"]) if shared else 0, act="relu2", shared_gate=False,
                                       weight_scale=float(r.get("scale", 1.0)))
        else:
            raise NotImplementedError(f"layer {index}: feed-forward kind {ml['kind']!r}")
        self.norm2, self.out2 = _vector(W, 1.0), OutputNorm(W, eps)

    def add_feed_forward(self, x: torch.Tensor, h: torch.Tensor, next_norm: torch.Tensor | None):
        if isinstance(self.mlp, SharedSparseMLP):
            return self.out2.add_experts_to(x, self.mlp, h, next_norm)
        return self.out2.add_to(x, self.mlp(h), next_norm)


class SikevikForCausalLM(nn.Module):
    hybrid_state = True   # ModelRunner takes the row-step path (the state slots of this design are empty)
    fp32_residual = True

    def __init__(self, config: SikevikConfig):
        super().__init__()
        self.config = config
        W = config.hidden_size
        self.embed = SinusoidEmbedding(config.vocab_size, W, config.embedding_scale)   # its table is the output projection too
        self.layers = nn.ModuleList([SikevikLayer(config, i) for i in range(len(config.layers))])
        self.final_norm = _vector(W, 1.0)
        self.pass_input = PassInput(W) if config.loop_times else None
        self.trace_layers: list | None = None  # bring-up hook: receives a copy of the residual stream after every layer run

    # ---- checkpoint names -> parameters (utils/loader.py) ------------------------------------------------------
    def map_checkpoint_name(self, name: str):
        """-> parameter path, (parameter path, shard) for tensors that land inside a merged / stacked parameter, or None
        for a tensor this configuration has no use for."""
        if name == "embed":
            return "embed.weight"
        if name == "final.norm":
            return "final_norm"
        if name == "loop.in":
            return "pass_input.weight" if self.pass_input is not None else None
        layer, rest = name.split(".", 1)
        i = int(layer[1:])
        pre, L = f"layers.{i}.", self.layers[i]
        norms = {"norm1": "norm1", "norm1b": "out1.weight", "norm2": "norm2", "norm2b": "out2.weight"}
        if rest in norms:
            return pre + norms[rest] if L.mlp is not None or rest.startswith("norm1") else None
        part, leaf = rest.split(".", 1)
        if part == "mix":
            if leaf in ("q", "k", "v"):
                return pre + "mix.qkv.weight", leaf
            return pre + "mix." + {"q.norm": "attn.q_norm", "k.norm": "attn.k_norm", "o": "o"}[leaf]
        if isinstance(L.mlp, DenseMLP):
            return pre + "mlp." + leaf           # up, down
        if leaf == "router":
            return pre + "mlp.router.weight", leaf
        expert, proj = leaf.split(".")
        return pre + "mlp.shared_" + proj if expert == "shared" else (pre + "mlp." + proj, int(expert[1:]))

    def synthetic_state(self, seed: int = 0):
        """Random tensors under the checkpoint's names (no-checkpoint mode: benchmarks)."""
        g = torch.Generator().manual_seed(seed)
        cfg, W = self.config, self.config.hidden_size

        def mat(*shape, std=None):
            return torch.randn(*shape, generator=g) * (std if std is not None else shape[-1] ** -0.5)

        def norm(n):
            return 1 + mat(n, std=0.05)

        yield "embed", mat(cfg.vocab_size, W, std=W ** -0.5)
        yield "final.norm", norm(W)
        if self.pass_input is not None:
            yield "loop.in", mat(W, 2 * W)
        for i, layer in enumerate(self.layers):
            a, p = layer.mix.attn, f"l{i}."
            yield p + "norm1", norm(W)
            yield p + "norm1b", norm(W)
            for n, rows in a.parts.items():
                yield p + "mix." + n, mat(rows, W)
            yield p + "mix.q.norm", norm(a.D)
            yield p + "mix.k.norm", norm(a.D)
            yield p + "mix.o", mat(W, a.out_features)
            ml = layer.mlp
            if ml is None:
                continue
            yield p + "norm2", norm(W)
            yield p + "norm2b", norm(W)
            if isinstance(ml, DenseMLP):
                yield p + "mlp.up", mat(*ml.up.shape)
                yield p + "mlp.down", mat(*ml.down.shape)
                continue
            yield p + "mlp.router", mat(ml.E, W)
            for e in range(ml.E):
                yield p + f"mlp.e{e}.up", mat(*ml.up.shape[1:])
                yield p + f"mlp.e{e}.down", mat(*ml.down.shape[1:])
            if ml.shared:
                yield p + "mlp.shared.up", mat(*ml.shared_up.shape)
                yield p + "mlp.shared.down", mat(*ml.shared_down.shape)

    # ---- cache and state ------------------------------------------------------------------------------------------
    def cache_bytes_per_block(self, block_size: int, itemsize: int) -> int:
        return block_size * itemsize * sum(l.lanes * l.mix.attn.G * (l.mix.attn.D + l.mix.attn.Dv) for l in self.layers)

    def state_bytes_per_slot(self) -> int:
        return 0

    def bind_cache(self, num_blocks: int, block_size: int, n_slots: int, dtype: torch.dtype, device) -> None:
        """Pages for the K / V rows (serving dtype), one set per pass of a looped layer.  Nothing has to be cleared when a
        page changes hands: no kernel reads a cache row its own sequence has not written."""
        for l in self.layers:
            ks, vs = l.mix.attn.cache_shapes(num_blocks, block_size)
            l.mix.attn.k_cache = [torch.zeros(ks, dtype=dtype, device=device) for _ in range(l.lanes)]
            l.mix.attn.v_cache = [torch.zeros(vs, dtype=dtype, device=device) for _ in range(l.lanes)]

    # ---- one step over the rows the context describes ----------------------------------------------------------------
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor | None = None) -> torch.Tensor:
        eps, runs = self.config.norm_eps, self.config.layer_runs
        x = self.embed(input_ids)
        fixed = self.pass_input.fixed_part(x) if any(begins is not None for _, _, begins in runs) else None
        h = None   # the normed stream, when the launch that last touched the stream made it already
        for n, (i, lane, begins) in enumerate(runs):
            layer = self.layers[i]
            if begins is not None:
                x, h = self.pass_input.begin(x, fixed, layer.norm1, eps)
            elif h is None:
                h = ops.add_rmsnorm_f32(x, None, 0.0, layer.norm1, eps)
            # what the stream is normed with after this layer: nothing at the end (the output's norm is taken of the wanted
            # rows only) and where a pass begins
            after = self.layers[runs[n + 1][0]].norm1 if n + 1 < len(runs) and runs[n + 1][2] is None else None
            h = layer.out1.add_to(x, layer.mix(h, lane), layer.norm2 if layer.mlp is not None else after)
            if layer.mlp is not None:
                h = layer.add_feed_forward(x, h, after)
            if self.trace_layers is not None:
                self.trace_layers.append(x.clone())
        return x

    def compute_logits(self, hidden: torch.Tensor, rows: torch.Tensor | None = None) -> torch.Tensor:
        """fp32 logits of the given rows (default: all): the embedding table, without its scale, is the projection."""
        if rows is not None:
            hidden = hidden.index_select(0, rows)
        h = ops.add_rmsnorm_f32(hidden, None, 0.0, self.final_norm, self.config.norm_eps)
        return ops.gemm_any(h, self.embed.weight)
