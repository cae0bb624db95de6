"""Host-side pieces of the Sikevik integration (no GPU): the configuration reader and the order of layer runs, the
checkpoint name map through the framework's loader, what a sequence needs in pages, the frequency table of the positions,
the bench models' weight bytes, and the plain statement's own consistency."""
import os

import pytest
import torch

from oracle import sikevik as S
from sikevik_harness import MIXED, attention, config, dense, moe, with_mlp, write_model_dir


@pytest.fixture(scope="module")
def model_dir():
    return write_model_dir(MIXED, S.random_model(MIXED, seed=1))


def test_config_is_read_from_the_directory(model_dir):
    from nanovllm.config import Config

    c = Config(model_dir, dtype="float32", max_model_len=128, max_num_batched_tokens=128)
    hf = c.hf_config
    assert c.hybrid_state and hf.architectures == ["Sikevik"]
    assert (hf.vocab_size, hf.hidden_size, hf.num_hidden_layers) == (MIXED["vocab"], MIXED["width"], 5)
    assert (hf.loop_start, hf.loop_stop, hf.loop_times) == (1, 4, 3)
    assert hf.norm_eps == 1e-5 and hf.embedding_scale == 3.0
    assert c.eos == -1 and c.max_model_len == 128


def test_order_of_layer_runs():
    """The same order as the plain statement's for a loop over a prefix, the middle, the tail, everything, nothing, one pass
    and no loop at all."""
    from nanovllm.models.sikevik import SikevikConfig

    layers = [with_mlp(attention(), None)] * 4
    for loop in ((0, 2, 2), (1, 3, 3), (2, 4, 2), (0, 4, 2), (0, 4, 1), (2, 2, 5), (0, 0, 0)):
        cfg = config(layers, loop=loop)
        c = SikevikConfig(cfg)
        assert [(i, t) for i, _, t in c.layer_runs] == S.layer_runs(cfg), loop
        for i, lane, t in c.layer_runs:
            assert 0 <= lane < c.lanes_of(i) and (t is None or t == lane)


def test_every_tensor_lands_in_a_parameter(model_dir):
    """Load through the framework's loader on the CPU: every parameter is written, merged, stacked and halved ones in the
    right ranges, and nothing of the checkpoint is left over."""
    from nanovllm.models.sikevik import SikevikConfig, SikevikForCausalLM
    from nanovllm.utils.loader import load_model
    from safetensors.torch import load_file

    model = SikevikForCausalLM(SikevikConfig.from_dir(model_dir))
    for p in model.parameters():
        p.data.fill_(float("nan"))
    load_model(model, model_dir)
    w = {k: v.float() for k, v in load_file(os.path.join(model_dir, "model.safetensors")).items()}
    for name, p in model.named_parameters():
        assert not torch.isnan(p).any(), name
    assert sum(p.numel() for p in model.parameters()) == sum(v.numel() for v in w.values())
    assert set(w) == set(S.tensor_shapes(MIXED))
    W = MIXED["width"]
    assert torch.equal(model.embed.weight, w["embed"]) and torch.equal(model.final_norm, w["final.norm"])
    assert torch.equal(model.pass_input.weight[0], w["loop.in"][:, :W]) and torch.equal(model.pass_input.weight[1], w["loop.in"][:, W:])
    for i, L in enumerate(model.layers):
        a, m = L.mix.attn, MIXED["layers"][i]["mixer"]
        for n in ("q", "k", "v"):
            off, rows = L.mix.qkv.offsets[n]
            assert torch.equal(L.mix.qkv.weight[off:off + rows], w[f"l{i}.mix.{n}"])
        assert torch.equal(a.q_norm, w[f"l{i}.mix.q.norm"]) and torch.equal(a.k_norm, w[f"l{i}.mix.k.norm"])
        assert torch.equal(L.mix.o, w[f"l{i}.mix.o"])
        assert torch.equal(L.norm1, w[f"l{i}.norm1"]) and torch.equal(L.out1.weight, w[f"l{i}.norm1b"])
        assert (a.H, a.G, a.D, a.Dv) == tuple(m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        assert (a.window, a.keep_first, a.scale) == (m["mask"]["size"], m["mask"]["keep_first"], m["scale"])
        assert a.rot_dims == 0 and a.unit_norm and torch.equal(a.sink, torch.zeros(a.H))
        if L.mlp is not None:
            assert torch.equal(L.norm2, w[f"l{i}.norm2"]) and torch.equal(L.out2.weight, w[f"l{i}.norm2b"])
    L0, L1, L3, L4 = (model.layers[i].mlp for i in (0, 1, 3, 4))
    assert torch.equal(L0.router.weight, w["l0.mlp.router"]) and torch.equal(L0.up[4], w["l0.mlp.e4.up"])
    assert torch.equal(L0.down[6], w["l0.mlp.e6.down"])
    assert torch.equal(L0.shared_up, w["l0.mlp.shared.up"]) and torch.equal(L0.shared_down, w["l0.mlp.shared.down"])
    assert (L0.E, L0.top_k, L0.weight_scale, L0.shared, L0.gated) == (7, 3, 1.75, True, False)
    assert (L1.E, L1.top_k, L1.shared) == (12, 1, False) and (L4.top_k, L4.shared_up.shape[0]) == (5, 72)
    assert model.layers[2].mlp is None and model.layers[2].norm2 is None
    assert torch.equal(L3.up, w["l3.mlp.up"]) and torch.equal(L3.down, w["l3.mlp.down"])


def test_pages_of_a_sequence(model_dir):
    from nanovllm.models.sikevik import SikevikConfig, SikevikForCausalLM

    model = SikevikForCausalLM(SikevikConfig.from_dir(model_dir))
    # K and V rows of every attention, three times for the layers inside the loop
    per_token = 2 * (24 + 20) + 3 * (4 * (32 + 16) + (64 + 48) + (10 + 6)) + 2 * (32 + 32)
    assert model.cache_bytes_per_block(16, 2) == 16 * per_token * 2 and model.state_bytes_per_slot() == 0
    assert model.layers[1].mix.attn.cache_shapes(7, 16) == ((7, 4, 16, 32), (7, 4, 16, 16))
    model.bind_cache(3, 16, 2, torch.float32, "cpu")
    assert [len(l.mix.attn.k_cache) for l in model.layers] == [1, 3, 3, 3, 1]


def test_synthetic_checkpoint_names_match_the_design(model_dir):
    from nanovllm.models.sikevik import SikevikConfig, SikevikForCausalLM

    model = SikevikForCausalLM(SikevikConfig.from_dir(model_dir))
    got = {name: tuple(t.shape) for name, t in model.synthetic_state(0)}
    assert got == {k: tuple(v) for k, v in S.tensor_shapes(MIXED).items()}


def test_absent_parts_are_absent():
    """No loop, no mask, no shared expert, no scales in the configuration."""
    from nanovllm.models.sikevik import SikevikConfig, SikevikForCausalLM

    m = moe(shared=0)
    del m["router"]["scale"]
    cfg = config([with_mlp(attention(window=None), m)])
    del cfg["embedding"]
    model = SikevikForCausalLM(SikevikConfig(cfg))
    a, ff = model.layers[0].mix.attn, model.layers[0].mlp
    assert model.pass_input is None and model.embed.scale == 1.0
    assert a.window > 2 ** 30 and a.keep_first == 0 and ff.weight_scale == 1.0 and not ff.shared
    assert model.map_checkpoint_name("loop.in") is None


def test_unknown_parts_are_refused():
    from nanovllm.models.sikevik import SikevikConfig, SikevikForCausalLM

    with pytest.raises(NotImplementedError):
        SikevikForCausalLM(SikevikConfig(config([{"type": "convolution", "mixer": {}, "mlp": None}])))
    with pytest.raises(NotImplementedError):
        SikevikForCausalLM(SikevikConfig(config([with_mlp(attention(), {"kind": "bilinear", "ff": 8})])))


def test_frequency_table():
    from nanovllm.layers.seqmix import SinusoidEmbedding

    for width in (1, 2, 7, 64):
        f = SinusoidEmbedding(3, width, 1.0).inv_freq
        assert f.dtype == torch.float32 and f.numel() == (width + 1) // 2
        for i, v in enumerate(f.tolist()):
            assert abs(v - 10000.0 ** (-2 * i / width)) <= 1e-7 * v


def test_bench_model_reads(model_dir):
    """The configuration `bench.py --design sikevik` serves is one of the design, and its weight bytes are those of a
    checkpoint of it when every expert is reached (looped layers twice, the table once as the head)."""
    import importlib.util

    path = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "nano-vllm-ascend_amd", "bench", "design_bench.py")
    spec = importlib.util.spec_from_file_location("design_bench", path)
    bench = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(bench)
    s = dict(bench.SIZES["w1024"], width=64, heads=4, kv_heads=2, dim=16, experts=6, ff=32, top=2, vocab=128, window=16)
    cfg = bench.sikevik_config(s)
    n = 0
    for name, shape in S.tensor_shapes(cfg).items():
        if len(shape) < 2:
            continue
        size = shape[0] * shape[1]
        if name == "loop.in":
            size = size // 2 * 3                    # the embedding's half once, the stream's in both passes
        elif name[0] == "l" and int(name[1:name.index(".")]) >= 2:
            size *= 2
        n += size
    assert bench.sikevik_decode_weight_bytes(cfg, 64) == 2.0 * n


# ---- the plain statement against itself -------------------------------------------------------------------------------
def test_plain_model_is_causal():
    cfg = config([with_mlp(attention(window=6), moe()), with_mlp(attention(), dense())], width=48, vocab=31, loop=(0, 2, 2))
    w = S.random_model(cfg, seed=2)
    toks = list(range(30))
    full = S.forward(cfg, w, toks)
    assert torch.allclose(S.forward(cfg, w, toks[:17]), full[:17], atol=1e-10)


def test_plain_visibility():
    ok = S.visible(9, 3, 2)
    assert [j for j in range(9) if ok[8, j]] == [0, 1, 6, 7, 8]
    assert [j for j in range(9) if ok[4, j]] == [0, 1, 2, 3, 4]
    assert [j for j in range(9) if ok[0, j]] == [0]
    assert bool((S.visible(9, None, 0) == S.visible(9, 100, 0)).all())
    assert bool((S.visible(9, 2, 9) == S.visible(9, None, 0)).all())


def test_plain_softmax_with_one():
    s = torch.tensor([[0.0, float("-inf")], [2.0, 1.0], [-300.0, -301.0], [400.0, 399.0]], dtype=torch.float64)
    p = S.softmax_with_one(s)
    assert torch.allclose(p[0], torch.tensor([0.5, 0.0], dtype=torch.float64))
    e = torch.exp(s[1])
    assert torch.allclose(p[1], e / (1 + e.sum())) and float(p[2].sum()) < 1e-100
    assert torch.allclose(p[3], torch.softmax(s[3], -1))


def test_plain_router_weights_sum_to_the_scale():
    torch.manual_seed(0)
    h, p = torch.randn(5, 8).double(), {"router": torch.randn(6, 8).double()}
    idx, w = S.route(h, p, {"top": 3, "scale": 1.75})
    assert torch.allclose(w.sum(-1), torch.full((5,), 1.75).double())
    z = h @ p["router"].T
    for t in range(5):
        assert idx[t].tolist() == z[t].argsort(descending=True)[:3].tolist()
        assert torch.allclose(w[t], 1.75 * torch.softmax(z[t, idx[t]], -1))


def test_plain_sinusoids():
    s = S.sinusoids(5, 6)
    for t in range(5):
        for i in range(3):
            a = torch.tensor(t * 10000.0 ** (-2 * i / 6), dtype=torch.float64)
            assert abs(s[t, 2 * i] - torch.sin(a)) < 1e-12 and abs(s[t, 2 * i + 1] - torch.cos(a)) < 1e-12
