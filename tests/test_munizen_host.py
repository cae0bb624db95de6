"""Host-side pieces of the Munizen integration (no GPU): the configuration reader and the order of layer runs, the checkpoint
name map through the framework's loader, what a sequence needs in pages and state slots, and the plain statement's own
consistency."""
import math
import os

import pytest
import torch

from oracle import munizen as M
from munizen_harness import MIXED, RANKS, attention, config, delta, dense, with_mlp, write_model_dir


@pytest.fixture(scope="module")
def model_dir():
    return write_model_dir(MIXED, M.random_model(MIXED, seed=1, rank=RANKS))


def test_config_is_read_from_the_directory(model_dir):
    from nanovllm.config import Config

    c = Config(model_dir, dtype="float32", max_model_len=128, max_num_batched_tokens=128)
    hf = c.hf_config
    assert c.hybrid_state and hf.architectures == ["Munizen"]
    assert (hf.vocab_size, hf.hidden_size, hf.num_hidden_layers) == (MIXED["vocab"], MIXED["width"], 5)
    assert (hf.loop_start, hf.loop_stop, hf.loop_times) == (1, 4, 3)
    assert (hf.norm_eps, hf.norm_groups, hf.streams) == (1e-5, 2, 3)
    assert [hf.rank_of(i) for i in (0, 2)] == [6, 5]      # from the checkpoint's header
    assert c.eos == -1 and c.max_model_len == 128


def test_order_of_layer_runs():
    from nanovllm.models.munizen import MunizenConfig

    layers = [with_mlp(attention(), None)] * 4
    for loop in ((0, 2, 2), (1, 3, 3), (2, 4, 2), (0, 4, 2), (0, 4, 1), (2, 2, 5), (0, 0, 0)):
        cfg = config(layers, loop=loop)
        c = MunizenConfig(cfg)
        assert [i for i, _, _ in c.layer_runs] == M.layer_runs(cfg), loop
        assert len({(i, lane) for i, lane, _ in c.layer_runs}) == len(c.layer_runs)     # a cache / state of its own per run
        for i, lane, _ in c.layer_runs:
            assert 0 <= lane < c.lanes_of(i)


def test_every_tensor_lands_in_a_parameter(model_dir):
    """Load through the framework's loader on the CPU: every parameter is written, merged ones in the right row ranges, the
    query rows in the attention's order, and nothing of the checkpoint is left over."""
    from nanovllm.models.munizen import MunizenConfig, MunizenForCausalLM
    from nanovllm.utils.loader import load_model
    from safetensors.torch import load_file

    model = MunizenForCausalLM(MunizenConfig.from_dir(model_dir))
    for n, p in model.named_parameters():
        if not n.endswith(".bias"):               # (biases of parts without one stay zero)
            p.data.fill_(float("nan"))
    load_model(model, model_dir)
    w = {k: v.float() for k, v in load_file(os.path.join(model_dir, "model.safetensors")).items()}
    for name, p in model.named_parameters():
        assert not torch.isnan(p).any(), name
    assert set(w) == set(M.tensor_shapes(MIXED, RANKS))
    dl, att = model.layers[0].mix, model.layers[1].mix

    def rows(m, name, of="weight"):
        off, n = m.offsets[name]
        return getattr(m, of)[off:off + n]

    for n in ("r", "k", "v", "g", "a", "w1"):
        assert torch.equal(rows(dl.proj, n), w["l0.mix." + n])
        b = rows(dl.proj, n, "bias")
        assert torch.equal(b, w["l0.mix.a.b"]) if n == "a" else not b.any()
    for n in ("w2", "w0", "norm", "o"):
        assert torch.equal(getattr(dl, n), w["l0.mix." + n])
    for n in ("k", "v", "g"):
        assert torch.equal(rows(att.qkvg, n), w["l1.mix." + n])
        b = rows(att.qkvg, n, "bias")
        assert not b.any() if n == "g" else torch.equal(b, w[f"l1.mix.{n}.b"])
    H, G, D = 6, 3, 24
    for of, src in (("weight", w["l1.mix.q"]), ("bias", w["l1.mix.q.b"])):
        got = rows(att.qkvg, "q", of).reshape(G, 2, H // G, D, -1)
        want = src.reshape(H, 2, D, -1)
        for h in range(H):
            for m in range(2):
                assert torch.equal(got[h // (H // G), m, h % (H // G)], want[h, m])
    for i, n in enumerate(("lq1", "lk1", "lq2", "lk2")):
        assert torch.equal(att.lam[i], w["l1.mix." + n])
    assert torch.equal(att.o, w["l1.mix.o"]) and torch.equal(att.o_b, w["l1.mix.o.b"])
    assert (att.chunk, att.diff, att.scale, att.rot_dims) == (17, 0.45, 0.3, 16) and model.layers[4].mix.chunk == 0
    L1 = model.layers[1]
    for q in ("hc1", "hc2"):
        c = getattr(L1, q)
        assert torch.equal(c.read, w[f"l1.{q}.in"]) and torch.equal(c.write, w[f"l1.{q}.out"]) and torch.equal(c.mix, w[f"l1.{q}.mix"])
    assert torch.equal(L1.norm1, w["l1.norm1"]) and torch.equal(L1.norm2, w["l1.norm2"]) and torch.equal(L1.shift.weight, w["l1.shift"])
    for n in ("gate", "up", "down"):
        assert torch.equal(getattr(L1.mlp, n), w["l1.mlp." + n])
    assert model.layers[2].mlp is None and model.layers[2].norm2 is None and model.layers[2].hc2 is None
    assert torch.equal(model.embed, w["embed"]) and torch.equal(model.head, w["head"]) and torch.equal(model.final_norm, w["final.norm"])


def test_pages_and_state_of_a_sequence(model_dir):
    from nanovllm.models.munizen import MunizenConfig, MunizenForCausalLM

    model = MunizenForCausalLM(MunizenConfig.from_dir(model_dir))
    # pages: both maps' K rows and the V rows of every attention, three times for the layers inside the loop
    per_token = 3 * ((2 * 3 * 24 + 3 * 20) + (2 * 4 * 32 + 4 * 16)) + (2 * 10 + 6)
    assert model.cache_bytes_per_block(16, 2) == 16 * per_token * 2
    # a slot: every layer's last shifted input and the delta rule's matrix states (the kernel keeps them padded: key
    # channels to 64, value channels to a multiple of 32), three times inside the loop
    W = MIXED["width"]
    assert model.state_bytes_per_slot() == 4 * ((W + 3 * 64 * 32) + 3 * W + 3 * (W + 2 * 64 * 64) + 3 * W + W)
    assert model.layers[1].mix.cache_shapes(7, 16) == ((7, 6, 16, 24), (7, 3, 16, 20))
    only_delta = MunizenForCausalLM(MunizenConfig(config([with_mlp(delta(), None)])))
    assert only_delta.cache_bytes_per_block(16, 2) == 0


def test_synthetic_checkpoint_names_match_the_design(model_dir):
    from nanovllm.models.munizen import MunizenConfig, MunizenForCausalLM

    model = MunizenForCausalLM(MunizenConfig.from_dir(model_dir))
    got = {name: tuple(t.shape) for name, t in model.synthetic_state(0)}
    assert got == {k: tuple(v) for k, v in M.tensor_shapes(MIXED, RANKS).items()}


def test_unknown_parts_are_refused():
    from nanovllm.models.munizen import MunizenConfig, MunizenForCausalLM

    with pytest.raises(NotImplementedError):
        MunizenForCausalLM(MunizenConfig(config([{"type": "convolution", "mixer": {}, "mlp": None}])))
    with pytest.raises(NotImplementedError):
        MunizenForCausalLM(MunizenConfig(config([with_mlp(attention(), {"kind": "moe", "ff": 8})])))
    with pytest.raises(AssertionError):
        MunizenConfig(config([with_mlp(attention(), None)], groups=5))      # 84 channels in five equal parts


# ---- the plain statement against itself -------------------------------------------------------------------------------
def test_plain_model_is_causal():
    cfg = config([with_mlp(delta(), dense()), with_mlp(attention(), None)], width=48, vocab=31, loop=(0, 2, 2))
    w = M.random_model(cfg, seed=2)
    toks = list(range(30))
    full = M.forward(cfg, w, toks)
    assert torch.allclose(M.forward(cfg, w, toks[:17]), full[:17], atol=1e-10)


def test_plain_chunks_do_not_see_each_other():
    """Scores depend on distances only and a chunk starts afresh: one attention layer over two equal chunks of inputs gives
    the same rows twice."""
    torch.manual_seed(0)
    m = attention(chunk=5)["mixer"]
    shapes = M.tensor_shapes(config([with_mlp(attention(chunk=5), None)]))
    p = {k[7:]: torch.randn(*s).double() for k, s in shapes.items() if k.startswith("l0.mix.")}
    h = torch.randn(5, 84).double()
    o = M.attention_mixer(torch.cat([h, h, h[:2]]), p, m, 1e-5)
    assert torch.allclose(o[5:10], o[:5], atol=1e-10) and torch.allclose(o[10:], o[:2], atol=1e-10)
    wide = M.attention_mixer(torch.cat([h, h]), p, dict(m, mask={"size": 10}), 1e-5)
    assert not torch.allclose(wide[5:], wide[:5], atol=1e-3)


def test_plain_delta_rule_in_special_cases():
    """No decay, removal rate one, unit keys: reading with the key just written gives its value back exactly; removal rate
    zero: linear attention, o_t = sum_s (r_t . k_s) v_s."""
    torch.manual_seed(1)
    T, H, D = 6, 2, 5
    r, k, v = (torch.randn(T, H, D).double() for _ in range(3))
    one, zero = torch.ones(T, H, D).double(), torch.zeros(T, H, D).double()
    ku = k / k.norm(dim=-1, keepdim=True)
    o = M.general_delta_scan(ku, ku, v, one, one)
    assert torch.allclose(o, v, atol=1e-5)      # (the unit key's 1e-6 under the root)
    o = M.general_delta_scan(r, k, v, one, zero)
    for t in range(T):
        want = sum((r[t] * k[s]).sum(-1, keepdim=True) * v[s] for s in range(t + 1))
        assert torch.allclose(o[t], want, atol=1e-10)


def test_plain_group_norm_and_shift():
    x = torch.randn(3, 6).double()
    y = M.group_norm(x, torch.ones(6).double(), 3, 0.0)
    for g in range(3):
        assert torch.allclose((y[:, 2 * g:2 * g + 2] ** 2).mean(-1), torch.ones(3).double())
    assert torch.equal(M.token_shift(x, torch.ones(6).double())[1:], x[1:] + (x[:-1] - x[1:]))
    assert torch.equal(M.token_shift(x, torch.zeros(6).double()), x)
    assert not M.token_shift(x, torch.ones(6).double())[0].any()


def test_plain_streams_keep_the_residual_sum():
    """One stream with weights of one is the plain residual sum; s equal streams read with weights 1 / s, written with ones
    and not mixed stay equal to it."""
    layers = [with_mlp(delta(), dense()), with_mlp(attention(), None)]
    one = config(layers, width=48, vocab=31, streams=1)
    w = M.random_model(one, seed=5)
    for k in list(w):
        if ".hc" in k:
            w[k] = torch.ones_like(w[k])
    four = dict(one, streams=4)
    w4 = dict(w)
    for k in w:
        if ".hc" in k:
            leaf = k.rsplit(".", 1)[1]
            w4[k] = torch.eye(4) if leaf == "mix" else torch.full((4,), 0.25 if leaf == "in" else 1.0)
    a, b = [], []
    M.forward(one, w, list(range(12)), collect=a)
    M.forward(four, w4, list(range(12)), collect=b)
    for x, y in zip(a, b):
        assert torch.allclose(4 * x, y, atol=1e-10)
    assert math.isclose(float(a[0].abs().max()), float(b[0].abs().max()) / 4, rel_tol=1e-9)
