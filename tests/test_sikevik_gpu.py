"""Sikevik on the GPU against the plain statement of its mechanisms in oracle/sikevik.py (float64, one sequence at a time,
dense scores).  Small configurations of the tests' own making, random bf16-representable weights; where random weights would
hide a fault the weights or inputs are shaped so that it shows.

Bars (sikevik_harness.assert_close): float32 serving mode 5e-5 on every row (row-wise rms difference / rms of the expected
logits), bfloat16 mode 2e-2 on the median row and 6e-2 on all but a few rows; two runs of the engine that differ only in the
cut (portions, batch, pages, slots) 2e-5 in float32."""
import pytest
import torch

from oracle import sikevik as S
from sikevik_harness import (F32_BAR, MIXED, Replay, assert_close, attention, config, dense, moe, rel_err, tokens_of, with_mlp,
                             write_model_dir)

pytestmark = pytest.mark.gpu

CUT_BAR = 2e-5


def expected(cfg, weights, tokens):
    return S.forward(cfg, weights, tokens, dtype=torch.float64)


@pytest.fixture(scope="module")
def mixed_model():
    w = S.random_model(MIXED, seed=3)
    return MIXED, w, write_model_dir(MIXED, w)


@pytest.fixture(scope="module", params=["float32", "bfloat16"])
def mixed_replay(request, mixed_model):
    r = Replay(mixed_model[2], request.param)
    yield request.param, r
    r.close()


# ------------------------------------------------------------------------------------------------ each mechanism alone
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,layers,kw", [
    ("attention", [with_mlp(attention(), None)], {}),
    ("attention_ungrouped", [with_mlp(attention(heads=3, kv_heads=3, dim=12, vdim=12), None)], {}),
    ("attention_one_head", [with_mlp(attention(heads=1, kv_heads=1, dim=16, vdim=8), None)], {}),
    ("attention_one_kv_head_odd_sizes", [with_mlp(attention(heads=5, kv_heads=1, dim=10, vdim=7), None)], {}),
    ("attention_matrix_core_sizes", [with_mlp(attention(heads=4, kv_heads=2, dim=32, vdim=48, window=20, kept=6), None)], {}),
    ("attention_twenty_heads_on_one", [with_mlp(attention(heads=20, kv_heads=1, dim=32, vdim=32, window=20, kept=6), None)], {}),
    ("attention_wide_heads", [with_mlp(attention(heads=2, kv_heads=1, dim=160, vdim=144, scale=0.05), None)], {}),
    ("attention_values_wider_than_keys", [with_mlp(attention(heads=4, kv_heads=2, dim=8, vdim=80, scale=0.4), None)], {}),
    ("attention_window_of_one", [with_mlp(attention(window=1, kept=2), None)], {}),
    ("attention_nothing_kept", [with_mlp(attention(kept=0), None)], {}),
    ("attention_more_kept_than_window", [with_mlp(attention(window=5, kept=19), None)], {}),
    ("attention_everything_kept", [with_mlp(attention(window=2, kept=500), None)], {}),
    ("attention_causal", [with_mlp(attention(window=None), None)], {}),
    ("dense_ff", [with_mlp(attention(), dense())], {}),
    ("sparse_ff", [with_mlp(attention(), moe())], {}),
    ("sparse_ff_no_shared_expert", [with_mlp(attention(), moe(shared=0))], {}),
    ("sparse_ff_top1_many_experts", [with_mlp(attention(), moe(ff=8, experts=70, top=1, scale=0.5, shared=100))], {}),
    ("sparse_ff_every_expert", [with_mlp(attention(), moe(ff=16, experts=4, top=4, scale=1.0))], {}),
    ("sparse_ff_one_expert", [with_mlp(attention(), moe(ff=16, experts=1, top=1, scale=3.0, shared=0))], {}),
    ("odd_width", [with_mlp(attention(), moe()), with_mlp(attention(), dense(33))], {"width": 61, "loop": (0, 2, 2)}),
    ("embedding_unscaled", [with_mlp(attention(), None)], {"scale": 1.0}),
    ("large_eps", [with_mlp(attention(), moe())], {"eps": 0.3}),
    ("loop_everything_twice", [with_mlp(attention(), moe()), with_mlp(attention(window=4), None)], {"loop": (0, 2, 2)}),
    ("loop_one_pass", [with_mlp(attention(), None), with_mlp(attention(kept=0), dense())], {"loop": (0, 2, 1)}),
    ("loop_middle_layer_thrice", [with_mlp(attention(), None), with_mlp(attention(window=6), moe()), with_mlp(attention(window=5), dense())],
     {"loop": (1, 2, 3)}),
    ("loop_tail", [with_mlp(attention(), dense()), with_mlp(attention(window=4), None)], {"loop": (1, 2, 2)}),
    ("no_loop", [with_mlp(attention(), moe()), with_mlp(attention(window=8), None), with_mlp(attention(window=8), dense())], {}),
    ("empty_loop", [with_mlp(attention(), None)], {"loop": (1, 1, 2)}),
])
def test_mechanism_alone(name, layers, kw, dtype):
    cfg = config(layers, **kw)
    w = S.random_model(cfg, seed=11)
    toks = tokens_of(45, cfg["vocab"], 5)
    r = Replay(write_model_dir(cfg, w), dtype)
    try:
        r.runner.model.trace_layers = []
        got = r.feed("a", toks, [45])
        want_layers = []
        want = S.forward(cfg, w, toks, collect=want_layers)
        assert len(r.runner.model.trace_layers) == len(want_layers) == len(S.layer_runs(cfg))
        for i, (a, b) in enumerate(zip(r.runner.model.trace_layers, want_layers)):
            assert_close(a.cpu(), b, dtype, f"the residual stream after layer run {i}")
        r.runner.model.trace_layers = None
        assert_close(got, want, dtype)
        # the same tokens again, one by one, through the pages of every pass
        assert_close(r.feed("b", toks, [3]), want, dtype)
    finally:
        r.close()


# ------------------------------------------------------------------------------------------------ operators
def _step_meta(lengths, starts):
    """cu_q, kv_lens of a step whose sequence s brings lengths[s] rows from position starts[s] on"""
    cu = [0]
    for n in lengths:
        cu.append(cu[-1] + n)
    kv = [a + n for a, n in zip(starts, lengths)]
    return torch.tensor(cu, dtype=torch.int32).cuda(), torch.tensor(kv, dtype=torch.int32).cuda()


@pytest.mark.parametrize("width", [1, 2, 7, 64, 530])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_embedding_with_positions(width, dtype):
    """Three sequences that continue at different places, far positions, odd widths.  (The angle is an fp32 product: at
    position p its rounding turns a channel by up to p * 2^-24 radians.)"""
    from nanovllm import ops
    from nanovllm.layers.seqmix import SinusoidEmbedding

    g = torch.Generator().manual_seed(width)
    V = 11
    table = torch.randn(V, width, generator=g).to(dtype)
    lengths, starts = [3, 1, 4], [0, 3000, 77]
    pos = [a + i for a, n in zip(starts, lengths) for i in range(n)]
    ids = torch.randint(0, V, (8,), generator=g)
    cu, kv = _step_meta(lengths, starts)
    f = SinusoidEmbedding(V, width, 1.0).inv_freq.cuda()
    got = ops.embedding_sinusoid_f32(ids.cuda(), table.cuda(), 2.5, f, cu, kv).cpu().double()
    want = table[ids].double() * 2.5 + S.sinusoids(3001, width)[pos]
    assert (got - want).abs().max() <= 3001 * 2.0 ** -23 + 1e-5


@pytest.mark.parametrize("H,G,D", [(3, 2, 24), (1, 1, 8), (5, 5, 130), (8, 2, 64)])
def test_head_norm_weights_and_pages(H, G, D):
    """Per-head norm with one weight for the query heads and another for the key heads, no rotation; keys and values in their
    page rows, a row with slot -1 storing nothing."""
    from nanovllm import _C, ops

    g = torch.Generator().manual_seed(D + H)
    rows, Dv, bs, eps = 8, 12, 16, 1e-3
    proj = torch.randn(rows, 7 + H * D + G * D + G * Dv, generator=g)
    q_off, k_off, v_off = 7, 7 + H * D, 7 + H * D + G * D
    qw, kw = 1 + torch.randn(D, generator=g), 1 + torch.randn(D, generator=g)
    cu, kv = _step_meta([5, 3], [300, 0])
    want_q = S.rms_norm(proj[:, q_off:k_off].double().view(rows, H, D), qw.double(), eps)
    want_k = S.rms_norm(proj[:, k_off:v_off].double().view(rows, G, D), kw.double(), eps)
    for dt in (torch.float32, torch.bfloat16):
        kc, vc = torch.full((4, G, bs, D), 9.0, dtype=dt).cuda(), torch.full((4, G, bs, Dv), 9.0, dtype=dt).cuda()
        slots = torch.tensor([2 * bs + 15, 3 * bs, 3 * bs + 1, 3 * bs + 2, -1, 5, 6, 7], dtype=torch.int32).cuda()
        p = proj.clone().cuda()
        ops.rotary_store(p, q_off, k_off, v_off, H, G, D, 0, _C.ROT_INTERLEAVED, torch.zeros(1).cuda(), 1.0, True, eps, 1.0, cu, kv,
                         kc, vc, slots, bs, q_norm=qw.cuda(), k_norm=kw.cuda())
        assert (p[:, q_off:k_off].cpu().double().view(rows, H, D) - want_q).abs().max() <= 1e-4
        tol = 1e-4 if dt == torch.float32 else 1e-2 * float(want_k.abs().max())
        for r_, s_ in enumerate(slots.tolist()):
            if s_ >= 0:
                assert (kc[s_ // bs, :, s_ % bs].cpu().double() - want_k[r_]).abs().max() <= tol
                assert (vc[s_ // bs, :, s_ % bs].cpu().double().reshape(-1) - proj[r_, v_off:].double()).abs().max() <= max(tol, 2e-2)
        written = torch.zeros(4 * bs, dtype=torch.bool)
        written[[s_ for s_ in slots.tolist() if s_ >= 0]] = True
        for c in (kc, vc):
            assert bool((c.cpu().float().permute(0, 2, 1, 3).reshape(4 * bs, -1)[~written] == 9.0).all())


def _paged(x, bs, n_blocks, table, dtype):
    """x [T, heads, d] -> a cache [n_blocks, heads, bs, d] holding token t at page table[t // bs], slot t % bs"""
    T, heads, d = x.shape
    c = torch.zeros(n_blocks, heads, bs, d)
    for t in range(T):
        c[table[t // bs], :, t % bs] = x[t]
    return c.to(dtype).cuda()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dv,window,kept,chunk", [
    (4, 2, 32, 16, 40, 4, 0), (4, 2, 32, 32, 1000, 7, 0), (6, 3, 12, 10, 70, 1, 0), (2, 2, 64, 64, 33, 32, 0), (3, 1, 7, 5, 64, 33, 0),
    (40, 2, 64, 48, 20, 5, 0), (2, 1, 160, 144, 50, 65, 0), (4, 2, 32, 32, 1, 1, 0), (4, 2, 32, 32, 17, 100, 0), (6, 2, 24, 24, 30, 16, 0),
    (4, 2, 32, 32, 1000, 6, 48), (6, 2, 24, 24, 25, 5, 40)])
def test_attention_with_kept_first_keys(dtype, H, G, D, Dv, window, kept, chunk):
    """The attention operator with kept first keys and one added to the denominator, in every form (matrix cores, 16-byte
    loads, element-wise; decode steps in one and in several workgroups per row and head): prompts from the start, portions on
    both sides of the place where the window leaves the kept keys, single rows, batches of both, scrambled pages; the kept
    keys beside a chunked mask too."""
    from nanovllm import ops

    g = torch.Generator().manual_seed(D * Dv + H + kept)
    T, bs, scale = 150, 16, 0.5
    n_blocks = 12
    table = torch.randperm(n_blocks - 1, generator=g)[:10].tolist()
    q, k, v = torch.randn(T, H, D, generator=g), torch.randn(T, G, D, generator=g), torch.randn(T, G, Dv, generator=g)
    if dtype == torch.bfloat16:
        k, v = k.bfloat16().float(), v.bfloat16().float()
    s = torch.einsum("ihd,jhd->hij", q.double(), k.double().repeat_interleave(H // G, 1)) * (scale / D ** 0.5)
    ok = S.visible(T, window, kept)
    if chunk:
        i = torch.arange(T)
        inside = (i.view(T, 1) // chunk == i.view(1, T) // chunk) & S.visible(T, window, 0)
        ok = inside | ((i.view(1, T) < kept) & (i.view(1, T) <= i.view(T, 1)))
    pr = S.softmax_with_one(s.masked_fill(~ok, float("-inf")))
    want = torch.einsum("hij,jhd->ihd", pr, v.double().repeat_interleave(H // G, 1)).reshape(T, H * Dv)
    kc, vc = _paged(k, bs, n_blocks, table, dtype), _paged(v, bs, n_blocks, table, dtype)
    tables = torch.tensor(table, dtype=torch.int32).repeat(4, 1)
    sink = torch.zeros(H).cuda()
    last = min(window + kept, T - 3)
    for lengths, starts in (([T], [0]), ([50], [100]), ([1], [149]), ([1, 1, 1], [149, 16, 0]), ([30, 1, 2], [120, 15, 31]),
                            ([2], [last]), ([3, 1], [max(window - 1, 0) % 140, last]), ([1, 1, 1, 1], [last, last + 1, min(kept, 149), 149])):
        cu, kv = _step_meta(lengths, starts)
        rows = [a + i for a, n in zip(starts, lengths) for i in range(n)]
        got = ops.paged_attention_f32(q[rows].reshape(len(rows), H * D).cuda(), kc, vc, Dv, tables[:len(lengths)].contiguous().cuda(),
                                      cu, kv, H, G, D, Dv, bs, window, scale / D ** 0.5, sink=sink, kept=kept, chunk=chunk)
        ref = want[rows]
        assert (got.cpu().double() - ref).abs().max() <= 1e-4 * max(1.0, float(ref.abs().max())), (lengths, starts)


@pytest.mark.parametrize("n,top", [(1, 1), (5, 5), (12, 2), (130, 9), (512, 8)])
def test_router_weights(n, top):
    from nanovllm import ops

    g = torch.Generator().manual_seed(n)
    z = torch.randn(9, n + 2, generator=g) * 4
    ids, wts = ops.route_topk(z.cuda(), n, top, 1.75)
    idx, want = S.route(z[:, :n].double(), {"router": torch.eye(n).double()}, {"top": top, "scale": 1.75})
    assert torch.equal(ids.cpu().long(), idx)
    assert (wts.cpu().double() - want).abs().max() <= 1e-5


@pytest.mark.parametrize("width", [5, 80, 300, 1030, 1100, 2048, 4100, 5000])
def test_output_norm_of_parts(width):
    """One part and several, with and without weights, a shared part and a following norm; widths that fit the registers of a
    workgroup and widths that are summed again, in 16-byte and in single loads; the residual a column slice."""
    from nanovllm import ops

    g = torch.Generator().manual_seed(width)
    rows, eps = 3, 1e-3
    for parts, weighted, with_shared, with_next in ((1, False, False, True), (1, False, False, False), (3, True, True, True),
                                                    (2, True, False, True), (4, False, True, False)):
        res, y = torch.randn(rows, width + 4, generator=g), torch.randn(rows * parts, width, generator=g)
        wts, shared = torch.rand(rows, parts, generator=g), torch.randn(rows, width, generator=g)
        w1, w2 = 1 + torch.randn(width, generator=g) * 0.3, 1 + torch.randn(width, generator=g) * 0.3
        v = y.double().view(rows, parts, width)
        v = (v * wts.double().unsqueeze(-1) if weighted else v).sum(1) + (shared.double() if with_shared else 0)
        want = res[:, :width].double() + S.rms_norm(v, w1.double(), eps)
        r = res.clone().cuda()
        h = ops.parts_norm_add_f32(r[:, :width], y.cuda(), w1.cuda(), eps, wts=wts.cuda() if weighted else None,
                                   shared=shared.cuda() if with_shared else None, w_next=w2.cuda() if with_next else None)
        assert (r[:, :width].cpu().double() - want).abs().max() <= 1e-4
        assert torch.equal(r[:, width:].cpu(), res[:, width:])
        assert (h is None) == (not with_next)
        if with_next:
            assert (h.cpu().double() - S.rms_norm(want, w2.double(), eps)).abs().max() <= 1e-4


@pytest.mark.parametrize("rows,dtype", [(1, torch.float32), (3, torch.bfloat16), (40, torch.float32), (40, torch.bfloat16),
                                        (200, torch.bfloat16), (700, torch.bfloat16), (1100, torch.float32)])
def test_squared_relu_in_every_gemm(rows, dtype):
    """Plain and grouped, in the kernels for few rows, decode batches, tiles and prompts, and the 32-bit ones."""
    from nanovllm import _C, ops

    g = torch.Generator().manual_seed(rows)
    K, N, E = 40, 136, 3
    x = torch.randn(rows, K, generator=g)
    if dtype == torch.bfloat16:
        x = x.bfloat16().float()
    w = (torch.randn(E, N, K, generator=g) * 0.4).to(dtype)
    want = S.relu_squared(x.double() @ w[0].double().T)
    got = ops.gemm_any_act(x.cuda(), w[0].contiguous().cuda(), act=_C.ACT_RELU2).cpu().double()
    assert (got - want).abs().max() <= 1e-4 * max(1.0, float(want.max())) and bool((got >= 0).all())
    ids = torch.randint(0, E, (rows, 1), generator=g).int()
    offsets, pair_token, pair_index = ops.moe_sort(ids.cuda(), E)
    got = ops.gemm_any_grouped_act(x.cuda(), pair_token, w.cuda(), None, _C.ACT_RELU2, offsets, rows, pair_index, rows).cpu().double()
    for t in range(0, rows, max(1, rows // 40)):
        ref = S.relu_squared(x[t].double() @ w[int(ids[t, 0])].double().T)
        assert (got[t] - ref).abs().max() <= 1e-4 * max(1.0, float(ref.max()))


def test_shared_part_without_a_gate():
    from nanovllm import ops

    g = torch.Generator().manual_seed(1)
    y, wts, shared = torch.randn(10, 33, generator=g), torch.rand(5, 2, generator=g), torch.randn(5, 33, generator=g)
    ids = torch.zeros(5, 2, dtype=torch.int32)
    got = ops.moe_combine_shared(y.cuda(), ids.cuda(), wts.cuda(), 33, shared.cuda())
    want = (y.view(5, 2, 33) * wts.unsqueeze(-1)).sum(1) + shared
    assert (got.cpu() - want).abs().max() <= 1e-5


# ------------------------------------------------------------------------------------------------ the engine's cuts
def test_whole_prompt(mixed_model, mixed_replay):
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(70, cfg["vocab"], 2)
    assert_close(r.feed("p", toks, [70]), expected(cfg, w, toks), dtype)


def test_prefill_then_token_by_token(mixed_model, mixed_replay):
    """Decoding through the pages of every pass: 20 prompt tokens, then 60 single tokens (across page borders at 32, 48, 64
    and out of the windows of 9, 13, 17 and 40)."""
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(80, cfg["vocab"], 2)
    assert_close(r.feed("d", toks, [20]), expected(cfg, w, toks), dtype)


def test_first_tokens_one_by_one(mixed_model, mixed_replay):
    """A sequence that starts with single tokens: windows that are not full yet, kept tokens that are still inside them."""
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(12, cfg["vocab"], 3)
    assert_close(r.feed("f", toks, []), expected(cfg, w, toks), dtype)


@pytest.mark.parametrize("cuts", [[2, 2, 2, 3, 5, 2, 16, 15, 17, 2], [31, 2, 33], [16, 16, 16, 16], [1, 2, 1, 2, 40],
                                  [6, 1, 7, 7, 6, 2, 14]])
def test_portions(mixed_model, mixed_replay, cuts):
    """Portions down to two tokens, ending on and off page borders (16), window edges and the kept tokens' end."""
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(75, cfg["vocab"], 6)
    got = r.feed("c", toks, cuts)
    assert_close(got, expected(cfg, w, toks), dtype)
    if dtype == "float32":
        assert rel_err(got, r.feed("w", toks, [75])) <= CUT_BAR


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_hundreds_of_keys(dtype):
    """330 tokens with head sizes of every attention kernel, long windows beside short ones, looped: whole, in portions,
    decoded (the attention kernels take keys 32 or 64 at a time)."""
    cfg = config([with_mlp(attention(heads=4, kv_heads=2, dim=32, vdim=48, window=250, kept=9), None),
                  with_mlp(attention(heads=4, kv_heads=2, dim=32, vdim=32, window=129, kept=64), moe(ff=16, experts=6, top=2)),
                  with_mlp(attention(heads=2, kv_heads=2, dim=12, vdim=12, window=64, kept=33), dense()),
                  with_mlp(attention(heads=3, kv_heads=1, dim=7, vdim=6, window=100, kept=2), None)],
                 width=96, vocab=61, loop=(0, 2, 2))
    w = S.random_model(cfg, seed=21)
    toks = tokens_of(330, 61, 8)
    want = expected(cfg, w, toks)
    r = Replay(write_model_dir(cfg, w), dtype, pages=48)
    try:
        assert_close(r.feed("a", toks, [330]), want, dtype)
        assert_close(r.feed("b", toks, [100, 3, 64, 65, 2, 70]), want, dtype)     # then 26 single tokens
        assert_close(r.feed("c", toks, [140] + [1] * 100 + [90]), want, dtype)
    finally:
        r.close()


def test_long_decoding(mixed_model, mixed_replay):
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(300, cfg["vocab"], 6)
    assert_close(r.feed("l", toks, [3]), expected(cfg, w, toks), dtype)


# ------------------------------------------------------------------------------------------------ batches, pages, slots
def test_unequal_batch_equals_alone(mixed_model, mixed_replay):
    """Four requests of unequal length in mixed steps (portions beside single tokens, a request left out of a step, one that
    ends and whose pages and slot the next one takes) against each request alone."""
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    V = cfg["vocab"]
    seqs = {"a": tokens_of(50, V, 10), "b": tokens_of(7, V, 5), "c": tokens_of(33, V, 12), "d": tokens_of(21, V, 15),
            "e": tokens_of(40, V, 2)}
    plan = [
        ([("a", 17), ("b", 2)], []),
        ([("a", 1), ("b", 3), ("c", 30)], []),
        ([("a", 1), ("c", 1), ("d", 21)], ["d"]),          # b left out
        ([("a", 16), ("b", 2), ("c", 1), ("e", 2)], ["b"]),  # e takes d's slot and pages
        ([("e", 30), ("c", 1), ("a", 15)], ["a", "c"]),
        ([("e", 8)], ["e"]),
    ]
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    slots_seen = {}
    for entries, end in plan:
        step = [(k, seqs[k][at[k]:at[k] + n]) for k, n in entries]
        out = r.step(step, end=[])
        for k, n in entries:
            got[k].append(out[k])
            at[k] += n
            slots_seen[k] = r.live[k].state_slot
        for k in end:
            assert at[k] == len(seqs[k])
            r.scheduler.finish(r.live.pop(k))
    assert slots_seen["e"] == slots_seen["d"], "the freed slot was not used again"
    for k, toks in seqs.items():
        both = torch.cat(got[k])
        assert_close(both, expected(cfg, w, toks), dtype)
        if dtype == "float32":
            assert rel_err(both, r.feed(k + "_alone", toks, [len(toks)])) <= CUT_BAR, k


def test_pages_and_slots_reused_without_clearing(mixed_model):
    """A pool of exactly one request's pages and ONE slot: every request runs in what the previous one left behind."""
    cfg, w, d = mixed_model
    r = Replay(d, "float32", pages=5, slots=1)
    try:
        for seed, cuts in ((20, [80]), (21, [40, 2, 30]), (22, [])):
            toks = tokens_of(80 if cuts != [] else 20, cfg["vocab"], seed)
            assert rel_err(r.feed("x", toks, cuts), expected(cfg, w, toks)) <= F32_BAR
            assert len(r.scheduler.block_manager.free_block_ids) == 5 and r.scheduler.state_slots.free == [0]
    finally:
        r.close()


# ------------------------------------------------------------------------------------------------ faults that random weights hide
def _spiky_model(window, kept, heads=2, dim=8, vdim=12, scale=1.5):
    """One layer whose keys and queries are a function of the token alone (a large embedding scale over the sinusoids): key
    channel 6 is large for token 1 only, every query of head 0 looks for it, and its score (scale * dim) stands out by far
    more than hundreds of other keys weigh together.  Head 1's queries turn away from every key (scores of -scale * dim, all
    of them under the one in the denominator): its read-out is next to nothing, and an output norm over both heads shows
    what the denominator does."""
    W = 32
    cfg = config([with_mlp(attention(heads=heads, kv_heads=1, dim=dim, vdim=vdim, window=window, kept=kept, scale=scale), None)],
                 width=W, vocab=8, scale=64.0)
    w = S.random_model(cfg, seed=6)
    e = torch.zeros(8, W)
    e[:, 0] = 1.0
    e[1, 1] = 6.0                                  # token 1 carries a large feature 1
    for t in range(2, 8):
        e[t, 2 + t % 4] = 1.0
    q, k = torch.zeros(heads * dim, W), torch.zeros(dim, W)
    q[6, 0] = 12.0                                 # head 0: channel 6, from the feature every token has
    for h in range(1, heads):
        q[h * dim + 6, 0] = q[h * dim + 7, 0] = -12.0
    k[6, 1] = 2.0                                  # the key's channel 6 = feature 1 (token 1 only)
    k[7, 0] = 1.0                                  # every other key lives in channel 7
    w.update({"embed": e, "l0.mix.q": q, "l0.mix.k": k, "l0.norm1": torch.ones(W), "l0.norm1b": torch.full((W,), 40.0),
              "l0.mix.q.norm": torch.ones(dim), "l0.mix.k.norm": torch.ones(dim)})
    return cfg, {n: t.bfloat16().float() for n, t in w.items()}


def _tokens_with_spike(n, p):
    toks = [2 + (i % 6) for i in range(n)]
    if p is not None:
        toks[p] = 1
    return toks


# head sizes of the element-wise form, the 16-byte form and (bf16 pages) the matrix cores
SHAPES = [dict(dim=8, vdim=12), dict(dim=8, vdim=7), dict(dim=32, vdim=32, scale=0.4), dict(dim=32, vdim=48, scale=0.4)]


@pytest.mark.parametrize("shape", SHAPES)
def test_a_far_key_among_hundreds(shape):
    """One dominant key at position p under a window that still holds it 390 rows on; every later row's output is that
    key's value: a page of the block table that is skipped, a chunk of keys that is dropped, or a first key that is lost
    shows at full size.  In a prompt, in portions, decoded; the key at position 0, at a page's last and first slot."""
    cfg, w = _spiky_model(100000, 2, **shape)
    r = Replay(write_model_dir(cfg, w), "float32", pages=30)
    try:
        n = 400
        without = expected(cfg, w, _tokens_with_spike(n, None))
        for p in (0, 15, 16, 130):
            toks = _tokens_with_spike(n, p)
            want = expected(cfg, w, toks)
            assert rel_err(without[n - 1:], want[n - 1:]) > 0.05, "the far key has no influence: the test's weights are wrong"
            for cuts in ([n], [p + 1, 2, 200, 2], [300] + [1] * 60 + [40], [129, 129, 129]):
                assert rel_err(r.feed("s", toks, cuts), want) <= F32_BAR, (p, cuts)
    finally:
        r.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window,kept", [(37, 0), (37, 4), (64, 1), (130, 16), (2, 3)])
@pytest.mark.parametrize("shape", SHAPES[1:3])
def test_window_edges(shape, window, kept, dtype):
    """The dominant key at position p (behind the kept tokens) is the OLDEST key of row p + window - 1 and just outside for
    row p + window: the two rows differ at full size in the plain statement, and the engine has to agree on both - in a
    prompt, when the edge falls on a portion's first or last row, and decoded token by token; p right behind the kept tokens,
    at a page's last and first slot and mid-page."""
    cfg, w = _spiky_model(window, kept, **shape)
    r = Replay(write_model_dir(cfg, w), dtype, pages=30)
    try:
        for p in sorted({kept, max(kept, 15), max(kept, 16), 41}):
            n = p + window + 20
            toks = _tokens_with_spike(n, p)
            want = expected(cfg, w, toks)
            inside, outside = p + window - 1, p + window
            assert rel_err(want[outside:outside + 1], want[inside:inside + 1]) > 0.05, "the edge does not show: the test's weights are wrong"
            for cuts in ([n], [inside, 1, 1], [inside + 1, 2], [outside, 2], [p + 1] + [1] * (window + 5),
                         [p + 2, max(window - 3, 1), 2, 2, 2]):
                got = r.feed("s", toks, cuts)
                assert rel_err(got, want) <= (F32_BAR if dtype == "float32" else 2e-2), (p, cuts)
    finally:
        r.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window,kept", [(37, 4), (20, 1), (64, 16), (12, 33), (1, 40)])
@pytest.mark.parametrize("shape", SHAPES[1:])
def test_first_tokens_stay_visible(shape, window, kept, dtype):
    """The dominant key as the last kept token shows in every later row; one position on, it leaves with the window.  Far
    behind both, in a prompt, at a portion's first and last row, decoded, and around the row whose window just leaves the
    kept tokens (where kept and window keys join without a hole or a doubled key)."""
    cfg, w = _spiky_model(window, kept, **shape)
    r = Replay(write_model_dir(cfg, w), dtype, pages=30)
    try:
        n = kept + window + 90
        rows = {}
        for p in sorted({0, kept - 1, kept, kept + 1}):
            toks = _tokens_with_spike(n, p)
            want = expected(cfg, w, toks)
            rows[p] = want[n - 1:]
            joint = kept + window - 1          # the last row whose window still reaches the kept tokens
            for cuts in ([n], [joint, 1, 1, 2], [joint + 1, 2, 40], [p + 1, 2, window, 3, 2], [joint - 1] + [1] * 50):
                got = r.feed("k", toks, [c for c in cuts if c > 0])
                assert rel_err(got, want) <= (F32_BAR if dtype == "float32" else 2e-2), (p, cuts)
        assert rel_err(rows[kept], rows[kept - 1]) > 0.05, "the last kept token does not show: the test's weights are wrong"
    finally:
        r.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("scale", [1.5, 0.05])
def test_one_in_the_denominator(scale, dtype, monkeypatch):
    """Scores far below zero (head 1: next to no weight is left for any key) and scores near zero with few keys (the first
    rows: half of the weight is nobody's): leaving the one out, or counting it once per chunk of keys, moves the rows by tens
    of percent through the balance of the two heads."""
    cfg, w = _spiky_model(1000, 0, scale=scale)
    n = 200
    toks = _tokens_with_spike(n, 70)
    want = expected(cfg, w, toks)
    with monkeypatch.context() as mp:
        mp.setattr(S, "softmax_with_one", lambda s: torch.softmax(s, -1))
        other = expected(cfg, w, toks)
        rows = slice(80, None) if scale > 1 else slice(0, 3)
        assert rel_err(other[rows], want[rows]) > 0.03, "the one has no influence: the test's weights are wrong"
    r = Replay(write_model_dir(cfg, w), dtype, pages=30)
    try:
        for cuts in ([n], [69, 2, 2, 100], [100] + [1] * 70 + [30], [2, 2, 2, 1, 1]):
            assert rel_err(r.feed("k", toks, cuts), want) <= (F32_BAR if dtype == "float32" else 2e-2), cuts
    finally:
        r.close()


def test_scores_without_positions_and_an_embedding_with_them():
    """All tokens equal: the layers see positions only through the sinusoids, which a large-scale embedding would bury; rows
    differ, and a portion that starts its positions at zero, or a decoded token at the wrong one, shows."""
    cfg = config([with_mlp(attention(), moe()), with_mlp(attention(window=50), dense())], vocab=17, scale=0.25, loop=(0, 2, 2))
    w = S.random_model(cfg, seed=8)
    toks = [5] * 60
    want = expected(cfg, w, toks)
    assert rel_err(want[30:31], want[2:3]) > 0.05
    r = Replay(write_model_dir(cfg, w), "float32")
    try:
        for cuts in ([60], [20, 2, 30], [16, 16, 16], []):
            assert rel_err(r.feed("p", toks, cuts), want) <= F32_BAR, cuts
        out = [r.step([("x", toks[:7]), ("y", toks[:20])]), r.step([("y", toks[20:21]), ("x", toks[7:30])])]
        for name, cut in (("x", (7, 30)), ("y", (20, 21))):
            assert rel_err(torch.cat([o[name] for o in out]), want[:cut[1]]) <= F32_BAR
            r.scheduler.finish(r.live.pop(name))
    finally:
        r.close()


def test_every_pass_begins_with_its_projection(monkeypatch):
    """A projection that mostly brings the embedding back, another that mostly keeps the stream: halves that are swapped, a
    pass that begins without it (the first one too) or with the stream instead of the embedding output move every row."""
    cfg = config([with_mlp(attention(), None), with_mlp(attention(window=6), moe()), with_mlp(attention(window=8), dense())], loop=(1, 3, 3))
    w = S.random_model(cfg, seed=14)
    W = cfg["width"]
    toks = tokens_of(30, 97, 4)
    g = torch.Generator().manual_seed(3)
    for a, b in ((1.0, 0.3), (0.2, 1.0)):
        half = [torch.eye(W) * c + torch.randn(W, W, generator=g) * 0.2 * W ** -0.5 for c in (a, b)]
        w["loop.in"] = torch.cat(half, 1).bfloat16().float()
        want = expected(cfg, w, toks)
        begin = S.begin_pass
        wrong = [lambda x, e, wl: begin(e, x, wl), lambda x, e, wl: begin(x, x, wl), lambda x, e, wl: x]
        for f in wrong:
            with monkeypatch.context() as mp:
                mp.setattr(S, "begin_pass", f)
                assert rel_err(expected(cfg, w, toks), want) > 0.05
        r = Replay(write_model_dir(cfg, w), "float32")
        try:
            assert rel_err(r.feed("v", toks, [17, 2]), want) <= F32_BAR
        finally:
            r.close()


def test_passes_do_not_share_their_pages():
    """Weights under which the second pass's keys differ much from the first's: a pass that reads another pass's pages shows
    in every row behind the first, whole, in portions and decoded."""
    cfg = config([with_mlp(attention(window=100, kept=3), None), with_mlp(attention(heads=4, kv_heads=2, dim=32, vdim=32, window=30), None)],
                 loop=(0, 2, 2))
    w = S.random_model(cfg, seed=15)
    for i in (0, 1):
        w[f"l{i}.norm1b"] = torch.full((80,), 2.0)
    toks = tokens_of(60, 97, 9)
    want = expected(cfg, w, toks)
    for dtype in ("float32", "bfloat16"):
        r = Replay(write_model_dir(cfg, w), dtype)
        try:
            for cuts in ([60], [30, 2, 20], [10]):
                assert_close(r.feed("v", toks, cuts), want, dtype, cuts)
        finally:
            r.close()


def test_head_norm_weights_differ_by_channel_and_side():
    """Query and key norm weights that each silence half of the channels: swapped, missing or one-plus weights show."""
    cfg = config([with_mlp(attention(heads=4, kv_heads=2, dim=16, vdim=16, window=40, scale=1.0), None)], width=48, vocab=31)
    w = S.random_model(cfg, seed=16)
    w["l0.norm1b"] = torch.full((48,), 4.0)
    w["l0.mix.q.norm"] = torch.cat([torch.full((12,), 1.5), torch.full((4,), 0.0)])
    w["l0.mix.k.norm"] = torch.cat([torch.full((4,), 0.0), torch.full((12,), 2.0)])
    w["l0.mix.k.norm"][5] = -3.0
    toks = tokens_of(50, 31, 2)
    want = expected(cfg, w, toks)
    swapped = dict(w)
    swapped["l0.mix.q.norm"], swapped["l0.mix.k.norm"] = w["l0.mix.q.norm"] + 1, w["l0.mix.k.norm"] + 1
    assert rel_err(expected(cfg, swapped, toks), want) > 0.05
    r = Replay(write_model_dir(cfg, w), "float32")
    try:
        for cuts in ([50], [20, 2, 2]):
            assert rel_err(r.feed("n", toks, cuts), want) <= F32_BAR
    finally:
        r.close()


# ------------------------------------------------------------------------------------------------ the engine's own entry point
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_llm(mixed_model, dtype):
    """LLM.generate: the scheduler's prefill and decode steps, its page and slot managers, captured decode steps, the sampler.
    Every generated token must be the plain model's best token given the same history (or within the sampler's bf16 logits
    of it); in the bfloat16 mode a router's near-tie now and then moves a row by more than that: two of the sixty may differ."""
    from nanovllm import LLM, SamplingParams

    cfg, w, d = mixed_model
    llm = LLM(d, dtype=dtype, kvcache_block_size=16, num_kvcache_blocks=40, max_num_seqs=3, max_model_len=256,
              max_num_batched_tokens=256, warmup=False)
    try:
        assert llm.model_runner.row_graphs
        prompts = [tokens_of(n, cfg["vocab"], 30 + n) for n in (5, 40, 17, 33, 2)]   # five requests over three slots
        outs = llm.generate(prompts, SamplingParams(max_tokens=12, greedy=True, ignore_eos=True), use_tqdm=False)
        assert len(outs) == 5
        off = []
        for prompt, out in zip(prompts, outs):
            gen = out["token_ids"]
            assert len(gen) == 12
            logits = expected(cfg, w, prompt + gen)
            for i, tok in enumerate(gen):
                row = logits[len(prompt) - 1 + i]
                if row.max() - row[tok] > 0.06 * max(1.0, float(row.abs().max())):
                    off.append((len(prompt), i, tok, int(row.argmax()), float(row.max() - row[tok])))
        assert len(off) <= (0 if dtype == "float32" else 2), off
    finally:
        llm.exit()


def test_captured_decode_steps_equal_eager(mixed_model):
    """Decode steps replay hipGraphs padded to a batch bucket (3 live requests in the bucket of 4): same tokens and the same
    logits as eager launches, over several replays with eager prefill steps between them."""
    from nanovllm import LLM, SamplingParams

    cfg, w, d = mixed_model
    prompts = [tokens_of(n, cfg["vocab"], 70 + n) for n in (9, 31, 16, 5, 22)]
    sp = SamplingParams(max_tokens=10, greedy=True, ignore_eos=True)
    runs, logits = [], []
    for eager in (True, False):
        llm = LLM(d, dtype="float32", kvcache_block_size=16, num_kvcache_blocks=40, max_num_seqs=4, max_model_len=128,
                  max_num_batched_tokens=128, warmup=False, enforce_eager=eager)
        try:
            assert bool(llm.model_runner.row_graphs) == (not eager)
            runs.append([o["token_ids"] for o in llm.generate(prompts[:3], sp, use_tqdm=False)])
            runs[-1] += [o["token_ids"] for o in llm.generate(prompts[3:], sp, use_tqdm=False)]
            logits.append(llm.model_runner.last_logits.float().cpu().clone())
        finally:
            llm.exit()
    assert runs[0] == runs[1]
    assert rel_err(logits[1], logits[0]) <= CUT_BAR


def test_engine_chunked_prefill_equals_whole_prompts(mixed_model):
    """Config.chunked_prefill: the engine's own scheduler cuts prompts into portions (24 rows per step) and batches them
    with the other requests' decoded tokens; the generated tokens are those of whole-prompt prefill steps."""
    from nanovllm import LLM, SamplingParams

    cfg, w, d = mixed_model
    prompts = [tokens_of(n, cfg["vocab"], 90 + n) for n in (70, 9, 41, 3, 26)]
    sp = SamplingParams(max_tokens=9, greedy=True, ignore_eos=True)
    runs = []
    for kw in (dict(max_num_batched_tokens=128), dict(max_num_batched_tokens=24, chunked_prefill=True)):
        llm = LLM(d, dtype="float32", kvcache_block_size=16, num_kvcache_blocks=40, max_num_seqs=3, max_model_len=128,
                  warmup=False, **kw)
        try:
            runs.append([o["token_ids"] for o in llm.generate(prompts, sp, use_tqdm=False)])
        finally:
            llm.exit()
    assert runs[0] == runs[1]


def test_trace_replay_program(mixed_model, tmp_path):
    """bin/trace_run end to end: steps on standard input, logits files and `done` lines out; two requests in one step."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np

    cfg, w, d = mixed_model
    toks, other = tokens_of(30, cfg["vocab"], 60), tokens_of(9, cfg["vocab"], 61)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[20:29], "want": []}, {"id": "o", "tokens": other[:8], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "o", "tokens": other[8:], "want": [0]}, {"id": "q", "tokens": toks[29:], "want": [0]}],
              "end": ["q", "o"]}]
    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run([sys.executable, os.path.join(repo, "bin", "trace_run"), "--model", d, "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "128"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want, want_o = expected(cfg, w, toks), expected(cfg, w, other)
    got0 = torch.from_numpy(np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, -1))
    got2 = torch.from_numpy(np.fromfile(tmp_path / "2.f32", dtype="<f4").reshape(2, -1))
    assert not (tmp_path / "1.f32").exists()
    assert rel_err(got0, want[[0, 19]]) <= F32_BAR
    assert rel_err(got2[:1], want_o[[8]]) <= F32_BAR and rel_err(got2[1:], want[[29]]) <= F32_BAR
