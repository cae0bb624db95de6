"""Munizen on the GPU against the plain statement of its mechanisms in oracle/munizen.py (float64, one sequence at a time,
dense scores, Python loops over time).  Small configurations of the tests' own making, random bf16-representable weights;
where random weights would hide a fault the weights or inputs are shaped so that it shows.

Bars (munizen_harness.assert_close): float32 serving mode 5e-5 on every row (row-wise rms difference / rms of the expected
logits), bfloat16 mode 6e-2 on every row and 2e-2 on the median; two runs of the engine that differ only in the cut (portions,
batch, pages, slots) 2e-5 in float32."""
import pytest
import torch

from oracle import munizen as M
from munizen_harness import (F32_BAR, MIXED, RANKS, Replay, assert_close, attention, config, delta, dense, rel_err, tokens_of,
                             with_mlp, write_model_dir)

pytestmark = pytest.mark.gpu

CUT_BAR = 2e-5


def expected(cfg, weights, tokens):
    return M.forward(cfg, weights, tokens, dtype=torch.float64)


@pytest.fixture(scope="module")
def mixed_model():
    w = M.random_model(MIXED, seed=3, rank=RANKS)
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
    ("attention_ungrouped_whole_head_rotated", [with_mlp(attention(heads=3, kv_heads=3, dim=12, vdim=12, dims=12), None)], {}),
    ("attention_one_kv_head", [with_mlp(attention(heads=5, kv_heads=1, dim=10, vdim=7, dims=6), None)], {}),
    ("attention_one_head", [with_mlp(attention(heads=1, kv_heads=1, dim=2, vdim=1, dims=2), None)], {}),
    ("attention_matrix_core_sizes", [with_mlp(attention(heads=4, kv_heads=2, dim=32, vdim=48, dims=32, chunk=50), None)], {}),
    ("attention_matrix_core_pairs", [with_mlp(attention(heads=8, kv_heads=2, dim=64, vdim=128, dims=20, chunk=19), None)], {}),
    ("attention_wide_heads", [with_mlp(attention(heads=2, kv_heads=1, dim=160, vdim=144, dims=64, scale=0.05), None)], {}),
    ("attention_chunk_of_one", [with_mlp(attention(chunk=1), None)], {}),
    ("attention_chunk_of_two", [with_mlp(attention(chunk=2, dim=32, vdim=32), None)], {}),
    ("attention_causal", [with_mlp(attention(chunk=0), None)], {}),
    ("attention_no_rotation", [with_mlp(attention(dims=0), None)], {}),
    ("attention_fast_rotation", [with_mlp(attention(dims=24, base=3.0), None)], {}),
    ("attention_no_difference_offset", [with_mlp(attention(diff=0.0), None)], {}),
    ("delta", [with_mlp(delta(), None)], {}),
    ("delta_one_head", [with_mlp(delta(heads=1, dim=7), None)], {"rank": 1}),
    ("delta_64", [with_mlp(delta(heads=2, dim=64), None)], {"rank": 16}),
    ("delta_100", [with_mlp(delta(heads=2, dim=100), None)], {"rank": 33}),
    ("delta_200", [with_mlp(delta(heads=1, dim=200), None)], {"rank": 8}),
    ("feed_forward", [with_mlp(attention(), dense())], {}),
    ("feed_forward_behind_the_delta_rule", [with_mlp(delta(), dense(ff=7))], {}),
    ("one_stream_one_group", [with_mlp(delta(), dense()), with_mlp(attention(), None)], {"streams": 1, "groups": 1}),
    ("eight_streams_seven_groups", [with_mlp(attention(), dense()), with_mlp(delta(), None)], {"streams": 8, "groups": 7}),
    ("two_streams_odd_width", [with_mlp(delta(), None), with_mlp(attention(), dense())], {"streams": 2, "groups": 3, "width": 87}),
    ("five_streams_many_groups", [with_mlp(attention(), None)], {"streams": 5, "groups": 12}),
    ("loop_everything_twice", [with_mlp(attention(), dense()), with_mlp(delta(), None)], {"loop": (0, 2, 2)}),
    ("loop_one_pass", [with_mlp(delta(), None), with_mlp(attention(), None)], {"loop": (0, 2, 1)}),
    ("loop_middle_layer_thrice", [with_mlp(attention(), None), with_mlp(delta(), dense()), with_mlp(attention(chunk=5), None)],
     {"loop": (1, 2, 3)}),
    ("loop_tail", [with_mlp(attention(), None), with_mlp(attention(chunk=4), None)], {"loop": (1, 2, 2)}),
    ("empty_loop", [with_mlp(attention(), None)], {"loop": (1, 1, 2)}),
])
def test_mechanism_alone(name, layers, kw, dtype):
    kw = dict(kw)
    rank = kw.pop("rank", 6)
    cfg = config(layers, **kw)
    w = M.random_model(cfg, seed=11, rank=rank)
    toks = tokens_of(45, cfg["vocab"], 5)
    r = Replay(write_model_dir(cfg, w), dtype)
    try:
        r.runner.model.trace_layers = []
        got = r.feed("a", toks, [45])
        want_layers = []
        want = M.forward(cfg, w, toks, collect=want_layers)
        assert len(r.runner.model.trace_layers) == len(want_layers) == len(M.layer_runs(cfg))
        for i, (a, b) in enumerate(zip(r.runner.model.trace_layers, want_layers)):
            assert_close(a.cpu(), b, dtype, f"the sum of the streams after layer run {i}")
        r.runner.model.trace_layers = None
        assert_close(got, want, dtype)
        # the same tokens again, one by one, through the caches / the states of every pass
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


@pytest.mark.parametrize("s,W,groups", [(1, 16, 1), (2, 36, 3), (3, 40, 2), (4, 2048, 2), (5, 9, 9), (6, 14, 7), (7, 300, 25),
                                        (8, 64, 8), (4, 7992, 1)])
@pytest.mark.parametrize("lengths,starts", [([1, 1, 1], [5, 0, 300]), ([4, 1, 6], [0, 9, 2]), ([2, 2], [1, 0])])
def test_stream_boundary(s, W, groups, lengths, starts):
    """Sublayer output into the streams, weighted sum, group norm, token shift, its carried rows: from the embedding's one
    row and from streams, in place (one row per sequence) and into another buffer; slots of other sequences untouched."""
    from nanovllm import ops

    g = torch.Generator().manual_seed(W + s)
    rows, n = sum(lengths), len(lengths)
    rand = lambda *sh: torch.randn(*sh, generator=g)
    coef = {"in": rand(s), "out": rand(s), "mix": rand(s, s)}
    norm_w, shift, y = rand(W), torch.rand(W, generator=g), rand(rows, W)
    cu, kv = _step_meta(lengths, starts)
    slots = torch.tensor([4, 0, 2][:n], dtype=torch.int32).cuda()
    state0 = rand(6, W)
    for broadcast in (False, True):
        X = rand(rows, s, W)
        if broadcast:
            X = X[:, :1].expand(rows, s, W)
        for with_y in (True, False):
            new = [X[:, i].double() for i in range(s)]
            dc = {k: v.double() for k, v in coef.items()}
            if with_y:
                new = M.streams_write(new, y.double(), dc)
            u = M.group_norm(M.streams_read(new, dc), norm_w.double(), groups, 1e-5)
            want, want_state = u.clone(), state0.double().clone()
            a = 0
            for q, (m, p) in enumerate(zip(lengths, starts)):
                prev = state0[int(slots[q])].double() if p > 0 else torch.zeros(W).double()
                ext = torch.cat([prev[None], u[a:a + m]])
                want[a:a + m] = u[a:a + m] + (ext[:-1] - u[a:a + m]) * shift.double()
                want_state[int(slots[q])] = u[a + m - 1]
                a += m
            src = X.cuda() if broadcast else X.clone().cuda()
            if broadcast:
                src = X[:, 0].contiguous().cuda().unsqueeze(1).expand(rows, s, W)
            in_place = max(lengths) == 1 and not broadcast
            dst = (src if in_place else torch.full((rows, s, W), 9.0).cuda()) if with_y else None
            st = state0.clone().cuda()
            dev = {k: v.cuda() for k, v in coef.items()}
            h = ops.stream_mix(src, dst, y.cuda() if with_y else None, dev["mix"], dev["out"], dev["in"], norm_w.cuda(), groups,
                               1e-5, shift.cuda(), st, cu, kv, slots, max(lengths))
            tol = 2e-5 * max(1.0, float(want.abs().max()))
            assert (h.cpu().double() - want).abs().max() <= tol, (broadcast, with_y)
            assert (st.cpu().double() - want_state).abs().max() <= tol
            if with_y:
                big = torch.stack(new, 1)
                assert (dst.cpu().double() - big).abs().max() <= 2e-5 * max(1.0, float(big.abs().max()))
            # without the shift; without the norm and with equal weights (the sum of the streams)
            src2 = X[:, 0].contiguous().cuda().unsqueeze(1).expand(rows, s, W) if broadcast else X.clone().cuda()
            h = ops.stream_mix(src2, None, y.cuda() if with_y else None, dev["mix"], dev["out"], dev["in"], norm_w.cuda(), groups, 1e-5)
            assert (h.cpu().double() - u).abs().max() <= tol
            h = ops.stream_mix(src2, None, y.cuda() if with_y else None, dev["mix"], dev["out"], None, None, 1, 1e-5)
            assert (h.cpu().double() - sum(new)).abs().max() <= 2e-5 * max(1.0, float(sum(new).abs().max()))


@pytest.mark.parametrize("rows", [2100, 8300])
def test_stream_boundary_over_many_rows(rows):
    """Prompt-sized steps: a workgroup takes two or eight rows in turn, its first row's predecessor computed again; sequence
    borders on and off the groups' borders."""
    from nanovllm import ops

    g = torch.Generator().manual_seed(rows)
    s, W = 3, 12
    lengths = [rows - 1000 - 7 - 8 - 1, 7, 8, 1, 1000]
    starts = [0, 3, 0, 50, 1]
    cu, kv = _step_meta(lengths, starts)
    slots = torch.tensor([3, 1, 0, 5, 4], dtype=torch.int32).cuda()
    X, y = torch.randn(rows, s, W, generator=g), torch.randn(rows, W, generator=g)
    coef = {"in": torch.randn(s, generator=g), "out": torch.randn(s, generator=g), "mix": torch.randn(s, s, generator=g)}
    norm_w, shift, state0 = torch.randn(W, generator=g), torch.rand(W, generator=g), torch.randn(6, W, generator=g)
    dc = {k: v.double() for k, v in coef.items()}
    new = M.streams_write([X[:, i].double() for i in range(s)], y.double(), dc)
    u = M.group_norm(M.streams_read(new, dc), norm_w.double(), 2, 1e-5)
    want, a = u.clone(), 0
    want_state = state0.double().clone()
    for q, (m, p) in enumerate(zip(lengths, starts)):
        prev = state0[int(slots[q])].double() if p > 0 else torch.zeros(W).double()
        ext = torch.cat([prev[None], u[a:a + m]])
        want[a:a + m] = u[a:a + m] + (ext[:-1] - u[a:a + m]) * shift.double()
        want_state[int(slots[q])] = u[a + m - 1]
        a += m
    st, dst = state0.clone().cuda(), torch.empty(rows, s, W).cuda()
    dev = {k: v.cuda() for k, v in coef.items()}
    h = ops.stream_mix(X.cuda(), dst, y.cuda(), dev["mix"], dev["out"], dev["in"], norm_w.cuda(), 2, 1e-5, shift.cuda(), st, cu, kv,
                       slots, max(lengths))
    assert (h.cpu().double() - want).abs().max() <= 1e-4
    assert (st.cpu().double() - want_state).abs().max() <= 1e-4
    assert (dst.cpu().double() - torch.stack(new, 1)).abs().max() <= 1e-4


@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 8, 12), (1, 1, 2, 1), (6, 1, 100, 70), (3, 3, 64, 130), (2, 1, 7, 300)])
def test_differential_heads(H, G, D, Dv):
    """Two maps' read-outs in the attention's order [kv head][map][query head of the group], lambda from its four vectors,
    the unit norm, (1 - diff), a gate number per head."""
    from nanovllm import ops

    g = torch.Generator().manual_seed(H * Dv)
    rows, diff = 5, 0.35
    a = torch.randn(2, rows, H, Dv, generator=g)
    lam = torch.randn(4, D, generator=g) * D ** -0.5
    gate = torch.randn(rows, H + 3, generator=g)
    p = dict(zip(("lq1", "lk1", "lq2", "lk2"), lam.double()))
    o = M.differential(a[0].double(), a[1].double(), p, diff, 1e-5)
    buf = a.view(2, rows, G, H // G, Dv).permute(1, 2, 0, 3, 4).reshape(rows, -1).contiguous().cuda()
    got = ops.diff_heads(buf, lam.cuda(), diff, 1e-5, None, H, G, Dv).cpu().double().view(rows, H, Dv)
    assert (got - o).abs().max() <= 1e-4 * float(o.abs().max())
    got = ops.diff_heads(buf, lam.cuda(), diff, 1e-5, gate.cuda()[:, 3:], H, G, Dv).cpu().double().view(rows, H, Dv)
    want = o * torch.sigmoid(gate[:, 3:].double()).unsqueeze(-1)
    assert (got - want).abs().max() <= 1e-4 * float(o.abs().max())


@pytest.mark.parametrize("H,D,Dv", [(2, 5, 3), (1, 64, 64), (2, 65, 33), (3, 128, 40), (1, 130, 32), (1, 256, 70)])
def test_general_delta_operator(H, D, Dv):
    """Three sequences in a step, one of which starts and two that continue from their slots, in portions around the walk's
    batches of rows, against the plain recurrence of the whole sequences; decays from 0 to 1, removal rates from 0 to 1."""
    from nanovllm import ops

    g = torch.Generator().manual_seed(D * Dv)
    T = {0: 40, 1: 23, 2: 36}
    n, nv = H * D, H * Dv
    data, want = {}, {}
    for i, t in T.items():
        r, k, v = torch.randn(t, n, generator=g), torch.randn(t, n, generator=g), torch.randn(t, nv, generator=g)
        w, a = torch.rand(t, n, generator=g).sqrt(), torch.rand(t, n, generator=g)
        w[:, ::5], a[:, ::7], w[:, 1::9] = 1.0, 1.0, 0.0
        data[i] = (r, k, v, w, a)
        want[i] = M.general_delta_scan(*(x.double().view(t, H, -1) for x in data[i])).reshape(t, nv)
    state = torch.full((4, ops.general_delta_state_elems(H, D, Dv)), 3.0).cuda()   # (a slot's old content must not matter)
    slot = {0: 2, 1: 0, 2: 3}
    at, got = {i: 0 for i in T}, {i: [] for i in T}
    for step in ([(0, 17), (1, 1)], [(1, 2), (2, 16), (0, 1)], [(2, 1)], [(0, 2), (1, 20), (2, 15)], [(2, 4), (0, 20)]):
        ids = [i for i, _ in step]
        lengths, starts = [m for _, m in step], [at[i] for i in ids]
        cu, kv = _step_meta(lengths, starts)
        part = [torch.cat([data[i][j][at[i]:at[i] + m] for i, m in step]) for j in range(5)]
        r, k, v, w, a = part
        proj = torch.cat([torch.zeros(r.shape[0], 3), r, v, a, k], 1).contiguous().cuda()
        out = ops.general_delta(proj, 3, 3 + n + nv + n, 3 + n, 3 + n + nv, w.cuda(), state, cu, kv,
                                torch.tensor([slot[i] for i in ids], dtype=torch.int32).cuda(), H, D, Dv).cpu()
        b = 0
        for i, m in step:
            got[i].append(out[b:b + m])
            b += m
            at[i] += m
    for i in T:
        assert at[i] == T[i]
        assert rel_err(torch.cat(got[i]), want[i]) <= 2e-5, i
    assert bool((state[1] == 3.0).all())


@pytest.mark.parametrize("rows,dtype", [(1, torch.float32), (6, torch.bfloat16), (40, torch.bfloat16), (100, torch.float32),
                                        (100, torch.bfloat16), (600, torch.bfloat16), (1100, torch.float32)])
@pytest.mark.parametrize("N,K", [(37, 20), (150, 72)])
def test_activation_segments(rows, dtype, N, K):
    """Features below the first border as they are, then sigmoid, then tanh; and the decay's activation over all of them; in
    every kernel of the GEMM family (the tile kernels round their input to bf16)."""
    from nanovllm import _C, ops

    g = torch.Generator().manual_seed(N + rows)
    x, w, b = torch.randn(rows, K, generator=g), (torch.randn(N, K, generator=g) * 0.4).to(dtype), torch.randn(N, generator=g)
    z = (x.to(dtype).double() if rows > 8 else x.double()) @ w.double().T + b.double()
    want = torch.cat([z[:, :11], torch.sigmoid(z[:, 11:30]), torch.tanh(z[:, 30:])], 1)
    got = ops.gemm_any_segments(x.cuda(), w.cuda(), b.cuda(), _C.ACT_SIGMOID, 11, _C.ACT_TANH, 30).cpu().double()
    assert (got - want).abs().max() <= 5e-5
    got = ops.gemm_any_segments(x.cuda(), w.cuda(), b.cuda(), _C.ACT_DECAY, 0).cpu().double()
    assert (got - torch.exp(-torch.exp(torch.tensor(-0.5).double()) * torch.sigmoid(z))).abs().max() <= 5e-5


def _paged(x, bs, n_blocks, table, dtype):
    """x [T, heads, d] -> a cache [n_blocks, heads, bs, d] holding token t at page table[t // bs], slot t % bs"""
    T, heads, d = x.shape
    c = torch.zeros(n_blocks, heads, bs, d)
    for t in range(T):
        c[table[t // bs], :, t % bs] = x[t]
    return c.to(dtype).cuda()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dv,chunk", [(4, 2, 32, 16, 40), (2, 1, 64, 64, 33), (6, 3, 12, 10, 70), (4, 2, 32, 32, 64),
                                            (3, 1, 7, 5, 1), (8, 4, 160, 144, 50), (4, 1, 96, 96, 45), (2, 2, 96, 80, 61), (2, 2, 40, 88, 1000), (2, 1, 16, 24, 5)])
def test_attention_in_chunks_with_shared_values(dtype, H, G, D, Dv, chunk):
    """The attention operator with chunked visibility and 2 G key heads over G value heads: prompt portions, single decoded
    rows and a batch of both, over scrambled pages, in every form (matrix cores, 16-byte loads, element-wise), rows on both
    sides of a chunk's border in one tile, against dense fp64 attention."""
    from nanovllm import ops

    g = torch.Generator().manual_seed(D * Dv + H)
    T, bs, scale = 150, 16, 0.5 * (8 / D) ** 0.5
    n_blocks = 12
    table = torch.randperm(n_blocks - 1, generator=g)[:10].tolist()
    q, k, v = torch.randn(T, H, 2, D, generator=g), torch.randn(T, G, 2, D, generator=g), torch.randn(T, G, Dv, generator=g)
    if dtype == torch.bfloat16:
        k, v = k.bfloat16().float(), v.bfloat16().float()
    maps = M.attention_maps(q.double(), k.double(), v.double(), {"scale": scale, "mask": {"size": chunk}})
    order = lambda x: x.view(T, G, H // G, 2, -1).transpose(2, 3).reshape(T, -1).contiguous()   # [kv head][map][head of the group]
    want = order(torch.stack(maps, 2))
    qr = order(q)
    kc, vc = _paged(k.reshape(T, 2 * G, D), bs, n_blocks, table, dtype), _paged(v, bs, n_blocks, table, dtype)
    tables = torch.tensor([table] * 3, dtype=torch.int32)
    edge = chunk if 10 < chunk < 130 else 64
    for lengths, starts in (([T], [0]), ([50], [100]), ([1], [149]), ([1, 1, 1], [149, 16, 0]), ([30, 1, 2], [120, 15, 31]),
                            ([1, 1, 1], [edge - 1, edge, edge + 1]), ([20], [edge - 7]), ([2, 2], [edge - 1, edge])):
        cu, kv = _step_meta(lengths, starts)
        rows = [a + i for a, n in zip(starts, lengths) for i in range(n)]
        got = ops.paged_attention_f32(qr[rows].cuda(), kc, vc, Dv, tables[:len(lengths)].contiguous().cuda(), cu, kv, 2 * H, 2 * G, D,
                                      Dv, bs, 2 ** 31 - 1, scale, value_heads=G, chunk=chunk)
        ref = want[rows]
        assert (got.cpu().double() - ref).abs().max() <= 1e-4 * max(1.0, float(ref.abs().max())), (lengths, starts)
    # a window on top: the nearer of the two limits counts
    window = 23
    cu, kv = _step_meta([T], [0])
    got = ops.paged_attention_f32(qr.cuda(), kc, vc, Dv, tables[:1].contiguous().cuda(), cu, kv, 2 * H, 2 * G, D, Dv, bs, window, scale,
                                  value_heads=G, chunk=chunk).cpu().double().view(T, G, 2, H // G, Dv)
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    ok = M.visible(T, chunk) & (i - j < window)
    for m in range(2):
        for h in range(H):
            s = (q[:, h, m].double() @ k[:, h // (H // G), m].double().T * scale).masked_fill(~ok, float("-inf"))
            ref = torch.softmax(s, -1) @ v[:, h // (H // G)].double()
            assert (got[:, h // (H // G), m, h % (H // G)] - ref).abs().max() <= 1e-4 * max(1.0, float(ref.abs().max()))


def test_head_norm_with_a_weight_of_its_own_per_head():
    from nanovllm import _C, ops

    g = torch.Generator().manual_seed(4)
    H, Dv = 3, 70
    o, gate, w = torch.randn(6, H * Dv, generator=g) * 3, torch.randn(6, H * Dv, generator=g), torch.randn(H * Dv, generator=g)
    want = M.unit(o.double().view(6, H, Dv), 1e-5).reshape(6, -1) * w.double() * torch.sigmoid(gate.double())
    got = o.clone().cuda()
    ops.head_norm_gate(got, gate.cuda(), _C.ACT_SIGMOID, w.cuda(), H, Dv, 1e-5)
    assert (got.cpu().double() - want).abs().max() <= 1e-5


# ------------------------------------------------------------------------------------------------ the engine's cuts
def test_whole_prompt(mixed_model, mixed_replay):
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(70, cfg["vocab"], 2)
    assert_close(r.feed("p", toks, [70]), expected(cfg, w, toks), dtype)


def test_prefill_then_token_by_token(mixed_model, mixed_replay):
    """Decoding through pages and state slots of every pass: 20 prompt tokens, then 60 single tokens (across page borders at
    32, 48, 64 and the borders of chunks of 9 and 17)."""
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(80, cfg["vocab"], 2)
    assert_close(r.feed("d", toks, [20]), expected(cfg, w, toks), dtype)


def test_first_tokens_one_by_one(mixed_model, mixed_replay):
    """A sequence that starts with single tokens: zero matrix states, no previous token, chunks that have just begun."""
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(20, cfg["vocab"], 3)
    assert_close(r.feed("f", toks, []), expected(cfg, w, toks), dtype)


@pytest.mark.parametrize("cuts", [[2, 2, 2, 3, 5, 2, 16, 15, 17, 2], [31, 2, 33], [16, 16, 16, 16], [1, 2, 1, 2, 40],
                                  [6, 1, 7, 7, 6, 2, 14], [9, 8, 17, 2, 9, 18], [8, 2, 16, 2, 9]])
def test_portions(mixed_model, mixed_replay, cuts):
    """Portions down to two tokens, ending on and off page borders (16), chunk borders (9, 17) and the recurrence's batches
    of rows (16)."""
    cfg, w, _ = mixed_model
    dtype, r = mixed_replay
    toks = tokens_of(75, cfg["vocab"], 6)
    got = r.feed("c", toks, cuts)
    assert_close(got, expected(cfg, w, toks), dtype)
    if dtype == "float32":
        assert rel_err(got, r.feed("w", toks, [75])) <= CUT_BAR


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_hundreds_of_keys(dtype):
    """330 tokens with head sizes of every attention kernel, no chunks beside short and long ones, looped: whole, in
    portions, decoded."""
    cfg = config([with_mlp(attention(heads=4, kv_heads=2, dim=32, vdim=48, dims=32, chunk=300), None),
                  with_mlp(delta(heads=2, dim=70), dense(ff=16)),
                  with_mlp(attention(heads=2, kv_heads=2, dim=12, vdim=10, dims=8, chunk=64), None),
                  with_mlp(attention(heads=4, kv_heads=2, dim=64, vdim=64, dims=64, chunk=0, scale=0.15), None),
                  with_mlp(attention(heads=3, kv_heads=1, dim=8, vdim=16, dims=8, chunk=100), None)],
                 width=96, vocab=61, loop=(0, 2, 2), streams=4)
    w = M.random_model(cfg, seed=21)
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
    """A pool of exactly one request's pages and ONE state slot: every request runs in what the previous one left behind."""
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
def _spiky_model(chunk, diff=0.3, far_map=0, heads=2, kv_heads=1, dim=8, vdim=12):
    """One attention layer whose keys and queries are a function of the token alone, in channels the rotation leaves alone:
    in map `far_map` key channel dim - 2 is large for token 1 only and every query looks for it, its score standing out by far
    more than hundreds of other keys weigh together; the other map weighs its keys nearly alike.  Two equal streams, no shift:
    the mixer reads the normed embedding."""
    W, V = 32, 8
    layer = attention(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, chunk=chunk, scale=1.5, diff=diff, dims=4)
    cfg = config([with_mlp(layer, None)], width=W, vocab=V, streams=2, groups=1)
    w = M.random_model(cfg, seed=6)
    e = torch.zeros(V, W)
    e[:, 0] = 0.5
    e[1, 1] = 0.6                                 # token 1 carries a large feature 1
    for t in range(2, V):
        e[t, 2 + t % 4] = 0.3
    w["embed"] = e
    q, k = torch.zeros(heads, 2, dim, W), torch.zeros(kv_heads, 2, dim, W)
    q[:, far_map, dim - 2, 0] = 3.0               # every query: this channel, from the feature every token has
    k[:, far_map, dim - 2, 1] = 1.5               # the key's channel = feature 1 (token 1 only)
    k[:, :, dim - 1, 0] = 1.0                     # every other key lives in another channel
    p = "l0.mix."
    w[p + "q"], w[p + "k"], w["l0.norm1"], w["l0.shift"] = q.reshape(-1, W), k.reshape(-1, W), torch.ones(W), torch.zeros(W)
    for n in ("q.b", "k.b"):
        w[p + n] = torch.zeros_like(w[p + n])
    w[p + "v"] = torch.cat([w[p + "v"][:, :1], 2 * w[p + "v"][:, 1:2], w[p + "v"][:, 2:]], 1)   # (its value stands out too)
    w["l0.hc1.in"], w["l0.hc1.out"], w["l0.hc1.mix"] = torch.full((2,), 0.5), torch.ones(2), 0.1 * torch.eye(2)
    return cfg, {n: t.bfloat16().float() for n, t in w.items()}


@pytest.mark.parametrize("far_map", [0, 1])
@pytest.mark.parametrize("shape", [{}, {"dim": 32, "vdim": 32, "heads": 4, "kv_heads": 2}])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_key_among_hundreds(far_map, shape, dtype):
    """One dominant key at position p in a chunk that still holds it 390 rows on, in either map: a page of the block table
    that is skipped, a batch of keys that is dropped, a first key that is lost, or the wrong map's keys show at full size.  In
    a prompt, in portions, decoded; the key at position 0, at a page's last and first slot."""
    cfg, w = _spiky_model(chunk=100000, far_map=far_map, **shape)
    r = Replay(write_model_dir(cfg, w), dtype, pages=30)
    try:
        for p in (0, 15, 16, 130):
            n = 400
            toks = [2 + (i % 6) for i in range(n)]
            toks[p] = 1
            plain = [2 + (i % 6) for i in range(n)]
            want, without = expected(cfg, w, toks), expected(cfg, w, plain)
            assert rel_err(without[n - 1:], want[n - 1:]) > 0.05, "the far key has no influence: the test's weights are wrong"
            for cuts in ([n], [p + 1, 2, 200, 2], [300] + [1] * 60 + [40], [129, 129, 129]):
                assert_close(r.feed("s", toks, cuts), want, dtype, (p, cuts))
    finally:
        r.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk", [37, 64, 130])
@pytest.mark.parametrize("shape", [{}, {"dim": 32, "vdim": 16}])
def test_chunk_edges(chunk, shape, dtype):
    """The dominant key in the first chunk is seen by that chunk's last row and not by the next chunk's first: the two rows
    differ at full size in the plain statement, and the engine has to agree on both - in a prompt, when the border falls on a
    portion's first or last row or inside it, and decoded token by token; the key as the chunk's first and last position.  Then
    in the second chunk: chunks are counted from the sequence's start, not from a portion's."""
    cfg, w = _spiky_model(chunk=chunk, **shape)
    r = Replay(write_model_dir(cfg, w), dtype, pages=30)
    try:
        for p in (0, 15, chunk - 1, chunk, chunk + 3):
            n = 2 * chunk + 20
            toks = [2 + (i % 6) for i in range(n)]
            toks[p] = 1
            want = expected(cfg, w, toks)
            last = chunk * (p // chunk + 1) - 1           # the last row that sees the key
            if p != last:
                assert rel_err(want[last + 1:last + 2], want[last:last + 1]) > 0.05, "the border does not show: the test's weights are wrong"
            for cuts in ([n], [last, 1, 1], [last + 1, 2], [last, 2, 2], [last - 1, 2, 2], [max(p, 1)] + [1] * (chunk + 5), [p + 2, 3, 2, 2]):
                got = r.feed("s", toks, cuts)
                assert_close(got, want, dtype, (p, cuts))
                assert rel_err(got[last - 1:last + 3], want[last - 1:last + 3]) <= (F32_BAR if dtype == "float32" else 3e-2), (p, cuts)
    finally:
        r.close()


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 8, 12), (4, 2, 32, 32), (6, 1, 32, 16)])
def test_the_two_maps_and_the_heads_are_told_apart(heads, kv_heads, dim, vdim):
    """Only ONE (head, map) pair looks for the dominant key, each in turn: a map taken for the other (a sign of lambda), heads
    regrouped, or another head's gate moves the rows at full size."""
    for h, m in ((0, 0), (0, 1), (heads - 1, 0), (heads - 1, 1), (1, 1)):
        cfg, w = _spiky_model(chunk=1000, far_map=m, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim)
        q = w["l0.mix.q"].view(heads, 2, dim, -1).clone()
        q[[i for i in range(heads) if i != h]] = 0.0
        w["l0.mix.q"] = q.reshape(-1, q.shape[-1])
        gate = torch.zeros(heads, 32)
        gate[h, 0] = 3.0                                         # the gates differ by head
        gate[(h + 1) % heads, 0] = -3.0
        w["l0.mix.g"] = gate.bfloat16().float()
        toks = [2 + (i % 6) for i in range(90)]
        toks[30] = 1
        want = expected(cfg, w, toks)
        other = dict(w)
        other["l0.mix.q"] = q.flip(1).reshape(-1, q.shape[-1])
        other["l0.mix.k"] = w["l0.mix.k"].view(kv_heads, 2, dim, -1).flip(1).reshape(-1, 32)
        assert rel_err(expected(cfg, other, toks)[40:], want[40:]) > 0.05, "the maps do not show: the test's weights are wrong"
        r = Replay(write_model_dir(cfg, w), "float32", pages=30)
        try:
            for cuts in ([90], [31, 2, 40], [35]):
                assert rel_err(r.feed("t", toks, cuts), want) <= F32_BAR, (h, m, cuts)
        finally:
            r.close()


def test_the_shift_reaches_over_portion_edges():
    """A shift of one: what a mixer reads is the PREVIOUS token's row alone.  Portions of one to three tokens take it from the
    slot; a row that is stored after its own shift, not advanced by a short portion, shared between passes or taken from
    another slot shows at full size.  In every kind of layer, under a loop."""
    cfg = config([with_mlp(delta(heads=2, dim=12), None), with_mlp(attention(heads=2, kv_heads=2, dim=12, vdim=12, dims=4, chunk=30), dense(ff=16))],
                 width=40, vocab=29, loop=(0, 2, 2))
    w = M.random_model(cfg, seed=12)
    flat = dict(w)
    for i in range(2):
        w[f"l{i}.shift"], flat[f"l{i}.shift"] = torch.ones(40), torch.zeros(40)
    toks = tokens_of(40, 29, 3)
    want = expected(cfg, w, toks)
    assert rel_err(expected(cfg, flat, toks)[8:], want[8:]) > 0.05, "the shift has no influence: the test's weights are wrong"
    r = Replay(write_model_dir(cfg, w), "float32")
    try:
        for cuts in ([40], [4, 1, 1, 1, 2, 3, 2, 4, 5, 6], [1, 1, 1, 1, 1, 35], [3, 3, 3, 3, 3, 2, 2, 2, 19], []):
            assert rel_err(r.feed("t", toks, cuts), want) <= F32_BAR, cuts
        a, b = tokens_of(30, 29, 4), tokens_of(30, 29, 5)     # two sequences side by side, portions of two; then single tokens
        for size in (2, 1, 7):
            got = {"a": [], "b": []}
            for at in range(0, 30, size):
                out = r.step([("a", a[at:at + size]), ("b", b[at:at + size])])
                got["a"].append(out["a"])
                got["b"].append(out["b"])
            for k in ("a", "b"):
                r.scheduler.finish(r.live.pop(k))
            assert rel_err(torch.cat(got["a"]), expected(cfg, w, a)) <= F32_BAR, size
            assert rel_err(torch.cat(got["b"]), expected(cfg, w, b)) <= F32_BAR, size
    finally:
        r.close()


def test_far_write_survives_in_the_state():
    """A delta rule that hardly fades or removes: what position 2 wrote still shows 150 tokens later; a state lost or cleared
    at a portion's start, a slot mixed up in a batch, or a pass reading another pass's state shows at full size."""
    cfg = config([with_mlp(delta(heads=2, dim=18), None)], width=48, vocab=31, loop=(0, 1, 2))
    w = M.random_model(cfg, seed=9)
    w["l0.mix.w0"], w["l0.mix.a.b"] = torch.full((36,), -9.0), torch.full((36,), -5.0)
    toks = tokens_of(160, 31, 7)
    other = list(toks)
    other[2] = (toks[2] + 1) % 31
    want, want_other = expected(cfg, w, toks), expected(cfg, w, other)
    assert rel_err(want_other[150:], want[150:]) > 1e-3, "the early token has no influence: the test's weights are wrong"
    r = Replay(write_model_dir(cfg, w), "float32", pages=24)
    try:
        assert rel_err(r.feed("a", toks, [160]), want) <= F32_BAR
        assert rel_err(r.feed("b", toks, [5, 70, 2, 2, 60]), want) <= F32_BAR
        for cut in (40, 1):   # two sequences that differ in the early token only, side by side in every step
            at, got = 0, {"x": [], "y": []}
            while at < 160:
                n = min(cut, 160 - at)
                out = r.step([("y", other[at:at + n]), ("x", toks[at:at + n])])
                got["x"].append(out["x"])
                got["y"].append(out["y"])
                at += n
            for k in ("x", "y"):
                r.scheduler.finish(r.live.pop(k))
            assert rel_err(torch.cat(got["x"]), want) <= F32_BAR and rel_err(torch.cat(got["y"]), want_other) <= F32_BAR
    finally:
        r.close()


def test_a_key_is_removed_along_itself_at_its_channels_rates():
    """Two tokens take turns, each always with the same key, no decay: with a removal rate of nearly one a repeated key
    replaces its value, with nearly zero the values pile up, with rates that differ by channel in between.  Removing along k
    instead of the unit key, or after the decay and the write, moves every row."""
    cfg = config([with_mlp(delta(heads=1, dim=24), None)], width=48, vocab=31, streams=1, groups=1)
    w0 = M.random_model(cfg, seed=10)
    w0["l0.mix.w0"], w0["l0.shift"] = torch.full((24,), -12.0), torch.zeros(48)
    w0["l0.mix.a"] = torch.zeros_like(w0["l0.mix.a"])
    toks = [3, 7] * 30 + tokens_of(10, 31, 2)
    rows = []
    for bias in (torch.full((24,), 6.0), torch.full((24,), -6.0), torch.linspace(-6, 6, 24)):
        w = dict(w0)
        w["l0.mix.a.b"] = bias.bfloat16().float()
        want = expected(cfg, w, toks)
        rows.append(want)
        r = Replay(write_model_dir(cfg, w), "float32")
        try:
            for cuts in ([70], [17, 2, 30], []):
                assert rel_err(r.feed("r", toks, cuts), want) <= F32_BAR, cuts
        finally:
            r.close()
    for a in range(3):
        for b in range(a):
            assert rel_err(rows[a][20:], rows[b][20:]) > 0.05, "the removal has no influence: the test's weights are wrong"


def test_streams_are_mixed_the_right_way_round():
    """A mix matrix that moves the streams in a cycle, unequal weights in and out: the transposed matrix, an update from
    streams that are already new, or one sublayer's coefficients used for the other move every row."""
    cfg = config([with_mlp(attention(), dense()), with_mlp(delta(), dense())], streams=4)
    w = M.random_model(cfg, seed=14)
    for i in range(2):
        for q, roll in (("hc1", 1), ("hc2", 2)):
            w[f"l{i}.{q}.mix"] = (torch.roll(torch.eye(4), roll, 1) + 0.25 * torch.eye(4)).bfloat16().float()
            w[f"l{i}.{q}.in"], w[f"l{i}.{q}.out"] = torch.tensor([1.0, 0.5, -0.25, 0.125]), torch.tensor([2.0, -1.0, 0.5, 0.25])
    toks = tokens_of(30, 97, 4)
    want = expected(cfg, w, toks)
    other = {k: (v.T.contiguous() if k.endswith("hc1.mix") else v) for k, v in w.items()}
    assert rel_err(expected(cfg, other, toks), want) > 0.05
    r = Replay(write_model_dir(cfg, w), "float32")
    try:
        for cuts in ([30], [17, 2], []):
            assert rel_err(r.feed("v", toks, cuts), want) <= F32_BAR
    finally:
        r.close()


# ------------------------------------------------------------------------------------------------ the engine's own entry point
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_llm(mixed_model, dtype):
    """LLM.generate: the scheduler's prefill and decode steps, its page and slot managers, captured decode steps, the sampler.
    Every generated token must be the plain model's best token given the same history (or within the sampler's bf16 logits
    of it)."""
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
                if row.max() - row[tok] > (0.02 if dtype == "float32" else 0.06) * max(1.0, float(row.abs().max())):
                    off.append((len(prompt), i, tok, int(row.argmax()), float(row.max() - row[tok])))
        assert not off, off
    finally:
        llm.exit()


def test_captured_decode_steps_equal_eager(mixed_model):
    """Decode steps replay hipGraphs padded to a batch bucket (3 live requests in the bucket of 4, the padded row writing the
    spare state slot): same tokens and the same logits as eager launches, over several replays with eager prefill steps
    between them."""
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


def test_recurrent_layers_only_through_llm():
    """A model without attention: pages cost nothing, the default pool size is what the longest sequences ask for."""
    from nanovllm import LLM, SamplingParams

    cfg = config([with_mlp(delta(), dense()), with_mlp(delta(heads=2, dim=40), None)], streams=2)
    w = M.random_model(cfg, seed=17)
    llm = LLM(write_model_dir(cfg, w), dtype="float32", kvcache_block_size=16, max_num_seqs=2, max_model_len=64,
              max_num_batched_tokens=128, warmup=False)
    try:
        prompts = [tokens_of(n, cfg["vocab"], 40 + n) for n in (5, 30, 12)]
        for prompt, out in zip(prompts, llm.generate(prompts, SamplingParams(max_tokens=6, greedy=True, ignore_eos=True), use_tqdm=False)):
            logits = expected(cfg, w, prompt + out["token_ids"])
            for i, tok in enumerate(out["token_ids"]):
                row = logits[len(prompt) - 1 + i]
                assert row.max() - row[tok] <= 0.02 * max(1.0, float(row.abs().max()))
    finally:
        llm.exit()


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
