"""Plain, slow statement of the Munizen design (torch on CPU, float64 by default): one function per mechanism.

TEST INFRASTRUCTURE: nothing of the product path imports this file and it imports nothing of the product path.
One sequence at a time, whole, with dense [T, T] score matrices and Python loops over time for the recurrence.

Notation (W x means `x @ W.T`, weights stored [out, in]; t = position, counted from 0; `.b` a bias):

  norm          n(x; w): x cut into `groups` equal consecutive parts, each part p / sqrt(mean(p^2) + eps); the whole times w
  streams       X_1 .. X_s, all the embedding row at the start.  A sublayer f with coefficients in [s], out [s], mix [s, s]:
                y = f(n(sum_i in_i X_i)),   X_j <- sum_i mix[i, j] X_i + out_j y   (all j from the old streams);
                at the end x = sum_i X_i
  layer         f_1 = mixer behind the token shift,  f_2 = feed-forward (a layer may have none)
  token shift   h_t <- h_t + (h_{t-1} - h_t) * shift per channel, h_{-1} = 0, h_{t-1} as it was before its own shift
  order         layers [0, start), then `times` passes over [start, stop) with the same weights, then [stop, n)
  rotation      a = t f_i,  f_i = base^(-2 i / dims); pairs (i, i + dims / 2) of the first `dims` channels:
                (u, v) -> (u cos a - v sin a, v cos a + u sin a)
  attention     q [heads][2][dim], k [kv_heads][2][dim], v [kv_heads][vdim] = W h + b, both maps of q and k rotated;
                map m of head h: s_ij = scale q_i . k_j over the keys j <= i of i's chunk (floor(i / size) = floor(j / size)),
                a_m = softmax(s) v;  lam = exp(lq1 . lk1) - exp(lq2 . lk2) + diff;  o = a_1 - lam a_2;
                o <- o / sqrt(mean(o^2) + eps) * (1 - diff);  o <- o sigmoid(W_g h)_head;  out = W_o concat(o) + b
  general delta r, k, v = W h;  w = exp(-exp(-1/2) sigmoid(W_2 tanh(W_1 h) + w0));  a = sigmoid(W_a h + b);
                u = k / sqrt(sum k^2 + 1e-6) per head;
                S_t = diag(w_t) S_{t-1} - (a_t u_t) (u_t^T S_{t-1}) + k_t v_t^T;   o_t = S_t^T r_t
                out = W_o (concat_h(o_h / sqrt(mean(o_h^2) + eps)) * norm * sigmoid(W_g h))
  dense ff      W_d (silu(W_gate h) * (W_up h))
  output        logits = head n(x; w_final)
"""
from __future__ import annotations

import math

import torch


def unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    return unit(x.reshape(*x.shape[:-1], groups, -1), eps).reshape(x.shape) * w


def silu(z):
    return z * torch.sigmoid(z)


def token_shift(h, shift):
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (prev - h) * shift


def streams_start(e, s):
    return [e.clone() for _ in range(s)]


def streams_read(X, p):
    return sum(p["in"][i] * X[i] for i in range(len(X)))


def streams_write(X, y, p):
    return [sum(p["mix"][i, j] * X[i] for i in range(len(X))) + p["out"][j] * y for j in range(len(X))]


def rotate(x, rot):
    """x [T, heads, dim] at positions 0 .. T - 1"""
    dims = int(rot["dims"]) if rot else 0
    if dims == 0:
        return x
    T, half = x.shape[0], dims // 2
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    ang = torch.arange(T, dtype=torch.float64).view(T, 1) * f
    cos, sin = torch.cos(ang).to(x.dtype).unsqueeze(1), torch.sin(ang).to(x.dtype).unsqueeze(1)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], -1)


def visible(T, chunk):
    """[T, T] bool: key j is seen from position i"""
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    ok = j <= i
    if chunk is not None:
        ok &= (i // chunk) == (j // chunk)
    return ok


def chunk_of(m):
    return int(m["mask"]["size"]) if m.get("mask") else None


def attention_maps(q, k, v, m):
    """q [T, H, 2, D], k [T, G, 2, D], v [T, G, Dv] (rotated) -> the two maps' read-outs [2][T, H, Dv]"""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    ok = visible(T, chunk_of(m))
    out = []
    for i in range(2):
        s = torch.einsum("ihd,jhd->hij", q[:, :, i], k[:, :, i]) * float(m["scale"])
        p = torch.softmax(s.masked_fill(~ok, float("-inf")), -1)
        out.append(torch.einsum("hij,jhd->ihd", p, v))
    return out


def differential(a1, a2, p, diff, eps):
    lam = torch.exp((p["lq1"] * p["lk1"]).sum()) - torch.exp((p["lq2"] * p["lk2"]).sum()) + diff
    return unit(a1 - lam * a2, eps) * (1 - diff)


def attention_mixer(h, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = h @ p["q"].T + p["q.b"], h @ p["k"].T + p["k.b"], h @ p["v"].T + p["v.b"]
    q = rotate(q.view(T, H * 2, D), m.get("rot")).view(T, H, 2, D)
    k = rotate(k.view(T, G * 2, D), m.get("rot")).view(T, G, 2, D)
    a1, a2 = attention_maps(q, k, v.view(T, G, Dv), m)
    o = differential(a1, a2, p, float(m["diff"]), eps)
    o = o * torch.sigmoid(h @ p["g"].T).unsqueeze(-1)
    return o.reshape(T, H * Dv) @ p["o"].T + p["o.b"]


def general_delta_scan(r, k, v, w, a):
    """all [T, H, D] -> o [T, H, D]"""
    T, H, D = r.shape
    u = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    S = torch.zeros(H, D, v.shape[-1], dtype=r.dtype)
    out = []
    for t in range(T):
        seen = torch.einsum("hdv,hd->hv", S, u[t])
        S = w[t].unsqueeze(-1) * S - (a[t] * u[t]).unsqueeze(-1) * seen.unsqueeze(1) + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out.append(torch.einsum("hdv,hd->hv", S, r[t]))
    return torch.stack(out)


def general_delta_mixer(h, p, m, eps):
    T = h.shape[0]
    H, D = int(m["heads"]), int(m["dim"])
    r, k, v = ((h @ p[n].T).view(T, H, D) for n in ("r", "k", "v"))
    w = torch.exp(-math.exp(-0.5) * torch.sigmoid(torch.tanh(h @ p["w1"].T) @ p["w2"].T + p["w0"])).view(T, H, D)
    a = torch.sigmoid(h @ p["a"].T + p["a.b"]).view(T, H, D)
    o = unit(general_delta_scan(r, k, v, w, a), eps).reshape(T, H * D)
    return (o * p["norm"] * torch.sigmoid(h @ p["g"].T)) @ p["o"].T


def dense_ff(h, p):
    return (silu(h @ p["gate"].T) * (h @ p["up"].T)) @ p["down"].T


def sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


MIXERS = {"attention": attention_mixer, "general_delta": general_delta_mixer}


def layer_runs(config):
    """layer indices in execution order"""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return list(range(n))
    a, b = int(loop["start"]), int(loop["stop"])
    return list(range(a)) + list(range(a, b)) * int(loop["times"]) + list(range(b, n))


def forward(config, weights, tokens, dtype=torch.float64, collect=None):
    """Logits [T, vocab] of one sequence; `collect` (a list) receives the sum of the streams after every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps, groups = float(config["norm"]["eps"]), int(config["norm"]["groups"])
    X = streams_start(w["embed"][torch.as_tensor(tokens, dtype=torch.long)], int(config["streams"]))
    for i in layer_runs(config):
        spec, p = config["layers"][i], sub(w, f"l{i}.")
        c = sub(p, "hc1.")
        h = token_shift(group_norm(streams_read(X, c), p["norm1"], groups, eps), p["shift"])
        X = streams_write(X, MIXERS[spec["type"]](h, sub(p, "mix."), spec["mixer"], eps), c)
        if spec.get("mlp") is not None:
            c = sub(p, "hc2.")
            X = streams_write(X, dense_ff(group_norm(streams_read(X, c), p["norm2"], groups, eps), sub(p, "mlp.")), c)
        if collect is not None:
            collect.append(sum(X))
    return group_norm(sum(X), w["final.norm"], groups, eps) @ w["head"].T


def tensor_shapes(config, rank=6):
    """name -> shape of a checkpoint of this configuration; rank: of the decay's low-rank projection (a number for every
    layer, or a dict layer -> number)"""
    W, V, s = int(config["width"]), int(config["vocab"]), int(config["streams"])
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    for i, spec in enumerate(config["layers"]):
        pre, m = f"l{i}.", spec["mixer"]
        mix = pre + "mix."
        out.update({pre + "norm1": (W,), pre + "shift": (W,)})
        if spec["type"] == "attention":
            H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
            for n, rows in (("q", H * 2 * D), ("k", G * 2 * D), ("v", G * Dv)):
                out.update({mix + n: (rows, W), mix + n + ".b": (rows,)})
            out.update({mix + n: (D,) for n in ("lq1", "lk1", "lq2", "lk2")})
            out.update({mix + "g": (H, W), mix + "o": (W, H * Dv), mix + "o.b": (W,)})
        elif spec["type"] == "general_delta":
            n = int(m["heads"]) * int(m["dim"])
            R = rank[i] if isinstance(rank, dict) else rank
            out.update({mix + x: (n, W) for x in ("r", "k", "v", "g", "a")})
            out.update({mix + "a.b": (n,), mix + "w1": (R, W), mix + "w2": (n, R), mix + "w0": (n,), mix + "norm": (n,),
                        mix + "o": (W, n)})
        else:
            raise ValueError(spec["type"])
        subs = ["hc1"]
        if spec.get("mlp") is not None:
            F = int(spec["mlp"]["ff"])
            out.update({pre + "norm2": (W,), pre + "mlp.gate": (F, W), pre + "mlp.up": (F, W), pre + "mlp.down": (W, F)})
            subs.append("hc2")
        for c in subs:
            out.update({pre + c + ".in": (s,), pre + c + ".out": (s,), pre + c + ".mix": (s, s)})
    return out


def random_model(config, seed=0, rank=6, overrides=None):
    """Random bf16-representable weights (so that a bf16 checkpoint of them is exact) under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config, rank).items():
        leaf, s = name.rsplit(".", 1)[-1], int(config["streams"])
        x = torch.randn(shape, generator=g)
        if "norm" in leaf:
            t = 1 + 0.2 * x
        elif leaf == "shift":
            t = torch.rand(shape, generator=g)
        elif leaf == "in":
            t = (1 + 0.4 * x) / s
        elif leaf == "out":
            t = 1 + 0.4 * x
        elif leaf == "mix" and len(shape) == 2 and name.split(".")[1].startswith("hc"):
            t = 0.85 * torch.eye(s) + 0.15 / s + 0.1 * x * s ** -0.5
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.5 * x * shape[0] ** -0.25
        elif leaf in ("b", "w0"):
            t = 0.7 * x
        elif name == "embed":
            t = 0.5 * x
        elif leaf in ("down", "o"):
            t = x * (0.7 * shape[-1] ** -0.5)
        else:
            t = x * (1.5 * shape[-1] ** -0.5)
        out[name] = t.to(torch.bfloat16).to(torch.float32)
    for k, v in (overrides or {}).items():
        out[k] = v.to(torch.bfloat16).to(torch.float32)
    return out
