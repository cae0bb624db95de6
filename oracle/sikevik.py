"""Plain, slow statement of the Sikevik design (torch on CPU, float64 by default): one function per mechanism.

TEST INFRASTRUCTURE: nothing of the product path imports this file and it imports nothing of the product path.
One sequence at a time, whole, with dense [T, T] score matrices.

Notation (W x means `x @ W.T`, weights stored [out, in]; t = position, counted from 0):

  norm          n(x; w) = x / sqrt(mean(x^2) + eps) * w
  embedding     e_t = scale * E[token_t] + s_t,  s_t[2i] = sin(t f_i),  s_t[2i + 1] = cos(t f_i),  f_i = 10000^(-2 i / width)
  layer         x <- x + n(mixer(n(x; w_1)); w_1b);   x <- x + n(ff(n(x; w_2)); w_2b)        (a layer may have no feed-forward)
  order         layers [0, start), then `times` passes over [start, stop) with the same weights, then [stop, n);
                every pass begins with  x <- W_loop [x | e]
  attention     q_h = n(W_q h; w_qn) per head of `dim` channels, k likewise with w_kn (one weight for all heads), no positions;
                s_ij = scale q_i . k_j  for the visible keys  j <= i and (i - j < window or j < kept);
                p_ij = exp(s_ij) / (1 + sum_j' exp(s_ij'));   out = W_o concat_h(sum_j p_ij v_j)
  dense ff      W_d gelu(W_u h),  gelu(z) = z / 2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))
  sparse ff     s = softmax(W_r h);  the `top` largest, weighing  a s_k / (sum of the chosen s + 1e-20);
                out = sum_k weight_k f(h; e_k) + f(h; shared),   f(h; e) = W_d (max(W_u h, 0))^2
  output        logits = E n(x; w_final)      (E: the embedding table, unscaled)
"""
from __future__ import annotations

import math

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return torch.clamp(z, min=0) ** 2


def sinusoids(T, width, dtype=torch.float64):
    """[T, width]: sine and cosine of position * frequency in neighbouring channels"""
    out = torch.zeros(T, width, dtype=dtype)
    t = torch.arange(T, dtype=dtype)
    for c in range(width):
        angle = t * 10000.0 ** (-2.0 * (c // 2) / width)
        out[:, c] = torch.sin(angle) if c % 2 == 0 else torch.cos(angle)
    return out


def embed(weights, tokens, scale):
    E = weights["embed"]
    return E[torch.as_tensor(tokens, dtype=torch.long)] * scale + sinusoids(len(tokens), E.shape[1], E.dtype)


def begin_pass(x, e, w_loop):
    return torch.cat([x, e], -1) @ w_loop.T


def visible(T, window, kept):
    """[T, T] bool: key j is seen from position i (window None: every key up to i)"""
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    if window is None:
        return j <= i
    return (j <= i) & ((i - j < window) | (j < kept))


def softmax_with_one(s):
    """exp(s) / (1 + sum exp(s)) along the last axis; masked scores are -inf"""
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0)
    ex = torch.exp(s - m)
    return ex / (torch.exp(-m) + ex.sum(-1, keepdim=True))


def attention_mixer(h, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rms_norm((h @ p["q"].T).view(T, H, D), p["q.norm"], eps)
    k = rms_norm((h @ p["k"].T).view(T, G, D), p["k.norm"], eps).repeat_interleave(H // G, 1)
    v = (h @ p["v"].T).view(T, G, Dv).repeat_interleave(H // G, 1)
    mask = m.get("mask") or {}
    ok = visible(T, int(mask["size"]) if mask else None, int(mask.get("keep_first", 0)))
    s = torch.einsum("ihd,jhd->hij", q, k) * float(m["scale"])
    pr = softmax_with_one(s.masked_fill(~ok, float("-inf")))
    return torch.einsum("hij,jhd->ihd", pr, v).reshape(T, H * Dv) @ p["o"].T


def dense_ff(h, p, ml):
    return gelu_tanh(h @ p["up"].T) @ p["down"].T


def expert_ff(h, p, name):
    return relu_squared(h @ p[name + ".up"].T) @ p[name + ".down"].T


def route(h, p, r):
    """-> (chosen experts [T, top], their weights [T, top])"""
    s = torch.softmax(h @ p["router"].T, -1)
    idx = torch.topk(s, int(r["top"]), dim=-1).indices
    w = torch.gather(s, 1, idx)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20) * float(r.get("scale", 1.0))


def sparse_ff(h, p, ml):
    idx, wts = route(h, p, ml["router"])
    out = expert_ff(h, p, "shared") if ml.get("shared") else torch.zeros_like(h)
    for t in range(h.shape[0]):
        for k in range(idx.shape[1]):
            out[t] = out[t] + wts[t, k] * expert_ff(h[t:t + 1], p, f"e{int(idx[t, k])}")[0]
    return out


def feed_forward(h, p, ml):
    return dense_ff(h, p, ml) if ml["kind"] == "dense" else sparse_ff(h, p, ml)


def sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


MIXERS = {"attention": attention_mixer}


def layer_runs(config):
    """[(layer index, pass number or None)] in execution order; the pass number is set on a pass's first layer"""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    runs = [(i, None) for i in range(a)]
    for t in range(times):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def forward(config, weights, tokens, dtype=torch.float64, collect=None):
    """Logits [T, vocab] of one sequence; `collect` (a list) receives the residual stream after every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    e = embed(w, tokens, float((config.get("embedding") or {}).get("scale", 1.0)))
    x = e
    for i, t in layer_runs(config):
        if t is not None:
            x = begin_pass(x, e, w["loop.in"])
        spec, p = config["layers"][i], sub(w, f"l{i}.")
        y = MIXERS[spec["type"]](rms_norm(x, p["norm1"], eps), sub(p, "mix."), spec["mixer"], eps)
        x = x + rms_norm(y, p["norm1b"], eps)
        if spec.get("mlp") is not None:
            y = feed_forward(rms_norm(x, p["norm2"], eps), sub(p, "mlp."), spec["mlp"])
            x = x + rms_norm(y, p["norm2b"], eps)
        if collect is not None:
            collect.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T


def tensor_shapes(config):
    """name -> shape of a checkpoint of this configuration"""
    W, V = int(config["width"]), int(config["vocab"])
    out = {"embed": (V, W), "final.norm": (W,)}
    if config.get("loop"):
        out["loop.in"] = (W, 2 * W)
    for i, spec in enumerate(config["layers"]):
        pre, m = f"l{i}.", spec["mixer"]
        if spec["type"] != "attention":
            raise ValueError(spec["type"])
        H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
        out.update({pre + "norm1": (W,), pre + "norm1b": (W,), pre + "mix.q": (H * D, W), pre + "mix.k": (G * D, W),
                    pre + "mix.v": (G * Dv, W), pre + "mix.q.norm": (D,), pre + "mix.k.norm": (D,), pre + "mix.o": (W, H * Dv)})
        ml = spec.get("mlp")
        if ml is None:
            continue
        out.update({pre + "norm2": (W,), pre + "norm2b": (W,)})

        def plain(name, ff):
            out.update({f"{pre}mlp.{name}up": (ff, W), f"{pre}mlp.{name}down": (W, ff)})

        if ml["kind"] == "dense":
            plain("", int(ml["ff"]))
            continue
        out[pre + "mlp.router"] = (int(ml["router"]["experts"]), W)
        for e in range(int(ml["router"]["experts"])):
            plain(f"e{e}.", int(ml["expert"]["ff"]))
        if ml.get("shared"):
            plain("shared.", int(ml["shared"]["ff"]))
    return out


def random_model(config, seed=0, overrides=None):
    """Random bf16-representable weights (so that a bf16 checkpoint of them is exact) under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm1b", "norm2b"):   # sublayer outputs below the stream: an expert swapped at a router's near-tie in
            t = (1 + torch.randn(shape, generator=g) * 0.2) * 0.25    # bf16 serving moves a row by little
        elif "norm" in leaf:
            t = 1 + torch.randn(shape, generator=g) * 0.2
        elif name == "embed":
            t = torch.randn(shape, generator=g) * 0.5
        else:
            t = torch.randn(shape, generator=g) * (1.2 * shape[-1] ** -0.5)
        out[name] = t.to(torch.bfloat16).to(torch.float32)
    for k, v in (overrides or {}).items():
        out[k] = v.to(torch.bfloat16).to(torch.float32)
    return out
