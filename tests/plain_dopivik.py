"""A plain implementation of the Dopivik decoder: whole sequences, no cache, one function per mechanism, token by token
where there is a recurrence, torch on the CPU in the precision of the tensors it is given (float32 or float64).  It
shares no code with the engine.  ``round_to`` (a 16-bit type) rounds the activations where a 16-bit engine stores them
(the rows that enter a product, q, k and v of the attention, the convolved rows, the values of time mixing, the
mixers' outputs before their last product) and nothing else: the difference to the unrounded run says how much of a 16-bit engine's error is that
rounding alone.

Notation: x is the residual stream [T, width]; LN(v) = (v - mean) / sqrt(var + eps) * w + b; N(v) = v / sqrt(mean(v^2) + eps).

    embedding:  x = table[token] * scale
    layer:      x <- x + LN_1b(mixer(LN_1(x)));   x <- x + LN_2b(W_down relu(W_up LN_2(x))^2)   (the second only with a feed-forward)
    parallel:   (N(left) w_left + N(right) w_right) / 2
      left:     softmax attention within chunks of positions, q and k turned in pairs (i, i + dims/2), scores
                c tanh(q.k scale / c), the heads' outputs times sigmoid(W_g h), then W_o
      right:    S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q   (q, k, v convolved, silu; q, k unit vectors)
    mamba1:     S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;  y_c = S[c] . C + D_c x_c
    wkv:        o = (S + diag(u) k v^T)^T r;  S <- diag(w) S + k v^T, inputs mixed with the token before
    logits:     W_head LN(x)
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F


def rounded(t, round_to):
    return t if round_to is None else t.to(round_to).to(t.dtype)


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


def frequencies(dims, base, dtype=torch.float64):
    i = torch.arange(dims // 2, dtype=torch.float64)
    return (torch.tensor(float(base), dtype=torch.float64) ** (-2.0 * i / dims)).to(dtype)


def rotate(x, positions, base, dims):
    """x [T, heads, d]: dimension i of the first ``dims`` is paired with i + dims / 2."""
    if dims == 0:
        return x
    half = dims // 2
    angle = positions.to(torch.float64)[:, None] * frequencies(dims, base)[None, :]
    cos, sin = torch.cos(angle).to(x.dtype)[:, None, :], torch.sin(angle).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def chunk_mask(n, size):
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i // size == j // size)


def capped(s, cap):
    return s if cap is None else cap * torch.tanh(s / cap)


def capped_attention(q, k, v, scale, cap, visible):
    """q [T, H, d], k [T, G, d], v [T, G, dv], visible [T, T] (row: query).  Returns [T, H, dv]."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = capped((q[:, h] @ k[:, g].T) * scale, cap).masked_fill(~visible, -math.inf)
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (e / e.sum(-1, keepdim=True)) @ v[:, g]
    return out


def gated_chunk_attention(h, W, m, eps, round_to=None):
    """The left mixer; ``W`` its tensors by local name."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ W["q"].T).view(T, H, d), (h @ W["k"].T).view(T, G, d), (h @ W["v"].T).view(T, G, dv)
    if m.get("rot"):
        pos = torch.arange(T)
        q, k = (rotate(t, pos, m["rot"]["base"], m["rot"]["dims"]) for t in (q, k))
    q, k, v = (rounded(t, round_to) for t in (q, k, v))
    o = capped_attention(q, k, v, m["scale"], m.get("softcap"), chunk_mask(T, m["mask"]["size"]))
    o = o.reshape(T, H * dv) * torch.sigmoid(h @ W["g"].T)
    return rounded(o, round_to) @ W["o"].T


def causal_conv(u, w, b=None):
    """u [T, C], w [C, taps]: y_t = b + sum_j w[:, j] u_(t - taps + 1 + j), zeros before the first token."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros((taps - 1, u.shape[1]), dtype=u.dtype), u], 0)
    y = sum(padded[j:j + u.shape[0]] * w[:, j] for j in range(taps))
    return y if b is None else y + b


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, beta, g, state=None):
    """q, k [T, G, d] (q already scaled), v [T, H, dv], beta, g [T, H].  Returns o [T, H, dv] and the state [H, d, dv]."""
    T, H, dv = v.shape
    G, d = k.shape[1:]
    S = torch.zeros((H, d, dv), dtype=v.dtype) if state is None else state.clone()
    idx = torch.arange(H) // (H // G)
    out = torch.zeros((T, H, dv), dtype=v.dtype)
    for t in range(T):
        kt, qt = k[t, idx], q[t, idx]
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, kt))
        S = S + kt[:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, qt)
    return out, S


def gated_delta(h, W, m, eps, round_to=None):
    """The right mixer."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W[n].T, W[n + ".conv"])) for n in ("q", "k", "v"))
    q, k, v = (rounded(t, round_to) for t in (q, k, v))
    q, k = unit(q.view(T, G, d)) * d ** -0.5, unit(k.view(T, G, d))
    beta = torch.sigmoid(h @ W["b"].T)
    g = torch.exp(-torch.exp(W["A_log"]) * F.softplus(h @ W["a"].T + W["dt_bias"]))
    o, _ = delta_rule(q, k, v.view(T, H, dv), beta, g)
    o = (rms(o, eps) * W["norm"]).reshape(T, H * dv) * silu(h @ W["g"].T)
    return rounded(o, round_to) @ W["o"].T


def sub(W, prefix):
    return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}


def parallel(h, W, m, eps, round_to=None):
    left = gated_chunk_attention(h, sub(W, "left."), m["left"], eps, round_to)
    right = gated_delta(h, sub(W, "right."), m["right"], eps, round_to)
    return 0.5 * (rms(left, eps) * W["left.out"] + rms(right, eps) * W["right.out"])


def selective_scan(x, dt, A, B, C, D, state=None):
    """x, dt [T, c], A [c, n], B, C [T, n], D [c].  Returns y [T, c] and the state [c, n]."""
    S = torch.zeros_like(A) if state is None else state.clone()
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba1(h, W, m, eps, round_to=None):
    inner, n, r = m["inner"], m["state"], m["dt_rank"]
    xz = h @ W["in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = rounded(silu(causal_conv(x, W["conv"], W["conv.b"])), round_to)
    dbc = x @ W["x"].T
    dt = F.softplus(rounded(dbc[:, :r], round_to) @ W["dt"].T + W["dt.b"])
    y, _ = selective_scan(x, dt, -torch.exp(W["A_log"]), dbc[:, r:r + n], dbc[:, r + n:], W["D"])
    return rounded(y * silu(z), round_to) @ W["o"].T


def wkv_rule(r, k, v, w, u, state=None):
    """r, k, v, w [T, H, d], u [H, d].  Returns o [T, H, d] and the state [H, d, d]."""
    T, H, d = r.shape
    S = torch.zeros((H, d, d), dtype=r.dtype) if state is None else state.clone()
    out = torch.zeros_like(r)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hkv,hk->hv", S + u[:, :, None] * kv, r[t])
        S = w[t][:, :, None] * S + kv
    return out, S


def wkv(h, W, m, eps, round_to=None):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]], 0)
    mix = {s: rounded(h + (before - h) * W["mu." + s], round_to) for s in "rkvgw"}
    r, k, v = ((mix[s] @ W[s].T).view(T, H, d) for s in "rkv")
    v = rounded(v, round_to)
    gate = silu(mix["g"] @ W["g"].T)
    w = torch.exp(-torch.exp(rounded(torch.tanh(mix["w"] @ W["w1"].T), round_to) @ W["w2"].T + W["w0"])).view(T, H, d)
    o, _ = wkv_rule(r, k, v, w, W["u"])
    o = rms(o, eps).reshape(T, H * d) * W["norm"] * gate
    return rounded(o, round_to) @ W["o"].T


MIXERS = {"parallel": parallel, "mamba1": mamba1, "wkv": wkv}


def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def run_layer(x, cfg, W, i, round_to=None):
    eps, lay = cfg["norm"]["eps"], cfg["layers"][i]
    w = sub(W, f"l{owner(cfg, i)}.")
    norm = lambda v, n: layer_norm(v, w[n], w[n + ".b"], eps)
    h = norm(x, "norm1")
    x = x + norm(MIXERS[lay["type"]](h if lay["type"] == "wkv" else rounded(h, round_to), sub(w, "mix."), lay["mixer"], eps, round_to), "norm1b")
    if lay.get("mlp") is not None:
        z = relu_squared(rounded(norm(x, "norm2"), round_to) @ w["mlp.up"].T)
        x = x + norm(rounded(z, round_to) @ w["mlp.down"].T, "norm2b")
    return x


def forward(W, cfg, tokens, round_to=None, layers_out=None):
    """Logits [T, vocab] of one whole sequence; ``layers_out``: a list that receives the stream after every layer."""
    x = W["embed"][torch.as_tensor(tokens)] * cfg.get("embedding", {}).get("scale", 1.0)
    for i in range(len(cfg["layers"])):
        x = run_layer(x, cfg, W, i, round_to)
        if layers_out is not None:
            layers_out.append(x)
    return rounded(layer_norm(x, W["final.norm"], W["final.norm.b"], cfg["norm"]["eps"]), round_to) @ W["head"].T


def greedy(W, cfg, prompt, n, margin=0.0):
    """``n`` greedy tokens after ``prompt``, or fewer: it ends where the two best logits lie within ``margin``."""
    toks, out = list(prompt), []
    for _ in range(n):
        last = forward(W, cfg, toks)[-1]
        top = torch.topk(last, 2).values
        if (top[0] - top[1]).item() <= margin:
            break
        out.append(int(last.argmax()))
        toks.append(out[-1])
    return out
