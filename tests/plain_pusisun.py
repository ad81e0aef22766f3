"""A plain implementation of the Pusisun decoder: whole sequences, no cache, one function per mechanism, torch on
the CPU in the precision of the tensors it is given (float32 or float64).  It shares no code with the engine.
``round_to`` (a 16-bit type) rounds the activations where a 16-bit engine stores them (the normed rows that enter a
product, the latents, q, k and v as they go to the attention, the heads' outputs, a feed-forward's hidden row) and
nothing else: the difference to the unrounded run says how much of a 16-bit engine's error is that rounding alone.

Notation: x is the residual stream [T, width]; N(v) = v / sqrt(mean(v^2) + eps).

    embedding:   x = e = table[token] * scale
    stretch:     layers start .. stop - 1 run `times` times with the same tensors; ahead of pass t: x <- x + e (t > 0), x <- x + step[t]
    layer:       x <- x + N(mixer(N(x) w1)) w1b;   x <- x + N(ff(N(x) w2)) w2b      (the second only with a feed-forward)
    latent:      c_q = N(W_dq h) w_q, q = W_uq c_q per head [d | rd];  W_dkv h = [c | k_rot], c <- N(c) w_c
                 k = [W_uk c | turn(k_rot)], v = W_uv c;  scores (q_d . k_d + turn(q_rd) . turn(k_rot)) * scale, softmax over j <= i
                 turn: pairs (i, i + rd / 2), frequencies stretched over a ramp of dimensions, both sine and cosine times a magnitude
    attention:   q = N(W_q h + b_q) w_q, k = N(W_k h + b_k) w_k over all rows at once, v = W_v h + b_v;  score * scale - slope_h (i - j)
                 position i sees j <= i with i - j < window or j < first;  p = exp(s_j) / (exp(sink_h) + sum_j' exp(s_j'))
    experts:     z = W_r h + b_r; the `top` largest, weighted by the softmax over them alone;  W_down (silu(W_gate h) * (W_up h))
    logits:      W_head (N(x) w)
"""
from __future__ import annotations

import math

import torch


def rounded(t, round_to):
    return t if round_to is None else t.to(round_to).to(t.dtype)


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def stretched_frequencies(dims: int, base: float, scaling: dict | None):
    """(frequencies of the dims / 2 pairs, factor of sine and cosine), float64.  With ``scaling`` the frequencies of
    the pairs below a ramp stay, those above it are divided by the factor, those on it are blended."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.tensor(float(base), dtype=torch.float64) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    factor, original, fast, slow = (float(scaling[k]) for k in ("factor", "original", "fast", "slow"))

    def dimension(turns):                       # the (fractional) pair that makes `turns` turns over `original` positions
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(dimension(fast)), 0)
    hi = min(math.ceil(dimension(slow)), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def turn(x, positions, freqs, magnitude: float):
    """x [T, heads, dims]: dimension i is paired with i + dims / 2."""
    half = freqs.numel()
    angle = positions.to(freqs.dtype)[:, None] * freqs[None, :]           # [T, half]
    cos = (torch.cos(angle) * magnitude).to(x.dtype)[:, None, :]
    sin = (torch.sin(angle) * magnitude).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., 2 * half:]], dim=-1)


def causal_mask(n: int):
    return torch.arange(n)[None, :] <= torch.arange(n)[:, None]


def window_mask(n: int, size: int | None, keep_first: int = 0):
    """Row i: the keys j <= i that are nearer than ``size`` or among the first ``keep_first``."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    near = torch.ones((n, n), dtype=torch.bool) if size is None else i - j < size
    return (j <= i) & (near | (j < keep_first))


def slopes(heads: int, dtype):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=dtype)


def softmax_attention(q, k, v, scale, visible, sink=None, distance_slopes=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv], visible [T, T] (row: query).  Returns [T, H, dv]."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    distance = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if distance_slopes is not None:
            s = s - distance_slopes[h] * distance
        s = s.masked_fill(~visible, -math.inf)
        m = s.max(-1).values
        if sink is not None:
            m = torch.maximum(m, sink[h].expand(T))
        e = torch.exp(s - m[:, None])
        total = e.sum(-1) if sink is None else e.sum(-1) + torch.exp(sink[h] - m)
        out[:, h] = (e / total[:, None]) @ v[:, g]
    return out


def latent_mixer(h, W, m, eps, round_to=None):
    T = h.shape[0]
    H, d, rd, dv, r = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    cq = rounded(rms_norm(h @ W["dq"].T, W["dq.norm"], eps), round_to)
    q = (cq @ W["uq"].T).view(T, H, d + rd)
    kv = h @ W["dkv"].T
    c = rounded(rms_norm(kv[:, :r], W["dkv.norm"], eps), round_to)
    q_flat, q_rot, k_rot = q[..., :d], q[..., d:], kv[:, None, r:]
    if rd:
        freqs, magnitude = stretched_frequencies(int(m["rot"]["dims"]), float(m["rot"]["base"]), m["rot"].get("scaling"))
        q_rot, k_rot = turn(q_rot, torch.arange(T), freqs, magnitude), turn(k_rot, torch.arange(T), freqs, magnitude)
    q_rot, k_rot = rounded(q_rot, round_to), rounded(k_rot, round_to)
    if round_to is None:
        k = torch.cat([(c @ W["uk"].T).view(T, H, d), k_rot.expand(T, H, rd)], -1)
        o = softmax_attention(torch.cat([q_flat, q_rot], -1), k, (c @ W["uv"].T).view(T, H, dv), float(m["scale"]), causal_mask(T))
    else:
        # a 16-bit engine takes the keys' up-projection into the query and the values' out of the sum: what is rounded is
        # the query in the latent's space and the latents' weighted sum
        qc = rounded(torch.einsum("thd,hdr->thr", q_flat, W["uk"].view(H, d, r)), round_to)
        mixed = softmax_attention(torch.cat([qc, q_rot], -1), torch.cat([c[:, None], k_rot], -1), c[:, None], float(m["scale"]), causal_mask(T))
        o = torch.einsum("thr,hvr->thv", rounded(mixed, round_to), W["uv"].view(H, dv, r))
    return rounded(o, round_to).reshape(T, -1) @ W["o"].T


def attention_mixer(h, W, m, eps, round_to=None):
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rms_norm(h @ W["q"].T + W["q.b"], W["q.norm"], eps).view(T, H, d)
    k = rms_norm(h @ W["k"].T + W["k.b"], W["k.norm"], eps).view(T, G, d)
    v = (h @ W["v"].T + W["v.b"]).view(T, G, dv)
    q, k, v = rounded(q, round_to), rounded(k, round_to), rounded(v, round_to)
    mask = m.get("mask") or {}
    seen = window_mask(T, mask.get("size"), int(mask.get("keep_first") or 0))
    o = softmax_attention(q, k, v, float(m["scale"]), seen, W["sink"], slopes(H, h.dtype))
    return rounded(o, round_to).reshape(T, -1) @ W["o"].T


def expert_weights(h, W, top: int):
    """[T, experts]: the softmax over the ``top`` largest logits, zero elsewhere."""
    z = h @ W["router"].T + W["router.b"]
    best = torch.topk(z, top, dim=-1)
    out = torch.zeros_like(z)
    return out.scatter(1, best.indices, torch.softmax(best.values, -1))


def experts(h, W, mlp, round_to=None):
    n, top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
    weights = expert_weights(h, W, top)
    out = torch.zeros_like(h)
    for e in range(n):
        rows = weights[:, e].nonzero()[:, 0]
        if rows.numel():
            he = h[rows]
            y = rounded(silu(he @ W[f"e{e}.gate"].T) * (he @ W[f"e{e}.up"].T), round_to)
            out[rows] += (y @ W[f"e{e}.down"].T) * weights[rows, e:e + 1]
    return out


def sub(W, prefix):
    return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}


def layer(x, L, spec, eps, round_to=None):
    h = rounded(rms_norm(x, L["norm1"], eps), round_to)
    mixer = {"latent_attention": latent_mixer, "attention": attention_mixer}[spec["type"]]
    x = x + rms_norm(mixer(h, sub(L, "mix."), spec["mixer"], eps, round_to), L["norm1b"], eps)
    if spec.get("mlp") is not None:
        h = rounded(rms_norm(x, L["norm2"], eps), round_to)
        x = x + rms_norm(experts(h, sub(L, "mlp."), spec["mlp"], round_to), L["norm2b"], eps)
    return x


def runs(config: dict) -> list:
    """(layer, pass that begins here or None) in the order in which they run."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    out = [(i, None) for i in range(a)]
    for t in range(int(loop["times"])):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(config: dict, W: dict, tokens, layers_out: list | None = None, round_to=None):
    """Logits [T, vocab] of one sequence.  ``W``: tensor name -> tensor in the dtype to compute in.  ``layers_out``:
    receives the residual stream after every run of a layer."""
    eps = float(config["norm"]["eps"])
    x0 = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float((config.get("embedding") or {}).get("scale", 1.0))
    x = x0
    for i, t in runs(config):
        if t is not None:
            if t > 0:
                x = x + x0
            x = x + W["loop.step"][t]
        x = layer(x, sub(W, f"l{i}."), config["layers"][i], eps, round_to)
        if layers_out is not None:
            layers_out.append(x.clone())
    return rounded(rms_norm(x, W["final.norm"], eps), round_to) @ W["head"].T
