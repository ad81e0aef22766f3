"""Small Pusisun configurations, random weights for them, and model folders: for the tests only, written without
the library (the safetensors package writes the files)."""
import json
import os

import torch


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, base=10000.0, scaling=None, scale=None):
    """``scaling``: (factor, original, fast, slow)."""
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
         "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}
    if rot_dim:
        m["rot"] = {"base": base, "dims": rot_dim}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return "latent_attention", m


def attention(heads, kv_heads, dim, vdim, window, keep_first=0, scale=None):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
                         "mask": {"size": window, "keep_first": keep_first}}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(mixer, mlp):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def config(width, vocab, layers, loop=None, eps=1e-5, scale=1.0):
    out = {"architecture": "Pusisun", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# a stretch of two layers three times; latents of sizes that are no multiples of 16; a window of 9 with 3 kept; one layer
# without feed-forward; two of five experts
TINY_A = config(96, 131, [
    layer(latent(3, 20, 12, 24, 28, 36, base=500.0, scaling=(4.0, 60, 8.0, 1.0)), moe(5, 2, 40)),
    layer(attention(4, 2, 24, 16, 9, 3), moe(3, 1, 24)),
    layer(attention(6, 1, 32, 32, 70, 66), None),
    layer(latent(2, 16, 8, 8, 16, 20), moe(4, 3, 33)),
], loop=(1, 3, 3), eps=1e-6, scale=2.5)

# a width that the matrix kernels cannot tile; the stretch begins with the first layer and ends with the last; one head of one;
# no rotated part; every expert chosen, and one of one; a window of 1 with one kept; as many kept as a page
TINY_B = config(72, 97, [
    layer(attention(1, 1, 8, 40, 7, 1), moe(4, 4, 8)),
    layer(latent(1, 8, 0, 5, 7, 3), moe(1, 1, 16)),
    layer(attention(5, 5, 16, 16, 1, 1), None),
    layer(attention(4, 4, 48, 40, 33, 64), moe(9, 3, 16)),
], loop=(0, 4, 2), eps=1e-4, scale=1.0)

# sizes of real layers, few of them: sixteen heads on one key head, a latent of 128 with 64 rotated, windows across pages, more
# experts than a wave; only the middle layer repeated, one pass more than there are layers
TINY_C = config(256, 211, [
    layer(attention(16, 1, 64, 64, 100, 5), moe(70, 3, 32)),
    layer(latent(4, 64, 64, 64, 128, 96, scaling=(40.0, 100, 32.0, 1.0)), moe(8, 2, 96)),
    layer(attention(8, 4, 128, 64, 130, 20), moe(6, 2, 64)),
], loop=(1, 2, 4), eps=1e-5, scale=3.0)

# no stretch at all; no frequencies stretched; nothing kept
TINY_D = config(64, 80, [layer(latent(2, 16, 16, 16, 32, 32), None), layer(attention(2, 1, 16, 32, 20, 0), moe(4, 2, 32))])

ALL = {"A": TINY_A, "B": TINY_B, "C": TINY_C, "D": TINY_D}


def mixer_weights(kind, m, w, g, dtype, sharp=1.0):
    """local name -> tensor of one mixer."""
    mat = lambda n, k, s=None: (torch.randn(n, k, generator=g) * (s if s is not None else k ** -0.5)).to(dtype)
    vec = lambda n, mean, s: (mean + s * torch.randn(n, generator=g)).to(dtype)
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    if kind == "latent_attention":
        rd, r, qr = m["rot_dim"], m["kv_rank"], m["q_rank"]
        return {"dq": mat(qr, w), "dq.norm": vec(qr, 1.0, 0.2), "uq": mat(H * (d + rd), qr, sharp * qr ** -0.5), "dkv": mat(r + rd, w),
                "dkv.norm": vec(r, 1.0, 0.2), "uk": mat(H * d, r, sharp * r ** -0.5), "uv": mat(H * dv, r), "o": mat(w, H * dv)}
    G = m["kv_heads"]
    out = {"sink": vec(H, 0.5, 1.0), "o": mat(w, H * dv), "q.norm": vec(H * d, 1.0, 0.2) * sharp, "k.norm": vec(G * d, 1.0, 0.2)}
    for name, n in (("q", H * d), ("k", G * d), ("v", G * dv)):
        out[name], out[name + ".b"] = mat(n, w), vec(n, 0.0, 0.3)
    return out


def mlp_weights(mlp, w, g, dtype, steady=False):
    """``steady``: the router's biases leave every token the same experts (their weights still differ)."""
    mat = lambda n, k, s=None: (torch.randn(n, k, generator=g) * (s if s is not None else k ** -0.5)).to(dtype)
    ff, E, top = mlp["expert"]["ff"], mlp["router"]["experts"], mlp["router"]["top"]
    out = {"router": mat(E, w, 1.5 * w ** -0.5)}
    b = 0.5 * torch.randn(E, generator=g)
    if steady:
        b[torch.randperm(E, generator=g)[:top]] += 24.0
    out["router.b"] = b.to(dtype)
    for e in range(E):
        out.update({f"e{e}.gate": mat(ff, w, 2.0 * w ** -0.5), f"e{e}.up": mat(ff, w, 2.0 * w ** -0.5), f"e{e}.down": mat(w, ff)})
    return out


def random_weights(cfg, seed, dtype=torch.bfloat16, sharp=1.0, steady=False):
    """name -> tensor as a file of the design holds it.  ``sharp`` scales what queries are made of."""
    g = torch.Generator().manual_seed(seed)
    w, V = cfg["width"], cfg["vocab"]
    vec = lambda mean, s: (mean + s * torch.randn(w, generator=g)).to(dtype)
    out = {"embed": torch.randn(V, w, generator=g).to(dtype), "final.norm": vec(1.0, 0.1),
           "head": (torch.randn(V, w, generator=g) * w ** -0.5).to(dtype)}
    if cfg.get("loop"):
        out["loop.step"] = torch.randn(cfg["loop"]["times"], w, generator=g).to(dtype)
    for i, layer_ in enumerate(cfg["layers"]):
        p = f"l{i}."
        out[p + "norm1"], out[p + "norm1b"] = vec(1.0, 0.2), vec(0.7, 0.2)
        out.update({p + "mix." + k: v for k, v in mixer_weights(layer_["type"], layer_["mixer"], w, g, dtype, sharp).items()})
        if layer_["mlp"] is not None:
            out[p + "norm2"], out[p + "norm2b"] = vec(1.0, 0.2), vec(0.7, 0.2)
            out.update({p + "mlp." + k: v for k, v in mlp_weights(layer_["mlp"], w, g, dtype, steady).items()})
    return out


def stand_out(weights, cfg, i, token, strength=6.0):
    """Makes the key of ``token`` stand out for every query of layer i, in place.  Every embedding row gets a common component
    along axis 0; for an 'attention' layer the last dimension of every query head reads that axis and the last dimension of
    every key head reads the direction of the token's own embedding row (as the layer's first norm leaves it); for a
    latent one the last latent dimension reads that direction and the last unrotated dimension of every query and key head
    reads the axis (through the last dimension of the queries' latent) and that latent dimension.  Layers ahead of i should
    leave the stream about as it is (i = 0 is exact)."""
    layer_ = cfg["layers"][i]
    m, dt = layer_["mixer"], weights["embed"].dtype
    e = weights["embed"].double()
    e[:, 0] = 3.0
    weights["embed"] = e.to(dt)
    n1 = weights[f"l{i}.norm1"].double()
    e = weights["embed"].double()                          # as rounded
    own = e[token] / e[token].norm()
    others = e.mean(0) / e.mean(0).norm()
    direction = (own - (own @ others) * others) / n1       # what the token has and the average row has not
    axis = torch.zeros_like(direction)
    axis[0] = 1.0 / n1[0]
    get = lambda k: weights[f"l{i}.mix.{k}"].double()

    def put(k, v):
        weights[f"l{i}.mix.{k}"] = v.to(dt)
    d = m["dim"]
    if layer_["type"] == "attention":
        q, k, qb, kb = get("q"), get("k"), get("q.b"), get("k.b")
        for h in range(m["heads"]):
            q[h * d + d - 1], qb[h * d + d - 1] = strength * axis, 0.0
        for g_ in range(m["kv_heads"]):
            k[g_ * d + d - 1], kb[g_ * d + d - 1] = strength * direction, 0.0
        put("q", q), put("k", k), put("q.b", qb), put("k.b", kb)
    else:
        rd = m["rot_dim"]
        dq, uq, dkv, uk = get("dq"), get("uq"), get("dkv"), get("uk")
        dq[-1] = strength * axis
        dkv[m["kv_rank"] - 1] = strength * direction
        uq[:, -1] *= 0.1                                   # nothing else of a query or key reads what was just made large
        uk[:, -1] *= 0.1
        for h in range(m["heads"]):
            uq[h * (d + rd) + d - 1], uk[h * d + d - 1] = 0.0, 0.0
            uq[h * (d + rd) + d - 1, -1], uk[h * d + d - 1, -1] = strength / 2, strength / 2
        put("dq", dq), put("uq", uq), put("dkv", dkv), put("uk", uk)
    return weights


def write_model(folder, cfg, weights):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))


def widen(weights, dtype=torch.float64):
    return {k: v.to(dtype) for k, v in weights.items()}


def with_mask(cfg, i, size=None, keep_first=None):
    """The configuration with another mask in layer i."""
    out = json.loads(json.dumps(cfg))
    mask = out["layers"][i]["mixer"]["mask"]
    if size is not None:
        mask["size"] = size
    if keep_first is not None:
        mask["keep_first"] = keep_first
    return out


def row_error(got, ref):
    """For each row the root mean square of the difference (its mean taken off), relative to the reference's own
    spread: the measure by which logits are compared.  The largest over the rows."""
    d = got.double() - ref.double()
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / ref.double().std()).max().item()


def tolerance(dtype, ref, ref_rounded=None, measure=row_error):
    """What a run in ``dtype`` may differ from the plain implementation's ``ref``: 1e-4 of its spread in float32; in
    bfloat16 3e-2, or three times what rounding the activations where a 16-bit engine stores them does to the plain
    implementation itself (``ref_rounded``), if that is more."""
    if dtype == "float32":
        return 1e-4
    return max(3e-2, 3.0 * measure(ref_rounded, ref)) if ref_rounded is not None else 3e-2
