"""Small Dopivik configurations, random weights for them, and model folders: for the tests only, written without
the library (the safetensors package writes the files)."""
import json
import os

import torch


def parallel(left, right):
    return "parallel", {"left": left, "right": right}


def left(heads, kv_heads, dim, vdim, chunk, dims=None, base=10000.0, scale=None, softcap=30.0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
         "scale": dim ** -0.5 if scale is None else scale, "softcap": softcap}
    dims = dim if dims is None else dims
    if dims:
        m["rot"] = {"base": base, "dims": dims}
    return m


def right(heads, kv_heads, dim, vdim, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def mamba(inner, state, dt_rank, conv=4):
    return "mamba1", {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def wkv(heads, dim):
    return "wkv", {"heads": heads, "dim": dim}


def layer(mixer, ff=None, weights_of=None):
    out = {"type": mixer[0], "mixer": mixer[1], "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def config(width, vocab, layers, eps=1e-5, scale=1.0):
    return {"architecture": "Dopivik", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


# grouped heads on both sides, keys and values of different sizes, a partial rotation, chunks below a page; a convolution of two
# taps; a layer without feed-forward; a later layer with the first one's weights
TINY_A = config(96, 131, [
    layer(parallel(left(4, 2, 24, 16, 50, dims=12, base=500.0, softcap=5.0), right(6, 2, 20, 24, conv=2)), 72),
    layer(mamba(80, 5, 7, conv=3), None),
    layer(wkv(3, 20), 40),
    layer(parallel(left(4, 2, 24, 16, 50, dims=12, base=500.0, softcap=5.0), right(6, 2, 20, 24, conv=2)), 72, weights_of=0),
    layer(wkv(3, 20), 40, weights_of=2),
], eps=1e-6, scale=2.5)

# a width that the matrix kernels cannot tile; one head of one; one tap; no rotation and no soft cap that bites; a state of one;
# the shared weights of a layer that comes twice more
TINY_B = config(72, 97, [
    layer(wkv(1, 7), 24),
    layer(parallel(left(1, 1, 16, 16, 7, dims=0, scale=0.4, softcap=1000.0), right(1, 1, 8, 5, conv=1)), None),
    layer(mamba(33, 1, 1, conv=1), 17),
    layer(mamba(33, 1, 1, conv=1), 17, weights_of=2),
    layer(mamba(33, 1, 1, conv=1), 17, weights_of=2),
], eps=1e-4)

# sizes of real layers, few of them: chunks beyond a page, heads of 64 and 128
TINY_C = config(256, 211, [
    layer(parallel(left(8, 2, 64, 64, 130, base=2e5, softcap=20.0), right(4, 2, 128, 64)), 320),
    layer(mamba(512, 16, 16), 128),
    layer(wkv(4, 64), 320),
    layer(parallel(left(8, 2, 64, 64, 130, base=2e5, softcap=20.0), right(4, 2, 128, 64)), 320, weights_of=0),
], scale=3.0)

ALL = {"A": TINY_A, "B": TINY_B, "C": TINY_C}


def _makers(g, dtype):
    mat = lambda n, k, s=None: (torch.randn(n, k, generator=g) * (s if s is not None else k ** -0.5)).to(dtype)
    vec = lambda n, mean, s: (mean + s * torch.randn(n, generator=g)).to(dtype)
    return mat, vec


def left_weights(m, w, g, dtype, sharp=1.0):
    mat, _ = _makers(g, dtype)
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    return {"q": mat(H * d, w, sharp * w ** -0.5), "k": mat(G * d, w, sharp * w ** -0.5), "v": mat(G * dv, w),
            "g": mat(H * dv, w, 2.0 * w ** -0.5), "o": mat(w, H * dv)}


def right_weights(m, w, g, dtype):
    mat, vec = _makers(g, dtype)
    H, G, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    conv = lambda n: (torch.randn(n, taps, generator=g) * 0.6).to(dtype)
    return {"q": mat(G * d, w), "k": mat(G * d, w), "v": mat(H * dv, w), "g": mat(H * dv, w), "b": mat(H, w, 2.0 * w ** -0.5),
            "a": mat(H, w, w ** -0.5), "q.conv": conv(G * d), "k.conv": conv(G * d), "v.conv": conv(H * dv),
            "A_log": vec(H, -1.0, 1.0), "dt_bias": vec(H, -2.0, 1.0), "norm": vec(dv, 1.0, 0.2), "o": mat(w, H * dv)}


def mamba_weights(m, w, g, dtype):
    mat, vec = _makers(g, dtype)
    c, n, r, taps = m["inner"], m["state"], m["dt_rank"], m["conv"]
    return {"in": mat(2 * c, w), "conv": (torch.randn(c, taps, generator=g) * 0.6).to(dtype), "conv.b": vec(c, 0.0, 0.3),
            "x": mat(r + 2 * n, c), "dt": mat(c, r), "dt.b": vec(c, -2.0, 1.0),
            "A_log": (torch.randn(c, n, generator=g) * 0.7 + 0.3).to(dtype), "D": vec(c, 1.0, 0.3), "o": mat(w, c)}


def wkv_weights(m, w, g, dtype, rank=11):
    mat, vec = _makers(g, dtype)
    H, d = m["heads"], m["dim"]
    c = H * d
    out = {"mu." + s: torch.rand(w, generator=g).to(dtype) for s in "rkvgw"}
    out.update({s: mat(c, w) for s in "rkvg"})
    out.update({"w1": mat(rank, w, 2.0 * w ** -0.5), "w2": mat(c, rank, rank ** -0.5), "w0": vec(c, -1.5, 1.0),
                "u": (torch.randn(H, d, generator=g) * 0.7).to(dtype), "norm": vec(c, 1.0, 0.2), "o": mat(w, c)})
    return out


def mixer_weights(mixer, w, g, dtype, sharp=1.0, rank=11):
    """local name -> tensor of one mixer."""
    kind, m = mixer
    if kind == "mamba1":
        return mamba_weights(m, w, g, dtype)
    if kind == "wkv":
        return wkv_weights(m, w, g, dtype, rank)
    _, vec = _makers(g, dtype)
    out = {"left." + k: v for k, v in left_weights(m["left"], w, g, dtype, sharp).items()}
    out.update({"right." + k: v for k, v in right_weights(m["right"], w, g, dtype).items()})
    out.update({"left.out": vec(w, 1.0, 0.3), "right.out": vec(w, 1.0, 0.3)})
    return out


def random_weights(cfg, seed, dtype=torch.bfloat16, sharp=1.0, rank=11):
    """name -> tensor as a file of the design holds it.  ``sharp`` scales the attention's query and key matrices, ``rank`` is that
    of the decays' two matrices (which the tensors alone say)."""
    g = torch.Generator().manual_seed(seed)
    w, V = cfg["width"], cfg["vocab"]
    mat, vec = _makers(g, dtype)
    norm = lambda name, mean: {name: vec(w, mean, 0.2), name + ".b": vec(w, 0.0, 0.2)}
    out = {"embed": torch.randn(V, w, generator=g).to(dtype), "head": mat(V, w), **norm("final.norm", 1.0)}
    for i, lay in enumerate(cfg["layers"]):
        if lay.get("weights_of") is not None:
            continue
        p = f"l{i}."
        out.update({p + k: v for n, mean in (("norm1", 1.0), ("norm1b", 0.7)) for k, v in norm(n, mean).items()})
        out.update({p + "mix." + k: v for k, v in mixer_weights((lay["type"], lay["mixer"]), w, g, dtype, sharp, rank).items()})
        if lay["mlp"] is not None:
            out.update({p + k: v for n, mean in (("norm2", 1.0), ("norm2b", 0.7)) for k, v in norm(n, mean).items()})
            out[p + "mlp.up"], out[p + "mlp.down"] = mat(lay["mlp"]["ff"], w, 2.0 * w ** -0.5), mat(w, lay["mlp"]["ff"])
    return out


def stand_out(weights, cfg, i, token, strength=6.0):
    """Makes the key of ``token`` stand out for every query of layer i's attention, in place: every embedding row gets a common
    component along axis 0, the last dimension of every query head reads that axis, and the last dimension of every key head
    reads the direction of the token's own embedding row (as the layer's first norm leaves it)."""
    m, w = cfg["layers"][i]["mixer"]["left"], cfg["width"]
    d = m["dim"]
    assert m.get("rot") is None or m["rot"]["dims"] < d, "the last dimension must not be turned"
    dt = weights["embed"].dtype
    e = weights["embed"].double()
    e[:, 0] = 3.0
    weights["embed"] = e.to(dt)
    p = f"l{i}."
    weights[p + "norm1.b"] = torch.zeros_like(weights[p + "norm1.b"])
    n1 = weights[p + "norm1"].double()
    e = weights["embed"].double()                          # as rounded
    e = e - e.mean(-1, keepdim=True)
    own = e[token] / e[token].norm()
    q, k = weights[p + "mix.left.q"].double(), weights[p + "mix.left.k"].double()
    for h in range(m["heads"]):
        q[h * d + d - 1] = 0.0
        q[h * d + d - 1, 0] = strength / n1[0]
    others = e.mean(0) / e.mean(0).norm()
    direction = own - (own @ others) * others              # what the token has and the average row has not
    for g_ in range(m["kv_heads"]):
        k[g_ * d + d - 1] = strength * direction / n1
    weights[p + "mix.left.q"], weights[p + "mix.left.k"] = q.to(dt), k.to(dt)
    return weights


def write_model(folder, cfg, weights):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))


def widen(weights, dtype=torch.float64):
    return {k: v.to(dtype) for k, v in weights.items()}


def with_chunk(cfg, i, size):
    """The configuration with another chunk size in layer i."""
    out = json.loads(json.dumps(cfg))
    out["layers"][i]["mixer"]["left"]["mask"]["size"] = size
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
