"""Dopivik configurations drawn at random (seeded): any order of the three mixers, layers with an earlier layer's weights,
with or without a feed-forward, sizes that are no multiples of anything, chunks from one position to beyond the prompt, one to
six taps, ranks of the decays from one on.  Each runs a whole prompt, portions, token-by-token decoding and a ragged batch in
float32 and bfloat16 against the plain implementation (in float32 the schedules also agree with each other to rounding).
Head sizes of the attention are drawn within the pairs whose matrix-core kernels the build entry compiles, so that no
test waits for a compiler."""
import random

import pytest
import torch

import dopivik_models as M
import plain_dopivik as P

pytestmark = pytest.mark.gpu
PAIRS = ((16, 32), (32, 32), (48, 64), (64, 64), (16, 64), (128, 64), (32, 64), (64, 32))     # (key size, value size) as padded


def draw(seed):
    r = random.Random(seed)
    width = r.choice([64, 72, 96, 100, 128, 160])
    layers = []
    for i in range(r.randint(1, 6)):
        own = [j for j, l in enumerate(layers) if l.get("weights_of") is None]
        if own and r.random() < 0.3:
            src = r.choice(own)
            layers.append(dict(layers[src], weights_of=src))
            continue
        kind = r.choice(["parallel", "parallel", "mamba1", "wkv"])
        if kind == "parallel":
            kp, vp = r.choice(PAIRS)
            G = r.choice([1, 2, 3])
            d, dv = r.randint(max(1, kp - 15), kp), r.randint(vp - 31, vp)
            if r.random() < 0.4:
                d = dv = r.choice([16, 32, 48, 64])                           # one size, a multiple of 16: the softmax decoder's kernels
            size = r.choice([1, 2, 5, 31, 32, 33, 64, 65, 100, 128, 200, 1000])
            g2 = r.choice([1, 2, 3])
            mixer = M.parallel(M.left(G * r.choice([1, 2, 4, 8]), G, d, dv, size, dims=r.choice([0, d // 2 * 2, d // 4 * 2]),
                                      base=r.choice([50.0, 10000.0, 1e6]), scale=r.uniform(0.05, 0.5), softcap=r.choice([None, 1.0, 4.0, 50.0])),
                               M.right(g2 * r.choice([1, 2, 3]), g2, r.randint(1, 140), r.randint(1, 140), conv=r.randint(1, 6)))
        elif kind == "mamba1":
            mixer = M.mamba(r.randint(1, 200), r.choice([1, 3, 8, 16, 31, 64]), r.randint(1, 24), conv=r.randint(1, 6))
        else:
            mixer = M.wkv(r.randint(1, 5), r.choice([1, 8, 16, 31, 32, 64, 65]))
        layers.append(M.layer(mixer, r.choice([None, 24, 50, 128])))
    return M.config(width, r.randint(40, 300), layers, eps=r.choice([1e-6, 1e-5, 1e-3]), scale=r.uniform(0.5, 20.0)), r.choice([1, 4, 9, 32])


@pytest.fixture(scope="module")
def lib():
    import llm_infer_amd
    return llm_infer_amd


def all_rows(n):
    return list(range(n))


@pytest.mark.parametrize("seed", range(16))
def test_a_random_configuration_in_every_schedule(lib, seed, tmp_path):
    cfg, rank = draw(5000 + seed)
    g = torch.Generator().manual_seed(seed)
    n = 150
    toks = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    short = torch.randint(0, cfg["vocab"], (37,), generator=g).tolist()
    W = M.random_weights(cfg, 7 + seed, sharp=2.0, rank=rank)
    Wd = M.widen(W)
    ref, ref_short = P.forward(Wd, cfg, toks), P.forward(Wd, cfg, short)
    rounded = P.forward(Wd, cfg, toks, round_to=torch.bfloat16), P.forward(Wd, cfg, short, round_to=torch.bfloat16)
    folder = str(tmp_path / "m")
    M.write_model(folder, cfg, W)
    for dtype in ("float32", "bfloat16"):
        tol = max(M.tolerance(dtype, ref, rounded[0]), M.tolerance(dtype, ref_short, rounded[1]))
        eng = lib.load(folder, dtype=dtype, max_tokens=1024)
        s = eng.alloc_slot()
        whole = eng.step([s], [toks], [all_rows(n)]).cpu()
        eng.free_slot(s)
        assert M.row_error(whole, ref) < tol, (cfg, dtype)
        # together with a shorter request, in slots used before, then both decoded
        a, b = eng.alloc_slot(), eng.alloc_slot()
        out = eng.step([a, b], [short[:30], toks[:140]], [all_rows(30), all_rows(140)]).cpu()
        rows_a, rows_b = [out[:30]], [out[30:]]
        for j in range(7):
            out = eng.step([a, b], [[short[30 + j]], [toks[140 + j]]], [[0], [0]]).cpu()
            rows_a.append(out[:1])
            rows_b.append(out[1:])
        eng.free_slot(a)
        rows_b += [eng.step([b], [[t]], [[0]]).cpu() for t in toks[147:]]
        eng.free_slot(b)
        got_a, got_b = torch.cat(rows_a), torch.cat(rows_b)
        assert M.row_error(got_a, ref_short) < tol and M.row_error(got_b, ref) < tol, (cfg, dtype)
        s = eng.alloc_slot()
        pieces, at = [], 0
        for k in (63, 2, 1, 34, n - 100):
            pieces.append(eng.step([s], [toks[at:at + k]], [all_rows(k)]).cpu())
            at += k
        eng.free_slot(s)
        assert M.row_error(torch.cat(pieces), ref) < tol, (cfg, dtype)
        if dtype == "float32":
            assert M.row_error(got_b, whole) < 5e-5 and M.row_error(torch.cat(pieces), whole) < 5e-5, cfg
