"""Pusisun configurations drawn at random (seeded): any order of the two mixers, stretches of layers anywhere that run once
to four times, with or without a feed-forward, sizes that are no multiples of anything, windows and kept tokens from one position
to beyond the prompt, stretched and plain frequencies, one to forty experts.  Each runs a whole prompt, portions, token-by-token
decoding and a ragged batch in float32 and bfloat16 against the plain implementation (in float32 the schedules also agree with
each other to rounding).  In bfloat16 the routers' biases settle the choice (see test_pusisun_gpu).  Head sizes are drawn within
the pairs whose matrix-core kernels the build entry compiles, so that no test waits for a compiler."""
import random

import pytest
import torch

import plain_pusisun as P
import pusisun_models as M

pytestmark = pytest.mark.gpu
PAIRS = ((16, 32), (32, 32), (48, 64), (64, 64), (16, 64), (128, 64), (32, 64), (64, 32))     # (key size, value size) as padded
LATENTS = ((16, 32), (32, 32), (48, 32), (64, 64), (80, 96), (128, 128), (192, 128))          # (key, latent) as padded


def draw(seed):
    r = random.Random(seed)
    width = r.choice([64, 72, 96, 100, 128, 160])
    layers = []
    for _ in range(r.randint(1, 4)):
        if r.random() < 0.5:
            kp, vp = r.choice(LATENTS)
            rank = r.randint(max(1, vp - 31), min(vp, kp))
            rd = r.randint(max(0, kp - 15 - rank), kp - rank) // 2 * 2
            while (rank + rd + 15) // 16 * 16 != kp:
                rank = r.randint(max(1, vp - 31), min(vp, kp))
                rd = r.randint(max(0, kp - 15 - rank), kp - rank) // 2 * 2
            scaling = None if r.random() < 0.3 else (r.uniform(1.5, 40.0), r.choice([20, 64, 300, 4096]), r.uniform(2.0, 40.0), r.uniform(0.3, 1.9))
            mixer = M.latent(r.choice([1, 2, 3, 5, 8, 33]), r.randint(1, 40), rd, r.randint(1, 48), rank, r.randint(1, 60),
                             base=r.choice([50.0, 10000.0, 1e6]), scaling=scaling, scale=r.uniform(0.05, 0.4))
        else:
            kp, vp = r.choice(PAIRS)
            G = r.choice([1, 2, 3])
            d, dv = r.randint(max(1, kp - 15), kp), r.randint(vp - 31, vp)
            if r.random() < 0.4:
                d = dv = r.choice([16, 32, 48, 64])                           # one size, a multiple of 16: the softmax decoder's kernels
            mixer = M.attention(G * r.choice([1, 2, 4, 8]), G, d, dv, r.choice([1, 2, 5, 31, 32, 33, 64, 65, 100, 128, 1000]),
                                r.choice([0, 0, 1, 3, 31, 32, 33, 64, 65, 140, 500]), scale=r.uniform(0.05, 0.5))
        E = r.choice([1, 2, 5, 8, 40])
        layers.append(M.layer(mixer, None if r.random() < 0.25 else M.moe(E, r.randint(1, min(E, 6)), r.randint(1, 70))))
    loop = None
    if r.random() < 0.8:
        a = r.randrange(len(layers))
        loop = (a, r.randint(a + 1, len(layers)), r.randint(1, 4))
    return M.config(width, r.randint(40, 300), layers, loop, eps=r.choice([1e-6, 1e-5, 1e-3]), scale=r.uniform(0.5, 20.0))


@pytest.fixture(scope="module")
def lib():
    import llm_infer_amd
    return llm_infer_amd


def all_rows(n):
    return list(range(n))


@pytest.mark.parametrize("seed", range(16))
def test_a_random_configuration_in_every_schedule(lib, seed, tmp_path):
    cfg = draw(9000 + seed)
    g = torch.Generator().manual_seed(seed)
    n = 150
    toks = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    short = torch.randint(0, cfg["vocab"], (37,), generator=g).tolist()
    for dtype in ("float32", "bfloat16"):
        W = M.random_weights(cfg, 7 + seed, sharp=2.0, steady=dtype != "float32")
        Wd = M.widen(W)
        ref, ref_short = P.forward(cfg, Wd, toks), P.forward(cfg, Wd, short)
        rounded = P.forward(cfg, Wd, toks, round_to=torch.bfloat16), P.forward(cfg, Wd, short, round_to=torch.bfloat16)
        folder = str(tmp_path / dtype)
        M.write_model(folder, cfg, W)
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
