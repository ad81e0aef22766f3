"""Pusisun on the GPU against the plain implementation: every kernel and mixer alone, whole prompts, prompts cut into
portions, decoding token by token, batches of unequal requests against each alone, slots and pages used again, keys far
away, at page borders and just inside and just outside a window, the first tokens that a window keeps and the next ones, the
first tokens of a sequence, long decoding, other sizes, stretches of layers that run several times, and greedy generation
through the library's entry point.

Where random weights would hide a fault, a token's key is made to stand out for every query (``pusisun_models.stand_out``)
and the test first shows, with the plain implementation alone, that the fault it looks for would move the result far
beyond the tolerance.

Routing: a float32 run follows the plain implementation's choices to rounding.  A bfloat16 run rounds the router's input, so
a token whose logits nearly tie could go either way, and what it then leaves in the caches reaches other rows; whole bfloat16
models therefore get router biases that settle the choice (the weights still differ from token to token), or a prompt whose
choices all have a clear margin; the choice itself is tested alone."""
import json
import os
import subprocess
import sys

import pytest
import torch

import plain_pusisun as P
import pusisun_models as M
import trace_util as TU

pytestmark = pytest.mark.gpu
DEV = "cuda"
SHOWS = {"float32": 20.0, "bfloat16": 2.0}      # a fault shows if it moves the result by this many tolerances
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16, "float16": torch.float16}


@pytest.fixture(scope="module")
def lib():
    import llm_infer_amd
    return llm_infer_amd


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, cfg in M.ALL.items():
        for dtype in ("float32", "bfloat16"):
            W = M.random_weights(cfg, 40 + ord(name), sharp=2.0, steady=dtype != "float32")
            folder = str(tmp_path_factory.mktemp(f"pusisun_{name}_{dtype}"))
            M.write_model(folder, cfg, W)
            out[name, dtype] = (folder, cfg, M.widen(W))
    return out


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def step_context(slots, lens_before, toks):
    from llm_infer_amd.engine.step import StepContext
    return StepContext(DEV, list(slots), [list(t) for t in toks], list(lens_before), [[] for _ in toks])


def error(got, ref):
    """Largest difference relative to the reference's spread."""
    return ((got.double() - ref.double()).abs().max() / ref.double().std()).item()


def rows(n):
    return list(range(n))


def load(lib, tmp_path, cfg, W, dtype, name="m", max_tokens=4096):
    folder = str(tmp_path / f"{name}_{dtype}")
    M.write_model(folder, cfg, W)
    return lib.load(folder, dtype=dtype, max_tokens=max_tokens)


def run_schedule(eng, reqs, schedule):
    """``schedule``: a list of steps, each {request: number of tokens it brings}; all rows wanted.  Returns
    {request: logits [n, vocab]}."""
    slot, at, out = {}, {r: 0 for r in reqs}, {r: [] for r in reqs}
    for step in schedule:
        rs = list(step)
        for r in rs:
            if r not in slot:
                slot[r] = eng.alloc_slot()
        res = eng.step([slot[r] for r in rs], [reqs[r][at[r]:at[r] + step[r]] for r in rs], [rows(step[r]) for r in rs]).cpu()
        for r, part in zip(rs, res.split([step[r] for r in rs])):
            out[r].append(part)
            at[r] += step[r]
            if at[r] == len(reqs[r]):
                eng.free_slot(slot.pop(r))
    return {r: torch.cat(v) for r, v in out.items()}


# ---------------------------------------------------------------------------- kernels alone
@pytest.mark.parametrize("width,n", [(96, 5), (70, 5), (8200, 3), (8192, 5), (1024, 100), (2052, 70), (5000, 3)])
def test_norm_with_the_residual_sum_takes_more_rows_and_pair_sums_along(lib, width, n):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(width + n)
    x, y, e = (torch.randn(n, width, generator=g) for _ in range(3))
    w, v, w2 = (torch.randn(width, generator=g) for _ in range(3))
    N = lambda z, eps: z / torch.sqrt(z.pow(2).mean(-1, keepdim=True) + eps)
    assert error(ops.add_rows(x.to(DEV), e.to(DEV), v.to(DEV)).cpu(), x.double() + e.double() + v.double()) < 1e-6
    assert error(ops.add_rows(x.to(DEV), None, v.to(DEV)).cpu(), x.double() + v.double()) < 1e-6
    for top in (0, 1, 3, 6):
        if top:
            pairs = torch.randn(n * top, width, generator=g)
            slot_of = torch.randperm(n * top, generator=g).to(torch.int32).view(n, top)
            if top == 3:
                slot_of[1, 2] = -1                                           # a token with fewer
            weights = torch.rand(n, top, generator=g)
            yy = sum(torch.where(slot_of[:, j:j + 1] >= 0, weights[:, j:j + 1], 0.0).double() * pairs[slot_of[:, j].clamp(min=0).long()].double()
                     for j in range(top))
            src = ops.PairSum(pairs.to(DEV), slot_of.to(DEV), weights.to(DEV))
            assert error(src.tensor().cpu(), yy) < 1e-6
            out = x.clone().to(DEV)
            src.add_to(out)
            assert error(out.cpu(), x.double() + yy) < 1e-6
        else:
            yy, src = y.double(), y.to(DEV)
        for also in (None, (None, v), (e, v)):
            ref = x.double() + N(yy, 1e-3) * w.double()
            if also is not None:
                ref = ref + v.double() + (0 if also[0] is None else e.double())
                also = (None if also[0] is None else e.to(DEV), v.to(DEV))
            for dt in (torch.float32, torch.bfloat16):
                xd, w2d = x.clone().to(DEV), w2.to(DEV)
                ops.rmsnorm_add(xd, src, w.to(DEV), 1e-3, None, (w2d, 1e-5, dt), also)
                assert error(xd.cpu(), ref) < 3e-6, (top, also is None)
                ready = ops.prepared_rmsnorm(xd, w2d, 1e-5, dt)
                assert torch.allclose(ready.cpu().double(), N(ref, 1e-5) * w2.double(), rtol=2e-5 if dt == torch.float32 else 2.0 ** -8, atol=3e-5)
            xd = x.clone().to(DEV)
            assert error(ops.rmsnorm_add(xd, src, w.to(DEV), 1e-3, also=also).cpu(), ref) < 3e-6


@pytest.mark.parametrize("H,d,rot", [(3, 20, 8), (2, 10, 0), (2, 10, 6), (5, 64, 64), (32, 128, 0), (1, 4, 4)])
def test_norm_over_all_of_q_on_the_way_to_the_cache_and_the_magnitude(lib, H, d, rot):
    """q as it comes back (keys and values take the same path and are checked through the mixers), in the kernel of four
    columns at a time and in the one of any size."""
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(H * d + rot)
    for n, pad in ((1, 0), (5, 3), (600, 0)):
        x = torch.randn(n, H * d + pad, generator=g)
        w = torch.randn(H * d, generator=g)
        pos = torch.randint(0, 900, (n,), generator=g, dtype=torch.int32)
        freqs = (1e4 ** (-torch.arange(max(rot // 2, 1)) / max(rot // 2, 1))).float()
        q = ops.rot_store(x.to(DEV), 0, 0, 0, freqs.to(DEV), rot, pos.to(DEV), torch.zeros(n, dtype=torch.int32, device=DEV), None, H, 0, d, d,
                          torch.float32, None, (w.to(DEV), None, 1e-4), 1.25).cpu()
        ref = P.rms_norm(x[:, :H * d].double(), w.double(), 1e-4).view(n, H, d)
        if rot:
            ref = P.turn(ref, pos, freqs.double()[:rot // 2], 1.25)
        assert error(q[:, :, :d], ref) < 5e-4, (n, pad)                      # (float32 angles up to 900)
        assert q.shape[2] == d or float(q[:, :, d:].abs().max()) == 0.0


@pytest.mark.parametrize("half", [False, True])
def test_latents_and_their_queries(lib, half):
    from llm_infer_amd.cache import Cache
    from llm_infer_amd.cache.specs import KVSpec
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(8)
    for H, d, rd, rot, r, qr, n in ((3, 5, 6, 6, 20, 9, 7), (2, 8, 12, 8, 40, 33, 300), (1, 3, 4, 0, 16, 40, 1)):
        rows_ = torch.randn(n, qr + r + rd + 2, generator=g)
        cq_w, kv_w = torch.randn(qr, generator=g), torch.randn(r, generator=g)
        q_rows = torch.randn(n, H * (d + rd), generator=g)
        freqs = (100.0 ** (-torch.arange(max(rot // 2, 1)) / 3.0)).float().to(DEV)
        turn = (freqs, rot, half, 1.3)
        cache = Cache([KVSpec(1, ops.padded_map_dim(r + rd), None, r, None, "maps")], 1024, 1024, torch.float32, DEV)
        slot = cache.alloc_slot()
        cache.grow([slot], [n])
        pos, slots = torch.arange(n, dtype=torch.int32, device=DEV), torch.full((n,), slot, dtype=torch.int32, device=DEV)
        kv = cache.view(0).as_tuple()
        cq = ops.latent_store(rows_.to(DEV), qr + 2, kv_w.to(DEV), 1e-3, turn, pos, slots, kv, d, rd, r, (1, cq_w.to(DEV))).cpu()
        assert error(cq, P.rms_norm(rows_[:, 1:1 + qr].double(), cq_w.double(), 1e-3)) < 1e-6
        q = ops.latent_queries(q_rows.to(DEV), 0, turn, pos, H, d, rd, r, torch.float32).cpu()
        both = ops.latent_store_queries(torch.cat([q_rows, rows_], 1).to(DEV), 0, H * (d + rd) + qr + 2, kv_w.to(DEV), 1e-3, turn, pos, slots, kv,
                                        H, d, rd, r).cpu()
        part = q_rows.view(n, H, d + rd)[..., d:].double()
        if rot and half:
            part = P.turn(part, torch.arange(n), freqs.double().cpu()[:rot // 2], 1.3)
        elif rot:                                                            # adjacent pairs: the same with the dimensions dealt out
            order = list(range(0, rot, 2)) + list(range(1, rot, 2)) + list(range(rot, rd))
            part[..., order] = P.turn(part[..., order], torch.arange(n), freqs.double().cpu()[:rot // 2], 1.3)
        for got in (q, both):
            assert error(got[:, :, r:r + rd], part) < 1e-4
            assert got.shape[2] == r + rd or float(got[:, :, r + rd:].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", ["bfloat16", "float16"])
def test_products_per_head_of_a_few_tokens(lib, dtype):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(9)
    for n, H, n_in, n_out in ((1, 3, 128, 192), (8, 2, 24, 40), (32, 1, 200, 33), (5, 4, 136, 7), (33, 2, 64, 64), (31, 2, 20, 16)):
        x, w = torch.randn(n, H * n_in, generator=g), torch.randn(H, n_out, n_in, generator=g).to(DT[dtype])
        gate = torch.randn(n, H * n_out, generator=g)
        ref = torch.einsum("thi,hji->thj", x.double().view(n, H, n_in), w.double())
        for gt in (None, gate):
            want = ref if gt is None else ref * torch.sigmoid(gt.double()).view(n, H, n_out)
            for src in (x, x.to(DT[dtype])):
                out = torch.zeros(n, H, n_out, dtype=DT[dtype], device=DEV)
                ops.head_linear(src.to(DEV), 0, n_in, w.to(DEV), out, 0, n_out, gate=None if gt is None else gt.to(DEV))
                assert error(out.cpu(), want) < (0.03 if src.dtype != torch.float32 else 0.02), (n, n_in, n_out)


@pytest.mark.parametrize("dtype", ["bfloat16", "float16", "float32"])
def test_queries_of_a_few_tokens_in_one_launch(lib, dtype):
    """The query taken into the latents' space beside its rotated part: in the launch of a few tokens and in two."""
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(10)
    for H, d, rd, rot, r, half in ((3, 8, 12, 8, 20, True), (2, 24, 4, 4, 33, False), (4, 64, 0, 0, 48, True), (1, 16, 8, 8, 40, True),
                                   (2, 10, 6, 6, 16, True), (2, 0, 16, 16, 16, True)):
        freqs = (50.0 ** (-torch.arange(max(rot // 2, 1)) / 3.0)).float().to(DEV)
        w = torch.randn(H, r, d, generator=g).to(DT[dtype]) if d else None
        for n in (1, 5, 32, 33):
            rows_ = torch.randn(n, H * (d + rd) + 4, generator=g)
            pos = torch.randint(0, 300, (n,), generator=g, dtype=torch.int32)
            q = ops.absorbed_queries(rows_.to(DEV), 4, None if w is None else w.to(DEV), (freqs if rot else None, rot, half, 1.3), pos.to(DEV), H, d,
                                     rd, r, DT[dtype]).cpu()
            part = rows_[:, 4:].view(n, H, d + rd).double()
            tol = 1e-4 if dtype == "float32" else 0.03
            if d:
                assert error(q[:, :, :r], torch.einsum("thd,hrd->thr", part[..., :d], w.double())) < tol, (H, d, n)
            else:
                assert float(q[:, :, :r].abs().max()) == 0.0
            turned = part[..., d:].clone()
            order = list(range(rot)) if half else list(range(0, rot, 2)) + list(range(1, rot, 2))
            if rot:
                turned[..., order] = P.turn(turned[..., order], pos, freqs.double().cpu()[:rot // 2], 1.3)
            if rd:
                assert error(q[:, :, r:r + rd], turned) < tol, (H, d, n)
            assert q.shape[2] == r + rd or float(q[:, :, r + rd:].abs().max()) == 0.0


def check_pairs(p, chosen, weights):
    """Sorted pairs against a choice [T, top] (experts ascending) and its weights, exactly."""
    T, top = chosen.shape
    counts, offsets = p.counts.cpu(), p.offsets.cpu()
    assert torch.equal(p.chosen.cpu().long(), chosen)
    assert torch.allclose(p.weights.cpu().double(), weights, atol=2e-6)
    want = torch.bincount(chosen.flatten(), minlength=p.n_experts)
    assert torch.equal(counts.long(), want) and torch.equal(offsets.long(), want.cumsum(0) - want)
    order = sorted(range(T * top), key=lambda i: (chosen.flatten()[i].item(), i))
    assert p.row_of.cpu().tolist() == [i // top for i in order]
    assert [p.slot_of.cpu().flatten()[i].item() for i in order] == list(range(T * top))


@pytest.mark.parametrize("dtype", ["bfloat16", "float16"])
@pytest.mark.parametrize("E,top", [(1, 1), (3, 2), (16, 4), (17, 17), (70, 3), (300, 8), (512, 1)])
def test_router_and_the_sorted_pairs(lib, E, top, dtype):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(E + top)
    K = 96
    bias = torch.randn(E, generator=g)
    for stored in (DT[dtype], torch.float32):                                # one 16-bit matrix, or the sum of several
        W = (torch.randn(E, K, generator=g) * 0.3).to(stored).float()
        wr = ops.router_weight(W.to(DEV), DT[dtype])
        assert (ops.matrix_shape(wr)[0] == (E + 15) // 16 * 16) == (stored != torch.float32)
        for T in (1, 5, 16, 17, 130):
            h = torch.randn(T, K, generator=g).to(DT[dtype])
            z = h.double() @ W.double().T + bias.double()
            best = torch.topk(z, min(top + 1, E), -1).values
            if E > top:                                                      # only rows without a close call
                keep = (best[:, top - 1] - best[:, top]) > 1e-4
                if keep.sum() == 0:
                    continue
                h, z = h[keep].contiguous(), z[keep]
            chosen = torch.topk(z, top, -1).indices.sort(-1).values
            weights = torch.softmax(z.gather(1, chosen), -1)
            p = ops.route_pairs(h.to(DEV), wr, bias.to(DEV), E, top)
            check_pairs(p, chosen, weights)
            p = ops.route_pairs(h.to(DEV), wr, None, E, top, 2.5)
            zz = z - bias.double()
            assert torch.allclose(p.weights.cpu().double(), 2.5 * torch.softmax(zz.gather(1, p.chosen.cpu().long()), -1), atol=5e-6)


def test_the_first_of_equal_logits_is_chosen_and_numbers_that_are_none_do_no_harm(lib):
    from llm_infer_amd.kernels import ops
    h = torch.ones(20, 32, dtype=torch.bfloat16, device=DEV)
    wr = ops.router_weight(torch.ones(6, 32, device=DEV), torch.bfloat16)
    p = ops.route_pairs(h, wr, None, 6, 3)
    check_pairs(p, torch.tensor([[0, 1, 2]] * 20), torch.full((20, 3), 1.0 / 3.0, dtype=torch.float64))
    for T in (3, 20):
        bad = h[:T].clone()
        bad[1, 3] = float("nan")
        p = ops.route_pairs(bad, wr, None, 6, 3)
        c = p.chosen.cpu()
        assert int(c.min()) >= 0 and int(c.max()) < 6 and all(len(set(r)) == 3 for r in c.tolist())
        assert int(p.counts.sum()) == 3 * T and sorted(p.slot_of.cpu().flatten().tolist()) == list(range(3 * T))


@pytest.mark.parametrize("dtype", ["bfloat16", "float16"])
def test_products_by_pairs_in_every_kernel(lib, dtype):
    """Experts with no pairs, with one, with a tile's worth and one more, and with nearly all; gathered rows and rows in
    place; stored and gated; every tile."""
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(12)
    for E, K, F_, counts in ((5, 64, 32, [1, 0, 3, 0, 0]), (4, 2080, 48, [0, 17, 1, 33]), (70, 96, 16, [0] * 30 + [2] + [0] * 30 + [40, 1] + [0] * 7),
                             (3, 128, 160, [129, 0, 400]), (9, 64, 64, [64, 65, 0, 128, 1, 127, 0, 63, 300])):
        n = sum(counts)
        T, top = n, 1
        p = ops.SortedPairs(T, top, E, DEV)
        chosen = torch.repeat_interleave(torch.arange(E), torch.tensor(counts))[torch.randperm(n, generator=g)].to(torch.int32)
        p.chosen.copy_(chosen.view(T, 1))
        p.weights.fill_(1.0)
        from llm_infer_amd.kernels.ops import _check, _ptr, _stream, experts
        _check(experts().li_sort_pairs(_ptr(p.chosen), n, top, E, _ptr(p.counts), _ptr(p.offsets), _ptr(p.row_of), _ptr(p.slot_of), _stream()), "sort")
        check_pairs(p, chosen.long().view(T, 1), torch.ones(T, 1, dtype=torch.float64))
        x = torch.randn(T, K, generator=g).to(DT[dtype])
        w = (torch.randn(E, 2 * F_, K, generator=g) * K ** -0.5 * 2).to(DT[dtype])
        wt = ops.prepare_weight(w.view(E * 2 * F_, K).to(DEV))
        row_of = p.row_of.cpu().long()
        for gather in (True, False):
            xr = x[row_of] if gather else x
            z = torch.stack([w[chosen[row_of[i]].long()].double() @ xr[i].double() for i in range(n)])
            h = P.silu(z[:, 0::2]) * z[:, 1::2]
            for force in (None, "gemv", "wreg:0:0", "wreg:1:0", "wreg:2:0", "wreg:2:1"):
                got = ops.linear_pairs(x.to(DEV), wt, p, ops.EPI_STORE, gather, torch.float32, force).cpu()
                assert error(got, z) < 2e-2, (E, gather, force)
                got = ops.linear_pairs(x.to(DEV), wt, p, ops.EPI_SWIGLU, gather, force=force).cpu()
                assert got.dtype == DT[dtype] and error(got, h) < 6e-2, (E, gather, force)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16", "float16"])
@pytest.mark.parametrize("width,ff,E,top", [(96, 40, 5, 2), (64, 33, 9, 9), (72, 24, 4, 2), (128, 64, 40, 3)])
def test_routed_experts_alone(lib, dtype, width, ff, E, top):
    """One step and many, by pairs (a width that tiles) or through every expert (one that does not, and float32), on
    tokens whose choice differs from token to token with a margin that no rounding can turn: a token's input has large
    entries where its experts' router rows have their only weights."""
    from llm_infer_amd.parts.feed_forward import RoutedExperts
    from llm_infer_amd.registry import config_from_dict
    from llm_infer_amd.weights.loader import place_tensor
    mlp = M.moe(E, top, ff)
    raw = M.config(width, 50, [M.layer(M.attention(1, 1, 16, 16, 8), mlp)])
    spec = config_from_dict(raw)._layer_spec(0, raw["layers"][0]).sublayers[1].part.with_prefix("")
    g = torch.Generator().manual_seed(31 + E)
    W = M.mlp_weights(mlp, width, g, torch.bfloat16)
    W["router"] = torch.zeros(E, width, dtype=torch.bfloat16)
    W["router"][torch.arange(E), torch.arange(E)] = 2.0
    W["router.b"] = (torch.randint(-2, 3, (E,), generator=g) * 0.125).to(torch.bfloat16)
    part = RoutedExperts(**spec.params, prefix="", dtype=DT[dtype], device=DEV)
    wanted = part.params()
    assert set(wanted) == set(W)
    part.bind({n: place_tensor(W[n], wanted[n].kind, DT[dtype], DEV) for n in wanted})
    assert part.paired == (dtype != "float32" and width % 32 == 0)
    for T in (1, 9, 70, 400):
        h = torch.randn(T, width, generator=g)
        h[:, :E] = torch.rand(T, E, generator=g).argsort(-1).argsort(-1).float()      # every token its own order of the experts
        h = (h * (4.0 / E)).to(torch.bfloat16)
        ref = P.experts(h.double(), M.widen(W), mlp)
        tol = M.tolerance("float32" if dtype == "float32" else "bfloat16", ref, P.experts(h.double(), M.widen(W), mlp, torch.bfloat16), error)
        res = torch.ones(T, width, device=DEV)
        part.forward(h.to(DEV).to(DT[dtype]), res)
        assert error(res.cpu() - 1.0, ref) < tol, T
        into = torch.full((T, width), 7.0, device=DEV)
        if part.makes_rows:
            into = part.forward_rows(h.to(DEV).to(DT[dtype])).tensor()
        else:
            part.forward_into(h.to(DEV).to(DT[dtype]), into)
        assert error(into.cpu(), ref) < tol, T


# ---------------------------------------------------------------------------- the mixers alone
def build_mixer(raw_cfg, i, weights, dtype):
    """Layer i's mixer as the configuration describes it, with the given tensors bound."""
    import llm_infer_amd.parts  # noqa: F401  (registers the parts)
    from llm_infer_amd.registry import config_from_dict, lookup
    from llm_infer_amd.weights.loader import place_tensor
    cfg = config_from_dict(raw_cfg)
    spec, position = cfg._mixer(raw_cfg["layers"][i], ""), cfg._position(raw_cfg["layers"][i])
    pos = None
    if position is not None:
        pos = lookup("position", position.kind)(**position.params, prefix="", dtype=DT[dtype], device=DEV)
    part = lookup("mixer", spec.kind)(**spec.params, position=pos, prefix="", dtype=DT[dtype], device=DEV)
    wanted = part.params()
    assert set(wanted) == set(weights), set(wanted) ^ set(weights)
    part.bind({n: place_tensor(weights[n], wanted[n].kind, DT[dtype], DEV) for n in wanted})
    return part


def run_mixer(part, h_of, schedule, dtype):
    """Runs a mixer over ``schedule`` (steps {request: tokens it brings}) on the inputs ``h_of[r]`` [n, width]; returns
    {r: what the mixer added, [n, width]}."""
    from llm_infer_amd.cache import Cache
    from llm_infer_amd.parts.base import cache_specs_of
    specs = cache_specs_of(part)
    cache = Cache(specs, 8192, 8192, DT[dtype], DEV)
    views = [cache.view(i) for i in range(len(specs))] if hasattr(part, "cache_specs") else cache.view(0)
    slot, at, out = {}, {r: 0 for r in h_of}, {r: [] for r in h_of}
    for step in schedule:
        rs = list(step)
        for r in rs:
            if r not in slot:
                slot[r] = cache.alloc_slot()
        cache.grow([slot[r] for r in rs], [at[r] + step[r] for r in rs], filled=True)
        ctx = step_context([slot[r] for r in rs], [at[r] for r in rs], [[0] * step[r] for r in rs])
        h = torch.cat([h_of[r][at[r]:at[r] + step[r]] for r in rs]).to(DEV).to(DT[dtype])
        res = torch.zeros((h.shape[0], h.shape[1]), dtype=torch.float32, device=DEV)
        part.forward(h, ctx, views, res)
        cache.trim_windows([slot[r] for r in rs])
        # what no sequence holds any more holds numbers that are none: whoever reads it shows
        if cache.groups[0].trims:
            free = sorted(set(range(1, cache.n_pages)) - cache.groups[0].pool.held())
            cache.groups[0].storage[free] = float("nan")
        for r, part_rows in zip(rs, res.cpu().split([step[r] for r in rs])):
            out[r].append(part_rows)
            at[r] += step[r]
        for r in rs:
            if at[r] == h_of[r].shape[0]:
                cache.free_slot(slot.pop(r))
    return {r: torch.cat(v) for r, v in out.items()}


SCHEDULES = {
    "whole": lambda n, m: [{"a": n}, {"b": m}],
    # portions down to two tokens and one, across page edges (64) and the masks' edges
    "portions": lambda n, m: [{"a": 61}, {"a": 2}, {"a": 1}, {"a": 2}, {"a": 70}, {"a": n - 136}, {"b": 1}, {"b": m - 1}],
    # unequal requests together, decoded together, the longer one alone, then a slot used again
    "together": lambda n, m: [{"a": n - 20, "b": m - 5}] + [{"a": 1, "b": 1}] * 5 + [{"a": 1}] * 15 + [{"c": 30}],
}

MIXERS = [
    M.latent(3, 20, 12, 24, 28, 36, base=500.0, scaling=(4.0, 60, 8.0, 1.0)),     # nothing a multiple of 16
    M.latent(40, 16, 16, 16, 32, 32, scaling=(16.0, 30, 4.0, 0.5)),               # two tiles of heads
    M.latent(1, 8, 0, 40, 16, 5),                                                 # nothing turned, one head
    M.latent(4, 64, 64, 64, 128, 96, scaling=(40.0, 4096, 32.0, 1.0)),
    M.latent(3, 16, 20, 16, 300, 40, scaling=(4.0, 60, 8.0, 1.0)),                # a latent beyond what the matrix-core kernel takes
    M.attention(2, 1, 272, 40, 30, 3),                                            # keys beyond it, with kept tokens
    M.attention(3, 1, 20, 9, 30, 3),                                              # a padded head, values narrower than keys
    M.attention(4, 4, 8, 40, 1, 2),                                               # only the token itself and the first two
    M.attention(16, 2, 64, 64, 70, 65),                                           # one size: the other kernels; more than a page kept
    M.attention(5, 1, 32, 32, 20, 1),
    M.attention(8, 8, 16, 32, 100, 7),                                            # one head each
    M.attention(6, 2, 48, 64, 64, 64),                                            # window = kept = page
    M.attention(4, 2, 32, 32, 1000, 5),                                           # a window never reached
    M.attention(4, 1, 16, 16, 33, 0),                                             # nothing kept
]


@pytest.mark.parametrize("schedule", sorted(SCHEDULES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mixer", MIXERS, ids=lambda m: f"{m[0]}-{m[1]['heads']}x{m[1]['dim']}-{m[1].get('mask', {}).get('size', m[1].get('kv_rank'))}")
def test_mixer_alone(lib, mixer, dtype, schedule):
    width, n, m_ = 96, 200, 40
    raw = M.config(width, 50, [M.layer(mixer, None)])
    g = torch.Generator().manual_seed(11)
    W = M.mixer_weights(mixer[0], mixer[1], width, g, torch.bfloat16, sharp=2.0)
    part = build_mixer(raw, 0, W, dtype)
    h_of = {r: torch.randn(k, width, generator=g).to(torch.bfloat16).float() for r, k in (("a", n), ("b", m_), ("c", 30))}
    sched = SCHEDULES[schedule](n, m_)
    got = run_mixer(part, {r: h_of[r] for r in {k for s in sched for k in s}}, sched, dtype)
    Wd = M.widen(W)
    fn = P.attention_mixer if mixer[0] == "attention" else P.latent_mixer
    for r, rows_ in got.items():
        ref = fn(h_of[r].double(), Wd, mixer[1], 1e-5)
        tol = M.tolerance(dtype, ref, fn(h_of[r].double(), Wd, mixer[1], 1e-5, torch.bfloat16), error)
        assert error(rows_, ref) < tol, r


def test_frequencies_and_magnitude_reach_the_latent_attention_in_every_setting(lib):
    """Far positions, where a wrong frequency shows, and a magnitude that shows at once."""
    for scaling in (None, (8.0, 64, 16.0, 1.0), (40.0, 4096, 32.0, 1.0)):
        mixer = M.latent(2, 4, 32, 16, 32, 32, base=1000.0, scaling=scaling)
        raw = M.config(64, 50, [M.layer(mixer, None)])
        g = torch.Generator().manual_seed(13)
        W = M.mixer_weights(mixer[0], mixer[1], 64, g, torch.bfloat16, sharp=3.0)
        h = torch.randn(500, 64, generator=g).to(torch.bfloat16).float()
        ref = P.latent_mixer(h.double(), M.widen(W), mixer[1], 1e-5)
        if scaling is not None:
            plain = dict(mixer[1], rot={"base": 1000.0, "dims": 32})
            assert error(P.latent_mixer(h.double(), M.widen(W), plain, 1e-5), ref) > 0.1
        got = run_mixer(build_mixer(raw, 0, W, "float32"), {"a": h}, [{"a": 450}] + [{"a": 1}] * 50, "float32")["a"]
        assert error(got, ref) < 5e-4                                        # (float32 angles of some hundred turns)


# ---------------------------------------------------------------------------- edges, kept tokens, far keys, sinks
# (keys and values of one size that is a multiple of 16 run on one pair of kernels, other sizes on another)
@pytest.mark.parametrize("vdim", [32, 16])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_just_inside_and_just_outside_the_window_in_prompts_portions_and_decoding(lib, dtype, vdim, tmp_path):
    size, n, at = 70, 180, 30
    mixer = M.attention(4, 2, 32, vdim, size, 5)
    cfg = M.config(64, 60, [M.layer(mixer, M.moe(3, 2, 32))], scale=0.3)
    W = M.stand_out(M.random_weights(cfg, 80, steady=True), cfg, 0, 7, strength=5.0)
    Wd = M.widen(W)
    toks = [t if t != 7 else 8 for t in tokens(cfg, n, 5)]
    toks[at] = 7
    last_seen = at + size - 1
    ref = P.forward(cfg, Wd, toks)
    tol = M.tolerance(dtype, ref, P.forward(cfg, Wd, toks, round_to=torch.bfloat16))
    # the plain implementation alone: a window of one more or less moves the rows at its edge far beyond the tolerance
    for wrong in (size - 1, size + 1):
        off = P.forward(M.with_mask(cfg, 0, size=wrong), Wd, toks)
        assert M.row_error(off[[last_seen, last_seen + 1]], ref[[last_seen, last_seen + 1]]) > SHOWS[dtype] * tol, wrong
    eng = load(lib, tmp_path, cfg, W, dtype)
    for name, sched in (("prompt", [{"a": n}]),
                        ("portions", [{"a": last_seen - 1}, {"a": 2}, {"a": 2}, {"a": n - last_seen - 3}]),
                        ("decoding", [{"a": last_seen - 3}] + [{"a": 1}] * 8 + [{"a": n - last_seen - 5}])):
        assert M.row_error(run_schedule(eng, {"a": toks}, sched)["a"], ref) < tol, name


@pytest.mark.parametrize("keep,at,kept", [(6, 5, True), (6, 6, False), (65, 64, True), (64, 64, False), (1, 0, True), (0, 0, False), (33, 31, True)])
@pytest.mark.parametrize("vdim", [32, 16])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_last_kept_token_and_the_next_one(lib, dtype, vdim, keep, at, kept, tmp_path):
    """A token that stands out as the last of those a window keeps, or right behind them, far from the window: in a prompt, in
    portions, decoded; across pages that were given back meanwhile."""
    n, size = 330, 40
    mixer = M.attention(4, 1, 32, vdim, size, keep)
    cfg = M.config(64, 60, [M.layer(mixer, None)], scale=0.3)
    W = M.stand_out(M.random_weights(cfg, 81), cfg, 0, 7, strength=7.0)
    Wd = M.widen(W)
    toks = [t if t != 7 else 8 for t in tokens(cfg, n, 6)]
    toks[at] = 7
    ref = P.forward(cfg, Wd, toks)
    tol = M.tolerance(dtype, ref, P.forward(cfg, Wd, toks, round_to=torch.bfloat16))
    far = list(range(120, n))
    wrong = P.forward(M.with_mask(cfg, 0, keep_first=at if kept else at + 1), Wd, toks)
    assert M.row_error(wrong[far], ref[far]) > SHOWS[dtype] * tol            # (one kept token more or less shows)
    eng = load(lib, tmp_path, cfg, W, dtype)
    for sched in ([{"a": n}], [{"a": 3}, {"a": 2}, {"a": 62}, {"a": 100}, {"a": n - 167}], [{"a": 100}] + [{"a": 1}] * (n - 100)):
        assert M.row_error(run_schedule(eng, {"a": toks}, sched)["a"], ref) < tol


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_key_among_hundreds_of_latents(lib, dtype, tmp_path):
    cfg = M.config(64, 60, [M.layer(M.latent(4, 16, 16, 16, 32, 32, scaling=(4.0, 100, 8.0, 1.0)), None)], scale=0.3)
    W = M.stand_out(M.random_weights(cfg, 78), cfg, 0, 7, strength=5.0)
    n = 700
    base = [t if t != 7 else 8 for t in tokens(cfg, n, 6)]
    toks = list(base)
    toks[3] = 7
    Wd = M.widen(W)
    ref, without = P.forward(cfg, Wd, toks), P.forward(cfg, Wd, base)
    tol = M.tolerance(dtype, ref, P.forward(cfg, Wd, toks, round_to=torch.bfloat16))
    far = list(range(600, 700))
    assert M.row_error(without[far], ref[far]) > SHOWS[dtype] * tol          # the rows far away feel the key at position 3
    eng = load(lib, tmp_path, cfg, W, dtype)
    for sched in ([{"a": n}], [{"a": 640}] + [{"a": 1}] * 60, [{"a": 130}, {"a": 500}, {"a": 70}]):
        assert M.row_error(run_schedule(eng, {"a": toks}, sched)["a"], ref) < tol


@pytest.mark.parametrize("vdim", [16, 32])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sinks_that_differ_widely_between_the_heads(lib, dtype, vdim, tmp_path):
    cfg = M.config(64, 60, [M.layer(M.attention(4, 2, 32, vdim, 90, 4), None)], scale=0.3)
    W = M.random_weights(cfg, 79, sharp=2.0)
    toks = tokens(cfg, 200, 7)
    ref0 = P.forward(cfg, M.widen(W), toks)
    W["l0.mix.sink"] = torch.tensor([-4.0, 9.0, 2.0, 30.0]).to(torch.bfloat16)
    Wd = M.widen(W)
    ref = P.forward(cfg, Wd, toks)
    tol = M.tolerance(dtype, ref, P.forward(cfg, Wd, toks, round_to=torch.bfloat16))
    assert M.row_error(ref0, ref) > SHOWS[dtype] * tol
    eng = load(lib, tmp_path, cfg, W, dtype)
    for sched in ([{"a": 200}], [{"a": 150}] + [{"a": 1}] * 50):
        assert M.row_error(run_schedule(eng, {"a": toks}, sched)["a"], ref) < tol


# ---------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("name", sorted(M.ALL))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_model_whole_first_tokens_portions_and_token_by_token(lib, models, dtype, name):
    folder, cfg, W = models[name, dtype]
    n = 210
    toks = tokens(cfg, n, 9)
    ref = P.forward(cfg, W, toks)
    tol = M.tolerance(dtype, ref, P.forward(cfg, W, toks, round_to=torch.bfloat16))
    eng = lib.load(folder, dtype=dtype, max_tokens=2048)
    reqs = {"a": toks}
    whole = run_schedule(eng, reqs, [{"a": n}])["a"]
    assert M.row_error(whole, ref) < tol
    for k in (1, 2, 3):                                                     # the first tokens alone
        assert M.row_error(run_schedule(eng, {"a": toks[:k]}, [{"a": k}])["a"], ref[:k]) < tol
    portions = run_schedule(eng, reqs, [{"a": 2}, {"a": 1}, {"a": 62}, {"a": 2}, {"a": 5}, {"a": 129}, {"a": n - 201}])["a"]
    one_by_one = run_schedule(eng, reqs, [{"a": 1}] * n)["a"]
    for got in (portions, one_by_one):
        assert M.row_error(got, ref) < tol
        if dtype == "float32":
            assert M.row_error(got, whole) < 2e-5


def test_a_bfloat16_model_whose_choices_differ_from_token_to_token(lib, tmp_path):
    """A short prompt on which every choice of experts has a clear margin in the plain implementation, rounded or not."""
    cfg = M.TINY_A
    top = {i: l["mlp"]["router"]["top"] for i, l in enumerate(cfg["layers"]) if l["mlp"]}

    def margins(W, toks, round_to):
        seen, plain = [], P.expert_weights

        def spy(h, Wm, k):
            z = h @ Wm["router"].T + Wm["router.b"]
            best = torch.topk(z, k + 1, -1).values
            seen.append(((best[:, k - 1] - best[:, k]).min().item(), plain(h, Wm, k) > 0))
            return plain(h, Wm, k)
        P.expert_weights = spy
        try:
            out = P.forward(cfg, W, toks, round_to=round_to)
        finally:
            P.expert_weights = plain
        return min(s for s, _ in seen), [c for _, c in seen], out
    for seed in range(300):
        W = M.random_weights(cfg, 500 + seed, sharp=1.5)
        Wd, toks = M.widen(W), tokens(cfg, 12, seed)
        gap, chosen, ref = margins(Wd, toks, None)
        if gap < 0.06:
            continue
        gap16, chosen16, ref16 = margins(Wd, toks, torch.bfloat16)
        if gap16 > 0.04 and all(torch.equal(a, b) for a, b in zip(chosen, chosen16)):
            break
    else:
        pytest.fail("no prompt with clear margins found")
    assert len(top) == 3 and any(not torch.equal(c, c[:1].expand_as(c)) for c in chosen)      # the choices do differ
    eng = load(lib, tmp_path, cfg, W, "bfloat16")
    for sched in ([{"a": 12}], [{"a": 5}] + [{"a": 1}] * 7):
        assert M.row_error(run_schedule(eng, {"a": toks}, sched)["a"], ref) < M.tolerance("bfloat16", ref, ref16)


@pytest.mark.parametrize("name", sorted(M.ALL))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_together_against_each_alone(lib, models, dtype, name):
    folder, cfg, W = models[name, dtype]
    reqs = {"a": tokens(cfg, 150, 12), "b": tokens(cfg, 1, 13), "c": tokens(cfg, 67, 14), "d": tokens(cfg, 230, 15),
            "e": tokens(cfg, 40, 16)}
    ref = {r: P.forward(cfg, W, t) for r, t in reqs.items()}
    tol = {r: M.tolerance(dtype, ref[r], P.forward(cfg, W, t, round_to=torch.bfloat16)) for r, t in reqs.items()}
    eng = lib.load(folder, dtype=dtype, max_tokens=1024, n_slots=4)
    # slots and pages used before, and given back in between
    first = run_schedule(eng, {"a": reqs["a"], "e": reqs["e"]}, [{"a": 150, "e": 40}])
    sched = [{"a": 140, "b": 1, "c": 60, "d": 190}] + [{"a": 1, "c": 1, "d": 1}] * 7 + [{"a": 1, "d": 1}] * 3 + \
        [{"d": 1, "e": 40}] + [{"d": 1}] * 29
    got = run_schedule(eng, reqs, sched)
    for r in reqs:
        assert M.row_error(got[r], ref[r]) < tol[r], r
    for r in first:
        assert M.row_error(first[r], ref[r]) < tol[r], r
    assert eng.cache.tokens_free() == (eng.cache.n_pages - 1) * 64         # every page came back


@pytest.mark.parametrize("name,dtype,graph", [("A", "float32", True), ("A", "bfloat16", True), ("A", "bfloat16", False), ("B", "float32", True),
                                              ("C", "bfloat16", True)])
def test_long_decoding_and_generation(lib, models, name, dtype, graph):
    """Greedy generation through the library's own loop (recorded and eager decode steps), across windows and pages that are
    given back, against the plain implementation's choice wherever its logits leave a margin."""
    folder, cfg, W = models[name, dtype]
    eng = lib.load(folder, dtype=dtype, max_tokens=4096)
    prompts = [tokens(cfg, 70, 21), tokens(cfg, 3, 22), tokens(cfg, 1, 23)]
    new = eng.generate(prompts, max_new_tokens=150, temperature=0.0, use_graph=graph)
    assert all(len(t) == 150 for t in new)
    if graph:
        assert eng.decode_counts["replayed"] > 100
    checked = 0
    for p, out in zip(prompts, new):
        logits = P.forward(cfg, W, list(p) + out)
        margin = (1e-3 if dtype == "float32" else 0.15) * logits.std().item()
        for k, t in enumerate(out):
            row = logits[len(p) - 1 + k]
            top2 = torch.topk(row, 2).values
            if (top2[0] - top2[1]).item() < margin:
                continue
            assert t == int(row.argmax()), (dtype, graph, k)
            checked += 1
    assert checked > (400 if dtype == "float32" else 100), checked


def test_recorded_steps_whose_experts_change_from_step_to_step(lib, models, tmp_path):
    """A recorded decode step is replayed with other tokens, lengths and so other experts: the same tokens as eager steps give."""
    cfg = M.TINY_C
    W = M.random_weights(cfg, 90, sharp=2.0)                                 # (no steady choice here)
    folder = str(tmp_path / "m")
    M.write_model(folder, cfg, W)
    prompts = [tokens(cfg, n, 60 + n) for n in (5, 40, 71)]
    outs = []
    for graph in (True, False):
        eng = lib.load(folder, dtype="bfloat16", max_tokens=2048)
        outs.append(eng.generate(prompts, max_new_tokens=60, temperature=0.0, use_graph=graph))
    assert outs[0] == outs[1]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_in_three_schedules(lib, models, dtype, tmp_path):
    folder, cfg, W = models["B", dtype]
    reqs = {"r1": tokens(cfg, 75, 41), "r2": tokens(cfg, 1, 42), "r3": tokens(cfg, 140, 43)}
    ref = {r: P.forward(cfg, W, t) for r, t in reqs.items()}
    tol = {r: M.tolerance(dtype, ref[r], P.forward(cfg, W, t, round_to=torch.bfloat16)) for r, t in reqs.items()}
    for k, (steps, where) in enumerate((TU.steps_whole(reqs), TU.steps_tail(reqs, 33), TU.steps_batches(reqs, 3, {"r1": 10, "r3": 70}))):
        out_dir = str(tmp_path / f"out{k}")
        got = TU.run_trace(folder, dtype, steps, where, cfg["vocab"], 300, out_dir)
        assert set(got) == {(r, p) for r, t in reqs.items() for p in range(len(t))}
        for r, t in reqs.items():
            g = torch.stack([torch.from_numpy(got[r, p].copy()) for p in range(len(t))])
            assert M.row_error(g, ref[r]) < tol[r], (k, r)


def test_command_line_reports_and_generates(lib, models):
    folder, cfg, W = models["A", "float32"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompts = [tokens(cfg, 9, 51), tokens(cfg, 2, 52)]
    cmd = [sys.executable, os.path.join(root, "bin", "infer"), folder, "-n", "6", "-t", "0", "--dtype", "float32", "-T", "64"]
    for p in prompts:
        cmd += ["--tokens", ",".join(map(str, p))]
    res = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert res.returncode == 0, res.stderr
    got = [json.loads(line.split("tokens: ", 1)[1]) for line in res.stdout.splitlines() if " tokens: [" in line]
    assert len(got) == 2
    for p, new in zip(prompts, got):
        toks = list(p)
        for t in new:
            last = P.forward(cfg, W, toks)[-1]
            top2 = torch.topk(last, 2).values
            if (top2[0] - top2[1]).item() > 1e-3:
                assert t == int(last.argmax())
            toks.append(t)
    for word in ("Dimensions: 96", "Vocab size: 131"):
        assert word in res.stdout, res.stdout
    info = subprocess.run([sys.executable, os.path.join(root, "bin", "model_info"), folder], capture_output=True, text=True,
                          timeout=300)
    assert info.returncode == 0 and "Architecture: Pusisun" in info.stdout and "The tensors fit the model." in info.stdout
