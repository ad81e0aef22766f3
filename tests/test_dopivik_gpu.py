"""Dopivik on the GPU against the plain implementation: every kernel and mixer alone, whole prompts, prompts cut into
portions, decoding token by token, batches of unequal requests against each alone, slots and pages used again, keys
far away, at page borders and just inside and just outside a chunk, the soft cap, the first tokens, long decoding, other
sizes, layers with another's weights, and greedy generation through the library's entry point.

Where random weights would hide a fault, a token's key is made to stand out for every query (``dopivik_models.stand_out``)
and the test first shows, with the plain implementation alone, that the fault it looks for would move the result far
beyond the tolerance."""
import json
import os
import subprocess
import sys

import pytest
import torch

import dopivik_models as M
import plain_dopivik as P
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
        W = M.random_weights(cfg, 40 + ord(name), sharp=2.0)
        folder = str(tmp_path_factory.mktemp(f"dopivik_{name}"))
        M.write_model(folder, cfg, W)
        out[name] = (folder, cfg, M.widen(W))
    return out


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def step_context(slots, lens_before, toks):
    from llm_infer_amd.engine.step import StepContext
    return StepContext(DEV, list(slots), [list(t) for t in toks], list(lens_before), [[] for _ in toks])


def error(got, ref):
    """Largest difference relative to the reference's spread."""
    return ((got.double().cpu() - ref.double()).abs().max() / ref.double().std()).item()


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


def in_portions(lengths, schedule, clear, run):
    """Walks ``schedule`` (steps {request: tokens it brings}) over slots of a state (request c takes a's slot): calls
    ``clear(slot)`` when a request starts and ``run(ctx, pick)`` a step, ``pick(x)`` the step's rows of {request: rows}; returns
    {request: rows of the results}."""
    slot = {"a": 2, "b": 0, "c": 2}
    at, got = {r: 0 for r in lengths}, {r: [] for r in lengths}
    for step in schedule:
        rs = list(step)
        for r in rs:
            if at[r] == 0:
                clear(slot[r])
        ctx = step_context([slot[r] for r in rs], [at[r] for r in rs], [[0] * step[r] for r in rs])
        res = run(ctx, lambda x: torch.cat([x[r][at[r]:at[r] + step[r]] for r in rs]).to(DEV))
        for r, part in zip(rs, res.split([step[r] for r in rs], dim=-2)):
            got[r].append(part.cpu())
            at[r] += step[r]
    return {r: torch.cat(v, dim=-2) for r, v in got.items()}


PORTIONS = ({"a": 1}, {"a": 2, "b": 5}, {"a": 1, "b": 1}, {"a": 37}, {"c": 1}, {"c": 33}, {"c": 1})
LENGTHS = {"a": 41, "b": 6, "c": 35}


# ---------------------------------------------------------------------------- kernels alone
@pytest.mark.parametrize("width", [96, 70, 1024, 1100, 4096, 8200, 20000])
def test_layer_norm_and_the_pass_behind_a_sub_layer(lib, width):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    for n in (3, 70):
        x, y, z = (torch.randn(n, width, generator=g) * s + 0.3 for s in (1.0, 3.0, 0.5))
        w, b, w1, w2, nw, nb = (torch.randn(width, generator=g) for _ in range(6))
        d = lambda t: t.double()
        dev = lambda t: t.clone().to(DEV)
        pick = torch.randint(0, n, (5,), generator=g, dtype=torch.int32)
        for dt in (torch.float32, torch.bfloat16):
            tol = dict(rtol=1e-5 if dt == torch.float32 else 2.0 ** -8, atol=2e-5)
            for bias in (None, b):
                ref = P.layer_norm(d(x), d(w), 0 if bias is None else d(bias), 1e-3)
                bd = None if bias is None else dev(bias)
                assert torch.allclose(d(ops.layernorm(dev(x), dev(w), 1e-3, dt, None, bd).cpu()), ref, **tol)
                assert torch.allclose(d(ops.layernorm(dev(x), dev(w), 1e-3, dt, pick.to(DEV), bd).cpu()), ref[pick.long()], **tol)
        pair = 0.5 * (P.rms(d(y), 1e-2) * d(w1) + P.rms(d(z), 1e-2) * d(w2))
        make = lambda: ops.NormedPair(dev(y), dev(w1), dev(z), dev(w2), 1e-2, 0.5)
        assert error(make().rows(), pair) < 3e-6
        for source, made in ((d(y), lambda: dev(y)), (pair, make)):
            ref = d(x) + P.layer_norm(source, d(w), d(b), 1e-3)
            xd = ops.layernorm_add(dev(x), made(), dev(w), dev(b), 1e-3)
            assert error(xd, ref) < 3e-6
            for dt in (torch.float32, torch.bfloat16):
                xd, nwd = dev(x), dev(nw)
                ops.layernorm_add(xd, made(), dev(w), None, 1e-3, (nwd, dev(nb), 1e-5, dt))
                ref = d(x) + P.layer_norm(source, d(w), 0, 1e-3)
                assert error(xd, ref) < 3e-6
                ready = ops.prepared_norm(xd, nwd, 1e-5, dt)
                assert ready is not None and ops.prepared_norm(xd, nwd, 1e-4, dt) is None
                assert torch.allclose(d(ready.cpu()), P.layer_norm(ref, d(nw), d(nb), 1e-5), rtol=1e-5 if dt == torch.float32 else 2.0 ** -8, atol=2e-5)
                ops.add_bias(xd, 0, nwd)                                  # anything written into the rows voids what was prepared
                assert ops.prepared_norm(xd, nwd, 1e-5, dt) is None


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
def test_convolution_with_silu_in_portions(lib, taps):
    """Portions shorter than the reach, two sequences at once, steps of one token each, a slot used again."""
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(4)
    C, extra = 10, 3
    w, b = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
    u = {r: torch.randn(n, C + extra, generator=g) for r, n in LENGTHS.items()}
    for bias in (None, b):
        hist = torch.full((4, max(taps - 1, 1), C), 7.0, device=DEV)           # what an earlier sequence left
        got = in_portions(LENGTHS, PORTIONS, lambda s: hist[s].zero_(),
                          lambda ctx, pick: ops.conv_silu(pick(u), 2, C, w.to(DEV), None if bias is None else bias.to(DEV), hist, ctx))
        for r in u:
            assert error(got[r], P.silu(P.causal_conv(u[r][:, 2:2 + C].double(), w.double(), None if bias is None else b.double()))) < 2e-6, r
    # many tokens at once: the form that walks several tokens a thread, over the edges of sequences
    lens = (300, 1, 2, 9, 40)
    u = [torch.randn(n, C, generator=g) for n in lens]
    hist = torch.zeros((5, max(taps - 1, 1), C), device=DEV)
    ctx = step_context(range(5), [0] * 5, [[0] * n for n in lens])
    got = ops.conv_silu(torch.cat(u).to(DEV), 0, C, w.to(DEV), b.to(DEV), hist, ctx).split(lens)
    for a, x in zip(got, u):
        assert error(a, P.silu(P.causal_conv(x.double(), w.double(), b.double()))) < 2e-6


@pytest.mark.parametrize("d", [20, 64])
def test_token_shift_with_several_mixes_in_portions(lib, d):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(5)
    mu = torch.rand(3, d, generator=g)
    x = {r: torch.randn(n, d, generator=g) for r, n in LENGTHS.items()}
    state = torch.full((4, d), 7.0, device=DEV)
    got = in_portions(LENGTHS, PORTIONS, lambda s: state[s].zero_(),
                      lambda ctx, pick: ops.token_shift(pick(x), mu.to(DEV), state, ctx.pos, ctx.tok_slot, torch.float32,
                                                        single=ctx.n_tokens == ctx.n_seqs))
    for r in x:
        before = torch.cat([torch.zeros(1, d), x[r][:-1]])
        ref = torch.stack([x[r] + (before - x[r]) * m for m in mu])
        assert got[r].shape == ref.shape and torch.allclose(got[r], ref, atol=1e-6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rows_", [3, 12, 40, 100, 300])
def test_products_with_an_activation_behind_them(lib, dtype, rows_):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(2 + rows_)
    for K, N in ((96, 70), (256, 200), (1024, 1536), (20, 33)):
        x = torch.randn(rows_, K, generator=g).to(torch.bfloat16)
        w = (torch.randn(N, K, generator=g) * K ** -0.5).to(torch.bfloat16)
        bias = torch.randn(N, generator=g)
        xd, wd = x.to(DEV).to(DT[dtype]), ops.prepare_weight(w.to(DEV).to(DT[dtype]))
        z = x.double() @ w.double().T
        for act, fn in (("relu2", P.relu_squared), ("tanh", torch.tanh)):
            for b in (None, bias):
                got = ops.linear(xd, wd, ops.EPI_BIAS, out_dtype=DT[dtype], params=ops.glu_params(None if b is None else b.to(DEV), act=act))
                ref = fn(z + (0 if b is None else b.double()))
                # (a 16-bit result: every element within that type's rounding)
                assert torch.allclose(got.double().cpu(), ref, rtol=1e-5 if dtype == "float32" else 2.0 ** -8, atol=3e-5), (K, N, act)


@pytest.mark.parametrize("m", [1, 5, 16, 20])
def test_several_products_of_few_rows_in_one_launch(lib, m):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(m)
    for K, R, last in ((64, 32, 7), (128, 96, 96), (256, 64, 20)):
        x = torch.randn(3, m, K, generator=g).to(torch.bfloat16)
        w = (torch.randn(2 * R + last, K, generator=g) * K ** -0.5).to(torch.bfloat16)
        tiled = ops.prepare_weight(w.to(DEV))
        got = ops.linear_groups(x.to(DEV), tiled, R).cpu()
        ref = torch.cat([x[i].double() @ w[i * R:(2 * R + last if i == 2 else (i + 1) * R)].double().T for i in range(3)], 1)
        assert error(got, ref) < 1e-5
        # the same storage cut into matrices of its own
        for i in range(3):
            part = tiled.rows_from(i * R, R if i < 2 else last)
            assert error(ops.linear(x[i].to(DEV), part, out_dtype=torch.float32), ref[:, i * R:i * R + (R if i < 2 else last)]) < 1e-5
        with pytest.raises(ValueError):
            tiled.rows_from(8, 16)


@pytest.mark.parametrize("dv,heads", [(7, 3), (32, 2), (64, 5), (128, 2), (256, 1), (130, 2)])
def test_head_norm_with_silu_gate_and_shared_weight(lib, dv, heads):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(dv)
    n = heads * dv
    y, gate = torch.randn(9, n, generator=g), torch.randn(9, n + 8, generator=g)
    for w in (torch.randn(dv, generator=g), torch.randn(n, generator=g)):
        o = P.rms(y.double().view(9, heads, dv), 1e-3)
        ref = (o * w.double().view(-1, dv)).reshape(9, n)
        for silu in (True, False):
            z = gate[:, 4:4 + n].double()
            got = ops.gated_head_norm(y.to(DEV), w.to(DEV), gate.to(DEV), 4, heads, 1e-3, torch.float32, gate_silu=silu)
            assert error(got, ref * (P.silu(z) if silu else torch.sigmoid(z))) < 5e-6


def decays(T, H, g, strong):
    """Logarithms of decays, most of them weak; with ``strong`` some tokens forget nearly everything or everything."""
    lg = -torch.rand(T, H, generator=g) * 0.3
    if strong:
        lg[T // 3], lg[T // 2] = -8.0, -60.0
    return lg


@pytest.mark.parametrize("H,G,d,dv", [(2, 1, 32, 64), (4, 2, 128, 128), (3, 3, 20, 9), (4, 1, 256, 40), (1, 1, 100, 33), (2, 2, 16, 200)])
def test_delta_rule_in_chunks_and_token_by_token(lib, H, G, d, dv):
    """Chunks of the matrix cores and the walk token by token, from a state that is not zero, sequences of every length around
    the chunk's, and the state they leave, against the plain recurrence."""
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(d)
    for lens, strong in (((77,), False), ((32, 5, 64, 1, 33), True), ((200,), True)):
        T = sum(lens)
        x = torch.randn(T, 2 * G * d + H * dv, generator=g).to(torch.bfloat16)
        q, k, v = (t.double() for t in (x[:, :G * d].view(T, G, d), x[:, G * d:2 * G * d].view(T, G, d), x[:, 2 * G * d:].view(T, H, dv)))
        rq, rk = d ** -0.5 / torch.sqrt((q * q).sum(-1) + 1e-6), 1 / torch.sqrt((k * k).sum(-1) + 1e-6)
        lg, beta = decays(T, H, g, strong), torch.rand(T, H, generator=g)
        qn, kn = q * rq[..., None], k * rk[..., None]
        start = torch.randn(len(lens), H, d, dv, generator=g)
        gates = torch.stack([lg, beta], -1).float().to(DEV).contiguous()
        norms = torch.stack([rq, rk], -1).float().to(DEV).contiguous()
        flat = torch.cat([qn.reshape(T, -1), kn.reshape(T, -1), v.reshape(T, -1)], 1).float().to(DEV).contiguous()
        weight, gate, eps = torch.randn(dv, generator=g), torch.randn(T, H * dv + 4, generator=g), 1e-3
        ctx = step_context(range(len(lens)), [0] * len(lens), [[0] * n for n in lens])
        runs = {"chunks": lambda st: ops.delta_chunks(x.to(DEV), gates, norms, st, ctx, H, G, d, dv),
                "scan": lambda st: ops.delta_scan(flat, gates, (qn * kn).sum(-1).float().to(DEV).contiguous(), st, ctx, H, G, d, dv)}
        if dv <= ops.SCAN_HEAD_LIMIT:
            runs["scan with the norm"] = lambda st: ops.delta_scan(flat, gates, (qn * kn).sum(-1).float().to(DEV).contiguous(), st, ctx, H, G, d,
                                                                   dv, (weight.to(DEV), gate.to(DEV), 4, eps, torch.float32))
        for name, run in runs.items():
            state = start.clone().to(DEV)
            y, at = run(state), 0
            for i, n in enumerate(lens):
                o, S = P.delta_rule(qn[at:at + n], kn[at:at + n], v[at:at + n], beta[at:at + n].double(), torch.exp(lg[at:at + n].double()), start[i].double())
                if name == "scan with the norm":
                    o = P.rms(o, eps) * weight.double() * P.silu(gate[at:at + n, 4:].double()).view(n, H, dv)
                # (sums of logarithms over a chunk that reach a hundred cost the chunked form some bits)
                tol = 1e-4 if strong and name == "chunks" else 1e-5
                assert error(y[at:at + n], o.reshape(n, -1)) < tol and error(state[i], S) < tol, (name, lens, n)
                at += n


@pytest.mark.parametrize("H,d", [(6, 32), (2, 64), (3, 20), (1, 256), (2, 100), (4, 128)])
def test_time_mixing_in_chunks_and_token_by_token(lib, H, d):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(d)
    for lens, strong in (((77,), False), ((32, 5, 64, 1, 33), True), ((200,), True)):
        T, c = sum(lens), H * d
        r, k, v = (torch.randn(T, c, generator=g) for _ in range(3))
        v = v.to(torch.bfloat16).float()
        raw = torch.randn(T, c, generator=g) * (1.0 if not strong else 2.0) - 1.5
        if strong:
            raw[T // 2] = 20.0                                             # e^-(e^20): everything is forgotten
            raw[T // 3, ::2] = -20.0                                       # nothing is
        u = torch.randn(H, d, generator=g)
        start = torch.randn(len(lens), H, d, d, generator=g)
        ctx = step_context(range(len(lens)), [0] * len(lens), [[0] * n for n in lens])
        dev = [t.to(DEV) for t in (r, k, v, raw, u)]
        wide = torch.cat([t.float() for t in (r, k, v)], 1).to(DEV)        # columns of wider rows
        weight, gate = torch.randn(c, generator=g), torch.randn(T, c, generator=g)
        runs = {"chunks": lambda st: ops.wkv_chunks(dev[0], dev[1], dev[2].to(torch.bfloat16), *dev[3:], st, ctx, H, d), "scan": lambda st: ops.wkv_scan(*dev, st, ctx, H, d),
                "scan of columns": lambda st: ops.wkv_scan(*(wide[:, i * c:(i + 1) * c] for i in range(3)), dev[3], dev[4], st, ctx, H, d)}
        if d <= ops.SCAN_HEAD_LIMIT:
            runs["scan with the norm"] = lambda st: ops.wkv_scan(*dev, st, ctx, H, d, (weight.to(DEV), gate.to(DEV), 0, 1e-3, torch.float32))
        w = torch.exp(-torch.exp(raw.double()))
        for name, run in runs.items():
            state = start.clone().to(DEV)
            y, at = run(state), 0
            for i, n in enumerate(lens):
                view = lambda t: t[at:at + n].double().view(n, H, d)
                o, S = P.wkv_rule(view(r), view(k), view(v), view(w), u.double(), start[i].double())
                if name == "scan with the norm":
                    o = P.rms(o, 1e-3).reshape(n, c) * weight.double() * P.silu(gate[at:at + n].double())
                # (sums of logarithms over a chunk that reach a thousand cost the chunked form some bits)
                assert error(y[at:at + n], o.reshape(n, -1)) < 2e-4 and error(state[i], S) < 2e-4, (name, lens, n)
                if name != "chunks" or not strong:
                    assert error(y[at:at + n], o.reshape(n, -1)) < 3e-5, (name, lens, n)
                at += n


@pytest.mark.parametrize("c,n", [(80, 5), (33, 1), (300, 16), (130, 33), (64, 256), (128, 64)])
def test_selective_scan_in_segments_and_in_order(lib, c, n):
    from llm_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(c)
    for lens, length in (((77,), 16), ((1, 40, 9, 23), 16), ((70, 3), None)):
        T = sum(lens)
        x, raw = torch.randn(T, c, generator=g), torch.randn(T, c, generator=g) * 2 - 1
        raw[T // 2] = 30.0                                                 # a large step: nearly everything is forgotten
        raw[T // 3] = -30.0                                                # none at all
        bias, Dk = torch.randn(c, generator=g) * 0.3, torch.randn(c, generator=g)
        A = -torch.exp(torch.randn(c, n, generator=g) * 0.7)
        bc, z = torch.randn(T, 3 + 2 * n, generator=g), torch.randn(T, c + 2, generator=g)
        start = torch.randn(len(lens), n, c, generator=g)
        a2 = (A.double() / torch.log(torch.tensor(2.0).double())).T.float().contiguous().to(DEV)
        ctx = step_context(range(len(lens)), [0] * len(lens), [[0] * k for k in lens])
        state = start.clone().to(DEV)
        y = ops.selective_scan(x.to(DEV), raw.to(DEV), bias.to(DEV), bc.to(DEV), 3, 3 + n, z.to(DEV), 2, a2, Dk.to(DEV), state, ctx,
                               None if length is None else ops.ssm_segments(ctx, length))
        dt, at = torch.nn.functional.softplus(raw.double() + bias.double()), 0
        for i, k in enumerate(lens):
            s = slice(at, at + k)
            o, S = P.selective_scan(x[s].double(), dt[s], A.double(), bc[s, 3:3 + n].double(), bc[s, 3 + n:].double(), Dk.double(), start[i].T.double())
            assert error(y[s], o * P.silu(z[s, 2:].double())) < 1e-5 and error(state[i], S.T) < 1e-5, (lens, k)
            at += k


# ---------------------------------------------------------------------------- the mixers alone
def build_mixer(mixer, width, weights, dtype):
    """A mixer as the configuration of a one-layer model describes it, with the given tensors bound."""
    import llm_infer_amd.parts  # noqa: F401  (registers the parts)
    from llm_infer_amd.parts.base import collect_params
    from llm_infer_amd.registry import config_from_dict, lookup
    from llm_infer_amd.weights.loader import place_tensor
    raw = M.config(width, 50, [M.layer(mixer)])
    cfg = config_from_dict(raw)
    spec, position = cfg._mixer(raw["layers"][0], ""), cfg._position(raw["layers"][0])
    pos = None
    if position is not None:
        pos = lookup("position", position.kind)(**position.params, prefix="", dtype=DT[dtype], device=DEV)
    part = lookup("mixer", spec.kind)(**spec.params, position=pos, prefix="", dtype=DT[dtype], device=DEV)
    table = collect_params(part)
    assert set(table) == set(weights), set(table) ^ set(weights)
    owners = {}
    for name, (p, local, _) in table.items():
        owners.setdefault(id(p), (p, {}))[1][local] = name
    for p, names in owners.values():
        p.bind({local: place_tensor(weights[n], table[n][2].kind, DT[dtype], DEV) for local, n in names.items()})
    if hasattr(part, "finish_bind"):
        part.finish_bind()
    return part


def run_mixer(part, h_of, schedule, dtype):
    """Runs a mixer over ``schedule`` (steps {request: tokens it brings}) on the inputs ``h_of[r]`` [n, width]; returns
    {r: what the mixer added, [n, width]}."""
    from llm_infer_amd.cache import Cache
    specs = part.cache_specs()
    cache = Cache(specs, 8192, 8192, DT[dtype], DEV)
    views = [cache.view(i) for i in range(len(specs))]
    slot, at, out = {}, {r: 0 for r in h_of}, {r: [] for r in h_of}
    for step in schedule:
        rs = list(step)
        for r in rs:
            if r not in slot:
                slot[r] = cache.alloc_slot()
        cache.grow([slot[r] for r in rs], [at[r] + step[r] for r in rs], filled=True)
        ctx = step_context([slot[r] for r in rs], [at[r] for r in rs], [[0] * step[r] for r in rs])
        h = torch.cat([h_of[r][at[r]:at[r] + step[r]] for r in rs]).to(DEV)
        h = h if getattr(part, "reads_float32", False) else h.to(DT[dtype])
        res = torch.zeros((h.shape[0], h.shape[1]), dtype=torch.float32, device=DEV)
        part.forward(h, ctx, views, res)
        cache.trim_windows([slot[r] for r in rs])
        for r, part_rows in zip(rs, res.cpu().split([step[r] for r in rs])):
            out[r].append(part_rows)
            at[r] += step[r]
        for r in rs:
            if at[r] == h_of[r].shape[0]:
                cache.free_slot(slot.pop(r))
    return {r: torch.cat(v) for r, v in out.items()}


SCHEDULES = {
    "whole": lambda n, m: [{"a": n}, {"b": m}],
    # portions down to two tokens and one, across page edges (64), the chunks of the masks and those of the recurrences (32)
    "portions": lambda n, m: [{"a": 61}, {"a": 2}, {"a": 1}, {"a": 2}, {"a": 70}, {"a": n - 136}, {"b": 1}, {"b": m - 1}],
    # unequal requests together, decoded together, the longer one alone, then a slot used again
    "together": lambda n, m: [{"a": n - 20, "b": m - 5}] + [{"a": 1, "b": 1}] * 5 + [{"a": 1}] * 15 + [{"c": 30}],
}
MIXERS = {
    "padded keys": M.parallel(M.left(4, 2, 24, 16, 50, dims=12, base=500.0, softcap=3.0), M.right(6, 2, 20, 24, conv=2)),
    "one size": M.parallel(M.left(8, 2, 64, 64, 130, base=2e5, softcap=2.0), M.right(4, 2, 128, 64)),
    "chunk is a page": M.parallel(M.left(3, 1, 32, 32, 64, dims=16, softcap=4.0), M.right(2, 2, 32, 16, conv=1)),
    "many heads on one": M.parallel(M.left(16, 1, 128, 64, 100, softcap=5.0), M.right(8, 1, 64, 130, conv=6)),
    "no rotation": M.parallel(M.left(2, 2, 16, 48, 7, dims=0, scale=0.5, softcap=1.0), M.right(1, 1, 256, 8, conv=3)),
    "no cap": M.parallel(M.left(6, 3, 48, 48, 1000, softcap=None), M.right(6, 3, 48, 48)),
    "mamba": M.mamba(80, 5, 7, conv=3), "mamba of ones": M.mamba(33, 1, 1, conv=1), "mamba wide": M.mamba(256, 40, 24),
    "wkv": M.wkv(3, 20), "wkv 64": M.wkv(4, 64), "wkv wide": M.wkv(1, 200), "wkv of one": M.wkv(5, 1),
}


@pytest.mark.parametrize("schedule", sorted(SCHEDULES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MIXERS))
def test_mixer_alone(lib, name, dtype, schedule):
    mixer, width, n, m_, eps = MIXERS[name], 96, 200, 40, 1e-5
    g = torch.Generator().manual_seed(11)
    W = M.mixer_weights(mixer, width, g, torch.bfloat16, sharp=2.0, rank=11 if name != "wkv 64" else 32)
    part = build_mixer(mixer, width, W, dtype)
    h_of = {r: torch.randn(k, width, generator=g).to(torch.bfloat16).float() for r, k in (("a", n), ("b", m_), ("c", 30))}
    sched = SCHEDULES[schedule](n, m_)
    got = run_mixer(part, {r: h_of[r] for r in {k for s in sched for k in s}}, sched, dtype)
    Wd, fn = M.widen(W), P.MIXERS[mixer[0]]
    for r, rows_ in got.items():
        ref = fn(h_of[r].double(), Wd, mixer[1], eps)
        tol = M.tolerance(dtype, ref, fn(h_of[r].double(), Wd, mixer[1], eps, round_to=torch.bfloat16), error)
        assert error(rows_, ref) < tol, r


# ---------------------------------------------------------------------------- edges, far keys, the soft cap
def edge_case(vdim, chunk, softcap=8.0, strength=8.0, seed=77, width=64):
    """A one-layer model whose token 7 has a key that stands out; keys and values of one size that is a multiple of 16 (vdim
    32) run on other kernels than other sizes."""
    cfg = M.config(width, 60, [M.layer(M.parallel(M.left(4, 2, 32, vdim, chunk, dims=16, base=300.0, softcap=softcap), M.right(2, 1, 16, 16)), 48)], scale=2.0)
    return cfg, M.stand_out(M.random_weights(cfg, seed), cfg, 0, 7, strength=strength)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("vdim", [32, 16])
def test_a_key_just_inside_and_just_outside_its_chunk_in_prompts_portions_and_decoding(lib, vdim, dtype, tmp_path):
    size, n = 70, 160
    cfg, W = edge_case(vdim, size)
    Wd = M.widen(W)
    toks = [t if t != 7 else 8 for t in tokens(cfg, n, 5)]
    toks[size - 3] = 7                                    # seen up to the chunk's last position, size - 1, and no more
    ref = P.forward(Wd, cfg, toks)
    tol = M.tolerance(dtype, ref, P.forward(Wd, cfg, toks, round_to=torch.bfloat16))
    for wrong in (size - 1, size + 1):                    # the plain implementation alone: one position off shows
        off = P.forward(Wd, M.with_chunk(cfg, 0, wrong), toks)
        assert M.row_error(off[size - 2:size + 2], ref[size - 2:size + 2]) > SHOWS[dtype] * tol, wrong
    eng = load(lib, tmp_path, cfg, W, dtype)
    for name, sched in (("prompt", [{"a": n}]), ("portions", [{"a": size - 2}, {"a": 2}, {"a": 2}, {"a": n - size - 2}]),
                        ("decoding", [{"a": size - 4}] + [{"a": 1}] * 8 + [{"a": n - size - 4}])):
        assert M.row_error(run_schedule(eng, {"a": toks}, sched)["a"], ref) < tol, name


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("vdim", [32, 16])
def test_a_far_key_among_hundreds_and_the_soft_cap_on_it(lib, vdim, dtype, tmp_path):
    # (the key's score is some 24, its share of the weights about a quarter under the cap and nearly all of them without it)
    n, cap = 500, 6.0
    cfg, W = edge_case(vdim, 1000, softcap=cap, strength=1.7, seed=78, width=256)
    Wd = M.widen(W)
    base = [t if t != 7 else 8 for t in tokens(cfg, n, 6)]
    toks = list(base)
    toks[3] = 7
    ref, without = P.forward(Wd, cfg, toks), P.forward(Wd, cfg, base)
    tol = M.tolerance(dtype, ref, P.forward(Wd, cfg, toks, round_to=torch.bfloat16))
    far = list(range(440, n))
    assert M.row_error(without[far], ref[far]) > SHOWS[dtype] * tol        # the rows far away feel the key at position 3
    other = json.loads(json.dumps(cfg))
    other["layers"][0]["mixer"]["left"]["softcap"] = None
    assert M.row_error(P.forward(Wd, other, toks)[far], ref[far]) > SHOWS[dtype] * tol      # and the cap on its score
    eng = load(lib, tmp_path, cfg, W, dtype)
    for sched in ([{"a": n}], [{"a": 450}] + [{"a": 1}] * 50, [{"a": 130}, {"a": 300}, {"a": 70}]):
        assert M.row_error(run_schedule(eng, {"a": toks}, sched)["a"], ref) < tol


# ---------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("name", sorted(M.ALL))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_model_whole_first_tokens_portions_and_token_by_token(lib, models, dtype, name):
    folder, cfg, W = models[name]
    n = 210
    toks = tokens(cfg, n, 9)
    ref = P.forward(W, cfg, toks)
    tol = M.tolerance(dtype, ref, P.forward(W, cfg, toks, round_to=torch.bfloat16))
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
            assert M.row_error(got, whole) < 5e-5


def test_model_in_float16(lib, models):
    """The other 16-bit type runs the same kernels (the recurrences' rows in bfloat16 all the same)."""
    folder, cfg, W = models["C"]
    toks = tokens(cfg, 150, 9)
    ref = P.forward(W, cfg, toks)
    eng = lib.load(folder, dtype="float16", max_tokens=1024)
    assert M.row_error(run_schedule(eng, {"a": toks}, [{"a": 130}] + [{"a": 1}] * 20)["a"], ref) < 3e-2


@pytest.mark.parametrize("name", sorted(M.ALL))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_together_against_each_alone(lib, models, dtype, name):
    folder, cfg, W = models[name]
    reqs = {"a": tokens(cfg, 150, 12), "b": tokens(cfg, 1, 13), "c": tokens(cfg, 67, 14), "d": tokens(cfg, 230, 15),
            "e": tokens(cfg, 40, 16)}
    ref = {r: P.forward(W, cfg, t) for r, t in reqs.items()}
    tol = {r: M.tolerance(dtype, ref[r], P.forward(W, cfg, t, round_to=torch.bfloat16)) for r, t in reqs.items()}
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


def test_a_batch_too_large_for_the_short_kernels(lib, models):
    """Twenty requests decoded together (more rows than the one-launch products of time mixing take), each against itself alone."""
    folder, cfg, W = models["C"]
    reqs = {f"r{i}": tokens(cfg, 20 + 3 * i, 60 + i) for i in range(20)}
    eng = lib.load(folder, dtype="bfloat16", max_tokens=4096, n_slots=24)
    sched = [{r: len(t) - 4 for r, t in reqs.items()}] + [{r: 1 for r in reqs}] * 4
    got = run_schedule(eng, reqs, sched)
    for r, t in reqs.items():
        ref = P.forward(W, cfg, t)
        assert M.row_error(got[r], ref) < M.tolerance("bfloat16", ref, P.forward(W, cfg, t, round_to=torch.bfloat16)), r


@pytest.mark.parametrize("dtype,graph", [("float32", True), ("bfloat16", True), ("bfloat16", False)])
@pytest.mark.parametrize("name", ["A", "C"])
def test_long_decoding_and_generation(lib, models, name, dtype, graph):
    """Greedy generation through the library's own loop (recorded and eager decode steps), across chunks and pages, against
    the plain implementation's choice wherever its logits leave a margin."""
    folder, cfg, W = models[name]
    eng = lib.load(folder, dtype=dtype, max_tokens=4096)
    prompts = [tokens(cfg, 70, 21), tokens(cfg, 3, 22), tokens(cfg, 1, 23)]
    new = eng.generate(prompts, max_new_tokens=150, temperature=0.0, use_graph=graph)
    assert all(len(t) == 150 for t in new)
    if graph:
        assert eng.decode_counts["replayed"] > 100
    checked = 0
    for p, out in zip(prompts, new):
        logits = P.forward(W, cfg, list(p) + out)
        margin = (1e-3 if dtype == "float32" else 0.15) * logits.std().item()
        for k, t in enumerate(out):
            row = logits[len(p) - 1 + k]
            top2 = torch.topk(row, 2).values
            if (top2[0] - top2[1]).item() < margin:
                continue
            assert t == int(row.argmax()), (dtype, graph, k)
            checked += 1
    assert checked > (400 if dtype == "float32" else 100), checked


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_recorded_steps_against_eager_ones(lib, models, dtype):
    """A recorded decode step replayed, with the engine's own eager work in between, gives the eager step's tokens."""
    folder, cfg, W = models["C"]
    a, b = (lib.load(folder, dtype=dtype, max_tokens=4096) for _ in range(2))
    prompts = [tokens(cfg, n, 70 + n) for n in (5, 40, 64)]
    for _ in range(3):
        one = a.generate(prompts, max_new_tokens=24, temperature=0.0, use_graph=True)
        two = b.generate(prompts, max_new_tokens=24, temperature=0.0, use_graph=False)
        assert one == two
    assert a.decode_counts["replayed"] > 40 and b.decode_counts["replayed"] == 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_in_three_schedules(lib, models, dtype, tmp_path):
    folder, cfg, W = models["B"]
    reqs = {"r1": tokens(cfg, 75, 41), "r2": tokens(cfg, 1, 42), "r3": tokens(cfg, 140, 43)}
    ref = {r: P.forward(W, cfg, t) for r, t in reqs.items()}
    tol = {r: M.tolerance(dtype, ref[r], P.forward(W, cfg, t, round_to=torch.bfloat16)) for r, t in reqs.items()}
    for k, (steps, where) in enumerate((TU.steps_whole(reqs), TU.steps_tail(reqs, 33), TU.steps_batches(reqs, 3, {"r1": 10, "r3": 70}))):
        got = TU.run_trace(folder, dtype, steps, where, cfg["vocab"], 300, str(tmp_path / f"out{k}"))
        assert set(got) == {(r, p) for r, t in reqs.items() for p in range(len(t))}
        for r, t in reqs.items():
            g = torch.stack([torch.from_numpy(got[r, p].copy()) for p in range(len(t))])
            assert M.row_error(g, ref[r]) < tol[r], (k, r)


def test_command_line_reports_and_generates(lib, models):
    folder, cfg, W = models["A"]
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
            last = P.forward(W, cfg, toks)[-1]
            top2 = torch.topk(last, 2).values
            if (top2[0] - top2[1]).item() > 1e-3:
                assert t == int(last.argmax())
            toks.append(t)
    for word in ("Dimensions: 96", "Vocab size: 131"):
        assert word in res.stdout, res.stdout
    info = subprocess.run([sys.executable, os.path.join(root, "bin", "model_info"), folder], capture_output=True, text=True,
                          timeout=300)
    assert info.returncode == 0 and "Architecture: Dopivik" in info.stdout and "The tensors fit the model." in info.stdout, info.stdout + info.stderr
