"""Pusisun without a GPU: the plain implementation pinned by library routines, closed forms and invariants; the
configuration's reading and refusals; the tensor table and the schedule of a repeated stretch; what the model asks of the
cache; pages of kept first tokens; the stretched frequencies; the random-weights folder."""
import json
import math

import pytest
import torch
import torch.nn.functional as F

import plain_pusisun as P
import pusisun_models as M

D = torch.float64


def rnd(*shape, seed=0, s=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=D) * s


# ---------------------------------------------------------------------------- the plain implementation, pinned
def test_norm_and_activation_against_torch():
    x, w = rnd(5, 24), rnd(24, seed=1)
    assert torch.allclose(P.rms_norm(x, w, 1e-5), F.rms_norm(x, (24,), w, 1e-5), atol=1e-12)
    assert torch.allclose(P.silu(x), F.silu(x), atol=1e-12)


def test_masks_at_their_edges():
    m = P.window_mask(30, 5, 3)
    assert m[10, 10] and m[10, 6] and not m[10, 5] and not m[10, 11]          # the window
    assert m[10, 2] and not m[10, 3] and m[29, 0] and m[29, 2] and not m[29, 3]   # the first three, and the next one
    assert m[1, 0] and not m[1, 2]                                            # kept tokens are not seen ahead of time
    assert P.window_mask(6, 1).equal(torch.eye(6, dtype=torch.bool))
    assert P.window_mask(6, 6, 2).equal(P.causal_mask(6)) and P.window_mask(6, 1, 6).equal(P.causal_mask(6))


def test_turning_half_pairs_with_a_magnitude():
    f, mag = P.stretched_frequencies(8, 100.0, None)
    assert mag == 1.0 and torch.allclose(f, torch.tensor([100.0 ** (-2 * i / 8) for i in range(4)], dtype=D))
    x = rnd(1, 1, 8)
    y = P.turn(x.expand(7, 1, 8), torch.arange(7), f, 1.5)
    assert torch.allclose(y[0], 1.5 * x[0])                                   # position 0: only the magnitude
    assert torch.allclose(y.norm(dim=-1), 1.5 * x.norm(dim=-1).expand(7, 1))
    a = f[1] * 3                                                              # pair (1, 5) at position 3
    assert torch.allclose(y[3, 0, 1], 1.5 * (x[0, 0, 1] * torch.cos(a) - x[0, 0, 5] * torch.sin(a)))
    assert torch.allclose(y[3, 0, 5], 1.5 * (x[0, 0, 5] * torch.cos(a) + x[0, 0, 1] * torch.sin(a)))
    q, k = rnd(1, 1, 8, seed=3), rnd(1, 1, 8, seed=4)
    s = lambda i, j: (P.turn(q, torch.tensor([i]), f, 1.2) * P.turn(k, torch.tensor([j]), f, 1.2)).sum()
    assert torch.allclose(s(9, 4), s(25, 20))


@pytest.mark.parametrize("scaling", [(6.0, 700, 30.0, 1.5), (2.0, 40, 3.0, 2.9), (40.0, 100000, 1.0, 0.5), (8.0, 10, 40.0, 20.0)])
def test_stretched_frequencies(scaling):
    sc = dict(zip(("factor", "original", "fast", "slow"), scaling))
    f0, (f, mag) = P.stretched_frequencies(40, 20000.0, None)[0], P.stretched_frequencies(40, 20000.0, sc)
    assert math.isclose(mag, 0.1 * math.log(sc["factor"]) + 1.0)
    assert (f <= f0 * (1 + 1e-12)).all() and (f >= f0 / sc["factor"] * (1 - 1e-12)).all()
    ratio = f / f0
    assert (ratio[1:] <= ratio[:-1] + 1e-12).all()                            # kept first, divided last
    # a pair that makes many more turns over the original positions than `fast` keeps its frequency; one that makes far
    # fewer than `slow` is divided
    turns = f0 * sc["original"] / (2 * math.pi)
    assert torch.allclose(ratio[turns > 1.8 * sc["fast"]], torch.ones((), dtype=D))
    few = turns < 0.5 * sc["slow"]
    few[0] = False                                                            # (the ramp never begins before the first pair)
    assert torch.allclose(ratio[few], torch.tensor(1.0 / sc["factor"], dtype=D))
    # the library's own table
    from llm_infer_amd.parts.position import scaled_by_ramp
    own, own_mag = scaled_by_ramp(20000.0, 40, sc)
    assert torch.allclose(own.double(), f, rtol=1e-6) and math.isclose(own_mag, mag)


def test_attention_against_scaled_dot_product():
    T, H, G, d, dv = 13, 4, 2, 8, 5
    q, k, v = rnd(T, H, d), rnd(T, G, d, seed=1), rnd(T, G, dv, seed=2)
    vis = P.window_mask(T, 6, 2)
    kk, vv = k.repeat_interleave(2, 1), v.repeat_interleave(2, 1)
    ref = F.scaled_dot_product_attention(q.transpose(0, 1), kk.transpose(0, 1), vv.transpose(0, 1), attn_mask=vis, scale=0.3)
    assert torch.allclose(P.softmax_attention(q, k, v, 0.3, vis), ref.transpose(0, 1), atol=1e-10)
    got = P.softmax_attention(q, k, v, 0.3, vis, torch.full((H,), -1e9, dtype=D))
    assert torch.allclose(got, ref.transpose(0, 1), atol=1e-10)


def test_a_sink_equal_to_the_only_score_halves_the_output_and_is_neither_scaled_nor_biased():
    q, k, v = torch.ones(1, 1, 4, dtype=D), torch.ones(1, 1, 4, dtype=D), rnd(1, 1, 3)
    out = P.softmax_attention(q, k, v, 0.5, torch.ones(1, 1, dtype=torch.bool), torch.tensor([2.0], dtype=D), torch.tensor([0.7], dtype=D))
    assert torch.allclose(out, 0.5 * v)                                  # score 4 * 0.5 = 2 = sink, distance 0


def test_distance_bias_counts_from_a_kept_tokens_true_position():
    s = P.slopes(4, D)
    assert torch.allclose(s, torch.tensor([2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8], dtype=D))
    T = 6
    q, k, v = torch.zeros(T, 1, 2, dtype=D), torch.zeros(T, 1, 2, dtype=D), torch.eye(T, dtype=D)[:, None, :]
    out = P.softmax_attention(q, k, v, 1.0, P.window_mask(T, 2, 1), None, torch.tensor([0.5], dtype=D))
    w = torch.exp(-0.5 * torch.tensor([5.0, 1.0, 0.0], dtype=D))        # the last row: position 0 (kept), 4 and 5
    want = torch.zeros(T, dtype=D)
    want[torch.tensor([0, 4, 5])] = w / w.sum()
    assert torch.allclose(out[5, 0], want)


def test_latent_attention_by_the_absorbed_form():
    """The one key [W_uk^T q . c] form gives the same as every head's own keys and values."""
    m = M.latent(3, 6, 4, 5, 7, 9, scaling=(4.0, 60, 8.0, 1.0))[1]
    W = M.widen(M.mixer_weights("latent_attention", m, 16, torch.Generator().manual_seed(1), torch.float32))
    h = rnd(11, 16)
    plain = P.latent_mixer(h, W, m, 1e-5)
    absorbed = P.latent_mixer(h, W, m, 1e-5, round_to=torch.float64)
    assert torch.allclose(plain, absorbed, atol=1e-10)


def test_q_and_k_are_normed_over_all_heads_at_once():
    m = M.attention(2, 1, 4, 3, 100)[1]
    W = M.widen(M.mixer_weights("attention", m, 8, torch.Generator().manual_seed(2), torch.float32))
    h = rnd(5, 8)
    a = P.attention_mixer(h, W, m, 1e-6)
    scaled = dict(W)
    for n in ("q", "k"):
        scaled[n], scaled[n + ".b"] = 3.0 * W[n], 3.0 * W[n + ".b"]      # a common factor of q, and of k, is divided out
    assert torch.allclose(P.attention_mixer(h, scaled, m, 1e-6), a, atol=1e-5)
    one = dict(W, q=W["q"].clone())
    one["q"][:4] *= 3.0                                                  # one head's alone is not
    assert not torch.allclose(P.attention_mixer(h, one, m, 1e-6), a, atol=1e-2)


def test_experts_are_weighted_by_the_softmax_over_the_chosen_and_the_bias_counts():
    w, mlp = 12, M.moe(4, 2, 6)
    W = M.widen(M.mlp_weights(mlp, w, torch.Generator().manual_seed(5), torch.float32))
    W["router.b"] = torch.tensor([0.0, 50.0, 0.0, 51.0], dtype=D)
    h = rnd(3, w)
    z = h @ W["router"].T + W["router.b"]
    p = torch.softmax(z[:, [1, 3]], -1)
    one = lambda e: (F.silu(h @ W[f"e{e}.gate"].T) * (h @ W[f"e{e}.up"].T)) @ W[f"e{e}.down"].T
    assert torch.allclose(P.experts(h, W, mlp), p[:, :1] * one(1) + p[:, 1:] * one(3), atol=1e-10)


def test_a_repeated_stretch_by_hand_and_causality():
    cfg = M.TINY_A
    W = M.widen(M.random_weights(cfg, 3))
    toks = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(1)).tolist()
    layers = []
    full = P.forward(cfg, W, toks, layers)
    assert len(layers) == 8 and torch.allclose(P.forward(cfg, W, toks[:25]), full[:25], atol=1e-9)
    x0 = W["embed"][torch.tensor(toks)] * 2.5
    eps, step = cfg["norm"]["eps"], lambda x, i: P.layer(x, P.sub(W, f"l{i}."), cfg["layers"][i], eps)
    x = step(x0, 0)
    x = step(step(x + W["loop.step"][0], 1), 2)
    x = step(step(x + x0 + W["loop.step"][1], 1), 2)
    x = step(step(x + x0 + W["loop.step"][2], 1), 2)
    x = step(x, 3)
    assert torch.allclose(x, layers[-1], atol=1e-9)


# ---------------------------------------------------------------------------- configuration, tensors, cache
def test_configuration_reading_and_refusals():
    from llm_infer_amd import ConfigError, config_from_dict
    cfg = config_from_dict(M.TINY_A)
    assert cfg.to_dict()["layers"] == M.TINY_A["layers"] and cfg.loop == (1, 3, 3)
    assert config_from_dict(cfg.to_dict()) == cfg
    assert config_from_dict(M.TINY_D).loop is None and "loop" not in config_from_dict(M.TINY_D).to_dict()

    def refused(change):
        bad = json.loads(json.dumps(M.TINY_A))
        change(bad)
        with pytest.raises(ConfigError):
            config_from_dict(bad)
    refused(lambda c: c["loop"].update(stop=5))
    refused(lambda c: c["loop"].update(times=0))
    refused(lambda c: c["loop"].update(start=3))
    refused(lambda c: c["layers"][1]["mixer"].update(kv_heads=3))
    refused(lambda c: c["layers"][1]["mixer"]["mask"].update(size=0))
    refused(lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1))
    refused(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14))
    refused(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("fast"))
    refused(lambda c: c["layers"][0]["mixer"].pop("q_rank"))
    refused(lambda c: c["layers"][0]["mlp"]["router"].update(top=6))
    refused(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    refused(lambda c: c["layers"][0].update(type="attention_3"))


@pytest.mark.parametrize("name", sorted(M.ALL))
def test_tensor_table_is_the_designs(name):
    from llm_infer_amd import config_from_dict
    from llm_infer_amd.engine.model import DecoderModel
    cfg = M.ALL[name]
    model = DecoderModel(config_from_dict(cfg).model_spec(), torch.float32, "cpu", allocate=False)
    W = M.random_weights(cfg, 1)
    assert {k: tuple(v.shape) for k, v in model.params().items()} == {k: tuple(v.shape) for k, v in W.items()}
    assert [(e.layer, e.pass_no if e.before is not None else None) for e in model.schedule] == P.runs(cfg)


def test_every_pass_keeps_a_cache_of_its_own():
    from llm_infer_amd import config_from_dict
    from llm_infer_amd.cache.specs import KVSpec
    from llm_infer_amd.engine.model import DecoderModel
    model = DecoderModel(config_from_dict(M.TINY_A).model_spec(), torch.float32, "cpu", allocate=False)
    specs = model.cache_specs()
    assert len(specs) == 8 and len({u for i in range(8) for u in model._seen[i, 0]}) == 8
    lat, near, wide = KVSpec(1, 48, None, 28, None, "maps"), KVSpec(2, 32, 9, 16, None, "maps", 3), KVSpec(1, 32, 70, 32, None, "maps", 66)
    assert specs == [lat, near, wide, near, wide, near, wide, KVSpec(1, 32, None, 16, None, "maps")]
    assert len(model.stream_parts) == 1                                       # one part, one tensor, for all three passes


def test_pages_of_kept_first_tokens_stay():
    from llm_infer_amd.cache import Cache
    from llm_infer_amd.cache.specs import KVSpec
    for keep, held in ((0, []), (1, [0]), (64, [0]), (65, [0, 1]), (130, [0, 1, 2])):
        cache = Cache([KVSpec(1, 16, 70, None, None, "maps", keep)], 64 * 20, 64 * 20, torch.float32, None, n_slots=2)
        group = cache.groups[0]
        slot = cache.alloc_slot()
        for n in (40, 130, 131, 400, 401, 1000):
            cache.grow([slot], [n])
            cache.trim_windows([slot])
            first = (n - 70 + 1) // 64 if n >= 70 else 0
            want = sorted(set(range(first, (n + 63) // 64)) | {p for p in held if p * 64 < n})
            assert sorted(group.pages_of[slot]) == want, (keep, n)
        cache.free_slot(slot)
        assert group.pool.n_free == group.n_pages - 1


def test_random_weights_folder(tmp_path):
    import llm_infer_amd
    from safetensors import safe_open
    cfg = llm_infer_amd.config_from_dict(M.TINY_B)
    llm_infer_amd.write_random_model(str(tmp_path), cfg, seed=4)
    back = llm_infer_amd.config_from_folder(str(tmp_path))
    assert back.to_dict()["layers"] == M.TINY_B["layers"] and back.loop == (0, 4, 2)
    with safe_open(str(tmp_path / "model.safetensors"), "pt") as f:
        W = {k: f.get_tensor(k) for k in f.keys()}
    assert W["l0.mlp.router"].dtype == torch.bfloat16
    out = P.forward(M.TINY_B, M.widen(W), [1, 2, 3, 4, 5, 6, 7, 8, 9])
    assert torch.isfinite(out).all()
