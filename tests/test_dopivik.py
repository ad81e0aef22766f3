"""Dopivik without a GPU: the plain implementation pinned by library routines, closed forms and invariants; the
configuration's reading and refusals; the tensor table (a rank that the checkpoint says); what the model asks of the cache
(a layer with another's weights has a cache and states of its own); the random-weights folder."""
import json
import math

import pytest
import torch
import torch.nn.functional as F

import dopivik_models as M
import plain_dopivik as P

D = torch.float64


def rnd(*shape, seed=0, s=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=D) * s


# ---------------------------------------------------------------------------- the plain implementation, pinned
def test_norms_and_activations_against_torch():
    x, w, b = rnd(5, 24), rnd(24, seed=1), rnd(24, seed=2)
    assert torch.allclose(P.layer_norm(x, w, b, 1e-5), F.layer_norm(x, (24,), w, b, 1e-5), atol=1e-12)
    assert torch.allclose(P.rms(x, 1e-5), F.rms_norm(x, (24,), None, 1e-5), atol=1e-12)
    assert torch.allclose(P.silu(x), F.silu(x)) and torch.allclose(P.relu_squared(x), F.relu(x) ** 2)
    u = P.unit(x)
    assert torch.allclose(u.norm(dim=-1), torch.ones(5, dtype=D), atol=1e-6)
    assert torch.allclose(P.unit(torch.zeros(1, 4, dtype=D)), torch.zeros(1, 4, dtype=D))


def test_chunk_mask_at_its_edges():
    c = P.chunk_mask(20, 5)
    assert c[9, 5] and not c[10, 9] and c[10, 10] and not c[9, 10] and c[4, 0] and not c[5, 4]
    assert P.chunk_mask(6, 1).equal(torch.eye(6, dtype=torch.bool))


def test_rotation_turns_half_pairs_and_scores_depend_on_distance():
    x = rnd(1, 1, 12)
    y = P.rotate(x.expand(7, 1, 12), torch.arange(7), 100.0, 8)
    assert torch.allclose(y[0], x[0]) and torch.allclose(y[..., 8:], x.expand(7, 1, 12)[..., 8:])
    a = torch.tensor(3 * 100.0 ** (-2.0 / 8), dtype=D)                  # pair (1, 5) at position 3
    assert torch.allclose(y[3, 0, 1], x[0, 0, 1] * torch.cos(a) - x[0, 0, 5] * torch.sin(a))
    assert torch.allclose(y[3, 0, 5], x[0, 0, 5] * torch.cos(a) + x[0, 0, 1] * torch.sin(a))
    q, k = rnd(1, 1, 8, seed=3), rnd(1, 1, 8, seed=4)
    s = lambda i, j: (P.rotate(q, torch.tensor([i]), 100.0, 8) * P.rotate(k, torch.tensor([j]), 100.0, 8)).sum()
    assert torch.allclose(s(9, 4), s(25, 20))


def test_attention_against_scaled_dot_product_and_the_soft_cap():
    T, H, G, d, dv = 13, 4, 2, 8, 5
    q, k, v = rnd(T, H, d), rnd(T, G, d, seed=1), rnd(T, G, dv, seed=2)
    vis = P.chunk_mask(T, 6)
    kk, vv = k.repeat_interleave(2, 1), v.repeat_interleave(2, 1)
    ref = F.scaled_dot_product_attention(q.transpose(0, 1), kk.transpose(0, 1), vv.transpose(0, 1), attn_mask=vis, scale=0.3)
    assert torch.allclose(P.capped_attention(q, k, v, 0.3, None, vis), ref.transpose(0, 1), atol=1e-10)
    assert torch.allclose(P.capped_attention(q, k, v, 0.3, 1e9, vis), ref.transpose(0, 1), atol=1e-6)
    s = torch.tensor([-1e4, -1.0, 0.0, 0.5, 1e4], dtype=D)
    assert torch.allclose(P.capped(s, 2.0), torch.tensor([-2.0, 2 * math.tanh(-0.5), 0.0, 2 * math.tanh(0.25), 2.0], dtype=D))


def test_convolution_against_conv1d():
    u, w, b = rnd(11, 6), rnd(6, 4, seed=2), rnd(6, seed=3)
    ref = F.conv1d(F.pad(u.T[None], (3, 0)), w[:, None, :], b, groups=6)[0].T
    assert torch.allclose(P.causal_conv(u, w, b), ref, atol=1e-12)
    assert torch.allclose(P.causal_conv(u, w)[0], u[0] * w[:, 3])       # the last tap is the current token's


def test_delta_rule_writes_what_it_reads():
    """beta = 1 and no decay: after a token its key reads back its value; a second token with the same key overwrites it."""
    k = P.unit(rnd(3, 1, 6)) / 1.0
    k[2] = k[1]
    v = rnd(3, 1, 4, seed=1)
    one = torch.ones(3, 1, dtype=D)
    o, S = P.delta_rule(k, k, v, one, one)
    assert torch.allclose(o[:, 0], v[:, 0], atol=1e-5)
    assert torch.allclose(torch.einsum("hdv,hd->hv", S, k[1]), v[2], atol=1e-5)
    # in two parts, the state handed over
    q, k, v = rnd(9, 2, 5, seed=3), P.unit(rnd(9, 2, 5, seed=4)), rnd(9, 4, 3, seed=5)
    beta, g = torch.sigmoid(rnd(9, 4, seed=6)), torch.sigmoid(rnd(9, 4, seed=7))
    o, S = P.delta_rule(q, k, v, beta, g)
    o1, S1 = P.delta_rule(q[:4], k[:4], v[:4], beta[:4], g[:4])
    o2, S2 = P.delta_rule(q[4:], k[4:], v[4:], beta[4:], g[4:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    # beta = 0 writes nothing, g scales what there is
    o0, S0 = P.delta_rule(q[:1], k[:1], v[:1], 0 * beta[:1], 0 * g[:1] + 0.5, S)
    assert torch.allclose(S0, 0.5 * S)


def test_selective_scan_against_a_sum_over_the_past():
    T, c, n = 6, 3, 2
    x, dt, B, C, Dk = rnd(T, c), torch.rand(T, c, dtype=D), rnd(T, n, seed=1), rnd(T, n, seed=2), rnd(c, seed=3)
    A = -torch.rand(c, n, dtype=D)
    y, S = P.selective_scan(x, dt, A, B, C, Dk)
    t = 4
    ref = Dk * x[t]
    for s in range(t + 1):
        decay = torch.exp(dt[s + 1:t + 1].sum(0)[:, None] * A)
        ref = ref + (decay * (dt[s] * x[s])[:, None] * B[s][None, :]) @ C[t]
    assert torch.allclose(y[t], ref)


def test_time_mixing_against_a_sum_over_the_past():
    T, H, d = 6, 2, 3
    r, k, v, u = rnd(T, H, d), rnd(T, H, d, seed=1), rnd(T, H, d, seed=2), rnd(H, d, seed=3)
    w = torch.sigmoid(rnd(T, H, d, seed=4))
    o, S = P.wkv_rule(r, k, v, w, u)
    t = 4
    ref = (r[t] * u * k[t]).sum(-1, keepdim=True) * v[t]
    for s in range(t):
        decay = torch.prod(w[s + 1:t], 0)                                # (the token's own decay comes after its read-out)
        ref = ref + (r[t] * decay * k[s]).sum(-1, keepdim=True) * v[s]
    assert torch.allclose(o[t], ref)
    o1, S1 = P.wkv_rule(r[:3], k[:3], v[:3], w[:3], u)
    o2, S2 = P.wkv_rule(r[3:], k[3:], v[3:], w[3:], u, S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)


def test_layers_with_anothers_weights_and_causality():
    cfg = M.TINY_A
    W = M.widen(M.random_weights(cfg, 3))
    toks = torch.randint(0, cfg["vocab"], (70,), generator=torch.Generator().manual_seed(1)).tolist()
    layers = []
    full = P.forward(W, cfg, toks, layers_out=layers)
    assert torch.allclose(P.forward(W, cfg, toks[:40]), full[:40], atol=1e-9)
    assert not any(k.startswith(("l3.", "l4.")) for k in W)
    assert torch.allclose(P.run_layer(layers[2], cfg, W, 0), layers[3])   # layer 3: layer 0's tensors on its own input
    h = P.layer_norm(layers[3], W["l2.norm1"], W["l2.norm1.b"], cfg["norm"]["eps"])
    first = P.wkv(h[:1], P.sub(W, "l2.mix."), cfg["layers"][4]["mixer"], cfg["norm"]["eps"])
    assert torch.allclose(first, P.wkv(h, P.sub(W, "l2.mix."), cfg["layers"][4]["mixer"], cfg["norm"]["eps"])[:1])


# ---------------------------------------------------------------------------- configuration, tensors, cache
def test_configuration_reading_and_refusals():
    from llm_infer_amd import ConfigError, config_from_dict
    cfg = config_from_dict(M.TINY_A)
    assert cfg.to_dict()["layers"] == M.TINY_A["layers"] and cfg.embedding_scale == 2.5
    assert config_from_dict(cfg.to_dict()) == cfg
    assert [cfg.owner(i) for i in range(5)] == [0, 1, 2, 0, 2]

    def refused(change):
        bad = json.loads(json.dumps(M.TINY_A))
        change(bad["layers"])
        with pytest.raises(ConfigError):
            config_from_dict(bad)
    refused(lambda L: L[3].update(weights_of=1))                            # another kind of layer
    refused(lambda L: L[3].update(weights_of=3))
    refused(lambda L: L[0].update(weights_of=3))                            # each the other's
    refused(lambda L: L[3]["mixer"]["left"]["mask"].update(size=51))        # the rest of its entry is its owner's
    refused(lambda L: L[0]["mixer"]["left"].update(kv_heads=3))
    refused(lambda L: L[0]["mixer"]["right"].update(conv=0))
    refused(lambda L: L[1].update(type="mamba3"))
    refused(lambda L: L[1]["mixer"].pop("dt_rank"))
    refused(lambda L: L[0]["mixer"]["left"]["rot"].update(dims=13))
    refused(lambda L: L[0]["mlp"].update(kind="moe"))


@pytest.mark.parametrize("name", sorted(M.ALL))
def test_tensor_table_is_the_designs(name, tmp_path):
    from llm_infer_amd import config_from_dict
    from llm_infer_amd.engine.model import DecoderModel
    from llm_infer_amd.weights.loader import Checkpoint, WeightError, check_tensors
    cfg = M.ALL[name]
    model = DecoderModel(config_from_dict(cfg).model_spec(), torch.float32, "cpu", allocate=False)
    W = M.random_weights(cfg, 1, rank=16)
    assert {k: tuple(v.shape) for k, v in model.params().items()} == {k: tuple(v.shape) for k, v in W.items()}
    # the rank of the decays is what the file says, any other size is not
    for rank in (1, 5):
        M.write_model(str(tmp_path / str(rank)), cfg, M.random_weights(cfg, 1, rank=rank))
        check_tensors(model.params(), Checkpoint(str(tmp_path / str(rank))))
    W["embed"] = W["embed"][:-1].contiguous()
    M.write_model(str(tmp_path / "bad"), cfg, W)
    with pytest.raises(WeightError):
        check_tensors(model.params(), Checkpoint(str(tmp_path / "bad")))


def test_what_the_model_asks_of_the_cache():
    from llm_infer_amd import config_from_dict
    from llm_infer_amd.cache import Cache
    from llm_infer_amd.cache.specs import KVSpec, StateSpec
    from llm_infer_amd.engine.model import DecoderModel
    model = DecoderModel(config_from_dict(M.TINY_A).model_spec(), torch.float32, "cpu", allocate=False)
    assert len(model.layers) == 3 and [e.layer for e in model.schedule] == [0, 1, 2, 0, 2]
    specs = model.cache_specs()
    par = [KVSpec(2, 32, None, 16, 50, "maps"), StateSpec((6, 20, 24)), StateSpec((1, 2 * 2 * 20 + 6 * 24))]
    assert specs[:3] == par and specs[7:10] == par                          # (layer 3: the same sizes, units of its own)
    assert specs[3:5] == [StateSpec((5, 80)), StateSpec((2, 80))]
    assert specs[5:7] == [StateSpec((3, 20, 20)), StateSpec((96,))] and specs[10:] == specs[5:7]
    seen = [u for i in range(5) for u in model._seen[i, 0]]
    assert seen == list(range(12))                                          # nobody reads another's
    cache = Cache(specs, 512, 512, torch.float32, None, n_slots=2)
    assert all(cache.view is not None for _ in seen) and cache.groups


def test_random_weights_folder(tmp_path):
    import llm_infer_amd
    from safetensors import safe_open
    cfg = llm_infer_amd.config_from_dict(M.TINY_A)
    llm_infer_amd.write_random_model(str(tmp_path), cfg, seed=4)
    assert llm_infer_amd.config_from_folder(str(tmp_path)).to_dict()["layers"] == M.TINY_A["layers"]
    with safe_open(str(tmp_path / "model.safetensors"), "pt") as f:
        W = {k: f.get_tensor(k) for k in f.keys()}
    assert W["l2.mix.w1"].shape == (16, 96) and W["l0.mix.right.A_log"].dtype == torch.float32
    assert torch.isfinite(P.forward(M.widen(W), M.TINY_A, [1, 2, 3, 4, 5, 6, 7, 8, 9])).all()
