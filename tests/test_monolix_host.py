"""Monolix on the CPU: properties of the oracle's mechanisms in closed form or in limiting cases (the oracle is what the GPU
tests compare with, so it is checked against arithmetic that does not share its code), mistakes planted in the oracle and
seen in its logits, the configuration reader, the registry, the pool shapes and the merges of load_weights.  No kernel runs."""
import json
import math

import pytest
import torch

from oracle import monolix as mo
from tests import monolix_util as U

D64 = dict(dtype=torch.float64)


def test_oracle_is_causal_and_hears_far_tokens():
    cfg = U.full_config()
    w = mo.random_weights(cfg, 3)
    toks = U.tokens(40, cfg["vocab"], 4)
    full = mo.forward(toks, w, cfg)
    assert torch.allclose(mo.forward(toks[:25], w, cfg), full[:25], atol=1e-9)
    other = list(toks)
    other[3] = (other[3] + 1) % cfg["vocab"]
    moved = mo.forward(other, w, cfg)
    assert torch.allclose(moved[:3], full[:3], atol=1e-9) and (moved[39] - full[39]).abs().max() > 1e-6


def test_norm_weight_is_the_distance_of_the_gain_from_one():
    x = torch.randn(5, 24, **D64) * 7
    y = mo.shifted_norm(x, torch.zeros(24, **D64), 0.0)
    assert torch.allclose((y * y).mean(-1), torch.ones(5, **D64))
    assert torch.allclose(mo.shifted_norm(x, torch.full((24,), 0.5, **D64), 0.0), 1.5 * y)
    assert float(mo.shifted_norm(torch.zeros(1, 24, **D64), torch.zeros(24, **D64), 1e-5).abs().max()) == 0.0


def attn_weights(W, H, G, D, seed=0):
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s: torch.randn(*s, generator=g, **D64)
    return {"a.q": rn(H * D, W), "a.k": rn(G * D, W), "a.q.b": rn(H * D), "a.k.b": rn(G * D), "a.q.norm": 1 + 0.3 * rn(D),
            "a.k.norm": 1 + 0.3 * rn(D), "a.o": torch.eye(H * D, **D64)}


def test_a_lone_token_returns_its_projected_key():
    """the value is W_k x + b: no norm, no rotation, no projection of its own"""
    H, G, D, W = 2, 1, 4, 6
    m = U.attention(H, G, D)["mixer"]
    w = attn_weights(W, H, G, D)
    x = torch.randn(1, W, **D64)
    out = mo.attention(x, w, "a", m, 1e-5)
    assert torch.allclose(out[0], (w["a.k"] @ x[0] + w["a.k.b"]).repeat(2))


def test_scores_by_hand():
    """two positions, one head: the score from the norm (before the rotation, weight per coordinate), the rotation of the
    first two of four coordinates, and the scale"""
    m = U.attention(1, 1, 4, dims=2, base=10.0, scale=0.7)["mixer"]
    w = attn_weights(4, 1, 1, 4, seed=5)
    x = torch.randn(2, 4, **D64)
    q, k = x @ w["a.q"].T + w["a.q.b"], x @ w["a.k"].T + w["a.k.b"]
    unit = lambda z, nw: [float(z[i]) / math.sqrt(sum(float(c) ** 2 for c in z) / 4 + 1e-5) * float(nw[i]) for i in range(4)]
    qn, k0, k1 = unit(q[1], w["a.q.norm"]), unit(k[0], w["a.k.norm"]), unit(k[1], w["a.k.norm"])
    turn = lambda z: [z[0] * math.cos(1) - z[1] * math.sin(1), z[1] * math.cos(1) + z[0] * math.sin(1), z[2], z[3]]
    qn, k1 = turn(qn), turn(k1)
    s0, s1 = 0.7 * sum(a * b for a, b in zip(qn, k0)), 0.7 * sum(a * b for a, b in zip(qn, k1))
    p0 = 1 / (1 + math.exp(s1 - s0))
    assert torch.allclose(mo.attention(x, w, "a", m, 1e-5)[1], p0 * k[0] + (1 - p0) * k[1])


def router(correction, count=1, keep=1, experts=4, identity=0, top=2):
    w = {"r.router": torch.eye(experts + identity, **D64), "r.correction": torch.tensor(correction, **D64)}
    return w, U.moe(experts, top, 8, identity, count, keep)["router"]


def test_router_weights_are_the_plain_scores():
    z = torch.tensor([[0.0, 1.0, 2.0, 3.0]], **D64)
    s = torch.softmax(z, -1)[0]
    w, r = router([0.0, 0.0, 0.0, 0.0])
    ids, wt = mo.route(z, w, "r", r)
    assert ids.tolist() == [[3, 2]] and torch.allclose(wt[0], s[[3, 2]])            # not renormalised
    w, r = router([2.0, 0.0, 0.0, -2.0])
    ids, wt = mo.route(z, w, "r", r)
    assert ids.tolist() == [[0, 2]] and torch.allclose(wt[0], s[[0, 2]])            # the correction chooses, it does not weigh


def test_groups_are_scored_by_their_best_member_and_the_others_cannot_win():
    z = torch.zeros(1, 6, **D64)
    w, r = router([0.5, -9.0, 0.4, 0.4, 0.0, 0.0], count=3, keep=1, experts=4, identity=2)
    ids, _ = mo.route(z, w, "r", r)
    assert ids.tolist() == [[0, 1]]               # by the sum of two the second group would win; -9 still beats a dropped group
    w, r = router([-3.0, -1.0, -2.0, -2.5], count=2, keep=1)
    assert mo.route(torch.zeros(1, 4, **D64), w, "r", r)[0].tolist() == [[1, 0]]      # every choice score negative


def test_identity_experts_hand_their_input_on_and_the_shared_gate_is_a_scalar():
    W = 4
    g = torch.Generator().manual_seed(1)
    rn = lambda *s: torch.randn(*s, generator=g, **D64)
    spec = U.moe(2, 1, 8, identity=2, shared=8)
    w = {"m.router": torch.zeros(4, W, **D64), "m.correction": torch.tensor([0.0, 0.0, 0.0, 1.0], **D64),
         "m.shared.up": rn(8, W), "m.shared.down": rn(W, 8), "m.shared.sg": rn(1, W)}
    for e in range(2):
        w[f"m.e{e}.up"], w[f"m.e{e}.down"] = rn(8, W), rn(W, 8)
    x = rn(3, W)
    dense = torch.stack([w["m.shared.down"] @ torch.relu(w["m.shared.up"] @ t) ** 2 / (1 + math.exp(-float(w["m.shared.sg"][0] @ t)))
                         for t in x])
    assert torch.allclose(mo.moe(x, w, "m", spec), 0.25 * x + dense)


@pytest.mark.parametrize("mistake", ["alpha", "scale1", "scale2", "plain-gain", "values", "norm-after", "group-sum", "renorm",
                                     "identity", "gate", "borrow"])
def test_mistakes_planted_in_the_oracle_show(mistake, monkeypatch):
    """each mechanism left out or done otherwise moves the logits by far more than the GPU tests' bar"""
    cfg = U.full_config()
    w = mo.random_weights(cfg, 11)
    toks = U.tokens(40, cfg["vocab"], 12)
    want = mo.forward(toks, w, cfg)
    if mistake == "alpha":
        cfg["postln_alpha"] = 1.0
    elif mistake in ("scale1", "scale2"):
        name = {"scale1": ".ls1", "scale2": ".ls2"}[mistake]
        w = {k: torch.ones_like(v) if k.endswith(name) else v for k, v in w.items()}
    elif mistake == "plain-gain":
        monkeypatch.setattr(mo, "shifted_norm", lambda x, g, eps: mo.rms(x, eps) * (1 + g.abs()))
    elif mistake in ("values", "norm-after"):
        def other(x, w, p, m, eps):
            T, (H, G, D) = x.shape[0], (int(m[k]) for k in ("heads", "kv_heads", "dim"))
            q = (x @ w[f"{p}.q"].T + w[f"{p}.q.b"]).reshape(T, H, D)
            k = (x @ w[f"{p}.k"].T + w[f"{p}.k.b"]).reshape(T, G, D)
            v = mo.rms(k, eps) if mistake == "values" else k
            if mistake == "values":
                q, k = (mo.rotate(mo.rms(t, eps) * w[f"{p}.{n}.norm"], m.get("rot")) for t, n in ((q, "q"), (k, "k")))
            else:
                q, k = (mo.rms(mo.rotate(t, m.get("rot")), eps) * w[f"{p}.{n}.norm"] for t, n in ((q, "q"), (k, "k")))
            s = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(H // G, 1)) * m["scale"]
            s = s.masked_fill(~torch.ones(T, T, dtype=torch.bool).tril(), -math.inf)
            return torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v.repeat_interleave(H // G, 1)).reshape(T, H * D) @ w[f"{p}.o"].T
        monkeypatch.setattr(mo, "attention", other)
    elif mistake in ("group-sum", "renorm", "identity"):
        route = mo.route

        def other(x, w, p, r):
            if mistake == "group-sum" and r.get("groups"):
                E, ident, top, count, keep = mo.router_sizes(r)
                s = torch.softmax(x @ w[f"{p}.router"].T, -1)
                choice = (s + w[f"{p}.correction"]).reshape(len(x), count, -1)
                kept = choice.topk(min(2, choice.shape[-1]), -1)[0].sum(-1).topk(keep, -1)[1]
                mask = torch.zeros(len(x), count, dtype=torch.bool).scatter(1, kept, True)
                ids = choice.masked_fill(~mask[..., None], -math.inf).flatten(1).topk(top, -1)[1]
                return ids, s.gather(1, ids)
            ids, wt = route(x, w, p, r)
            if mistake == "renorm":
                wt = wt / wt.sum(-1, keepdim=True)
            if mistake == "identity":
                wt = wt * (ids < int(r["experts"]))
            return ids, wt
        monkeypatch.setattr(mo, "route", other)
    elif mistake == "gate":
        monkeypatch.setattr(mo, "shared_expert", mo.expert)
    elif mistake == "borrow":
        monkeypatch.setattr(mo, "weight_owner", lambda layers, i: 4 if i == 3 else (0 if i == 5 else i if i != 6 else 2))
    try:
        got = mo.forward(toks, w, cfg)
    except RuntimeError:
        assert mistake == "borrow"                       # another layer's tensors do not even fit
        return
    assert U.rel(got, want) > 1e-2


def test_configuration_registry_and_pool_shapes(tmp_path):
    from scratchpad_amd import registry
    raw = U.full_config()
    folder, _ = U.make_model(tmp_path, raw, seed=1)
    cfg = registry.load_config(folder, context_len=128)
    assert type(cfg).__name__ == "MonolixConfig" and registry.model_class_for(cfg).__name__ == "MonolixForCausalLM"
    assert cfg.owners == [0, 1, 2, 0, 4, 0, 2] and cfg.alpha == 1.7 and cfg.shift_layers() == [] and cfg.named_state() == {}
    assert cfg.window_cache() == {0: (2, 24, 24, False), 1: (2, 40, 40, False), 2: (1, 16, 16, False), 3: (2, 24, 24, False),
                                  4: (3, 32, 32, False), 5: (2, 24, 24, False), 6: (1, 16, 16, False)}
    assert cfg.cache_bytes_per_token(torch.bfloat16) == 2 * 2 * (3 * 2 * 24 + 2 * 40 + 2 * 16 + 3 * 32)


@pytest.mark.parametrize("spoil", ["vdim", "type", "mlp", "circle", "nowhere"])
def test_configurations_that_cannot_be_served_are_refused(spoil):
    from scratchpad_amd.monolix import MonolixConfig
    raw = U.full_config()
    if spoil == "vdim":
        raw["layers"][1]["mixer"]["vdim"] = 24
    elif spoil == "type":
        raw["layers"][1]["type"] = "mamba2"
    elif spoil == "mlp":
        raw["layers"][0]["mlp"]["kind"] = "dense"
    elif spoil == "circle":
        raw["layers"][0]["weights_of"] = 3
    else:
        raw["layers"][0]["weights_of"] = 9
    with pytest.raises(ValueError):
        MonolixConfig(raw)


def test_router_module_refuses_groups_that_cannot_hold_the_choice():
    from scratchpad_amd.moe import SoftmaxRouter
    SoftmaxRouter(8, 12, 3, groups=4, keep=1)
    for bad in (dict(top=4, groups=4, keep=1), dict(top=2, groups=5, keep=2), dict(top=2, groups=3, keep=4)):
        with pytest.raises(ValueError):
            SoftmaxRouter(8, 12, bad["top"], groups=bad["groups"], keep=bad["keep"])


def test_model_loads_a_checkpoint_on_cpu(tmp_path):
    """names and merges of load_weights (no kernel runs): merged projections hold the checkpoint's rows in order, norms hold
    the gain, a borrowing layer has no parameters"""
    from scratchpad_amd import distributed, registry
    from scratchpad_amd.monolix import MonolixForCausalLM
    if not distributed.model_parallel_is_initialized():
        distributed.initialize_model_parallel(1)
    raw = U.full_config()
    folder, w = U.make_model(tmp_path, raw, seed=2)
    cfg = registry.load_config(folder, context_len=64)
    model = MonolixForCausalLM(cfg, dtype=torch.float32)
    registry.load_weights(model, folder)
    assert sorted(model.layers) == ["0", "1", "2", "4"] and model.layers["1"].mlp is None
    l0 = model.layers["0"]
    assert torch.equal(l0.mix.qk[6 * 24:].double(), w["l0.mix.k"]) and torch.equal(l0.mix.k_bias.double(), w["l0.mix.k.b"])
    assert torch.equal(l0.mix.attn.k_norm.double(), w["l0.mix.k.norm"]) and l0.mix.attn.qk_norm == 2
    assert torch.allclose(l0.norm2.weight.double(), 1 + w["l0.norm2"], atol=1e-7) and torch.equal(l0.norm2.scale.double(), w["l0.ls2"])
    assert torch.equal(l0.mlp.router.weight[:10].double(), w["l0.mlp.router"]) and torch.equal(l0.mlp.router.weight[10:].double(), w["l0.mlp.shared.sg"])
    assert torch.equal(l0.mlp.experts.up[6].double(), w["l0.mlp.e6.up"]) and torch.equal(l0.mlp.experts.down[2].double(), w["l0.mlp.e2.down"])
    assert torch.equal(l0.mlp.shared.down.double(), w["l0.mlp.shared.down"]) and l0.mlp.outputs == 10
    assert model.layers["2"].mlp.shared is None and model.layers["2"].mlp.router.weight.shape[0] == 4
    assert torch.equal(model.lm_head.weight[:cfg.vocab_size].double(), w["head"]) and torch.equal(model.embed.double(), w["embed"])
    assert torch.allclose(model.norm.weight.double(), 1 + w["final.norm"], atol=1e-7)
    assert json.load(open(folder + "/config.json"))["architecture"] == "Monolix"
