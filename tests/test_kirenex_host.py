"""Kirenex on the CPU: properties of the oracle's mechanisms in closed form or in limiting cases (the oracle is what the GPU
tests compare with, so it is checked against arithmetic that does not share its code), mistakes planted in the oracle and
seen in its logits, the configuration reader, the registry, the pool shapes and the merges of load_weights.  No kernel runs."""
import copy
import json
import math

import pytest
import torch

from oracle import kirenex as ko
from tests import kirenex_util as U

D64 = dict(dtype=torch.float64)


def gen(seed=0):
    g = torch.Generator().manual_seed(seed)
    return lambda *s: torch.randn(*s, generator=g, **D64)


def test_oracle_is_causal_and_hears_far_tokens():
    cfg = U.full_config()
    w = ko.random_weights(cfg, 3)
    toks = U.tokens(60, cfg["vocab"], 4)
    full = ko.forward(toks, w, cfg)
    assert torch.allclose(ko.forward(toks[:25], w, cfg), full[:25], atol=1e-9)
    other = list(toks)
    other[3] = (other[3] + 1) % cfg["vocab"]
    moved = ko.forward(other, w, cfg)
    assert torch.allclose(moved[:3], full[:3], atol=1e-9) and (moved[59] - full[59]).abs().max() > 1e-6


def test_positions_are_added_unscaled():
    w = {"embed": torch.eye(4, **D64) * 3, "pos": torch.arange(20, **D64).reshape(5, 4)}
    assert ko.embed([2, 2], w).tolist() == [[0, 1, 5, 3], [4, 5, 9, 7]]


def test_gelu_is_the_tanh_form():
    z = torch.tensor([-3.0, -0.5, 0.0, 1.0, 2.5], **D64)
    assert torch.allclose(ko.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert not torch.allclose(ko.gelu_tanh(z), torch.nn.functional.gelu(z), atol=1e-5)


def test_window_and_kept_tokens_by_enumeration():
    m = ko.window_mask(9, {"size": 3, "keep_first": 2})
    seen = [[j for j in range(9) if m[i, j]] for i in range(9)]
    assert seen == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 3, 4, 5], [0, 1, 4, 5, 6], [0, 1, 5, 6, 7],
                    [0, 1, 6, 7, 8]]
    assert torch.equal(ko.window_mask(6, {"size": 1, "keep_first": 0}), torch.eye(6, dtype=torch.bool))
    assert torch.equal(ko.window_mask(6, None), torch.ones(6, 6, dtype=torch.bool).tril())


def test_frequencies_by_wavelength():
    f = ko.rotary_frequencies({"dims": 8, "base": 10.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 32}})
    plain = [10.0 ** (-2 * i / 8) for i in range(4)]
    turns = [32 * p / (2 * math.pi) for p in plain]                       # 5.09, 2.86, 1.61, 0.91
    want = [plain[0]] + [(1 - s) * p / 4 + s * p for p, s in ((plain[i], (turns[i] - 1) / 3) for i in (1, 2))] + [plain[3] / 4]
    assert torch.allclose(f, torch.tensor(want, **D64))


def test_the_two_rotations_pair_other_coordinates():
    x = torch.zeros(2, 1, 6, **D64)
    x[1, 0, 0] = 1.0
    rot = {"dims": 4, "base": 10.0}
    half, near = ko.rotate_halves(x, rot)[1, 0], ko.rotate_neighbours(x, rot)[1, 0]
    c, s = math.cos(1.0), math.sin(1.0)
    assert torch.allclose(half, torch.tensor([c, 0, s, 0, 0, 0], **D64)) and torch.allclose(near, torch.tensor([c, s, 0, 0, 0, 0], **D64))


def test_latent_scores_depend_on_distance_only_and_a_lone_token_returns_its_value():
    rn = gen(1)
    m = U.latent(2, 4, 6, 5, 8)["mixer"]
    W = 7
    w = {"a.q": rn(20, W), "a.dkv": rn(14, W), "a.dkv.norm": 1 + 0.3 * rn(8), "a.uk": rn(8, 8), "a.uv": rn(10, 8), "a.g": rn(10, W),
         "a.o": torch.eye(10, **D64)}
    x = rn(1, W)
    c, kr = ko.latent(x, w, "a", m, 1e-5)
    z = (w["a.dkv"] @ x[0])[:8]
    assert torch.allclose(c[0], z / torch.sqrt((z * z).mean() + 1e-5) * w["a.dkv.norm"])
    want = (w["a.uv"] @ c[0]) / (1 + torch.exp(-(w["a.g"] @ x[0])))
    assert torch.allclose(ko.latent_attention(x, w, "a", m, (c, kr))[0], want)
    # equal tokens at every position: the rotated parts of query and key turn together
    xs = x.repeat(9, 1)
    qr = ko.rotate_neighbours((xs @ w["a.q"].T).reshape(9, 2, 10)[..., 4:], m["rot"])
    krs = ko.latent(xs, w, "a", m, 1e-5)[1]
    s = qr[:, 0] @ krs.T
    assert torch.allclose(s[5, 2], s[8, 5]) and not torch.allclose(s[5, 2], s[5, 3])


def test_delta_rule_recalls_what_it_stored():
    """a full write (step size 1, no decay) under a unit key returns the value; a second write under the same key replaces it;
    decay halves what is read"""
    e = torch.eye(3, **D64)
    v = torch.tensor([[1.0, 2.0], [5.0, 7.0], [9.0, 9.0]], **D64)
    one = torch.ones(3, **D64)
    out = ko.delta_scan(e[[0, 0, 0]], e[[0, 1, 0]], v, one, one)
    assert torch.allclose(out, torch.stack([v[0], v[0], v[2]]))
    out = ko.delta_scan(e[[0, 0, 0]], e[[0, 1, 1]], v, one, torch.tensor([1.0, 0.5, 0.5], **D64))
    assert torch.allclose(out, torch.stack([v[0], v[0] / 2, v[0] / 4]))


def test_convolution_by_hand():
    u, k = torch.tensor([[1.0], [2.0], [3.0]], **D64), torch.tensor([[100.0, 10.0, 1.0]], **D64)
    assert ko.causal_conv(u, k)[:, 0].tolist() == [1.0, 12.0, 123.0]


def test_post_norm_and_average():
    rn = gen(2)
    x, y, w = rn(4, 6), rn(4, 6), rn(6)
    z = 2.5 * x + y
    assert torch.allclose(ko.post_norm(x, y, w, 2.5, 1e-5)[3], z[3] / math.sqrt(float((z[3] ** 2).mean()) + 1e-5) * w)
    one = torch.ones(6, **D64)
    avg = ko.average_of_normed(x, 100 * x, one, 3 * one, 0.0)
    assert torch.allclose(avg, 2 * ko.rms(x, 0.0))


@pytest.mark.parametrize("mistake", ["alpha", "positions", "branch-norm", "keep", "window+1", "window-1", "norm-after-rotation",
                                     "halves-for-neighbours", "no-scaling", "gate", "latent-norm", "own-rows", "decay", "beta",
                                     "silu-gate", "gelu", "conv", "unit", "pre-norm"])
def test_mistakes_planted_in_the_oracle_show(mistake, monkeypatch):
    """each mechanism left out or done otherwise moves the logits by far more than the GPU tests' bar"""
    cfg = U.full_config()
    w = ko.random_weights(cfg, 11)
    toks = U.tokens(60, cfg["vocab"], 12)
    want = ko.forward(toks, w, cfg)
    cfg = copy.deepcopy(cfg)
    left = cfg["layers"][0]["mixer"]["left"]
    if mistake == "alpha":
        cfg["postln_alpha"] = 1.0
    elif mistake == "positions":
        w = {**w, "pos": torch.zeros_like(w["pos"])}
    elif mistake == "branch-norm":
        monkeypatch.setattr(ko, "average_of_normed", lambda a, b, wa, wb, eps: 0.5 * (a * wa + b * wb))
    elif mistake == "keep":
        left["mask"]["keep_first"] = 0
    elif mistake.startswith("window"):
        left["mask"]["size"] += 1 if mistake.endswith("+1") else -1
    elif mistake == "norm-after-rotation":
        rot = ko.rotate_halves
        # the weight after the turn instead of before it
        def attn(h, w, p, m, eps, plain=ko.window_attention):
            one = {**w, f"{p}.q.norm": torch.ones_like(w[f"{p}.q.norm"])}
            monkeypatch.setattr(ko, "rotate_halves", lambda x, r: rot(x, r) * (w[f"{p}.q.norm"] if x.shape[1] == int(m["heads"]) else 1.0))
            out = plain(h, one, p, m, eps)
            monkeypatch.setattr(ko, "rotate_halves", rot)
            return out
        monkeypatch.setattr(ko, "window_attention", attn)
    elif mistake == "halves-for-neighbours":
        monkeypatch.setattr(ko, "rotate_neighbours", ko.rotate_halves)
    elif mistake == "no-scaling":
        left["rot"].pop("scaling")
    elif mistake == "gate":
        w = {k: (torch.zeros_like(v) if k.endswith("l1.mix.g") else v) for k, v in w.items()}
    elif mistake == "latent-norm":
        w = {k: (torch.ones_like(v) if k.endswith("dkv.norm") else v) for k, v in w.items()}
    elif mistake == "own-rows":
        latent = ko.latent_attention
        monkeypatch.setattr(ko, "latent_attention", lambda h, w, p, m, kept: latent(
            h, w, p, m, ko.latent(h, w, "l1.mix", m, 1e-5) if m.get("kv_from") is not None else kept))
    elif mistake in ("decay", "beta"):
        scan = ko.delta_scan
        monkeypatch.setattr(ko, "delta_scan", lambda q, k, v, b, g: scan(q, k, v, *((b, torch.ones_like(g)) if mistake == "decay"
                                                                                   else (torch.ones_like(b), g))))
    elif mistake == "silu-gate":
        silu = ko.silu
        monkeypatch.setattr(ko, "silu", lambda z: torch.sigmoid(z) if z.shape[1] == 96 else silu(z))       # layer 0's gate rows
    elif mistake == "gelu":
        monkeypatch.setattr(ko, "gelu_tanh", lambda z: z * torch.sigmoid(z))
    elif mistake == "conv":
        monkeypatch.setattr(ko, "causal_conv", lambda u, k: u * k[:, -1])
    elif mistake == "unit":
        monkeypatch.setattr(ko, "unit", lambda x: x)
    elif mistake == "pre-norm":
        monkeypatch.setattr(ko, "post_norm", lambda x, y, weight, alpha, eps: alpha * x + ko.rms(y, eps) * weight)
    assert U.rel(ko.forward(toks, w, cfg), want) > 1e-2


def test_configuration_registry_and_pool_shapes(tmp_path):
    from scratchpad_amd import registry
    from scratchpad_amd.pool import WindowKVPool
    raw = U.full_config()
    folder, _ = U.make_model(tmp_path, raw, seed=1)
    cfg = registry.load_config(folder, context_len=128)
    assert type(cfg).__name__ == "KirenexConfig" and registry.model_class_for(cfg).__name__ == "KirenexForCausalLM"
    assert cfg.alpha == 1.7 and cfg.shift_layers() == [] and cfg.context_len == 128
    assert registry.load_config(folder, context_len=9999).context_len == 420              # the learned positions bound it
    assert registry.load_config(folder).context_len == 420
    assert cfg.window_cache() == {0: (2, 24, 40, False), 3: (4, 16, 16, False), 5: (1, 40, 24, False)}
    assert cfg.latent_cache() == {1: (72, 8), 2: (40, 12)}                                 # the readers keep nothing
    assert cfg.named_state() == {0: {"S": (4, 16, 24), "conv": (3, 160)}, 3: {"S": (3, 40, 16), "conv": (1, 128)},
                                 5: {"S": (2, 8, 40), "conv": (0, 112)}}
    assert cfg.cache_bytes_per_token(torch.bfloat16) == 2 * (2 * 64 + 4 * 32 + 64 + 80 + 52)
    pool = WindowKVPool(10, torch.float32, cfg.window_cache(), "cpu", latent=cfg.latent_cache())
    assert pool.layer_num == 5 and pool.get_key_buffer(1).shape == (11, 80) and pool.get_value_buffer(1).shape == (11, 72)
    assert pool.get_kv_buffer(0)[1].shape == (11, 80) and sum(pool.get_kv_size_bytes()) == 11 * 2 * cfg.cache_bytes_per_token(torch.bfloat16)
    src = [torch.randn_like(b) for b in pool._all()]
    pool.transfer(torch.arange(11), src)
    assert all(torch.equal(a, b) for a, b in zip(pool.get_flat_data(torch.arange(11)), src))
    with pytest.raises(ValueError):
        WindowKVPool(10, torch.float32, {1: (1, 8, 8, False)}, "cpu", latent={1: (8, 4)})


@pytest.mark.parametrize("spoil", ["type", "mlp", "later", "chain", "rank", "rot", "parallel"])
def test_configurations_that_cannot_be_served_are_refused(spoil):
    from scratchpad_amd.kirenex import KirenexConfig
    raw = U.full_config()
    m = raw["layers"][4]["mixer"]
    if spoil == "type":
        raw["layers"][1]["type"] = "mamba2"
    elif spoil == "mlp":
        raw["layers"][0]["mlp"]["kind"] = "moe"
    elif spoil == "later":
        m["kv_from"] = 6
    elif spoil == "chain":
        raw["layers"][6]["mixer"]["kv_from"] = 4
    elif spoil == "rank":
        m["kv_rank"] = 64
    elif spoil == "rot":
        m["rot"]["base"] = 7.0
    else:
        m["kv_from"] = 3
    with pytest.raises(ValueError):
        KirenexConfig(raw)


def test_window_layer_and_splits_helpers():
    from scratchpad_amd import _native
    from scratchpad_amd.attention import PooledWindowAttention
    assert PooledWindowAttention(2, 1, 8, 8, 1.0, 0, window=None, keep_first=4).keep_first == 0
    with pytest.raises(ValueError):
        PooledWindowAttention(2, 1, 8, 8, 1.0, 0, window=16, block=4, keep_first=4)
    assert _native.latent_splits(16 * 8, 8, True, 8192) == 32 and _native.latent_splits(16 * 8, 8, True, 100) == 2
    assert _native.latent_splits(4096 * 16, 8, False, 8192) == 1 and _native.latent_splits(6 * 3, 2, False, 4096) == 32


def test_model_loads_a_checkpoint_on_cpu(tmp_path):
    """names and merges of load_weights (no kernel runs): merged projections hold the checkpoint's rows in order, per-head
    up-projections are stored the way the products read them, a layer that reads another's rows has no latent parameters"""
    from scratchpad_amd import distributed, registry
    from scratchpad_amd.kirenex import KirenexForCausalLM
    if not distributed.model_parallel_is_initialized():
        distributed.initialize_model_parallel(1)
    raw = U.full_config()
    folder, w = U.make_model(tmp_path, raw, seed=2)
    cfg = registry.load_config(folder, context_len=64)
    model = KirenexForCausalLM(cfg, dtype=torch.float32)
    registry.load_weights(model, folder)
    l0, l1, l4 = (model.layers[i] for i in (0, 1, 4))
    assert torch.equal(l1.mix.in_proj[:96].double(), w["l1.mix.q"]) and torch.equal(l1.mix.in_proj[96:176].double(), w["l1.mix.dkv"])
    assert torch.equal(l1.mix.in_proj[176:].double(), w["l1.mix.g"]) and torch.equal(l1.mix.latent_norm.double(), w["l1.mix.dkv.norm"])
    assert torch.equal(l1.mix.uk_t[2].double(), w["l1.mix.uk"].view(3, 24, 72)[2].T) and torch.equal(l1.mix.uv[1].double(), w["l1.mix.uv"][40:80])
    assert l4.mix.latent_norm is None and l4.mix.attn.layer_id == 1 and l4.mix.in_proj.shape[0] == 2 * 48 + 48
    assert torch.equal(l4.mix.in_proj[96:].double(), w["l4.mix.g"]) and l1.mix.attn.layer_id == 1
    assert torch.equal(l0.mix.in_proj[144:192].double(), w["l0.mix.left.k"]) and l0.mix.attn.keep_first == 3 and l0.mix.attn.window == 11
    assert torch.equal(l0.mix.in_proj[272:304].double(), w["l0.mix.right.q"]) and torch.equal(l0.mix.in_proj[-96:].double(), w["l0.mix.right.g"])
    assert torch.equal(l0.mix.right.gates[:4].double(), w["l0.mix.right.b"]) and torch.equal(l0.mix.right.gates[4:].double(), w["l0.mix.right.a"])
    assert torch.equal(l0.mix.right.conv[64:].double(), w["l0.mix.right.v.conv"]) and l0.mix.right.gates.dtype == torch.float32
    assert torch.equal(l0.norm1.branch_weight[1].double(), w["l0.mix.right.out"]) and l1.norm1.branch_weight is None
    assert torch.equal(l0.mlp.gate_up[120:].double(), w["l0.mlp.up"]) and model.layers[2].mlp is None
    assert torch.equal(model.pos.double(), w["pos"]) and torch.equal(model.lm_head.weight[:cfg.vocab_size].double(), w["head"])
    assert model.layers[5].mix.rotary is None and model.layers[5].mix.attn.window == 0
    assert json.load(open(folder + "/config.json"))["architecture"] == "Kirenex"
