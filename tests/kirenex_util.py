"""Helpers of the Kirenex tests: small configurations whose sizes differ from one another (key width unlike value width, query
heads unlike key/value heads, rotations narrower than the head, latent ranks that are no power of two, windows shorter than the
prompts, layers that read another layer's latent rows), a checkpoint folder written from the oracle's random weights, and the
comparison used throughout."""
import torch

from oracle import kirenex as ko
from tests.tizalorn_util import rel, tokens, write_checkpoint  # noqa: F401  (the checkpoint writer is format-only)


def latent(heads, dim, rot_dim, vdim, kv_rank, base=300.0, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale or (dim + rot_dim) ** -0.5,
         "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def parallel(heads, kv_heads, dim, vdim, rheads, rkv, rdim, rvdim, size=11, keep=2, dims=None, scaling=True, base=500.0, conv=3,
             scale=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if size:
        left["mask"] = {"size": size, "keep_first": keep}
    if dims != 0:
        left["rot"] = {"base": base, "dims": dims or dim}
        if scaling:
            left["rot"]["scaling"] = {"factor": 3.0, "low": 1.0, "high": 3.0, "original": 40}
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": rheads, "kv_heads": rkv, "dim": rdim, "vdim": rvdim,
                                                                  "conv": conv}}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def config(layers, width=80, vocab=173, eps=1e-5, alpha=1.7, positions=420):
    return {"architecture": "Kirenex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha,
            "max_positions": positions, "layers": [{**spec, "mlp": mlp} for spec, mlp in layers]}


def full_config():
    """both mixers in an order of their own, sizes unlike each other; two latent caches of different widths, the first read by
    two later layers; windows of 11, 24 and none; a layer without a feed-forward"""
    return config([
        (parallel(6, 2, 24, 40, 4, 2, 16, 24, size=11, keep=3, dims=16, conv=4), dense(120)),
        (latent(3, 24, 8, 40, 72), dense(56)),
        (latent(5, 16, 12, 8, 40, base=50.0), None),
        (parallel(4, 4, 16, 16, 3, 1, 40, 16, size=24, keep=1, scaling=False, conv=2), dense(72)),
        (latent(2, 40, 8, 24, 72, kv_from=1), dense(40)),
        (parallel(2, 1, 40, 24, 2, 2, 8, 40, size=None, dims=0, conv=1), dense(24)),
        (latent(4, 8, 8, 16, 72, kv_from=1, scale=0.4), dense(64)),
    ], width=96)


def make_model(tmp_path, cfg, seed=0, name="m"):
    w = ko.random_weights(cfg, seed)
    return write_checkpoint(str(tmp_path / name), cfg, w), w


def greedy(prompt, w, cfg, n):
    """n tokens of greedy generation by the oracle (the whole sequence again for every token)"""
    seq, out = list(prompt), []
    for _ in range(n):
        t = int(torch.argmax(ko.forward(seq, w, cfg, last_only=True)[-1]))
        out.append(t)
        seq.append(t)
    return out


def random_config(seed: int):
    """a design drawn at random: layer order, shared rows, every size and constant"""
    import random
    r = random.Random(seed)
    layers = []
    for i in range(r.randint(2, 6)):
        owners = [j for j, (s, _) in enumerate(layers) if s["type"] == "latent_attention" and "kv_from" not in s["mixer"]]
        if r.random() < 0.5:
            heads, dim, vdim = r.choice([1, 2, 3, 4, 6, 9]), r.choice([8, 16, 24, 64]), r.choice([8, 16, 40, 72])
            scale = r.choice([None, 0.3, 0.11])
            if owners and r.random() < 0.5:
                j = r.choice(owners)
                m = layers[j][0]["mixer"]
                spec = latent(heads, dim, m["rot_dim"], vdim, m["kv_rank"], m["rot"]["base"], scale, kv_from=j)
            else:
                spec = latent(heads, dim, r.choice([2, 8, 16, 24]), vdim, r.choice([8, 24, 40, 64, 136]),
                              r.choice([100.0, 10000.0, 1e6]), scale)
        else:
            heads = r.choice([1, 2, 3, 4, 6])
            kv = r.choice([d for d in range(1, heads + 1) if heads % d == 0])
            dim = r.choice([8, 16, 24, 64])
            rheads = r.choice([1, 2, 4, 6])
            spec = parallel(heads, kv, dim, r.choice([8, 16, 40, 64]), rheads,
                            r.choice([d for d in range(1, rheads + 1) if rheads % d == 0]), r.choice([8, 16, 20, 40]),
                            r.choice([8, 24, 64]), size=r.choice([None, 1, 5, 16, 33]), keep=r.choice([0, 1, 4, 7]),
                            dims=r.choice([0, dim, dim // 2]), scaling=r.random() < 0.6, base=r.choice([100.0, 10000.0]),
                            conv=r.choice([1, 2, 4, 5]), scale=r.choice([None, 0.3]))
        layers.append((spec, None if r.random() < 0.2 else dense(r.choice([8, 24, 40, 100]))))
    return config(layers, width=r.choice([48, 64, 96, 100]), vocab=r.choice([61, 130, 257]), eps=r.choice([1e-6, 1e-5]),
                  alpha=r.choice([1.0, 1.9, 4.0]), positions=r.choice([128, 200]))
