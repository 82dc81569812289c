"""Helpers of the Monolix tests: small configurations whose sizes differ from one another (query heads unlike key/value
heads, a rotation narrower than the head, widths that are no power of two, groups of several sizes, layers that borrow
another's tensors), a checkpoint folder written from the oracle's random weights, and the comparison used throughout."""
import torch

from oracle import monolix as mo
from tests.tizalorn_util import rel, tokens, write_checkpoint  # noqa: F401  (the checkpoint writer is format-only)


def attention(heads, kv_heads, dim, dims=None, base=500.0, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale or dim ** -0.5}
    if dims != 0:
        m["rot"] = {"base": base, "dims": dims or dim}
    return {"type": "attention", "mixer": m}


def moe(experts, top, ff, identity=0, count=None, keep=None, shared=None):
    router = {"experts": experts, "top": top, "identity": identity}
    if count:
        router["groups"] = {"count": count, "keep": keep}
    out = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def config(layers, width=80, vocab=173, eps=1e-5, alpha=1.7):
    """layers: (mixer, mlp), or the number of the layer whose tensors this one uses"""
    out = []
    for spec in layers:
        if isinstance(spec, int):
            out.append({**out[spec], "weights_of": spec})
        else:
            out.append({**spec[0], "mlp": spec[1]})
    return {"architecture": "Monolix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "layers": out}


def full_config():
    """four layers of unlike sizes and three that borrow tensors (one of them from a borrower); groups with and without
    pruning, a router without identity experts, one without a shared expert, a layer without a feed-forward"""
    return config([
        (attention(6, 2, 24, dims=16), moe(7, 3, 40, identity=3, count=5, keep=2, shared=56)),
        (attention(2, 2, 40, dims=0, scale=0.3), None),
        (attention(4, 1, 16, dims=8, base=10000.0), moe(4, 1, 24)),
        0,
        (attention(3, 3, 32), moe(5, 4, 16, identity=7, count=3, keep=1, shared=24)),
        3,
        2,
    ], width=96)


def make_model(tmp_path, cfg, seed=0, name="m"):
    w = mo.random_weights(cfg, seed)
    return write_checkpoint(str(tmp_path / name), cfg, w), w


def greedy(prompt, w, cfg, n):
    """n tokens of greedy generation by the oracle (the whole sequence again for every token)"""
    seq, out = list(prompt), []
    for _ in range(n):
        t = int(torch.argmax(mo.forward(seq, w, cfg, last_only=True)[-1]))
        out.append(t)
        seq.append(t)
    return out


def random_config(seed: int):
    """a design drawn at random: layer order, borrowed tensors, every size and constant"""
    import random
    r = random.Random(seed)
    layers = []
    for i in range(r.randint(2, 6)):
        if i and r.random() < 0.35:
            layers.append(r.randrange(i))
            continue
        heads = r.choice([1, 2, 3, 4, 6])
        kv = r.choice([d for d in range(1, heads + 1) if heads % d == 0])
        dim = r.choice([8, 16, 24, 32, 64, 72])
        spec = attention(heads, kv, dim, dims=r.choice([0, dim, dim // 2 // 2 * 2]), base=r.choice([50.0, 10000.0, 1e6]),
                         scale=r.choice([None, 0.3, 0.11]))
        e, ident = r.choice([(2, 2), (4, 0), (6, 3), (9, 3), (12, 4), (5, 1)])
        count = r.choice([d for d in (1, 2, 3, 4, 6) if (e + ident) % d == 0])
        keep = r.randint(1, count)
        top = r.randint(1, min(4, keep * ((e + ident) // count)))
        mlp = None if r.random() < 0.15 else moe(e, top, r.choice([8, 24, 40, 64]), ident, count, keep,
                                                 r.choice([None, 16, 72]))
        layers.append((spec, mlp))
    return config(layers, width=r.choice([48, 64, 96, 100]), vocab=r.choice([61, 130, 257]), eps=r.choice([1e-6, 1e-5]),
                  alpha=r.choice([1.0, 1.9, 4.0]))
