"""Monolix: a decoder-only design of sequential post-norm sublayers over an fp32 residual stream,
    x <- N(alpha x + s1 * mixer(x)) (1 + w1);    x <- N(alpha x + s2 * ff(x)) (1 + w2),
N being division by the row's root mean square, alpha one constant of the model, s1 and s2 learned vectors: every sublayer
reads the stream itself.  The mixer is grouped-query softmax attention without a value projection - the values are the keys
as projected, with their bias, before norm and rotation; q and k have biases, are normed per head with a learned weight
shared by the heads, and then rotated on part of each head (rotate-half pairs).  The feed-forward is a mixture of
relu-square experts under one softmax router: the choice adds a learned correction to the scores and is confined to the best
groups of neighbouring outputs, the weights are the plain scores; the last outputs stand for identity experts, which hand
their input on.  A shared expert behind a scalar sigmoid gate runs for every token.  A layer may use another layer's
tensors; it then has a cache of its own.  Embedding and head are separate tables.

Everything that differs between models of the design comes from config.json (``MonolixConfig``); the model is assembled from
the framework's mechanisms - PostNorm / HalfAngleRotary (layers.py), PooledWindowAttention + SequenceBackend (attention.py),
IdentityMoE (moe.py), WindowKVPool (pool.py), LogitsProcessor (llama.py) - and served by the ModelRunner like the other model
classes.  A cache layer's id is the index in the configuration's layer list, whoever owns the weights."""
from typing import Iterable, List, Optional, Tuple

import torch
from torch import nn

from . import _native
from .attention import PooledWindowAttention
from .forward_info import ForwardBatch
from .layers import GroupRMSNorm, HalfAngleRotary, PostNorm
from .llama import LogitsProcessor, LogitsProcessorOutput, ParallelLMHead
from .moe import IdentityMoE


class MonolixConfig:
    """config.json of the design, plus what the runner asks of any model configuration (vocab_size, context_len,
    num_hidden_layers, is_encoder_decoder) and what it builds the pools from."""
    architecture = "Monolix"
    is_encoder_decoder = False
    vision_config = None
    tie_word_embeddings = False

    def __init__(self, raw: dict, context_len: int = 8192):
        self.raw = raw
        self.vocab_size = int(raw["vocab"])
        self.hidden_size = int(raw["width"])
        self.layers: List[dict] = raw["layers"]
        self.num_hidden_layers = len(self.layers)
        self.rms_norm_eps = float(raw["norm"]["eps"])
        self.alpha = float(raw["postln_alpha"])
        self.context_len = context_len
        self.owners = [self._owner(i) for i in range(self.num_hidden_layers)]     # whose tensors layer i uses
        for layer in self.layers:
            if layer["type"] != "attention":
                raise ValueError(f"unknown layer type {layer['type']!r}")
            if layer.get("mlp") is not None and layer["mlp"]["kind"] != "moe":
                raise ValueError(f"unknown feed-forward kind {layer['mlp']['kind']!r}")
            if int(layer["mixer"]["dim"]) != int(layer["mixer"]["vdim"]):
                raise ValueError("the values are the keys: vdim must equal dim")

    def _owner(self, i: int) -> int:
        seen = set()
        while self.layers[i].get("weights_of") is not None:
            if i in seen:
                raise ValueError("weights_of goes in a circle")
            seen.add(i)
            i = int(self.layers[i]["weights_of"])
            if not 0 <= i < self.num_hidden_layers:
                raise ValueError("weights_of names no layer")
        return i

    # ---- what the runner builds its pools from
    def window_cache(self):
        """{layer id: (kv_heads, dim, vdim, pooled)} of the layers that keep a key/value row per token"""
        return {i: (int(l["mixer"]["kv_heads"]), int(l["mixer"]["dim"]), int(l["mixer"]["vdim"]), False)
                for i, l in enumerate(self.layers)}

    def shift_layers(self):
        return []                                     # no mixer reads the previous token's input

    def named_state(self):
        return {}                                     # nothing is carried besides the cache

    def cache_bytes_per_token(self, kv_dtype: torch.dtype) -> int:
        per = sum(g * (d + dv) for g, d, dv, _ in self.window_cache().values())
        return max(1, per * torch.finfo(kv_dtype).bits // 8)


class MonolixAttention(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, dtype=None):
        super().__init__()
        H, G, D = (int(m[k]) for k in ("heads", "kv_heads", "dim"))
        self.heads, self.kv_heads, self.dim, self.eps = H, G, D, eps
        self.qk = nn.Parameter(torch.empty((H + G) * D, width, dtype=dtype), requires_grad=False)
        f32 = dict(dtype=torch.float32)
        self.q_bias = nn.Parameter(torch.zeros(H * D, **f32), requires_grad=False)
        self.k_bias = nn.Parameter(torch.zeros(G * D, **f32), requires_grad=False)
        self.o = nn.Parameter(torch.empty(width, H * D, dtype=dtype), requires_grad=False)
        rot = m.get("rot")
        self.rotary = None
        if rot and int(rot["dims"]) > 0:
            if int(rot["dims"]) > D:
                raise ValueError("rot.dims exceeds the head size")
            self.rotary = HalfAngleRotary(int(rot["dims"]), float(rot["base"]))
        self.attn = PooledWindowAttention(H, G, D, D, float(m["scale"]), None, norm_values=False, qk_norm="before",
                                          keys_as_values=True)

    def forward(self, positions, h: torch.Tensor, forward_batch: ForwardBatch, cache_id: int) -> torch.Tensor:
        nq = self.heads * self.dim
        qk = _native.linear(h, self.qk)
        q = qk[:, :nq]
        self.attn.store(q, qk[:, nq:], None, self.rotary, positions, self.eps, forward_batch, cache_id=cache_id,
                        biases=(self.q_bias.data, self.k_bias.data, None))
        return _native.linear(self.attn(q, forward_batch, cache_id=cache_id), self.o)


class MonolixLayer(nn.Module):
    """the tensors of one layer; it may run in several places of the layer list, with a cache for each"""

    def __init__(self, config: MonolixConfig, layer_id: int, dtype=None):
        super().__init__()
        spec, W, eps = config.layers[layer_id], config.hidden_size, config.rms_norm_eps
        self.mix = MonolixAttention(W, spec["mixer"], eps, dtype)
        self.norm1 = PostNorm(W, eps, config.alpha, layer_scale=True)
        self.mlp = None
        mlp = spec.get("mlp")
        if mlp is not None:
            r, groups, shared = mlp["router"], mlp["router"].get("groups") or {}, mlp.get("shared")
            self.mlp = IdentityMoE(W, int(r["experts"]), int(r.get("identity", 0)), int(r["top"]), int(mlp["expert"]["ff"]),
                                   int(groups.get("count", 1)), int(groups.get("keep", 1)),
                                   None if shared is None else int(shared["ff"]), dtype)
            self.norm2 = PostNorm(W, eps, config.alpha, layer_scale=True)

    def forward(self, positions, x: torch.Tensor, h: torch.Tensor, forward_batch: ForwardBatch, cache_id: int, dtype,
                want_lo: bool) -> Optional[torch.Tensor]:
        """x: the fp32 stream, updated in place; h = x in the projections' dtype.  Returns the new x in that dtype."""
        y = self.mix(positions, h, forward_batch, cache_id)
        if self.mlp is None:
            return self.norm1(x, y, dtype, want_lo)
        h = self.norm1(x, y, dtype)
        return self.norm2(x, self.mlp(h, x), dtype, want_lo)


class MonolixForCausalLM(nn.Module):
    # parameters keep the dtypes they are declared with (fp32 norms, biases, router) whatever the runner's dtype
    keeps_parameter_dtypes = True
    supports_tensor_parallel = False
    # Largest decode step that is captured into a HIP graph (the step has no host synchronisation and no data-dependent
    # shape); larger steps run eagerly.
    max_graph_batch = 64
    # sources of the HIP library this model's path needs beyond the core (scratchpad_amd.build.build_native(only=...));
    # ssm.hip: the fp32 product of few rows that routers share with step sizes
    NATIVE_SOURCES = ["stream_norm.hip", "window_attention.hip", "moe.hip", "ssm.hip"]

    def __init__(self, config: MonolixConfig, dtype=None):
        super().__init__()
        self.config = config
        self.dtype = dtype or torch.get_default_dtype()
        self.layers = nn.ModuleDict({str(i): MonolixLayer(config, i, dtype) for i in sorted(set(config.owners))})
        self.norm = GroupRMSNorm(config.hidden_size, 1, config.rms_norm_eps)
        self.embed = nn.Parameter(torch.empty(config.vocab_size, config.hidden_size, dtype=dtype), requires_grad=False)
        self.lm_head = ParallelLMHead(config.vocab_size, config.hidden_size, dtype)
        self.logits_processor = LogitsProcessor(config)
        self.capture_layers: Optional[list] = None     # set to a list to collect the stream after every layer

    @torch.no_grad()
    def forward(self, input_ids, positions, forward_batch: ForwardBatch, input_embeds=None) -> LogitsProcessorOutput:
        dtype = self.embed.dtype
        x, h = _native.embed_scale(self.embed.data, input_ids, 1.0, want_lo=True)
        last = len(self.config.owners) - 1
        for i, owner in enumerate(self.config.owners):
            h = self.layers[str(owner)](positions, x, h, forward_batch, i, dtype, i < last)
            if self.capture_layers is not None:
                self.capture_layers.append(x.clone())
        return self.logits_processor(input_ids, self.norm(x, dtype), self.lm_head, forward_batch)

    # ---- weights --------------------------------------------------------------------------------------------------
    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> None:
        """Checkpoint names of the design ('embed', 'head', 'final.norm', 'l<i>.norm1|norm2|ls1|ls2', 'l<i>.mix.q|k' with
        '.b' and '.norm', 'l<i>.mix.o', 'l<i>.mlp.router|correction', 'l<i>.mlp.e<j>.up|down', 'l<i>.mlp.shared.up|down|sg')
        -> this module's (partly merged) parameters.  The layer norms' and the final norm's weights are stored as their
        distance from one; the parameters hold the gain itself."""
        w = dict(weights)
        used = set()

        def take(name):
            used.add(name)
            return w[name]

        def put(param: nn.Parameter, value: torch.Tensor):
            value = value.reshape(param.shape) if value.numel() == param.numel() and value.dim() != param.dim() else value
            if value.shape != param.shape:
                raise RuntimeError(f"shape {tuple(value.shape)} does not fit parameter {tuple(param.shape)}")
            param.data.copy_(value.to(param.dtype))

        def gain(param: nn.Parameter, name: str):
            put(param, 1.0 + take(name).to(torch.float32))

        put(self.embed, take("embed"))
        put(self.lm_head.weight, self.lm_head.shard_from_full(take("head")))
        gain(self.norm.weight, "final.norm")
        for key, layer in self.layers.items():
            p, mix = f"l{key}", layer.mix
            M = f"{p}.mix"
            put(mix.qk, torch.cat([take(f"{M}.q"), take(f"{M}.k")], 0))
            put(mix.q_bias, take(f"{M}.q.b"))
            put(mix.k_bias, take(f"{M}.k.b"))
            put(mix.attn.q_norm, take(f"{M}.q.norm"))
            put(mix.attn.k_norm, take(f"{M}.k.norm"))
            put(mix.o, take(f"{M}.o"))
            gain(layer.norm1.weight, f"{p}.norm1")
            put(layer.norm1.scale, take(f"{p}.ls1"))
            if layer.mlp is None:
                continue
            gain(layer.norm2.weight, f"{p}.norm2")
            put(layer.norm2.scale, take(f"{p}.ls2"))
            mlp, F = layer.mlp, f"{p}.mlp"
            for e in range(mlp.experts.experts):
                mlp.experts.put(e, take(f"{F}.e{e}.up"), take(f"{F}.e{e}.down"))
            router = take(f"{F}.router")
            if mlp.shared is not None:
                router = torch.cat([router, take(f"{F}.shared.sg").to(router.dtype)], 0)
                put(mlp.shared.up, take(f"{F}.shared.up"))
                put(mlp.shared.down, take(f"{F}.shared.down"))
            put(mlp.router.weight, router)
            put(mlp.router.correction, take(f"{F}.correction"))
        extra = set(w) - used
        if extra:
            import warnings
            warnings.warn(f"checkpoint tensors no part of the configured model reads: {sorted(extra)[:8]}")

    def init_random(self, generator: torch.Generator) -> None:
        """random weights of a plausible scale (benchmarks and tests of the host path: no checkpoint)"""
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("scale", "q_norm", "k_norm") or (leaf == "weight" and p.dim() == 1):
                p.data.fill_(1.0)
            elif leaf == "embed":
                p.data.normal_(0.0, 1.0, generator=generator)
            elif p.dim() >= 2:
                p.data.normal_(0.0, 1.0 / (p.shape[-1] ** 0.5), generator=generator)
            else:
                p.data.normal_(0.0, 0.01, generator=generator)
