"""Tedenex: a decoder around a fp32 residual stream whose sublayers sit between two zero-centred RMS
norms, x <- x + norm_b(f(norm_a x)), and whose layers end with an input of the token's own.  The
layers - in whatever order the configuration lists them - carry one of three mixers and an optional
feed-forward, and a stretch of them may run several times in a row with the same weights (every
pass with its own caches and state; ahead of every pass but the first the embedding output is added
to the stream again).

* ``attention``         biased q / k / v on grouped heads, a short causal filter over time on every
                        projected channel, per-head RMS norms of q and k, no rotation, a distance
                        penalty per head, keys of the query's own chunk of positions only
                        (``layers.attention.FilteredHeads`` + ``SinkAttention`` with a chunk and
                        without its sink);
* ``wkv``               RWKV-style time mixing (``layers.linear_attention.TokenShiftWKV``);
* ``latent_attention``  one cached latent and one rotated key part per token, queries through a
                        normed latent of their own, neighbouring pairs turned
                        (``layers.attention.LatentAttention``);
* feed-forward          W_down relu(W_up h)^2, or none;
* token input           ``layers.embedding_head.LayerTokenInput`` behind the feed-forward: its norm
                        has a plain weight.

The head is tied: final norm, then the embedding table.  Stream update, addition of the embedding at
a pass's end and the next sublayer's norm (or the rounding of the stream for the token input's gate)
are one kernel (``ops.post_norm_residual``).  ``TedenexConfig.from_dict`` reads the family's
``config.json``; the rank of the decay's low-rank projection comes from the checkpoint's tensor
shapes.  One rank only.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F

from minivllm_amd import ops
from minivllm_amd.layers.activation import ReluSquared
from minivllm_amd.layers.attention import FilteredHeads, LatentAttention, SinkAttention
from minivllm_amd.layers.embedding_head import LayerTokenInput, ScaledTiedHead
from minivllm_amd.layers.layernorm import OffsetRMSNorm
from minivllm_amd.layers.linear_attention import TokenShiftWKV
from minivllm_amd.layers.rotary_embedding import NeighbourRotation
from minivllm_amd.utils.context import get_context

MIXER_TYPES = ("attention", "wkv", "latent_attention")


# ------------------------------------------------------------------ configuration
@dataclass
class TedenexLayerSpec:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]]


@dataclass
class TedenexConfig:
    vocab_size: int
    hidden_size: int
    layers: List[TedenexLayerSpec] = field(default_factory=list)
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    side_dim: int = 0                    # numbers per layer of the token's own input; 0: none
    rms_norm_epsilon: float = 1e-6
    max_position: int = 1 << 20          # no table depends on it: positions enter as fp32 numbers
    name: str = "tedenex"
    architecture: str = "tedenex"
    tie_word_embeddings: bool = True

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def passes(self, i: int) -> int:
        """How often layer i runs per token."""
        return self.loop_times if self.loop_start <= i < self.loop_stop else 1

    def run_order(self) -> List[Tuple[int, int, bool]]:
        """(layer, pass, the embedding is added ahead of it) in the order the layers run."""
        a, b = self.loop_start, self.loop_stop
        out = [(i, 0, False) for i in range(a)]
        for p in range(self.loop_times if b > a else 0):
            out += [(i, p, i == a and p > 0) for i in range(a, b)]
        return out + [(i, 0, False) for i in range(b, len(self.layers))]

    @classmethod
    def from_dict(cls, c: dict, name: str = "tedenex") -> "TedenexConfig":
        layers = []
        for L in c["layers"]:
            if L["type"] not in MIXER_TYPES:
                raise ValueError(f"unknown layer type {L['type']!r}")
            f = L.get("mlp")
            if f and f.get("kind") != "dense":
                raise ValueError(f"unknown feed-forward kind {f.get('kind')!r}")
            layers.append(TedenexLayerSpec(L["type"], L["mixer"], f or None))
        loop = c.get("loop") or {}
        start, stop = int(loop.get("start", 0)), int(loop.get("stop", 0))
        times = int(loop.get("times", 1))
        if not (0 <= start <= stop <= len(layers)) or times < 1:
            raise ValueError("the loop must be a stretch of the layers that runs at least once")
        return cls(vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers,
                   loop_start=start, loop_stop=stop, loop_times=times if stop > start else 1,
                   side_dim=int((c.get("token_side") or {}).get("dim", 0)),
                   rms_norm_epsilon=float(c["norm"]["eps"]),
                   max_position=int(c.get("max_position", 1 << 20)), name=name)

    def validate_engine(self, engine_cfg) -> None:
        if engine_cfg.tp_degree != 1:
            raise ValueError("Tedenex runs on one rank (its mixers are not sharded)")
        for L in self.layers:
            m = L.mixer
            if L.type == "attention":
                H, G, D, E = _attention_sizes(m)
                if H % G:
                    raise ValueError("heads must be a multiple of kv_heads")
                if D > 1024 or E > 1024:
                    raise ValueError("the attention kernels take keys and values of at most 1024 "
                                     "numbers per head")
                if int(m["conv"]) < 1 or int((m.get("mask") or {}).get("size", 0)) < 0:
                    raise ValueError("conv must be at least 1 and mask.size not negative")
            elif L.type == "wkv":
                if int(m["dim"]) > 256:
                    raise ValueError("the recurrence kernel takes heads of at most 256 numbers")
            else:
                if int(m["rot"]["dims"]) > int(m["rot_dim"]) or int(m["rot"]["dims"]) % 2:
                    raise ValueError("rot.dims must be even and at most rot_dim")
                if int(m["kv_rank"]) + int(m["rot_dim"]) > 1024:
                    raise ValueError("attention over the latent runs with key rows of at most 1024 "
                                     "numbers (kv_rank + rot_dim)")


def _attention_sizes(m: dict) -> Tuple[int, int, int, int]:
    H, D = int(m["heads"]), int(m["dim"])
    return H, int(m.get("kv_heads", H)), D, int(m.get("vdim", D))


def _param(t: torch.Tensor, like: torch.Tensor) -> nn.Parameter:
    return nn.Parameter(t.to(device=like.device, dtype=like.dtype).contiguous(), requires_grad=False)


def _take(w: dict, key: str, shape, where: str) -> torch.Tensor:
    """``shape``: an entry of None matches any size."""
    if key not in w:
        raise KeyError(f"checkpoint lacks {where}{key}")
    t = w.pop(key)
    if len(shape) != t.dim() or any(s is not None and s != n for s, n in zip(shape, t.shape)):
        raise ValueError(f"shape mismatch for {where}{key}: expected {tuple(shape)}, checkpoint "
                         f"has {tuple(t.shape)}")
    return t


def _up8(n: int) -> int:
    return n + (-n % 8)


def _pad_rows(rows: List[torch.Tensor]) -> None:
    """Zero rows so that the fused projection's output has rows of whole runs of eight."""
    pad = -sum(r.shape[0] for r in rows) % 8
    if pad:
        rows.append(torch.zeros((pad,) + tuple(rows[0].shape[1:]), dtype=rows[0].dtype))


# ------------------------------------------------------------------ mixers
# ``forward(h, which)``: the normed input -> [T, W]; ``which`` is the pass of a looped layer.
class TedenexAttentionMixer(nn.Module):
    def __init__(self, W: int, m: dict, eps: float, passes: int):
        super().__init__()
        self.W = W
        H, G, D, E = _attention_sizes(m)
        slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=torch.float32)
        self.cores = nn.ModuleList([
            SinkAttention(H, G, D, E, float(m["scale"]), sink=False, distance_slopes=slopes,
                          chunk=int((m.get("mask") or {}).get("size", 0))) for _ in range(passes)])
        self.heads = FilteredHeads(H, G, D, E, int(m["conv"]), eps, passes)
        self.in_proj = nn.Parameter(torch.zeros(1, W), requires_grad=False)
        self.in_bias = nn.Parameter(torch.zeros(1), requires_grad=False)
        self.o_proj = nn.Parameter(torch.zeros(W, H * E), requires_grad=False)

    def attention_cores(self):
        return list(self.cores)

    def state_cores(self):
        return list(self.heads.slots)

    def forward(self, h: torch.Tensor, which: int) -> torch.Tensor:
        core = self.cores[which]
        q = self.heads(F.linear(h, self.in_proj, self.in_bias), core, which)
        return F.linear(core(q, None), self.o_proj)

    def load(self, w: dict, where: str, like) -> None:
        W, f = self.W, self.heads
        H, G, D, E = f.sizes
        sizes = (("q", H * D), ("k", G * D), ("v", G * E))
        rows = [_take(w, k, (n, W), where) for k, n in sizes]
        bias = [_take(w, k + ".b", (n,), where) for k, n in sizes]
        f.conv_weight.copy_(torch.cat([_take(w, k + ".conv", (n, f.taps), where) for k, n in sizes], 0))
        f.q_norm.copy_(_take(w, "q.norm", (D,), where))
        f.k_norm.copy_(_take(w, "k.norm", (D,), where))
        _pad_rows(rows)
        _pad_rows(bias)
        self.in_proj, self.in_bias = _param(torch.cat(rows, 0), like), _param(torch.cat(bias, 0), like)
        self.o_proj = _param(_take(w, "o", (W, H * E), where), like)

    @staticmethod
    def shapes(W, m, rank):
        H, G, D, E = _attention_sizes(m)
        out = []
        for k, n in (("q", H * D), ("k", G * D), ("v", G * E)):
            out += [(k, (n, W)), (k + ".b", (n,)), (k + ".conv", (n, int(m["conv"])))]
        return out + [("q.norm", (D,)), ("k.norm", (D,)), ("o", (W, H * E))]


class TedenexTimeMixer(nn.Module):
    def __init__(self, W: int, m: dict, eps: float, passes: int):
        super().__init__()
        self.W = W
        H, D = int(m["heads"]), int(m["dim"])
        self.unit = TokenShiftWKV(W, H, D, eps, passes)
        self.o_proj = nn.Parameter(torch.zeros(W, H * D), requires_grad=False)

    def attention_cores(self):
        return []

    def state_cores(self):
        return list(self.unit.slots)

    def forward(self, h: torch.Tensor, which: int) -> torch.Tensor:
        return F.linear(self.unit(h, which), self.o_proj)

    def load(self, w: dict, where: str, like) -> None:
        W, u = self.W, self.unit
        H, D = u.num_heads, u.head_dim
        u.mu.copy_(torch.stack([_take(w, "mu." + k, (W,), where) for k in u.MIXES], 0))
        u.proj = _param(torch.stack([_take(w, k, (H * D, W), where).t() for k in "rkvg"], 0), like)
        u.decay_down = _param(_take(w, "w1", (None, W), where), like)
        u.decay_up = _param(_take(w, "w2", (H * D, u.decay_down.shape[0]), where), like)
        u.decay_bias.copy_(_take(w, "w0", (H * D,), where))
        u.bonus.copy_(_take(w, "u", (H, D), where))
        u.norm_weight.copy_(_take(w, "norm", (H * D,), where))
        self.o_proj = _param(_take(w, "o", (W, H * D), where), like)

    @staticmethod
    def shapes(W, m, rank):
        H, D = int(m["heads"]), int(m["dim"])
        return ([("mu." + k, (W,)) for k in TokenShiftWKV.MIXES] + [(k, (H * D, W)) for k in "rkvg"]
                + [("w1", (rank, W)), ("w2", (H * D, rank)), ("w0", (H * D,)), ("u", (H, D)),
                   ("norm", (H * D,)), ("o", (W, H * D))])


class TedenexLatentMixer(nn.Module):
    def __init__(self, W: int, m: dict, eps: float, passes: int):
        super().__init__()
        self.W, self.eps, self.q_rank = W, eps, int(m["q_rank"])
        H, D, P, E, R = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        rot = NeighbourRotation(int(m["rot"]["dims"]), float(m["rot"]["base"]))
        self.attn = LatentAttention(H, D, P, E, R, float(m["scale"]), 0, rot, eps)
        self.later = nn.ModuleList([LatentAttention.make_core(H, P, R, float(m["scale"]), 0)
                                    for _ in range(passes - 1)])
        self.q_norm = nn.Parameter(torch.ones(self.q_rank, dtype=torch.float32), requires_grad=False)
        # W_dq's rows, padded so that the latent's block starts on a run of eight columns
        self.in_proj = nn.Parameter(torch.zeros(1, W), requires_grad=False)
        self.up_q = nn.Parameter(torch.zeros(H * (D + P), self.q_rank), requires_grad=False)
        self.o_proj = nn.Parameter(torch.zeros(W, H * E), requires_grad=False)

    def attention_cores(self):
        return [self.attn.core] + list(self.later)

    def state_cores(self):
        return []

    def forward(self, h: torch.Tensor, which: int) -> torch.Tensor:
        a, Q = self.attn, self.q_rank
        T, at = h.shape[0], _up8(Q)
        proj = F.linear(h, self.in_proj)
        q = F.linear(ops.rms_norm_rows(proj[:, :Q], self.q_norm, self.eps, h.dtype), self.up_q)
        o = a(q.view(T, a.num_heads, a.head_dim + a.rot_dim), proj[:, at:at + a.kv_rank + a.rot_dim],
              self.attention_cores()[which])
        return F.linear(o.view(T, -1), self.o_proj)

    def load(self, w: dict, where: str, like) -> None:
        W, a, Q = self.W, self.attn, self.q_rank
        H, D, P, E, R = a.num_heads, a.head_dim, a.rot_dim, a.v_head_dim, a.kv_rank
        rows = [_take(w, "dq", (Q, W), where)]
        _pad_rows(rows)
        rows.append(_take(w, "dkv", (R + P, W), where))
        _pad_rows(rows)
        self.in_proj = _param(torch.cat(rows, 0), like)
        self.q_norm.copy_(_take(w, "dq.norm", (Q,), where))
        self.up_q = _param(_take(w, "uq", (H * (D + P), Q), where), like)
        a.latent_norm.copy_(_take(w, "dkv.norm", (R,), where))
        a.load_expansions(_take(w, "uk", (H * D, R), where), _take(w, "uv", (H * E, R), where), like)
        self.o_proj = _param(_take(w, "o", (W, H * E), where), like)

    @staticmethod
    def shapes(W, m, rank):
        H, D, P, E, R, Q = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
        return [("dq", (Q, W)), ("dq.norm", (Q,)), ("uq", (H * (D + P), Q)), ("dkv", (R + P, W)),
                ("dkv.norm", (R,)), ("uk", (H * D, R)), ("uv", (H * E, R)), ("o", (W, H * E))]


_MIXERS = {"attention": TedenexAttentionMixer, "wkv": TedenexTimeMixer,
           "latent_attention": TedenexLatentMixer}


# ------------------------------------------------------------------ layers
class TedenexFeedForward(nn.Module):
    def __init__(self, W: int, ff: int):
        super().__init__()
        self.W, self.ff, self.act = W, ff, ReluSquared()
        self.up = nn.Parameter(torch.zeros(ff, W), requires_grad=False)
        self.down = nn.Parameter(torch.zeros(W, ff), requires_grad=False)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(self.act(F.linear(h, self.up)), self.down)


class TedenexLayer(nn.Module):
    def __init__(self, cfg: TedenexConfig, spec: TedenexLayerSpec, number: int):
        super().__init__()
        W, eps = cfg.hidden_size, cfg.rms_norm_epsilon
        self.W, self.kind = W, spec.type
        self.norm1, self.norm1b = OffsetRMSNorm(W, eps), OffsetRMSNorm(W, eps)
        self.mix = _MIXERS[spec.type](W, spec.mixer, eps, cfg.passes(number))
        self.ff = TedenexFeedForward(W, int(spec.mlp["ff"])) if spec.mlp else None
        if self.ff is not None:
            self.norm2, self.norm2b = OffsetRMSNorm(W, eps), OffsetRMSNorm(W, eps)
        self.side = LayerTokenInput(W, cfg.side_dim, number * cfg.side_dim) if cfg.side_dim else None

    def load(self, w: dict, where: str, like) -> None:
        W = self.W
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if self.ff is not None else ()):
            getattr(self, n).weight.copy_(_take(w, n, (W,), where))
        mw = {k[4:]: w.pop(k) for k in [k for k in w if k.startswith("mix.")]}
        self.mix.load(mw, where + "mix.", like)
        if mw:
            raise KeyError(f"checkpoint tensor {where}mix.{next(iter(mw))} has no parameter")
        if self.ff is not None:
            self.ff.up = _param(_take(w, "mlp.up", (self.ff.ff, W), where), like)
            self.ff.down = _param(_take(w, "mlp.down", (W, self.ff.ff), where), like)
        if self.side is not None:
            n = self.side.dim
            self.side.gate = _param(_take(w, "side.gate", (n, W), where), like)
            self.side.proj = _param(_take(w, "side.proj", (W, n), where), like)
            self.side.norm_weight.copy_(_take(w, "side.norm", (W,), where))
        if w:
            raise KeyError(f"checkpoint tensor {where}{next(iter(w))} has no parameter")


class TedenexModel(nn.Module):
    def __init__(self, cfg: TedenexConfig):
        super().__init__()
        W = cfg.hidden_size
        self.embed = nn.Embedding(cfg.vocab_size, W)
        self.embed.weight.requires_grad_(False)
        self.side_table = (nn.Parameter(torch.zeros(cfg.vocab_size, cfg.num_layers * cfg.side_dim),
                                        requires_grad=False) if cfg.side_dim else None)
        self.layers = nn.ModuleList([TedenexLayer(cfg, s, i) for i, s in enumerate(cfg.layers)])
        self.order = cfg.run_order()
        self.eps = cfg.rms_norm_epsilon
        self.act_dtype = self.embed.weight.dtype
        # observer for tests: called with (index of the layer run, fp32 stream) after every run
        self.layer_hook = None

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Returns the fp32 residual stream [T, W] after the last layer (the final norm belongs
        to the head: only the rows whose logits are wanted go through it)."""
        dt, eps, order = self.act_dtype, self.eps, self.order
        table, hook = self.embed.weight, self.layer_hook
        x = ops.embed_sum(input_ids, None, table, None)
        h = self.layers[order[0][0]].norm1(x, dt) if order else None
        for n, (i, which, _) in enumerate(order):
            L = self.layers[i]
            nxt, again = None, None
            if n + 1 < len(order):
                j, _, adds = order[n + 1]
                nxt, again = self.layers[j].norm1.weight, (input_ids, table) if adds else None
            # an observer sees the stream before the embedding joins it: the next input is formed apart
            apart = hook is not None and again is not None
            last = dict(w_next=None if apart else nxt, extra=None if apart else again)

            def update(y, w, final, **kw):
                return ops.post_norm_residual(y, w, x, eps, out_dtype=dt, **kw, **(last if final else {}))
            side = L.side is not None
            rest = dict(raw=True, w_next=None) if side else {}
            y, wb = L.mix(h, which), L.norm1b.weight
            if L.ff is not None:
                y, wb = L.ff(update(y, wb, False, w_next=L.norm2.weight)), L.norm2b.weight
            h = update(y, wb, not side, **rest)
            if side:
                h = update(L.side(h, input_ids, self.side_table), L.side.norm_weight, True, plain=True)
            if hook is not None:
                hook(n, x)
            if apart:
                x.add_(ops.embed_sum(input_ids, None, table, None))
                h = self.layers[order[n + 1][0]].norm1(x, dt)
        return x


class TedenexForCausalLM(nn.Module):
    needs_aux_rows = False
    # (a model with filters or time mixing has state, and is then not cached by prefix; the latent
    # rows of every pass are functions of the prefix alone)
    prefix_cacheable = True

    def __init__(self, config: TedenexConfig):
        super().__init__()
        self.config = config
        self.model = TedenexModel(config)
        self.lm_head = ScaledTiedHead(self.model.embed, config.rms_norm_epsilon, offset=1.0)
        self.has_recurrent_state = bool(self.state_layers())

    def forward(self, input_ids, positions=None):
        if positions is None:
            positions = get_context().positions
        return self.model(input_ids, positions)

    def compute_logits(self, hidden):
        return self.lm_head(hidden)

    def compute_local_logits(self, hidden):
        return self.lm_head.local_logits(hidden)

    # ---- what the engine needs to know about caches and state ---------------------------
    def attention_layers(self):
        """Every (layer, pass) cache holder: a looped layer owns one cache per pass."""
        return [a for l in self.model.layers for a in l.mix.attention_cores()]

    def state_layers(self):
        return [c for l in self.model.layers for c in l.mix.state_cores()]

    # ---- weights -----------------------------------------------------------------------
    @torch.no_grad()
    def load_weights(self, items) -> int:
        """``items``: iterable of (checkpoint name, tensor).  The tensors of a layer are collected
        and then stacked into its fused parameters; unknown, missing or mis-shaped tensors raise
        with their name."""
        like, side = self.model.embed.weight, self.model.side_table
        per_layer: List[dict] = [dict() for _ in self.model.layers]
        top: Dict[str, torch.Tensor] = {}
        n = 0
        for name, t in items:
            n += 1
            li, _, rest = name.partition(".")
            if li.startswith("l") and li[1:].isdigit() and int(li[1:]) < len(per_layer):
                per_layer[int(li[1:])][rest] = t
            else:
                top[name] = t
        like.copy_(_take(top, "embed", like.shape, ""))
        if side is not None:
            side.copy_(_take(top, "side.embed", side.shape, ""))
        self.lm_head.load_norm(_take(top, "final.norm", like.shape[1:], "").to(device=like.device, dtype=torch.float32))
        if top:
            raise KeyError(f"checkpoint tensor {next(iter(top))!r} has no parameter")
        for i, (layer, w) in enumerate(zip(self.model.layers, per_layer)):
            layer.load(w, f"l{i}.", like)
        return n

    def checkpoint_shapes(self, rank: int = 64):
        """(name, shape) of every tensor a checkpoint of this configuration holds; ``rank``: the
        inner size of the decay's low-rank projection (a checkpoint's own shapes decide when
        loading)."""
        c = self.config
        W = c.hidden_size
        yield "embed", (c.vocab_size, W)
        if c.side_dim:
            yield "side.embed", (c.vocab_size, c.num_layers * c.side_dim)
        for i, L in enumerate(c.layers):
            p = f"l{i}."
            for nm in ("norm1", "norm1b") + (("norm2", "norm2b") if L.mlp else ()):
                yield p + nm, (W,)
            for nm, shape in _MIXERS[L.type].shapes(W, L.mixer, rank):
                yield p + "mix." + nm, shape
            if L.mlp:
                yield p + "mlp.up", (int(L.mlp["ff"]), W)
                yield p + "mlp.down", (W, int(L.mlp["ff"]))
            if c.side_dim:
                yield p + "side.gate", (c.side_dim, W)
                yield p + "side.proj", (W, c.side_dim)
                yield p + "side.norm", (W,)
        yield "final.norm", (W,)

    def random_checkpoint(self, seed: int = 0, rank: int = 64):
        """Seeded random tensors (values exactly representable in bfloat16) of every checkpoint
        name, scaled so that activations stay O(1) through the stack."""
        g = torch.Generator().manual_seed(seed)
        out = {}
        for name, shape in self.checkpoint_shapes(rank):
            leaf = name.rsplit(".", 1)[-1]
            r = torch.randn(shape, generator=g)
            if leaf in ("norm1", "norm1b", "norm2", "norm2b") or name == "final.norm":
                t = 0.1 * r
            elif leaf == "norm":
                t = 1.0 + 0.1 * r
            elif leaf == "conv":
                t = 0.5 * r
            elif leaf == "b":
                t = 0.1 * r
            elif ".mu." in name:
                t = torch.sigmoid(r)
            elif leaf == "w0":
                t = -2.0 + r
            elif leaf == "u":
                t = 0.5 * r
            elif leaf == "embed":
                t = r
            else:
                t = r * (shape[-1] ** -0.5)
            out[name] = t.to(torch.bfloat16)
        return out

    def init_random_weights(self, seed: int = 0, std: float = 0.02) -> None:
        self.load_weights(self.random_checkpoint(seed).items())
