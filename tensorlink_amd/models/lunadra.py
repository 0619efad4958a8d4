"""Lunadra model family: a layered decoder with parallel sublayers whose
``config.json`` lists every layer. A layer has ONE norm; its mixer and its
feed-forward both read that norm's output and enter the fp32 residual
together,

    h = norm1(x);  x <- x + m * (mixer(h) + ff(h))           (ff optional)

with RMS norms (plain weights) and m a constant of the model. Mixers:

``mlstm``, ``mlstm_2``  matrix memory with exponential gates, fp32 state per
               sequence (the two names differ in sizes only);
``parallel``   windowed grouped-query attention with rotate-half positions
               beside a gated delta rule, a weighted sum of the two.

The feed-forward is a dense gated one (relu) or a mixture of experts with
identity experts, a clamped activation, scores from a softmax over all
experts, a correction that acts on the choice only, and optionally a shared
expert. The input embedding is a token embedding plus a hashed bigram
embedding; the id of a sequence's last token is part of its state.

Because everything in a layer reads the same h, a layer runs one fused
projection in the serving dtype — [mixer | feed-forward or shared expert] —
and one thin projection with fp32 results — [gates or step sizes | router].

The blocks live in :mod:`tensorlink_amd.models.mixers`; this file reads the
configuration, assembles them, maps checkpoint tensor names and runs the
stage over a flat ragged batch through the stage interface of
:class:`~tensorlink_amd.models.layered.LayeredStage`. One stage (PP = 1).
"""

from __future__ import annotations

import json
import math
import os
from dataclasses import dataclass, field
from typing import List, Optional

import torch
import torch.nn as nn

from tensorlink_amd.models.configs import ModelConfig
from tensorlink_amd.models.dense import TLLinear
from tensorlink_amd.models.layered import (LayeredStage, load_named_tensors,
                                           tensor_shapes)
from tensorlink_amd.models.mixers import (GatedDeltaMixer, GatedFF, GatedMoE,
                                          MLSTMMixer, ParallelMixer,
                                          RMSWeight, WindowAttention, _F32Cache,
                                          align_cols, pad_cols)
from tensorlink_amd.ops import mixers as mx

MIXERS = ("mlstm", "mlstm_2", "parallel")
FEED_FORWARDS = ("dense", "moe")
SWISH_ALPHA = 1.702         # of the experts' clamped swish
# ranks that are a tensor's shape, not a key of config.json: mixer key ->
# the tensor whose row count it is
RANKS = {"decay_rank": "a1", "gate_rank": "g1"}


@dataclass
class LunadraConfig(ModelConfig):
    """Flat ModelConfig fields are filled for the planner and the engine;
    ``layer_specs`` (the checkpoint's ``layers`` list) is authoritative. The
    ranks of a delta rule's low-rank projections are read from the
    checkpoint's header into its ``decay_rank`` and ``gate_rank`` (a
    configuration built by hand gives them)."""
    layer_specs: List[dict] = field(default_factory=list)
    bigram_buckets: int = 1
    bigram_mul_prev: int = 1
    bigram_mul_cur: int = 1
    residual_mult: float = 1.0
    architecture: str = "lunadra"

    @classmethod
    def from_dict(cls, cfg: dict, name: str = "lunadra") -> "LunadraConfig":
        if "layer_specs" in cfg:                     # own to_json round trip
            known = {f.name for f in cls.__dataclass_fields__.values()}
            return cls(**{k: v for k, v in cfg.items() if k in known})
        layers = json.loads(json.dumps(cfg["layers"]))       # own copy
        shapes = None
        for i, lc in enumerate(layers):
            if lc["type"] not in MIXERS:
                raise KeyError(f"layer {i}: unknown mixer {lc['type']!r}")
            cls._check_ff(i, lc.get("mlp"))
            if lc["type"] != "parallel":
                continue
            for side in ("left", "right"):
                if lc["mixer"][side]["heads"] % lc["mixer"][side]["kv_heads"]:
                    raise KeyError(f"layer {i}: heads must be a multiple of "
                                   "kv_heads")
            rot = lc["mixer"]["left"].get("rot")
            if rot and (rot["dims"] % 2
                        or rot["dims"] > lc["mixer"]["left"]["dim"]):
                raise KeyError(f"layer {i}: rot.dims must be even and at "
                               "most dim")
            for rank, tensor in RANKS.items():
                if rank in lc["mixer"]["right"]:
                    continue
                if shapes is None:
                    shapes = tensor_shapes(name)
                key = f"l{i}.mix.right.{tensor}"
                if key not in shapes:
                    raise KeyError(f"layer {i}: {rank} is neither configured "
                                   "nor in a checkpoint")
                lc["mixer"]["right"][rank] = int(shapes[key][0])
        att = [lc["mixer"].get("left", lc["mixer"]) for lc in layers]
        big = cfg["embedding"]["bigram"]
        return cls(
            name=name, vocab_size=cfg["vocab"], hidden_size=cfg["width"],
            intermediate_size=max(
                (cls._ff_width(lc["mlp"]) for lc in layers
                 if lc.get("mlp") is not None), default=cfg["width"]),
            num_hidden_layers=len(layers),
            num_attention_heads=max(m["heads"] for m in att),
            num_key_value_heads=max(m.get("kv_heads", 1) for m in att),
            head_dim=max(m["dim"] for m in att),
            rms_norm_eps=cfg["norm"]["eps"], tie_word_embeddings=False,
            layer_specs=layers, bigram_buckets=int(big["buckets"]),
            bigram_mul_prev=int(big["mul_prev"]),
            bigram_mul_cur=int(big["mul_cur"]),
            residual_mult=float(cfg["residual_mult"]))

    @staticmethod
    def _check_ff(i: int, mlp: Optional[dict]) -> None:
        if mlp is None:
            return
        if mlp.get("kind") not in FEED_FORWARDS:
            raise KeyError(f"layer {i}: unknown feed-forward "
                           f"{mlp.get('kind')!r}")
        if mlp["kind"] == "moe":
            r = mlp["router"]
            if not 1 <= r["top"] <= r["experts"] + r.get("identity", 0):
                raise KeyError(f"layer {i}: need 1 <= top <= experts + "
                               "identity")

    @staticmethod
    def _ff_width(mlp: dict) -> int:
        if mlp["kind"] == "dense":
            return mlp["ff"]
        return (mlp["router"]["experts"] * mlp["expert"]["ff"]
                + (mlp.get("shared") or {"ff": 0})["ff"])

    def param_count(self, include_embeddings: bool = True) -> int:
        w = self.hidden_size
        total = w
        for lc in self.layer_specs:
            mc, mlp = lc["mixer"], lc.get("mlp")
            total += w
            if lc["type"] == "parallel":
                L, R = mc["left"], mc["right"]
                total += w * (L["heads"] * L["dim"] + L["kv_heads"]
                              * (L["dim"] + L["vdim"])
                              + L["heads"] * L["vdim"])
                cc = 2 * R["kv_heads"] * R["dim"] + R["heads"] * R["vdim"]
                hd, hv = R["heads"] * R["dim"], R["heads"] * R["vdim"]
                total += cc * (w + R["conv"]) + R["heads"] * (w + 1) \
                    + R["decay_rank"] * (w + hd) + hd \
                    + R["gate_rank"] * (w + hv) + R["vdim"] + hv * w
            else:
                H, D, V = mc["heads"], mc["dim"], mc["vdim"]
                total += w * (2 * H * D + 3 * H * V) + H * V \
                    + 2 * H * (w + 1)
            if mlp is None:
                continue
            if mlp["kind"] == "dense":
                total += 3 * w * mlp["ff"]
            else:
                r = mlp["router"]
                total += (r["experts"] + r.get("identity", 0)) * (w + 1) \
                    + 3 * r["experts"] * w * mlp["expert"]["ff"]
                if mlp.get("shared"):
                    total += 3 * w * mlp["shared"]["ff"]
        if include_embeddings:
            total += (2 * self.vocab_size + self.bigram_buckets + 1) * w
        return total


def build_mixer(lc: dict, width: int, eps: float) -> nn.Module:
    mc = lc["mixer"]
    if lc["type"] != "parallel":
        return MLSTMMixer(width, mc["heads"], mc["dim"], mc["vdim"],
                          mc["gate_cap"], eps, hosted=True)
    L, R = mc["left"], mc["right"]
    rot = L.get("rot") or {"dims": 0, "base": 1.0}
    left = WindowAttention(width, L["heads"], L["kv_heads"], L["dim"],
                           L["vdim"], L["scale"], rot["dims"], rot["base"],
                           (L.get("mask") or {"size": 0})["size"], eps,
                           sink=False, talk=False, qk_norm=False, hosted=True)
    right = GatedDeltaMixer(width, R["heads"], R["kv_heads"], R["dim"],
                            R["vdim"], R["conv"], R["decay_rank"],
                            R["gate_rank"], eps)
    return ParallelMixer(width, left, right, hosted=True,
                         scales=(mc["left_scale"], mc["right_scale"]))


def build_ff(mlp: dict, width: int) -> nn.Module:
    if mlp["kind"] == "dense":
        return GatedFF(width, mlp["ff"], act="relu", hosted=True)
    r, shared = mlp["router"], mlp.get("shared") or {"ff": 0, "limit": 0.0}
    return GatedMoE(width, mlp["expert"]["ff"], r["experts"], r["top"],
                    shared["ff"], scores=True, hosted=True,
                    identity=r.get("identity", 0), shared_gate=False,
                    act=("clamped_swish", mlp["expert"]["limit"],
                         SWISH_ALPHA),
                    shared_act=("clamped_swish", shared["limit"],
                                SWISH_ALPHA))


class LunadraLayer(nn.Module, _F32Cache):
    """Norm, the two fused input projections, mixer, feed-forward."""

    def __init__(self, config: LunadraConfig, idx: int):
        super().__init__()
        lc = config.layer_specs[idx]
        w, eps = config.hidden_size, config.rms_norm_eps
        self.mult = config.residual_mult
        self.norm1 = RMSWeight(w, one_plus=False)
        self.mix = build_mixer(lc, w, eps)
        self.mlp = (build_ff(lc["mlp"], w)
                    if lc.get("mlp") is not None else None)
        # columns of the fused projection [mixer | ff]
        self.ff_col = align_cols(self.mix.in_cols)
        ff_in = self.mlp.in_cols if self.mlp is not None else 0
        self.proj = TLLinear(w, pad_cols(self.ff_col + ff_in), bias=False)
        # fp32 columns [mixer | router]
        self.router_col = self.mix.thin_cols
        thin = self.router_col + (self.mlp.thin_cols
                                  if self.mlp is not None else 0)
        self.thin = nn.Parameter(torch.zeros((thin + 15) // 16 * 16, w))
        self.thin_b = nn.Parameter(torch.zeros(self.thin.shape[0])) \
            if self.mix.kind == "mlstm" else None

    def forward(self, h, meta, cache, run: int):
        """The layer's terms of the residual sum, [(tensor, factor), ...],
        from its normed input h."""
        p = self.proj(h)
        t = mx.thin_linear(h, self.thin, self._f32("thin_b")
                           if self.thin_b is not None else None)
        m = self.mult
        if self.mix.kind == "mlstm":
            terms = [(self.mix(p, meta, cache, run, 0, t), m)]
        else:
            a, b = self.mix(p, meta, cache.k[run], cache.v[run],
                            cache.state[run], 0, t)
            ls, rs = self.mix.scales
            terms = [(a, m * ls), (b, m * rs)]
        if self.mlp is None:
            return terms
        if self.mlp.kind == "dense":
            y = self.mlp(p, self.ff_col)
        else:
            y = self.mlp(h, p, self.ff_col, t, self.router_col)
        return terms + [(y, m)]


class LunadraStageModel(LayeredStage):
    """Whole-model stage (embedding, every layer, final norm + head)."""

    def __init__(self, config: LunadraConfig, layer_start: int,
                 layer_end: int, has_embedding: bool, has_head: bool):
        super().__init__()
        if not (has_embedding and has_head and layer_start == 0
                and layer_end == config.num_hidden_layers):
            raise ValueError("the Lunadra family runs as a single stage "
                             "(fp32 residual); use world=1")
        self.config = config
        self.layer_start, self.layer_end = layer_start, layer_end
        self.has_embedding = self.has_head = True
        w = config.hidden_size
        self.embed_tokens = nn.Embedding(config.vocab_size, w)
        self.bigram = nn.Parameter(torch.zeros(config.bigram_buckets + 1, w))
        self.layers = nn.ModuleList([LunadraLayer(config, i)
                                     for i in range(config.num_hidden_layers)])
        self.norm = RMSWeight(w, one_plus=False)
        self.lm_head = TLLinear(w, config.vocab_size, bias=False)
        self.layer_sums = None      # list -> residual after every layer

    def cache_specs(self):
        """One entry per layer, then the last token of every sequence."""
        return super().cache_specs() + [{"kind": "last_token"}]

    def head(self, hidden: torch.Tensor) -> torch.Tensor:
        """Final norm and vocabulary projection of residual rows [..., W]
        (fp32); fp32 logits."""
        shape = hidden.shape
        x = hidden.reshape(-1, shape[-1]).float()
        h = mx.rms_scale(x, self.norm.w32(), self.config.rms_norm_eps, False,
                         out_dtype=self.lm_head.weight.dtype)
        return self.lm_head(h).float().reshape(*shape[:-1], -1)

    @torch.no_grad()
    def forward(self, hidden_or_ids, positions, kv_cache=None,
                training: bool = False, return_logits: bool = True):
        if training:
            raise NotImplementedError(
                "the Lunadra family is served, not trained, by this build")
        B, S = hidden_or_ids.shape[:2]
        dev = hidden_or_ids.device
        dtype = self.lm_head.weight.dtype
        cfg = self.config
        eps = cfg.rms_norm_eps
        if kv_cache is None:
            kv_cache = self.make_kv_cache(B, int(positions.max()) + 1, dev,
                                          dtype)
        meta = self._meta(kv_cache, positions, B, S)
        (last,) = kv_cache.state[-1]
        X = mx.bigram_embed(hidden_or_ids, self.embed_tokens.weight,
                            self.bigram, last, meta, cfg.bigram_mul_prev,
                            cfg.bigram_mul_cur)
        # a layer's terms are added by the NEXT layer's norm
        terms = []
        for i, layer in enumerate(self.layers):
            h = self._add(X, terms, layer.norm1.w32(), eps, dtype)
            terms = layer(h, meta, kv_cache, i)
        self._add(X, terms, None, eps, dtype)
        kv_cache.advance(S)
        u = X.view(B, S, -1)
        return self.head(u) if return_logits else u

    def _add(self, X, terms, w, eps, dtype):
        y, s = terms[0] if terms else (None, 1.0)
        h = mx.add_rms(X, y, w, eps, dtype, y_scale=s, more=terms[1:])
        if terms and self.layer_sums is not None:
            self.layer_sums.append(X.clone())
        return h


# ------------------------------------------------------------------ weights
def _name_map(stage: LunadraStageModel):
    """(checkpoint tensor name -> (parameter, row offset or expert index
    [, row offset inside the expert])), parameters, and the parameters that
    a checkpoint fills only in part (fused projections are padded with zero
    rows, thin ones biased only where the design has a bias)."""
    P = dict(stage.named_parameters())
    w = stage.config.hidden_size
    m = {"embed": ("embed_tokens.weight", 0), "bigram": ("bigram", 0),
         "head": ("lm_head.weight", 0), "final.norm": ("norm.weight", 0)}
    partial = {}
    for i, layer in enumerate(stage.layers):
        a, b = f"l{i}.", f"layers.{i}."
        m[f"{a}norm1"] = (f"{b}norm1.weight", 0)
        rows, thin, biased = [], [], 0
        mix, x, y = layer.mix, f"{a}mix.", f"{b}mix."
        if mix.kind == "mlstm":
            H, hd, hv = mix.H, mix.H * mix.D, mix.H * mix.V
            rows += [(f"{x}{n}", c, k) for n, c, k in zip(
                "qkvg", mix.offs, (hd, hd, hv, hv))]
            thin += [(f"{x}i", 0, H), (f"{x}f", H, H)]
            m[f"{x}i.b"] = (f"{b}thin_b", 0)
            m[f"{x}f.b"] = (f"{b}thin_b", H)
            partial[f"{b}thin_b"] = 2 * H
            m[f"{x}norm"] = (f"{y}norm", 0)
            m[f"{x}o"] = (f"{y}o_proj.weight", 0)
        else:
            L, R, c = mix.left, mix.right, mix.right_col
            rows += [(f"{x}left.q", 0, L.q_cols),
                     (f"{x}left.k", L.q_cols, L.k_cols),
                     (f"{x}left.v", L.q_cols + L.k_cols, L.v_cols)]
            m[f"{x}left.o"] = (f"{y}left.o_proj.weight", 0)
            qk, hv = R.G * R.D, R.H * R.V
            for n, off, k in zip("qkv", R.offs, (qk, qk, hv)):
                rows.append((f"{x}right.{n}", c + off, k))
                m[f"{x}right.{n}.conv"] = (f"{y}right.conv", off)
            rows += [(f"{x}right.a1", c + R.a_col, R.R),
                     (f"{x}right.g1", c + R.g_col, R.GR)]
            thin.append((f"{x}right.b", 0, R.H))
            for n in ("A_log", "a2", "dt_bias", "g2", "norm"):
                m[f"{x}right.{n}"] = (f"{y}right.{n}", 0)
            m[f"{x}right.o"] = (f"{y}right.o_proj.weight", 0)
        mlp, x, y = layer.mlp, f"{a}mlp.", f"{b}mlp."
        c = layer.ff_col
        if mlp is not None and mlp.kind == "dense":
            rows += [(f"{x}gate", c, mlp.ff), (f"{x}up", c + mlp.ff, mlp.ff)]
            m[f"{x}down"] = (f"{y}down.weight", 0)
        elif mlp is not None:
            if mlp.sff:
                rows += [(f"{x}shared.gate", c, mlp.sff),
                         (f"{x}shared.up", c + mlp.sff, mlp.sff)]
                m[f"{x}shared.down"] = (f"{y}shared_down.weight", 0)
            thin.append((f"{x}router", layer.router_col, mlp.thin_cols))
            m[f"{x}correction"] = (f"{y}correction", 0)
            for e in range(mlp.E):
                m[f"{x}e{e}.gate"] = (f"{y}gate_up", e, 0)
                m[f"{x}e{e}.up"] = (f"{y}gate_up", e, mlp.ff)
                m[f"{x}e{e}.down"] = (f"{y}down", e, 0)
        for param, parts in ((f"{b}proj.weight", rows), (f"{b}thin", thin)):
            for name, row, _ in parts:
                m[name] = (param, row)
            partial[param] = w * sum(n for _, _, n in parts)
    return m, P, partial


@torch.no_grad()
def load_lunadra_weights(stage: LunadraStageModel, ckpt_dir: str,
                         dtype=torch.bfloat16) -> int:
    """Fill the stage from ``model.safetensors``; every tensor of the
    checkpoint must be consumed and every parameter filled (padding rows and
    rows without a bias stay zero)."""
    names, P, partial = _name_map(stage)
    for k in partial:
        P[k].zero_()
    return load_named_tensors(P, names, ckpt_dir, partial=partial)


@torch.no_grad()
def init_lunadra_random(stage: LunadraStageModel, seed: int = 0) -> None:
    """Scaled-normal matrices, norm weights near one, taps near a delta on
    the current token, open forget gates, decays in the usual range: finite
    activations at any depth for benchmarks and tests."""
    g = torch.Generator().manual_seed(seed)
    for name, p in stage.named_parameters():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.empty(p.shape, dtype=torch.float32)
        if leaf == "norm" or ".norm" in name or name == "norm.weight":
            t = 1.0 + 0.1 * torch.randn(p.shape, generator=g)
        elif leaf == "conv":
            t = 0.3 * torch.randn(p.shape, generator=g)
            t[:, -1] += 1.0
        elif leaf == "thin_b":
            t = 1.0 + torch.randn(p.shape, generator=g)
        elif leaf == "dt_bias":
            t = torch.rand(p.shape, generator=g) * 3.0 - 4.0
        elif leaf == "A_log":
            t = torch.log(1.0 + 7.0 * torch.rand(p.shape, generator=g))
        elif leaf == "correction":
            t = 0.02 * torch.randn(p.shape, generator=g)
        elif name in ("embed_tokens.weight", "bigram"):
            t.normal_(0.0, 1.0, generator=g)
        else:
            t.normal_(0.0, 1.0 / math.sqrt(p.shape[-1]), generator=g)
        p.copy_(t.to(p.dtype))


def read_config(path: str) -> Optional[LunadraConfig]:
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    if cfg.get("architecture") in ("Lunadra", "lunadra"):
        return LunadraConfig.from_dict(cfg, name=path)
    return None
