"""Mogisun model family: a pre-norm layered decoder whose ``config.json``
lists every layer. Each sublayer's result is added through an element-wise
sigmoid gate that reads the sublayer's own input,

    h = norm1(x);  x <- x + sigmoid(R1 h + r1) * mixer(h)
    h = norm2(x);  x <- x + sigmoid(R2 h + r2) * ff(h)        (ff optional)

with RMS norms (plain weights) and an fp32 residual. Two mixers:

``gla``        gated linear attention, one decay per key channel and token,
               fp32 state per sequence;
``attention``  position-free grouped-query attention over the paged pool:
               biased projections, unit-RMS queries and keys, a query
               temperature that grows with the position, one output gate per
               head.

The feed-forward is a dense SwiGLU or a mixture of them with a shared
expert. A span of layers may run several times in a row with the same
weights (``loop``); every pass has its own pages and state and starts with
x <- W_in [x; x0], x0 the token embedding. Logits are scaled and
soft-capped.

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
from typing import List, Optional, Tuple

import torch
import torch.nn as nn

from tensorlink_amd.models.configs import ModelConfig
from tensorlink_amd.models.dense import TLLinear
from tensorlink_amd.models.layered import (LayeredStage, load_named_tensors,
                                           looped_runs, read_loop,
                                           tensor_shapes)
from tensorlink_amd.models.mixers import (GatedFF, GatedLinearAttention,
                                          GatedMoE, RMSWeight,
                                          WindowAttention)
from tensorlink_amd.ops import mixers as mx

MIXERS = ("gla", "attention")
FEED_FORWARDS = ("dense", "moe")


@dataclass
class MogisunConfig(ModelConfig):
    """Flat ModelConfig fields are filled for the planner and the engine;
    ``layer_specs`` (the checkpoint's ``layers`` list) is authoritative.
    The rank of a ``gla`` layer's decay projection is no key of config.json:
    it is a tensor's shape, read from the checkpoint's header into the
    mixer's ``decay_rank`` (a configuration built by hand gives it)."""
    layer_specs: List[dict] = field(default_factory=list)
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 0                 # 0 = no looped span
    logit_scale: float = 1.0
    logit_softcap: float = 0.0          # 0 = none
    architecture: str = "mogisun"

    @classmethod
    def from_dict(cls, cfg: dict, name: str = "mogisun") -> "MogisunConfig":
        if "layer_specs" in cfg:                     # own to_json round trip
            known = {f.name for f in cls.__dataclass_fields__.values()}
            return cls(**{k: v for k, v in cfg.items() if k in known})
        layers = json.loads(json.dumps(cfg["layers"]))       # own copy
        shapes = None
        for i, lc in enumerate(layers):
            if lc["type"] not in MIXERS:
                raise KeyError(f"layer {i}: unknown mixer {lc['type']!r}")
            mlp, mc = lc.get("mlp"), lc["mixer"]
            if mlp is not None and mlp.get("kind") not in FEED_FORWARDS:
                raise KeyError(f"layer {i}: unknown feed-forward "
                               f"{mlp.get('kind')!r}")
            if mlp is not None and mlp["kind"] == "moe" and not (
                    1 <= mlp["router"]["top"] <= mlp["router"]["experts"]):
                raise KeyError(f"layer {i}: need 1 <= top <= experts")
            if lc["type"] == "attention":
                if mc["heads"] % mc["kv_heads"]:
                    raise KeyError(f"layer {i}: heads must be a multiple of "
                                   "kv_heads")
            elif "decay_rank" not in mc:
                if shapes is None:
                    shapes = tensor_shapes(name)
                key = f"l{i}.mix.a1"
                if key not in shapes:
                    raise KeyError(f"layer {i}: the decay projection's rank "
                                   "is neither configured nor in a "
                                   "checkpoint")
                mc["decay_rank"] = int(shapes[key][0])
        start, stop, times = read_loop(cfg, len(layers))
        inter = max((cls._ff_width(lc["mlp"]) for lc in layers
                     if lc.get("mlp") is not None), default=cfg["width"])
        return cls(
            name=name, vocab_size=cfg["vocab"], hidden_size=cfg["width"],
            intermediate_size=inter, num_hidden_layers=len(layers),
            num_attention_heads=max(lc["mixer"]["heads"] for lc in layers),
            num_key_value_heads=max(lc["mixer"].get("kv_heads", 1)
                                    for lc in layers),
            head_dim=max(lc["mixer"]["dim"] for lc in layers),
            rms_norm_eps=cfg["norm"]["eps"], tie_word_embeddings=False,
            layer_specs=layers, loop_start=start, loop_stop=stop,
            loop_times=times,
            logit_scale=float(cfg.get("logit_scale", 1.0)),
            logit_softcap=float(cfg.get("logit_softcap") or 0.0))

    @staticmethod
    def _ff_width(mlp: dict) -> int:
        if mlp["kind"] == "dense":
            return mlp["ff"]
        return (mlp["router"]["experts"] * mlp["expert"]["ff"]
                + (mlp.get("shared") or {"ff": 0})["ff"])

    def layer_runs(self) -> List[Tuple[int, Optional[int]]]:
        """(layer index, pass number or None) in execution order; every
        run has its own cache entry."""
        return looped_runs(len(self.layer_specs), self.loop_start,
                           self.loop_stop, self.loop_times)

    def param_count(self, include_embeddings: bool = True) -> int:
        w = self.hidden_size
        total = w + (2 * w * w if self.loop_times else 0)
        for lc in self.layer_specs:
            mc, mlp = lc["mixer"], lc.get("mlp")
            H, D, V = mc["heads"], mc["dim"], mc["vdim"]
            total += w + w * (w + 1)                     # norm1, rg1
            if lc["type"] == "gla":
                R = mc["decay_rank"]
                total += w * (2 * H * D + 2 * H * V + R) + H * D * (R + 1) \
                    + V + H * V * w
            else:
                G = mc["kv_heads"]
                total += (w + 1) * (H * D + G * D + G * V) + w * H \
                    + (H * V + 1) * w
            if mlp is None:
                continue
            total += w + w * (w + 1)                     # norm2, rg2
            if mlp["kind"] == "dense":
                total += 3 * w * mlp["ff"]
            else:
                E = mlp["router"]["experts"]
                total += E * w + 3 * E * w * mlp["expert"]["ff"]
                if mlp.get("shared"):
                    total += 3 * w * mlp["shared"]["ff"] + w
        if include_embeddings:
            total += 2 * self.vocab_size * w
        return total


def build_mixer(lc: dict, width: int, eps: float,
                side_cols: int = 0) -> nn.Module:
    mc = lc["mixer"]
    if lc["type"] == "gla":
        return GatedLinearAttention(width, mc["heads"], mc["dim"], mc["vdim"],
                                    mc["decay_rank"], mc["tau"], eps,
                                    side_cols=side_cols)
    qt = mc.get("q_temp")
    return WindowAttention(width, mc["heads"], mc["kv_heads"], mc["dim"],
                           mc["vdim"], mc["scale"], 0, 1.0, 0, eps,
                           sink=False, talk=False, qk_norm=False,
                           unit_norm=True, head_gate=True, bias=True,
                           q_temp=(qt["coef"], qt["every"]) if qt else None,
                           side_cols=side_cols)


def build_ff(mlp: dict, width: int, side_cols: int = 0) -> nn.Module:
    if mlp["kind"] == "dense":
        return GatedFF(width, mlp["ff"], act="silu", side_cols=side_cols)
    return GatedMoE(width, mlp["expert"]["ff"], mlp["router"]["experts"],
                    mlp["router"]["top"],
                    (mlp.get("shared") or {"ff": 0})["ff"],
                    side_cols=side_cols)


class MogisunLayer(nn.Module):
    """Every sublayer's fused input projection also holds the rows of its
    residual gate, which reads the same input."""

    def __init__(self, config: MogisunConfig, idx: int):
        super().__init__()
        lc = config.layer_specs[idx]
        w, eps = config.hidden_size, config.rms_norm_eps
        self.norm1 = RMSWeight(w, one_plus=False)
        self.mix = build_mixer(lc, w, eps, side_cols=w)
        self.mlp = None
        if lc.get("mlp") is not None:
            self.norm2 = RMSWeight(w, one_plus=False)
            self.mlp = build_ff(lc["mlp"], w, side_cols=w)


class MogisunStageModel(LayeredStage):
    """Whole-model stage (embedding, every layer run, final norm + head)."""

    def __init__(self, config: MogisunConfig, layer_start: int,
                 layer_end: int, has_embedding: bool, has_head: bool):
        super().__init__()
        if not (has_embedding and has_head and layer_start == 0
                and layer_end == config.num_hidden_layers):
            raise ValueError("the Mogisun family runs as a single stage "
                             "(fp32 residual); use world=1")
        self.config = config
        self.layer_start, self.layer_end = layer_start, layer_end
        self.has_embedding = self.has_head = True
        w = config.hidden_size
        self.embed_tokens = nn.Embedding(config.vocab_size, w)
        self.layers = nn.ModuleList([MogisunLayer(config, i)
                                     for i in range(config.num_hidden_layers)])
        self.loop_in = (nn.Parameter(torch.zeros(w, 2 * w))
                        if config.loop_times else None)
        self.norm = RMSWeight(w, one_plus=False)
        self.lm_head = TLLinear(w, config.vocab_size, bias=False)
        self.runs = config.layer_runs()
        self.layer_sums = None      # list -> residual after every layer run

    def cache_specs(self):
        """One cache entry per layer RUN: a looped layer's passes do not
        share pages or state."""
        return [self.layers[i].mix.cache_spec() for i, _ in self.runs]

    def head(self, hidden: torch.Tensor) -> torch.Tensor:
        """Final norm, vocabulary projection, scale and soft cap of
        residual rows [..., W] (fp32); fp32 logits."""
        shape, cfg = hidden.shape, self.config
        x = hidden.reshape(-1, shape[-1]).float()
        h = mx.rms_scale(x, self.norm.w32(), cfg.rms_norm_eps, False,
                         out_dtype=self.lm_head.weight.dtype)
        z = self.lm_head(h).float()
        if cfg.logit_softcap or cfg.logit_scale != 1.0:
            z = mx.soft_cap_(z, cfg.logit_softcap, cfg.logit_scale)
        return z.reshape(*shape[:-1], -1)

    @torch.no_grad()
    def forward(self, hidden_or_ids, positions, kv_cache=None,
                training: bool = False, return_logits: bool = True):
        if training:
            raise NotImplementedError(
                "the Mogisun family is served, not trained, by this build")
        B, S = hidden_or_ids.shape[:2]
        dev = hidden_or_ids.device
        dtype = self.lm_head.weight.dtype
        cfg = self.config
        eps = cfg.rms_norm_eps
        if kv_cache is None:
            kv_cache = self.make_kv_cache(B, int(positions.max()) + 1, dev,
                                          dtype)
        meta = self._meta(kv_cache, positions, B, S)
        x0 = self.embed_tokens(hidden_or_ids.reshape(-1))
        X = x0.float().clone()
        # a sublayer's gated output is added by the NEXT sublayer's norm:
        # (output, the projection that holds its gate, the gate's column)
        y, proj, col = None, None, 0
        x0_part = None
        for run, (li, t) in enumerate(self.runs):
            layer = self.layers[li]
            if t is not None and li == cfg.loop_start:
                if y is not None:
                    mx.add_rms(X, y, None, eps, dtype, gate=proj,
                               gate_col=col)
                    self._note(X)
                    y = proj = None
                X, x0_part = mx.pair_linear(X, x0, self.loop_in, x0_part)
            h = mx.add_rms(X, y, layer.norm1.w32(), eps, dtype, gate=proj,
                           gate_col=col)
            if y is not None:
                self._note(X)
            y, proj, col = layer.mix(h, meta, kv_cache, run)
            if layer.mlp is not None:
                h = mx.add_rms(X, y, layer.norm2.w32(), eps, dtype,
                               gate=proj, gate_col=col)
                y, proj, col = layer.mlp(h)
        if y is not None:
            mx.add_rms(X, y, None, eps, dtype, gate=proj, gate_col=col)
            self._note(X)
        if kv_cache is not None:
            kv_cache.advance(S)
        u = X.view(B, S, -1)
        return self.head(u) if return_logits else u

    def _note(self, X: torch.Tensor) -> None:
        if self.layer_sums is not None:
            self.layer_sums.append(X.clone())


# ------------------------------------------------------------------ weights
def _name_map(stage: MogisunStageModel):
    """(checkpoint tensor name -> (parameter, row offset or expert index
    [, row offset inside the expert])), parameters, and the parameters that
    a checkpoint fills only in part: fused projections are padded with zero
    rows and biased only where the design has a bias."""
    P = dict(stage.named_parameters())
    partial = {}
    m = {"embed": ("embed_tokens.weight", 0), "head": ("lm_head.weight", 0),
         "final.norm": ("norm.weight", 0)}
    if stage.loop_in is not None:
        m["loop.in"] = ("loop_in", 0)
    w = stage.config.hidden_size

    def fused(mod, parts, biased):
        """Rows of a padded fused projection: (tensor, first row, rows);
        the names in ``biased`` have a bias row range too."""
        for nm, row, n in parts:
            m[nm] = (f"{mod}.weight", row)
            if nm in biased:
                m[nm + ".b"] = (f"{mod}.bias", row)
        partial[f"{mod}.weight"] = w * sum(n for _, _, n in parts)
        partial[f"{mod}.bias"] = sum(n for nm, _, n in parts if nm in biased)

    for i, layer in enumerate(stage.layers):
        a, b = f"l{i}.", f"layers.{i}."
        m[f"{a}norm1"] = (f"{b}norm1.weight", 0)
        mix, x = layer.mix, f"{a}mix."
        if mix.kind == "gla":
            hd, hv = mix.H * mix.D, mix.H * mix.V
            fused(f"{b}mix.proj", [
                (f"{x}q", mix.offs[0], hd), (f"{x}k", mix.offs[1], hd),
                (f"{x}v", mix.offs[2], hv), (f"{x}g", mix.g_col, hv),
                (f"{a}rg1", mix.side_col, w), (f"{x}a1", mix.a_col, mix.R)],
                {f"{a}rg1"})
            m[f"{x}a2"] = (f"{b}mix.a2", 0)
            m[f"{x}a2.b"] = (f"{b}mix.a2_b", 0)
            m[f"{x}norm"] = (f"{b}mix.norm", 0)
        else:
            fused(f"{b}mix.qkv", [
                (f"{x}q", 0, mix.q_cols), (f"{x}k", mix.q_cols, mix.k_cols),
                (f"{x}v", mix.q_cols + mix.k_cols, mix.v_cols),
                (f"{a}rg1", mix.side_col, w),
                (f"{x}g", mix.g_col, mix.g_cols)],
                {f"{x}q", f"{x}k", f"{x}v", f"{a}rg1"})
            m[f"{x}o.b"] = (f"{b}mix.o_proj.bias", 0)
        m[f"{x}o"] = (f"{b}mix.o_proj.weight", 0)
        mlp, x = layer.mlp, f"{a}mlp."
        if mlp is None:
            continue
        m[f"{a}norm2"] = (f"{b}norm2.weight", 0)
        if mlp.kind == "dense":
            fused(f"{b}mlp.gate_up", [
                (f"{x}gate", 0, mlp.ff), (f"{x}up", mlp.ff, mlp.ff),
                (f"{a}rg2", mlp.side_col, w)], {f"{a}rg2"})
            m[f"{x}down"] = (f"{b}mlp.down.weight", 0)
            continue
        parts = [(f"{a}rg2", mlp.side_col, w)]
        if mlp.sff:
            parts += [(f"{x}shared.gate", 0, mlp.sff),
                      (f"{x}shared.up", mlp.sff, mlp.sff),
                      (f"{x}shared.sg", mlp.sg_col, 1)]
            m[f"{x}shared.down"] = (f"{b}mlp.shared_down.weight", 0)
        fused(f"{b}mlp.dense", parts, {f"{a}rg2"})
        m[f"{x}router"] = (f"{b}mlp.router", 0)
        for e in range(mlp.E):
            m[f"{x}e{e}.gate"] = (f"{b}mlp.gate_up", e, 0)
            m[f"{x}e{e}.up"] = (f"{b}mlp.gate_up", e, mlp.ff)
            m[f"{x}e{e}.down"] = (f"{b}mlp.down", e, 0)
    return m, P, partial


@torch.no_grad()
def load_mogisun_weights(stage: MogisunStageModel, ckpt_dir: str,
                         dtype=torch.bfloat16) -> int:
    """Fill the stage from ``model.safetensors``; every tensor of the
    checkpoint must be consumed and every parameter filled (padding rows and
    rows without a bias stay zero)."""
    names, P, partial = _name_map(stage)
    for k in partial:
        P[k].zero_()
    return load_named_tensors(P, names, ckpt_dir, partial=partial)


@torch.no_grad()
def init_mogisun_random(stage: MogisunStageModel, seed: int = 0) -> None:
    """Scaled-normal matrices, norm weights near one, small biases, decays
    in the usual range: finite activations at any depth for benchmarks and
    tests."""
    g = torch.Generator().manual_seed(seed)
    for name, p in stage.named_parameters():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.empty(p.shape, dtype=torch.float32)
        if ".norm" in name or name == "norm.weight":
            t = 1.0 + 0.1 * torch.randn(p.shape, generator=g)
        elif leaf == "a2_b":
            t = 1.0 + torch.randn(p.shape, generator=g)
        elif leaf == "bias":
            t = 0.2 * torch.randn(p.shape, generator=g)
        elif name == "embed_tokens.weight":
            t.normal_(0.0, 1.0, generator=g)
        else:
            t.normal_(0.0, 1.0 / math.sqrt(p.shape[-1]), generator=g)
        p.copy_(t.to(p.dtype))


def read_config(path: str) -> Optional[MogisunConfig]:
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    if cfg.get("architecture") in ("Mogisun", "mogisun"):
        return MogisunConfig.from_dict(cfg, name=path)
    return None
