"""Lunadra family against the plain oracle (tests/lunadra_oracle.py).

Every test builds its own small configuration and random checkpoint,
loads it through the framework's registry and loader, and drives the
framework's stage, cache and batcher. The same bodies run on the CPU tier
(torch ops) and, marked ``gpu``, on the HIP kernels in fp32 and bf16.
"""

import json
import math
import os
import random

import numpy as np
import pytest
import torch

import lunadra_oracle as O
from tensorlink_amd.engine.batcher import ContinuousBatcher
from tensorlink_amd.models.paged import PAGE, HybridSlotCache
from tensorlink_amd.ops import mixers as mx
from tensorlink_amd.parallel.pipeline import PipelineRunner, SamplingParams
from tensorlink_amd.parallel.planner import plan_for_world

CPU32 = pytest.param("cpu", torch.float32, id="cpu-f32")
GPU32 = pytest.param("cuda", torch.float32, id="gpu-f32",
                     marks=pytest.mark.gpu)
GPU16 = pytest.param("cuda", torch.bfloat16, id="gpu-bf16",
                     marks=pytest.mark.gpu)
ALL = [CPU32, GPU32, GPU16]


def tol(dtype):
    return 3e-4 if dtype == torch.float32 else 8e-2


# ------------------------------------------------------------ fixtures
def ml(heads, dim, vdim, cap=15.0, name="mlstm"):
    return {"type": name, "mixer": {"heads": heads, "dim": dim,
                                    "vdim": vdim, "gate_cap": cap}}


def win(heads, kv, dim, vdim, rot, size, base=10000.0, scale=None):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "scale": 2.0 * dim ** -0.5 if scale is None else scale,
            "rot": {"dims": rot, "base": base}, "mask": {"size": size}}


def delta(heads, kv, dim, vdim, conv=4, ra=6, rg=5):
    """``decay_rank`` and ``gate_rank`` are tensors' shapes and live in the
    checkpoint, not in config.json (see file_config)."""
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "conv": conv, "decay_rank": ra, "gate_rank": rg}


def par(left, right, ls=0.7, rs=0.4):
    return {"type": "parallel", "mixer": {
        "left": left, "right": right, "left_scale": ls, "right_scale": rs}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, identity=1, limit=1.2, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
         "router": {"experts": experts, "top": top, "identity": identity}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def model_cfg(layers, vocab, width, mult=0.6, buckets=101, mp=31, mc=7,
              eps=1e-5):
    return {"architecture": "Lunadra", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "residual_mult": mult, "layers": layers,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mp,
                                     "mul_cur": mc}}}


def cfg_mixed():
    """Every mixer and feed-forward, one layer without any, key groups on
    both sides of a pair, partial rotation, vdim != dim."""
    return model_cfg([
        layer(ml(3, 8, 20), moe(5, 2, 24, 2, shared=(16, 0.8))),
        layer(par(win(4, 2, 12, 10, 6, 21), delta(4, 2, 8, 12)), dense(40)),
        layer(ml(2, 12, 10, cap=4.0, name="mlstm_2"), None),
        layer(par(win(3, 1, 16, 20, 16, 70), delta(2, 2, 12, 8, conv=2),
                  1.1, 0.3), moe(4, 3, 20, 3))], 90, 48)


def cfg_ones():
    """Values that could hide a fault by being equal or 1: one head, one
    expert, no identity expert, ranks, taps and scales of 1, a window of
    one, a window longer than any sequence, one bucket."""
    return model_cfg([
        layer(par(win(1, 1, 16, 16, 16, 1, scale=1.0),
                  delta(1, 1, 16, 16, 1, 1, 1), 1.0, 1.0),
              moe(1, 1, 16, 0, 1.0, (16, 1.0))),
        layer(ml(1, 16, 16, cap=1.0), dense(16)),
        layer(par(win(2, 2, 8, 8, 2, 4096), delta(2, 1, 8, 8, 3, 8, 8),
                  0.0, 1.0), moe(2, 1, 16, 1)),
        layer(ml(2, 8, 8, name="mlstm_2"), moe(1, 2, 8, 1, 9.0))],
        40, 32, mult=1.0, buckets=1, mp=1, mc=1, eps=1e-6)


def cfg_wide():
    """Head sizes beyond one wave's columns, key sizes of the 32-token chunk
    form, a key group of four, many experts."""
    return model_cfg([
        layer(ml(2, 136, 72), dense(64)),
        layer(par(win(8, 2, 24, 136, 8, 100), delta(4, 1, 72, 40)),
              moe(9, 4, 32, 5, shared=(64, 2.0))),
        layer(par(win(2, 1, 40, 8, 40, 130), delta(1, 1, 136, 72, 4, 10)),
              dense(24)),
        layer(ml(1, 40, 200, name="mlstm_2"), None)], 64, 64, eps=1e-6)


def cfg_tiles():
    """Sizes that the MFMA kernels serve in bf16."""
    return model_cfg([
        layer(par(win(4, 2, 24, 48, 16, 64), delta(2, 2, 16, 32, 4, 8, 8)),
              moe(6, 2, 32, 2, shared=(32, 1.0))),
        layer(ml(4, 16, 32), moe(8, 3, 64, 1, shared=(64, 1.0))),
        layer(par(win(4, 1, 32, 16, 32, 150), delta(4, 2, 64, 64, 4, 16,
                                                    16)), dense(96)),
        layer(ml(1, 64, 128, name="mlstm_2"), dense(64))], 128, 64,
        buckets=200, eps=1e-6)


def cfg_plain():
    """No router (bf16 runs of it can be held tightly everywhere)."""
    return model_cfg([
        layer(ml(2, 32, 48), dense(80)),
        layer(par(win(6, 3, 16, 32, 8, 50), delta(3, 3, 24, 16)), None),
        layer(ml(1, 24, 32, cap=8.0, name="mlstm_2"), dense(48))], 80, 64,
        eps=1e-6)


def cfg_odd():
    """Sizes that are multiples of 2 at most, or odd."""
    return model_cfg([
        layer(ml(3, 10, 6, cap=5.5), moe(3, 2, 10, 2, shared=(14, 0.5))),
        layer(par(win(6, 2, 6, 14, 4, 19), delta(3, 1, 7, 9, 5, 3, 7)),
              dense(26)),
        layer(par(win(2, 2, 9, 7, 2, 33), delta(2, 2, 10, 6, 3, 5, 3)),
              moe(5, 2, 7, 1))], 37, 36, buckets=53, mp=3, mc=5)


def mixer_weights(lc, w, rnd):
    """Checkpoint tensors of one mixer (names without the layer prefix)."""
    mc, P, s = lc["mixer"], {}, w ** -0.5
    if lc["type"] != "parallel":
        H, D, V = mc["heads"], mc["dim"], mc["vdim"]
        for nm, n, k in (("q", H * D, 2), ("k", H * D, 1), ("v", H * V, 2),
                         ("g", H * V, 2), ("i", H, 2), ("f", H, 2)):
            P[nm] = rnd(n, w, std=k * s)
        P["i.b"], P["f.b"] = rnd(H), 2.0 + rnd(H)
        P["norm"] = 1.0 + rnd(H * V, std=0.2)
        P["o"] = rnd(w, H * V, std=(H * V) ** -0.5)
        return P
    L, R = mc["left"], mc["right"]
    for nm, n in (("q", L["heads"] * L["dim"]),
                  ("k", L["kv_heads"] * L["dim"]),
                  ("v", L["kv_heads"] * L["vdim"])):
        P["left." + nm] = rnd(n, w, std=2 * s)
    hv = L["heads"] * L["vdim"]
    P["left.o"] = rnd(w, hv, std=hv ** -0.5)
    H, D, V, K = R["heads"], R["dim"], R["vdim"], R["conv"]
    hv = H * V
    for nm, n in (("q", R["kv_heads"] * D), ("k", R["kv_heads"] * D),
                  ("v", hv)):
        P["right." + nm] = rnd(n, w, std=2 * s)
        P[f"right.{nm}.conv"] = rnd(n, K, std=0.5)
        P[f"right.{nm}.conv"][:, -1] += 0.7
    P["right.b"] = rnd(H, w, std=2 * s)
    P["right.A_log"] = rnd(H, std=0.5)
    P["right.a1"] = rnd(R["decay_rank"], w, std=s)
    P["right.a2"] = rnd(H * D, R["decay_rank"],
                        std=2 * R["decay_rank"] ** -0.5)
    P["right.dt_bias"] = rnd(H * D) - 2.0
    P["right.g1"] = rnd(R["gate_rank"], w, std=s)
    P["right.g2"] = rnd(hv, R["gate_rank"], std=2 * R["gate_rank"] ** -0.5)
    P["right.norm"] = 1.0 + rnd(V, std=0.2)
    P["right.o"] = rnd(w, hv, std=hv ** -0.5)
    return P


def ff_weights(mlp, w, rnd):
    def expert(pre, ff):
        return {pre + "gate": rnd(ff, w, std=2 * w ** -0.5),
                pre + "up": rnd(ff, w, std=2 * w ** -0.5),
                pre + "down": rnd(w, ff, std=ff ** -0.5)}
    if mlp["kind"] == "dense":
        return expert("", mlp["ff"])
    n = mlp["router"]["experts"] + mlp["router"]["identity"]
    P = {"router": rnd(n, w, std=3 * w ** -0.5),
         "correction": rnd(n, std=0.2)}
    for e in range(mlp["router"]["experts"]):
        P.update(expert(f"e{e}.", mlp["expert"]["ff"]))
    if mlp.get("shared"):
        P.update(expert("shared.", mlp["shared"]["ff"]))
    return P


def make_weights(cfg, seed=0):
    """Random checkpoint tensors (bf16-representable fp32), named as in a
    checkpoint file."""
    g = torch.Generator().manual_seed(seed)
    w = cfg["width"]

    def rnd(*shape, std=1.0):
        return (torch.randn(*shape, generator=g) * std).bfloat16().float()

    P = {"embed": rnd(cfg["vocab"], w),
         "bigram": rnd(cfg["embedding"]["bigram"]["buckets"] + 1, w),
         "head": rnd(cfg["vocab"], w, std=3 * w ** -0.5),
         "final.norm": 1.0 + rnd(w, std=0.1)}
    for i, lc in enumerate(cfg["layers"]):
        a = f"l{i}."
        P[a + "norm1"] = 1.0 + rnd(w, std=0.1)
        subs = [("mix.", mixer_weights(lc, w, rnd))]
        if lc.get("mlp") is not None:
            subs.append(("mlp.", ff_weights(lc["mlp"], w, rnd)))
        for pre, Q in subs:
            P.update({a + pre + k: v for k, v in Q.items()})
    return {k: v.bfloat16().float() for k, v in P.items()}


def file_config(cfg):
    """The configuration as a checkpoint's config.json holds it."""
    out = json.loads(json.dumps(cfg))
    for lc in out["layers"]:
        if lc["type"] == "parallel":
            for k in ("decay_rank", "gate_rank"):
                lc["mixer"]["right"].pop(k, None)
    return out


def write_checkpoint(path, cfg, P):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(file_config(cfg), f)
    save_file({k: v.bfloat16().contiguous() for k, v in P.items()},
              os.path.join(path, "model.safetensors"))


def np64(P):
    return {k: v.double().numpy() for k, v in P.items()}


def oracle(cfg, P, toks, layers=None):
    return torch.from_numpy(O.forward(cfg, np64(P), toks, layers))


_CACHE = {}


def model(tmp_path_factory, cfg_fn, device, dtype, seed=0):
    """(runner, oracle weights, cfg) — checkpoint written once per
    configuration, loaded through the registry by directory name."""
    key = (cfg_fn.__name__, seed)
    if key not in _CACHE:
        cfg = cfg_fn()
        P = make_weights(cfg, seed)
        d = str(tmp_path_factory.mktemp(cfg_fn.__name__))
        write_checkpoint(d, cfg, P)
        _CACHE[key] = (d, cfg, P)
    d, cfg, P = _CACHE[key]
    runner = PipelineRunner(plan_for_world(d, 1), 0, 1,
                            device=torch.device(device), init="checkpoint",
                            ckpt_dir=d, dtype=dtype)
    return runner, P, cfg


def batcher(runner, max_ctx=512, pool_pages=None, slots=4):
    return ContinuousBatcher(runner, max_slots=slots, max_ctx=max_ctx,
                             pool_pages=pool_pages)


def rel_err(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std(-1).clamp_min(1e-6)


def close(got, want, dtype, cfg):
    """fp32: every position within tolerance of the oracle. bf16: without a
    router every position, the worst one loosely; with one, a close routing
    decision that falls the other way after 16-bit rounding changes single
    positions altogether, so the bulk is held. Exactness is the fp32 runs'
    job, bf16 runs show that the same path works in that dtype."""
    e = rel_err(got, want).reshape(-1)
    routed = any((lc.get("mlp") or {}).get("kind") == "moe"
                 for lc in cfg["layers"])
    if dtype == torch.float32:
        ok = float(e.max()) < tol(dtype)
    elif routed:
        ok = (float(e.median()) < tol(dtype)
              and float(e.quantile(0.75)) < 2 * tol(dtype))
    else:
        ok = (float(e.median()) < tol(dtype) / 2
              and float(e.quantile(0.9)) < tol(dtype)
              and float(e.max()) < 4 * tol(dtype))
    if not ok:
        print("rel err: median %.3g p90 %.3g max %.3g at %d" % (
            float(e.median()), float(e.quantile(0.9)), float(e.max()),
            int(e.argmax())))
    return ok


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def run_schedule(b, toks, cuts, rid="r"):
    """Feed ``toks`` in portions of the given sizes (rest one by one);
    returns logits at every position."""
    outs, at = [], 0
    sizes = list(cuts)
    while at < len(toks):
        n = sizes.pop(0) if sizes else 1
        n = min(n, len(toks) - at)
        last = at + n == len(toks)
        outs.append(b.forced_step([(rid, toks[at:at + n], list(range(n)))],
                                  [rid] if last else []))
        at += n
    return torch.cat(outs)


def _rnd(seed):
    g = torch.Generator().manual_seed(seed)
    return lambda *shape, std=1.0: (torch.randn(*shape, generator=g)
                                    * std).bfloat16().float()


# ------------------------------------------------- mechanisms, one by one
class Hosted:
    """A framework mixer of a layer spec, filled from oracle tensors ``P``
    (names without prefix), and the two projections that its layer runs for
    it. ``scale`` = False leaves a pair's two outputs apart."""

    def __init__(self, lc, width, eps, P, device, dtype):
        from tensorlink_amd.models.lunadra import build_mixer
        self.mod = mod = build_mixer(lc, width, eps)
        W = torch.zeros(mod.in_cols, width)
        thin = torch.zeros(mod.thin_cols, width)
        self.bias = None

        def put(M, row, t):
            M[row:row + t.shape[0]] = t

        with torch.no_grad():
            if mod.kind == "mlstm":
                for nm, off in zip("qkvg", mod.offs):
                    put(W, off, P[nm])
                put(thin, 0, torch.cat([P["i"], P["f"]]))
                self.bias = torch.cat([P["i.b"], P["f.b"]]).to(device)
                mod.norm.copy_(P["norm"])
                mod.o_proj.weight.copy_(P["o"])
            else:
                L, R, c = mod.left, mod.right, mod.right_col
                for nm, off in (("q", 0), ("k", L.q_cols),
                                ("v", L.q_cols + L.k_cols)):
                    put(W, off, P["left." + nm])
                L.o_proj.weight.copy_(P["left.o"])
                for nm, off in zip("qkv", R.offs):
                    put(W, c + off, P["right." + nm])
                    put(R.conv, off, P[f"right.{nm}.conv"])
                put(W, c + R.a_col, P["right.a1"])
                put(W, c + R.g_col, P["right.g1"])
                put(thin, 0, P["right.b"])
                for nm in ("A_log", "a2", "dt_bias", "g2", "norm"):
                    getattr(R, nm).copy_(P["right." + nm])
                R.o_proj.weight.copy_(P["right.o"])
        self.W = W.to(device, dtype)
        self.thin = thin.to(device, dtype)
        mod.to(device=device, dtype=dtype)

    def __call__(self, h, meta, cache):
        p = torch.nn.functional.linear(h, self.W)
        t = mx.thin_linear(h, self.thin, self.bias)
        if self.mod.kind == "mlstm":
            return self.mod(p, meta, cache, 0, 0, t)
        a, b = self.mod(p, meta, cache.k[0], cache.v[0], cache.state[0], 0,
                        t)
        ls, rs = self.mod.scales
        return ls * a.float() + rs * b.float()


def run_mixer(mod, h, cuts, device, dtype, pages=4, slot=1):
    """One mixer over one sequence cut into portions, in a slot whose state
    and pages hold the leavings of another sequence."""
    T = h.shape[0]
    pages = max(pages, (T + PAGE - 1) // PAGE + 1)
    cache = HybridSlotCache([mod.mod.cache_spec()], 2, pages, pages * PAGE,
                            device, dtype)
    for group in (cache.k, cache.v, *cache.state):
        for t in group or ():
            if t is not None and t.numel():
                t.normal_(0.0, 3.0)
    outs, at, sizes = [], 0, list(cuts)
    while at < T:
        n = min(sizes.pop(0) if sizes else 1, T - at)
        cache.ensure(slot, at + n)
        meta = mx.RaggedMeta([n], [at], [slot], cache.table[[slot]], device)
        with torch.no_grad():
            y = mod(h[at:at + n].to(device=device, dtype=dtype), meta, cache)
        outs.append(y.float().cpu())
        at += n
    return torch.cat(outs)


def mixer_close(got, want, dtype, lim16=4e-2):
    """A mixer's output rows against the oracle's: row errors over the
    typical row size. fp32: the worst row. bf16: the bulk of the rows
    tightly and the worst one loosely."""
    want = torch.as_tensor(want)
    err = (got.double() - want).norm(dim=-1) / want.norm(dim=-1).median()
    if dtype == torch.float32:
        ok = float(err.max()) < 2e-4
    else:
        ok = (float(err.quantile(0.9)) < lim16
              and float(err.max()) < 5 * lim16)
    if not ok:
        print("mixer err max %.3g at row %d, p90 %.3g" % (
            float(err.max()), int(err.argmax()), float(err.quantile(0.9))))
    return ok


def oracle_mixer(lc, h, P, eps):
    fn = O.parallel if lc["type"] == "parallel" else O.mlstm
    return fn(h.double().numpy(), np64(P), lc["mixer"], eps)


@pytest.mark.parametrize("hdv,cap", [
    ((3, 8, 20), 15.0), ((1, 16, 16), 1.0), ((2, 136, 72), 15.0),
    ((1, 40, 200), 3.0), ((4, 16, 32), 30.0), ((3, 10, 6), 5.5),
    ((2, 7, 9), 8.0), ((2, 64, 128), 15.0), ((1, 200, 12), 4.0),
    ((1, 24, 300), 15.0)], ids=lambda x: str(x).replace(" ", ""))
@pytest.mark.parametrize("device,dtype", ALL)
def test_mlstm_against_oracle(device, dtype, hdv, cap):
    """The matrix memory alone: whole (chunk form on the GPU), in portions
    down to two tokens, token by token; a slot that holds another
    sequence's state."""
    w, eps, T = 40, 1e-5, 290
    lc = ml(*hdv, cap=cap)
    rnd = _rnd(5)
    P = mixer_weights(lc, w, rnd)
    h = rnd(T, w)
    want = oracle_mixer(lc, h, P, eps)
    mod = Hosted(lc, w, eps, P, device, dtype)
    for cuts in ([T], [140, 2, 3, 130], [257, 2], [3]):
        got = run_mixer(mod, h, cuts, device, dtype)
        assert mixer_close(got, want, dtype), cuts


@pytest.mark.parametrize("case", ["open", "shut", "floor", "swing"])
@pytest.mark.parametrize("device,dtype", ALL)
def test_mlstm_gate_extremes(device, dtype, case):
    """Gates at their limits: a memory that keeps a token written early to
    the end (open), one that forgets at once (shut), gates so low that the
    normaliser's floor decides from the first token on — the running
    maximum starts at 0 — (floor), and input gates that jump by the whole
    cap between tokens (swing)."""
    w, eps, T = 40, 1e-5, 330
    lc = ml(2, 16, 24, cap=12.0)
    rnd = _rnd(21)
    P = mixer_weights(lc, w, rnd)
    h = rnd(T, w)
    for nm in ("i", "f"):
        P[nm] = P[nm] * (30.0 if case == "swing" and nm == "i" else 0.1)
    P["f.b"] = torch.full((2,), {"open": 30.0, "swing": 4.0}.get(case, -6.0))
    P["i.b"] = torch.full((2,), {"floor": -30.0}.get(case, 0.0))
    if case == "open":
        P["k"] = P["k"] * 0.1
        h[3] *= 12.0
    want = oracle_mixer(lc, h, P, eps)
    if case == "open":
        h2 = h.clone()
        h2[3] = rnd(w)
        alt = oracle_mixer(lc, h2, P, eps)
        assert np.linalg.norm(alt[-1] - want[-1]) > \
            0.3 * np.linalg.norm(want[-1])
    mod = Hosted(lc, w, eps, P, device, dtype)
    for cuts in ([T], [200, 2, 100], [64, 150]):
        got = run_mixer(mod, h, cuts, device, dtype)
        assert mixer_close(got, want, dtype, 8e-2), cuts


@pytest.mark.parametrize("shape", [
    (4, 2, 8, 12, 4, 6, 5), (1, 1, 16, 16, 1, 1, 1), (4, 1, 72, 40, 4, 6, 5),
    (1, 1, 136, 72, 4, 10, 5), (2, 2, 32, 64, 3, 20, 8),
    (3, 1, 7, 9, 5, 3, 7), (4, 2, 64, 64, 4, 16, 16), (2, 1, 10, 6, 2, 5, 3),
    (1, 1, 270, 20, 4, 4, 4), (2, 2, 128, 33, 9, 33, 2),
    (1, 1, 24, 140, 4, 70, 3), (2, 1, 250, 16, 3, 4, 4)],
    ids=lambda x: "x".join(map(str, x)))
@pytest.mark.parametrize("device,dtype", ALL)
def test_delta_rule_against_oracle(device, dtype, shape):
    """The gated delta rule alone (the pair's other half weighs nothing):
    whole (chunk form on the GPU), portions down to two tokens, token by
    token; key groups, taps of 1 to 9, ranks of 1 to 70."""
    w, eps, T = 40, 1e-5, 210
    lc = par(win(1, 1, 8, 8, 8, 5), delta(*shape), 0.0, 1.0)
    rnd = _rnd(7)
    P = mixer_weights(lc, w, rnd)
    h = rnd(T, w)
    want = oracle_mixer(lc, h, P, eps)
    mod = Hosted(lc, w, eps, P, device, dtype)
    for cuts in ([T], [140, 2, 3, 60], [129, 2, 64], [3]):
        got = run_mixer(mod, h, cuts, device, dtype)
        assert mixer_close(got, want, dtype), cuts


@pytest.mark.parametrize("case", ["kept", "fast", "vanishing", "repeat"])
@pytest.mark.parametrize("device,dtype", ALL)
def test_delta_rule_extremes(device, dtype, case):
    """Decays from none over a long sequence (kept: an early token must
    still be there at the end) over strong (fast) to gone at once
    (vanishing: running sums of log-decays leave the range of fp32's
    exponential inside one tile); the same key again and again with step
    sizes near one, so that every write corrects the last (repeat)."""
    w, eps, T, D = 40, 1e-5, 330, 24
    lc = par(win(1, 1, 8, 8, 8, 5), delta(2, 1, D, 16, 2, 4, 4), 0.0, 1.0)
    rnd = _rnd(12)
    P = mixer_weights(lc, w, rnd)
    h = rnd(T, w)
    if case in ("kept", "repeat"):
        P["right.a1"] = P["right.a1"] * 0.1
        P["right.dt_bias"] = torch.full((2 * D,), -12.0)
    else:
        f = 3.0 if case == "fast" else 40.0
        P["right.a2"] = P["right.a2"] * f
        P["right.A_log"] = P["right.A_log"] + math.log(f)
    if case == "kept":
        # later tokens write little
        P["right.b"] = P["right.b"] * 0.0
        P["right.b"][:, 0] = 4.0
        h[:, 0] = -2.0
        h[3, 0] = 2.0
    if case == "repeat":
        P["right.b"] = P["right.b"] * 0.0
        P["right.b"][:, 0] = 4.0
        P["right.k"] = P["right.k"] * 0.02
        P["right.k"][:, 0] += 3.0 * rnd(D).abs()
        h[:, 0] = 2.0
    want = oracle_mixer(lc, h, P, eps)
    if case == "kept":
        h2 = h.clone()
        h2[3, 1:] = rnd(w)[1:]
        alt = oracle_mixer(lc, h2, P, eps)
        assert np.linalg.norm(alt[-1] - want[-1]) > \
            0.3 * np.linalg.norm(want[-1])
    mod = Hosted(lc, w, eps, P, device, dtype)
    for cuts in ([T], [200, 2, 100], [64, 150]):
        got = run_mixer(mod, h, cuts, device, dtype)
        if dtype == torch.float32:
            assert mixer_close(got, want, dtype), cuts
        else:
            # bf16 rounding before a large a2, or of nearly parallel keys,
            # moves single rows: the typical row is held
            err = (got.double() - torch.from_numpy(want)).norm(dim=-1) \
                / torch.from_numpy(want).norm(dim=-1).median()
            assert float(err.median()) < 6e-2, cuts


@pytest.mark.parametrize("H,G,D,V", [(4, 2, 20, 12), (2, 2, 64, 40),
                                     (2, 1, 100, 36)])
@pytest.mark.parametrize("device,dtype", ALL)
def test_delta_state_across_a_batch(device, dtype, H, G, D, V):
    """The op on a ragged batch of fresh and continued sequences in
    shuffled slots, chunk form and token walk: read-outs and the states
    left behind equal each sequence alone; untouched slots stay."""
    R = 5
    g = torch.Generator().manual_seed(2)
    new, pos0, slots = [150, 1, 257, 2], [0, 70, 5, 0], [4, 0, 3, 1]
    T, C = sum(new), 2 * G * D + H * V
    x = torch.randn(T, C + 2, generator=g)
    proj = torch.randn(T, R + 3, generator=g).to(dtype)
    b = torch.randn(T, H + 1, generator=g)
    a2t = torch.randn(R, H * D, generator=g) * 0.5
    dt = torch.randn(H * D, generator=g) - 2.0
    A = torch.randn(H, generator=g) * 0.5
    S0 = torch.randn(5, H, D, V, generator=g)
    f = x.double().numpy()[:, 1:]
    dec = np.exp(-np.exp(A.double().numpy())[:, None] * O.softplus(
        proj.double().numpy()[:, 2:2 + R] @ a2t.double().numpy()
        + dt.double().numpy()).reshape(T, H, D))
    beta = O.sigmoid(b.double().numpy()[:, 1:])
    q = O.unit(f[:, :G * D].reshape(T, G, D)) / math.sqrt(D)
    k = O.unit(f[:, G * D:2 * G * D].reshape(T, G, D))
    v = f[:, 2 * G * D:C].reshape(T, H, V)
    want, states, at = np.zeros((T, H, V)), {}, 0
    for n, p, s in zip(new, pos0, slots):
        st = np.zeros((H, D, V)) if p == 0 else S0[s].double().numpy()
        for t in range(at, at + n):
            for h in range(H):
                kk, qq = k[t, h // (H // G)], q[t, h // (H // G)]
                S = dec[t, h][:, None] * st[h]
                S = S + np.outer(kk, beta[t, h] * (v[t, h] - S.T @ kk))
                st[h] = S
                want[t, h] = S.T @ qq
        states[s] = st
        at += n
    want = want.reshape(T, H * V)
    meta = mx.RaggedMeta(new, pos0, slots, torch.zeros(4, 2,
                         dtype=torch.int32).to(device), device)
    for chunks in (True, False):
        if not chunks:
            os.environ["TL_NO_SCAN_CHUNKS"] = "1"
        try:
            S = S0.to(device).clone()
            got = mx.delta_scan(
                x.to(device), (1, 1 + G * D, 1 + 2 * G * D), proj.to(device),
                2, b.to(device), 1, a2t.to(device), dt.to(device),
                A.to(device), S, meta, H, G, D, V)
        finally:
            os.environ.pop("TL_NO_SCAN_CHUNKS", None)
        assert np.abs(got.cpu().numpy() - want).max() < \
            1e-4 * np.abs(want).max()
        for s, st in states.items():
            assert np.abs(S[s].cpu().numpy() - st).max() < \
                1e-4 * np.abs(st).max()
        assert torch.equal(S[2].cpu(), S0[2])


@pytest.mark.parametrize("H,D,V", [(3, 20, 12), (2, 64, 80), (1, 100, 132),
                                   (2, 7, 9)])
@pytest.mark.parametrize("device,dtype", ALL)
def test_mlstm_state_across_a_batch(device, dtype, H, D, V):
    """The op on a ragged batch of fresh and continued sequences in
    shuffled slots, chunk forms and token walk: outputs and the states
    left behind equal each sequence alone; untouched slots stay."""
    g = torch.Generator().manual_seed(9)
    new, pos0, slots = [150, 1, 257, 2], [0, 70, 5, 0], [4, 0, 3, 1]
    T, cap, eps = sum(new), 15.0, 1e-5
    offs = (0, H * D, 2 * H * D, 2 * H * D + H * V)
    proj = torch.randn(T, offs[3] + H * V + (4 if D % 4 == 0 else 3),
                       generator=g).to(dtype)
    gates = torch.randn(T, 2 * H + 3, generator=g) * 3
    nw = 1.0 + 0.2 * torch.randn(H * V, generator=g)
    S0 = torch.randn(5, H, D, V, generator=g)
    n0, m0 = torch.randn(5, H, D, generator=g), torch.rand(5, H, generator=g)
    f, gt = proj.double().numpy(), gates.double().numpy()
    want, states, at = np.zeros((T, H, V)), {}, 0
    for cnt, p, s in zip(new, pos0, slots):
        S, n, m = (x[s].double().numpy().copy() * (p > 0)
                   for x in (S0, n0, m0))
        for t in range(at, at + cnt):
            for h in range(H):
                q, k, v, _ = (f[t, o + h * w:o + (h + 1) * w]
                              for o, w in zip(offs, (D, D, V, V)))
                li = cap * math.tanh(gt[t, h] / cap)
                lf = -O.softplus(-cap * math.tanh(gt[t, H + h] / cap))
                top = max(lf + m[h], li)
                a, b = math.exp(lf + m[h] - top), math.exp(li - top)
                S[h] = a * S[h] + b * np.outer(k, v)
                n[h] = a * n[h] + b * k
                m[h] = top
                q = q / math.sqrt(D)
                want[t, h] = (S[h].T @ q) / (
                    max(abs(n[h] @ q), math.exp(-top)) + 1e-6)
        states[s] = (S, n, m)
        at += cnt
    want = O.rms(want, eps).reshape(T, H * V) * nw.double().numpy() \
        * O.sigmoid(f[:, offs[3]:offs[3] + H * V])
    meta = mx.RaggedMeta(new, pos0, slots, torch.zeros(4, 2,
                         dtype=torch.int32).to(device), device)
    lim = 2e-4 if dtype == torch.float32 else 2e-2
    for chunks in (True, False):
        if not chunks:
            os.environ["TL_NO_SCAN_CHUNKS"] = "1"
        try:
            S, n, m = (x.to(device).clone() for x in (S0, n0, m0))
            got = mx.mlstm_scan(proj.to(device), offs, gates.to(device),
                                nw.to(device), S, n, m, meta, H, D, V, cap,
                                eps)
        finally:
            os.environ.pop("TL_NO_SCAN_CHUNKS", None)
        # a normaliser near zero makes single rows ill-conditioned
        err = np.abs(got.float().cpu().numpy() - want).max(-1)
        assert np.quantile(err, 0.98) < lim * np.abs(want).max()
        for s, st in states.items():
            for x, y in zip((S, n, m), st):
                assert np.abs(x[s].cpu().numpy() - y).max() < \
                    1e-4 * np.abs(y).max()
        assert torch.equal(S[2].cpu(), S0[2])
        assert torch.equal(m[2].cpu(), m0[2])


@pytest.mark.parametrize("device,dtype", ALL)
def test_short_convolution(device, dtype):
    """The convolution with silu on a ragged batch, one to nine taps, with
    and without the vector path: portions shorter and longer than the taps,
    slots that hold another sequence's inputs before the first step."""
    g = torch.Generator().manual_seed(8)
    for N, K, col in ((12, 1, 4), (8, 2, 0), (16, 4, 8), (2052, 4, 4),
                      (12, 9, 4), (7, 3, 1), (10, 5, 2), (12, 6, 8)):
        seqs = [torch.randn(n, N + col + 4, generator=g).to(dtype)
                for n in (40, 3, 17)]
        taps = torch.randn(N, K, generator=g)
        want = [O.short_conv_silu(s[:, col:col + N].double().numpy(),
                                  taps.double().numpy()) for s in seqs]
        hist = torch.randn(5, K - 1, N, generator=g).to(device)
        slots, at = [3, 0, 4], [0, 0, 0]
        for step in ([9, 1, 2], [1, 1, 1], [30, 0, 14], [0, 1, 0]):
            live = [i for i in range(3) if step[i]]
            meta = mx.RaggedMeta(
                [step[i] for i in live], [at[i] for i in live],
                [slots[i] for i in live],
                torch.zeros(len(live), 1, dtype=torch.int32).to(device),
                device)
            src = torch.cat([seqs[i][at[i]:at[i] + step[i]] for i in live])
            got = mx.conv_rope_rows(src.to(device), col, 1, N,
                                    taps.to(device), hist, meta, silu=True)
            ref = np.concatenate([want[i][at[i]:at[i] + step[i]]
                                  for i in live])
            assert np.abs(got.cpu().numpy() - ref).max() < 2e-5, (N, K)
            for i in live:
                at[i] += step[i]


@pytest.mark.parametrize("hgdv,rot,size", [
    ((4, 2, 12, 10), 6, 21), ((1, 1, 16, 16), 16, 1),
    ((8, 2, 24, 136), 8, 100), ((4, 2, 24, 48), 24, 64),
    ((4, 1, 32, 16), 32, 4096), ((6, 2, 6, 14), 4, 19),
    ((5, 5, 40, 8), 2, 2), ((6, 1, 40, 96), 40, 128)],
    ids=lambda x: str(x).replace(" ", ""))
@pytest.mark.parametrize("device,dtype", ALL)
def test_window_attention_against_oracle(device, dtype, hgdv, rot, size):
    """The attention alone (the pair's other half weighs nothing) across a
    page border: partial and full rotation, windows of one, two, around a
    page and longer than the sequence."""
    w, eps, T = 40, 1e-5, 170
    lc = par(win(*hgdv, rot, size, base=500.0), delta(1, 1, 8, 8), 1.3, 0.0)
    rnd = _rnd(6)
    P = mixer_weights(lc, w, rnd)
    h = rnd(T, w)
    want = oracle_mixer(lc, h, P, eps)
    mod = Hosted(lc, w, eps, P, device, dtype)
    for cuts in ([T], [100, 27, 2, 2], [130]):
        got = run_mixer(mod, h, cuts, device, dtype)
        assert mixer_close(got, want, dtype), cuts


@pytest.mark.parametrize("device,dtype", ALL)
def test_window_edges_and_far_keys(device, dtype):
    """One key answers one query: just inside and just outside the window,
    at page borders, at the first token; read from inside a prompt portion
    and decoded alone. Inside, the output is another without it; outside it
    makes no difference at all."""
    w, eps, D = 40, 1e-6, 32
    cases = [(qpos, qpos - size + 1 - out, size)
             for qpos, size in ((2 * PAGE + 9, PAGE + 10), (PAGE + 20, 40),
                                (70, 70), (PAGE, 2), (2 * PAGE, PAGE))
             for out in (0, 1) if qpos - size + 1 - out >= 0]
    cases += [(2 * PAGE + 9, PAGE - 1, 500), (2 * PAGE + 9, PAGE, 500),
              (2 * PAGE, 0, 500), (PAGE - 1, 0, 500)]
    for n, (qpos, kpos, size) in enumerate(cases):
        lc = par(win(2, 1, D, 8, 0, size, scale=1.0), delta(1, 1, 8, 8), 1.0,
                 0.0)
        rnd = _rnd(40 + n)
        P = mixer_weights(lc, w, rnd)
        T = qpos + 2
        h = rnd(T, w)
        # an input row whose key points where the query's heads point
        q = (P["left.q"] @ h[qpos]).view(2, D).double().sum(0)
        row = torch.linalg.pinv(P["left.k"].double()) @ (
            60.0 * q / q.norm())
        h[kpos] = row.float().bfloat16().float()
        want = oracle_mixer(lc, h, P, eps)
        h2 = h.clone()
        h2[kpos] = rnd(w)
        alt = oracle_mixer(lc, h2, P, eps)
        d = np.linalg.norm(want[qpos] - alt[qpos])
        if qpos - kpos < size:
            assert d > 0.3 * np.linalg.norm(want[qpos])
        else:
            assert d == 0.0
        mod = Hosted(lc, w, eps, P, device, dtype)
        for cuts in ([T], [qpos], [max(1, qpos - 5), 2, 20]):
            got = run_mixer(mod, h, cuts, device, dtype)
            e = (got[qpos].double() - torch.from_numpy(want[qpos])).norm()
            lim = 2e-4 if dtype == torch.float32 else 6e-2
            assert float(e) < lim * np.linalg.norm(want[qpos]), \
                (qpos, kpos, size, cuts)


@pytest.mark.parametrize("device,dtype", ALL)
def test_first_tokens_reach_the_end(device, dtype):
    """Both mixers' states carry a sequence's first tokens: changing token
    0 changes a far output, and the framework follows; the first output
    rows (convolution before its first taps, one visible key) are exact."""
    w, eps, T = 40, 1e-5, 150
    for lc in (ml(2, 16, 12), par(win(2, 1, 8, 8, 8, 400),
                                  delta(2, 2, 16, 12, conv=6), 0.5, 0.5)):
        rnd = _rnd(33)
        P = mixer_weights(lc, w, rnd)
        if "f" in P:
            P["f.b"] = torch.full((2,), 20.0)
            P["f"] = P["f"] * 0.1
        else:
            P["right.dt_bias"] = P["right.dt_bias"] - 9.0
            P["right.a1"] = P["right.a1"] * 0.1
        h = rnd(T, w)
        h2 = h.clone()
        h2[0] = rnd(w)
        w1, w2 = (oracle_mixer(lc, x, P, eps) for x in (h, h2))
        mod = Hosted(lc, w, eps, P, device, dtype)
        g1, g2 = (run_mixer(mod, x, [140, 2], device, dtype)
                  for x in (h, h2))
        assert mixer_close(g1, w1, dtype) and mixer_close(g2, w2, dtype)
        assert mixer_close(g1[:8], w1[:8], dtype)
        if dtype == torch.float32:
            dw = torch.from_numpy(w2 - w1)[-1]
            assert float(dw.norm()) > 1e-3 * np.linalg.norm(w1[-1])
            assert float(((g2 - g1)[-1].double() - dw).norm()) < \
                2e-2 * float(dw.norm()) + 1e-5 * np.linalg.norm(w1[-1])


@pytest.mark.parametrize("device,dtype", ALL)
def test_bigram_embedding(device, dtype):
    """Rows of the bigram table on a ragged batch: a sequence's first token,
    the token before a portion from its slot (one that holds another
    sequence's token before), portions of one token, products beyond 32
    bits; the slots left holding the last tokens, others untouched."""
    g = torch.Generator().manual_seed(3)
    for V, n, mp, mc, W in ((50, 13, 5, 3, 12), (30, 1, 1, 1, 7),
                            (40000, 997, 131071, 65537, 36)):
        embed = torch.randn(V, W, generator=g).to(dtype)
        table = torch.randn(n + 1, W, generator=g).to(dtype)
        seqs = [torch.randint(0, V, (k,), generator=g).tolist()
                for k in (20, 3, 9, 30)]
        spec = {"buckets": n, "mul_prev": mp, "mul_cur": mc}
        want = [embed[s].double() + table[O.bigram_rows(s, spec)].double()
                for s in seqs]
        slots = [5, 0, 3, 1]
        prev = torch.full((6,), 7, dtype=torch.int32, device=device)
        at = [0] * 4
        for step in ([0, 1, 5, 2], [1, 1, 1, 1], [19, 0, 3, 27], [0, 1, 0, 0]):
            live = [i for i in range(4) if step[i]]
            meta = mx.RaggedMeta(
                [step[i] for i in live], [at[i] for i in live],
                [slots[i] for i in live],
                torch.zeros(len(live), 1, dtype=torch.int32).to(device),
                device)
            toks = [t for i in live for t in seqs[i][at[i]:at[i] + step[i]]]
            X = mx.bigram_embed(torch.tensor([toks], device=device),
                                embed.to(device), table.to(device), prev,
                                meta, mp, mc)
            ref = torch.cat([want[i][at[i]:at[i] + step[i]] for i in live])
            assert X.dtype == torch.float32
            assert (X.double().cpu() - ref).abs().max() < 1e-6
            for i in live:
                at[i] += step[i]
                assert int(prev[slots[i]]) == seqs[i][at[i] - 1]
        assert prev[2] == 7 and prev[4] == 7


@pytest.mark.parametrize("device,dtype", ALL)
def test_row_ops(device, dtype):
    """Residual sums of several scaled terms with the norm, per-head norm
    with a sigmoid gate, the two activations on columns of a wider
    projection, thin projections with fp32 results: against the oracle's
    formulas, sizes with and without the vector paths."""
    g = torch.Generator().manual_seed(4)
    a = 3e-5 if dtype == torch.float32 else 2e-2
    for W in (48, 33, 1028, 2304):
        for n in (0, 1, 2, 3):
            X = torch.randn(5, W, generator=g) * 3
            ys = [torch.randn(5, W, generator=g).to(dtype)
                  for _ in range(n)]
            fs = [0.5, -1.3, 0.07][:n]
            wn = 1.0 + 0.2 * torch.randn(W, generator=g)
            want = X.double().numpy() + sum(
                f * y.double().numpy() for f, y in zip(fs, ys))
            for with_w in (True, False):
                Xd = X.to(device).clone()
                h = mx.add_rms(
                    Xd, ys[0].to(device) if n else None,
                    wn.to(device) if with_w else None, 1e-5, dtype,
                    y_scale=fs[0] if n else 1.0,
                    more=[(y.to(device), f)
                          for y, f in zip(ys[1:], fs[1:])])
                assert np.abs(Xd.cpu().numpy() - want).max() < 1e-5
                if with_w:
                    hw = O.rms(want, 1e-5) * wn.double().numpy()
                    assert np.abs(h.float().cpu().numpy() - hw).max() < a * 4
    for H, V, col in ((3, 20, 4), (2, 128, 0), (1, 9, 1), (5, 64, 8)):
        x = torch.randn(4, H * V, generator=g)
        p = torch.randn(4, H * V + 10, generator=g).to(dtype)
        wn = 1.0 + 0.2 * torch.randn(V, generator=g)
        want = O.rms(x.double().numpy().reshape(4, H, V), 1e-6) \
            * wn.double().numpy()
        want = want.reshape(4, -1) * O.sigmoid(
            p[:, col:col + H * V].double().numpy())
        got = mx.rms_scale(x.to(device), wn.to(device), 1e-6, False,
                           gate=p.to(device), gate_col=col, out_dtype=dtype,
                           heads=H, gate_act="sigmoid").float().cpu().numpy()
        assert np.abs(got - want).max() < a * 4
    for N, col, extra in ((24, 8, 8), (7, 3, 2), (16, 0, 0)):
        p = (3.0 * torch.randn(6, col + 2 * N + extra, generator=g)).to(dtype)
        f = p.double().numpy()
        gt, up = f[:, col:col + N], f[:, col + N:col + 2 * N]
        got = mx.act_gate(p.to(device), "relu", N, col).float().cpu().numpy()
        assert np.abs(got - np.maximum(gt, 0) * up).max() < a * 20
        for lim, alpha in ((1.1, 1.702), (0.3, 1.0), (50.0, 3.0)):
            c = np.minimum(gt, lim)
            want = c * O.sigmoid(alpha * c) * (np.clip(up, -lim, lim) + 1)
            got = mx.act_gate(p.to(device), ("clamped_swish", lim, alpha), N,
                              col).float().cpu().numpy()
            assert np.abs(got - want).max() < a * 20
    for T, W, N in ((1, 40, 5), (7, 33, 16), (64, 64, 130), (65, 40, 32),
                    (200, 48, 16)):
        h = torch.randn(T, W, generator=g).to(dtype)
        w = torch.randn(N, W, generator=g).to(dtype)
        b = torch.randn(N, generator=g)
        want = h.double() @ w.double().t()
        for bias in (None, b):
            got = mx.thin_linear(h.to(device), w.to(device),
                                 None if bias is None else bias.to(device))
            assert got.dtype == torch.float32
            ref = want if bias is None else want + b.double()
            assert (got.double().cpu() - ref).abs().max() < 1e-4


def routed_ff(spec, w, P, device, dtype):
    """The framework's mixture of a spec and the two projections its layer
    runs for it."""
    from tensorlink_amd.models.lunadra import build_ff
    mod = build_ff(spec, w)
    with torch.no_grad():
        mod.correction.copy_(P["correction"])
        for e in range(spec["router"]["experts"]):
            mod.gate_up[e].copy_(torch.cat([P[f"e{e}.gate"], P[f"e{e}.up"]]))
            mod.down[e].copy_(P[f"e{e}.down"])
        W = torch.zeros(max(1, mod.in_cols), w)
        if spec.get("shared"):
            W.copy_(torch.cat([P["shared.gate"], P["shared.up"]]))
            mod.shared_down.weight.copy_(P["shared.down"])
    mod = mod.to(device=device, dtype=dtype)
    W, R = W.to(device, dtype), P["router"].to(device, dtype)

    def run(h):
        h = h.to(device=device, dtype=dtype)
        with torch.no_grad():
            return mod(h, torch.nn.functional.linear(h, W), 0,
                       mx.thin_linear(h, R), 0)
    return run


@pytest.mark.parametrize("T", [1, 9, 100, 2500])
@pytest.mark.parametrize("device,dtype", ALL)
def test_routed_experts(device, dtype, T):
    """The mixture alone: few rows and many, identity experts (none, some,
    more than real ones), experts that nobody chooses, all chosen at once,
    sizes for the MFMA products and odd ones, with and without a shared
    expert of another limit."""
    for n, (w, spec) in enumerate([
            (64, moe(6, 2, 32, 2, shared=(64, 0.5))), (36, moe(5, 2, 10, 3)),
            (64, moe(70, 3, 64, 4)), (24, moe(1, 1, 8, 0, shared=(8, 3.0))),
            (32, moe(2, 6, 16, 4, 0.7, shared=(6, 1.0)))]):
        if T == 2500 and n not in (0, 1):
            continue
        rnd = _rnd(60 + n)
        P = ff_weights(spec, w, rnd)
        if n == 2:
            P["correction"][5:40] -= 3.0
        run = routed_ff(spec, w, P, device, dtype)
        rows = min(T, 300)
        h = rnd(rows, w)
        want = torch.from_numpy(O.moe(h.double().numpy(), np64(P), spec))
        reps = (T + rows - 1) // rows
        got = run(h.repeat(reps, 1)[:T]).double().cpu()
        want = want.repeat(reps, 1)[:T]
        err = (got - want).norm(dim=-1) / want.norm(dim=-1).median()
        lim = 1e-5 if dtype == torch.float32 else 2e-2
        assert float(err.quantile(0.75)) < lim, (n, float(err.max()))
        assert float(err.max()) < lim * 20, (n, float(err.max()))


@pytest.mark.parametrize("device,dtype", ALL)
def test_all_choices_identity(device, dtype):
    """A correction that sends every token to the identity experts only:
    the output is the input times their scores, and the correction is not
    in the weights."""
    w, spec = 32, moe(3, 2, 16, 2)
    rnd = _rnd(70)
    P = ff_weights(spec, w, rnd)
    P["correction"] = torch.tensor([-5.0, -5.0, -5.0, 0.5, 0.25])
    for T in (1, 70):
        h = rnd(T, w)
        want = torch.from_numpy(O.moe(h.double().numpy(), np64(P), spec))
        s = torch.softmax(h.double() @ P["router"].double().t(), -1)
        assert torch.allclose(want, h.double() * s[:, 3:].sum(-1, True))
        got = routed_ff(spec, w, P, device, dtype)(h).double().cpu()
        lim = 1e-5 if dtype == torch.float32 else 2e-2
        assert float((got - want).abs().max()) < lim


@pytest.mark.parametrize("device,dtype", [CPU32, GPU32])
def test_router_correction_ties_and_columns(device, dtype):
    """Choice by score + correction, weights without it and not
    renormalised; equal choice scores: the lower index first; logits in
    columns of a wider tensor; more experts than a wave has lanes."""
    E = 130
    z = torch.zeros(2, E + 5)
    z[0, 3 + 7] = z[0, 3 + 100] = z[0, 3 + 9] = 2.0
    z[0, 3 + 64] = 1.0
    corr = torch.zeros(E)
    s = torch.softmax(z[:, 3:3 + E], -1)
    for rep in (1, 60):
        zz = z.repeat(rep, 1).to(device)
        wt, idx = mx.score_router(zz, 3, E, None, 4)
        assert idx[0].tolist() == [7, 9, 100, 64]
        assert torch.allclose(wt[0].cpu(), s[0, [7, 9, 100, 64]], atol=1e-7)
        assert idx[1].tolist() == [0, 1, 2, 3]
        corr[129], corr[9] = 1.0, -1.0
        wt, idx = mx.score_router(zz, 3, E, corr.to(device), 3)
        assert idx[0].tolist() == [129, 7, 100]
        assert torch.allclose(wt[0].cpu(), s[0, [129, 7, 100]], atol=1e-7)
        assert idx[1].tolist() == [129, 0, 1]
        corr.zero_()


# ---------------------------------------------------------- whole model
CFGS = [cfg_mixed, cfg_ones, cfg_wide, cfg_tiles, cfg_odd, cfg_plain]


@pytest.mark.parametrize("cfg_fn", CFGS, ids=lambda f: f.__name__)
@pytest.mark.parametrize("device,dtype", ALL)
def test_whole_prompt_and_layers(tmp_path_factory, device, dtype, cfg_fn):
    """Logits of a whole prompt and the residual after every layer."""
    runner, P, cfg = model(tmp_path_factory, cfg_fn, device, dtype)
    toks = tokens(cfg, 150, 1)
    layers = []
    want = oracle(cfg, P, toks, layers)
    stage = runner.stage
    stage.layer_sums = []
    try:
        got = run_schedule(batcher(runner), toks, [len(toks)])
        sums = [s.cpu() for s in stage.layer_sums]
    finally:
        stage.layer_sums = None
    assert close(got, want, dtype, cfg)
    assert len(sums) == len(cfg["layers"])
    for li, (s, wl) in enumerate(zip(sums, layers)):
        wl = torch.from_numpy(wl)
        err = (s.double() - wl).norm(dim=-1) / wl.norm(dim=-1)
        if dtype == torch.float32:
            assert float(err.max()) < 1e-4, li
        else:
            assert float(err.quantile(0.75)) < 8e-2, li


@pytest.mark.parametrize("cfg_fn", CFGS, ids=lambda f: f.__name__)
@pytest.mark.parametrize("device,dtype", ALL)
def test_portions_and_decoding(tmp_path_factory, device, dtype, cfg_fn):
    """Prefill against token-by-token decoding from the first token, and
    portions of several sizes down to two tokens, cut inside pages, windows
    and chunks; then long decoding across a page border."""
    runner, P, cfg = model(tmp_path_factory, cfg_fn, device, dtype)
    toks = tokens(cfg, 2 * PAGE + 30, 2)
    want = oracle(cfg, P, toks)
    b = batcher(runner, max_ctx=512)
    for cuts in ([], [1, 2, 61, 2, 64, 3, 130], [PAGE, PAGE, 2], [97]):
        got = run_schedule(b, toks if cuts else toks[:70], cuts)
        assert close(got, want[:got.shape[0]], dtype, cfg), cuts


@pytest.mark.parametrize("cfg_fn", [cfg_mixed, cfg_tiles, cfg_plain],
                         ids=lambda f: f.__name__)
@pytest.mark.parametrize("device,dtype", ALL)
def test_mixed_batches_reuse_pages_and_slots(tmp_path_factory, device,
                                             dtype, cfg_fn):
    """Unequal requests in one batch against each alone: portions beside
    single tokens, five requests through three slots and a pool of five
    pages, so pages and state slots are used again; one request is left out
    of steps and goes on later."""
    runner, P, cfg = model(tmp_path_factory, cfg_fn, device, dtype)
    reqs = {"a": tokens(cfg, 150, 3), "b": tokens(cfg, 40, 4),
            "c": tokens(cfg, 131, 5), "d": tokens(cfg, 9, 6),
            "e": tokens(cfg, 200, 7)}
    want = {k: oracle(cfg, P, v) for k, v in reqs.items()}
    b = batcher(runner, max_ctx=256, pool_pages=5, slots=3)
    at = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    plan = [[("a", 100), ("b", 2)], [("a", 1), ("b", 30), ("d", 9)],
            [("a", 49), ("b", 8), ("c", 2)], [("c", 127), ("e", 3)],
            [("c", 2), ("e", 60)], [("e", 2)], [("e", 135)]]
    for step in plan:
        entries, end = [], []
        for rid, n in step:
            t = reqs[rid][at[rid]:at[rid] + n]
            entries.append((rid, t, list(range(n))))
            at[rid] += n
            if at[rid] == len(reqs[rid]):
                end.append(rid)
        out = b.forced_step(entries, end)
        o = 0
        for rid, t, _ in entries:
            got[rid].append(out[o:o + len(t)])
            o += len(t)
    assert b.cache.available_pages() == 5
    for rid in reqs:
        assert at[rid] == len(reqs[rid])
        assert close(torch.cat(got[rid]), want[rid], dtype, cfg), rid


@pytest.mark.parametrize("device,dtype", ALL)
def test_greedy_generation(tmp_path_factory, device, dtype):
    """Greedy continuation through submit() -> scheduler thread and
    through PipelineRunner.generate equals the oracle's, token for token
    (fp32; in bf16 a near-tie may flip, so only the first tokens are
    held)."""
    runner, P, cfg = model(tmp_path_factory, cfg_plain, device, dtype)
    prompts = [tokens(cfg, 21, 8), tokens(cfg, 50, 9)]
    n_new = 12
    want = []
    for p in prompts:
        seq = list(p)
        for _ in range(n_new):
            seq.append(int(oracle(cfg, P, seq)[-1].argmax()))
        want.append(seq[len(p):])
    keep = n_new if dtype == torch.float32 else 2
    b = batcher(runner, max_ctx=256).start()
    try:
        rs = [b.submit(torch.tensor(p), max_new_tokens=n_new,
                       temperature=0.0) for p in prompts]
        outs = [r.result(timeout=120) for r in rs]
    finally:
        b.stop()
    for o, wv in zip(outs, want):
        assert list(o)[:keep] == wv[:keep]
    out = runner.generate(torch.tensor([prompts[0]]),
                          SamplingParams(temperature=0.0,
                                         max_new_tokens=n_new))
    assert out[0].tolist()[:keep] == want[0][:keep]


@pytest.mark.parametrize("device,dtype", ALL)
def test_trace_runner(tmp_path_factory, tmp_path, device, dtype):
    """bin/trace_run as a user starts it: steps on standard input, three
    requests through a small pool (the first ends before the third starts),
    portions beside single tokens, logits files for the wanted places only,
    a line per step."""
    import subprocess
    import sys
    _, P, cfg = model(tmp_path_factory, cfg_plain, "cpu", torch.float32)
    d = _CACHE[("cfg_plain", 0)][0]
    reqs = {"a": tokens(cfg, 100, 11), "b": tokens(cfg, 130, 12),
            "c": tokens(cfg, 90, 13)}
    want = {k: oracle(cfg, P, v) for k, v in reqs.items()}
    plan = [[("a", 60, [0, 59])], [("a", 39, [38]), ("b", 2, [])],
            [("a", 1, [0]), ("b", 127, [5, 126])], [("b", 1, [0]),
                                                    ("c", 88, [87])],
            [("c", 1, [])], [("c", 1, [0])]]
    at = {k: 0 for k in reqs}
    lines, rows = [], []
    for n, step in enumerate(plan):
        entries, end, asked = [], [], []
        for rid, cnt, wanted in step:
            entries.append({"id": rid, "want": wanted,
                            "tokens": reqs[rid][at[rid]:at[rid] + cnt]})
            asked += [(rid, at[rid] + k) for k in wanted]
            at[rid] += cnt
            if at[rid] == len(reqs[rid]):
                end.append(rid)
        lines.append(json.dumps({"step": n, "entries": entries, "end": end}))
        rows.append(asked)
    exe = os.path.join(os.path.dirname(os.path.dirname(
        os.path.abspath(__file__))), "bin", "trace_run")
    out = str(tmp_path / "out")
    r = subprocess.run(
        [sys.executable, exe, "--model", d, "--out", out, "--device", device,
         "--dtype", "float32" if dtype == torch.float32 else "bfloat16",
         "--max-tokens", "320"], input="\n".join(lines) + "\n",
        capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    done = [ln for ln in r.stdout.splitlines() if ln.startswith("done ")]
    assert done == ["done %d" % n for n in range(len(plan))]
    for n, asked in enumerate(rows):
        f = os.path.join(out, "%d.f32" % n)
        if not asked:
            assert not os.path.exists(f)
            continue
        got = torch.from_numpy(np.fromfile(f, dtype="<f4").reshape(
            len(asked), cfg["vocab"]).copy())
        ref = torch.stack([want[rid][p] for rid, p in asked])
        assert close(got, ref, dtype, cfg), n


def random_cfg(rng):
    """A random model of the design: 2-5 layers in any order, head sizes
    below, at and above a wave's 64 columns, not all multiples of 8."""
    w = rng.choice([24, 40, 64, 96, 128])
    layers = []
    for _ in range(rng.randint(2, 5)):
        if rng.random() < 0.5:
            m = ml(rng.randint(1, 5), rng.choice([6, 8, 16, 24, 48, 130]),
                   rng.choice([5, 8, 16, 48, 96, 140]),
                   rng.choice([2.0, 8.0, 20.0]),
                   rng.choice(["mlstm", "mlstm_2"]))
        else:
            G, g = rng.randint(1, 3), rng.randint(1, 2)
            D = rng.choice([6, 8, 24, 48, 96])
            m = par(win(G * rng.choice([1, 2, 3, 4]), G, D,
                        rng.choice([6, 16, 48, 96, 130]),
                        2 * rng.randint(1, D // 2),
                        rng.choice([1, 7, 33, 64, 100, 1000]),
                        rng.choice([100.0, 10000.0])),
                    delta(g * rng.choice([1, 2, 3]), g,
                          rng.choice([5, 8, 16, 32, 48, 80, 130]),
                          rng.choice([6, 16, 33, 64, 100]),
                          rng.randint(1, 6), rng.choice([1, 4, 9, 24]),
                          rng.choice([1, 4, 9, 24])),
                    rng.choice([0.2, 0.7, 1.5]), rng.choice([0.2, 0.7, 1.5]))
        E, ident = rng.choice([2, 5, 9]), rng.choice([0, 1, 4])
        mlp = rng.choice([
            None, dense(rng.choice([16, 50, 128])),
            moe(E, rng.choice([1, 2, 3]) if E + ident > 2 else 1,
                rng.choice([8, 32, 50]), ident, rng.choice([0.5, 2.0, 7.0]),
                rng.choice([None, (10, 0.7), (64, 3.0)]))])
        layers.append(layer(m, mlp))
    return model_cfg(layers, rng.choice([37, 64, 200]), w,
                     rng.choice([0.3, 0.8, 1.0]),
                     rng.choice([2, 61, 1000]), rng.choice([1, 40, 1009]),
                     rng.choice([1, 23, 999]), rng.choice([1e-5, 1e-6]))


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8])
@pytest.mark.parametrize("device,dtype", ALL)
def test_random_configurations(tmp_path, device, dtype, seed):
    """Other sizes, orders and constants: whole, portioned and decoded
    against the oracle."""
    cfg = random_cfg(random.Random(seed))
    P = make_weights(cfg, seed)
    d = str(tmp_path / "m")
    write_checkpoint(d, cfg, P)
    toks = tokens(cfg, 140, seed)
    want = oracle(cfg, P, toks)
    runner = PipelineRunner(plan_for_world(d, 1), 0, 1,
                            device=torch.device(device), init="checkpoint",
                            ckpt_dir=d, dtype=dtype)
    for cuts in ([140], [90, 2, 3, 40]):
        got = run_schedule(batcher(runner, max_ctx=256), toks, cuts)
        if dtype == torch.float32:
            e = rel_err(got, want)
            assert float(e.median()) < 2e-5 and float(e.max()) < 1e-3, \
                (seed, cuts, float(e.median()), float(e.max()))
        else:
            assert close(got, want, dtype, cfg), (seed, cuts)


# --------------------------------------------------- configuration, loader
def test_registry_and_strict_loading(tmp_path):
    from tensorlink_amd.models.configs import ModelConfig, get_config
    from tensorlink_amd.models.lunadra import LunadraConfig
    cfg = cfg_mixed()
    c = ModelConfig.from_hf_config(cfg)
    assert isinstance(c, LunadraConfig) and c.residual_mult == 0.6
    assert c.num_hidden_layers == 4 and c.bigram_buckets == 101
    c2 = LunadraConfig.from_dict(json.loads(c.to_json()))
    assert c2.layer_specs == c.layer_specs and c2.bigram_mul_prev == 31
    for fn in CFGS:
        cf, Pf = fn(), make_weights(fn())
        assert ModelConfig.from_hf_config(cf).param_count() == \
            sum(v.numel() for v in Pf.values()), fn.__name__
    P = make_weights(cfg)
    # the ranks come from the checkpoint when config.json has none
    d = str(tmp_path / "ok")
    write_checkpoint(d, cfg, P)
    got = [lc["mixer"].get("right", {}) for lc in get_config(d).layer_specs]
    assert [(m.get("decay_rank"), m.get("gate_rank")) for m in got] == \
        [(None, None), (6, 5), (None, None), (6, 5)]
    with pytest.raises(KeyError):
        ModelConfig.from_hf_config(file_config(cfg))       # no checkpoint
    for path, value in ((("layers", 0, "type"), "conv"),
                        (("layers", 0, "mlp", "kind"), "conv"),
                        (("layers", 1, "mixer", "left", "kv_heads"), 3),
                        (("layers", 1, "mixer", "right", "kv_heads"), 3),
                        (("layers", 1, "mixer", "left", "rot", "dims"), 14),
                        (("layers", 0, "mlp", "router", "top"), 8)):
        bad = json.loads(json.dumps(cfg))
        node = bad
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = value
        with pytest.raises(KeyError):
            ModelConfig.from_hf_config(bad)
    for n, (drop, extra) in enumerate((
            ("l0.mix.g", None), ("l0.mix.f.b", None), ("bigram", None),
            ("l0.mlp.e4.up", None), ("l0.mlp.correction", None),
            ("l1.mix.right.a1", None), ("l1.mix.right.k.conv", None),
            ("l1.mix.left.o", None), (None, "l1.mix.right.b.b"),
            (None, "l2.norm2"))):
        Q = dict(P)
        if drop:
            del Q[drop]
        if extra:
            Q[extra] = torch.zeros(3)
        d = str(tmp_path / f"x{n}")
        write_checkpoint(d, cfg, Q)
        with pytest.raises(KeyError):
            PipelineRunner(plan_for_world(d, 1), 0, 1,
                           device=torch.device("cpu"), init="checkpoint",
                           ckpt_dir=d, dtype=torch.float32)


def test_optional_parts_may_be_absent(tmp_path):
    """No mask (plain causal), no rotation, no identity experts and no
    shared expert in config.json."""
    cfg = cfg_mixed()
    del cfg["layers"][1]["mixer"]["left"]["mask"]
    del cfg["layers"][3]["mixer"]["left"]["rot"]
    P = make_weights(cfg, 5)
    ref = json.loads(json.dumps(cfg))
    ref["layers"][1]["mixer"]["left"]["mask"] = {"size": 10 ** 6}
    ref["layers"][3]["mixer"]["left"]["rot"] = {"dims": 0, "base": 1.0}
    d = str(tmp_path / "m")
    write_checkpoint(d, cfg, P)
    runner = PipelineRunner(plan_for_world(d, 1), 0, 1,
                            device=torch.device("cpu"), init="checkpoint",
                            ckpt_dir=d, dtype=torch.float32)
    toks = tokens(cfg, 60, 3)
    got = run_schedule(batcher(runner), toks, [40, 2])
    assert close(got, oracle(ref, P, toks), torch.float32, cfg)


def test_random_init_runs():
    """init='random' (benchmarks) gives finite logits."""
    from tensorlink_amd.models.configs import ModelConfig
    c = ModelConfig.from_hf_config(cfg_wide())
    runner = PipelineRunner(plan_for_world(c, 1), 0, 1,
                            device=torch.device("cpu"), init="random",
                            dtype=torch.float32)
    out = run_schedule(batcher(runner), tokens(cfg_wide(), 20, 1), [17])
    assert torch.isfinite(out).all() and float(out.std()) > 0
