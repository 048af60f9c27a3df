"""Kikurax (sigmoid attention beside a gated delta rule, Mamba-2 scans, rotary
attention with blended values) against the plain oracle in kikurax_oracle.py.

Every test builds its own small configuration and random checkpoint, loads
it through the engine's own entry points (config reader, weight loader,
scheduler, cache and state managers) and compares logits with the oracle.
The scenarios run on the CPU (torch reference ops) and, marked ``gpu``, on
the HIP kernels in fp32 (sharp) and bf16.

Expert routing is a discrete choice: a bf16 run rounds the router's input,
so a near-tie may fall the other way than in the float64 oracle. Whole-model
bf16 scenarios therefore use mixtures in which every expert is chosen (the
logits still weigh the outputs); the choice itself is checked in fp32 at
model level and at op level, where the oracle sees the same inputs.
"""

from __future__ import annotations

import json
import math

import pytest
import torch

import kikurax_oracle as oracle
from llmq_amd import ops
from llmq_amd.engine.config import EngineConfig
from llmq_amd.engine.engine import LLMEngine
from llmq_amd.engine.sampling_params import SamplingParams


# --------------------------------------------------------------- fixtures --

def moe_cfg(experts=5, top=2, ff=24, limit=1.2):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "top": top}}


def attn(heads=4, kv_heads=2, dim=16, vdim=12, rot_dims=8, base=5000.0, scale=0.8, softcap=6.0,
         v_mix=True, scaling=(4.0, 1.0, 3.0, 40), mlp=None):
    rot = {"base": base, "dims": rot_dims}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
        "softcap": softcap, "v_mix": v_mix, "rot": rot}}


def par(heads=4, kv_heads=2, dim=8, vdim=12, scale=0.4, coef=0.5, every=9, conv=3, dheads=4,
        dkv=2, ddim=8, dvdim=12, mlp=None):
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                 "q_temp": {"coef": coef, "every": every}},
        "right": {"heads": dheads, "kv_heads": dkv, "dim": ddim, "vdim": dvdim, "conv": conv}}}


def ssd(heads=4, vdim=8, state=12, groups=2, norm_groups=2, conv=4, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {
        "heads": heads, "vdim": vdim, "state": state, "groups": groups,
        "norm_groups": norm_groups, "conv": conv}}


def make_config(layers, width=48, vocab=128, eps=1e-5, groups=3, emb=3.0):
    return {"architecture": "Kikurax", "embedding": {"scale": emb}, "layers": layers,
            "norm": {"eps": eps, "groups": groups}, "vocab": vocab, "width": width}


def make_tensors(cfg, seed=0, ranks=(10, 6)):
    g = torch.Generator().manual_seed(seed)

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).to(torch.bfloat16)

    def lin(out, inn, gain=1.0):
        return rnd(out, inn, std=gain / math.sqrt(inn))

    W, V = cfg["width"], cfg["vocab"]
    t = {"embed": rnd(V, W, std=0.5), "final.norm": rnd(W, std=0.1, mean=0.9)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        t[p + "norm1"] = rnd(W, std=0.1, mean=1.1)
        if layer["type"] == "attention":
            H, G, D, DV = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for name, rows in (("q", H * D), ("k", G * D), ("v", G * DV)):
                t[f"{p}mix.{name}"], t[f"{p}mix.{name}.b"] = lin(rows, W, 2.0), rnd(rows, std=0.4)
            t[p + "mix.temp"] = rnd(H, std=0.4, mean=1.3)
            t[p + "mix.vmix"] = torch.tensor(0.3 + 0.1 * (i % 4)).to(torch.bfloat16)
            t[p + "mix.o"] = lin(W, H * DV, 2.0)
        elif layer["type"] == "mamba2":
            H, DV, N, G, K = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
            inner, ch = H * DV, H * DV + 2 * G * N
            t[p + "mix.in"] = lin(inner + ch + H, W, 1.5)
            t[p + "mix.conv"] = rnd(ch, K, std=0.9 / math.sqrt(K))
            t[p + "mix.conv.b"] = rnd(ch, std=0.3)
            t[p + "mix.dt_bias"] = rnd(H, std=0.7, mean=-1.0)
            t[p + "mix.A_log"] = rnd(H, std=0.7, mean=-1.0)
            t[p + "mix.D"] = rnd(H, std=0.3, mean=0.7)
            t[p + "mix.norm"] = rnd(inner, std=0.1, mean=1.0)
            t[p + "mix.o"] = lin(W, inner, 1.5)
        else:
            a, r = m["left"], m["right"]
            H, G, D, DV = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            lf, rt = p + "mix.left.", p + "mix.right."
            for name, rows in (("q", H * D), ("k", G * D), ("v", G * DV), ("g", H * DV)):
                t[lf + name] = lin(rows, W, 2.0)
            t[lf + "pb"] = rnd(H, std=0.6, mean=-2.0)
            t[lf + "o"], t[lf + "out"] = lin(W, H * DV, 1.5), rnd(W, std=0.1, mean=0.9)
            H, G, D, DV, K = r["heads"], r["kv_heads"], r["dim"], r["vdim"], r["conv"]
            for name, rows in (("q", G * D), ("k", G * D), ("v", H * DV)):
                t[rt + name] = lin(rows, W, 2.0)
                t[rt + name + ".conv"] = rnd(rows, K, std=0.9 / math.sqrt(K))
            t[rt + "b"], t[rt + "A_log"] = lin(H, W, 1.5), rnd(H, std=0.7, mean=-1.0)
            t[rt + "a1"], t[rt + "a2"] = lin(ranks[0], W, 1.0), lin(H * D, ranks[0], 1.0)
            t[rt + "g1"], t[rt + "g2"] = lin(ranks[1], W, 1.5), lin(H * DV, ranks[1], 1.5)
            t[rt + "dt_bias"] = rnd(H * D, std=0.7, mean=-1.0)
            t[rt + "norm"] = rnd(DV, std=0.1, mean=1.0)
            t[rt + "o"], t[rt + "out"] = lin(W, H * DV, 1.5), rnd(W, std=0.1, mean=0.8)
        mlp = layer["mlp"]
        if mlp is None:
            continue
        t[p + "norm2"] = rnd(W, std=0.1, mean=1.0)
        E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        t[p + "mlp.router"], t[p + "mlp.router.b"] = lin(E, W, 2.0), rnd(E, std=0.5)
        for e in range(E):
            ep = f"{p}mlp.e{e}."
            t[ep + "gate"], t[ep + "up"] = lin(ff, W, 1.5), lin(ff, W, 1.5)
            t[ep + "down"] = lin(W, ff, 1.5)
    return t


def write_checkpoint(path, cfg, tensors):
    from safetensors.torch import save_file

    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(path / "model.safetensors"))
    return str(path)


def mixed_layers(route):
    """Every switch at once: the three mixers, grouped and ungrouped heads,
    q/k size != v size, partial rotation with and without scaled frequencies,
    value blending that skips a layer, layers with and without experts."""
    moe = (lambda **kw: moe_cfg(experts=5, top=2, **kw)) if route else \
        (lambda **kw: moe_cfg(experts=3, top=3, **kw))
    return [
        attn(heads=2, kv_heads=1, dim=12, vdim=20, rot_dims=12, scale=0.3, v_mix=False, scaling=None),
        par(mlp=moe()),
        attn(scale=0.4, mlp=moe(limit=0.7)),
        ssd(mlp=moe(ff=17)),
        par(heads=3, kv_heads=3, dim=16, vdim=8, coef=0.2, every=16, conv=4, dheads=3, dkv=3,
            ddim=20, dvdim=4),
        attn(heads=6, kv_heads=2, dim=8, vdim=12, rot_dims=4, softcap=2.5, base=100.0),
        ssd(heads=6, vdim=12, state=5, groups=3, norm_groups=1, conv=2),
        attn(heads=2, kv_heads=2, dim=24, vdim=12, rot_dims=24, scale=0.2, softcap=30.0, mlp=moe()),
    ]


def tokens_for(n, vocab, seed):
    g = torch.Generator().manual_seed(4000 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


DEVICES = [
    pytest.param(("cpu", "float32"), id="cpu"),
    pytest.param(("cuda", "float32"), id="hip-fp32", marks=pytest.mark.gpu),
    pytest.param(("cuda", "bfloat16"), id="hip-bf16", marks=pytest.mark.gpu),
]


def make_engine(path, target, blocks=64, block_size=16, max_seqs=4, prefill_budget=4096,
                max_len=1024):
    device, dtype = target
    return LLMEngine(EngineConfig(
        model=path, device=device, dtype=dtype, max_num_seqs=max_seqs, max_model_len=max_len,
        num_kv_blocks=blocks, kv_block_size=block_size, max_prefill_tokens=prefill_budget))


def assert_close(got, want, target, what=""):
    """Relative rms error per row: fp32 is the sharp comparison; bf16 rounds
    every GEMM input and output of a deep stack and has to stay at rounding
    level (nine rows in ten, and the median: a memory read-out is divided by
    its own root mean square, so a row whose query meets little that was
    written has its direction decided by rounding)."""
    got, want = got.double().cpu(), want.double()
    err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()
    if target[1] == "bfloat16":
        worst = float(err.quantile(0.9)) if err.numel() >= 10 else float(err.min())
        mean, lim_worst, lim_mean = float(err.median()), 1e-1, 4e-2
    else:
        worst, mean, lim_worst, lim_mean = float(err.max()), float(err.mean()), 2e-4, 5e-5
    assert worst < lim_worst, f"{what}: worst row error {worst:.3e} at row {int(err.argmax())}"
    assert mean < lim_mean, f"{what}: mean row error {mean:.3e}"


def replay(engine, rid, toks, cuts, end=True):
    """One request alone, cut into the given portion sizes; all logits."""
    out, at = [], 0
    for n in cuts:
        last = at + n == len(toks)
        out.append(engine.replay_step(
            [{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}],
            end=[rid] if (last and end) else []))
        at += n
    assert at == len(toks)
    return torch.cat(out)


def f64(tensors):
    return {k: v.double() for k, v in tensors.items()}


_MODELS = {}


@pytest.fixture(scope="module")
def mixed_model(tmp_path_factory):
    """(config, tensors, path) of the all-switches model; bf16 targets get the
    variant in which every expert is chosen."""
    def get(target):
        route = target[1] != "bfloat16"
        if route not in _MODELS:
            cfg = make_config(mixed_layers(route))
            tensors = make_tensors(cfg, seed=11)
            path = write_checkpoint(tmp_path_factory.mktemp("kx") / "m", cfg, tensors)
            _MODELS[route] = (cfg, f64(tensors), path)
        return _MODELS[route]
    return get


_WANT = {}


def oracle_logits(cfg, tensors, toks):
    key = (id(tensors), tuple(toks))
    if key not in _WANT:
        _WANT[key] = oracle.forward(cfg, tensors, toks)
    return _WANT[key]


def dev_dtype(target):
    return target[0], (torch.bfloat16 if target[1] == "bfloat16" else torch.float32)


# ------------------------------------------------------ config and layout --

def test_config_reader_takes_everything_from_config(tmp_path):
    from llmq_amd.engine.model_specs import resolve_spec

    cfg = make_config(mixed_layers(True))
    tensors = make_tensors(cfg)
    path = write_checkpoint(tmp_path / "m", cfg, tensors)
    spec = resolve_spec(path)
    assert spec.family == "kikurax" and spec.num_layers == 8 and spec.hidden_size == 48
    assert (spec.rms_eps, spec.norm_groups, spec.embedding_scale) == (1e-5, 3, 3.0)
    assert [ls.mixer.kind for ls in spec.layers] == [
        "attention", "parallel", "attention", "mamba2", "parallel", "attention", "mamba2",
        "attention"]
    a = spec.layers[2].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.softcap, a.v_mix) == \
        (4, 2, 16, 12, 0.4, 6.0, True)
    assert (a.rot.base, a.rot.dims) == (5000.0, 8)
    sc = a.rot_scaling
    assert (sc.factor, sc.low, sc.high, sc.original) == (4.0, 1.0, 3.0, 40.0)
    assert spec.layers[0].mixer.rot_scaling is None and spec.first_v_mix() == 2
    lt, rt = spec.layers[4].mixer.left, spec.layers[4].mixer.right
    assert (lt.heads, lt.kv_heads, lt.dim, lt.vdim, lt.scale, lt.temp_coef, lt.temp_every) == \
        (3, 3, 16, 8, 0.4, 0.2, 16)
    assert (rt.heads, rt.kv_heads, rt.dim, rt.vdim, rt.conv, rt.decay_rank, rt.gate_rank) == \
        (3, 3, 20, 4, 4, 10, 6)
    m = spec.layers[6].mixer
    assert (m.heads, m.vdim, m.state, m.groups, m.norm_groups, m.conv, m.inner) == \
        (6, 12, 5, 3, 1, 2, 72)
    e = spec.layers[2].moe
    assert (e.experts, e.top, e.ff, e.limit) == (5, 2, 24, 0.7)
    assert spec.layers[0].moe is None and spec.layers[3].moe.ff == 17
    # the checkpoint holds a blend factor for the unblended layer too
    assert spec.param_count() == sum(v.numel() for v in tensors.values()) - 1
    eng = make_engine(path, ("cpu", "float32"))
    assert eng.kv_cache.k[3] is None and eng.state_cache.state[2] is None
    assert eng.kv_cache.k[1].shape[1:] == (2, 16, 8) and eng.kv_cache.v[1].shape[1:] == (2, 16, 12)
    S, tail = eng.state_cache.state[1]
    assert S.shape[1:] == (4, 8, 12) and tail.shape[1:] == (2, 80)
    S, tail = eng.state_cache.state[3]
    assert S.shape[1:] == (4, 12, 8) and tail.shape[1:] == (3, 80)
    for bad in (dict(attn(), type="lstm"), ssd(heads=4, groups=3), ssd(norm_groups=5),
                attn(heads=4, kv_heads=3), attn(mlp=moe_cfg(experts=2, top=3))):
        with pytest.raises(ValueError):
            resolve_spec(write_checkpoint(tmp_path / "bad", make_config([bad]), {}))
    with pytest.raises(ValueError):      # blended values of different shapes
        resolve_spec(write_checkpoint(tmp_path / "bad", make_config([attn(), attn(vdim=8)]), {}))


def test_a_missing_tensor_is_refused(tmp_path):
    cfg = make_config([par(), attn()])
    tensors = make_tensors(cfg)
    del tensors["l0.mix.right.k.conv"]
    with pytest.raises(KeyError):
        make_engine(write_checkpoint(tmp_path / "m", cfg, tensors), ("cpu", "float32"))


@pytest.mark.parametrize("scaling", [None, (8.0, 1.0, 4.0, 64), (3.0, 2.0, 2.0, 100),
                                     (4.0, 1.0, 4.0, 8192), (2.0, 1.0, 8.0, 1)])
def test_scaled_frequencies(scaling):
    """Long waves slowed, short waves kept, a blend between; a context so long
    or so short that one branch takes every frequency; an empty blend range."""
    from llmq_amd.engine.model_specs import RotaryScaling
    from llmq_amd.engine.models.kikurax import scaled_inv_freq

    rot = attn(rot_dims=16, scaling=scaling)["mixer"]["rot"]
    got = scaled_inv_freq(rot["base"], rot["dims"], RotaryScaling(*map(float, scaling)) if scaling
                          else None)
    want = torch.tensor(oracle.frequencies(rot), dtype=torch.float64)
    assert ((got.double() - want).abs() / want).max() < 1e-6


# ------------------------------------------------------ mechanisms alone --

@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("layers,kw", [
    ([attn()], {}),
    ([attn(heads=3, kv_heads=3, dim=8, vdim=8, rot_dims=8, softcap=50.0, scaling=None)], {"groups": 1}),
    ([attn(heads=8, kv_heads=1, dim=16, vdim=24, rot_dims=2, scale=2.0, softcap=1.0)], {}),
    ([attn(v_mix=False), attn(), attn(), attn(v_mix=False), attn()], {}),
    ([attn(v_mix=False), attn(v_mix=False)], {"emb": 1.0}),
    ([attn(heads=1, kv_heads=1, dim=2, vdim=1, rot_dims=2)], {}),
    ([par()], {}),
    ([par(heads=6, kv_heads=1, dim=20, vdim=4, coef=0.0, every=1, conv=1, dheads=2, dkv=1, ddim=32,
          dvdim=32)], {"groups": 1}),
    ([par(heads=1, kv_heads=1, dim=32, vdim=32, every=1, coef=1.0, dheads=1, dkv=1, ddim=4, dvdim=70,
          conv=8)], {}),
    ([par(heads=5, kv_heads=5, scale=1.5, every=37, dheads=6, dkv=3, ddim=40, dvdim=20, conv=2)],
     {"groups": 6}),
    ([ssd()], {}),
    ([ssd(heads=1, vdim=24, state=1, groups=1, norm_groups=1, conv=1)], {"groups": 1}),
    ([ssd(heads=6, vdim=5, state=33, groups=6, norm_groups=3, conv=6)], {}),
    ([ssd(heads=3, vdim=40, state=70, groups=1, norm_groups=8, conv=3)], {}),
    ([attn(mlp=moe_cfg(experts=4, top=4))], {}),
    ([ssd(mlp=moe_cfg(experts=1, top=1, ff=7, limit=0.3))], {}),
    ([par(mlp=moe_cfg(experts=2, top=2, ff=40, limit=100.0))], {}),
], ids=["attn", "attn-loose", "attn-one-kv-head-tight-cap", "blend-skips-layers", "no-blend",
        "attn-ones", "pair", "pair-no-temp-no-conv", "pair-ones", "pair-odd", "ssd", "ssd-ones",
        "ssd-groups-equal-heads", "ssd-wide", "experts-all", "expert-single", "experts-loose"])
def test_mechanism_alone(tmp_path, target, layers, kw):
    cfg = make_config(layers, **kw)
    tensors = make_tensors(cfg, seed=3)
    path = write_checkpoint(tmp_path / "m", cfg, tensors)
    toks = tokens_for(37, cfg["vocab"], 1)
    eng = make_engine(path, target)
    eng.model.taps = []
    got = replay(eng, "a", toks, [37])
    taps = []
    want = oracle.forward(cfg, f64(tensors), toks, taps)
    for i, (g, w) in enumerate(zip(eng.model.taps, taps)):
        assert_close(g, w, target, f"stream after layer {i}")
    assert_close(got, want, target, "logits")
    eng.model.taps = None
    assert_close(replay(eng, "b", toks, [5, 1, 2, 20, 1, 1, 7]), want, target, "portions")


@pytest.mark.parametrize("target", DEVICES)
def test_sizes_that_fit_no_vector_width(tmp_path, target):
    layers = [par(heads=3, kv_heads=1, dim=6, vdim=10, conv=3, dheads=3, dkv=1, ddim=5, dvdim=7,
                  mlp=moe_cfg(experts=3, top=3, ff=9)),
              ssd(heads=3, vdim=7, state=9, groups=3, norm_groups=7, conv=5),
              attn(heads=3, kv_heads=1, dim=10, vdim=6, rot_dims=6),
              attn(heads=3, kv_heads=1, dim=10, vdim=6, rot_dims=10, mlp=moe_cfg(experts=2, top=2, ff=5))]
    cfg = make_config(layers, width=27, vocab=61, groups=3)
    tensors = make_tensors(cfg, seed=5, ranks=(3, 5))
    path = write_checkpoint(tmp_path / "m", cfg, tensors)
    toks = tokens_for(41, 61, 2)
    want = oracle.forward(cfg, f64(tensors), toks)
    eng = make_engine(path, target)
    assert_close(replay(eng, "a", toks, [41]), want, target, "whole")
    assert_close(replay(eng, "b", toks, [7, 1, 1, 30, 2]), want, target, "portions")


@pytest.mark.parametrize("target", DEVICES[:2])
@pytest.mark.parametrize("experts,top", [(5, 1), (6, 3), (2, 1), (13, 4), (9, 8)])
def test_expert_choice_in_the_model(tmp_path, target, experts, top):
    cfg = make_config([attn(mlp=moe_cfg(experts=experts, top=top)),
                       ssd(mlp=moe_cfg(experts=experts, top=top, ff=10))])
    tensors = make_tensors(cfg, seed=experts * 10 + top)
    path = write_checkpoint(tmp_path / "m", cfg, tensors)
    toks = tokens_for(33, cfg["vocab"], 6)
    assert_close(replay(make_engine(path, target), "a", toks, [30, 1, 1, 1]),
                 oracle.forward(cfg, f64(tensors), toks), target, f"{experts} experts, top {top}")


@pytest.mark.parametrize("target", DEVICES)
def test_wider_model_with_other_sizes(tmp_path, target):
    """Head sizes that take the 16-byte paths and the matrix-core tiles, more
    keys than one tile, whole, cut and in a batch."""
    layers = [par(heads=6, kv_heads=2, dim=32, vdim=40, scale=0.2, every=50, conv=4, dheads=4, dkv=2,
                  ddim=48, dvdim=64, mlp=moe_cfg(experts=3, top=3, ff=64)),
              attn(heads=8, kv_heads=1, dim=40, vdim=32, rot_dims=32, scale=0.3, softcap=20.0,
                   scaling=(8.0, 1.0, 4.0, 128)),
              ssd(heads=8, vdim=16, state=48, groups=2, norm_groups=4, conv=4,
                  mlp=moe_cfg(experts=2, top=2, ff=80)),
              attn(heads=8, kv_heads=1, dim=64, vdim=32, rot_dims=16, softcap=9.0)]
    cfg = make_config(layers, width=160, vocab=300, groups=5)
    tensors = make_tensors(cfg, seed=9, ranks=(16, 24))
    path = write_checkpoint(tmp_path / "m", cfg, tensors)
    t64 = f64(tensors)
    a, b = tokens_for(200, 300, 80), tokens_for(90, 300, 81)
    want_a, want_b = oracle.forward(cfg, t64, a), oracle.forward(cfg, t64, b)
    eng = make_engine(path, target, blocks=24)
    assert_close(replay(eng, "w", a, [200]), want_a, target, "whole")
    assert_close(replay(eng, "c", a, [63, 2, 65, 1, 1, 1, 1, 30, 36]), want_a, target, "cut")
    # b's portions beside a's single tokens, then b's single tokens beside a's portion
    got_a = [eng.replay_step([{"id": "a", "tokens": a[:120], "want": list(range(120))}])]
    got_b = []
    for k in range(40):
        out = eng.replay_step([{"id": "a", "tokens": [a[120 + k]], "want": [0]},
                               {"id": "b", "tokens": b[2 * k:2 * k + 2], "want": [0, 1]}])
        got_a.append(out[:1])
        got_b.append(out[1:])
    out = eng.replay_step([{"id": "b", "tokens": [b[80]], "want": [0]},
                           {"id": "a", "tokens": a[160:], "want": list(range(40))}])
    got_b.append(out[:1])
    got_a.append(out[1:])
    got_b.append(eng.replay_step([{"id": "b", "tokens": b[81:], "want": list(range(9))}],
                                 end=["a", "b"]))
    assert_close(torch.cat(got_a), want_a, target, "a in the batch")
    assert_close(torch.cat(got_b), want_b, target, "b in the batch")
    assert eng.allocator.num_free == 24


# ------------------------------------------- schedules: cuts, batches, reuse --

@pytest.mark.parametrize("target", DEVICES)
def test_prefill_equals_token_by_token(mixed_model, target):
    cfg, tensors, path = mixed_model(target)
    toks = tokens_for(90, cfg["vocab"], 2)
    want = oracle_logits(cfg, tensors, toks)
    eng = make_engine(path, target)
    assert_close(replay(eng, "w", toks, [90]), want, target, "whole prompt")
    assert_close(replay(eng, "d", toks, [1] * 90), want, target, "token by token")
    assert eng.allocator.num_free == eng.allocator.num_blocks
    assert eng.slot_allocator.num_free == 4


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("cuts", [
    [2] * 45,
    [1, 2, 3, 5, 8, 13, 21, 34, 3],
    [16, 16, 16, 16, 16, 10],                  # at page borders
    [15, 2, 15, 17, 31, 1, 1, 8],              # around page borders
    [64, 1, 1, 1, 1, 1, 1, 1, 1, 1, 17],
    [3, 87],
], ids=["twos", "growing", "pages", "around-pages", "decode-then-portion", "short-first"])
def test_portions(mixed_model, target, cuts):
    cfg, tensors, path = mixed_model(target)
    toks = tokens_for(90, cfg["vocab"], 3)
    want = oracle_logits(cfg, tensors, toks)
    eng = make_engine(path, target)
    assert_close(replay(eng, "c", toks, cuts), want, target, f"cuts {cuts}")


@pytest.mark.parametrize("target", DEVICES)
def test_mixed_batches_equal_alone_and_reuse(mixed_model, target):
    """Six unequal requests through four slots and a pool that cannot hold
    them all at once: portions beside single tokens, requests that pause,
    blocks and slots handed on to later requests."""
    cfg, tensors, path = mixed_model(target)
    lens = {"a": 70, "b": 9, "c": 41, "d": 130, "e": 25, "f": 3}
    toks = {r: tokens_for(n, cfg["vocab"], 10 + i) for i, (r, n) in enumerate(lens.items())}
    want = {r: oracle_logits(cfg, tensors, t) for r, t in toks.items()}
    eng = make_engine(path, target, blocks=14, block_size=16)
    at = {r: 0 for r in lens}
    got = {r: [] for r in lens}
    plan = [
        {"a": 33, "b": 2, "c": 17},
        {"a": 1, "b": 1, "c": 24, "d": 40},
        {"a": 1, "b": 6, "d": 2},              # c pauses at its end; b ends
        {"a": 35, "d": 1, "e": 25},            # e takes b's slot and blocks
        {"d": 1},
        {"d": 86, "f": 3},                     # a, c, e ended; f reuses
    ]
    ends = [[], [], ["b"], ["a", "e"], ["c"], ["d", "f"]]
    slots_seen = set()
    for step, end in zip(plan, ends):
        entries = [{"id": r, "tokens": toks[r][at[r]:at[r] + n], "want": list(range(n))}
                   for r, n in step.items()]
        out = eng.replay_step(entries, end=[])
        for s in eng._seqs.values():
            slots_seen.add(s.state_slot)
        eng.replay_step([], end=end)
        k = 0
        for ent in entries:
            n = len(ent["tokens"])
            got[ent["id"]].append(out[k:k + n])
            at[ent["id"]] += n
            k += n
    assert at == lens
    assert slots_seen <= {0, 1, 2, 3}
    for r in lens:
        assert_close(torch.cat(got[r]), want[r], target, f"request {r}")
    assert eng.allocator.num_free == 14 and eng.slot_allocator.num_free == 4


@pytest.mark.parametrize("target", DEVICES)
def test_stale_pages_and_slots_do_not_leak(mixed_model, target):
    """A request that runs in blocks and a slot another one just left sees
    nothing of it: same logits as in a fresh engine."""
    cfg, tensors, path = mixed_model(target)
    first = tokens_for(64, cfg["vocab"], 30)
    second = tokens_for(50, cfg["vocab"], 31)
    want = oracle_logits(cfg, tensors, second)
    eng = make_engine(path, target, blocks=4, max_seqs=1)
    replay(eng, "x", first, [60, 1, 1, 1, 1])
    assert_close(replay(eng, "y", second, [3, 1, 1, 45]), want, target, "after reuse")


@pytest.mark.parametrize("target", DEVICES)
def test_long_decode_across_pages_and_temperature_steps(mixed_model, target):
    cfg, tensors, path = mixed_model(target)
    toks = tokens_for(5 + 150, cfg["vocab"], 4)
    want = oracle_logits(cfg, tensors, toks)
    eng = make_engine(path, target)
    assert_close(replay(eng, "l", toks, [5] + [1] * 150), want, target, "long decode")


@pytest.mark.parametrize("target", DEVICES)
def test_first_tokens(mixed_model, target):
    """Requests of one to four tokens: nothing before the start, no
    convolution full."""
    cfg, tensors, path = mixed_model(target)
    eng = make_engine(path, target)
    for n in (1, 2, 3, 4):
        toks = tokens_for(n, cfg["vocab"], 70 + n)
        assert_close(replay(eng, f"n{n}", toks, [n]), oracle_logits(cfg, tensors, toks), target,
                     f"{n} tokens")


# ------------------------------------------ edges made visible by design --

def _needle(device, dtype, key_pos, query_pos, decode, H=2, G=1, D=16, DV=8, raw=8.0, page=16,
            **kw):
    """Every key scores 0 and has value 0, but the needle at key_pos: raw
    score `raw`, value 1 in channel 1; behind the query lie stale rows of score
    30 and value 50. The output's channel 1 is then the weight the needle gets.
    Pages are handed out in reverse order."""
    n = query_pos + 1
    nblocks = (n + page - 1) // page
    kc = torch.zeros(nblocks + 2, G, page, D, dtype=dtype)
    vc = torch.zeros(nblocks + 2, G, page, DV, dtype=dtype)
    table = torch.arange(nblocks + 1, 0, -1, dtype=torch.int32).view(1, -1)
    for pos, score, value in [(j, 30.0, 50.0) for j in range(n, nblocks * page)] + \
            [(key_pos, raw, 1.0)]:
        b, o = int(table[0, pos // page]), pos % page
        kc[b, :, o, 0] = score
        vc[b, :, o, 1] = value
    kc, vc, table = kc.to(device), vc.to(device), table.to(device)
    if decode:
        q = torch.zeros(1, H, D, dtype=dtype, device=device)
        q[0, :, 0] = 1.0
        out = ops.window_attn_decode(
            q, kc, vc, DV, table, torch.tensor([n], dtype=torch.int32, device=device), 0, 1.0, **kw)
        return float(out[0, H - 1, 1])
    start = max(0, query_pos - 4)            # a portion whose last row is the query
    rows = query_pos - start + 1
    q = torch.zeros(rows, H, D, dtype=dtype, device=device)
    q[:, :, 0] = 1.0
    out = ops.window_attn_prefill(
        q, kc, vc, DV, table, torch.tensor([0, rows], dtype=torch.int32, device=device),
        torch.tensor([start], dtype=torch.int32, device=device), rows, 0, 1.0, **kw)
    return float(out[-1, H - 1, 1])


def _positions(query_pos):
    return sorted({k for k in (0, 1, 15, 16, 17, 63, 64, 65, query_pos - 64, query_pos - 1, query_pos)
                   if 0 <= k <= query_pos})


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("decode", [False, True], ids=["portion", "single"])
@pytest.mark.parametrize("H,G,D,DV", [(2, 1, 16, 8), (8, 1, 64, 48), (6, 2, 72, 136), (5, 5, 10, 6),
                                      (2, 2, 24, 300)])
def test_sigmoid_weight_of_one_key_among_many(target, decode, H, G, D, DV):
    """Sigmoid weights: a far, a near and the query's own key among hundreds,
    at page and tile borders; a weight does not depend on the other keys and
    the stale rows behind the query weigh nothing."""
    device, dtype = dev_dtype(target)
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    wb = torch.linspace(2.0, -9.0, H, device=device)
    for query_pos in (0, 16, 200, 1030):
        for key_pos in _positions(query_pos):
            got = _needle(device, dtype, key_pos, query_pos, decode, H, G, D, DV, sigmoid=True,
                          wbias=wb)
            want = 1.0 / (1.0 + math.exp(-(8.0 + float(wb[-1]))))
            assert abs(got - want) < tol * want, (query_pos, key_pos, got, want)


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("decode", [False, True], ids=["portion", "single"])
def test_sigmoid_weights_far_from_zero(target, decode):
    """Scores where a sigmoid saturates, without a bias and with a cap."""
    device, dtype = dev_dtype(target)
    for raw in (-120.0, -20.0, 0.0, 30.0, 120.0):
        for cap in (0.0, 5.0):
            got = _needle(device, dtype, 3, 80, decode, raw=raw, sigmoid=True, softcap=cap)
            s = cap * math.tanh(raw / cap) if cap else raw
            want = 1.0 / (1.0 + math.exp(-s))
            assert abs(got - want) < 1e-2 * want + 1e-12, (raw, cap, got, want)


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("decode", [False, True], ids=["portion", "single"])
@pytest.mark.parametrize("H,G,D,DV", [(2, 1, 16, 8), (8, 1, 64, 48), (16, 1, 72, 24), (6, 2, 40, 136),
                                      (4, 4, 10, 6)])
def test_softmax_with_one_in_the_denominator(target, decode, H, G, D, DV):
    """The zero-score sink: most visible where all scores are far below 0 or
    few keys are seen; and the needle's weight among hundreds of keys, capped
    and not."""
    device, dtype = dev_dtype(target)
    tol = 2e-2 if dtype == torch.bfloat16 else 1e-5
    sink = torch.zeros(H, device=device)
    for query_pos in (0, 1, 63, 64, 700):
        for key_pos in _positions(query_pos):
            for cap in (0.0, 6.0):
                got = _needle(device, dtype, key_pos, query_pos, decode, H, G, D, DV, sink=sink,
                              softcap=cap)
                s = cap * math.tanh(8.0 / cap) if cap else 8.0
                want = math.exp(s) / (1.0 + math.exp(s) + query_pos)
                assert abs(got - want) < tol * want, (query_pos, key_pos, cap, got, want)
    got = _needle(device, dtype, 0, 0, decode, H, G, D, DV, raw=-6.0, sink=sink)
    assert abs(got - math.exp(-6.0) / (1.0 + math.exp(-6.0))) < tol * math.exp(-6.0)


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("per_head", [False, True])
@pytest.mark.parametrize("H,G,D,DV", [(4, 2, 16, 24), (3, 1, 10, 7), (2, 1, 24, 1)])
def test_output_gate(target, per_head, H, G, D, DV):
    """sigmoid(gate) per channel of every head, or per head, in a mixed set of
    rows: gate rows are column slices of a wider matrix."""
    device, dtype = dev_dtype(target)
    g = torch.Generator().manual_seed(H)
    n, cols = 70, H if per_head else H * DV
    q = torch.randn(n, H, D, generator=g).to(dtype).to(device)
    wide = (torch.randn(n, cols + 16, generator=g) * 2).to(dtype).to(device)
    gate = wide[:, 8:8 + cols]
    kc = torch.randn(6, G, 16, D, generator=g).to(dtype).to(device)
    vc = torch.randn(6, G, 16, DV, generator=g).to(dtype).to(device)
    table = torch.tensor([[4, 0, 2, 1, 5]], dtype=torch.int32, device=device)
    cu = torch.tensor([0, n], dtype=torch.int32, device=device)
    start = torch.tensor([0], dtype=torch.int32, device=device)
    sg = torch.sigmoid(gate.double().cpu())
    sg = sg.unsqueeze(-1) if per_head else sg.view(n, H, DV)
    tol = 2e-2 if dtype == torch.bfloat16 else 1e-5
    for kw in ({}, {"sigmoid": True}):
        plain = ops.window_attn_prefill(q, kc, vc, DV, table, cu, start, n, 0, 0.2, **kw)
        got = ops.window_attn_prefill(q, kc, vc, DV, table, cu, start, n, 0, 0.2, gate=gate, **kw)
        want = plain.double().cpu() * sg
        assert (got.double().cpu() - want).abs().max() < tol * want.abs().max()
        one = ops.window_attn_decode(q[-1:], kc, vc, DV, table,
                                     torch.tensor([n], dtype=torch.int32, device=device), 0, 0.2,
                                     gate=gate[-1:], **kw)
        assert (one.double().cpu() - want[-1:]).abs().max() < tol * want.abs().max()


# ------------------------------------------------------ ops against oracle --

@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("H,G,D,DV,rot", [(4, 2, 64, 48, 32), (8, 1, 128, 128, 0), (3, 1, 40, 24, 16),
                                          (2, 2, 16, 10, 6), (5, 1, 136, 136, 32), (1, 1, 2, 1, 2)])
def test_unit_norm_rotate_blend_scatter_op(target, H, G, D, DV, rot):
    """The per-token kernel between projections and attention: unit-RMS q and
    k, rotation, a factor per head and one per position (around its steps),
    and values blended with another matrix's, on column slices of a wider
    matrix; a padding row writes nothing."""
    device, dtype = dev_dtype(target)
    g = torch.Generator().manual_seed(D + DV)
    T, page, eps, base, coef, every, first = 21, 16, 1e-5, 300.0, 0.7, 5, 93
    wide = torch.randn(T, 8 + H * D + G * D + G * DV, generator=g).to(dtype).to(device)
    q = wide[:, 8:8 + H * D].unflatten(1, (H, D))
    k = wide[:, 8 + H * D:8 + (H + G) * D].unflatten(1, (G, D))
    v = wide[:, 8 + (H + G) * D:].unflatten(1, (G, DV))
    vf = torch.randn(T, 16 + G * DV, generator=g).to(dtype).to(device)[:, 16:].unflatten(1, (G, DV))
    q0, k0, v0 = q.double().cpu(), k.double().cpu(), v.double().cpu()
    rotc = {"base": base, "dims": rot, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0,
                                                   "original": 100}}
    table = torch.tensor(oracle.frequencies(rotc), dtype=torch.float64).float().to(device)
    hs = torch.rand(H, generator=g) + 0.5
    kc = torch.zeros(3, G, page, D, dtype=dtype, device=device)
    vc = torch.zeros(3, G, page, DV, dtype=dtype, device=device)
    pos = torch.arange(first, first + T, dtype=torch.long, device=device)
    slots = torch.arange(5, 5 + T, dtype=torch.long, device=device)
    slots[4] = -1
    ops.qkv_norm_rope_cache(q, k, v, None, None, table if rot else None, rot, pos, kc, vc, slots, eps,
                            qk_unit_norm=True, head_scale=hs.to(device), temp_coef=coef,
                            temp_every=every, v_first=vf, mix=0.3)
    f = torch.tensor([oracle.query_temperature(first + t, coef, every) for t in range(T)],
                     dtype=torch.float64)
    want_q = oracle.rms(oracle.rotate_half(q0, rotc, first), eps) * hs.double().view(1, H, 1) * \
        f.view(T, 1, 1)
    want_k = oracle.rms(oracle.rotate_half(k0, rotc, first), eps)
    want_v = 0.7 * v0 + 0.3 * vf.double().cpu()
    for w in (want_k, want_v):
        w[4] = 0.0
    got_k = kc.permute(0, 2, 1, 3).reshape(-1, G, D)[5:5 + T].double().cpu()
    got_v = vc.permute(0, 2, 1, 3).reshape(-1, G, DV)[5:5 + T].double().cpu()
    tol = 1e-2 if dtype == torch.bfloat16 else 5e-5
    for got, want in ((q.double().cpu(), want_q), (got_k, want_k), (got_v, want_v)):
        assert (got - want).abs().max().item() < tol * want.abs().max().item()
    assert float(kc.reshape(-1, G, page, D)[0, :, :5].abs().max()) == 0.0   # rows before the slots


def _packed(lens, part, total):
    """Row spans of call `part` (0 or 1) over sequences cut once."""
    return [(0, n) if part == 0 else (n, f) for n, f in zip(lens, total)]


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("H,G,D,DV,lens", [
    (2, 1, 8, 12, [70, 1, 3, 40]), (1, 1, 32, 32, [300]), (6, 2, 5, 7, [17, 33]),
    (4, 4, 64, 48, [5, 1, 1]), (2, 2, 16, 31, [1, 1, 1]), (2, 1, 128, 68, [21, 16]),
    (1, 1, 200, 20, [18]), (16, 8, 40, 64, [1] * 20)])
def test_gated_delta_rule_against_token_by_token(target, H, G, D, DV, lens):
    """Unequal packed sequences, each cut in two calls through its state slot
    (whose stale contents a fresh sequence ignores), against the plain
    recurrence over the whole sequence."""
    device, dtype = dev_dtype(target)
    g = torch.Generator().manual_seed(H * 100 + D)
    B, total = len(lens), [n * 2 + 1 for n in lens]
    data = [dict(q=torch.randn(n, G, D, generator=g), k=torch.randn(n, G, D, generator=g),
                 v=torch.randn(n, H, DV, generator=g), z=torch.randn(n, H, D, generator=g) * 2,
                 b=torch.randn(n, H, generator=g) * 2) for n in total]
    zb, rate = torch.randn(H * D, generator=g) - 1.0, torch.rand(H, generator=g) + 0.1
    S = torch.full((B + 1, H, D, DV), 7.0, device=device)
    slots = torch.tensor(list(range(B - 1, -1, -1)), dtype=torch.int32, device=device)
    outs = [[] for _ in range(B)]
    for part in range(2):
        spans = _packed(lens, part, total)
        cu = torch.tensor([0] + list(torch.tensor([e - s for s, e in spans]).cumsum(0)),
                          dtype=torch.int32, device=device)
        cat = lambda key: torch.cat([d[key][s:e] for d, (s, e) in zip(data, spans)]).to(dtype).to(device)
        fresh = torch.full((B,), 1 - part, dtype=torch.int32, device=device)
        o = ops.gated_delta_rule(cat("q"), cat("k"), cat("v"), cat("z"), zb.to(device),
                                 rate.to(device), cat("b"), S, cu, slots, fresh, D ** -0.5)
        for b in range(B):
            outs[b].append(o[int(cu[b]):int(cu[b + 1])].cpu())
    tol = 1e-4                      # inputs are exact in both; the recurrence itself is fp32
    for b, d in enumerate(data):
        r = {k: t.to(dtype).double() for k, t in d.items()}
        q = r["q"] / torch.sqrt((r["q"] ** 2).sum(-1, keepdim=True) + 1e-6) * D ** -0.5
        k = r["k"] / torch.sqrt((r["k"] ** 2).sum(-1, keepdim=True) + 1e-6)
        dec = torch.exp(-rate.double().view(1, H, 1) *
                        oracle.softplus(r["z"] + zb.double().view(1, H, D)))
        beta = oracle.sigmoid(r["b"])
        want = torch.zeros(total[b], H, DV, dtype=torch.float64)
        for a in range(H):
            ga = a // (H // G)
            M = torch.zeros(D, DV, dtype=torch.float64)
            for t in range(total[b]):
                M = dec[t, a].view(D, 1) * M
                u = beta[t, a] * (r["v"][t, a] - M.T @ k[t, ga])
                M = M + torch.outer(k[t, ga], u)
                want[t, a] = M.T @ q[t, ga]
            got_S = S[int(slots[b]), a].double().cpu()
            assert (got_S - M).abs().max() < tol * M.abs().max().clamp(min=0.1), (b, a)
        got = torch.cat(outs[b]).double()
        err = (got - want).abs().max() / want.abs().max()
        assert err < tol, (b, float(err))


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("H,G,N,DV,ng,lens", [
    (4, 2, 8, 12, 2, [70, 1, 3, 40]), (1, 1, 1, 24, 1, [100]), (6, 6, 33, 5, 3, [17, 33]),
    (3, 1, 70, 40, 8, [5, 1, 1]), (2, 1, 128, 64, 1, [40, 9]), (2, 2, 200, 31, 2, [1, 1]),
    (40, 8, 16, 64, 1, [3, 1]), (4, 2, 24, 72, 2, [130, 64, 1, 65]), (2, 2, 64, 16, 1, [300]),
    (1, 1, 8, 8, 1, [63, 200]), (8, 1, 96, 136, 1, [150, 31]), (16, 2, 128, 64, 4, [64, 127])])
def test_ssd_scan_and_read_out_against_token_by_token(target, H, G, N, DV, ng, lens):
    """Unequal packed sequences, each cut in two calls through its state slot:
    short portions and odd sizes walk token by token, long bf16 portions of
    whole granules run in chunks on the matrix cores."""
    device, dtype = dev_dtype(target)
    g = torch.Generator().manual_seed(H * 100 + N)
    B, total, eps = len(lens), [n * 2 + 1 for n in lens], 1e-5
    data = [dict(x=torch.randn(n, H * DV, generator=g), B=torch.randn(n, G, N, generator=g),
                 C=torch.randn(n, G, N, generator=g), dt=torch.randn(n, H, generator=g) * 2,
                 z=torch.randn(n, H * DV, generator=g)) for n in total]
    dtb, rate = torch.randn(H, generator=g), torch.rand(H, generator=g) + 0.1
    Dh = torch.randn(H, generator=g)
    w = (torch.randn(H * DV, generator=g) * 0.1 + 1).to(dtype)
    S = torch.full((B + 1, H, N, DV), -5.0, device=device)
    slots = torch.tensor(list(range(B - 1, -1, -1)), dtype=torch.int32, device=device)
    outs = [[] for _ in range(B)]
    for part in range(2):
        spans = _packed(lens, part, total)
        cu = torch.tensor([0] + list(torch.tensor([e - s for s, e in spans]).cumsum(0)),
                          dtype=torch.int32, device=device)
        cat = lambda key: torch.cat([d[key][s:e] for d, (s, e) in zip(data, spans)]).to(dtype).to(device)
        fresh = torch.full((B,), 1 - part, dtype=torch.int32, device=device)
        x = cat("x")
        o = ops.ssd_scan(x.unflatten(1, (H, DV)), cat("B"), cat("C"), cat("dt"), dtb.to(device),
                         rate.to(device), S, cu, slots, fresh)
        y = ops.ssd_out_gate_norm(o, x, Dh.to(device), cat("z"), w.to(device), eps, ng, dtype)
        for b in range(B):
            outs[b].append((o[int(cu[b]):int(cu[b + 1])].cpu(), y[int(cu[b]):int(cu[b + 1])].cpu()))
    tol = 2e-2 if dtype == torch.bfloat16 else 2e-4
    for b, d in enumerate(data):
        r = {k: t.to(dtype).double() for k, t in d.items()}
        n = total[b]
        step = oracle.softplus(r["dt"] + dtb.double())
        x = r["x"].view(n, H, DV)
        want = torch.zeros(n, H, DV, dtype=torch.float64)
        for a in range(H):
            ga, M = a // (H // G), torch.zeros(N, DV, dtype=torch.float64)
            for t in range(n):
                M = torch.exp(-rate[a].double() * step[t, a]) * M + \
                    step[t, a] * torch.outer(r["B"][t, ga], x[t, a])
                want[t, a] = M.T @ r["C"][t, ga]
            got_S = S[int(slots[b]), a].double().cpu()
            assert (got_S - M).abs().max() < 1e-4 * M.abs().max().clamp(min=0.1), (b, a)
        # inputs are exact in both: the recurrence itself is at fp32 level
        got_o = torch.cat([oo for oo, _ in outs[b]]).double()
        assert (got_o - want).abs().max() < 1e-4 * want.abs().max(), b
        want = want + Dh.double().view(1, H, 1) * x
        want = oracle.group_norm(want.reshape(n, H * DV) * oracle.silu(r["z"]), w.double(), eps, ng)
        got = torch.cat([y for _, y in outs[b]]).double()
        err = (got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()
        assert err < tol, (b, float(err))


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("decay", [1e-4, 0.3, 40.0], ids=["slow", "middle", "fast"])
def test_ssd_scan_one_write_far_back(target, decay):
    """A single write read hundreds of tokens later survives (or fades) by
    exactly the decays between, across the chunks of a long portion."""
    device, dtype = dev_dtype(target)
    T, H, N, DV, at = 400, 2, 16, 8, 37
    x = torch.zeros(T, H, DV, dtype=dtype)
    Bm = torch.zeros(T, 1, N, dtype=dtype)
    x[at], Bm[at, :, 3] = 1.0, 2.0
    Cm = torch.zeros(T, 1, N, dtype=dtype)
    Cm[:, :, 3] = 0.5
    dt = torch.full((T, H), 1.0, dtype=dtype)
    step = math.log1p(math.exp(1.0))
    S = torch.zeros(1, H, N, DV, device=device)
    o = ops.ssd_scan(x.to(device), Bm.to(device), Cm.to(device), dt.to(device),
                     torch.zeros(H, device=device), torch.full((H,), decay / step, device=device), S,
                     torch.tensor([0, T], dtype=torch.int32, device=device),
                     torch.tensor([0], dtype=torch.int32, device=device),
                     torch.tensor([1], dtype=torch.int32, device=device))
    o = o.double().cpu()[:, :, 0]
    for t in (0, at - 1):
        assert float(o[t].abs().max()) == 0.0
    for t in (at, at + 1, 63, 64, 65, 127, 128, 399):
        want = step * math.exp(-decay * (t - at))
        assert float((o[t] - want).abs().max()) < 2e-4 * want + 1e-30, (t, o[t], want)


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("W,groups", [(48, 3), (27, 3), (2048, 4), (2056, 1), (1536, 1), (3072, 2),
                                      (6000, 1), (9000, 1)])
def test_grouped_residual_join(target, W, groups):
    device, dtype = dev_dtype(target)
    g = torch.Generator().manual_seed(W)
    T, eps = 19, 1e-5
    y = torch.randn(T, W, generator=g).to(dtype)
    y2 = torch.randn(T, W, generator=g).to(dtype)
    res = torch.randn(T, W, generator=g)
    w = (torch.randn(W, generator=g) * 0.1 + 1).to(dtype)
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    for second, a2 in ((None, 0.0), (y2, -0.5)):
        r = res.clone().to(device)
        h = ops.scaled_add_norm(r, y.to(device), None if second is None else second.to(device), 1.5,
                                a2, w.to(device), eps, dtype, groups)
        want_r = res.double() + 1.5 * y.double() + a2 * y2.double()
        want_h = oracle.group_norm(want_r, w.double(), eps, groups)
        assert (r.double().cpu() - want_r).abs().max() < 1e-5
        assert (h.double().cpu() - want_h).abs().max() < tol * want_h.abs().max()


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("E,top,T", [(7, 3, 9), (20, 4, 130), (2, 1, 5), (5, 5, 33), (130, 2, 40)])
def test_router_softmax_over_the_chosen(target, E, top, T):
    device, _ = dev_dtype(target)
    g = torch.Generator().manual_seed(E + top)
    logits = torch.randn(T, E, generator=g) * 4
    idx, w = ops.softmax_topk(logits.to(device), top, 1.0, renorm=True)
    for t in range(T):
        order = sorted(range(E), key=lambda e: (-float(logits[t, e]), e))[:top]
        assert idx[t].tolist() == order
        want = torch.softmax(logits[t, order].double(), 0)
        assert (w[t].double().cpu() - want).abs().max() < 1e-5


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("sigmoid", [False, True])
@pytest.mark.parametrize("H,DV", [(3, 7), (4, 64), (2, 130)])
def test_head_norm_gate(target, sigmoid, H, DV):
    device, dtype = dev_dtype(target)
    g = torch.Generator().manual_seed(DV)
    T, eps = 11, 1e-5
    o = torch.randn(T, H, DV, generator=g)
    gate = torch.randn(T, H * DV, generator=g).to(dtype)
    w = (torch.randn(DV, generator=g) * 0.1 + 1).to(dtype)
    got = ops.gla_out_norm_gate(o.to(device), w.to(device), gate.to(device), eps, dtype, sigmoid=sigmoid)
    act = oracle.sigmoid if sigmoid else oracle.silu
    want = (oracle.rms(o.double(), eps) * w.double()).reshape(T, H * DV) * act(gate.double())
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    assert (got.double().cpu() - want).abs().max() < tol * want.abs().max()


@pytest.mark.parametrize("target", DEVICES)
@pytest.mark.parametrize("C,K,bias", [(5, 4, True), (64, 3, False), (300, 8, True), (7, 2, True),
                                      (40, 1, False), (24, 5, False), (33, 16, True)])
def test_convolution_across_short_cuts(target, C, K, bias):
    """The convolution with SiLU, its tail carried through cuts shorter than
    its reach, with a second sequence packed in front."""
    device, dtype = dev_dtype(target)
    g = torch.Generator().manual_seed(C * K)
    n, other = 600, 3
    x = torch.randn(n, C, generator=g).to(dtype)
    w = torch.randn(C, K, generator=g) / math.sqrt(K)
    b = torch.randn(C, generator=g) if bias else None
    want = oracle.silu(oracle.causal_conv(x.double(), w.double(), None if b is None else b.double()))
    tail = torch.full((3, K - 1, C), 9.0, device=device)
    got, at = [], 0
    for cut in (1, 1, 2, 1, 5, 1, 12, 540, 37):
        cu = torch.tensor([0, other, other + cut], dtype=torch.int32, device=device)
        xs = torch.cat([torch.full((other, C), 4.0, dtype=dtype), x[at:at + cut]]).to(device)
        out = ops.causal_conv_silu(
            xs, w.to(device), None if b is None else b.to(device), tail, cu,
            torch.tensor([2, 1], dtype=torch.int32, device=device),
            torch.tensor([0, int(at == 0)], dtype=torch.int32, device=device))
        got.append(out[other:])
        at += cut
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    assert (torch.cat(got).double().cpu() - want).abs().max().item() < tol * want.abs().max().item()


# -------------------------------------------- generation and entry points --

@pytest.mark.parametrize("target", DEVICES[:2])
def test_greedy_generation_through_the_scheduler(mixed_model, target):
    """add_request / step: the scheduler's own admission, chunked prefill
    (a budget smaller than the prompts), decode batching and sampler."""
    cfg, tensors, path = mixed_model(target)
    prompts = {"p": tokens_for(21, cfg["vocab"], 40), "q": tokens_for(5, cfg["vocab"], 41),
               "r": tokens_for(34, cfg["vocab"], 42)}
    eng = make_engine(path, target, prefill_budget=16)
    params = SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True)
    for rid, toks in prompts.items():
        eng.add_request(rid, prompt_token_ids=toks, params=params)
    got = {rid: [] for rid in prompts}
    while eng.has_unfinished():
        for out in eng.step():
            got[out.request_id].extend(out.new_token_ids)
    for rid, toks in prompts.items():
        assert got[rid] == oracle.greedy(cfg, tensors, toks, 6), rid
    assert eng.allocator.num_free == eng.allocator.num_blocks


def test_preset_runs_through_generate():
    eng = LLMEngine(EngineConfig(model="tiny-kikurax", device="cpu", max_num_seqs=2,
                                 max_model_len=64, num_kv_blocks=8))
    assert eng.spec.param_count() == sum(
        int(lw.t[n].numel()) for lw in eng.model.layers for n in lw.t
        if n not in ("in", "in_b", "conv_w", "conv_b")) + eng.model.embedding.numel() + \
        eng.model.final_norm.numel() + sum(
            rows * (64 + (lw.t["conv_w"].shape[1] if "conv_w" in lw.t and
                          at < lw.conv_cols else 0) +
                    int("in_b" in lw.t) + int("conv_b" in lw.t and at < lw.conv_cols))
            for lw in eng.model.layers for at, rows in lw.seg.values())
    out = eng.generate_batch(["ab", "c"], SamplingParams(temperature=0.0, max_tokens=4,
                                                         ignore_eos=True))
    assert len(out) == 2


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_graph_replays_equal_eager(mixed_model, dtype):
    """Captured decode steps replayed several times, with eager work between
    the replays, against the same steps run eagerly."""
    target = ("cuda", dtype)
    cfg, tensors, path = mixed_model(target)
    toks = {r: tokens_for(n, cfg["vocab"], 50 + i) for i, (r, n) in enumerate(
        {"a": 30, "b": 12, "c": 19, "d": 9, "e": 25, "f": 14, "g": 11, "h": 21}.items())}
    results = []
    for eager in (True, False):
        eng = LLMEngine(EngineConfig(model=path, device="cuda", dtype=dtype, max_num_seqs=8,
                                     max_model_len=256, num_kv_blocks=32, enforce_eager=eager))
        assert eng.runner.use_graphs == (not eager)
        rows = []
        eng.replay_step([{"id": r, "tokens": t[:-8], "want": []} for r, t in toks.items()])
        for k in range(8, 0, -1):
            rows.append(eng.replay_step(
                [{"id": r, "tokens": [t[len(t) - k]], "want": [0]} for r, t in toks.items()]))
            torch.cuda.synchronize()
        results.append(torch.cat(rows))
    diff = (results[0] - results[1]).abs().max() / results[0].abs().max()
    assert diff < (3e-2 if dtype == "bfloat16" else 1e-4)
    want = torch.cat([torch.stack([oracle_logits(cfg, tensors, t)[len(t) - k] for t in toks.values()])
                      for k in range(8, 0, -1)])
    assert_close(results[1], want, target, "graph replays")


def test_trace_runner_cli(tmp_path, mixed_model):
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    cfg, tensors, path = mixed_model(("cpu", "float32"))
    toks = tokens_for(20, cfg["vocab"], 60)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": toks[:13], "want": [0, 12]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": toks[13:15], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": toks[15:], "want": [4]}], "end": ["a"]},
    ]
    out = tmp_path / "out"
    root = Path(__file__).resolve().parent.parent
    proc = subprocess.run(
        [sys.executable, str(root / "bin" / "trace_run"), "--model", path, "--dtype", "float32",
         "--out", str(out), "--max-tokens", "64"],
        input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
        timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [ln for ln in proc.stdout.splitlines() if ln.startswith("done")] == \
        ["done 0", "done 1", "done 2"]
    want = oracle_logits(cfg, tensors, toks)
    a = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1).copy())
    b = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(1, -1).copy())
    assert not (out / "1.f32").exists()
    assert_close(torch.cat([a, b]), want[[0, 12, 19]], ("cpu", "float32"), "trace runner")
