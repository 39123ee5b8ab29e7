"""Fedinex in the framework against the plain oracle (tests/fedinex_oracle.py).

Every test builds its own small configuration and random checkpoint, runs it
through the framework's ops / model / cache / executor (and, for generation,
the shard runtime's slot scheduler and the trace replay CLI) and compares with
the oracle, which is written from the equations, runs whole sequences without
any cache and shares no code with dnet_amd. Tests run on the CPU reference-op
path and, marked ``gpu``, on the HIP kernels.
"""
import copy
import json
import subprocess
import sys
from pathlib import Path

import pytest
import torch

import fedinex_oracle as O
from dnet_amd.models import ModelConfig
from dnet_amd.models.config import fedinex_config
from dnet_amd.parallel.ring import RingExecutor

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
F64 = torch.float64
V = 83
W = 48


def base_cfg(**kw):
    """Seven layers: three that mix values (the second one with other heads
    and another mask), one attention layer that does not, two parallel ones of
    different sizes, a gated linear one; one layer without a feed-forward."""
    args = dict(pattern="gapaapa", layers=7, heads=4, kv_heads=2, dim=10,
                vdim=6, rot_dims=6, window=9, keep_first=2, left_heads=3,
                left_kv_heads=1, left_dim=14, left_vdim=10, conv=3,
                left_rot_dims=8, mem_heads=2, mem_dim=9, mem_vdim=13,
                gate_cap=4.0, gla_heads=3, gla_dim=7, gla_vdim=11, tau=5.0,
                ff=40, limit=1.2, experts=9, top=2, expert_ff=20, groups=3,
                keep_groups=2, rot_base=300.0, left_rot_base=900.0, eps=1e-5)
    args.update(kw)
    cfg = copy.deepcopy(fedinex_config(W, V, **args))
    if args["pattern"] == "gapaapa":
        L = cfg["layers"]
        L[2]["mlp"] = None
        L[3]["mixer"].update(heads=6, dim=5, scale=0.6,
                             rot={"base": 70.0, "dims": 4},
                             mask={"size": 4, "keep_first": 7})
        L[4]["mixer"].update(heads=2, kv_heads=1, vdim=9, v_mix=False)
        L[4]["mixer"].pop("mask")
        L[5]["mixer"]["left"].update(heads=2, kv_heads=2, vdim=4, conv=5)
        L[5]["mixer"]["right"].update(heads=3, dim=4, vdim=5, gate_cap=9.0)
        L[5]["mixer"].update(left_scale=1.1, right_scale=0.35)
    return cfg


def steady_cfg(dtype, **kw):
    """The base stack; for bfloat16 runs a shallower one (every layer of
    these tiny random models multiplies rounding noise)."""
    if dtype == "bfloat16":
        kw = dict(dict(pattern="apg", layers=3), **kw)
    return base_cfg(**kw)


def checkpoint(cfg, seed, dtype="float32"):
    """Random weights; for bfloat16 runs with smaller sublayer results, and
    corrections wide enough that rounding does not move a routing choice."""
    if dtype == "float32":
        return O.make_checkpoint(cfg, seed)
    sd = O.make_checkpoint(cfg, seed, out_gain=0.5)
    return {k: v * 16 if k.endswith("correction") else v
            for k, v in sd.items()}


def tokens(n, seed, vocab=V):
    return torch.randint(0, vocab, (n,),
                         generator=torch.Generator().manual_seed(seed))


def executor(cfg, sd, device, dtype="float32", slots=3, smax=160, **kw):
    mc = ModelConfig.from_hf(cfg)
    mc.compute_dtype = dtype
    ex = RingExecutor(mc, 0, 1, torch.device(device), mb_size=slots,
                      smax=smax, init_weights=False,
                      use_graphs=kw.pop("use_graphs", False), **kw)
    ex.model.load_state_dict(sd)
    return ex


def close(got, want, dtype="float32"):
    got, want = got.detach().cpu().to(F64), want.to(F64)
    scale = float(want.pow(2).mean().sqrt())
    if dtype == "float32":
        err = float((got - want).abs().max())
        assert err <= 2e-3 * scale, f"max err {err:.3g} vs scale {scale:.3g}"
        rms = float((got - want).pow(2).mean().sqrt())
        assert rms <= 5e-4 * scale, f"rms err {rms:.3g} vs {scale:.3g}"
        return
    # bfloat16: rows by their own error; a close routing call may fall the
    # other way in a single row
    err = (got - want).pow(2).mean(-1).sqrt().reshape(-1) / scale
    assert float(err.median()) <= 0.08, err
    assert int((err > 0.25).sum()) <= max(1, len(err) // 10), err


def decode_step(ex, slot_tokens):
    """One slot-batch decode step {slot: token}; other rows sit it out."""
    tb = ex.tokbuf[0].cpu()
    for s, t in slot_tokens.items():
        tb[s] = int(t)
    ex.tokbuf[0].copy_(tb)
    idle = torch.ones(ex.mb_size, dtype=torch.bool)
    idle[list(slot_tokens)] = False
    idle = idle.to(ex.device)
    ex.slot_step_compute(park=idle)
    lg = ex.logits_buf[0].float().cpu().clone()
    ex.kvs[0].pos.add_((~idle).to(torch.int32))
    return lg


def oracle(toks, cfg, sd, **kw):
    return O.forward([int(t) for t in toks], sd, cfg, F64, **kw)


def sub64(sd, prefix):
    return {k: v.to(F64) for k, v in O.sub(sd, prefix).items()}


# ---------- configuration ----------

def test_config_registry_and_cache_layout():
    from dnet_amd.models import FedinexRingModel, get_ring_model
    cfg = base_cfg()
    mc = ModelConfig.from_hf(cfg)
    assert mc.model_type == "fedinex" and mc.num_layers == 7
    assert get_ring_model("fedinex") is FedinexRingModel
    assert mc.num_experts == 9 and mc.num_experts_per_tok == 2
    assert mc.moe_intermediate_size == 20
    ex = executor(cfg, checkpoint(cfg, 1), "cpu")
    kv = ex.kvs[0]
    assert ex.hidden_width == W and ex.model.v_layer == 1
    assert kv.k[0] is None and kv.state[0]["S"].shape == (3, 3, 7, 11)
    assert kv.k[1].shape == (3, 2, 160, 10) and kv.v[1].shape[3] == 6
    assert kv.k[3].shape == (3, 2, 160, 5) and not kv.state[3]
    assert kv.k[2].shape == (3, 1, 160, 14)
    st = kv.state[2]
    assert st["conv"].shape == (3, 2, 3 * 14 + 14 + 10)
    assert st["S"].shape == (3, 2, 9, 13) and st["m"].shape == (3, 2, 1)
    assert st["n"].shape == (3, 2, 1, 9)
    assert all(kv.state[i][n].dtype == torch.float32
               for i in (0, 2, 5) for n in kv.state[i] if n != "conv")

    def broken(change):
        c = base_cfg()
        change(c["layers"])
        with pytest.raises(ValueError):
            ModelConfig.from_hf(c)

    broken(lambda l: l[1].update(type="mystery"))
    broken(lambda l: l[1]["mixer"].pop("scale"))
    broken(lambda l: l[1]["mixer"].update(kv_heads=3))
    broken(lambda l: l[3]["mixer"].update(vdim=5))      # mixes other values
    broken(lambda l: l[1]["mixer"]["rot"].update(dims=12))
    broken(lambda l: l[1]["mixer"]["rot"].update(dims=3))
    broken(lambda l: l[1]["mixer"]["mask"].update(size=0))
    broken(lambda l: l[2]["mixer"].pop("left_scale"))
    broken(lambda l: l[2]["mixer"]["left"].update(conv=0))
    broken(lambda l: l[2]["mixer"]["right"].pop("gate_cap"))
    broken(lambda l: l[0]["mixer"].pop("tau"))
    broken(lambda l: l[1]["mlp"]["router"].update(top=7))   # 2 groups of 3
    broken(lambda l: l[1]["mlp"]["router"]["groups"].update(count=2))
    broken(lambda l: l[1]["mlp"]["router"]["groups"].update(keep=4))
    broken(lambda l: l[0]["mlp"].update(kind="mystery"))
    broken(lambda l: l[0]["mlp"].pop("limit"))


# ---------- mechanisms alone ----------

def _mixer_alone(device, cfg, sd, u, T0, portion=None, lid=0):
    """Run a mixer on given inputs u [T, W] through the cache: the first T0
    rows as one prompt portion (or portions), then row by row, in a slot whose
    cache and state hold another sequence's leftovers."""
    T = u.shape[0]
    ex = executor(cfg, sd, device, smax=max(160, T))
    m, kv = ex.model, ex.kvs[0]
    for t in [*kv.k, *kv.v, *(t for st in kv.state for t in st.values())]:
        if t is not None:
            t.fill_(3.0)
    slot = torch.tensor([2], dtype=torch.int32, device=device)
    steps, p = [], 0
    while p < T0:
        n = min(portion or T0, T0 - p)
        steps.append((p, n))
        p += n
    steps += [(t, 1) for t in range(T0, T)]
    fn = {"attention": m._attention, "parallel": m._parallel,
          "gla": m._gla}[m.cfg.layer_specs[lid]["type"]]
    outs = []
    for p0, n in steps:
        pos = torch.tensor([p0], dtype=torch.int32, device=device)
        ln = torch.tensor([n], dtype=torch.int32, device=device)
        x = u[p0:p0 + n].to(torch.float32).to(device).contiguous()
        o = fn(x, m.layers[lid], lid, kv, pos, n, ln, slot, None)
        outs.append(o.float().cpu())
    return torch.cat(outs)


def _want(u, cfg, sd, lid=0, **change):
    """The oracle's mixer ``lid`` on u; ``change`` edits its sizes."""
    spec = cfg["layers"][lid]
    m = copy.deepcopy(spec["mixer"])
    m.update(change)
    p, eps = sub64(sd, f"l{lid}.mix."), cfg["norm"]["eps"]
    u = u.to(F64)
    if spec["type"] == "attention":
        return O.biased_attention(u, p, m)[0]
    return (O.parallel if spec["type"] == "parallel" else O.gla)(u, p, m, eps)


def far_apart(a, b):
    return float((a - b).abs().max()) > 0.2 * float(b.pow(2).mean().sqrt())


def inputs(T, seed, std=1.0):
    return torch.randn(T, W, generator=torch.Generator().manual_seed(seed)) \
        * std


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [
    {}, dict(heads=1, kv_heads=1, dim=3, vdim=1, rot_dims=2, window=1,
             keep_first=1),
    dict(heads=6, kv_heads=1, dim=8, vdim=8, rot_dims=8, keep_first=0),
    dict(heads=16, kv_heads=1, dim=8, vdim=16, rot_dims=4, window=5,
         keep_first=12),
    dict(heads=2, kv_heads=2, dim=33, vdim=40, rot_dims=0, window=0),
    dict(window=100, keep_first=50)])
def test_attention_alone(device, kw):
    """Biased projections, half-split rotation, window with kept first
    tokens: prompt portion, then token by token through the cache."""
    cfg = base_cfg(**dict(dict(pattern="a", layers=1), **kw))
    sd = checkpoint(cfg, 3)
    u = inputs(41, 9)
    want = _want(u, cfg, sd)
    for T0, portion in ((29, None), (30, 7), (2, 2), (41, None)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,kept", [(64, 3), (65, 64), (63, 65), (130, 33),
                                       (32, 31), (7, 100)])
def test_window_and_kept_edges(device, size, kept):
    """Peaky scores, so that one key more or less at the window's edge or
    behind the kept tokens shows: the oracle with a size one off differs
    grossly, the framework equals the true one at every position (page and
    tile borders of 32 and 64 keys among them)."""
    T = 210
    cfg = base_cfg(pattern="a", layers=1, heads=8, kv_heads=2, dim=12,
                   vdim=16, window=size, keep_first=kept)
    cfg["layers"][0]["mixer"]["scale"] = 2.5
    sd = checkpoint(cfg, 4)
    u = inputs(T, 5, 0.8)
    u[kept - 1:kept + 1] *= 2.5             # the keys on the kept border
    want = _want(u, cfg, sd)
    masks = [dict(size=size + 1, keep_first=kept),
             dict(size=max(1, size - 1), keep_first=kept),
             dict(size=size, keep_first=kept + 1),
             dict(size=size, keep_first=kept - 1),
             dict(size=size, keep_first=0)]
    for other in masks:
        assert far_apart(_want(u, cfg, sd, mask=other), want), other
    for T0, portion in ((T, None), (T - 90, None), (T - 20, 33), (5, None)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_kept_and_far_keys_stand_out(device):
    """Queries at the end aimed at one key far back: a kept one in the
    windowed layer, any one in the full causal half of a parallel layer. The
    key's turn by its true position matters: aimed one position off, the
    weight is another."""
    T, far = 330, 2
    cfg = base_cfg(pattern="a", layers=1, heads=2, kv_heads=1, dim=16, vdim=8,
                   rot_dims=12, rot_base=40.0, window=20, keep_first=4)
    cfg["layers"][0]["mixer"]["scale"] = 1.0
    sd = checkpoint(cfg, 7)
    u = inputs(T, 12, 0.7)
    p = sub64(sd, "l0.mix.")
    m = cfg["layers"][0]["mixer"]

    def keys(at=None):
        k = (u.to(F64) @ p["k"].T + p["k.b"]).view(T, 1, 16)
        return O.turn(k, m["rot"], "halves")[:, 0]

    # the query that, turned to the last position, lies along the far key
    aim = keys()[far]
    # (turned back by the last position's angles)
    n = 6
    ang = (T - 1) * 40.0 ** (-2.0 * torch.arange(n, dtype=F64) / 12)
    q0 = aim.clone()
    q0[:n] = aim[:n] * torch.cos(ang) + aim[n:2 * n] * torch.sin(ang)
    q0[n:2 * n] = aim[n:2 * n] * torch.cos(ang) - aim[:n] * torch.sin(ang)
    u[T - 1] = (torch.linalg.pinv(p["q"][:16])
                @ (q0 * 3 - p["q.b"][:16])).float()
    want = _want(u, cfg, sd)
    assert far_apart(_want(u, cfg, sd, mask={"size": 20, "keep_first": 2})[-1],
                     want[-1])
    assert far_apart(_want(u, cfg, sd, rot={"dims": 12, "base": 400.0})[-1],
                     want[-1])
    for T0, portion in ((T, None), (T - 1, None), (T - 5, 64), (13, 12)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [
    {}, dict(conv=1, left_heads=1, left_kv_heads=1, left_dim=2, left_vdim=1,
             left_rot_dims=2),
    dict(conv=2, left_heads=6, left_kv_heads=3, left_dim=8, left_vdim=16,
         left_rot_dims=8),
    dict(conv=4, left_heads=16, left_kv_heads=1, left_dim=16, left_vdim=8,
         left_rot_dims=0),
    dict(conv=7, left_heads=2, left_kv_heads=2, left_dim=24, left_vdim=32,
         left_rot_dims=12)])
def test_convolved_attention_alone(device, kw):
    """The left half of a parallel layer (the right one scaled by 0): short
    convolution with its tail across portions and decode steps, interleaved
    rotation, full causal softmax, per-head gate and the half's factor."""
    cfg = base_cfg(**dict(dict(pattern="p", layers=1, right_scale=0.0,
                               left_scale=0.6), **kw))
    sd = checkpoint(cfg, 5)
    u = inputs(45, 9)
    want = _want(u, cfg, sd)
    flat = dict(sd)
    flat["l0.mix.left.g"] = torch.zeros_like(sd["l0.mix.left.g"])
    assert far_apart(_want(u, cfg, flat), want)
    if int(cfg["layers"][0]["mixer"]["left"]["conv"]) > 1:
        late = dict(sd)                     # the taps in the other order
        late["l0.mix.left.k.conv"] = sd["l0.mix.left.k.conv"].flip(1)
        assert far_apart(_want(u, cfg, late), want)
    for T0, portion in ((33, None), (30, 7), (2, 2), (1, None), (45, 9),
                        (44, 2)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_far_key_through_the_convolution(device):
    """A dominating key hundreds of positions back in the full causal half;
    without it, or with the convolution left out, the last row is another."""
    T, far = 320, 9
    cfg = base_cfg(pattern="p", layers=1, right_scale=0.0, left_heads=2,
                   left_kv_heads=1, left_dim=16, left_vdim=8, conv=4,
                   left_rot_dims=0)
    cfg["layers"][0]["mixer"]["left"]["scale"] = 1.0
    sd = checkpoint(cfg, 8)
    u = inputs(T, 12, 0.6)
    u[far] *= 5
    p = sub64(sd, "l0.mix.left.")
    k = O.short_conv(u.to(F64) @ p["k"].T, p["k.conv"])
    # solve for the last input so that head 0's convolved query is the far key
    q = O.short_conv(u.to(F64) @ p["q"].T, p["q.conv"])
    w = p["q"][:16] * p["q.conv"][:16, -1:]
    u[T - 1] += (torch.linalg.pinv(w)
                 @ (1.0 * k[far] - q[T - 1, :16])).float()
    want = _want(u, cfg, sd)
    quiet = u.clone()
    quiet[far] = u[far + 1]
    assert far_apart(_want(quiet, cfg, sd)[-1], want[-1])
    for T0, portion in ((T, None), (T - 1, None), (T - 5, 64), (13, 12)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [
    {}, dict(mem_heads=1, mem_dim=1, mem_vdim=1),
    dict(mem_heads=5, mem_dim=16, mem_vdim=70),
    dict(mem_heads=2, mem_dim=130, mem_vdim=64, gate_cap=15.0),
    dict(mem_heads=3, mem_dim=64, mem_vdim=33, gate_cap=1.0)])
def test_matrix_memory_alone(device, kw):
    """The right half of a parallel layer (the left one scaled by 0)."""
    cfg = base_cfg(**dict(dict(pattern="p", layers=1, left_scale=0.0,
                               right_scale=0.8), **kw))
    sd = checkpoint(cfg, 6)
    u = inputs(83, 9)
    want = _want(u, cfg, sd)
    for T0, portion in ((71, None), (70, 7), (2, 2), (83, 16)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("ib,fb", [(-8.0, 1.0), (6.0, -6.0), (0.0, 12.0)])
def test_memory_gates_and_the_first_tokens(device, ib, fb):
    """Gates far to either side: the running maximum starts at 0, so weak
    input gates meet the floor exp(-m) of the normalizer from the first token
    on (started at minus infinity the oracle gives another result); the cap
    bends large gates."""
    cfg = base_cfg(pattern="p", layers=1, left_scale=0.0, mem_heads=2,
                   mem_dim=6, mem_vdim=5, gate_cap=7.0)
    sd = checkpoint(cfg, 6)
    sd["l0.mix.right.i.b"] = torch.full((2,), ib, dtype=torch.bfloat16)
    sd["l0.mix.right.f.b"] = torch.full((2,), fb, dtype=torch.bfloat16)
    u = inputs(40, 10)
    want = _want(u, cfg, sd)
    p = sub64(sd, "l0.mix.right.")
    g = 7.0 * torch.tanh((u.to(F64) @ p["i"].T + p["i.b"]) / 7.0)
    f = O.log_sigmoid(7.0 * torch.tanh(
        (u.to(F64) @ p["f"].T + p["f.b"]) / 7.0))
    q, k, v = (torch.randn(40, 2, n, dtype=F64) for n in (6, 6, 5))
    a = O.matrix_memory(q, k, v, g, f)
    if ib < 0:          # the same with everything shifted: no floor at 0
        b = O.matrix_memory(q, k, v, g + 8.0, f)
        assert far_apart(a[:3], b[:3])
    for T0, portion in ((40, None), (1, None), (33, 2)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["p", "g"])
def test_far_token_through_the_recurrent_state(device, kind):
    """Gates that keep almost everything: what one standout token wrote is
    still most of the state 300 tokens on, in a prompt, across portions and
    in decoding. The oracle without that token differs grossly."""
    cfg = base_cfg(pattern=kind, layers=1, left_scale=0.0, gate_cap=15.0,
                   mem_dim=6, gla_dim=6)
    sd = checkpoint(cfg, 6)
    if kind == "p":
        sd["l0.mix.right.f.b"] = torch.full((2,), 12.0).to(torch.bfloat16)
        sd["l0.mix.right.f"] = sd["l0.mix.right.f"] * 0.1
    else:
        sd["l0.mix.a2.b"] = torch.full((18,), 9.0).to(torch.bfloat16)
    T = 310
    u = inputs(T, 11, 0.3)
    u[5] = u[5] * 60
    want = _want(u, cfg, sd)
    quiet = u.clone()
    quiet[5] = u[6]
    assert far_apart(_want(quiet, cfg, sd)[-1], want[-1])
    for T0, portion in ((T, None), (T - 10, 33), (7, None)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [
    {}, dict(gla_heads=1, gla_dim=1, gla_vdim=1, tau=1.0),
    dict(gla_heads=2, gla_dim=64, gla_vdim=130),
    dict(gla_heads=3, gla_dim=40, gla_vdim=64, tau=0.5),
    dict(gla_heads=2, gla_dim=140, gla_vdim=7)])
def test_gated_linear_attention_alone(device, kw):
    cfg = base_cfg(**dict(dict(pattern="g", layers=1), **kw))
    sd = checkpoint(cfg, 5)
    m = cfg["layers"][0]["mixer"]
    u = inputs(83, 9)
    want = _want(u, cfg, sd)
    assert far_apart(_want(u, cfg, sd, tau=m["tau"] * 1.5), want)
    for T0, portion in ((71, None), (70, 7), (2, 2), (83, 16)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_value_mixing(device):
    """Later mixing layers take the first one's own values of the same token
    (not its mixed ones, not another token's, not those of a layer that does
    not mix); run as one window and layer by layer, in portions and decoding."""
    cfg = base_cfg(pattern="aagaa", layers=5, experts=0)
    cfg["layers"][0]["mixer"]["v_mix"] = False
    cfg["layers"][0]["mixer"].update(kv_heads=1, vdim=7)
    sd = checkpoint(cfg, 21)
    for i, lam in ((1, -3.0), (3, 0.7), (4, 1.3)):
        sd[f"l{i}.mix.vmix"] = torch.tensor(lam, dtype=torch.bfloat16)
    a = tokens(40, 22)
    want = oracle(a, cfg, sd)
    for i in (3, 4):
        off = dict(sd)
        off[f"l{i}.mix.vmix"] = torch.tensor(0.0)
        assert far_apart(oracle(a, cfg, off), want)
    unused = dict(sd)                   # the first mixing layer's factor
    unused["l1.mix.vmix"] = torch.tensor(9.0)
    assert torch.equal(oracle(a, cfg, unused), want)
    ex = executor(cfg, sd, device)
    assert ex.model.v_layer == 1 and ex.model.layers[1].lam is None
    got = ex.prefill_slots([1], [a[:30]], want=[list(range(30))], chunk=7)[0]
    close(got, want[:30])
    for t in range(30, 40):
        close(decode_step(ex, {1: a[t]})[1:2], want[t].view(1, -1))
    layers = []
    oracle(a, cfg, sd, layers_out=layers)
    m, kv = ex.model, ex.kvs[0]
    h = m.embed_tokens(a.view(1, -1).to(device)).clone()
    ln = torch.tensor([40], dtype=torch.int32, device=device)
    slot = torch.tensor([2], dtype=torch.int32, device=device)
    for lid in range(5):
        m.prefill_window(h, [lid], kv, 0, lens=ln, slots=slot)
        close(h[0], layers[lid])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("rows", [1, 3, 40, 90])
@pytest.mark.parametrize("kw", [
    {}, dict(top=1, keep_groups=1), dict(top=6),
    dict(groups=0, experts=5, top=3), dict(groups=1, keep_groups=1, experts=4, top=4),
    dict(groups=5, keep_groups=3, experts=5, top=2),
    dict(groups=2, keep_groups=1, experts=12, top=4, router_scale=0.7),
    dict(experts=1, top=1, groups=1, keep_groups=1)])
def test_experts_alone(device, rows, kw):
    """Mixture of experts on every row-count path: chosen by the corrected
    score inside the best groups, weighted by the plain score times the
    constant, not renormalized. Choice scores are negative for many experts
    (a group that drops out must not come back as zeros), and the correction
    alone moves the choice."""
    cfg = base_cfg(**dict(dict(pattern="gg", layers=2), **kw))
    sd = checkpoint(cfg, 9)
    ff = cfg["layers"][1]["mlp"]
    E, r = ff["router"]["experts"], ff["router"]
    sd["l1.mlp.correction"] = torch.linspace(-1.5, -0.6, E).to(torch.bfloat16)
    h = inputs(rows, 15, 2.0)
    p64 = sub64(sd, "l1.mlp.")
    want = O.moe(h.to(F64), p64, ff)
    if rows >= 40 and r["top"] < E:
        plain = dict(p64, correction=p64["correction"] * 0)
        assert far_apart(O.moe(h.to(F64), plain, ff), want)
        g = r.get("groups")
        if g and r["top"] > 1 and 1 < g["count"] < E and g["keep"] < g["count"]:
            free = copy.deepcopy(ff)
            free["router"].pop("groups")
            assert far_apart(O.moe(h.to(F64), p64, free), want)
    for dtype in ("float32", "bfloat16"):
        ex = executor(cfg, sd, device, dtype)
        m = ex.model
        u = h.to(device).to(m.wdtype)
        for step in (False, True):
            got = m._moe(u, m.layers[1], ff, step)
            if dtype == "float32":
                close(got, want)
            else:
                rel = (got.float().cpu().to(F64) - want).pow(2).mean(-1) \
                    .sqrt() / want.pow(2).mean().sqrt()
                assert float(rel.median()) < 0.03 and \
                    float((rel > 0.1).float().mean()) <= 0.1, rel


@pytest.mark.parametrize("device", DEVICES)
def test_dense_feed_forward_alone(device):
    """Clamps that bite: inputs large enough that the limit shows on both
    sides of the gate and of the other half."""
    cfg = base_cfg(pattern="g", layers=1, ff=37, limit=0.8)
    sd = checkpoint(cfg, 10)
    h = inputs(6, 16, 3.0)
    p = sub64(sd, "l0.mlp.")
    want = O.clamped_ff(h.to(F64), p, "", 0.8)
    assert far_apart(O.clamped_ff(h.to(F64), p, "", 1.6), want)
    m = executor(cfg, sd, device).model
    close(m._ff(h.to(device), m.layers[0], cfg["layers"][0]["mlp"], False),
          want)


# ---------- the whole model ----------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompt_logits_first_tokens_and_layers(device, dtype):
    cfg = steady_cfg(dtype)
    sd = checkpoint(cfg, 6, dtype)
    a = tokens(37, 1)
    layers = []
    want = oracle(a, cfg, sd, layers_out=layers)
    ex = executor(cfg, sd, device, dtype)
    got = ex.prefill_slots([1], [a], want=[list(range(37))])[0]
    close(got, want, dtype)
    if dtype == "float32":
        # the residual after every layer
        m, kv = ex.model, ex.kvs[0]
        ln = torch.tensor([37], dtype=torch.int32, device=device)
        slot = torch.tensor([2], dtype=torch.int32, device=device)
        h = m.embed_tokens(a.view(1, -1).to(device)).clone()
        for lid in range(len(cfg["layers"])):
            m.prefill_window(h, [lid], kv, 0, lens=ln, slots=slot)
            close(h[0], layers[lid])
    # single-token prompts and the very first positions
    one = ex.prefill_slots([0], [a[:1]])[0]
    close(one, want[:1], dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_prefill_vs_token_by_token_and_long_decode(device):
    cfg = base_cfg()
    sd = checkpoint(cfg, 7)
    a = tokens(150, 2)
    want = oracle(a, cfg, sd)
    ex = executor(cfg, sd, device)
    got = [ex.prefill_slots([2], [a[:1]])[0].float().cpu()]
    for t in range(1, 150):                 # decode from the second token on
        got.append(decode_step(ex, {2: a[t]})[2:3])
    close(torch.cat(got), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("chunk", [2, 3, 16, 33])
def test_portions(device, chunk):
    """A prompt cut into portions (executor chunking and continued requests)
    gives the logits of the whole prompt."""
    cfg = base_cfg()
    sd = checkpoint(cfg, 8)
    a = tokens(45, 3)
    want = oracle(a, cfg, sd)
    ex = executor(cfg, sd, device)
    got = ex.prefill_slots([1], [a], want=[list(range(45))], chunk=chunk)[0]
    close(got, want)
    # the same through continued calls of unequal size
    rows, p = [], 0
    for n in (chunk, 2, 45):
        n = min(n, 45 - p)
        if n <= 0:
            break
        rows.append(ex.prefill_slots([0], [a[p:p + n]],
                                     want=[list(range(n))], start=[p])[0])
        p += n
    close(torch.cat(rows), want[:p])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batch_equals_each_alone(device, dtype):
    cfg = steady_cfg(dtype)
    sd = checkpoint(cfg, 9, dtype)
    a, b, c = tokens(40, 4), tokens(5, 5), tokens(1, 6)
    if dtype == "float32":
        wa, wb, wc = (oracle(t, cfg, sd) for t in (a, b, c))
    else:
        # each request alone through the framework, whole and in one step
        wa, wb, wc = (executor(cfg, sd, device, dtype).prefill_slots(
            [0], [t], want=[list(range(len(t)))])[0].float().cpu()
            for t in (a, b, c))
    ex = executor(cfg, sd, device, dtype, slots=4)
    got = ex.prefill_slots([3, 1, 0], [a[:30], b[:3], c],
                           want=[[0, 29], [2], [0]])
    close(got[0], wa[[0, 29]], dtype)
    close(got[1], wb[2:3], dtype)
    close(got[2], wc, dtype)
    for i in range(2):                      # decoded together
        lg = decode_step(ex, {3: a[30 + i], 1: b[3 + i]})
        close(lg[3:4], wa[30 + i].view(1, -1), dtype)
        close(lg[1:2], wb[3 + i].view(1, -1), dtype)
    for i in range(32, 40):                 # the shorter request has ended
        lg = decode_step(ex, {3: a[i]})
        close(lg[3:4], wa[i].view(1, -1), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_slot_freed_and_used_again(device):
    """A slot that held a long request is taken by a new one without any
    reset: cache rows, recurrent states and convolution tails of the
    old request do not leak."""
    cfg = base_cfg()
    sd = checkpoint(cfg, 10)
    a, b = tokens(60, 7), tokens(20, 8)
    ex = executor(cfg, sd, device, slots=2)
    ex.prefill_slots([1], [a[:50]])
    for t in range(50, 60):
        decode_step(ex, {1: a[t]})
    wb = oracle(b, cfg, sd)
    ex.kvs[0].pos[1] = 0
    got = ex.prefill_slots([1], [b[:12]], want=[[0, 5, 11]])[0]
    close(got, wb[[0, 5, 11]])
    for t in range(12, 20):
        close(decode_step(ex, {1: b[t]})[1:2], wb[t].view(1, -1))


OTHER = [
    # everything of size 1 that can be, dense only
    dict(pattern="apg", layers=3, heads=1, kv_heads=1, dim=2, vdim=1,
         rot_dims=2, window=1, keep_first=0, left_heads=1, left_kv_heads=1,
         left_dim=1, left_vdim=1, left_rot_dims=0, conv=1, mem_heads=1,
         mem_dim=1, mem_vdim=1, gla_heads=1, gla_dim=1, gla_vdim=1, ff=1,
         experts=0),
    # no attention layer; every expert taken
    dict(pattern="ggp", layers=3, experts=3, top=3, groups=1, keep_groups=1,
         expert_ff=5, conv=2),
    # only attention, no value mixing, no mask, no rotation
    dict(pattern="aa", layers=2, v_mix=False, window=0, rot_dims=0,
         experts=4, top=1, groups=0),
    # parallel layers only; wide states in several column tiles; one key/value
    # head for sixteen (the grouped-heads decode kernel in bf16)
    dict(pattern="pp", layers=2, left_heads=16, left_kv_heads=1, left_dim=8,
         left_vdim=24, left_rot_dims=8, mem_dim=20, mem_vdim=150,
         expert_ff=8),
    # window and kept tokens longer than the prompt, every layer kind last
    dict(pattern="pga", layers=3, window=64, keep_first=40, conv=6,
         gla_vdim=70, tau=1.0, gate_cap=1.5),
    # no feed-forward in the dense layers
    dict(pattern="gapa", layers=4, ff=0, eps=0.01, groups=9, keep_groups=5),
]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", OTHER)
def test_other_sizes(device, kw):
    cfg = base_cfg(**kw)
    sd = checkpoint(cfg, 11)
    a, b = tokens(33, 9), tokens(7, 10)
    wa, wb = oracle(a, cfg, sd), oracle(b, cfg, sd)
    ex = executor(cfg, sd, device, slots=2)
    got = ex.prefill_slots([0, 1], [a[:25], b[:4]],
                           want=[list(range(25)), [3]], chunk=9)
    close(got[0], wa[:25])
    close(got[1], wb[3:4])
    for i in range(3):
        lg = decode_step(ex, {0: a[25 + i], 1: b[4 + i]})
        close(lg[0:1], wa[25 + i].view(1, -1))
        close(lg[1:2], wb[4 + i].view(1, -1))


@pytest.mark.parametrize("device", DEVICES)
def test_cache_filled_to_its_last_row(device):
    """A request that ends on the cache's last position, its prompt padded
    beside a longer one."""
    cfg = base_cfg()
    sd = checkpoint(cfg, 14)
    a, b = tokens(64, 13), tokens(50, 14)
    wa, wb = oracle(a, cfg, sd), oracle(b, cfg, sd)
    ex = executor(cfg, sd, device, smax=64)
    got = ex.prefill_slots([0, 2], [a[:60], b[:45]], want=[[59], [44]])
    close(got[0], wa[59:60])
    close(got[1], wb[44:45])
    for i in range(4):
        lg = decode_step(ex, {0: a[60 + i], 2: b[45 + i]})
        close(lg[0:1], wa[60 + i].view(1, -1))
        close(lg[2:3], wb[45 + i].view(1, -1))


@pytest.mark.gpu
def test_decode_graph_replays_match_eager():
    """Captured decode steps, replayed with eager prefills and host syncs in
    between, equal the eager steps every time (warm-up runs of the capture
    must not advance any slot's state)."""
    cfg = steady_cfg("bfloat16")
    sd = checkpoint(cfg, 12, "bfloat16")
    a, b = tokens(40, 31), tokens(30, 32)
    runs = []
    for graphs in (False, True):
        ex = executor(cfg, sd, "cuda:0", "bfloat16", use_graphs=graphs)
        out = [ex.prefill_slots([1], [a[:30]], want=[[0, 29]])[0].float().cpu()]
        for t in range(30, 35):
            out.append(decode_step(ex, {1: a[t]})[1:2])
        out.append(ex.prefill_slots([2], [b[:25]],
                                    want=[[3, 24]])[0].float().cpu())
        for t in range(5):
            lg = decode_step(ex, {1: a[35 + t], 2: b[25 + t]})
            out.append(lg[1:3])
            torch.cuda.synchronize()
        runs.append(torch.cat(out))
    torch.testing.assert_close(runs[1], runs[0], atol=2e-2, rtol=2e-2)


# ---------- generation through the scheduler, trace replay ----------

def write_checkpoint(path: Path, cfg, sd):
    from safetensors.torch import save_file
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in sd.items()},
              str(path / "model.safetensors"))


def oracle_greedy(prompt, n, cfg, sd):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(oracle(seq, cfg, sd)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_slot_scheduler(tmp_path, device,
                                                  monkeypatch):
    """Requests queued at the shard runtime are admitted into slots (more
    requests than slots), prefilled, decoded as one batch with idle rows in
    it and sampled greedily; every token equals the oracle's argmax."""
    if device == "cpu":
        monkeypatch.setattr(torch.cuda, "is_available", lambda: False)
    from dnet_amd.core.types import ShardLoadModelRequest
    from dnet_amd.shard.runtime import ShardRuntime
    cfg = base_cfg()
    cfg["vocab"] = 59
    sd = checkpoint(cfg, 15)
    write_checkpoint(tmp_path / "m", cfg, sd)
    emitted: dict = {}

    class Cap:
        def send(self, frame):
            emitted.setdefault(frame["nonce"], []).append(
                (frame["token_id"], frame["finished"]))

        def close(self):
            pass

    rt = ShardRuntime("probe")
    monkeypatch.setattr(rt.settings.storage, "repack_on_load", False)
    rt._load(ShardLoadModelRequest(
        model_path=str(tmp_path / "m"), total_layers=7,
        layers=list(range(7)), max_batch=2, max_seq=96, dtype="float32"))
    assert (rt.executor.device.type == "cuda") == device.startswith("cuda")
    rt._callback = Cap()
    prompts = {"a": tokens(9, 1, 59), "b": tokens(2, 2, 59),
               "c": tokens(23, 3, 59)}
    n_new = {"a": 6, "b": 9, "c": 4}
    for name in ("a", "b", "c"):            # c waits for a slot to free up
        rt.infer_q.put({"nonce": name, "prompt_len": len(prompts[name]),
                        "tokens": prompts[name].to(torch.int32).numpy()
                        .tobytes(), "max_tokens": n_new[name],
                        "stop_ids": [], "params": {}})
    for _ in range(60):
        rt._slots_tick()
        if all(emitted.get(k) and emitted[k][-1][1] for k in prompts):
            break
    for name, p in prompts.items():
        got = [t for t, _ in emitted[name]]
        assert got == oracle_greedy(p.tolist(), n_new[name], cfg, sd), name
    rt._unload()


def test_repacked_weights_load(tmp_path, monkeypatch):
    """The per-layer repacked weight cache holds every tensor of the family:
    a second load reads it and gives the same logits."""
    monkeypatch.setattr(torch.cuda, "is_available", lambda: False)
    monkeypatch.setenv("DNET_REPACK_DIR", str(tmp_path / "repack"))
    from dnet_amd.core.types import ShardLoadModelRequest
    from dnet_amd.shard.runtime import ShardRuntime
    cfg = base_cfg()
    sd = checkpoint(cfg, 17)
    write_checkpoint(tmp_path / "m", cfg, sd)
    a = tokens(12, 5)
    outs = []
    for _ in range(2):
        rt = ShardRuntime("probe")
        rt._load(ShardLoadModelRequest(
            model_path=str(tmp_path / "m"), total_layers=7,
            layers=list(range(7)), max_batch=2, max_seq=64, dtype="float32"))
        outs.append(rt.executor.prefill_slots([0], [a])[0].float().cpu())
        rt._unload()
    close(outs[0], oracle(a, cfg, sd)[-1:])
    assert torch.equal(outs[0], outs[1])


@pytest.mark.gpu
def test_trace_replay_cli_gpu(tmp_path):
    test_trace_replay_cli(tmp_path, "bfloat16")
    test_trace_replay_cli(tmp_path / "f", "float32")


def test_trace_replay_cli(tmp_path, dtype="float32"):
    """bin/trace_run on a tiny checkpoint: a prompt batch of unequal
    requests (more than the initial slot count), decode steps together, a
    request that sits steps out, requests that end early, a slot used
    again by a new request."""
    cfg = steady_cfg(dtype)
    cfg["vocab"] = 53
    sd = checkpoint(cfg, 16, dtype)
    write_checkpoint(tmp_path / "m", cfg, sd)
    a, b = tokens(14, 1, 53).tolist(), tokens(4, 2, 53).tolist()
    c, d = tokens(12, 3, 53).tolist(), tokens(6, 4, 53).tolist()
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:11], "want": [0, 10]},
                                {"id": "b", "tokens": b[:2], "want": []},
                                {"id": "c", "tokens": c[:10], "want": [9]}],
         "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[11:12], "want": [0]},
                                {"id": "b", "tokens": b[2:3], "want": [0]}],
         "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[12:13], "want": []},
                                {"id": "b", "tokens": b[3:4], "want": [0]}],
         "end": ["b"]},
        {"step": 3, "entries": [{"id": "a", "tokens": a[13:14], "want": [0]}],
         "end": ["a"]},
        {"step": 4, "entries": [{"id": "c", "tokens": c[10:11], "want": [0]}],
         "end": []},
        {"step": 5, "entries": [{"id": "d", "tokens": d[:5], "want": [4]}],
         "end": []},
        {"step": 6, "entries": [{"id": "c", "tokens": c[11:12], "want": [0]},
                                {"id": "d", "tokens": d[5:6], "want": [0]}],
         "end": ["c", "d"]},
    ]
    root = Path(__file__).resolve().parents[1]
    import os

    import numpy as np

    def replay(out, hide_gpu=False):
        env = dict(os.environ)
        if hide_gpu:
            env["HIP_VISIBLE_DEVICES"] = env["CUDA_VISIBLE_DEVICES"] = ""
        r = subprocess.run(
            [sys.executable, str(root / "bin" / "trace_run"), "--model",
             str(tmp_path / "m"), "--dtype", dtype, "--out", str(out),
             "--max-tokens", "48", "--max-batch", "2"],
            input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
            capture_output=True, timeout=600, env=env)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [l for l in r.stdout.splitlines() if l.startswith("done")] \
            == [f"done {i}" for i in range(7)]
        return [torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4")
                                 .reshape(-1, 53)) for i in range(7)]

    got = replay(tmp_path / "out")
    if dtype == "float32":
        w = {n: oracle(t, cfg, sd) for n, t in
             (("a", a), ("b", b), ("c", c), ("d", d))}
        want = [torch.cat([w["a"][[0, 10]], w["c"][9:10]]),
                torch.stack([w["a"][11], w["b"][2]]), w["b"][3:4],
                w["a"][13:14], w["c"][10:11], w["d"][4:5],
                torch.stack([w["c"][11], w["d"][5]])]
    else:
        # bfloat16: the same replay on the CPU reference ops
        want = replay(tmp_path / "ref", hide_gpu=True)
    for g, x in zip(got, want):
        close(g, x, dtype)


# ---------- pipeline stages (gloo, two processes) ----------

def _ring_run(rank, world):
    cfg = base_cfg(pattern="gapgaa", layers=6)      # cut: g a p | g a a
    mc = ModelConfig.from_hf(cfg)
    mc.compute_dtype = "float32"
    ex = RingExecutor(mc, rank, world, "cpu", mb_count=1, mb_size=2, smax=64,
                      seed=7, use_graphs=False)
    if world == 2:
        assert ex.hidden_width == W + 2 * 6
        assert (1 in ex.kvs[0].local) == (rank == 0)
    g = torch.Generator().manual_seed(21)
    first = ex.prefill(torch.randint(0, V, (1, 2, 13), generator=g), chunk=5)
    steps = []
    ex.decode_stream(6, on_token=lambda s, t, last: steps.append(t.clone()))
    if rank:
        return None
    return torch.cat([first.view(2, 1)] + [t.view(2, 1) for t in steps], -1)


def _ring_rank_main(rank, world, port, q):
    import os
    os.environ.update(RANK=str(rank), WORLD_SIZE=str(world),
                      MASTER_ADDR="127.0.0.1", MASTER_PORT=str(port),
                      LOCAL_RANK=str(rank))
    import torch.distributed as dist
    dist.init_process_group("gloo", rank=rank, world_size=world)
    out = _ring_run(rank, world)
    if rank == 0:
        q.put(out.tolist())
    dist.destroy_process_group()


@pytest.mark.timeout(360)
def test_two_stage_ring_matches_single():
    """Layers split over two pipeline stages between the first value-mixing
    layer and those that read its values: the step's values ride the hops
    beside the fp32 residual, and the generated tokens equal the single-stage
    run."""
    import multiprocessing as mp
    import socket
    ctx = mp.get_context("spawn")

    def run(world):
        s = socket.socket()
        s.bind(("127.0.0.1", 0))
        port = s.getsockname()[1]
        s.close()
        q = ctx.Queue()
        procs = [ctx.Process(target=_ring_rank_main, args=(r, world, port, q))
                 for r in range(world)]
        for p in procs:
            p.start()
        out = q.get(timeout=200)
        for p in procs:
            p.join(timeout=60)
            assert p.exitcode == 0
        return out

    single, out = run(1), run(2)
    assert len(single) == 2 and len(single[0]) >= 6
    assert out == single


def test_synthetic_preset_runs():
    """The preset builds with seeded random weights and generates the same
    tokens whatever the slot a prompt sits in."""
    from dnet_amd.models import PRESETS
    mc = ModelConfig.from_hf(dict(PRESETS["fedinex-tiny"]))
    ex = RingExecutor(mc, 0, 1, "cpu", mb_size=2, smax=96, seed=3,
                      use_graphs=False)
    toks = torch.randint(0, 256, (1, 2, 30),
                         generator=torch.Generator().manual_seed(1))
    toks[0, 1] = toks[0, 0]
    first = ex.prefill(toks)
    gen = ex.decode_rounds(6)
    assert torch.equal(first[0, 0], first[0, 1])
    assert torch.equal(gen[0, 0], gen[0, 1])
    with pytest.raises(NotImplementedError):
        RingExecutor(mc, 0, 1, "cpu", mb_size=1, smax=32, residency=2,
                     use_graphs=False)
