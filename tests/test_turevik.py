"""Turevik in the framework against the plain oracle (tests/turevik_oracle.py).

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

import turevik_oracle as O
from dnet_amd import ops
from dnet_amd.models import ModelConfig
from dnet_amd.models.config import turevik_config
from dnet_amd.parallel.ring import RingExecutor

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
F64 = torch.float64
V = 83
W = 48


def base_cfg(**kw):
    """Six layers: rows of its own, shared rows, minGRU without a
    feed-forward, own, minGRU, shared; the two sharing layers have other
    heads, sizes and scales than the owners; a dense feed-forward first, then
    mixtures (the last one without a shared expert)."""
    args = dict(pattern="lsglgs", layers=6, heads=3, dim=10, rot_dim=6,
                vdim=14, kv_rank=22, gru_width=56, ff=40, experts=5, top=2,
                expert_ff=20, shared_ff=28, rot_base=300.0, eps=1e-5)
    args.update(kw)
    cfg = copy.deepcopy(turevik_config(W, V, **args))
    if args["pattern"] == "lsglgs":
        cfg["layers"][2]["mlp"] = None
        cfg["layers"][5]["mlp"].pop("shared", None)
        for i, h, d, dv in ((1, 2, 12, 6), (5, 5, 4, 10)):
            m = cfg["layers"][i]["mixer"]
            m.update(heads=h, dim=d, vdim=dv, scale=0.9 * m["scale"])
    return cfg


def steady_cfg(dtype, **kw):
    """The base stack; for bfloat16 runs a shallower one (every layer of
    these tiny random models multiplies rounding noise)."""
    if dtype == "bfloat16":
        kw = dict(dict(pattern="lsg", layers=3), **kw)
    return base_cfg(**kw)


def checkpoint(cfg, seed, dtype="float32"):
    return O.make_checkpoint(cfg, seed,
                             out_gain=1.0 if dtype == "float32" else 0.5)


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
    from dnet_amd.models import TurevikRingModel, get_ring_model
    cfg = base_cfg()
    mc = ModelConfig.from_hf(cfg)
    assert mc.model_type == "turevik" and mc.num_layers == 6
    assert get_ring_model("turevik") is TurevikRingModel
    assert mc.num_experts == 5 and mc.num_experts_per_tok == 2
    assert mc.shared_expert_intermediate_size == 28
    ex = executor(cfg, checkpoint(cfg, 1), "cpu")
    kv = ex.kvs[0]
    assert ex.hidden_width == W
    owns = [0, 3]
    for i in range(6):
        if i in owns:           # one row per token, no separate values
            assert kv.k[i].shape == (3, 1, 160, 28) and kv.v[i] is None
        else:
            assert kv.k[i] is None
        assert kv.state[i]["h"].shape == (3, W)
    assert kv.state[2]["S"].shape == (3, 56)
    assert all(t.dtype == torch.float32 for st in kv.state
               for t in st.values())
    for bad in ("x", "sl"):
        with pytest.raises(ValueError):
            base_cfg(pattern=bad, layers=2)

    def broken(change):
        c = base_cfg()
        change(c["layers"])
        with pytest.raises(ValueError):
            ModelConfig.from_hf(c)

    broken(lambda l: l[1].update(type="mystery"))
    broken(lambda l: l[1]["mixer"].update(kv_from=1))       # itself
    broken(lambda l: l[1]["mixer"].update(kv_from=3))       # a later layer
    broken(lambda l: l[5]["mixer"].update(kv_from=1))       # not an owner
    broken(lambda l: l[5]["mixer"].update(kv_from=2))       # another kind
    broken(lambda l: l[5]["mixer"].update(kv_rank=23))
    broken(lambda l: l[0]["mixer"].pop("scale"))
    broken(lambda l: l[0]["mixer"]["rot"].update(dims=4))
    broken(lambda l: l[3]["mlp"]["router"].update(top=6))
    broken(lambda l: l[0]["mlp"].update(kind="mystery"))


# ---------- mechanisms alone ----------

def _mixer_alone(device, cfg, sd, u, T0, portion=None, lids=(0,)):
    """Run mixers on given inputs u [T, W] through the cache: the first T0
    rows as one prompt portion (or portions), then row by row. Returns the
    last listed layer's output."""
    T = u.shape[0]
    ex = executor(cfg, sd, device, smax=max(160, T))
    m, kv = ex.model, ex.kvs[0]
    slot = torch.tensor([2], dtype=torch.int32, device=device)
    steps, p = [], 0
    while p < T0:
        n = min(portion or T0, T0 - p)
        steps.append((p, n))
        p += n
    steps += [(t, 1) for t in range(T0, T)]
    outs = []
    for p0, n in steps:
        pos = torch.tensor([p0], dtype=torch.int32, device=device)
        ln = torch.tensor([n], dtype=torch.int32, device=device)
        x = u[p0:p0 + n].to(torch.float32).to(device).contiguous()
        for lid in lids:
            fn = {"latent_attention": m._latent_attention,
                  "mingru": m._mingru}[m.cfg.layer_specs[lid]["type"]]
            o = fn(x, m.layers[lid], lid, kv, pos, n, ln, slot)
        outs.append(o.float().cpu())
    return torch.cat(outs)


def _attention_want(u, cfg, sd, lid=0):
    m, eps = cfg["layers"][lid]["mixer"], cfg["norm"]["eps"]
    src = m.get("kv_from", lid)
    rows = O.latent_rows(u.to(F64), sub64(sd, f"l{src}.mix."),
                         cfg["layers"][src]["mixer"], eps)
    return O.latent_attention(u.to(F64), sub64(sd, f"l{lid}.mix."), m, eps,
                              rows)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [
    {}, dict(heads=1, dim=3, rot_dim=2, vdim=1, kv_rank=5),
    dict(heads=16, dim=8, rot_dim=4, vdim=6, kv_rank=12),
    dict(heads=2, dim=5, rot_dim=16, vdim=33, kv_rank=40, rot_base=5e4)])
def test_latent_attention_alone(device, kw):
    """Latent attention on its own inputs: prompt portion, then token by
    token through the cache, equals the oracle's whole-sequence result."""
    cfg = base_cfg(**dict(dict(pattern="l", layers=1), **kw))
    sd = checkpoint(cfg, 3)
    u = torch.randn(41, W, generator=torch.Generator().manual_seed(9))
    want = _attention_want(u, cfg, sd)
    for T0, portion in ((29, None), (30, 7), (2, 2)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_layer_reading_another_layers_rows(device):
    """A layer without rows of its own: the owner's rows, with its own
    queries, up-projections, scale and sinks (other head counts and sizes)."""
    cfg = base_cfg()
    sd = checkpoint(cfg, 4)
    u = torch.randn(37, W, generator=torch.Generator().manual_seed(8))
    for lids in ((0, 1), (3, 5)):
        want = _attention_want(u, cfg, sd, lids[1])
        for T0, portion in ((25, None), (24, 5), (1, None)):
            close(_mixer_alone(device, cfg, sd, u, T0, portion, lids), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("width", [56, 48, 1, 130])
def test_mingru_alone(device, width):
    cfg = base_cfg(pattern="g", layers=1, gru_width=width)
    sd = checkpoint(cfg, 5)
    T = 83
    u = torch.randn(T, W, generator=torch.Generator().manual_seed(9))
    want = O.mingru(u.to(F64), sub64(sd, "l0.mix."),
                    cfg["layers"][0]["mixer"], cfg["norm"]["eps"])
    for T0, portion in ((71, None), (70, 7), (2, 2)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_far_token_through_the_recurrent_state(device):
    """Gates that stay almost shut after one standout token: what it wrote
    is still most of the state 300 tokens on, in a prompt, across portions
    and in decoding. The oracle without that token differs grossly."""
    cfg = base_cfg(pattern="g", layers=1, gru_width=24)
    sd = checkpoint(cfg, 6)
    sd["l0.mix.z.b"] = torch.full((24,), -9.0, dtype=torch.bfloat16)
    T = 310
    u = torch.randn(T, W, generator=torch.Generator().manual_seed(11)) * 0.3
    u[5] = u[5] * 60
    spec = cfg["layers"][0]["mixer"]
    p64 = sub64(sd, "l0.mix.")
    want = O.mingru(u.to(F64), p64, spec, 1e-5)
    quiet = u.clone()
    quiet[5] = u[6]
    other = O.mingru(quiet.to(F64), p64, spec, 1e-5)
    assert float((other[-1] - want[-1]).abs().max()) \
        > 0.5 * float(want[-1].abs().max())
    for T0, portion in ((T, None), (T - 10, 33), (7, None)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_far_key_stands_out(device):
    """One key hundreds of positions back, met by a matching query at the
    end, carries that row; with the keys one position off (a rotation or an
    append that is one row out) the row would be something else."""
    cfg = base_cfg(pattern="l", layers=1, heads=2, dim=24, rot_dim=8, vdim=8,
                   kv_rank=32, rot_base=40.0)
    sd = checkpoint(cfg, 7)
    T, far = 320, 11
    u = torch.randn(T, W, generator=torch.Generator().manual_seed(12))
    m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    p = sub64(sd, "l0.mix.")
    c, kr = O.latent_rows(u.to(F64), p, m, eps)
    k = (c @ p["uk"].T).view(T, 2, 24)
    # head 0's query at the end: along the far token's plain key, and along
    # its rotated key part once turned to the last position
    aim = torch.cat([k[far, 0], O.turn_pairs(kr[far], -(T - 1), 40.0, 8)])
    u[T - 1] = (torch.linalg.pinv(p["q"][:32]) @ aim).float()
    m["scale"] = 1.0
    want = _attention_want(u, cfg, sd)
    c, kr = O.latent_rows(u.to(F64), p, m, eps)
    k = (c @ p["uk"].T).view(T, 2, 24)
    q = (u.to(F64)[-1] @ p["q"].T).view(2, 32)

    def far_weight(at):
        qr = O.turn_pairs(q[0, 24:], at, 40.0, 8)
        return float(O.sink_softmax(k[:, 0] @ q[0, :24] + kr @ qr,
                                    p["sink"][0])[far])
    assert far_weight(T - 1) > 0.9 and far_weight(T) < far_weight(T - 1)
    for T0, portion in ((T, None), (T - 1, None), (T - 5, 64), (13, 12)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_sink_is_counted_once_and_unscaled(device):
    """Sinks of the scores' size: leaving them out, scaling them or counting
    them per key changes the oracle's result grossly (most at the first
    tokens); the framework equals the true one."""
    cfg = base_cfg(pattern="l", layers=1)
    sd = checkpoint(cfg, 8)
    sd["l0.mix.sink"] = torch.tensor([1.5, 3.0, -2.0], dtype=torch.bfloat16)
    u = torch.randn(40, W, generator=torch.Generator().manual_seed(13))
    want = _attention_want(u, cfg, sd)
    for wrong in ([-1e4] * 3, [0.4, 0.8, -0.5]):
        other = dict(sd)
        other["l0.mix.sink"] = torch.tensor(wrong)
        d = (_attention_want(u, cfg, other) - want).abs()
        assert float(d[0].max()) > 0.2 * float(want.abs().mean())
    for T0, portion in ((40, None), (1, None), (33, 2)):
        close(_mixer_alone(device, cfg, sd, u, T0, portion), want)


@pytest.mark.parametrize("device", DEVICES)
def test_norm_and_token_shift_alone(device):
    """Norm weights around zero, the shift towards the token before (across
    portions, decode steps and slots with stale state, zero before the first
    token), and the residual update that goes with it in decode steps."""
    g = torch.Generator().manual_seed(14)
    T = 23
    x = torch.randn(T, W, generator=g) * 3
    w, mu = torch.randn(W, generator=g) * 0.3, torch.rand(W, generator=g)
    wa = torch.randn(W, generator=g) * 0.3
    a = torch.randn(T, W, generator=g)
    after = x.to(F64) + O.norm_around_one(a.to(F64), wa.to(F64), 1e-5)
    want = O.token_shift(O.norm_around_one(after, w.to(F64), 1e-5),
                         mu.to(F64))
    slot = torch.tensor([1], dtype=torch.int32, device=device)
    for cuts in ((23,), (5, 1, 1, 2, 14), (1, 22), (2, 2, 17, 2)):
        prev = torch.full((3, W), 7.0, device=device)       # stale state
        out, res, p = [], [], 0
        for n in cuts:
            xs = x[p:p + n].clone().to(device)
            out.append(ops.resid_norm_token_shift(
                xs, a[p:p + n].to(device).contiguous(), (1 + wa).to(device),
                (1 + w).to(device), mu.to(device), prev,
                torch.tensor([p], dtype=torch.int32, device=device), n, 1e-5,
                torch.float32,
                torch.tensor([n], dtype=torch.int32, device=device),
                slot).cpu())
            res.append(xs.cpu())
            p += n
        close(torch.cat(out), want)
        close(torch.cat(res), after)
        assert bool((prev[[0, 2]] == 7.0).all())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("rows", [1, 3, 40, 90])
@pytest.mark.parametrize("kw", [
    {}, dict(top=1), dict(top=5), dict(shared_ff=0, experts=9, top=3),
    dict(experts=1, top=1, shared_ff=4)])
def test_experts_alone(device, rows, kw):
    """Mixture of experts on every row-count path (few rows, grouped, sorted
    prompts; as a captured-style decode step too): scores neither
    renormalized nor applied to the output, shared expert behind its gate."""
    cfg = base_cfg(**dict(dict(pattern="lg", layers=2), **kw))
    sd = checkpoint(cfg, 9)
    # scores well inside (0, 1)
    sd["l1.mlp.router"] = sd["l1.mlp.router"] * 0.25
    ff = cfg["layers"][1]["mlp"]
    h = torch.randn(rows, W, generator=torch.Generator().manual_seed(15)) * 2
    p64 = sub64(sd, "l1.mlp.")
    want = O.moe(h.to(F64), p64, ff)
    # the weight on the output instead of the input is another function
    s = O.sigmoid(h.to(F64) @ p64["router"].T)
    wrong = torch.zeros_like(want)
    for t in range(rows):
        for e in torch.topk(s[t], ff["router"]["top"]).indices.tolist():
            wrong[t] += s[t, e] * O.gated_ff(h[t].to(F64), p64, f"e{e}.",
                                             O.silu)
    if ff.get("shared"):
        wrong += O.sigmoid(h.to(F64) @ p64["shared.sg"].T) * O.gated_ff(
            h.to(F64), p64, "shared.", O.silu)
    assert float((wrong - want).pow(2).mean().sqrt()) > \
        0.05 * float(want.pow(2).mean().sqrt())
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
    cfg = base_cfg(pattern="l", layers=1, ff=37)
    sd = checkpoint(cfg, 10)
    h = torch.randn(6, W, generator=torch.Generator().manual_seed(16)) * 3
    want = O.gated_ff(h.to(F64), sub64(sd, "l0.mlp."), "", O.gelu_tanh)
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
    reset: cache rows, recurrent states and shift inputs of the old
    request do not leak."""
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
    # one head everywhere, everything of size 1 that can be, dense only
    dict(pattern="lsg", layers=3, heads=1, dim=1, rot_dim=2, vdim=1,
         kv_rank=1, gru_width=1, ff=1, experts=0),
    # no recurrent layer, two sharers in a row, every expert taken
    dict(pattern="lss", layers=3, heads=4, dim=7, rot_dim=4, vdim=5,
         kv_rank=9, experts=3, top=3, expert_ff=5, shared_ff=1),
    # recurrent layers only at the start, an owner nobody shares
    dict(pattern="ggl", layers=4, gru_width=100, experts=12, top=1,
         shared_ff=0, expert_ff=8),
    # sixteen heads on one row (the grouped-heads decode kernel in bf16), a
    # single expert, value size above the key size
    dict(pattern="lgs", layers=3, heads=16, dim=8, rot_dim=8, vdim=24,
         kv_rank=24, experts=1, top=1, gru_width=W, rot_base=7.0),
    # no feed-forward at all in the first layer
    dict(pattern="lsgs", layers=4, ff=0, experts=4, top=2, eps=0.01),
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
def test_rows_wider_than_the_kernels_key_row(device, monkeypatch):
    """When the latent row does not fit one key row of the attention kernels
    every layer that reads it caches per-head keys and values: same logits,
    through ragged prompts, portions, batched decode with an idle row."""
    from dnet_amd.models import TurevikRingModel
    monkeypatch.setattr(TurevikRingModel, "MAX_LATENT_ROW", 20)
    cfg = base_cfg()                        # rows of 22 + 6
    sd = checkpoint(cfg, 13)
    a, b = tokens(33, 11), tokens(6, 12)
    wa, wb = oracle(a, cfg, sd), oracle(b, cfg, sd)
    ex = executor(cfg, sd, device, slots=3)
    assert ex.kvs[0].state[1]["xk"].shape == (3, 2, 160, 18)
    got = ex.prefill_slots([2, 0], [a[:25], b[:3]],
                           want=[list(range(25)), [2]], chunk=7)
    close(got[0], wa[:25])
    close(got[1], wb[2:3])
    for i in range(3):
        lg = decode_step(ex, {2: a[25 + i], 0: b[3 + i]})
        close(lg[2:3], wa[25 + i].view(1, -1))
        close(lg[0:1], wb[3 + i].view(1, -1))
    for i in range(28, 33):
        close(decode_step(ex, {2: a[i]})[2:3], wa[i].view(1, -1))
    with pytest.raises(NotImplementedError):
        monkeypatch.setattr(TurevikRingModel, "MAX_LATENT_ROW", 4)
        executor(cfg, sd, device)


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
        model_path=str(tmp_path / "m"), total_layers=6,
        layers=list(range(6)), max_batch=2, max_seq=96, dtype="float32"))
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
            model_path=str(tmp_path / "m"), total_layers=6,
            layers=list(range(6)), max_batch=2, max_seq=64, dtype="float32"))
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
    cfg = base_cfg(pattern="lggsls", layers=6)      # cut: l g g | s l s
    mc = ModelConfig.from_hf(cfg)
    mc.compute_dtype = "float32"
    ex = RingExecutor(mc, rank, world, "cpu", mb_count=1, mb_size=2, smax=64,
                      seed=7, use_graphs=False)
    if world == 2:
        assert ex.hidden_width == W + 28 + 28
        assert ex.model.foreign == ([0] if rank else [])
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
    """Layers split over two pipeline stages between a row-owning layer and
    one that reads its rows: the step's rows ride the hops beside the fp32
    residual, and the generated tokens equal the single-stage run."""
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
    mc = ModelConfig.from_hf(dict(PRESETS["turevik-tiny"]))
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
