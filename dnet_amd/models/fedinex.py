"""Fedinex ring model: windowed attention with value mixing, convolved attention
beside a matrix memory, and gated linear attention on an fp32 residual.

    x <- x + mixer(rmsnorm(x) * g1)
    x <- x + ff(rmsnorm(x) * g2)
    logits = head (rmsnorm(x) * gf)

Mixers (``cfg.layer_specs[l]["type"]``):

* ``attention``: grouped heads with projection biases, half-split rotation of
  the first channels of a head, softmax over a sliding window plus the first
  ``mask.keep_first`` tokens (at their true positions). Value mixing: in every
  layer with ``v_mix`` but the first such one, v <- (1 - lam) v + lam v_first,
  v_first being that first layer's values of the same token; the mixed values
  are what is cached.
* ``parallel``: two mixers read the same input and their results, each times a
  constant, are added. Left: full causal attention whose q, k and v run
  through a short causal convolution, interleaved rotation, one sigmoid gate
  per head on the result. Right: matrix memory with exponential gates
  (soft-capped) and a running maximum, per-head RMS norm, sigmoid gate.
* ``gla``: linear attention with a decay per key channel,
  sigmoid(A2 A1 h + b)^(1/tau); per-head RMS norm, silu gate.

Feed-forwards: a dense clamped gated unit or a mixture of such experts:
sigmoid router, chosen by score + correction among the best groups of
neighbouring experts, weighted by the plain score times a constant.

Both halves of a parallel layer share one input product and one output
product: the left heads leave the attention kernel already gated and scaled,
the right heads are scaled through their norm weight, side by side in one
buffer.

Per-slot state lives in the framework's cache object: keys and values in
``KVCache.k`` / ``KVCache.v``, the convolution's input tail and the fp32
recurrent states (matrix, normalizer, maximum) in ``KVCache.state``. State is
taken as zero at position 0 and never touched by padding or idle rows, so
slots are reused without a reset and a ragged batch equals each row alone.

v_first is read back from the first mixing layer's value cache. A pipeline
stage without that layer gets the step's values beside the residual on the
hops (``hidden_width``).

Checkpoint names: ``embed``, ``head``, ``final.norm``, ``l<i>.norm{1,2}``,
``l<i>.mix.{q,q.b,k,k.b,v,v.b,vmix,o,o.b}``,
``l<i>.mix.left.{q,q.conv,k,k.conv,v,v.conv,g,o}``,
``l<i>.mix.right.{q,k,v,g,i,i.b,f,f.b,norm,o}``,
``l<i>.mix.{q,k,v,g,a1,a2,a2.b,norm,o}``, ``l<i>.mlp.{gate,up,down}``,
``l<i>.mlp.{router,correction,e<j>.{gate,up,down}}``.

``cfg.compute_dtype == "float32"`` runs weights, activations, caches and every
product in true fp32.
"""
from __future__ import annotations

from typing import Optional, Sequence

import torch

from .. import ops
from .base import KVCache, LayerWeights, Linear, RingModel
from .config import ModelConfig

GLU_ALPHA = 1.702               # sigmoid slope of the clamped gated unit


class FedinexRingModel(RingModel):
    model_type = "fedinex"
    model_types = ["fedinex"]
    act_dtype = torch.float32          # residual stream / ring hops
    ragged_prefill = True
    supports_float32 = True
    stateful = True                    # idle decode rows must not step
    supports_offload = False           # layer kinds hold different tensors
    MAX_HEAD = 256                     # the attention kernels' key / value row
    MAX_STATE_ROWS = 512               # key size of the recurrences' kernels
    # rows up to which the experts run as grouped products over all rows
    # (weights read once, no host sync); above, rows are sorted by expert
    GROUPED_MAX_T = 64

    def __init__(self, cfg: ModelConfig, layer_ids: Sequence[int], device,
                 is_first: bool, is_last: bool, smax: int = 4096, **kw):
        if kw.get("tp_size", 1) > 1 or kw.get("cp_size", 1) > 1:
            raise NotImplementedError(
                "fedinex: tensor/context parallelism inside a stage is not "
                "implemented")
        assert cfg.layer_specs is not None, "fedinex needs per-layer specs"
        assert cfg.quant is None, "fedinex: bf16 / fp32 weights only"
        super().__init__(cfg, layer_ids, device, is_first, is_last,
                         smax=smax, **kw)
        self.wdtype = (torch.float32 if cfg.compute_dtype == "float32"
                       else torch.bfloat16)
        self.logits_dtype = self.wdtype
        mixing = [i for i, s in enumerate(cfg.layer_specs)
                  if s["type"] == "attention" and s["mixer"].get("v_mix")]
        # the layer whose values the later mixing layers read
        self.v_layer: Optional[int] = mixing[0] if mixing else None
        # columns of the hops that carry those values between stages (none
        # when one stage holds the whole stack, or nobody reads them)
        self._v_width = 0
        if len(mixing) > 1 and not (is_first and is_last):
            m = cfg.layer_specs[mixing[0]]["mixer"]
            self._v_width = m["kv_heads"] * m["vdim"]
        for lid in self.layer_ids:
            s = self._spec(lid)
            m = s["mixer"]
            at = m if s["type"] == "attention" else m.get("left")
            if at is not None and max(at["dim"], at["vdim"]) > self.MAX_HEAD:
                raise NotImplementedError(
                    f"fedinex layer {lid}: head sizes {at['dim']} / "
                    f"{at['vdim']} exceed the attention kernels' row of "
                    f"{self.MAX_HEAD}")
            rec = m if s["type"] == "gla" else m.get("right")
            if rec is not None and rec["dim"] > self.MAX_STATE_ROWS:
                raise NotImplementedError(
                    f"fedinex layer {lid}: key size {rec['dim']} exceeds the "
                    f"recurrence kernels' {self.MAX_STATE_ROWS}")

    def _init_positional(self):
        pass        # angles are computed from positions inside the kernels

    @property
    def hidden_width(self) -> int:
        return self.cfg.hidden_size + self._v_width

    # ---------- per-layer sizes ----------

    def _spec(self, lid: int) -> dict:
        return self.cfg.layer_specs[lid]

    @staticmethod
    def _qkv_cols(m: dict) -> int:
        return m["heads"] * m["dim"] + m["kv_heads"] * (m["dim"] + m["vdim"])

    def make_kv_cache(self, batch: int, smax: int) -> KVCache:
        dims, states = [], []
        for lid in self.layer_ids:
            s = self._spec(lid)
            m = s["mixer"]
            st = {}
            if s["type"] == "gla":
                dims.append(None)
                st["S"] = ((m["heads"], m["dim"], m["vdim"]), torch.float32)
            elif s["type"] == "attention":
                dims.append((m["kv_heads"], m["dim"], m["vdim"]))
            else:
                lf, rt = m["left"], m["right"]
                dims.append((lf["kv_heads"], lf["dim"], lf["vdim"]))
                nt = ops.scan_tiles(rt["dim"], rt["vdim"])
                st = {"conv": ((int(lf["conv"]) - 1, self._qkv_cols(lf)),
                               self.wdtype),
                      "S": ((rt["heads"], rt["dim"], rt["vdim"]),
                            torch.float32),
                      "n": ((rt["heads"], nt, rt["dim"]), torch.float32),
                      "m": ((rt["heads"], nt), torch.float32)}
            states.append(st)
        return KVCache(self.cfg, self.layer_ids, batch, smax, self.device,
                       layer_dims=dims, dtype=self.wdtype,
                       layer_state=states)

    # ---------- weights ----------

    def _mat(self, w: torch.Tensor) -> torch.Tensor:
        return w.to(self.wdtype).to(self.device).contiguous()

    def _lin(self, w: torch.Tensor, bias=None) -> Linear:
        return Linear(self._mat(w), None if bias is None else self._mat(bias))

    def _vec(self, t: torch.Tensor) -> torch.Tensor:
        # small per-channel / per-head parameters feed fp32 math directly
        return t.to(torch.float32).to(self.device).contiguous()

    def _freq(self, m: dict) -> Optional[torch.Tensor]:
        rot = m.get("rot")
        n = int(rot["dims"]) if rot else 0
        if n < 2:
            return None
        return torch.tensor(
            [float(rot["base"]) ** (-2.0 * i / n) for i in range(n // 2)],
            dtype=torch.float32, device=self.device)

    def _build_layer(self, lid: int, get) -> LayerWeights:
        """``get(name)`` returns the tensor ``l<lid>.<name>``."""
        s = self._spec(lid)
        m = s["mixer"]
        W = self.cfg.hidden_size
        lw = LayerWeights(attn_norm=self._vec(get("norm1")))
        assert lw.attn_norm.shape == (W,), f"layer {lid}: norm shape"
        if s["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            w = torch.cat([get("mix." + n) for n in "qkv"])
            assert w.shape == (self._qkv_cols(m), W), f"layer {lid}: q/k/v"
            lw.qkv = self._lin(w)
            # added in fp32 where the rows are rotated and appended
            lw.qkv_bias = self._vec(torch.cat([get(f"mix.{n}.b")
                                               for n in "qkv"]))
            lw.rot_freq = self._freq(m)
            lw.lam = None
            if m.get("v_mix") and lid != self.v_layer:
                lw.lam = self._vec(get("mix.vmix").reshape(1))
            lw.o = self._lin(get("mix.o"), get("mix.o.b"))
            assert lw.o.w.shape == (W, H * dv), f"layer {lid}: o"
        elif s["type"] == "parallel":
            lf, rt = m["left"], m["right"]
            H, d, dv = rt["heads"], rt["dim"], rt["vdim"]
            parts = [get("mix.left." + n) for n in "qkv"] \
                + [get("mix.right." + n) for n in "qkvg"] \
                + [get("mix.left.g"), get("mix.right.i"), get("mix.right.f")]
            assert [p.shape[0] for p in parts] == [
                lf["heads"] * lf["dim"], lf["kv_heads"] * lf["dim"],
                lf["kv_heads"] * lf["vdim"], H * d, H * d, H * dv, H * dv,
                lf["heads"], H, H], f"layer {lid}: projection shapes"
            # columns of the product: q k v | q k v g | left gate, i, f
            at = [0]
            for p in parts:
                at.append(at[-1] + p.shape[0])
            lw.cols = dict(zip(("rq", "rk", "rv", "rg", "lg", "ri", "rf"),
                               at[3:10]))
            pad = -at[-1] % 16
            parts.append(torch.zeros(pad, W, dtype=parts[0].dtype,
                                     device=parts[0].device))
            lw.qkv = self._lin(torch.cat(parts))
            lw.conv_w = self._vec(torch.cat([get(f"mix.left.{n}.conv")
                                             for n in "qkv"]))
            assert lw.conv_w.shape == (self._qkv_cols(lf), int(lf["conv"])), \
                f"layer {lid}: convolution shape"
            lw.rot_freq = self._freq(lf)
            lw.i_bias = self._vec(get("mix.right.i.b"))
            lw.f_bias = self._vec(get("mix.right.f.b"))
            # the right half's factor rides on its norm weight
            lw.mix_norm = self._vec(get("mix.right.norm")) \
                * float(m["right_scale"])
            assert lw.mix_norm.shape == (H * dv,), f"layer {lid}: norm"
            lw.o = self._lin(torch.cat([get("mix.left.o"),
                                        get("mix.right.o")], dim=1))
        else:
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            parts = [get("mix." + n) for n in ("q", "k", "v", "g", "a1")]
            assert [p.shape[0] for p in parts[:4]] == [H * d, H * d, H * dv,
                                                       H * dv], \
                f"layer {lid}: projection shapes"
            pad = -sum(p.shape[0] for p in parts) % 16
            parts.append(torch.zeros(pad, W, dtype=parts[0].dtype,
                                     device=parts[0].device))
            lw.qkv = self._lin(torch.cat(parts))    # [q | k | v | g | a1]
            # second half of the decay's projection, fp32 and transposed
            lw.a2t = self._vec(get("mix.a2").float().t())
            lw.a2_b = self._vec(get("mix.a2.b"))
            assert lw.a2t.shape == (parts[4].shape[0], H * d) \
                and lw.a2_b.shape == (H * d,), f"layer {lid}: decay shapes"
            # the heads share one weight vector
            assert get("mix.norm").shape == (dv,), f"layer {lid}: norm"
            lw.mix_norm = self._vec(get("mix.norm").repeat(H))
            lw.o = self._lin(get("mix.o"))
        ff = s.get("mlp")
        if ff is None:
            return lw
        lw.mlp_norm = self._vec(get("norm2"))
        if ff["kind"] == "dense":
            gate, up = get("mlp.gate"), get("mlp.up")
            assert gate.shape == up.shape == (ff["ff"], W), f"layer {lid}: ff"
            lw.gateup = self._lin(torch.cat([gate, up]))
            lw.down = self._lin(get("mlp.down"))
            return lw
        E = int(ff["router"]["experts"])
        lw.router_w = self._vec(get("mlp.router"))
        lw.correction = self._vec(get("mlp.correction"))
        assert lw.router_w.shape == (E, W) and lw.correction.shape == (E,), \
            f"layer {lid}: router shapes"
        lw.gateup_w = self._mat(torch.stack(
            [torch.cat([get(f"mlp.e{e}.gate"), get(f"mlp.e{e}.up")])
             for e in range(E)]))                            # [E, 2I, W]
        lw.down_w = self._mat(torch.stack(
            [get(f"mlp.e{e}.down") for e in range(E)]))      # [E, W, I]
        assert lw.gateup_w.shape[1] == 2 * ff["expert"]["ff"]
        return lw

    def _finish_ends(self, embed, final_norm, head):
        if self.is_first:
            self.embed = self._mat(embed)
        if self.is_last:
            self.final_norm = self._vec(final_norm)
            self.lm_head = self._lin(head)

    def load_state_dict(self, sd: dict):
        for lid in self.layer_ids:
            self.layers[lid] = self._build_layer(
                lid, lambda n, p=f"l{lid}.": sd[p + n])
        self._finish_ends(sd.get("embed"), sd.get("final.norm"),
                          sd.get("head"))

    def init_random(self, seed: int = 0):
        """Seeded per layer id (any sharding of one (model, seed) holds the
        same global weights); scales keep every branch of comparable size."""
        c = self.cfg
        W = c.hidden_size
        gdev = self.device if self.device.type == "cuda" else "cpu"

        def gen(sub):
            g = torch.Generator(device=gdev)
            g.manual_seed(seed * 100003 + sub)
            return g

        def rn(g, *shape, std=1.0):
            return (torch.randn(*shape, generator=g, device=gdev)
                    * std).to(torch.bfloat16)

        def lin(g, out, inp):
            return rn(g, out, inp, std=inp ** -0.5)

        for lid in self.layer_ids:
            g = gen(lid)
            s = self._spec(lid)
            m = s["mixer"]
            t = {n: 1 + rn(g, W, std=0.1) for n in ("norm1", "norm2")}
            if s["type"] == "attention":
                H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
                for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                    t["mix." + n] = lin(g, rows, W)
                    t[f"mix.{n}.b"] = rn(g, rows, std=0.1)
                t.update({"mix.vmix": rn(g, 1, std=0.1) + 0.5,
                          "mix.o": lin(g, W, H * dv),
                          "mix.o.b": rn(g, W, std=0.1)})
            elif s["type"] == "parallel":
                lf, rt = m["left"], m["right"]
                H, G, d, dv = (lf[n] for n in ("heads", "kv_heads", "dim",
                                               "vdim"))
                for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                    t["mix.left." + n] = lin(g, rows, W)
                    t[f"mix.left.{n}.conv"] = rn(g, rows, int(lf["conv"]),
                                                 std=0.5)
                t.update({"mix.left.g": lin(g, H, W),
                          "mix.left.o": lin(g, W, H * dv)})
                H, d, dv = rt["heads"], rt["dim"], rt["vdim"]
                for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv),
                                ("g", H * dv), ("i", H), ("f", H)):
                    t["mix.right." + n] = lin(g, rows, W)
                t.update({"mix.right.i.b": rn(g, H),
                          "mix.right.f.b": rn(g, H) + 3.0,
                          "mix.right.norm": 1 + rn(g, H * dv, std=0.1),
                          "mix.right.o": lin(g, W, H * dv)})
            else:
                H, d, dv = m["heads"], m["dim"], m["vdim"]
                rank = 16
                for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv),
                                ("g", H * dv), ("a1", rank)):
                    t["mix." + n] = lin(g, rows, W)
                t.update({"mix.a2": lin(g, H * d, rank),
                          "mix.a2.b": rn(g, H * d),
                          "mix.norm": 1 + rn(g, dv, std=0.1),
                          "mix.o": lin(g, W, H * dv)})
            ff = s.get("mlp")
            parts = []
            if ff is not None and ff["kind"] == "dense":
                parts = [("", ff["ff"])]
            elif ff is not None:
                E = int(ff["router"]["experts"])
                t["mlp.router"] = lin(g, E, W)
                t["mlp.correction"] = rn(g, E, std=0.1)
                parts = [(f"e{e}.", ff["expert"]["ff"]) for e in range(E)]
            for n, I in parts:
                t.update({f"mlp.{n}gate": lin(g, I, W),
                          f"mlp.{n}up": lin(g, I, W),
                          f"mlp.{n}down": lin(g, W, I)})
            self.layers[lid] = self._build_layer(lid, t.__getitem__)
        self._finish_ends(rn(gen(99991), c.vocab_size, W),
                          1 + rn(gen(99993), W, std=0.1),
                          lin(gen(99992), c.vocab_size, W))

    # ---------- forward ----------

    def embed_tokens(self, tokens: torch.Tensor) -> torch.Tensor:
        """fp32 residual rows [..., hidden_width] (the hops' value columns
        are filled behind the layer that owns the values)."""
        assert self.embed is not None, "this shard does not own the embedding"
        x = torch.nn.functional.embedding(tokens, self.embed).to(
            torch.float32)
        if self._v_width:
            x = torch.nn.functional.pad(x, (0, self._v_width))
        return x

    def _attention(self, u, lw, lid, kv, pos, T, lens, slots, v_hop):
        """``v_hop``: the step's first-layer values [M, kv_heads*vdim] that
        came with the hop, None when that layer's cache is here."""
        m = self._spec(lid)["mixer"]
        li = kv.local[lid]
        vf = None
        if lw.lam is not None:
            vf = kv.v[kv.local[self.v_layer]] if v_hop is None else v_hop
        q = ops.qkv_rope_append(
            lw.qkv(u), 0, m["heads"], m["kv_heads"], m["dim"], m["vdim"],
            kv.k[li], kv.v[li], pos, T, lens, slots, bias=lw.qkv_bias,
            rot_freq=lw.rot_freq, half=True, vf=vf, lam=lw.lam)
        mask = m.get("mask") or {}
        a = ops.attn_mod(q, kv.k[li], kv.v[li], pos, T, float(m["scale"]),
                         lens, slots, window=int(mask.get("size") or 0),
                         keep=int(mask.get("keep_first") or 0), wide=True)
        return lw.o(a)

    def _parallel(self, u, lw, lid, kv, pos, T, lens, slots, v_hop):
        m = self._spec(lid)["mixer"]
        lf, rt = m["left"], m["right"]
        li, c = kv.local[lid], lw.cols
        st = kv.state[li]
        p = lw.qkv(u)
        # both halves' heads side by side: one output product
        nl, nr = lf["heads"] * lf["vdim"], rt["heads"] * rt["vdim"]
        y = (torch.zeros if lens is not None else torch.empty)(
            u.shape[0], nl + nr, dtype=u.dtype, device=u.device)
        q = ops.qkv_rope_append(
            p, 0, lf["heads"], lf["kv_heads"], lf["dim"], lf["vdim"],
            kv.k[li], kv.v[li], pos, T, lens, slots, conv_w=lw.conv_w,
            conv_state=st["conv"], rot_freq=lw.rot_freq)
        ops.attn_mod(q, kv.k[li], kv.v[li], pos, T, float(lf["scale"]), lens,
                     slots, gate=p, gate_col=c["lg"],
                     gate_scale=float(m["left_scale"]), out=y[:, :nl],
                     wide=True)
        ops.mlstm_heads(p, c["rq"], c["rk"], c["rv"], c["ri"], c["rf"],
                        lw.i_bias, lw.f_bias, float(rt["gate_cap"]),
                        rt["dim"] ** -0.5, st["S"], st["n"], st["m"], pos, T,
                        lens, slots, lw.mix_norm, c["rg"], "sigmoid",
                        self.cfg.rms_eps, out=y[:, nl:])
        return lw.o(y)

    def _gla(self, u, lw, lid, kv, pos, T, lens, slots, v_hop):
        m = self._spec(lid)["mixer"]
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        p = lw.qkv(u)                              # [q | k | v | g | a1]
        g0 = 2 * H * d + H * dv
        return lw.o(ops.gla_heads(
            p, 0, H * d, 2 * H * d, g0 + H * dv, lw.a2t, lw.a2_b,
            1.0 / float(m["tau"]), d ** -0.5, kv.state[kv.local[lid]]["S"],
            pos, T, lens, slots, lw.mix_norm, g0, "silu", self.cfg.rms_eps))

    def _moe(self, u, lw, ff, step: bool):
        """Routed experts, their results weighted. ``step``: a decode step,
        which must not sync with the host (it may be captured)."""
        r = ff["router"]
        groups = r.get("groups") or {"count": 1, "keep": 1}
        E, top = int(r["experts"]), int(r["top"])
        limit = float(ff["expert"]["limit"])
        M, W = u.shape
        I = lw.gateup_w.shape[1] // 2
        idx, val, we, _ = ops.moe_router(
            u, lw.router_w, E, top, lw.correction, int(groups["count"]),
            int(groups["keep"]), float(r.get("scale", 1.0)))
        if step or M <= self.GROUPED_MAX_T:
            if self.wdtype == torch.bfloat16 and W % 8 == 0 and I % 8 == 0:
                act = ops.moe_clamped_rows(u, lw.gateup_w, we, GLU_ALPHA,
                                           limit)
                y = ops.moe_down_rows(act, lw.down_w, we)
            else:
                # every expert on every row; rows that did not choose it
                # have weight 0 and are not merged
                y = torch.stack([
                    ops.gated_act(u @ lw.gateup_w[e].t(), "clamped",
                                  we[:, e].contiguous(), GLU_ALPHA, limit)
                    @ lw.down_w[e].t() for e in range(E)])
            return ops.moe_merge(y, idx, None, None, self.wdtype)
        # prompts: rows sorted by expert, one product per expert and half
        order, at, counts = ops.moe_plan(idx, E)
        xs, scale = ops.moe_gather(u, order, val)
        gu = torch.empty(M * top, 2 * I, dtype=u.dtype, device=u.device)
        y = torch.empty(M * top, W, dtype=u.dtype, device=u.device)
        n = counts.tolist()
        ends = [sum(n[:e + 1]) for e in range(E)]
        spans = [(e, ends[e] - n[e], ends[e]) for e in range(E) if n[e]]
        for e, a, b in spans:
            torch.mm(xs[a:b], lw.gateup_w[e].t(), out=gu[a:b])
        act = ops.gated_act(gu, "clamped", scale, GLU_ALPHA, limit)
        for e, a, b in spans:
            torch.mm(act[a:b], lw.down_w[e].t(), out=y[a:b])
        return ops.moe_merge(y, at, None, None, self.wdtype)

    def _ff(self, u, lw, ff, step: bool):
        if ff["kind"] == "dense":
            return lw.down(ops.gated_act(lw.gateup(u), "clamped", None,
                                         GLU_ALPHA, float(ff["limit"])))
        return self._moe(u, lw, ff, step)

    def _window(self, x: torch.Tensor, layer_ids: Sequence[int], kv: KVCache,
                pos: torch.Tensor, T: int, lens, slots, step: bool,
                v_hop=None) -> None:
        """Run the layers of one window over x [B*T, W] fp32 (in place).
        Token (b, t) sits at position pos[b]+t of cache row slots[b]."""
        eps, wdt = self.cfg.rms_eps, self.wdtype
        mixers = {"attention": self._attention, "parallel": self._parallel,
                  "gla": self._gla}
        u = None
        layer_ids = list(layer_ids)
        for i, lid in enumerate(layer_ids):
            lw = self._layer(lid)
            s = self._spec(lid)
            if u is None:
                u = ops.rmsnorm_rows(x, lw.attn_norm, eps, wdt)
            a = mixers[s["type"]](u, lw, lid, kv, pos, T, lens, slots, v_hop)
            if s.get("mlp") is not None:
                u, _ = ops.resid_branches_rmsnorm(
                    x, a, None, None, None, 1.0, None, lw.mlp_norm, eps, wdt)
                a = self._ff(u, lw, s["mlp"], step)
            nxt = (self._layer(layer_ids[i + 1]).attn_norm
                   if i + 1 < len(layer_ids) else None)
            u, _ = ops.resid_branches_rmsnorm(x, a, None, None, None, 1.0,
                                              None, nxt, eps, wdt)
            if self._obs_sync:
                self._profile_layer_sync(lid)

    def _step_values(self, kv, pos, T, slots):
        """The first mixing layer's cached values of this step's tokens,
        [B*T, kv_heads*vdim] (rows of padding tokens hold anything)."""
        v = kv.v[kv.local[self.v_layer]]
        B = pos.shape[0]
        at = (pos.view(B, 1).long()
              + torch.arange(T, device=v.device)).clamp_(max=v.shape[2] - 1)
        sl = (slots.long() if slots is not None
              else torch.arange(B, device=v.device)).view(B, 1)
        return v[sl, :, at].reshape(B * T, -1)

    def _run(self, h, layer_ids, kv, pos, T, lens, slots, step):
        """One window over h [B*T, hidden_width]: values that came with the
        hop are handed to the mixing layers, this stage's own are packed for
        the next one."""
        if not self._v_width:
            self._window(h, layer_ids, kv, pos, T, lens, slots, step)
            return
        W = self.cfg.hidden_size
        own = self.v_layer in kv.local
        x = h[:, :W].contiguous()
        v_hop = None if own else h[:, W:].to(self.wdtype).contiguous()
        self._window(x, layer_ids, kv, pos, T, lens, slots, step, v_hop)
        h[:, :W].copy_(x)
        if self.v_layer in layer_ids:
            h[:, W:] = self._step_values(kv, pos[:h.shape[0] // T], T,
                                         slots).float()

    def decode_window(self, h: torch.Tensor, layer_ids: Sequence[int],
                      kv: KVCache) -> torch.Tensor:
        """One decode step. h [B, hidden_width] fp32, modified in place;
        kv.pos holds each row's write position; rows flagged in kv.idle keep
        their state (they run as padding)."""
        if layer_ids:
            self._run(h, layer_ids, kv, kv.pos, 1,
                      (~kv.idle).to(torch.int32), None, True)
        return h

    def prefill_window(self, h: torch.Tensor, layer_ids: Sequence[int],
                       kv: KVCache, p0, lens: Optional[torch.Tensor] = None,
                       slots: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Prefill h [B, T, hidden_width] fp32 in place. ``p0``: first
        position, an int (every row) or an int32 tensor [B]. ``lens`` [B]
        int32: real token count per row (rows are right-padded to T; padding
        never reaches the cache or any state and its outputs are
        meaningless). ``slots`` [B] int32: cache row of each batch row
        (default: row b)."""
        if not layer_ids:
            return h
        B, T, HW = h.shape
        if not torch.is_tensor(p0):
            p0 = torch.full((B,), int(p0), dtype=torch.int32,
                            device=h.device)
        self._run(h.view(B * T, HW), layer_ids, kv, p0, T, lens, slots, False)
        return h

    def normalize_project(self, h: torch.Tensor) -> torch.Tensor:
        assert self.final_norm is not None and self.lm_head is not None
        if self._v_width:
            h = h[:, :self.cfg.hidden_size].contiguous()
        y = ops.rmsnorm_rows(h, self.final_norm, self.cfg.rms_eps,
                             self.wdtype)
        return self.lm_head(y)

    def weight_bytes(self) -> int:
        """Bytes of every tensor and linear the resident layers hold (the
        layer kinds carry different sets of them)."""
        def size(v) -> int:
            if isinstance(v, Linear):
                return v.nbytes()
            if torch.is_tensor(v):
                return v.numel() * v.element_size()
            return 0
        return sum(size(v) for lw in self.layers.values()
                   for v in vars(lw).values())
