"""Turevik ring model: shared-latent attention and minGRU layers with a token
shift, norms on both sides of every sublayer, mixtures of experts.

    h  = rmsnorm(x) * (1 + g1)                 (norm weights stored around 0)
    h <- h + (h_prev - h) * mu                 (token shift, per element)
    x <- x + rmsnorm(mixer(h)) * (1 + g1b)
    x <- x + rmsnorm(ff(rmsnorm(x) * (1 + g2))) * (1 + g2b)
    logits = embed (rmsnorm(x) * (1 + gf))     (the embedding table, tied)

``h_prev`` is the previous token's h before its own shift (zero for a
sequence's first token); every layer keeps it per slot.

Mixers (``cfg.layer_specs[l]["type"]``):

* ``latent_attention``: one cached row per token serves all heads as key and
  value: [RMS-normed latent | rotated key part] (interleaved rotation). Each
  head's plain query part is carried through its key up-projection, the
  scores are taken against the cached rows, the weighted sum of the latents
  goes through the head's value up-projection. Full causal softmax with a
  learned sink per head in the denominator. A layer with ``kv_from`` = j owns
  no rows: it reads those of the earlier layer j with its own queries,
  up-projections and sinks.
* ``mingru``: S <- (1 - z) S + z * candidate per channel, with z and the
  candidate computed from the step's input alone (no state feedback, so a
  prompt is a scan of affine maps); output gated by silu.

Feed-forwards: dense (gelu-gated) or a mixture of silu-gated experts: sigmoid
router, the largest ``top`` scores kept as they are, each score multiplying
its expert's INPUT; an optional shared expert behind a sigmoid gate. The
router and that gate are one fp32 product.

Per-slot state lives in the framework's cache object: the latent rows in
``KVCache.k`` (layers that own rows), the fp32 shift input and the fp32
recurrent state in ``KVCache.state``. State is taken as zero at position 0
and never touched by padding or idle rows, so slots are reused without a
reset and a ragged batch equals each row alone.

When a latent row is wider than the attention kernels' key row, every layer
that reads it also caches per-head keys and values formed from it.

Pipeline stages may separate a layer from the one whose rows it reads: the
rows of this step's tokens then ride the hops beside the residual
(``hidden_width``), and the later stage appends them to a cache of its own.

Checkpoint names: ``embed``, ``final.norm``, ``l<i>.norm{1,1b,2,2b}``,
``l<i>.shift``, ``l<i>.mix.{q,dkv,dkv.norm,uk,uv,sink,o}``,
``l<i>.mix.{z,z.b,x,x.b,g,o}``, ``l<i>.mlp.{gate,up,down}``,
``l<i>.mlp.{router,e<j>.{gate,up,down},shared.{gate,up,down,sg}}``.

``cfg.compute_dtype == "float32"`` runs weights, activations, caches and every
product in true fp32.
"""
from __future__ import annotations

from typing import Optional, Sequence

import torch

from .. import ops
from .base import KVCache, LayerWeights, Linear, RingModel
from .config import ModelConfig


class TurevikRingModel(RingModel):
    model_type = "turevik"
    model_types = ["turevik"]
    act_dtype = torch.float32          # residual stream / ring hops
    ragged_prefill = True
    supports_float32 = True
    stateful = True                    # idle decode rows must not step
    supports_offload = False           # layer kinds hold different tensors
    # the attention kernels hold one key row of at most this many entries
    MAX_LATENT_ROW = 256
    # rows up to which the experts run as grouped products over all rows
    # (weights read once, no host sync); above, rows are sorted by expert
    GROUPED_MAX_T = 64

    def __init__(self, cfg: ModelConfig, layer_ids: Sequence[int], device,
                 is_first: bool, is_last: bool, smax: int = 4096, **kw):
        if kw.get("tp_size", 1) > 1 or kw.get("cp_size", 1) > 1:
            raise NotImplementedError(
                "turevik: tensor/context parallelism inside a stage is not "
                "implemented")
        assert cfg.layer_specs is not None, "turevik needs per-layer specs"
        assert cfg.quant is None, "turevik: bf16 / fp32 weights only"
        super().__init__(cfg, layer_ids, device, is_first, is_last,
                         smax=smax, **kw)
        self.wdtype = (torch.float32 if cfg.compute_dtype == "float32"
                       else torch.bfloat16)
        self.logits_dtype = self.wdtype
        # columns of the hops that carry shared rows between stages: one
        # span per row-owning layer that another layer reads, the same on
        # every stage (none when one stage holds the whole stack)
        self.row_cols: dict = {}
        self._row_width = 0
        if not (is_first and is_last):
            for s in cfg.layer_specs:
                j = s["mixer"].get("kv_from")
                if j is not None and j not in self.row_cols:
                    self.row_cols[j] = cfg.hidden_size + self._row_width
                    self._row_width += self._row_size(
                        cfg.layer_specs[j]["mixer"])
        # owners on earlier stages whose rows layers here read
        self.foreign = sorted({self._owner(l) for l in self.layer_ids
                               if self._spec(l)["type"] == "latent_attention"}
                              - set(self.layer_ids))
        for lid in self.layer_ids:
            m = self._spec(lid)["mixer"]
            if self._spec(lid)["type"] == "latent_attention" \
                    and not self._row_fits(m) and max(
                        m["dim"] + m["rot_dim"], m["vdim"]) \
                    > self.MAX_LATENT_ROW:
                raise NotImplementedError(
                    f"turevik layer {lid}: neither the latent row "
                    f"({self._row_size(m)}) nor the per-head key / value "
                    f"sizes fit the attention kernels' row of "
                    f"{self.MAX_LATENT_ROW}")

    def _init_positional(self):
        pass        # angles are computed from positions inside the kernels

    @property
    def hidden_width(self) -> int:
        return self.cfg.hidden_size + self._row_width

    # ---------- per-layer sizes ----------

    def _spec(self, lid: int) -> dict:
        return self.cfg.layer_specs[lid]

    def _owner(self, lid: int) -> int:
        """The layer whose latent rows layer ``lid`` reads."""
        j = self._spec(lid)["mixer"].get("kv_from")
        return lid if j is None else int(j)

    @staticmethod
    def _row_size(m: dict) -> int:
        return m["kv_rank"] + m["rot_dim"]

    def _row_fits(self, m: dict) -> bool:
        return self._row_size(m) <= self.MAX_LATENT_ROW

    def make_kv_cache(self, batch: int, smax: int) -> KVCache:
        W = self.cfg.hidden_size
        dims, states = [], []
        for lid in self.layer_ids:
            s = self._spec(lid)
            m = s["mixer"]
            st = {"h": ((W,), torch.float32)}
            own = None
            if s["type"] == "mingru":
                st["S"] = ((m["width"],), torch.float32)
            else:
                if self._owner(lid) == lid:
                    own = (1, self._row_size(m), 0)
                if not self._row_fits(m):
                    st["xk"] = ((m["heads"], smax, m["dim"] + m["rot_dim"]),
                                self.wdtype)
                    st["xv"] = ((m["heads"], smax, m["vdim"]), self.wdtype)
            dims.append(own)
            states.append(st)
        # caches for the rows of layers on earlier stages, filled from the
        # hops; they sit behind the local layers
        for j in self.foreign:
            dims.append((1, self._row_size(self._spec(j)["mixer"]), 0))
            states.append({})
        return KVCache(self.cfg, self.layer_ids + self.foreign, batch, smax,
                       self.device, layer_dims=dims, dtype=self.wdtype,
                       layer_state=states)

    # ---------- weights ----------

    def _mat(self, w: torch.Tensor) -> torch.Tensor:
        return w.to(self.wdtype).to(self.device).contiguous()

    def _lin(self, w: torch.Tensor) -> Linear:
        return Linear(self._mat(w))

    def _vec(self, t: torch.Tensor) -> torch.Tensor:
        # small per-channel / per-head parameters feed fp32 math directly
        return t.to(torch.float32).to(self.device).contiguous()

    def _build_layer(self, lid: int, get) -> LayerWeights:
        """``get(name)`` returns the tensor ``l<lid>.<name>``."""
        s = self._spec(lid)
        m = s["mixer"]
        W = self.cfg.hidden_size
        # norm weights are stored around zero: the kernels take 1 + w
        lw = LayerWeights(attn_norm=self._vec(get("norm1")) + 1.0)
        lw.post_norm = self._vec(get("norm1b")) + 1.0
        lw.shift = self._vec(get("shift"))
        assert lw.attn_norm.shape == lw.post_norm.shape == lw.shift.shape \
            == (W,), f"layer {lid}: norm / shift shapes"
        if s["type"] == "mingru":
            D = m["width"]
            z, x, g = (get("mix." + n) for n in "zxg")
            assert z.shape == x.shape == g.shape == (D, W), \
                f"layer {lid}: recurrence shapes"
            lw.qkv = self._lin(torch.cat([z, x, g]))        # [z | x | g]
            lw.z_bias = self._vec(get("mix.z.b"))
            lw.x_bias = self._vec(get("mix.x.b"))
            assert lw.z_bias.shape == lw.x_bias.shape == (D,)
        else:
            H, d, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
            R = m["kv_rank"]
            q, uk, uv = get("mix.q"), get("mix.uk"), get("mix.uv")
            assert q.shape == (H * (d + rd), W) and uk.shape == (H * d, R) \
                and uv.shape == (H * dv, R), f"layer {lid}: attention shapes"
            if self._owner(lid) == lid:
                dkv = get("mix.dkv")
                assert dkv.shape == (R + rd, W), f"layer {lid}: dkv shape"
                q = torch.cat([q, dkv])                     # [q | dkv]
                lw.kv_a_norm = self._vec(get("mix.dkv.norm"))
            lw.qkv = self._lin(q)
            # per-head up-projections as batched operands: keys [H, d, R]
            # (query side: q_h W_uk,h), values [H, R, dv]
            lw.uk = self._mat(uk).view(H, d, R)
            lw.uv = self._mat(self._mat(uv).view(H, dv, R).transpose(1, 2))
            if not self._row_fits(m):
                lw.kv_b = self._lin(torch.cat([uk, uv]))    # [uk ; uv]
            lw.sinks = self._vec(get("mix.sink"))
            assert lw.sinks.shape == (H,)
            n = int(m["rot"]["dims"])
            lw.rot_freq = torch.tensor(
                [float(m["rot"]["base"]) ** (-2.0 * i / n)
                 for i in range(n // 2)],
                dtype=torch.float32, device=self.device)
        lw.o = self._lin(get("mix.o"))
        ff = s.get("mlp")
        if ff is None:
            return lw
        lw.mlp_norm = self._vec(get("norm2")) + 1.0
        lw.ff_post_norm = self._vec(get("norm2b")) + 1.0
        if ff["kind"] == "dense":
            gate, up = get("mlp.gate"), get("mlp.up")
            assert gate.shape == up.shape == (ff["ff"], W)
            lw.gateup = self._lin(torch.cat([gate, up]))
            lw.down = self._lin(get("mlp.down"))
            return lw
        E = int(ff["router"]["experts"])
        router = [get("mlp.router")]
        assert router[0].shape == (E, W), f"layer {lid}: router shape"
        if ff.get("shared"):
            # the shared expert's gate is one more row of the fp32 product
            router.append(get("mlp.shared.sg"))
            lw.shared_gateup = self._lin(torch.cat(
                [get("mlp.shared.gate"), get("mlp.shared.up")]))
            lw.shared_down = self._lin(get("mlp.shared.down"))
        lw.router_w = self._vec(torch.cat([r.float() for r in router]))
        lw.gateup_w = self._mat(torch.stack(
            [torch.cat([get(f"mlp.e{e}.gate"), get(f"mlp.e{e}.up")])
             for e in range(E)]))                            # [E, 2I, W]
        lw.down_w = self._mat(torch.stack(
            [get(f"mlp.e{e}.down") for e in range(E)]))      # [E, W, I]
        assert lw.gateup_w.shape[1] == 2 * ff["expert"]["ff"]
        return lw

    def _finish_ends(self, embed, final_norm):
        emb = self._mat(embed)
        if self.is_first:
            self.embed = emb
        if self.is_last:
            self.final_norm = self._vec(final_norm) + 1.0
            self.lm_head = Linear(emb)

    def load_state_dict(self, sd: dict):
        for lid in self.layer_ids:
            self.layers[lid] = self._build_layer(
                lid, lambda n, p=f"l{lid}.": sd[p + n])
        if self.is_first or self.is_last:
            self._finish_ends(sd["embed"], sd.get("final.norm"))

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
            t = {n: rn(g, W, std=0.1)
                 for n in ("norm1", "norm1b", "norm2", "norm2b")}
            t["shift"] = torch.rand(W, generator=g, device=gdev) \
                .to(torch.bfloat16)
            if s["type"] == "mingru":
                D = m["width"]
                t.update({"mix.z": lin(g, D, W), "mix.z.b": rn(g, D),
                          "mix.x": lin(g, D, W),
                          "mix.x.b": rn(g, D, std=0.5),
                          "mix.g": lin(g, D, W), "mix.o": lin(g, W, D)})
            else:
                H, d, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
                R = m["kv_rank"]
                t.update({"mix.q": lin(g, H * (d + rd), W),
                          "mix.dkv": lin(g, R + rd, W),
                          "mix.dkv.norm": 1 + rn(g, R, std=0.1),
                          "mix.uk": lin(g, H * d, R),
                          "mix.uv": lin(g, H * dv, R),
                          "mix.sink": rn(g, H), "mix.o": lin(g, W, H * dv)})
            ff = s.get("mlp")
            if ff is not None and ff["kind"] == "dense":
                t.update({"mlp.gate": lin(g, ff["ff"], W),
                          "mlp.up": lin(g, ff["ff"], W),
                          "mlp.down": lin(g, W, ff["ff"])})
            elif ff is not None:
                t["mlp.router"] = lin(g, ff["router"]["experts"], W)
                parts = [(f"e{e}", ff["expert"]["ff"])
                         for e in range(ff["router"]["experts"])]
                if ff.get("shared"):
                    parts.append(("shared", ff["shared"]["ff"]))
                    t["mlp.shared.sg"] = lin(g, 1, W)
                for n, I in parts:
                    t.update({f"mlp.{n}.gate": lin(g, I, W),
                              f"mlp.{n}.up": lin(g, I, W),
                              f"mlp.{n}.down": lin(g, W, I)})
            self.layers[lid] = self._build_layer(lid, t.__getitem__)
        if self.is_first or self.is_last:
            self._finish_ends(rn(gen(99991), c.vocab_size, W),
                              rn(gen(99993), W, std=0.1))

    # ---------- forward ----------

    def embed_tokens(self, tokens: torch.Tensor) -> torch.Tensor:
        """fp32 residual rows [..., hidden_width] (columns of the hops that
        carry shared rows are filled by the layers that own them)."""
        assert self.embed is not None, "this shard does not own the embedding"
        x = torch.nn.functional.embedding(tokens, self.embed).to(
            torch.float32)
        if self._row_width:
            x = torch.nn.functional.pad(x, (0, self._row_width))
        return x

    def _latent_attention(self, u, lw, lid, kv, pos, T, lens, slots):
        m = self._spec(lid)["mixer"]
        H, d, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
        R = m["kv_rank"]
        M = u.shape[0]
        nq = H * (d + rd)
        p = lw.qkv(u)                                  # [q | dkv]
        owner = self._owner(lid)
        rows = kv.k[kv.local[owner]]
        if owner == lid:
            ops.latent_append(p, nq, lw.kv_a_norm, self.cfg.rms_eps, R,
                              lw.rot_freq, rows, pos, T, lens, slots)
        # plain query parts, head by head (a strided view)
        qh = p[:, :nq].view(M, H, d + rd)[:, :, :d].transpose(0, 1)
        if not self._row_fits(m):
            return self._expanded_attention(p, qh, rows, lw, lid, kv, pos, T,
                                            lens, slots)
        qabs = torch.bmm(qh, lw.uk)                    # [H, M, R]
        qf = ops.latent_q_pack(p, qabs, lw.rot_freq, pos, T, H, d)
        ol = ops.attn_mod(qf, rows, None, pos, T, float(m["scale"]), lens,
                          slots, sinks=lw.sinks, v_dim=R)    # [M, H*R]
        ov = torch.bmm(ol.view(M, H, R).transpose(0, 1), lw.uv)
        return lw.o(ov.transpose(0, 1).reshape(M, H * dv))

    def _step_rows(self, rows, pos, T, slots):
        """The cached rows of this step's tokens, [B*T, D] (rows of padding
        tokens hold anything)."""
        B = pos.shape[0]
        at = (pos.view(B, 1).long()
              + torch.arange(T, device=rows.device)).clamp_(
                  max=rows.shape[2] - 1)
        sl = (slots.long() if slots is not None
              else torch.arange(B, device=rows.device)).view(B, 1)
        return rows[sl, 0, at].reshape(B * T, -1)

    def _expanded_attention(self, p, qh, rows, lw, lid, kv, pos, T, lens,
                            slots):
        """Latent rows too wide for one key row of the kernels: per-head keys
        [plain | rotated shared part] and values are formed from this step's
        rows and cached beside them."""
        m = self._spec(lid)["mixer"]
        H, d, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
        R = m["kv_rank"]
        M = p.shape[0]
        st = kv.state[kv.local[lid]]
        B = M // T
        row = self._step_rows(rows, pos[:B], T, slots)
        kvu = lw.kv_b(row[:, :R].contiguous())         # [ku (H*d) | v (H*dv)]
        k = torch.cat([kvu[:, :H * d].view(M, H, d),
                       row[:, R:].view(M, 1, rd).expand(M, H, rd)],
                      dim=-1).reshape(M, H * (d + rd)).contiguous()
        ops.cache_append(k, 0, st["xk"], pos, T, lens, slots)
        ops.cache_append(kvu, H * d, st["xv"], pos, T, lens, slots)
        # the query pack turns the rotated parts and copies the plain ones
        q = ops.latent_q_pack(p, qh.contiguous(), lw.rot_freq, pos, T, H, d)
        return lw.o(ops.attn_mod(q, st["xk"], st["xv"], pos, T,
                                 float(m["scale"]), lens, slots,
                                 sinks=lw.sinks))

    def _mingru(self, u, lw, lid, kv, pos, T, lens, slots):
        D = self._spec(lid)["mixer"]["width"]
        y = ops.mingru_scan(lw.qkv(u), 0, D, 2 * D, lw.z_bias, lw.x_bias,
                            kv.state[kv.local[lid]]["S"], pos, T, lens, slots)
        return lw.o(y)

    def _moe(self, u, lw, ff, step: bool):
        """Routed experts (inputs scaled by their scores) plus the gated
        shared expert. ``step``: a decode step, which must not sync with the
        host (it may be captured)."""
        E, top = int(ff["router"]["experts"]), int(ff["router"]["top"])
        M, W = u.shape
        I = lw.gateup_w.shape[1] // 2
        idx, val, we, gate = ops.moe_router(u, lw.router_w, E, top)
        shared = None
        if gate is not None:
            shared = lw.shared_down(ops.gated_act(lw.shared_gateup(u),
                                                  "silu"))
        if step or M <= self.GROUPED_MAX_T:
            if self.wdtype == torch.bfloat16 and W % 8 == 0 and I % 8 == 0:
                act = ops.moe_gateup_rows(u, lw.gateup_w, we)
                y = ops.moe_down_rows(act, lw.down_w, we)
            else:
                # every expert on every row; rows that did not choose it
                # have scale 0 and are not merged
                y = torch.stack([
                    ops.gated_act(u @ lw.gateup_w[e].t(), "silu",
                                  we[:, e].contiguous())
                    @ lw.down_w[e].t() for e in range(E)])
            return ops.moe_merge(y, idx, shared, gate, self.wdtype)
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
        act = ops.gated_act(gu, "silu", scale)
        for e, a, b in spans:
            torch.mm(act[a:b], lw.down_w[e].t(), out=y[a:b])
        return ops.moe_merge(y, at, shared, gate, self.wdtype)

    def _ff(self, u, lw, ff, step: bool):
        if ff["kind"] == "dense":
            return lw.down(ops.gated_act(lw.gateup(u), "gelu_tanh"))
        return self._moe(u, lw, ff, step)

    def _window(self, x: torch.Tensor, layer_ids: Sequence[int], kv: KVCache,
                pos: torch.Tensor, T: int, lens, slots, step: bool) -> None:
        """Run the layers of one window over x [B*T, W] fp32 (in place).
        Token (b, t) sits at position pos[b]+t of cache row slots[b]."""
        eps, wdt = self.cfg.rms_eps, self.wdtype
        mixers = {"latent_attention": self._latent_attention,
                  "mingru": self._mingru}
        u = None
        layer_ids = list(layer_ids)
        for i, lid in enumerate(layer_ids):
            lw = self._layer(lid)
            s = self._spec(lid)
            if u is None:
                u = ops.norm_token_shift(
                    x, lw.attn_norm, lw.shift, kv.state[kv.local[lid]]["h"],
                    pos, T, eps, wdt, lens, slots)
            a = mixers[s["type"]](u, lw, lid, kv, pos, T, lens, slots)
            post = lw.post_norm
            if s.get("mlp") is not None:
                u2, _ = ops.resid_branches_rmsnorm(
                    x, a, post, None, None, 1.0, None, lw.mlp_norm, eps, wdt)
                a = self._ff(u2, lw, s["mlp"], step)
                post = lw.ff_post_norm
            nxt = layer_ids[i + 1] if i + 1 < len(layer_ids) else None
            if nxt is not None:
                ln = self._layer(nxt)
                u = ops.resid_norm_token_shift(
                    x, a, post, ln.attn_norm, ln.shift,
                    kv.state[kv.local[nxt]]["h"], pos, T, eps, wdt, lens,
                    slots)
            else:
                ops.resid_branches_rmsnorm(x, a, post, None, None, 1.0, None,
                                           None, eps, wdt)
            if self._obs_sync:
                self._profile_layer_sync(lid)

    def _run(self, h, layer_ids, kv, pos, T, lens, slots, step):
        """One window over h [B*T, hidden_width]: unpack the rows that came
        with the hop, run the layers, pack the rows this window made."""
        if not self._row_width:
            self._window(h, layer_ids, kv, pos, T, lens, slots, step)
            return
        W = self.cfg.hidden_size
        here = {self._owner(l) for l in layer_ids
                if self._spec(l)["type"] == "latent_attention"}
        for j in self.foreign:
            if j in here:
                ops.cache_append(h, self.row_cols[j], kv.k[kv.local[j]], pos,
                                 T, lens, slots)
        x = h[:, :W].contiguous()
        self._window(x, layer_ids, kv, pos, T, lens, slots, step)
        h[:, :W].copy_(x)
        for j, c in self.row_cols.items():
            if j in layer_ids:
                rows = kv.k[kv.local[j]]
                h[:, c:c + rows.shape[3]] = self._step_rows(
                    rows, pos[:h.shape[0] // T], T, slots).float()

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
        if self._row_width:
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
