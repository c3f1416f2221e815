"""Kolotar decoder over the mixer op layer (``ops.mixers``).

Post-norm layers: the fp32 residual itself is normed after every sum, ``x = rms(alpha x +
mixer(x)) w1`` then ``x = rms(alpha x + experts(x)) w2``; the sub-layers read x.  Mixers:

* ``attention`` - grouped-query softmax attention inside a sliding window with biased
  projections, per-head q / k norms, YaRN-scaled rotate-half positions, values normed per head
  and mixed with the first mixing layer's values of the same token, a learned sink per head and
  a sigmoid output gate per head;
* ``latent_attention`` - softmax attention inside a sliding window over ONE cached latent per
  token plus a rotated key part shared by the heads (interleaved pairs), element-wise sigmoid
  output gate;
* ``parallel`` - unnormalised sigmoid attention over all earlier keys (soft-capped scores, a
  number per head, head mixing, q / k normed over the whole projection, a query temperature that
  grows with the position) next to a gated delta rule; the branches are mixed with two
  configured weights.

The feed-forward is a set of SiLU-GLU experts: the largest router logits choose, their softmax
weights the outputs.  The embedding table is the output head.

MI355X layout: every projection that reads a mixer's input is one fused library GEMM (blocks
padded to 8 rows so the kernels read 16-byte aligned slices in place; a fused bias row where the
mixer has biases).  The weighted sum of a layer boundary, its norm and the 16-bit copy the next
GEMM reads are one kernel; the router reads the fp32 residual.  q / k norm, rotation and the K
pages are one kernel, value norm, value mixing and the channel-major V pages another; gates of
the window attention sit in the attention kernel's store.  Latent attention runs absorbed (key
up-projection on the queries, value up-projection on the output), i.e. as multi-query attention
over compressed pages.  The experts run as two grouped matrix-core products over rows sorted by
expert on the device, so a decode step stays capturable as a hipGraph.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from pathlib import Path

import torch
import torch.nn.functional as F

from ..config import KolotarConfig
from ..engine.state_cache import HybridCache, LayerCacheSpec
from ..ops import mixers as mx


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


@dataclass
class KolotarLayerWeights:
    norm1: torch.Tensor
    w_in: torch.Tensor = None                  # fused projections of the mixer's input
    b_in: torch.Tensor | None = None           # fused bias of the same rows
    seg: dict = field(default_factory=dict)    # block name -> (column offset, width)
    q_norm: torch.Tensor | None = None
    k_norm: torch.Tensor | None = None
    inv_freq: torch.Tensor | None = None
    rot_mult: float = 1.0                      # factor on cos and sin
    w_o: torch.Tensor | None = None
    b_o: torch.Tensor | None = None
    # window attention
    sink: torch.Tensor | None = None           # fp32 [H]
    v_lambda: float = 0.0
    # latent attention
    c_norm: torch.Tensor | None = None
    uk: torch.Tensor | None = None             # [H, dim, kv_rank]
    uv_t: torch.Tensor | None = None           # [H, kv_rank, vdim]
    # sigmoid attention
    head_bias: torch.Tensor | None = None      # fp32 [H]
    talk: torch.Tensor | None = None           # fp32 [H, H]
    # delta rule
    conv_w: torch.Tensor | None = None         # [2 G d + H dv, taps] (q, k, v channels)
    a_log: torch.Tensor | None = None          # fp32 [H]
    dt_bias: torch.Tensor | None = None        # fp32 [H]
    out_norm: torch.Tensor | None = None
    delta_o: torch.Tensor | None = None
    # experts
    norm2: torch.Tensor | None = None
    router: torch.Tensor | None = None         # fp32 [E, W]
    router_b: torch.Tensor | None = None       # fp32 [E]
    e_gu: torch.Tensor | None = None           # [E, 2 ff, W]: gate rows, then up rows
    e_down: torch.Tensor | None = None         # [E, W, ff]


class KolotarModel:
    family = "kolotar"
    has_state = True

    def __init__(self, cfg: KolotarConfig, dtype=torch.bfloat16, device="cuda", tp_rank: int = 0,
                 tp_size: int = 1, tp_group=None, quantization: str = ""):
        if tp_size != 1:
            raise ValueError("Kolotar runs on one GPU per replica (tensor_parallel_size 1)")
        if quantization:
            raise ValueError("Kolotar weights are 16-bit or 32-bit; no quantization")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Kolotar activations are bfloat16 or float32")
        self.cfg = cfg
        self.dtype = dtype
        self.device = torch.device(device)
        self.tp_rank, self.tp_size, self.tp_group = 0, 1, None
        self.layers: list[KolotarLayerWeights] = []
        self.embed = self.final_norm = None
        self.vocab_shard = cfg.vocab_size
        if self.dtype == torch.float32 and self.device.type == "cuda":
            # fp32 serving is exact fp32: no reduced-precision matrix mode
            torch.backends.cuda.matmul.allow_tf32 = False
            torch.backends.cudnn.allow_tf32 = False

    # ---------------------------------------------------------------------------------
    def tensor_shapes(self) -> dict:
        """Checkpoint tensor name -> shape for this configuration."""
        c = self.cfg
        W = c.hidden_size
        out = {"embed": (c.vocab_size, W), "final.norm": (W,)}
        for i, L in enumerate(c.layers):
            p, m = f"l{i}.", L.mixer
            x = p + "mix."
            out[p + "norm1"] = (W,)
            if L.kind == "attention":
                nq, nk, nv = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
                out.update({x + "q": (nq, W), x + "q.b": (nq,), x + "k": (nk, W), x + "k.b": (nk,),
                            x + "v": (nv, W), x + "v.b": (nv,), x + "q.norm": (m.dim,),
                            x + "k.norm": (m.dim,), x + "sink": (m.heads,), x + "g": (m.heads, W),
                            x + "o": (W, m.heads * m.vdim), x + "o.b": (W,)})
                if m.v_mix:
                    out[x + "vmix"] = ()
            elif L.kind == "latent_attention":
                out.update({x + "q": (m.heads * (m.dim + m.rot_dim), W),
                            x + "dkv": (m.kv_rank + m.rot_dim, W), x + "dkv.norm": (m.kv_rank,),
                            x + "uk": (m.heads * m.dim, m.kv_rank),
                            x + "uv": (m.heads * m.vdim, m.kv_rank),
                            x + "g": (m.heads * m.vdim, W), x + "o": (W, m.heads * m.vdim)})
            else:
                l, r, d = x + "left.", x + "right.", L.delta
                nq, nk = m.heads * m.dim, m.kv_heads * m.dim
                out.update({l + "q": (nq, W), l + "k": (nk, W), l + "v": (m.kv_heads * m.vdim, W),
                            l + "q.norm": (nq,), l + "k.norm": (nk,), l + "pb": (m.heads,),
                            l + "talk": (m.heads, m.heads), l + "o": (W, m.heads * m.vdim)})
                qk, vv = d.kv_heads * d.dim, d.heads * d.vdim
                out.update({r + "q": (qk, W), r + "q.conv": (qk, d.conv), r + "k": (qk, W),
                            r + "k.conv": (qk, d.conv), r + "v": (vv, W),
                            r + "v.conv": (vv, d.conv), r + "b": (d.heads, W),
                            r + "a": (d.heads, W), r + "A_log": (d.heads,),
                            r + "dt_bias": (d.heads,), r + "norm": (d.vdim,), r + "g": (vv, W),
                            r + "o": (W, vv)})
            if L.moe:
                f = p + "mlp."
                out.update({p + "norm2": (W,), f + "router": (L.moe.experts, W),
                            f + "router.b": (L.moe.experts,)})
                for e in range(L.moe.experts):
                    out.update({f"{f}e{e}.gate": (L.moe.ff, W), f"{f}e{e}.up": (L.moe.ff, W),
                                f"{f}e{e}.down": (W, L.moe.ff)})
        return out

    def random_state(self, seed: int = 0) -> dict:
        """Seeded random tensors under the checkpoint's names (bf16-representable values)."""
        g = torch.Generator().manual_seed(24680 + seed)
        st = {}
        for name, shape in self.tensor_shapes().items():
            r = torch.randn(shape, generator=g)
            leaf = name.split(".")[-1]
            if name == "embed":
                t = r
            elif leaf.startswith("norm"):
                t = 1.0 + 0.1 * r
            elif leaf == "b" and len(shape) == 1:
                t = 0.1 * r
            elif leaf == "conv":
                t = 0.5 * r
            elif leaf == "A_log":
                t = torch.log(0.25 + 2.0 * torch.rand(shape, generator=g))
            elif leaf == "dt_bias":
                t = r - 1.0
            elif leaf == "sink":
                t = r
            elif leaf == "pb":
                t = r - 6.0
            elif leaf == "talk":
                t = torch.eye(shape[0]) + 0.2 * r
            elif leaf == "vmix":
                t = torch.rand(shape, generator=g)
            elif leaf == "router":
                t = 4.0 * r / math.sqrt(shape[-1])
            else:
                t = r / math.sqrt(shape[-1])
            st[name] = t.to(torch.bfloat16)
        return st

    def init_random(self, seed: int = 0):
        return self.load_state(self.random_state(seed))

    def load_safetensors(self, path: str):
        from safetensors import safe_open

        files = sorted(Path(path).glob("*.safetensors"))
        if not files:
            raise FileNotFoundError(f"no safetensors in {path}")
        st = {}
        for f in files:
            with safe_open(str(f), framework="pt") as sf:
                for k in sf.keys():
                    st[k] = sf.get_tensor(k)
        return self.load_state(st)

    def load_state(self, st: dict):
        """Build the fused device weights from checkpoint-named tensors."""
        c, dev, dt = self.cfg, self.device, self.dtype
        W = c.hidden_size
        shapes = self.tensor_shapes()

        def get(name):
            t = st[name]
            if tuple(t.shape) != tuple(shapes[name]):
                raise ValueError(f"{name}: shape {tuple(t.shape)}, configuration wants "
                                 f"{tuple(shapes[name])}")
            return t

        def act(name):
            return get(name).to(dt).to(dev).contiguous()

        def f32(name):
            return get(name).float().to(dev).contiguous()

        def fuse(lw, blocks, biases=None):
            """blocks (name, weight [n, W]); biases name -> [n] (absent: zero)."""
            rows, bias, off = [], [], 0
            for name, t in blocks:
                n, pad = t.shape[0], _pad8(t.shape[0])
                lw.seg[name] = (off, n)
                rows += [t, t.new_zeros(pad - n, W)]
                b = (biases or {}).get(name)
                bias += [t.new_zeros(n) if b is None else b, t.new_zeros(pad - n)]
                off += pad
            lw.w_in = torch.cat(rows).contiguous()
            lw.b_in = torch.cat(bias).contiguous() if biases else None

        self.embed = act("embed")
        self.final_norm = act("final.norm")
        self.layers = []
        for i, L in enumerate(c.layers):
            p, m = f"l{i}.", L.mixer
            x = p + "mix."
            lw = KolotarLayerWeights(norm1=act(p + "norm1"))
            if L.kind == "attention":
                fuse(lw, [(n, act(x + n)) for n in ("q", "k", "v", "g")],
                     {n: act(f"{x}{n}.b") for n in ("q", "k", "v")})
                lw.q_norm, lw.k_norm = act(x + "q.norm"), act(x + "k.norm")
                lw.sink = f32(x + "sink")
                lw.w_o, lw.b_o = act(x + "o"), act(x + "o.b")
                if m.rot_dims:
                    lw.inv_freq, lw.rot_mult = mx.yarn_inv_freq(m.rot_dims, m.rot_base,
                                                                m.rot_scaling, dev)
                if m.v_mix and i != c.first_v_mix:
                    lw.v_lambda = float(get(x + "vmix"))
            elif L.kind == "latent_attention":
                fuse(lw, [(n, act(x + n)) for n in ("q", "dkv", "g")])
                lw.c_norm = act(x + "dkv.norm")
                lw.uk = act(x + "uk").view(m.heads, m.dim, m.kv_rank)
                lw.uv_t = act(x + "uv").view(m.heads, m.vdim, m.kv_rank).transpose(1, 2).contiguous()
                lw.inv_freq = mx.inv_freq(m.rot_dims, m.rot_base, dev)
                lw.w_o = act(x + "o")
            elif L.kind == "parallel":
                l, r = x + "left.", x + "right."
                # q, k, v of the delta branch stay adjacent: one convolution launch covers them
                fuse(lw, [("q", act(l + "q")), ("k", act(l + "k")), ("v", act(l + "v")),
                          ("dqkv", torch.cat([act(r + n) for n in "qkv"])), ("beta", act(r + "b")),
                          ("a", act(r + "a")), ("gate", act(r + "g"))])
                lw.q_norm, lw.k_norm = act(l + "q.norm"), act(l + "k.norm")
                lw.head_bias, lw.talk = f32(l + "pb"), f32(l + "talk")
                lw.w_o = act(l + "o")
                lw.conv_w = torch.cat([act(f"{r}{n}.conv") for n in "qkv"]).contiguous()
                lw.a_log, lw.dt_bias = f32(r + "A_log"), f32(r + "dt_bias")
                lw.out_norm, lw.delta_o = act(r + "norm"), act(r + "o")
            else:
                raise ValueError(L.kind)
            if L.moe:
                f = p + "mlp."
                lw.norm2 = act(p + "norm2")
                lw.router, lw.router_b = f32(f + "router"), f32(f + "router.b")
                E = range(L.moe.experts)
                lw.e_gu = torch.stack([torch.cat([act(f"{f}e{e}.gate"), act(f"{f}e{e}.up")])
                                       for e in E])
                lw.e_down = torch.stack([act(f"{f}e{e}.down") for e in E])
            self.layers.append(lw)
        return self

    def prepare_decode_weights(self):
        return self

    def decode_copy_bytes(self) -> int:
        return 0

    def weight_bytes(self) -> int:
        ts = [self.embed, self.final_norm]
        for L in self.layers:
            ts += [v for v in vars(L).values() if isinstance(v, torch.Tensor)]
        return sum(t.numel() * t.element_size() for t in ts if t is not None)

    # ---------------------------------------------------------------------------------
    def cache_specs(self) -> list[LayerCacheSpec]:
        specs = []
        for L in self.cfg.layers:
            m = L.mixer
            if L.kind == "latent_attention":
                specs.append(LayerCacheSpec(kv_heads=1, kdim=m.kv_rank + m.rot_dim, vdim=m.kv_rank))
                continue
            kw = {}
            if L.kind == "parallel":
                d = L.delta
                kw = dict(state_heads=d.heads, state_dim=d.dim, state_vdim=d.vdim,
                          conv_channels=2 * d.kv_heads * d.dim + d.heads * d.vdim,
                          conv_taps=d.conv)
            specs.append(LayerCacheSpec(kv_heads=m.kv_heads, kdim=m.dim, vdim=m.vdim, **kw))
        return specs

    @property
    def attn_tile_tokens(self) -> int:
        return mx.ATTN_TILE_TOKENS

    # ---------------------------------------------------------------------------------
    @staticmethod
    def _cut(P, seg, name):
        o, n = seg[name]
        return P[:, o:o + n]

    @staticmethod
    def _table(md, lw, m, tables, scaling=None):
        """cos / sin of the step's positions, once per rotary setting."""
        key = (m.rot_dims, m.rot_base, scaling)
        if key not in tables:
            tables[key] = mx.rotary_table(md.positions, lw.inv_freq, lw.rot_mult)
        return tables[key]

    def _attention(self, h, lw, m, md, lc, tables, step):
        T = h.shape[0]
        P = F.linear(h, lw.w_in, lw.b_in)
        q, k, v, g = (self._cut(P, lw.seg, n) for n in ("q", "k", "v", "g"))
        table = (self._table(md, lw, m, tables, m.rot_scaling) if m.rot_dims else
                 torch.zeros(T, 0, dtype=torch.float32, device=h.device))
        first = v_out = None
        if m.v_mix:     # the first mixing layer keeps its values for the step's later ones
            first = step.get("v_first")
            if first is None:
                v_out = step["v_first"] = torch.empty(T, m.kv_heads * m.vdim, dtype=h.dtype,
                                                      device=h.device)
        q = mx.qk_norm_rope_cache(q, k, v, lw.q_norm, lw.k_norm, self.cfg.rms_norm_eps,
                                  md.positions, md.slot_mapping, table, lc.k, lc.v, m.heads,
                                  m.kv_heads, m.dim, m.vdim, rotate_half_pairs=True, v_norm=True,
                                  v_first=first, v_lambda=lw.v_lambda, v_out=v_out)
        a = mx.sink_attention(q, lc.k, lc.v, md.block_tables, md.seq_kvlen, md.seq_qstart,
                              md.tile_seq, md.tile_qoff, m.scale, True, md.num_decode,
                              md.max_decode_kv, sink_values=lw.sink, window=m.window, gate=g)
        return F.linear(a.view(T, m.heads * m.vdim), lw.w_o, lw.b_o)

    def _latent_attention(self, h, lw, m, md, lc, tables):
        T = h.shape[0]
        P = F.linear(h, lw.w_in)
        q = self._cut(P, lw.seg, "q").unflatten(1, (m.heads, m.dim + m.rot_dim))
        # absorbed queries: q_unrotated W_uk per head, then [ . | rotated part ]
        q_lat = torch.bmm(q[:, :, :m.dim].transpose(0, 1), lw.uk)
        qa = mx.latent_rope_cache(q_lat, q, self._cut(P, lw.seg, "dkv"), lw.c_norm,
                                  self.cfg.rms_norm_eps, md.slot_mapping,
                                  self._table(md, lw, m, tables), lc.k, lc.v,
                                  rotate_half_pairs=False)
        a = mx.sink_attention(qa, lc.k, lc.v, md.block_tables, md.seq_kvlen, md.seq_qstart,
                              md.tile_seq, md.tile_qoff, m.scale, False, md.num_decode,
                              md.max_decode_kv, window=m.window)
        o = torch.bmm(a.transpose(0, 1), lw.uv_t)           # [H, T, vdim]
        return F.linear(mx.head_gate(o.contiguous(), self._cut(P, lw.seg, "g")), lw.w_o)

    def _parallel(self, h, lw, m, d, md, lc):
        """The two branches' projected outputs (their weights are applied in the layer sum)."""
        T, eps = h.shape[0], self.cfg.rms_norm_eps
        P = F.linear(h, lw.w_in)
        q, k, v, qkv, beta, decay, gate = (self._cut(P, lw.seg, n) for n in
                                           ("q", "k", "v", "dqkv", "beta", "a", "gate"))
        table = torch.zeros(T, 0, dtype=torch.float32, device=h.device)   # no rotation
        q = mx.qk_norm_rope_cache(q, k, v, lw.q_norm, lw.k_norm, eps, md.positions,
                                  md.slot_mapping, table, lc.k, lc.v, m.heads, m.kv_heads, m.dim,
                                  m.vdim, whole_norm=True,
                                  q_temp=(m.temp_coef, m.temp_every) if m.temp_coef else None)
        a = mx.sigmoid_attention(q, lc.k, lc.v, md.block_tables, md.seq_kvlen, md.seq_qstart,
                                 md.tile_seq, md.tile_qoff, m.scale, m.softcap, lw.head_bias,
                                 lw.talk, md.num_decode, md.max_decode_kv)
        left = F.linear(a.view(T, m.heads * m.vdim), lw.w_o)
        qkv = mx.short_conv_silu(qkv, lw.conv_w, lc.conv, md.positions, md.seq_qstart, md.seq_slot)
        o = mx.gated_delta_rule(qkv, beta, decay, lw.a_log, lw.dt_bias, lc.state, md.positions,
                                md.seq_qstart, md.seq_slot, d.heads, d.kv_heads, d.dim, d.vdim)
        o = mx.gated_rms_norm(o, gate, lw.out_norm, eps, "silu", self.dtype)
        return left, F.linear(o, lw.delta_o)

    @staticmethod
    def _experts(x, h, lw, mo):
        idx, wts = mx.moe_route(F.linear(x, lw.router, lw.router_b), mo.top, "logit")
        return mx.moe_experts(h, idx, wts, lw.e_gu, lw.e_down, glu="silu")

    def forward(self, input_ids, md, cache: HybridCache, rows=None, layer_out=None):
        """One step over a decode-first batch of portions; returns the final-normed hidden rows
        (all, or ``rows``).  ``layer_out``: a list that receives a copy of the fp32 residual
        stream after every layer (debugging / tests)."""
        c = self.cfg
        eps, alpha = c.rms_norm_eps, c.alpha
        x = mx.embed_scale(self.embed, input_ids, 1.0)            # [T, W] fp32
        h = x.to(self.dtype)
        tables, step = {}, {}
        for li, (L, lw) in enumerate(zip(c.layers, self.layers)):
            lc, b, sa, sb = cache.layers[li], None, 1.0, 1.0
            if L.kind == "attention":
                a = self._attention(h, lw, L.mixer, md, lc, tables, step)
            elif L.kind == "latent_attention":
                a = self._latent_attention(h, lw, L.mixer, md, lc, tables)
            else:
                a, b = self._parallel(h, lw, L.mixer, L.delta, md, lc)
                sa, sb = L.left_scale, L.right_scale
            h = mx.post_norm(x, alpha, a, sa, b, sb, lw.norm1, eps, self.dtype)
            if L.moe:
                h = mx.post_norm(x, alpha, self._experts(x, h, lw, L.moe), 1.0, None, 1.0, lw.norm2,
                                 eps, self.dtype)
            if layer_out is not None:
                layer_out.append(x.clone())
        if rows is not None:
            x = x.index_select(0, rows)
        return mx.rms_norm_f32(x, self.final_norm, eps, False, self.dtype)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.embed).float()
