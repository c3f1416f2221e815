"""Tofodra decoder over the mixer op layer (``ops.mixers``).

Sandwich-norm layers on an fp32 residual stream with a per-channel scale on every branch:
``x += s1 * rms(mixer(rms(x)))`` then ``x += s2 * rms(ff(rms(x)))``.  Mixers:

* ``retention`` - linear attention with one fixed decay per head (no softmax, no denominator),
  rotate-half positions on q and k, fp32 state per sequence, each head's output divided by its
  root mean square, SiLU gate;
* ``attention`` - differential attention: two softmax maps over the same values, the second
  subtracted with one learned weight per layer; biased projections, no rotation, a sliding window
  that keeps the sequence's first tokens, element-wise sigmoid output gate;
* ``latent_attention`` - softmax attention over ONE cached latent per token plus a rotated key part
  shared by the heads (interleaved pairs); a layer may read an earlier layer's cache.

The feed-forward is a dense clamped GLU or routed SiLU-GLU experts (sigmoid scores, normalised and
scaled weights) with a shared expert.

MI355X layout: every projection that reads a mixer's input is one fused library GEMM (blocks
padded to 8 rows so the kernels read 16-byte aligned slices in place); the rows of the attention's
query projection are ordered (KV head, map, head of the group) at load time, so the attention
kernel reads its queries straight from the GEMM's output with the heads that share keys adjacent.
The post-norm of a branch, its scale, the residual sum and the next pre-norm are one kernel.
Latent attention runs absorbed (key up-projection on the queries, value up-projection on the
output), i.e. as multi-query attention over compressed pages.  The experts run as two grouped
matrix-core products over rows sorted by expert on the device, so a decode step stays capturable
as a hipGraph.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from pathlib import Path

import torch
import torch.nn.functional as F

from ..config import TofodraConfig
from ..engine.state_cache import HybridCache, LayerCacheSpec
from ..ops import mixers as mx


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


@dataclass
class TofodraLayerWeights:
    norm1: torch.Tensor
    norm1b: torch.Tensor
    ls1: torch.Tensor                          # per-channel scale of the mixer's branch
    w_in: torch.Tensor = None                  # fused projections of the mixer's input
    b_in: torch.Tensor | None = None           # fused bias of the same rows
    seg: dict = field(default_factory=dict)    # block name -> (column offset, width)
    w_o: torch.Tensor | None = None
    inv_freq: torch.Tensor | None = None
    powers: torch.Tensor | None = None         # retention: fp32 powers of every head's decay
    lam: float = 0.0                           # differential attention: weight of the second map
    # latent attention
    c_norm: torch.Tensor | None = None
    uk: torch.Tensor | None = None             # [H, dim, kv_rank]
    uv_t: torch.Tensor | None = None           # [H, kv_rank, vdim]
    # feed-forward
    norm2: torch.Tensor | None = None
    norm2b: torch.Tensor | None = None
    ls2: torch.Tensor | None = None
    gu: torch.Tensor | None = None             # dense or shared expert: fused gate | up
    gu_seg: dict = field(default_factory=dict)
    down: torch.Tensor | None = None
    router: torch.Tensor | None = None         # fp32 [E, W]
    e_gu: torch.Tensor | None = None           # [E, 2 ff, W]: gate rows, then up rows
    e_down: torch.Tensor | None = None         # [E, W, ff]


class TofodraModel:
    family = "tofodra"
    has_state = True

    def __init__(self, cfg: TofodraConfig, dtype=torch.bfloat16, device="cuda", tp_rank: int = 0,
                 tp_size: int = 1, tp_group=None, quantization: str = ""):
        if tp_size != 1:
            raise ValueError("Tofodra runs on one GPU per replica (tensor_parallel_size 1)")
        if quantization:
            raise ValueError("Tofodra weights are 16-bit or 32-bit; no quantization")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Tofodra activations are bfloat16 or float32")
        self.cfg = cfg
        self.dtype = dtype
        self.device = torch.device(device)
        self.tp_rank, self.tp_size, self.tp_group = 0, 1, None
        self.layers: list[TofodraLayerWeights] = []
        self.embed = self.final_norm = self.head = None
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
        out = {"embed": (c.vocab_size, W), "final.norm": (W,), "head": (c.vocab_size, W)}
        for i, L in enumerate(c.layers):
            p, m = f"l{i}.", L.mixer
            x, f = p + "mix.", p + "mlp."
            out.update({p + "norm1": (W,), p + "norm1b": (W,), p + "ls1": (W,)})
            if L.kind == "retention":
                nq, nv = m.heads * m.dim, m.heads * m.vdim
                out.update({x + "q": (nq, W), x + "k": (nq, W), x + "v": (nv, W), x + "g": (nv, W),
                            x + "o": (W, nv)})
            elif L.kind == "attention":
                nq, nk = m.heads * 2 * m.dim, m.kv_heads * 2 * m.dim
                nv, no = m.kv_heads * m.vdim, m.heads * m.vdim
                out.update({x + "q": (nq, W), x + "q.b": (nq,), x + "k": (nk, W), x + "k.b": (nk,),
                            x + "v": (nv, W), x + "v.b": (nv,), x + "g": (no, W), x + "o": (W, no)})
                out.update({x + n: (m.dim,) for n in ("lq1", "lk1", "lq2", "lk2")})
            else:
                out.update({x + "q": (m.heads * (m.dim + m.rot_dim), W),
                            x + "uk": (m.heads * m.dim, m.kv_rank),
                            x + "uv": (m.heads * m.vdim, m.kv_rank), x + "o": (W, m.heads * m.vdim)})
                if m.kv_from < 0:
                    out.update({x + "dkv": (m.kv_rank + m.rot_dim, W), x + "dkv.norm": (m.kv_rank,)})
            if L.ff or L.moe:
                out.update({p + "norm2": (W,), p + "norm2b": (W,), p + "ls2": (W,)})
            if L.ff:
                out.update({f + "gate": (L.ff, W), f + "up": (L.ff, W), f + "down": (W, L.ff)})
            if L.moe:
                out[f + "router"] = (L.moe.experts, W)
                for e in range(L.moe.experts):
                    out.update({f"{f}e{e}.gate": (L.moe.ff, W), f"{f}e{e}.up": (L.moe.ff, W),
                                f"{f}e{e}.down": (W, L.moe.ff)})
                if L.moe.shared_ff:
                    n = L.moe.shared_ff
                    out.update({f + "shared.gate": (n, W), f + "shared.up": (n, W),
                                f + "shared.down": (W, n)})
        return out

    def random_state(self, seed: int = 0) -> dict:
        """Seeded random tensors under the checkpoint's names (bf16-representable values)."""
        g = torch.Generator().manual_seed(86420 + seed)
        st = {}
        for name, shape in self.tensor_shapes().items():
            r = torch.randn(shape, generator=g)
            leaf = name.split(".")[-1]
            if name == "embed":
                t = r / self.cfg.embed_scale
            elif leaf.startswith("norm"):
                t = 1.0 + 0.1 * r
            elif leaf in ("ls1", "ls2"):
                t = 0.5 + 0.1 * r
            elif leaf == "b":
                t = 0.1 * r
            elif leaf in ("lq1", "lk1", "lq2", "lk2"):
                t = 0.1 * r
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

        def fuse(seg, blocks, biases=None):
            """blocks (name, weight [n, W]); biases name -> [n] (absent: zero)."""
            rows, bias, off = [], [], 0
            for name, t in blocks:
                n, pad = t.shape[0], _pad8(t.shape[0])
                seg[name] = (off, n)
                rows += [t, t.new_zeros(pad - n, W)]
                b = (biases or {}).get(name)
                bias += [t.new_zeros(n) if b is None else b, t.new_zeros(pad - n)]
                off += pad
            return torch.cat(rows).contiguous(), torch.cat(bias).contiguous() if biases else None

        def glu(lw, f):
            lw.gu, _ = fuse(lw.gu_seg, [("gate", act(f + "gate")), ("up", act(f + "up"))])
            lw.down = act(f + "down")

        self.embed, self.head = act("embed"), act("head")
        self.final_norm = act("final.norm")
        self.layers = []
        for i, L in enumerate(c.layers):
            p, m = f"l{i}.", L.mixer
            x, f = p + "mix.", p + "mlp."
            lw = TofodraLayerWeights(act(p + "norm1"), act(p + "norm1b"), act(p + "ls1"))
            lw.w_o = act(x + "o")
            if L.kind == "retention":
                lw.w_in, _ = fuse(lw.seg, [(n, act(x + n)) for n in "qkvg"])
                lw.powers = mx.retention_powers(m.decay, dev)
                lw.inv_freq = mx.inv_freq(m.rot_dims, m.rot_base, dev)
            elif L.kind == "attention":
                def grouped(t):
                    """rows (head, map, channel) -> (KV head, map, head of the group, channel)"""
                    t = t.view(m.kv_heads, m.heads // m.kv_heads, 2, m.dim, -1)
                    return t.transpose(1, 2).reshape(m.heads * 2 * m.dim, -1)

                lw.w_in, lw.b_in = fuse(
                    lw.seg, [("q", grouped(act(x + "q")))] + [(n, act(x + n)) for n in "kvg"],
                    {"q": grouped(act(x + "q.b")).flatten(), "k": act(x + "k.b"),
                     "v": act(x + "v.b")})
                a, b = (float(torch.exp((get(x + "lq" + n).double() * get(x + "lk" + n).double())
                                        .sum())) for n in "12")
                lw.lam = a - b + m.diff
            elif L.kind == "latent_attention":
                own = m.kv_from < 0
                lw.w_in, _ = fuse(lw.seg, [(n, act(x + n)) for n in (("q", "dkv") if own else ("q",))])
                lw.c_norm = act(x + "dkv.norm") if own else None
                lw.uk = act(x + "uk").view(m.heads, m.dim, m.kv_rank)
                lw.uv_t = act(x + "uv").view(m.heads, m.vdim, m.kv_rank).transpose(1, 2).contiguous()
                lw.inv_freq = mx.inv_freq(m.rot_dims, m.rot_base, dev)
            else:
                raise ValueError(L.kind)
            if L.ff or L.moe:
                lw.norm2, lw.norm2b, lw.ls2 = act(p + "norm2"), act(p + "norm2b"), act(p + "ls2")
            if L.ff:
                glu(lw, f)
            if L.moe:
                lw.router = get(f + "router").float().to(dev).contiguous()
                E = range(L.moe.experts)
                lw.e_gu = torch.stack([torch.cat([act(f"{f}e{e}.gate"), act(f"{f}e{e}.up")])
                                       for e in E])
                lw.e_down = torch.stack([act(f"{f}e{e}.down") for e in E])
                if L.moe.shared_ff:
                    glu(lw, f + "shared.")
            self.layers.append(lw)
        return self

    def prepare_decode_weights(self):
        return self

    def decode_copy_bytes(self) -> int:
        return 0

    def weight_bytes(self) -> int:
        ts = [self.embed, self.final_norm, self.head]
        for L in self.layers:
            ts += [v for v in vars(L).values() if isinstance(v, torch.Tensor)]
        return sum(t.numel() * t.element_size() for t in ts if t is not None)

    # ---------------------------------------------------------------------------------
    def cache_specs(self) -> list[LayerCacheSpec]:
        specs = []
        for L in self.cfg.layers:
            m = L.mixer
            if L.kind == "retention":
                specs.append(LayerCacheSpec(state_heads=m.heads, state_dim=m.dim,
                                            state_vdim=m.vdim))
            elif L.kind == "attention":   # a K head per map, the values shared by both
                specs.append(LayerCacheSpec(kv_heads=2 * m.kv_heads, kdim=m.dim, vdim=m.vdim,
                                            v_heads=m.kv_heads))
            else:
                specs.append(LayerCacheSpec(kv_heads=1, kdim=m.kv_rank + m.rot_dim, vdim=m.kv_rank,
                                            kv_from=m.kv_from))
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
    def _table(md, lw, m, tables):
        """cos / sin of the step's positions, once per rotary setting."""
        key = (m.rot_dims, m.rot_base)
        if key not in tables:
            tables[key] = (mx.rotary_table(md.positions, lw.inv_freq) if m.rot_dims else
                           torch.zeros(md.positions.shape[0], 0, dtype=torch.float32,
                                       device=md.positions.device))
        return tables[key]

    def _retention(self, h, lw, m, md, lc, tables):
        P = F.linear(h, lw.w_in)
        q, k, v, g = (self._cut(P, lw.seg, n) for n in "qkvg")
        o = mx.retention(q, k, v, lw.powers, self._table(md, lw, m, tables), lc.state, md.positions,
                         md.seq_qstart, md.seq_slot, m.heads, m.dim, m.vdim, md.num_decode)
        o = mx.gated_rms_norm(o, g, None, self.cfg.rms_norm_eps, "silu", self.dtype)
        return F.linear(o, lw.w_o)

    def _attention(self, h, lw, m, md, lc):
        P = F.linear(h, lw.w_in, lw.b_in)
        q, k, v, g = (self._cut(P, lw.seg, n) for n in "qkvg")
        mx.kv_cache_write(k, v, md.slot_mapping, lc.k, lc.v)
        o = mx.differential_attention(q.unflatten(1, (2 * m.heads, m.dim)), lc.k, lc.v,
                                      md.block_tables, md.seq_kvlen, md.seq_qstart, md.tile_seq,
                                      md.tile_qoff, m.scale, lw.lam, m.diff, self.cfg.rms_norm_eps,
                                      g, md.num_decode, md.max_decode_kv, m.window, m.keep_first)
        return F.linear(o, lw.w_o)

    def _latent_attention(self, h, lw, m, md, lc, tables):
        P = F.linear(h, lw.w_in)
        q = self._cut(P, lw.seg, "q").unflatten(1, (m.heads, m.dim + m.rot_dim))
        # absorbed queries: q_unrotated W_uk per head, then [ . | rotated part ]
        q_lat = torch.bmm(q[:, :, :m.dim].transpose(0, 1), lw.uk)
        qa = mx.latent_rope_cache(q_lat, q, self._cut(P, lw.seg, "dkv") if m.kv_from < 0 else None,
                                  lw.c_norm, self.cfg.rms_norm_eps, md.slot_mapping,
                                  self._table(md, lw, m, tables), lc.k, lc.v,
                                  rotate_half_pairs=False)
        a = mx.sink_attention(qa, lc.k, lc.v, md.block_tables, md.seq_kvlen, md.seq_qstart,
                              md.tile_seq, md.tile_qoff, m.scale, False, md.num_decode,
                              md.max_decode_kv)
        o = torch.bmm(a.transpose(0, 1), lw.uv_t)           # [H, T, vdim]
        return F.linear(mx.head_gate(o.contiguous(), None), lw.w_o)

    @staticmethod
    def _gate_up(h, lw):
        P = F.linear(h, lw.gu)
        (og, n), (ou, _) = lw.gu_seg["gate"], lw.gu_seg["up"]
        return P[:, og:og + n], P[:, ou:ou + n]

    def _experts(self, h, lw, mo):
        logits = F.linear(h.float(), lw.router)       # fp32 router on the (rounded) input
        idx, wts = mx.moe_route(logits, mo.top, "sigmoid", renorm=True, scale=mo.scale)
        shared = None
        if mo.shared_ff:
            gate, up = self._gate_up(h, lw)
            shared = F.linear(mx.gate_mul(up, gate, "silu"), lw.down)
        return mx.moe_experts(h, idx, wts, lw.e_gu, lw.e_down, glu="silu", addend=shared)

    def forward(self, input_ids, md, cache: HybridCache, rows=None, layer_out=None):
        """One step over a decode-first batch of portions; returns the final-normed hidden rows
        (all, or ``rows``).  ``layer_out``: a list that receives a copy of the fp32 residual
        stream after every layer (debugging / tests)."""
        c = self.cfg
        eps, dt = c.rms_norm_eps, self.dtype
        x = mx.embed_scale(self.embed, input_ids, c.embed_scale)            # [T, W] fp32
        h = (mx.norm_add_norm(x, None, None, self.layers[0].norm1, eps, "rms", dt)
             if self.layers else None)
        tables = {}
        for li, (L, lw) in enumerate(zip(c.layers, self.layers)):
            lc = cache.layers[li]
            if L.kind == "retention":
                y = self._retention(h, lw, L.mixer, md, lc, tables)
            elif L.kind == "attention":
                y = self._attention(h, lw, L.mixer, md, lc)
            else:
                y = self._latent_attention(h, lw, L.mixer, md, lc, tables)
            post, scale = lw.norm1b, lw.ls1
            if L.ff or L.moe:   # post-norm, scale, residual sum and the feed-forward's norm at once
                h = mx.norm_add_norm(x, y, post, lw.norm2, eps, "rms", dt, post_scale=scale)
                if L.ff:
                    gate, up = self._gate_up(h, lw)
                    y = F.linear(mx.clamped_gate_mul(up, gate, L.limit), lw.down)
                else:
                    y = self._experts(h, lw, L.moe)
                post, scale = lw.norm2b, lw.ls2
            nxt = self.layers[li + 1].norm1 if li + 1 < len(self.layers) else None
            h = mx.norm_add_norm(x, y, post, nxt, eps, "rms", dt, post_scale=scale)
            if layer_out is not None:
                layer_out.append(x.clone())
        if rows is not None:
            x = x.index_select(0, rows)
        return mx.norm_add_norm(x, None, None, self.final_norm, eps, "rms", dt)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.head).float()
