"""HIP mixer kernels against the plain fp32 PyTorch reference of the same op
(ops/mixers_reference.py), on ragged batches with reused state slots and paged caches."""
import numpy as np
import pytest
import torch

from agentic_traffic_testing_amd.ops import mixers as mx
from agentic_traffic_testing_amd.ops import mixers_reference as mref

pytestmark = pytest.mark.gpu

DTYPES = [torch.bfloat16, torch.float32]


def tol(dt):
    return dict(atol=3e-2, rtol=3e-2) if dt == torch.bfloat16 else dict(atol=2e-5, rtol=2e-5)


def ragged(lens, starts, slots, tile=64, bs=16, width=12, seed=0):
    """Metadata of a batch of portions: lens / starts (tokens already cached) / state slots."""
    rng = np.random.default_rng(seed)
    pos, qstart, kvlen, tseq, toff = [], [0], [], [], []
    nblk = [-(-(s + n) // bs) for s, n in zip(starts, lens)]
    pages = rng.permutation(sum(nblk) + 3)
    bt = np.zeros((len(lens), width), dtype=np.int32)
    slot_map, p0 = [], 0
    for i, (n, s) in enumerate(zip(lens, starts)):
        bt[i, :nblk[i]] = pages[p0:p0 + nblk[i]]
        p0 += nblk[i]
        for j in range(n):
            p = s + j
            pos.append(p)
            slot_map.append(bt[i, p // bs] * bs + p % bs)
        qstart.append(qstart[-1] + n)
        kvlen.append(s + n)
        for o in range(0, n, tile):
            tseq.append(i)
            toff.append(o)
    i32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32)  # noqa: E731
    return dict(positions=i32(pos), seq_qstart=i32(qstart), seq_slot=i32(slots),
                seq_kvlen=i32(kvlen), slot_mapping=i32(slot_map), block_tables=i32(bt),
                tile_seq=i32(tseq), tile_qoff=i32(toff), num_pages=len(pages))


def cuda(d):
    return {k: (v.cuda() if torch.is_tensor(v) else v) for k, v in d.items()}


LENS, STARTS, SLOTS = [1, 1, 37, 2, 16], [0, 70, 0, 31, 5], [3, -1, 0, 2, 1]


@pytest.mark.parametrize("dt", DTYPES)
def test_embed_norm_elementwise(dt):
    torch.manual_seed(0)
    md = ragged(LENS, STARTS, SLOTS)
    T, W, V, B = int(md["seq_qstart"][-1]), 96, 50, 13
    table, pair = torch.randn(V, W).to(dt), torch.randn(B + 1, W).to(dt)
    ids = torch.randint(0, V, (T,), dtype=torch.int32)
    prev = torch.randint(0, V, (5,), dtype=torch.int32)
    prev_g = prev.cuda()
    mdg = cuda(md)
    want = mref.embed_pair(table, pair, ids, md["positions"], md["seq_qstart"], md["seq_slot"],
                           prev, 29, 5, B)
    got = mx.embed_pair(table.cuda(), pair.cuda(), ids.cuda(), mdg["positions"],
                        mdg["seq_qstart"], mdg["seq_slot"], prev_g, 29, 5, B)
    assert torch.equal(got.cpu(), want)
    assert torch.equal(prev_g.cpu(), prev)
    x = torch.randn(T, W) * 3
    w = (0.1 * torch.randn(W)).to(dt)
    for one_plus in (True, False):
        a = mx.rms_norm_f32(x.cuda(), w.cuda(), 1e-5, one_plus, dt).cpu().float()
        b = mref.rms_norm_f32(x, w, 1e-5, one_plus, dt).float()
        assert torch.allclose(a, b, **tol(dt))
    big = torch.randn(T, 3 * W).to(dt)
    assert torch.allclose(mx.relu_sq(big.cuda()[:, 8:8 + W]).cpu().float(),
                          mref.relu_sq(big[:, 8:8 + W]).float(), **tol(dt))
    a_, b_, c_ = (torch.randn(T, W).to(dt) for _ in range(3))
    for bb, cc in ((b_, c_), (None, c_), (b_, None), (None, None)):
        xr = mref.residual_add(x.clone(), a_, 0.8, bb, 0.5, cc)
        xg = mx.residual_add(x.clone().cuda(), a_.cuda(), 0.8, None if bb is None else bb.cuda(),
                             0.5, None if cc is None else cc.cuda())
        assert torch.allclose(xg.cpu(), xr, atol=1e-5, rtol=1e-5)
    o = torch.randn(T, 3, 40)
    gate = torch.randn(T, 200).to(dt)
    wn = (1 + 0.1 * torch.randn(40)).to(dt)
    for act in ("silu", "sigmoid"):
        a = mx.gated_rms_norm(o.cuda(), gate.cuda()[:, 16:136], wn.cuda(), 1e-5, act, dt)
        b = mref.gated_rms_norm(o, gate[:, 16:136], wn, 1e-5, act, dt)
        assert torch.allclose(a.cpu().float(), b.float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("W", [64, 1024, 4096, 100, 12288])
def test_norm_kernels_vector_and_scalar_widths(dt, W):
    torch.manual_seed(W)
    T = 5
    x = torch.randn(T, W) * 2
    w = (0.1 * torch.randn(W)).to(dt)
    a, b, c = (torch.randn(T, W).to(dt) for _ in range(3))
    got = mx.rms_norm_f32(x.cuda(), w.cuda(), 1e-5, True, dt).cpu().float()
    assert torch.allclose(got, mref.rms_norm_f32(x, w, 1e-5, True, dt).float(), **tol(dt))
    for bb, cc in ((b, c), (None, c), (b, None)):
        xr, xg = x.clone(), x.clone().cuda()
        hr = mref.rms_norm_f32(mref.residual_add(xr, a, 0.7, bb, 1.2, cc), w, 1e-5, True, dt)
        hg = mx.add_norm(xg, a.cuda(), 0.7, None if bb is None else bb.cuda(), 1.2,
                         None if cc is None else cc.cuda(), w.cuda(), 1e-5, True, dt)
        assert torch.allclose(xg.cpu(), xr, atol=1e-5, rtol=1e-5)
        assert torch.allclose(hg.cpu().float(), hr.float(), **tol(dt))
    big = torch.randn(T, W + 32).to(dt)
    assert torch.allclose(mx.relu_sq(big.cuda()[:, 16:16 + W]).cpu().float(),
                          mref.relu_sq(big[:, 16:16 + W]).float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,rot", [(6, 2, 64, 96, 32), (4, 1, 48, 80, 32),
                                              (8, 8, 128, 128, 128), (2, 2, 32, 16, 16)])
def test_rope_cache_and_attention(dt, H, G, dim, vdim, rot):
    torch.manual_seed(1)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T, nb, bs = int(md["seq_qstart"][-1]), md["num_pages"], 16
    P = torch.randn(T, (H + G) * dim + G * vdim + 24).to(dt)
    qx, kx = P[:, 8:8 + H * dim], P[:, 8 + H * dim:8 + (H + G) * dim]
    vx = P[:, 16 + (H + G) * dim:16 + (H + G) * dim + G * vdim]
    qn, kn = (1 + 0.1 * torch.randn(dim)).to(dt), (1 + 0.1 * torch.randn(dim)).to(dt)
    inv = mx.inv_freq(rot, 10000.0, "cpu")
    kc, vc = torch.randn(nb, G, bs, dim).to(dt), torch.randn(nb, G, vdim, bs).to(dt)
    kcg, vcg = kc.cuda(), vc.cuda()
    Pg = P.cuda()
    tab = mref.rotary_table(md["positions"], inv)
    tab_g = mx.rotary_table(mdg["positions"], inv.cuda())
    assert torch.allclose(tab_g.cpu(), tab, atol=2e-6)
    qr = mref.qk_norm_rope_cache(qx, kx, vx, qn, kn, 1e-5, md["positions"], md["slot_mapping"],
                                 tab, kc, vc, H, G, dim, vdim)
    qg = mx.qk_norm_rope_cache(Pg[:, 8:8 + H * dim], Pg[:, 8 + H * dim:8 + (H + G) * dim],
                               Pg[:, 16 + (H + G) * dim:16 + (H + G) * dim + G * vdim], qn.cuda(),
                               kn.cuda(), 1e-5, mdg["positions"], mdg["slot_mapping"], tab_g,
                               kcg, vcg, H, G, dim, vdim)
    assert torch.allclose(qg.cpu().float(), qr.float(), **tol(dt))
    assert torch.allclose(kcg.cpu().float(), kc.float(), **tol(dt))
    assert torch.equal(vcg.cpu(), vc)
    for sink in (True, False):
        want = mref.sink_attention(qr, kc, vc, md["block_tables"], md["seq_kvlen"],
                                   md["seq_qstart"], 0.2, sink)
        got = mx.sink_attention(qr.cuda(), kc.cuda(), vc.cuda(), mdg["block_tables"],
                                mdg["seq_kvlen"], mdg["seq_qstart"], mdg["tile_seq"],
                                mdg["tile_qoff"], 0.2, sink)
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))
        # the rows kernel on every shape (the matrix-core kernel takes bf16 with fitting widths)
        mx.ATTENTION_MFMA = False
        try:
            got = mx.sink_attention(qr.cuda(), kc.cuda(), vc.cuda(), mdg["block_tables"],
                                    mdg["seq_kvlen"], mdg["seq_qstart"], mdg["tile_seq"],
                                    mdg["tile_qoff"], 0.2, sink)
        finally:
            mx.ATTENTION_MFMA = True
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim", [(6, 2, 64, 96), (4, 1, 48, 80), (8, 2, 128, 128)])
def test_attention_long_prefill_and_partitioned_decode(dt, H, G, dim, vdim):
    """Decode sequences first (one row each, contexts across several key partitions), then
    prefill portions that start inside a context and span several tiles and pages."""
    torch.manual_seed(4)
    lens, starts = [1, 1, 1, 150, 70], [0, 255, 700, 333, 0]
    md = ragged(lens, starts, [0, 1, 2, 3, 4], width=64)
    # only the prefill portions are tiled
    keep = md["tile_seq"] >= 3
    md["tile_seq"], md["tile_qoff"] = md["tile_seq"][keep], md["tile_qoff"][keep]
    mdg = cuda(md)
    T, nb = int(md["seq_qstart"][-1]), md["num_pages"]
    q = torch.randn(T, H, dim).to(dt)
    kc, vc = torch.randn(nb, G, 16, dim).to(dt), torch.randn(nb, G, vdim, 16).to(dt)
    for sink in (True, False):
        want = mref.sink_attention(q, kc, vc, md["block_tables"], md["seq_kvlen"],
                                   md["seq_qstart"], 0.15, sink)
        got = mx.sink_attention(q.cuda(), kc.cuda(), vc.cuda(), mdg["block_tables"],
                                mdg["seq_kvlen"], mdg["seq_qstart"], mdg["tile_seq"],
                                mdg["tile_qoff"], 0.15, sink, num_decode=3, max_decode_kv=701)
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 4])
def test_short_conv(dt, taps):
    torch.manual_seed(2)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T, C = int(md["seq_qstart"][-1]), 300
    C = 304 if taps == 4 else C            # a multiple of 8 takes the 8-channel kernel
    P = torch.randn(T, C + 16).to(dt)
    w = (0.5 * torch.randn(C, taps)).to(dt)
    st = torch.randn(5, taps - 1, C).to(dt)
    stg = st.cuda()
    want = mref.short_conv_silu(P[:, 8:8 + C], w, st, md["positions"], md["seq_qstart"],
                                md["seq_slot"])
    got = mx.short_conv_silu(P.cuda()[:, 8:8 + C], w.cuda(), stg, mdg["positions"],
                             mdg["seq_qstart"], mdg["seq_slot"])
    live = [r for s in range(len(LENS)) if SLOTS[s] >= 0
            for r in range(int(md["seq_qstart"][s]), int(md["seq_qstart"][s + 1]))]
    assert torch.allclose(got.cpu().float()[live], want.float()[live], **tol(dt))
    assert torch.equal(stg.cpu(), st)


@pytest.mark.parametrize("dt", DTYPES)
def test_short_conv_prefill_sized_step(dt):
    """More than 1024 rows: the kernel walks eight rows per workgroup, across portion borders."""
    torch.manual_seed(7)
    lens, starts, slots = [700, 1, 401, 30], [0, 9, 50, 0], [2, 0, 3, 1]
    md = ragged(lens, starts, slots, width=64)
    mdg = cuda(md)
    T, C, taps = int(md["seq_qstart"][-1]), 72, 4
    P = torch.randn(T, C + 16).to(dt)
    w = (0.5 * torch.randn(C, taps)).to(dt)
    st = torch.randn(4, taps - 1, C).to(dt)
    stg = st.cuda()
    want = mref.short_conv_silu(P[:, 8:8 + C], w, st, md["positions"], md["seq_qstart"],
                                md["seq_slot"])
    got = mx.short_conv_silu(P.cuda()[:, 8:8 + C], w.cuda(), stg, mdg["positions"],
                             mdg["seq_qstart"], mdg["seq_slot"])
    assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))
    assert torch.equal(stg.cpu(), st)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,per_channel", [(6, 2, 32, 96, False), (2, 1, 64, 48, True),
                                                      (4, 2, 128, 128, True), (3, 1, 48, 72, False),
                                                      (2, 1, 80, 16, True)])
def test_gated_delta_rule(dt, H, G, dim, vdim, per_channel):
    torch.manual_seed(3)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T = int(md["seq_qstart"][-1])
    qkv = torch.randn(T, 2 * G * dim + H * vdim).to(dt)
    side = torch.randn(T, 8 + H + 8 + (H * dim if per_channel else H)).to(dt)
    beta, decay = side[:, 8:8 + H], side[:, 16 + H:]
    a_log = torch.log(0.25 + 2 * torch.rand(H))
    dt_bias = torch.randn(decay.shape[1]) - 1
    st = torch.randn(5, H, dim, vdim)
    stg = st.cuda()
    want = mref.gated_delta_rule(qkv, beta, decay, a_log, dt_bias, st, md["positions"],
                                 md["seq_qstart"], md["seq_slot"], H, G, dim, vdim)
    sg = side.cuda()
    got = mx.gated_delta_rule(qkv.cuda(), sg[:, 8:8 + H], sg[:, 16 + H:], a_log.cuda(),
                              dt_bias.cuda(), stg, mdg["positions"], mdg["seq_qstart"],
                              mdg["seq_slot"], H, G, dim, vdim)
    live = [r for s in range(len(LENS)) if SLOTS[s] >= 0
            for r in range(int(md["seq_qstart"][s]), int(md["seq_qstart"][s + 1]))]
    assert torch.allclose(got.cpu()[live], want[live], atol=2e-4, rtol=2e-4)
    assert torch.allclose(stg.cpu(), st, atol=2e-4, rtol=2e-4)


def live_rows(md, lens, slots):
    return [r for s in range(len(lens)) if slots[s] >= 0
            for r in range(int(md["seq_qstart"][s]), int(md["seq_qstart"][s + 1]))]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,qdim,rot,rank,dims", [(4, 48, 32, 96, 32), (8, 128, 64, 192, 64),
                                                  (3, 8, 12, 24, 8), (20, 16, 8, 40, 4)])
def test_latent_front_end_and_absorbed_attention(dt, H, qdim, rot, rank, dims):
    """Latent norm + rotate-half + compressed page writes, then multi-query attention with a
    learned sink per head over those pages: prefill tiles, partitioned decode, matrix-core
    and rows kernels, more than 16 query heads on the one key head."""
    torch.manual_seed(8)
    lens, starts = [1, 1, 1, 150, 70], [0, 255, 700, 333, 0]
    md = ragged(lens, starts, [0, 1, 2, 3, 4], width=64)
    keep = md["tile_seq"] >= 3
    md["tile_seq"], md["tile_qoff"] = md["tile_seq"][keep], md["tile_qoff"][keep]
    mdg = cuda(md)
    T, nb, bs = int(md["seq_qstart"][-1]), md["num_pages"], 16
    q_lat, qx = torch.randn(H, T, rank).to(dt), torch.randn(T, H, qdim + rot).to(dt)
    P = torch.randn(T, rank + rot + 16).to(dt)
    w = (1 + 0.1 * torch.randn(rank)).to(dt)
    sink = torch.randn(H)
    kc, vc = torch.randn(nb, 1, bs, rank + rot).to(dt), torch.randn(nb, 1, rank, bs).to(dt)
    kcg, vcg = kc.cuda(), vc.cuda()
    inv = mx.inv_freq(dims, 30000.0, "cpu")
    tab = mref.rotary_table(md["positions"], inv)
    qr = mref.latent_rope_cache(q_lat, qx, P[:, 8:8 + rank + rot], w, 1e-6, md["slot_mapping"],
                                tab, kc, vc)
    qg = mx.latent_rope_cache(q_lat.cuda(), qx.cuda(), P.cuda()[:, 8:8 + rank + rot], w.cuda(),
                              1e-6, mdg["slot_mapping"], tab.cuda(), kcg, vcg)
    assert torch.allclose(qg.cpu().float(), qr.float(), **tol(dt))
    assert torch.allclose(kcg.cpu().float(), kc.float(), **tol(dt))
    assert torch.allclose(vcg.cpu().float(), vc.float(), **tol(dt))
    want = mref.sink_attention(qr, kc, vc, md["block_tables"], md["seq_kvlen"], md["seq_qstart"],
                               0.1, True, sink)
    for mfma in (True, False):
        mx.ATTENTION_MFMA = mfma
        try:
            got = mx.sink_attention(qr.cuda(), kc.cuda(), vc.cuda(), mdg["block_tables"],
                                    mdg["seq_kvlen"], mdg["seq_qstart"], mdg["tile_seq"],
                                    mdg["tile_qoff"], 0.1, True, num_decode=3, max_decode_kv=701,
                                    sink_values=sink.cuda())
        finally:
            mx.ATTENTION_MFMA = True
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt)), mfma


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,dk,dv", [(4, 56, 64), (2, 128, 128), (3, 10, 20), (1, 200, 33)])
def test_forget_gate_scan(dt, H, dk, dv):
    torch.manual_seed(9)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T = int(md["seq_qstart"][-1])
    P = torch.randn(T, 2 * H * dk + H * dv + 24).to(dt)
    q, f = P[:, 8:8 + H * dk], P[:, 8 + H * dk:8 + 2 * H * dk]
    v = P[:, 16 + 2 * H * dk:16 + 2 * H * dk + H * dv]
    fb, lower = torch.randn(H * dk), torch.rand(H * dk)
    st = torch.randn(5, H, dk, dv)
    stg, Pg = st.cuda(), P.cuda()
    want = mref.forget_gate_scan(q, f, v, fb, lower, st, md["positions"], md["seq_qstart"],
                                 md["seq_slot"], H, dk, dv)
    got = mx.forget_gate_scan(Pg[:, 8:8 + H * dk], Pg[:, 8 + H * dk:8 + 2 * H * dk],
                              Pg[:, 16 + 2 * H * dk:16 + 2 * H * dk + H * dv], fb.cuda(),
                              lower.cuda(), stg, mdg["positions"], mdg["seq_qstart"],
                              mdg["seq_slot"], H, dk, dv)
    live = live_rows(md, LENS, SLOTS)
    assert torch.allclose(got.cpu()[live], want[live], atol=2e-4, rtol=2e-4)
    assert torch.allclose(stg.cpu(), st, atol=2e-4, rtol=2e-4)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,N,dv", [(6, 3, 40, 32), (8, 1, 128, 64), (5, 5, 7, 12), (4, 2, 16, 100)])
def test_state_space_scan(dt, H, G, N, dv):
    torch.manual_seed(10)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T = int(md["seq_qstart"][-1])
    xbc = torch.randn(T, H * dv + 2 * G * N).to(dt)
    dtr = torch.randn(T, H + 8).to(dt)
    bias, a_log, skip = torch.randn(H) - 1, torch.log(0.25 + 2 * torch.rand(H)), torch.randn(H)
    st = torch.randn(5, H, N, dv)
    stg, xg, dg = st.cuda(), xbc.cuda(), dtr.cuda()
    i, gn = H * dv, G * N
    want = mref.state_space_scan(xbc[:, :i], xbc[:, i:i + gn], xbc[:, i + gn:], dtr[:, 8:], bias,
                                 a_log, skip, st, md["positions"], md["seq_qstart"],
                                 md["seq_slot"], H, G, N, dv)
    got = mx.state_space_scan(xg[:, :i], xg[:, i:i + gn], xg[:, i + gn:], dg[:, 8:], bias.cuda(),
                              a_log.cuda(), skip.cuda(), stg, mdg["positions"], mdg["seq_qstart"],
                              mdg["seq_slot"], H, G, N, dv)
    live = live_rows(md, LENS, SLOTS)
    assert torch.allclose(got.cpu()[live], want[live], atol=3e-4, rtol=3e-4)
    assert torch.allclose(stg.cpu(), st, atol=3e-4, rtol=3e-4)


@pytest.mark.parametrize("dt", DTYPES)
def test_biased_conv_gated_group_norm_xielu_head_gate(dt):
    torch.manual_seed(11)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T, C, taps = int(md["seq_qstart"][-1]), 304, 4
    P = torch.randn(T, C + 16).to(dt)
    w, b = (0.5 * torch.randn(C, taps)).to(dt), torch.randn(C).to(dt)
    st = torch.randn(5, taps - 1, C).to(dt)
    stg = st.cuda()
    want = mref.short_conv_silu(P[:, 8:8 + C], w, st, md["positions"], md["seq_qstart"],
                                md["seq_slot"], b)
    got = mx.short_conv_silu(P.cuda()[:, 8:8 + C], w.cuda(), stg, mdg["positions"],
                             mdg["seq_qstart"], mdg["seq_slot"], bias=b.cuda())
    live = live_rows(md, LENS, SLOTS)
    assert torch.allclose(got.cpu().float()[live], want.float()[live], **tol(dt))
    assert torch.equal(stg.cpu(), st)
    y, gate = torch.randn(T, 192), torch.randn(T, 200).to(dt)
    for parts, wn in ((2, torch.randn(192)), (1, torch.randn(192)), (6, torch.randn(32))):
        for g in (gate[:, 8:], None):
            a = mx.group_rms_norm(y.cuda(), None if g is None else g.cuda(), wn.to(dt).cuda(),
                                  parts, 1e-6, dt).cpu().float()
            r = mref.group_rms_norm(y, g, wn.to(dt), parts, 1e-6, dt).float()
            assert torch.allclose(a, r, **tol(dt))
    for N in (384, 100):
        z, zb = (2 * torch.randn(T, N + 8)).to(dt), torch.randn(N).to(dt)
        a = mx.xielu_bias(z.cuda()[:, 8:], zb.cuda(), 0.8, 0.3).cpu().float()
        assert torch.allclose(a, mref.xielu_bias(z[:, 8:], zb, 0.8, 0.3).float(), **tol(dt))
    o, hg = torch.randn(4, T, 32).to(dt), torch.randn(T, 12).to(dt)
    a = mx.head_gate(o.cuda(), hg.cuda()[:, 8:]).cpu().float()
    assert torch.allclose(a, mref.head_gate(o, hg[:, 8:]).float(), **tol(dt))
    table = torch.randn(50, 96).to(dt)
    ids = torch.randint(0, 50, (T,), dtype=torch.int32)
    assert torch.allclose(mx.embed_scale(table.cuda(), ids.cuda(), 0.5).cpu(),
                          mref.embed_scale(table, ids, 0.5))
    x = torch.randn(T, 136).to(dt)
    wr = (1 + 0.1 * torch.randn(128)).to(dt)
    assert torch.allclose(mx.rms_norm_rows(x.cuda()[:, 8:], wr.cuda(), 1e-6).cpu().float(),
                          mref.rms_norm_rows(x[:, 8:], wr, 1e-6).float(), **tol(dt))


# ---- multi-stream residual, token shift, window attention, minGRU, routed experts ------------

@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("ns,W", [(2, 96), (3, 1024), (1, 100), (4, 4096), (2, 20000)])
def test_hyper_update_norm(dt, ns, W):
    torch.manual_seed(11)
    T = 9
    xs = torch.randn(T, ns, W) * 2
    y = torch.randn(T, W).to(dt)
    mix, w_out, w_in = torch.randn(ns, ns), torch.randn(ns), torch.randn(ns)
    w = (1 + 0.1 * torch.randn(W)).to(dt)
    for out_dt in (dt, torch.float32):
        xr, xg = xs.clone(), xs.clone().cuda()
        want = mref.hyper_norm(mref.hyper_update(xr, y, mix, w_out), w_in, w, 1e-6, out_dt)
        got = mx.hyper_update_norm(xg, y.cuda(), mix.cuda(), w_out.cuda(), w_in.cuda(), w.cuda(),
                                   1e-6, out_dt)
        assert got.dtype == out_dt
        assert torch.allclose(xg.cpu(), xr, atol=1e-4, rtol=1e-5)
        assert torch.allclose(got.cpu().float(), want.float(), **tol(out_dt if out_dt == dt else
                                                                     torch.float32))
        # norm only / update only
        a = mx.hyper_norm(xg, w_in.cuda(), w.cuda(), 1e-6, out_dt)
        assert torch.allclose(a.cpu().float(), want.float(), **tol(dt))
    x2 = xs.clone().cuda()
    assert mx.hyper_update_norm(x2, y.cuda(), mix.cuda(), w_out.cuda(), None, None, 1e-6) is None
    assert torch.allclose(x2.cpu(), mref.hyper_update(xs.clone(), y, mix, w_out), atol=1e-4,
                          rtol=1e-5)


@pytest.mark.parametrize("dt", DTYPES)
def test_token_shift_gate_gelu(dt):
    torch.manual_seed(12)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T, W = int(md["seq_qstart"][-1]), 72
    n, mu = torch.randn(T, W), torch.rand(W)
    st = torch.randn(5, W)
    st_g = st.clone().cuda()
    want = mref.token_shift(n, mu, st, md["positions"], md["seq_qstart"], md["seq_slot"], dt)
    got = mx.token_shift(n.cuda(), mu.cuda(), st_g, mdg["positions"], mdg["seq_qstart"],
                         mdg["seq_slot"], dt)
    rows = live_rows(md, LENS, SLOTS)
    assert torch.allclose(got.cpu().float()[rows], want.float()[rows], **tol(dt))
    assert torch.equal(st_g.cpu(), st)
    for N, off in ((96, 8), (50, 3)):
        big = torch.randn(T, 2 * N + 16).to(dt)
        a = torch.randn(T, N).to(dt)
        for act in ("sigmoid", "silu"):
            assert torch.allclose(mx.gate_mul(a.cuda(), big.cuda()[:, off:off + N], act).cpu().float(),
                                  mx.gate_mul(a, big[:, off:off + N], act).float(), **tol(dt))
        for tanh_form in (False, True):
            assert torch.allclose(mx.gelu(big.cuda()[:, off:off + N], tanh_form).cpu().float(),
                                  mref.gelu(big[:, off:off + N], tanh_form).float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,rot", [(6, 2, 64, 24), (4, 1, 48, 48), (8, 2, 128, 64), (2, 2, 32, 0)])
def test_rotate_half_norm_last_front_end(dt, H, G, dim, rot):
    """Rotate-half pairs, rotation before a weightless norm, values = the raw key projection."""
    torch.manual_seed(13)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T, nb, bs = int(md["seq_qstart"][-1]), md["num_pages"], 16
    P = torch.randn(T, (H + G) * dim + 16).to(dt)
    sl = (slice(None), slice(8, 8 + H * dim)), (slice(None), slice(8 + H * dim, 8 + (H + G) * dim))
    inv = mx.scaled_inv_freq(rot, 30000.0, (3.0, 1.0, 5.0, 256.0), "cpu")
    tab = mref.rotary_table(md["positions"], inv)
    kc, vc = torch.randn(nb, G, bs, dim).to(dt), torch.randn(nb, G, dim, bs).to(dt)
    kcg, vcg, Pg = kc.cuda(), vc.cuda(), P.cuda()
    qr = mref.qk_norm_rope_cache(P[sl[0]], P[sl[1]], P[sl[1]], None, None, 1e-6, md["positions"],
                                 md["slot_mapping"], tab, kc, vc, H, G, dim, dim, True, True)
    qg = mx.qk_norm_rope_cache(Pg[sl[0]], Pg[sl[1]], Pg[sl[1]], None, None, 1e-6,
                               mdg["positions"], mdg["slot_mapping"], tab.cuda(), kcg, vcg, H, G,
                               dim, dim, True, True)
    assert torch.allclose(qg.cpu().float(), qr.float(), **tol(dt))
    assert torch.allclose(kcg.cpu().float(), kc.float(), **tol(dt))
    assert torch.equal(vcg.cpu(), vc)


def test_scaled_inv_freq_bands():
    f = mx.inv_freq(32, 10000.0, "cpu").double()
    g = mx.scaled_inv_freq(32, 10000.0, (8.0, 1.0, 4.0, 64.0), "cpu").double()
    wave = 2 * np.pi / f
    for i in range(16):
        if wave[i] < 16:
            assert abs(g[i] - f[i]) < 1e-7 * f[i]
        elif wave[i] > 64:
            assert abs(g[i] - f[i] / 8) < 1e-7 * f[i]
        else:
            assert f[i] / 8 < g[i] < f[i]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim", [(6, 2, 64, 64), (4, 1, 48, 80), (8, 2, 128, 128)])
@pytest.mark.parametrize("window", [1, 31, 80, 128, 300])
def test_window_attention(dt, H, G, dim, vdim, window):
    """Windows shorter and longer than a tile, a partition and the contexts; decode rows whose
    window starts inside, at the edge of and before their first partition."""
    torch.manual_seed(14)
    lens, starts = [1, 1, 1, 1, 150, 70, 2], [0, 127, 128, 700, 333, 0, 71]
    md = ragged(lens, starts, list(range(7)), width=64)
    keep = md["tile_seq"] >= 4
    md["tile_seq"], md["tile_qoff"] = md["tile_seq"][keep], md["tile_qoff"][keep]
    mdg = cuda(md)
    T, nb = int(md["seq_qstart"][-1]), md["num_pages"]
    q = torch.randn(T, H, dim).to(dt)
    kc, vc = torch.randn(nb, G, 16, dim).to(dt), torch.randn(nb, G, vdim, 16).to(dt)
    want = mref.sink_attention(q, kc, vc, md["block_tables"], md["seq_kvlen"], md["seq_qstart"],
                               0.15, False, None, window)
    for mfma in (True, False):
        mx.ATTENTION_MFMA = mfma
        try:
            got = mx.sink_attention(q.cuda(), kc.cuda(), vc.cuda(), mdg["block_tables"],
                                    mdg["seq_kvlen"], mdg["seq_qstart"], mdg["tile_seq"],
                                    mdg["tile_qoff"], 0.15, False, num_decode=4, max_decode_kv=701,
                                    window=window)
        finally:
            mx.ATTENTION_MFMA = True
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt)), (mfma, window)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("C", [200, 64, 100, 1024])
def test_mingru_scan(dt, C):
    torch.manual_seed(15)
    lens, starts, slots = [1, 1, 37, 2, 600, 17], [0, 70, 0, 31, 5, 3], [3, -1, 0, 2, 1, 4]
    md = ragged(lens, starts, slots, width=64)
    mdg = cuda(md)
    T = int(md["seq_qstart"][-1])
    P = torch.randn(T, 3 * C + 24).to(dt) * 2
    cut = lambda t: (t[:, 8:8 + C], t[:, 8 + C:8 + 2 * C], t[:, 16 + 2 * C:16 + 3 * C])  # noqa: E731
    st = torch.randn(6, 1, 1, C)
    st_g = st.clone().cuda()
    want = mref.mingru_scan(*cut(P), st, md["positions"], md["seq_qstart"], md["seq_slot"], dt)
    got = mx.mingru_scan(*cut(P.cuda()), st_g, mdg["positions"], mdg["seq_qstart"],
                         mdg["seq_slot"], dt)
    rows = live_rows(md, lens, slots)
    assert torch.allclose(got.cpu().float()[rows], want.float()[rows], **tol(dt))
    assert torch.allclose(st_g.cpu(), st, atol=1e-4, rtol=1e-4)
    # a decode-sized step takes the one-wave path
    md1 = ragged([1, 1, 1], [5, 0, 9], [2, 0, -1])
    P1 = torch.randn(3, 3 * C + 24).to(dt)
    st1 = st.clone()
    st1_g = st.clone().cuda()
    want = mref.mingru_scan(*cut(P1), st1, md1["positions"], md1["seq_qstart"], md1["seq_slot"], dt)
    m1 = cuda(md1)
    got = mx.mingru_scan(*cut(P1.cuda()), st1_g, m1["positions"], m1["seq_qstart"], m1["seq_slot"],
                         dt)
    assert torch.allclose(got.cpu().float()[:2], want.float()[:2], **tol(dt))
    assert torch.allclose(st1_g.cpu(), st1, atol=1e-5)


@pytest.mark.parametrize("E,top", [(10, 1), (6, 2), (70, 4), (3, 3)])
def test_moe_route(E, top):
    torch.manual_seed(16)
    logits = torch.randn(200, E) * 3
    logits[5, :] = 0.0              # all equal: the lowest indices win
    idx, wts = mx.moe_route(logits.cuda(), top)
    ri, rw = mref.moe_route(logits, top)
    assert torch.equal(idx.cpu(), ri)
    assert torch.allclose(wts.cpu(), rw, atol=1e-6)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,E,top,ff,W", [(150, 10, 1, 72, 328), (3, 6, 2, 48, 96), (700, 4, 2, 200, 136),
                                          (65, 5, 3, 30, 50), (1, 8, 1, 128, 256), (5, 6, 2, 1024, 128),
                                          (2, 3, 1, 584, 64)])
def test_moe_experts(dt, T, E, top, ff, W):
    """Matrix-core kernels (bf16, widths % 8 == 0; small and large tiles) and the rows kernels
    (fp32, odd widths); tiles of one row and full tiles; clamps on both sides active; few tiles
    with a long down product (its K range cut over several workgroups); the library path of
    large steps against the grouped kernels."""
    torch.manual_seed(17)
    h = torch.randn(T, W).to(dt)
    wgu = (torch.randn(E, 2 * ff, W) * 2 / W ** 0.5).to(dt)
    wd = (torch.randn(E, W, ff) / ff ** 0.5).to(dt)
    idx, wts = mref.moe_route(torch.randn(T, E) * 2, top)
    want = mref.moe_experts(h, idx, wts, wgu, wd, 1.5, 1.702)
    t = dict(atol=6e-2, rtol=3e-2) if dt == torch.bfloat16 else dict(atol=5e-5, rtol=5e-5)
    for library_from in (0, 1):
        old, mx.MOE_LIBRARY_FLOPS = mx.MOE_LIBRARY_FLOPS, library_from
        try:
            got = mx.moe_experts(h.cuda(), idx.cuda(), wts.cuda(), wgu.cuda(), wd.cuda(), 1.5, 1.702)
        finally:
            mx.MOE_LIBRARY_FLOPS = old
        assert torch.allclose(got.cpu().float(), want.float(), **t), library_from


# ---- sandwich-norm boundary, whole-projection q / k norm, grouped routing, SiLU-GLU experts ----
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("W", [96, 100, 1024, 4096, 20000])
@pytest.mark.parametrize("kind", ["layer", "rms"])
def test_norm_add_norm(dt, W, kind):
    """Vector and plain kernel, both norms; rows with a common offset so the mean matters; every
    combination of (branch added or not) x (next norm or not) that a model uses."""
    torch.manual_seed(18)
    T = 7
    x = torch.randn(T, W) * 2 + 3
    y = (torch.randn(T, W) * 5 - 20).to(dt)
    wp, wn = (torch.rand(W) + 0.5).to(dt), (torch.rand(W) + 0.5).to(dt)
    t = dict(atol=4e-2, rtol=2e-2) if dt == torch.bfloat16 else dict(atol=3e-5, rtol=3e-5)
    for add, nxt in ((True, True), (False, True), (True, False)):
        xr, xg = x.clone(), x.clone().cuda()
        hr = mref.norm_add_norm(xr, y if add else None, wp if add else None, wn if nxt else None,
                                1e-5, kind == "layer", dt)
        hg = mx.norm_add_norm(xg, y.cuda() if add else None, wp.cuda() if add else None,
                              wn.cuda() if nxt else None, 1e-5, kind, dt)
        assert torch.allclose(xg.cpu(), xr, atol=3e-5, rtol=3e-5), (add, nxt)
        assert (hg is None) == (hr is None)
        if nxt:
            assert torch.allclose(hg.cpu().float(), hr.float(), **t), (add, nxt)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,rot", [(6, 2, 64, 48, 24), (4, 1, 48, 48, 48),
                                               (8, 2, 128, 128, 64), (3, 3, 10, 6, 0),
                                               (3, 1, 9, 5, 4)])
def test_whole_projection_norm_front_end(dt, H, G, dim, vdim, rot):
    """q and k normed over all their heads at once with weights per row of the projection
    (slices of a fused projection, aligned and not), then rotate-half positions."""
    torch.manual_seed(19)
    md = ragged(LENS, STARTS, SLOTS)
    mdg = cuda(md)
    T, nb, bs = int(md["seq_qstart"][-1]), md["num_pages"], 16
    nq, nk, nv = H * dim, G * dim, G * vdim
    P = torch.randn(T, nq + nk + nv + 16).to(dt)
    P[:, 8:8 + dim] *= 20                         # one large head: a per-head norm would differ
    sq = (slice(None), slice(8, 8 + nq))
    sk = (slice(None), slice(8 + nq, 8 + nq + nk))
    sv = (slice(None), slice(8 + nq + nk, 8 + nq + nk + nv))
    qw, kw = (torch.rand(nq) + 0.5).to(dt), (torch.rand(nk) + 0.5).to(dt)
    tab = (mref.rotary_table(md["positions"], mx.inv_freq(rot, 30000.0, "cpu")) if rot else
           torch.zeros(T, 0))
    kc, vc = torch.randn(nb, G, bs, dim).to(dt), torch.randn(nb, G, vdim, bs).to(dt)
    kcg, vcg, Pg = kc.cuda(), vc.cuda(), P.cuda()
    qr = mref.qk_norm_rope_cache(P[sq], P[sk], P[sv], qw, kw, 1e-6, md["positions"],
                                 md["slot_mapping"], tab, kc, vc, H, G, dim, vdim, True, False, True)
    qg = mx.qk_norm_rope_cache(Pg[sq], Pg[sk], Pg[sv], qw.cuda(), kw.cuda(), 1e-6,
                               mdg["positions"], mdg["slot_mapping"], tab.cuda(), kcg, vcg, H, G,
                               dim, vdim, rotate_half_pairs=True, whole_norm=True)
    assert torch.allclose(qg.cpu().float(), qr.float(), **tol(dt))
    assert torch.allclose(kcg.cpu().float(), kc.float(), **tol(dt))
    assert torch.equal(vcg.cpu(), vc)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("window", [0, 40, 128])
def test_learned_sink_with_window(dt, window):
    """The per-head sink score together with a window, in prefill tiles and in decode rows whose
    window covers one or several partitions (the combine adds the sink once)."""
    torch.manual_seed(20)
    H, G, dim, vdim = 6, 2, 64, 64
    lens, starts = [1, 1, 1, 150, 70], [0, 130, 700, 333, 0]
    md = ragged(lens, starts, list(range(5)), width=64)
    keep = md["tile_seq"] >= 3
    md["tile_seq"], md["tile_qoff"] = md["tile_seq"][keep], md["tile_qoff"][keep]
    mdg = cuda(md)
    T, nb = int(md["seq_qstart"][-1]), md["num_pages"]
    q = torch.randn(T, H, dim).to(dt)
    kc, vc = torch.randn(nb, G, 16, dim).to(dt), torch.randn(nb, G, vdim, 16).to(dt)
    sink = torch.tensor([-20.0, -1.0, 0.0, 2.0, 6.0, 30.0])
    want = mref.sink_attention(q, kc, vc, md["block_tables"], md["seq_kvlen"], md["seq_qstart"],
                               0.15, True, sink, window)
    for mfma in (True, False):
        mx.ATTENTION_MFMA = mfma
        try:
            got = mx.sink_attention(q.cuda(), kc.cuda(), vc.cuda(), mdg["block_tables"],
                                    mdg["seq_kvlen"], mdg["seq_qstart"], mdg["tile_seq"],
                                    mdg["tile_qoff"], 0.15, True, num_decode=3, max_decode_kv=701,
                                    sink_values=sink.cuda(), window=window)
        finally:
            mx.ATTENTION_MFMA = True
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt)), (mfma, window)


@pytest.mark.parametrize("E,top,groups,keep", [(10, 1, 1, 1), (20, 3, 5, 2), (64, 6, 8, 3),
                                               (70, 4, 5, 2), (256, 8, 8, 4), (300, 5, 300, 7),
                                               (1024, 8, 16, 2), (3, 3, 3, 3)])
@pytest.mark.parametrize("softmax", [True, False])
def test_moe_route_grouped(E, top, groups, keep, softmax):
    """All three register tiers of the route kernel (<= 64, <= 256, <= 1024 experts), row counts
    that leave waves of the last workgroup without a row, with and without correction."""
    torch.manual_seed(21)
    for T in (1, 6, 203):
        logits = torch.randn(T, E) * 3
        corr = torch.randn(E) * (0.3 / E if softmax else 0.2)
        for c in (corr, None):
            for renorm in (True, False):
                idx, wts = mx.moe_route(logits.cuda(), top, "softmax" if softmax else "sigmoid",
                                        None if c is None else c.cuda(), groups, keep, renorm)
                ri, rw = mref.moe_route(logits, top, "softmax" if softmax else "sigmoid", c, groups,
                                            keep, renorm)
                # the order among the chosen is by choice score; compare as sets with weights
                so, ro = torch.argsort(idx.cpu(), 1), torch.argsort(ri, 1)
                same = (torch.gather(idx.cpu(), 1, so) == torch.gather(ri, 1, ro)).all(1)
                assert same.float().mean() > 0.97     # fp32 ties between near-equal scores aside
                gw, ww = torch.gather(wts.cpu(), 1, so), torch.gather(rw, 1, ro)
                assert torch.allclose(gw[same], ww[same], atol=1e-6, rtol=1e-5)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,E,ident,top,ff,W", [(150, 10, 0, 1, 72, 328), (3, 6, 2, 2, 48, 96),
                                                (700, 4, 1, 2, 200, 136), (65, 5, 3, 3, 30, 50),
                                                (1, 8, 0, 1, 128, 256), (5, 6, 2, 2, 1024, 128),
                                                (2, 1, 3, 2, 584, 64)])
def test_moe_experts_silu_identity(dt, T, E, ident, top, ff, W):
    """The SiLU-GLU form with the weights on the outputs, identity experts and an added row, in
    all tile forms of the grouped kernels (small, large, split down product, rows kernels) and on
    the library path."""
    torch.manual_seed(22)
    h = torch.randn(T, W).to(dt)
    wgu = (torch.randn(E, 2 * ff, W) * 2 / W ** 0.5).to(dt)
    wd = (torch.randn(E, W, ff) / ff ** 0.5).to(dt)
    idx, wts = mref.moe_route(torch.randn(T, E + ident) * 2, top, "softmax", None, 1, 1, True)
    add = torch.randn(T, W).to(dt)
    t = dict(atol=6e-2, rtol=3e-2) if dt == torch.bfloat16 else dict(atol=5e-5, rtol=5e-5)
    for addend in (add, None):
        want = mref.moe_experts(h, idx, wts, wgu, wd, 0.0, 0.0, True, addend)
        for library_from in (0, 1):
            old, mx.MOE_LIBRARY_FLOPS = mx.MOE_LIBRARY_FLOPS, library_from
            try:
                got = mx.moe_experts(h.cuda(), idx.cuda(), wts.cuda(), wgu.cuda(), wd.cuda(),
                                     glu="silu", addend=None if addend is None else addend.cuda())
            finally:
                mx.MOE_LIBRARY_FLOPS = old
            assert torch.allclose(got.cpu().float(), want.float(), **t), library_from


@pytest.mark.parametrize("dt", DTYPES)
def test_strided_glu_and_softcap(dt):
    torch.manual_seed(23)
    for T, n, pad in ((5, 72, 8), (3, 50, 6), (300, 1024, 0)):
        P = (torch.randn(T, 2 * n + pad) * 3).to(dt)
        g, u = P[:, :n], P[:, n + pad:]
        for act, code in (("gelu_tanh", 2), ("silu", 0), ("sigmoid", 1)):
            got = mx.gate_mul(P.cuda()[:, n + pad:], P.cuda()[:, :n], act)
            assert torch.allclose(got.cpu().float(), mref.gate_mul(u, g, code).float(), **tol(dt))
    z = (torch.randn(9, 1000) * 40).to(dt)
    for scale, cap in ((0.3, 12.0), (1.0, 0.0), (2.0, 50.0)):
        got = mx.scale_softcap(z.cuda(), scale, cap)
        assert got.dtype == torch.float32
        assert torch.allclose(got.cpu(), mref.scale_softcap(z, scale, cap), atol=2e-5, rtol=1e-5)


# ---- sigmoid attention, post-norm boundary, value path, gates ------------------------------------

def ragged_pages(md, G, dim, vdim, bs, dt, seed=0):
    g = torch.Generator().manual_seed(seed)
    nb = md["num_pages"]
    return (torch.randn(nb, G, bs, dim, generator=g).to(dt),
            torch.randn(nb, G, vdim, bs, generator=g).to(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,bs,cap", [
    (6, 6, 40, 48, 16, 7.0), (8, 2, 64, 64, 16, 0.0), (12, 4, 128, 128, 32, 20.0),
    (24, 8, 128, 96, 8, 15.0), (32, 8, 128, 128, 16, 30.0), (3, 1, 16, 16, 16, 5.0),
    (20, 2, 72, 32, 16, 9.0), (5, 5, 13, 9, 16, 4.0), (40, 8, 32, 16, 16, 6.0),
    (4, 2, 32, 32, 12, 6.0), (8, 8, 192, 160, 16, 11.0), (1, 1, 8, 16, 16, 0.0)])
def test_sigmoid_attention(dt, H, G, dim, vdim, bs, cap, monkeypatch):
    torch.manual_seed(1)
    lens, starts = [1, 1, 37, 2, 150, 64, 16], [0, 170, 0, 131, 45, 200, 15]
    md = ragged(lens, starts, list(range(7)), bs=bs, width=48)
    T = int(md["seq_qstart"][-1])
    q = torch.randn(T, H, dim).to(dt)
    kc, vc = ragged_pages(md, G, dim, vdim, bs, dt)
    bias = torch.randn(H) - 3.0
    talk = (torch.eye(H) + 0.3 * torch.randn(H, H)).to(torch.bfloat16).float()
    scale = 1.7 * dim ** -0.5
    want = mref.sigmoid_attention(q, kc, vc, md["block_tables"], md["seq_kvlen"],
                                  md["seq_qstart"], scale, cap, bias, talk).float()
    g = cuda(md)
    # the single-row portions in the tile kernel, then as decode rows; with and without key shares
    for nd, shares in ((0, 4), (2, 4), (2, 1), (0, 7)):
        monkeypatch.setattr(mx, "SIGMOID_MAX_SPLIT", shares)
        keep = md["tile_seq"] >= nd
        got = mx.sigmoid_attention(q.cuda(), kc.cuda(), vc.cuda(), g["block_tables"],
                                   g["seq_kvlen"], g["seq_qstart"],
                                   md["tile_seq"][keep].cuda(), md["tile_qoff"][keep].cuda(),
                                   scale, cap, bias.cuda(), talk.cuda(), nd,
                                   int(md["seq_kvlen"][:max(nd, 1)].max())).cpu().float()
        err = (got - want).abs() / (want.abs() + want.pow(2).mean().sqrt())
        bf = dt == torch.bfloat16
        assert float(err.max()) < (4e-2 if bf else 2e-5), (nd, float(err.max()))
        assert float(err.mean()) < (4e-3 if bf else 2e-6), (nd, float(err.mean()))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("W", [40, 100, 1024, 4096, 33000])
def test_post_norm(dt, W):
    torch.manual_seed(2)
    T = 9
    x = 3 * torch.randn(T, W)
    a, b = torch.randn(T, W).to(dt), torch.randn(T, W).to(dt)
    w = (1 + 0.1 * torch.randn(W)).to(dt)
    for bb in (b, None):
        xr, xg = x.clone(), x.clone().cuda()
        want = mref.post_norm(xr, 1.7, a, 0.6, bb, 0.9, w, 1e-5, dt)
        got = mx.post_norm(xg, 1.7, a.cuda(), 0.6, None if bb is None else bb.cuda(), 0.9,
                           w.cuda(), 1e-5, dt)
        assert torch.allclose(xg.cpu(), xr, atol=2e-5, rtol=2e-5)
        assert got.dtype == dt
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("G,vdim,bs", [(2, 48, 16), (3, 20, 16), (1, 130, 8), (2, 9, 12)])
def test_values_normed_mixed_and_temperature(dt, G, vdim, bs):
    torch.manual_seed(3)
    H, dim = 2 * G, 24
    md = ragged(LENS, STARTS, SLOTS, bs=bs, width=20)
    md["slot_mapping"][1] = -1
    g = cuda(md)
    T = int(md["seq_qstart"][-1])
    P = torch.randn(T, H * dim + G * dim + G * vdim + 8).to(dt)
    qn, kn = torch.randn(H * dim).to(dt), torch.randn(G * dim).to(dt)
    first = torch.randn(T, G * vdim).to(dt)
    table = mref.rotary_table(md["positions"], mx.inv_freq(10, 50.0, "cpu"), 1.3)
    tg = mx.rotary_table(g["positions"], mx.inv_freq(10, 50.0, "cuda"), 1.3)
    assert torch.allclose(tg.cpu(), table, atol=1e-5, rtol=1e-5)
    cut = lambda t: (t[:, :H * dim], t[:, H * dim:(H + G) * dim],  # noqa: E731
                     t[:, (H + G) * dim:(H + G) * dim + G * vdim])
    for norm, fst in ((True, None), (True, first), (False, first), (False, None)):
        kc, vc = ragged_pages(md, G, dim, vdim, bs, dt, 5)
        kg, vg = kc.clone().cuda(), vc.clone().cuda()
        vo, vog = torch.zeros(T, G * vdim, dtype=dt), torch.zeros(T, G * vdim, dtype=dt).cuda()
        kw = dict(rotate_half_pairs=True, whole_norm=True, q_temp=(0.4, 7.0), v_norm=norm,
                  v_lambda=0.3)
        want = mref.qk_norm_rope_cache(*cut(P), qn, kn, 1e-5, md["positions"], md["slot_mapping"],
                                       table, kc, vc, H, G, dim, vdim, v_first=fst, v_out=vo, **kw)
        got = mx.qk_norm_rope_cache(*cut(P.cuda()), qn.cuda(), kn.cuda(), 1e-5, g["positions"],
                                    g["slot_mapping"], tg, kg, vg, H, G, dim, vdim,
                                    v_first=None if fst is None else fst.cuda(), v_out=vog, **kw)
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))
        assert torch.allclose(kg.cpu().float(), kc.float(), **tol(dt))
        assert torch.allclose(vg.cpu().float(), vc.float(), **tol(dt))
        live = md["slot_mapping"][:T] >= 0
        assert torch.allclose(vog.cpu().float()[live], vo.float()[live], **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
def test_gates_and_interleaved_latent_front_end(dt):
    torch.manual_seed(4)
    md = ragged(LENS, STARTS, SLOTS)
    g = cuda(md)
    T, H = int(md["seq_qstart"][-1]), 3
    for dv in (16, 20):
        o, wide = torch.randn(H, T, dv).to(dt), torch.randn(T, H * dv + 8).to(dt)
        for gate in (wide[:, :H], wide[:, :H * dv]):
            got = mx.head_gate(o.cuda(), wide.cuda()[:, :gate.shape[1]])
            assert torch.allclose(got.cpu().float(), mref.head_gate(o, gate).float(), **tol(dt))
    # interleaved pairs on the rotated part of row-strided queries
    rank, rot, qd, bs = 24, 12, 16, 16
    wide = torch.randn(T, H * (qd + rot) + 8).to(dt)
    q_lat, kvx = torch.randn(H, T, rank).to(dt), torch.randn(T, rank + rot).to(dt)
    cn = torch.randn(rank).to(dt)
    table = mref.rotary_table(md["positions"], mx.inv_freq(10, 50.0, "cpu"))
    res = []
    for dev, m_ in (("cpu", md), ("cuda", g)):
        qx = wide.to(dev)[:, :H * (qd + rot)].unflatten(1, (H, qd + rot))
        kc = torch.zeros(md["num_pages"], 1, bs, rank + rot, dtype=dt, device=dev)
        vc = torch.zeros(md["num_pages"], 1, rank, bs, dtype=dt, device=dev)
        q = mx.latent_rope_cache(q_lat.to(dev), qx, kvx.to(dev), cn.to(dev), 1e-5,
                                 m_["slot_mapping"], table.to(dev), kc, vc, False)
        res.append([t.cpu().float() for t in (q, kc, vc)])
    for a, b in zip(*res):
        assert torch.allclose(a, b, **tol(dt))
    # per-head gate in the attention kernels' store: tiles and decode rows
    for dim, vdim in ((32, 64), (20, 12)):
        G = 3
        q = torch.randn(T, H, dim).to(dt)
        kc, vc = ragged_pages(md, G, dim, vdim, 16, dt)
        gate = torch.randn(T, 11).to(dt)
        want = mref.sink_attention(q, kc, vc, md["block_tables"], md["seq_kvlen"],
                                   md["seq_qstart"], 0.2, False, None, 9, gate[:, 8:])
        keep = md["tile_seq"] >= 2
        got = mx.sink_attention(q.cuda(), kc.cuda(), vc.cuda(), g["block_tables"], g["seq_kvlen"],
                                g["seq_qstart"], md["tile_seq"][keep].cuda(),
                                md["tile_qoff"][keep].cuda(), 0.2, False, 2, 71, None, 9,
                                gate.cuda()[:, 8:])
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))


@pytest.mark.parametrize("E,top", [(16, 2), (5, 5), (70, 3), (300, 4), (3, 1)])
def test_route_by_logit(E, top):
    logits = 40 * torch.randn(50, E)
    logits[3] -= 500.0          # a softmax over the row would leave no second choice
    logits[3, 1] += 900.0
    got = mx.moe_route(logits.cuda(), top, "logit")
    want = mref.moe_route(logits, top, "logit")
    assert torch.equal(got[0].cpu(), want[0])
    assert torch.allclose(got[1].cpu(), want[1], atol=1e-6, rtol=1e-5)


# ---- retention, differential attention, windows that keep the first tokens ------------------------
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,dk,dv,nf", [(3, 64, 64, 32), (2, 128, 128, 32), (4, 24, 20, 8), (2, 32, 80, 16),
                                        (1, 256, 64, 64), (3, 48, 72, 0), (2, 9, 5, 2), (1, 1, 1, 0)])
def test_retention(dt, H, dk, dv, nf):
    torch.manual_seed(dk + dv)
    lens, starts, slots = [1, 1, 70, 2, 64, 129, 200, 3], [5, 0, 0, 11, 0, 64, 7, 0], [3, 1, 0, 2, -1, 5, 4, 6]
    md = ragged(lens, starts, slots, width=24)
    T = int(md["seq_qstart"][-1])
    P = torch.randn(T, 2 * H * dk + H * dv + 24).to(dt)
    state = torch.randn(8, H, dk, dv)
    state_g = state.cuda()
    tab = (mref.rotary_table(md["positions"], mx.inv_freq(2 * nf, 1000.0, "cpu")) if nf else
           torch.zeros(T, 0))
    pw = mx.retention_powers([0.9, 0.97, 0.999, 0.5][:H], "cpu")

    def cut(X):
        return (X[:, 8:8 + H * dk], X[:, 8 + H * dk:8 + 2 * H * dk],
                X[:, 8 + 2 * H * dk:8 + 2 * H * dk + H * dv])

    g = cuda(md)
    a = mref.retention(*cut(P), pw[:, 1], tab, state, md["positions"], md["seq_qstart"],
                       md["seq_slot"], H, dk, dv)
    b = mx.retention(*cut(P.cuda()), pw.cuda(), tab.cuda(), state_g, g["positions"], g["seq_qstart"],
                     g["seq_slot"], H, dk, dv, 2)
    live = torch.ones(T, dtype=torch.bool)
    live[int(md["seq_qstart"][4]):int(md["seq_qstart"][5])] = False
    scale = float(a.abs().max())
    assert float((a - b.cpu())[live].abs().max()) < 1e-5 * scale      # fp32 inside for both dtypes
    assert float((state - state_g.cpu()).abs().max()) < 1e-5 * float(state.abs().max())


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,window,keep", [(4, 2, 32, 64, 40, 5), (6, 1, 16, 32, 0, 0),
                                                  (2, 2, 64, 128, 150, 140), (8, 4, 12, 20, 17, 30),
                                                  (3, 3, 80, 96, 130, 2), (2, 1, 48, 160, 9, 1)])
def test_differential_attention(dt, H, G, d, dv, window, keep):
    """Decode rows, portions and pages in one ragged batch; the pair form and the two-step path."""
    torch.manual_seed(H * d)
    lens, starts = [1, 1, 1, 37, 2, 130], [0, 290, 128, 0, 140, 60]
    md = ragged(lens, starts, [0, 1, 2, 3, 4, 5], width=24)
    T, nb = int(md["seq_qstart"][-1]), md["num_pages"]
    k, v = torch.randn(nb, 2 * G, 16, d).to(dt), torch.randn(nb, G, dv, 16).to(dt)
    wide = torch.randn(T, 2 * H * d + H * dv + 32).to(dt)
    tiles = md["tile_seq"] >= 3
    md["tile_seq"], md["tile_qoff"] = md["tile_seq"][tiles], md["tile_qoff"][tiles]
    g = cuda(md)

    def run(w, kc, vc, m, **kw):
        q = w[:, 8:8 + 2 * H * d].unflatten(1, (2 * H, d))
        gate = w[:, 8 + 2 * H * d + 8:8 + 2 * H * d + 8 + H * dv]
        return mx.differential_attention(q, kc, vc, m["block_tables"], m["seq_kvlen"], m["seq_qstart"],
                                         m["tile_seq"], m["tile_qoff"], d ** -0.5, 0.7, 0.3, 1e-5,
                                         gate, 3, 291, window, keep)

    want, got = run(wide, k, v, md), run(wide.cuda(), k.cuda(), v.cuda(), g).cpu()
    t = dict(atol=4e-2, rtol=4e-2) if dt == torch.bfloat16 else dict(atol=2e-5, rtol=1e-4)
    assert torch.allclose(got.float(), want.float(), **t)
    if dt == torch.bfloat16 and mx.mfma_attention_ok(wide[:, :d].view(T, 1, d), k, v):
        was, mx.ATTENTION_MFMA = mx.ATTENTION_MFMA, False
        try:
            rows = run(wide.cuda(), k.cuda(), v.cuda(), g).cpu()
        finally:
            mx.ATTENTION_MFMA = was
        assert torch.allclose(rows.float(), want.float(), **t)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("d,dv", [(32, 64), (20, 28)])
@pytest.mark.parametrize("window,keep", [(40, 5), (140, 300), (16, 16), (1, 1)])
def test_kept_tokens_with_sink_and_gate(dt, d, dv, window, keep):
    torch.manual_seed(window)
    lens, starts = [1, 1, 37, 2, 130], [290, 0, 0, 140, 60]
    md = ragged(lens, starts, [0, 1, 2, 3, 4], width=24)
    T, nb, H, G = int(md["seq_qstart"][-1]), md["num_pages"], 4, 2
    q, gate = torch.randn(T, H, d).to(dt), torch.randn(T, H).to(dt)
    k, v = torch.randn(nb, G, 16, d).to(dt), torch.randn(nb, G, dv, 16).to(dt)
    sink = torch.randn(H)
    tiles = md["tile_seq"] >= 2
    md["tile_seq"], md["tile_qoff"] = md["tile_seq"][tiles], md["tile_qoff"][tiles]
    want = mref.sink_attention(q, k, v, md["block_tables"], md["seq_kvlen"], md["seq_qstart"], 0.2,
                               True, sink, window, gate, keep)
    g = cuda(md)
    got = mx.sink_attention(q.cuda(), k.cuda(), v.cuda(), g["block_tables"], g["seq_kvlen"],
                            g["seq_qstart"], g["tile_seq"], g["tile_qoff"], 0.2, True, 2, 291,
                            sink.cuda(), window, gate.cuda(), keep)
    assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
def test_branch_scale_norms_and_glu(dt):
    torch.manual_seed(4)
    for W in (64, 100, 2048):
        x = torch.randn(5, W)
        y, w, s, wn = (torch.randn(*n).to(dt) for n in ((5, W), (W,), (W,), (W,)))
        xg = x.cuda()
        want = mref.norm_add_norm(x, y, w, wn, 1e-5, False, dt, s)
        got = mx.norm_add_norm(xg, y.cuda(), w.cuda(), wn.cuda(), 1e-5, "rms", dt, post_scale=s.cuda())
        assert torch.allclose(xg.cpu(), x, atol=2e-5, rtol=2e-5)
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))
    for dv in (12, 64, 128, 136, 600):
        o, gate, w = torch.randn(7, 3, dv), torch.randn(7, 3 * dv + 8).to(dt), torch.randn(dv).to(dt)
        for wt in (None, w):
            for act in ("silu", "sigmoid"):
                want = mref.gated_rms_norm(o, gate[:, 8:], wt, 1e-5, act, dt)
                got = mx.gated_rms_norm(o.cuda(), gate.cuda()[:, 8:], wt.cuda() if wt is not None else None,
                                        1e-5, act, dt)
                assert torch.allclose(got.cpu().float(), want.float(), **tol(dt)), (dv, act)
    for n, off in ((64, 8), (33, 1), (2048, 0)):
        p = (3.0 * torch.randn(6, 2 * n + off)).to(dt)
        want = mref.clamped_gate_mul(p[:, off + n:], p[:, off:off + n], 2.0)
        pg = p.cuda()
        got = mx.clamped_gate_mul(pg[:, off + n:], pg[:, off:off + n], 2.0)
        assert torch.allclose(got.cpu().float(), want.float(), **tol(dt))


@pytest.mark.parametrize("E,top,scale", [(16, 4, 2.5), (5, 5, 1.0), (70, 3, 0.5), (300, 8, 7.0)])
def test_scaled_sigmoid_route(E, top, scale):
    logits = 2.0 * torch.randn(33, E, generator=torch.Generator().manual_seed(E))
    idx, w = mx.moe_route(logits.cuda(), top, "sigmoid", renorm=True, scale=scale)
    ri, rw = mref.moe_route(logits, top, "sigmoid", renorm=True, scale=scale)
    assert torch.equal(idx.cpu(), ri) and torch.allclose(w.cpu(), rw, atol=1e-5, rtol=1e-5)
    assert torch.allclose(w.cpu().sum(1), torch.full((33,), scale), rtol=1e-4)
