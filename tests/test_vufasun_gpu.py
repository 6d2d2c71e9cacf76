"""Vufasun on the GPU against the plain statement in ``oracle/vufasun.py``: every mechanism alone, then whole models
through the engine -- the streams after every layer run, whole prompts, token-by-token decoding, portions down to two
tokens, mixed batches, pages and state slots that are reused, greedy generation through ``LLM.generate``, the replay entry
point.

The models are small and random (``tests/vufasun_util.py``); where random numbers would hide a fault (one far key among
hundreds, a key on a page border, a missing sink, a state that fades) the inputs are built so that it shows.
"""
import random
from types import SimpleNamespace

import pytest
import torch

import vufasun_util as vu
from mixer_harness import DEV, attention_case, ops, paged, ragged, steps_of, tol_of
from oracle import vufasun as oracle

pytestmark = pytest.mark.gpu
F64 = torch.float64
BOTH = [torch.float32, torch.bfloat16]


# ------------------------------------------------------------------ the streams
def _connection(s, g):
    return 0.6 * torch.eye(s) + 0.4 * torch.randn(s, s, generator=g), torch.randn(s, generator=g), torch.randn(s, generator=g)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("width", [22, 48, 260, 516, 1030, 2560, 8200])
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 8])
def test_a_step_of_the_streams(streams, width, dtype):
    """The write to all streams from the old ones, the next read and its norm; addends in every combination; a row small
    enough for eps to count; outputs into place, neighbours in memory untouched."""
    g = torch.Generator().manual_seed(width + streams)
    rows, eps = 5, 1e-5
    x = torch.randn(rows, streams, width, generator=g) * 3
    mix, writes, reads = _connection(streams, g)
    wide = (torch.randn(rows, 2 * width + 4, generator=g)).to(dtype)
    a, b, c = wide[:, 4:4 + width], wide[:, 4 + width:], torch.randn(rows, width, generator=g)
    x[3], wide[3], c[3] = x[3] * 1e-4, wide[3] * 1e-4, c[3] * 1e-4
    w = torch.randn(width, generator=g) * 0.3 + 1.0
    dev = lambda t: t.to(DEV)                                            # noqa: E731
    wide_d = dev(wide)
    for use in [(1, 0, 0), (1, 0, 1), (1, 1, 1), (0, 0, 1), (0, 0, 0)]:
        got = dev(x.clone())
        out = torch.full((rows, width), float("nan"), dtype=dtype, device=DEV)
        parts = [t if u else None for t, u in zip((wide_d[:, 4:4 + width], wide_d[:, 4 + width:], dev(c)), use)]
        ops().hyper_step(got, out, eps, None, dev(mix), dev(writes), *parts, reads=dev(reads), weight=dev(w))
        y = sum((t.double() for t, u in zip((a, b, c), use) if u), torch.zeros(rows, width, dtype=F64))
        want = oracle.write_streams(x.double().transpose(0, 1), mix.double(), writes.double(), y)
        torch.testing.assert_close(got.cpu().double(), want.transpose(0, 1), atol=2e-5, rtol=2e-5)
        read = oracle.rms_norm(oracle.read_streams(want, reads.double()), w.double(), eps)
        torch.testing.assert_close(out.cpu().double(), read, **tol_of(dtype))
    # without an output: only the write
    got2 = dev(x.clone())
    ops().hyper_step(got2, None, eps, None, dev(mix), dev(writes), wide_d[:, 4:4 + width])
    y = oracle.write_streams(x.double().transpose(0, 1), mix.double(), writes.double(), a.double())
    torch.testing.assert_close(got2.cpu().double(), y.transpose(0, 1), atol=2e-5, rtol=2e-5)
    # without a write: the streams stay
    got3, out = dev(x.clone()), torch.empty(rows, width, dtype=dtype, device=DEV)
    ops().hyper_step(got3, out, eps, reads=dev(reads), weight=dev(w))
    assert torch.equal(got3.cpu(), x)
    read = oracle.rms_norm(oracle.read_streams(x.double().transpose(0, 1), reads.double()), w.double(), eps)
    torch.testing.assert_close(out.cpu().double(), read, **tol_of(dtype))


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("width", [22, 48, 1030, 2560, 4096])
def test_mean_of_two_normed_outputs_goes_into_the_streams(width, dtype):
    g = torch.Generator().manual_seed(width)
    rows, s, eps = 6, 4, 1e-5
    x = torch.randn(rows, s, width, generator=g)
    mix, writes, reads = _connection(s, g)
    a, b = torch.randn(rows, width, generator=g).to(dtype), (torch.randn(rows, width, generator=g) * 30).to(dtype)
    a[2] *= 1e-3                                                         # small enough for eps to count
    wa, wb, w = (torch.randn(width, generator=g) * 0.4 + 1.0 for _ in range(3))
    got, out = x.clone().to(DEV), torch.empty(rows, width, dtype=dtype, device=DEV)
    ops().hyper_step(got, out, eps, None, mix.to(DEV), writes.to(DEV), a.to(DEV), b.to(DEV), norms=(wa.to(DEV), wb.to(DEV)),
                     blend=0.5, reads=reads.to(DEV), weight=w.to(DEV))
    y = 0.5 * (oracle.rms_norm(a.double(), wa.double(), eps) + oracle.rms_norm(b.double(), wb.double(), eps))
    want = oracle.write_streams(x.double().transpose(0, 1), mix.double(), writes.double(), y)
    torch.testing.assert_close(got.cpu().double(), want.transpose(0, 1), atol=2e-5, rtol=2e-5)
    torch.testing.assert_close(out.cpu().double(), oracle.rms_norm(oracle.read_streams(want, reads.double()), w.double(), eps),
                               **tol_of(dtype))


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("width,streams", [(22, 3), (48, 1), (1030, 2), (2560, 4)])
def test_streams_begin_in_the_embedding_table(width, streams, dtype):
    """The first read and the first write take the old streams from the table; an id beyond it shows as NaN."""
    from splitwise_amd.model_executor.layers.basic import HyperConnection, OffsetRMSNorm
    g = torch.Generator().manual_seed(width)
    table = torch.randn(31, width, generator=g).to(dtype)
    ids = torch.tensor([0, 30, 7, 7, 12, 31, -1])
    norm, first = OffsetRMSNorm(width, 1e-5, 0.0), HyperConnection(streams)
    norm.weight.data.copy_(torch.randn(width, generator=g) * 0.3 + 1.0)
    mix, writes, reads = _connection(streams, g)
    for t, v in ((first.mix, mix), (first.writes, writes), (first.reads, reads)):
        t.data.copy_(v)
    norm, first = norm.to(DEV), first.to(DEV)
    origin = (ids.to(DEV), table.to(DEV))
    h = HyperConnection.begin(origin, first.reads.data, norm)
    e = table[ids[:5]].double()
    X = torch.stack([e] * streams)
    w = norm.weight.cpu().double()
    torch.testing.assert_close(h[:5].cpu().double(), oracle.rms_norm(oracle.read_streams(X, reads.double()), w, 1e-5), **tol_of(dtype))
    y = torch.randn(7, width, generator=g).to(dtype)
    x = torch.full((7, streams, width), float("nan"), device=DEV)
    nxt = torch.randn(streams, generator=g)
    h2 = first.step(x, nxt.to(DEV), norm, dtype, a=y.to(DEV), origin=origin)
    want = oracle.write_streams(X, mix.double(), writes.double(), y[:5].double())
    torch.testing.assert_close(x[:5].cpu().double(), want.transpose(0, 1), atol=2e-5, rtol=2e-5)
    torch.testing.assert_close(h2[:5].cpu().double(), oracle.rms_norm(oracle.read_streams(want, nxt.double()), w, 1e-5), **tol_of(dtype))
    assert torch.isnan(h[5:]).all() and torch.isnan(h2[5:]).all()


def test_stream_counts_and_widths_beyond_the_kernel_are_refused():
    x, w = torch.zeros(1, 9, 16, device=DEV), torch.ones(16, device=DEV)
    with pytest.raises(RuntimeError, match="streams"):
        ops().hyper_step(x, torch.empty(1, 16, device=DEV), 1e-5, reads=torch.ones(9, device=DEV), weight=w)
    wide = torch.zeros(1, 1, 16392, device=DEV)
    with pytest.raises(RuntimeError, match="too wide"):
        ops().hyper_step(wide, torch.empty(1, 16392, device=DEV), 1e-5, reads=torch.ones(1, device=DEV), weight=torch.ones(16392, device=DEV))


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("kind", ["silu", "gelu_tanh"])
@pytest.mark.parametrize("ff", [33, 40, 2112])
def test_gated_activations(ff, kind, dtype):
    from splitwise_amd.model_executor.layers.basic import GatedActivation
    g = torch.Generator().manual_seed(ff)
    x = (torch.randn(9, 2 * ff, generator=g) * 3).to(dtype)
    x[0, :8] = torch.tensor([-1e4, -40.0, -9.0, -1e-3, 0.0, 1e-3, 9.0, 1e4])        # both tails
    act = {"silu": oracle.silu, "gelu_tanh": oracle.gelu_tanh}[kind]
    want = act(x[:, :ff].double()) * x[:, ff:].double()
    torch.testing.assert_close(GatedActivation(kind)(x.to(DEV)).cpu().double(), want, **tol_of(dtype))
    wide = torch.full((9, ff + 8), 7.0, dtype=dtype, device=DEV)
    ops().gated_act(wide[:, 8:], x.to(DEV), {"silu": ops().GATE_SILU, "gelu_tanh": ops().GATE_GELU_TANH}[kind])
    torch.testing.assert_close(wide[:, 8:].cpu().double(), want, **tol_of(dtype))
    assert (wide[:, :8] == 7.0).all()


# ------------------------------------------------------------------ rotated operands
@pytest.mark.parametrize("H,G,d,dv,dims,lead", [(4, 2, 16, 12, 16, 0), (3, 1, 7, 5, 4, 3), (6, 3, 24, 20, 16, 4), (2, 2, 64, 32, 24, 8),
                                                (2, 1, 12, 8, 12, 4), (1, 1, 512, 3, 512, 0), (4, 4, 8, 8, 0, 0)])
@pytest.mark.parametrize("R,rd,rdims", [(3, 8, 8), (2, 5, 2), (1, 20, 16)])
@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("normed", [False, True])
def test_rotated_operands_of_one_mixer_and_of_two(H, G, d, dv, dims, lead, R, rd, rdims, dtype, normed):
    """Queries and keys of both sides against the oracle at positions up to 70000; one norm over ALL heads before the rotation
    where there is one; rows without a slot; neighbours in the cache untouched; either side alone."""
    g = torch.Generator().manual_seed(H * 100 + d + R)
    rows, page, eps = 7, 8, 1e-5
    positions = torch.tensor([0, 1, 7, 300, 2047, 9, 70000])
    sizes = [H * d, G * d, G * dv, R * rd, R * rd]
    proj = torch.randn(rows, lead + sum(sizes) + 1, generator=g).to(dtype)
    proj = torch.cat([proj, proj.new_zeros(rows, -proj.shape[1] % 4)], 1)
    cut = [lead + sum(sizes[:i]) for i in range(6)]
    proj[3, cut[0]:cut[2]] *= 1e-3                                       # small enough for eps to count
    q, k, v, rq, rk = (proj[:, lo:hi] for lo, hi in zip(cut, cut[1:]))
    pd = proj.to(DEV)
    qd, kd, vd, rqd, rkd = (pd[:, lo:hi] for lo, hi in zip(cut, cut[1:]))
    f = oracle.rotary_frequencies({"dims": dims, "base": 30.0, "scaling": vu.scaling()})
    rf = oracle.rotary_frequencies({"dims": rdims, "base": 500.0})
    inv, rinv = (torch.tensor(x, dtype=torch.float32, device=DEV) for x in (f, rf))
    wq, wk = torch.randn(H * d, generator=g), torch.randn(G * d, generator=g)
    slots = torch.tensor([9, -1, 17, 31, 16, 8, 0])
    kc, vc = torch.full((4, page, G * d), 5.0, dtype=dtype, device=DEV), torch.full((4, page, G * dv), 5.0, dtype=dtype, device=DEV)

    def check(att, lin):
        q_out = torch.full((rows, H * d), float("nan"), device=DEV)
        lq, lk = (torch.full((rows, R * rd), float("nan"), device=DEV) for _ in range(2))
        ops().rope_operands(positions.to(DEV), (q_out, qd, kd, vd, inv, H, G, d, dv, kc, vc, slots.to(DEV)) if att else None,
                            (lq, lk, rqd, rkd, rinv, R, rd, 0.37) if lin else None, wq.to(DEV) if normed and att else None,
                            wk.to(DEV) if normed and att else None, eps if normed else 0.0)

        def turned(x, heads, size, freqs, w=None):
            x = x.double()
            x = oracle.rms_norm(x, w.double(), eps) if w is not None else x
            return torch.stack([oracle.rotate_halves(x[t].view(heads, size), int(positions[t]), freqs) for t in range(rows)]).flatten(1)
        exact = dict(atol=3e-5, rtol=3e-5)
        if att:
            torch.testing.assert_close(q_out.cpu().double(), turned(q, H, d, f, wq if normed else None), **exact)
            want = turned(k, G, d, f, wk if normed else None)
            kf, vf = kc.cpu().view(-1, G * d), vc.cpu().view(-1, G * dv)
            for t, slot in enumerate(slots.tolist()):
                if slot >= 0:
                    torch.testing.assert_close(kf[slot].double(), want[t], **tol_of(dtype))
                    assert torch.equal(vf[slot], v[t])
            rest = [s for s in range(32) if s not in slots.tolist()]
            assert (kf[rest] == 5.0).all() and (vf[rest] == 5.0).all()   # the row without a slot wrote nowhere
        if lin:
            torch.testing.assert_close(lq.cpu().double(), turned(rq, R, rd, rf), **exact)
            torch.testing.assert_close(lk.cpu().double(), 0.37 * turned(rk, R, rd, rf), **exact)
    check(True, True)
    check(True, False)
    if not normed:
        check(False, True)


# ------------------------------------------------------------------ attention with a learned sink
@pytest.mark.parametrize("H,G,d,dv,page", [(4, 2, 16, 12, 16), (3, 1, 7, 5, 8), (6, 6, 8, 24, 16), (8, 2, 64, 32, 16), (6, 2, 20, 40, 32),
                                           (16, 1, 24, 72, 16)])
@pytest.mark.parametrize("mode", ["prompt", "decode", "pairs", "portions"])
@pytest.mark.parametrize("dtype", BOTH)
def test_attention_with_a_learned_sink_per_head(H, G, d, dv, page, mode, dtype):
    """Keys far away, on both sides of a page border and of a 32-key tile, the query's own key, the sequence's first key;
    sinks of every size, one so large that it takes nearly everything and one so small that it takes nothing; each head
    must use its own."""
    n = 300
    last = n - 1
    spikes = [(last, 2, 0), (last - 1, page - 1, H - 1), (last - 2, page, 0), (last - 3, 31, H - 1), (last - 4, 32, 0),
              (last - 5, last - 5, H - 1), (100, 0, 0), (129, 127, H - 1), (128, 128, 0), (40, 39, H - 1), (last - 45, 0, H - 1)]
    q, k, v = attention_case(H, G, d, dv, n, spikes, seed=H * 1000 + d)
    sink = torch.linspace(-2.0, 9.0, H)
    sink[H // 2] = 40.0
    if H > 3:
        sink[1] = -200.0
    kc, vc, table = paged(k.reshape(n, -1), v.reshape(n, -1), page, dtype, seed=d)
    kk = torch.stack([kc.cpu().double()[table[t // page], t % page].view(G, d) for t in range(n)])
    vv = torch.stack([vc.cpu().double()[table[t // page], t % page].view(G, dv) for t in range(n)])
    scale = 0.3
    want = oracle.causal_attention(q.double(), kk, vv, scale, sink.double()).reshape(n, H * dv)
    for wrong in (None, 0 * sink.double(), sink.double().roll(1)):         # no sink, a sink of 0, the neighbour's: all show
        if H > 1:
            assert (oracle.causal_attention(q[:9].double(), kk, vv, scale, wrong).reshape(9, H * dv) - want[:9]).abs().max() > 0.1
    seqs, rows = steps_of(mode, n, table)
    qd = q[rows].reshape(len(rows), H * d).float().contiguous().to(DEV)
    wide = torch.full((len(rows), H * dv + 9), 3.0, dtype=dtype, device=DEV)
    ops().capped_attention(wide[:, 5:5 + H * dv], qd, kc, vc, None, ragged(seqs), H, G, d, dv, scale, sink=sink.to(DEV))
    tol = dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=2e-2)
    torch.testing.assert_close(wide[:, 5:5 + H * dv].cpu().double(), want[rows], **tol)
    assert (wide[:, :5] == 3.0).all() and (wide[:, 5 + H * dv:] == 3.0).all()


@pytest.mark.parametrize("dtype", BOTH)
def test_a_learned_sink_where_workgroups_share_the_keys(dtype):
    """Decode steps of few sequences with long contexts and many query heads per key: the join launch takes each head's
    sink once."""
    n, page, H, d, dv = 1500, 16, 16, 24, 40
    rows = [n - 1, 1201, 700]
    q, k, v = attention_case(H, 1, d, dv, n, [(n - 1, 3, 0), (1201, 650, H - 1), (700, 699, 5)], seed=7)
    sink = torch.linspace(2.0, 12.0, H)
    kc, vc, table = paged(k.reshape(n, d), v.reshape(n, dv), page, dtype, seed=5)
    kk = torch.stack([kc.cpu().double()[table[t // page], t % page].view(1, d) for t in range(n)])
    vv = torch.stack([vc.cpu().double()[table[t // page], t % page].view(1, dv) for t in range(n)])
    want = torch.stack([oracle.causal_attention(q[t:t + 1].double(), kk, vv, 0.9, sink.double(), first_position=t)[0] for t in rows])
    from splitwise_amd import _C_mixers
    assert _C_mixers.load_library().swm_masked_attention_workspace_floats(3, 3, 1, H, 1, dv, page, len(table), 0, 0) > 0
    out = torch.empty(3, H * dv, dtype=dtype, device=DEV)
    ops().capped_attention(out, q[rows].reshape(3, H * d).contiguous().to(DEV), kc, vc, None,
                           ragged([(t, 1, 0, table) for t in rows]), H, 1, d, dv, 0.9, sink=sink.to(DEV))
    tol = dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=2e-2)
    torch.testing.assert_close(out.cpu().double(), want.reshape(3, H * dv), **tol)


@pytest.mark.parametrize("mode", ["prompt", "decode", "pairs", "portions"])
@pytest.mark.parametrize("H,G,d,dv,dims,page,whole", [(4, 2, 16, 12, 10, 16, True), (6, 2, 20, 40, 16, 8, False), (3, 3, 9, 6, 4, 16, True)])
def test_rotary_attention_layer(H, G, d, dv, dims, page, whole, mode):
    """From the projections to the heads, fp32, with scores so peaked that single far keys carry the output (asserted)."""
    from splitwise_amd.model_executor.layers.attention import RotaryPagedAttention
    g = torch.Generator().manual_seed(H + d)
    n, eps = 300, 1e-5
    sizes = [H * d, G * d, G * dv]
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": 1.1, "rot": {"dims": dims, "base": 200.0, "scaling": vu.scaling()}}
    h = torch.randn(n, sum(sizes), generator=g)                          # "projections" that pick columns of the input
    eye = torch.eye(sum(sizes)).split(sizes)
    w = dict(zip(("q", "k", "v"), eye), o=torch.eye(H * dv))
    w["q.norm"], w["k.norm"] = torch.randn(H * d, generator=g) * 0.3 + 1.0, torch.randn(G * d, generator=g) * 0.3 + 1.0
    w["sink"] = torch.randn(H, generator=g) * 2 + 2

    def plain(x):
        args = (x.double(), {k: v.double() for k, v in w.items()}, m)
        return oracle.normed_attention(*args, eps) if whole else oracle.attention_mixer(*args)
    want = plain(h)
    freqs = torch.tensor(oracle.rotary_frequencies(m["rot"]), dtype=torch.float32)
    layer = RotaryPagedAttention(H, G, d, dv, 1.1, freqs, whole_norm_eps=eps if whole else None, sink=not whole)
    for t, name in ((layer.q_norm, "q.norm"), (layer.k_norm, "k.norm"), (layer.sink, "sink")):
        if t is not None:
            t.data.copy_(w[name])
    layer = layer.to(DEV)
    pages = -(-n // page)
    table = list(range(pages + 3))
    random.Random(d).shuffle(table)
    table = table[:pages]
    kc, vc = (torch.full((pages + 3, page, G * s), float("nan"), device=DEV) for s in (d, dv))
    slot_of = torch.tensor([table[t // page] * page + t % page for t in range(n)])

    def run(batch, rows):
        q, k, v = h[rows].to(DEV).split(sizes, 1)
        md = SimpleNamespace(ragged=batch, slot_mapping=slot_of[rows].to(DEV))
        return layer(q, k, v, torch.tensor(rows, device=DEV), kc, vc, md).cpu().double()
    torch.testing.assert_close(run(ragged([(0, n, 0, table)]), list(range(n))), want, atol=2e-4, rtol=2e-4)     # fills the cache
    seqs, rows = steps_of(mode, n, table)
    torch.testing.assert_close(run(ragged(seqs), rows), want[rows], atol=2e-4, rtol=2e-4)
    # far keys carry rows: without the first half of the sequence, late rows come out otherwise by far
    late = plain(torch.cat([torch.zeros(150, sum(sizes)), h[150:]]))
    assert ((late - want)[200:].abs().amax(-1) > 0.2).float().mean() > 0.5


# ------------------------------------------------------------------ retention
@pytest.mark.parametrize("H,d,dv,decay", [(3, 8, 12, (0.9, 0.98, 0.75)), (2, 5, 7, (1.0, 0.999)), (1, 40, 70, (0.01,)), (2, 33, 256, (0.95, 0.99)),
                                          (4, 64, 64, (0.97, 0.9, 0.5, 0.9995)), (1, 256, 40, (0.99,))])
@pytest.mark.parametrize("cuts", [[400], [2] * 200, [1] * 30 + [33, 2, 31, 32, 64, 208], [300, 2, 1, 97]])
@pytest.mark.parametrize("dtype", BOTH)
def test_retention_in_every_cut(H, d, dv, decay, cuts, dtype):
    """A sequence in portions beside another in one piece, in slots that a longer sequence used before; runs long enough to
    be cut into segments; decays from 0.01 to 1."""
    g = torch.Generator().manual_seed(H * 10 + d)
    n = 400
    assert sum(cuts) == n
    q, k = torch.randn(n, H, d, generator=g), torch.randn(n, H, d, generator=g) * d ** -0.5
    v = torch.randn(n, H, dv, generator=g).to(dtype)
    want, S = oracle.retention(q.double(), k.double(), v.double(), list(decay))
    state = torch.randn(3, H, d, dv, generator=g).to(DEV) * 50           # what earlier owners left behind
    lam = torch.tensor(decay, device=DEV)
    got, at = [], 0
    for i, size in enumerate(cuts):
        beside = i == len(cuts) - 1                                      # the whole sequence again, from the start, in slot 1
        part = slice(at, at + size)
        pick = lambda x: torch.cat([x, x[part]] if beside else [x[part]]).flatten(1).contiguous().to(DEV)      # noqa: E731
        wide = torch.cat([pick(v), pick(v)], 1)
        batch = ragged(([(0, n, 1, [])] if beside else []) + [(at, size, 2, [])])
        out = torch.full((wide.shape[0], H * dv), float("nan"), device=DEV)
        ops().retention(out, pick(q), pick(k), wide[:, H * dv:], lam, state, batch, H, d, dv)
        if beside:
            torch.testing.assert_close(out[:n].cpu().double().view(n, H, dv), want, atol=2e-4, rtol=2e-4)
        got.append(out[-size:].cpu().double().view(size, H, dv))
        at += size
    scale = want.abs().max()
    assert (torch.cat(got) - want).abs().max() < 3e-6 * scale * max(1.0, d ** 0.5)
    torch.testing.assert_close(state[1:].cpu().double(), torch.stack([S, S]), atol=2e-4 * float(S.abs().max()), rtol=2e-4)


@pytest.mark.parametrize("dtype", BOTH)
def test_retention_remembers_one_far_token(dtype):
    """One token's key and value tower over silence: 250 tokens later what is left is exactly its decayed share."""
    H, d, dv, n = 2, 8, 6, 300
    q, k, v = torch.zeros(n, H, d), torch.zeros(n, H, d), torch.zeros(n, H, dv)
    q[:, :, 0], k[40, :, 0], v[40] = 1.0, 3.0, 2.0
    decay = [0.99, 0.999]
    state = torch.full((1, H, d, dv), 9.0, device=DEV)
    out = torch.empty(n, H * dv, device=DEV)
    ops().retention(out, q.flatten(1).to(DEV), k.flatten(1).to(DEV), v.flatten(1).to(dtype).to(DEV), torch.tensor(decay, device=DEV), state,
                    ragged([(0, n, 0, [])]), H, d, dv)
    o = out.cpu().view(n, H, dv)
    assert (o[:40] == 0).all()
    for t in (40, 41, 71, 72, 168, 290):
        for a in range(H):
            torch.testing.assert_close(o[t, a], torch.full((dv,), 6.0 * decay[a] ** (t - 40)), atol=1e-6, rtol=2e-4)


@pytest.mark.parametrize("dtype", BOTH)
def test_retention_mixer_alone(dtype):
    """Rotation, key scale, recurrence, head norm and gate together, in portions."""
    from splitwise_amd.model_executor.layers.recurrent import RetentionMixer
    H, d, dv, n, eps = 3, 12, 10, 90, 1e-5
    g = torch.Generator().manual_seed(4)
    m = {"heads": H, "dim": d, "vdim": dv, "rot": {"dims": 8, "base": 40.0}, "decay": [0.9, 0.99, 0.6]}
    sizes = [H * d, H * d, H * dv, H * dv]
    h = torch.randn(n, sum(sizes), generator=g).to(dtype)
    h[5] *= 1e-3
    w = dict(zip(("q", "k", "v", "g"), torch.eye(sum(sizes), dtype=F64).split(sizes)), o=torch.eye(H * dv, dtype=F64))
    want = oracle.retention_mixer(h.double(), w, m, eps)
    mixer = RetentionMixer(H, d, dv, m["decay"], torch.tensor(oracle.rotary_frequencies(m["rot"])), eps).to(DEV)
    for cuts in ([90], [1] * 20 + [2, 33, 35]):
        state = torch.full((2, *mixer.state_shapes()[0]), float("nan"), device=DEV)
        got, at = [], 0
        for size in cuts:
            q, k, v, gate = h[at:at + size].to(DEV).split(sizes, 1)
            md = SimpleNamespace(ragged=ragged([(at, size, 1, [])]))
            got.append(mixer(q, k, v, gate, torch.arange(at, at + size, device=DEV), state, md).cpu().double())
            at += size
        torch.testing.assert_close(torch.cat(got), want, **(dict(atol=1e-4, rtol=1e-4) if dtype == torch.float32 else tol_of(dtype)))


# ------------------------------------------------------------------ router and experts
@pytest.mark.parametrize("dtype,width,ff,experts,top,shared", [
    (torch.float32, 48, 24, 5, 2, 20), (torch.bfloat16, 48, 24, 5, 2, None), (torch.bfloat16, 64, 96, 8, 1, 48),
    (torch.float32, 22, 9, 7, 3, 11), (torch.bfloat16, 22, 9, 7, 7, 5), (torch.bfloat16, 128, 32, 4, 4, 64), (torch.float32, 40, 17, 3, 1, None),
    (torch.float32, 32, 16, 256, 8, 8)])
def test_experts_weighed_on_their_input(dtype, width, ff, experts, top, shared):
    from splitwise_amd.model_executor.layers.moe import GroupRoutedExperts
    g = torch.Generator().manual_seed(width + ff)
    rows = 77
    w = {}
    for e, size in [(f"e{e}", ff) for e in range(experts)] + ([("shared", shared)] if shared else []):
        w[e + ".gate"], w[e + ".up"] = ((torch.randn(size, width, generator=g) * 2 * width ** -0.5).to(dtype) for _ in range(2))
        w[e + ".down"] = (torch.randn(width, size, generator=g) * 2 * size ** -0.5).to(dtype)
    w["router"] = torch.randn(experts, width, generator=g).bfloat16().to(dtype) * 0.2
    h = torch.randn(rows, width, generator=g).to(dtype)
    layer = GroupRoutedExperts(width, experts, top, ff, shared, 1, 1, 1.0, dtype, None, score="sigmoid", normalize=False,
                               activation="clamped_glu", glu_alpha=1.0, glu_shift=0.0, router_dtype=dtype, weigh_input=True)
    layer.load_named(w)
    layer = layer.to(DEV)
    own, got = layer(h.to(DEV))
    wd = {k: v.double() for k, v in w.items()}
    mlp = {"router": {"top": top}}
    want = oracle.moe_ff(h.double(), wd, mlp)
    bound = 2e-5 if dtype == torch.float32 else 2e-2
    assert got.dtype == torch.float32 and (got.cpu().double() - want).abs().max() < bound * want.abs().max()
    chosen, weights = oracle.route(h.double(), wd["router"], top)
    behind = torch.stack([sum(p * oracle.gated_ff(h[t].double(), wd[f"e{e}.gate"], wd[f"e{e}.up"], wd[f"e{e}.down"], oracle.silu)
                              for e, p in zip(chosen[t].tolist(), weights[t])) for t in range(rows)])
    assert (behind - want).abs().max() > 0.05 * want.abs().max()         # a weight on the output would show
    if shared is None:
        assert own is None
    else:
        ws = oracle.gated_ff(h.double(), wd["shared.gate"], wd["shared.up"], wd["shared.down"], oracle.silu)
        assert (own.cpu().double() - ws).abs().max() < bound * ws.abs().max()


# --------------------------------------------------------------- whole models through the engine
FP32_TOL = 2e-4


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name in vu.MODELS:
        cfg, sd, reqs = vu.load(name)
        path = vu.write_model(str(tmp_path_factory.mktemp("vufasun_" + name)), cfg, sd)
        out[name] = SimpleNamespace(cfg=cfg, sd=sd, path=path, reqs=reqs,
                                    want={rid: oracle.logits(cfg, sd, toks, dtype=F64) for rid, toks in reqs.items()})
    return out


@pytest.fixture(scope="module")
def engines(models):
    cache = {}

    def get(name, dtype, **kw):
        key = (name, dtype, tuple(sorted(kw.items())))
        if key not in cache:
            cache[key] = vu.make_engine(models[name].path, dtype, **kw)
        return cache[key]
    return get


@pytest.mark.parametrize("name", sorted(vu.MODELS))
def test_streams_after_every_layer_run(models, engines, name):
    m = models[name]
    engine = engines(name, "float32")
    model = engine.model_executor.driver_worker.model_runner.model
    toks = m.reqs["r4"]
    _, want = oracle.logits(m.cfg, m.sd, toks, dtype=F64, keep_streams=True)
    model.keep_residuals = []
    try:
        vu.Replayer(engine, {"r4": toks}).run_alone("r4", [len(toks)])
        got = [r.cpu().double() for r in model.keep_residuals]
    finally:
        model.keep_residuals = None
    assert len(got) == len(want) == len(oracle.layer_order(m.cfg))
    for i, (a, b) in enumerate(zip(got, want)):
        assert (a - b).abs().max() < 1e-4 * b.abs().max(), f"run {i}"


@pytest.mark.parametrize("name", sorted(vu.MODELS))
def test_whole_prompts_match_the_plain_statement(models, engines, name):
    m = models[name]
    for rid, toks in m.reqs.items():
        got = vu.Replayer(engines(name, "float32"), {rid: toks}).run_alone(rid, [len(toks)])
        assert vu.row_error(got, m.want[rid]) < FP32_TOL, rid


@pytest.mark.parametrize("name", sorted(vu.MODELS))
def test_decoding_token_by_token(models, engines, name):
    """Most of a prompt at once and then 45 (and 100) tokens one by one, and a sequence fed one token at a time from its
    very first."""
    m = models[name]
    for rid, first in (("r0", 25), ("r6", 50)):
        toks = m.reqs[rid]
        got = vu.Replayer(engines(name, "float32"), {rid: toks}).run_alone(rid, [first] + [1] * (len(toks) - first))
        assert vu.row_error(got, m.want[rid]) < FP32_TOL
    toks = m.reqs["r2"]
    got = vu.Replayer(engines(name, "float32"), {"r2": toks}).run_alone("r2", [1] * len(toks))
    assert vu.row_error(got, m.want["r2"]) < FP32_TOL


@pytest.mark.parametrize("name", sorted(vu.MODELS))
@pytest.mark.parametrize("portions", [[2] * 35, [3, 2, 16, 1, 2, 7, 17, 2, 2, 18], [15, 1, 16, 17, 2, 19], [33, 31, 2, 4]])
def test_portions_of_prompts(models, engines, name, portions):
    m = models[name]
    toks = m.reqs["r0"]
    assert sum(portions) == len(toks)
    got = vu.Replayer(engines(name, "float32"), {"r0": toks}).run_alone("r0", portions)
    assert vu.row_error(got, m.want["r0"]) < FP32_TOL


@pytest.mark.parametrize("name,dtype,tol", [(n, "float32", FP32_TOL) for n in sorted(vu.MODELS)] + [("e", "bfloat16", 0.08)])
def test_mixed_batches_reuse_pages_and_slots(models, engines, name, dtype, tol):
    """Six unequal requests over three places and a pool of 9 pages: portions beside single tokens, requests that sit out
    steps, pages and state slots handed on as requests end.  Every request must come out as it does alone."""
    m = models[name]
    reqs = {r: t for r, t in m.reqs.items() if r != "r6"}
    engine = engines(name, dtype, max_tokens=144, max_requests=3)
    rp = vu.Replayer(engine, reqs)
    free_before = engine.scheduler.block_manager.get_num_free_gpu_blocks()
    steps = [{"r0": 3, "r2": 16}, {"r0": 16, "r2": 1, "r3": 1}, {"r0": 2, "r1": 29, "r2": 1}, {"r0": 17, "r1": 2},
             {"r0": 30, "r1": 1}, {"r1": 9, "r0": 1}, {"r0": 1, "r4": 20}]
    for step in steps:
        rp.step(step)
    rnd = random.Random(7)
    pending = ["r5"]
    while any(rp.at[r] < len(reqs[r]) for r in reqs):
        live = [r for r in rp.live if rp.at[r] < len(reqs[r])]
        while pending and len(live) < 3:
            nxt = pending[0]
            need = -(-len(reqs[nxt]) // 16)
            held = sum(-(-len(reqs[r]) // 16) for r in live)
            if held + need > 9:
                break
            live.append(pending.pop(0))
        step = {}
        for r in live:
            left = len(reqs[r]) - rp.at[r]
            step[r] = min(left, rnd.choice([1, 1, 2, 3, 16, 21]))
        if rnd.random() < 0.3 and len(step) > 1:
            step.pop(rnd.choice(sorted(step)))                  # somebody sits this step out
        rp.step(step)
    for rid in reqs:
        assert vu.row_error(rp.result(rid), m.want[rid]) < tol, rid
    assert engine.scheduler.block_manager.get_num_free_gpu_blocks() == free_before
    assert engine.scheduler.state_slots.num_free() == 3


def test_bfloat16_is_close_and_does_not_depend_on_the_cut(models, engines):
    """On a model whose routers choose all their experts, so that nothing discrete can fall the other way."""
    m = models["e"]
    toks = m.reqs["r0"]
    whole = vu.Replayer(engines("e", "bfloat16"), {"r0": toks}).run_alone("r0", [len(toks)])
    cut = vu.Replayer(engines("e", "bfloat16"), {"r0": toks}).run_alone("r0", [2, 3, 16, 1, 1, 30, 17])
    assert vu.row_error(whole, m.want["r0"]) < 0.08
    assert vu.row_error(cut, m.want["r0"]) < 0.08
    assert vu.row_error(cut, whole) < 0.05


@pytest.mark.parametrize("name", sorted(vu.MODELS))
def test_greedy_generation_through_the_entry_point(models, name):
    """``LLM.generate`` with the scheduler's own policy: a token budget of 16 cuts the prompts into portions that run
    beside other requests' decoded tokens.  Every generated token must be (within rounding) the arg-max of the plain
    statement's logits for the text before it, with that row's log-probability."""
    from splitwise_amd import LLM, SamplingParams
    m = models[name]
    llm = LLM(model=m.path, dtype="float32", block_size=16, max_model_len=128, max_num_seqs=3,
              max_num_batched_tokens=16, num_gpu_blocks_override=20, swap_space=0, enforce_eager=True)
    prompts = [m.reqs["r1"], m.reqs["r2"], m.reqs["r3"], m.reqs["r4"][:20]]
    outs = llm.generate(prompt_token_ids=prompts, sampling_params=SamplingParams(temperature=0.0, max_tokens=12, logprobs=1,
                                                                                 ignore_eos=True))
    assert len(outs) == len(prompts)
    for prompt, out in zip(prompts, outs):
        new = out.outputs[0].token_ids
        assert len(new) == 12
        full = oracle.logits(m.cfg, m.sd, list(prompt) + list(new), dtype=F64)
        for k, tok in enumerate(new):
            row = full[len(prompt) + k - 1]
            assert row[tok] >= row.max() - 1e-3 * (row.max() - row.min()), (k, tok, int(row.argmax()))
            lp = out.outputs[0].logprobs[k][tok]
            assert abs(float(getattr(lp, "logprob", lp)) - float(torch.log_softmax(row, -1)[tok])) < 5e-3
    sched = llm.llm_engine.scheduler
    assert sched.state_slots.num_free() == 3 and not sched.running and not sched.waiting


def test_trace_run_replays_a_schedule(models, tmp_path):
    """``bin/trace_run`` as a user starts it: steps on standard input, ``done <step>`` after each, logits files in the
    order of the entries; requests that sit out a step, end, and hand their pages on."""
    import json
    import os
    import subprocess
    import numpy as np
    m = models["b"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b, c = m.reqs["r1"], m.reqs["r2"], m.reqs["r4"]
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:7], "want": [0, 6]}, {"id": "b", "tokens": b[:2], "want": []}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [15]}, {"id": "a", "tokens": a[7:8], "want": [0]}], "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": a[8:], "want": [len(a) - 9]}, {"id": "c", "tokens": c, "want": [0, len(c) - 1]}],
         "end": ["a", "c"]},
        {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [len(b) - 1]}], "end": ["b"]},        # the name comes back
    ]
    out = tmp_path / "out"
    proc = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", m.path, "--dtype", "float32", "--out", str(out),
                           "--max-tokens", "128", "--max-requests", "2"],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    vocab = m.cfg["vocab"]
    want = {0: [m.want["r1"][0], m.want["r1"][6]], 1: [m.want["r2"][17], m.want["r1"][7]],
            2: [m.want["r1"][len(a) - 1], m.want["r4"][0], m.want["r4"][len(c) - 1]], 3: [m.want["r2"][len(b) - 1]]}
    for step, rows in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(-1, vocab))
        assert got.shape[0] == len(rows)
        assert vu.row_error(got, torch.stack(rows)) < FP32_TOL, step
