"""Each Ralepel mechanism alone: the engine's ops and modules (in portions,
through scattered and previously used pages) against the float64 oracle in
tests/oracle_ralepel.py, and, marked gpu, the HIP kernels against the
reference ops."""

import pytest
import torch

import oracle_ralepel as O
from production_stack_amd import ops
from production_stack_amd.engine.models import registry
from production_stack_amd.engine.models.llama import BatchMeta
from production_stack_amd.ops import reference as R
from ralepel_util import (TOL, attn, dense, latent, make_cfg, make_weights,
                          moe, rel_err, save_checkpoint)

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = ["float32", "bfloat16"]
TD = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64

pytestmark = pytest.mark.filterwarnings("ignore::UserWarning")


def rnd(shape, seed, scale=1.0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def relerr(got, want):
    got, want = got.detach().cpu().to(F64), want.detach().cpu().to(F64)
    return float((got - want).norm() / want.norm().clamp_min(1e-12))


def load_model(cfg, W, dtype, device):
    """A model read through the registry, as the engine reads it."""
    import tempfile

    with tempfile.TemporaryDirectory() as d:
        save_checkpoint(d, cfg, W)
        model = registry.build_model(registry.config_from_dir(d), dtype)
        registry.load_weights(model, d)
    return model.to(device)


class Harness:
    """Mixers over one paged cache full of stale rows and scattered pages."""

    def __init__(self, mx, device, dtype, n_seqs=3, max_len=320, bs=16):
        self.mixer, self.device, self.bs = mx, device, bs
        per = (max_len + bs - 1) // bs
        g = torch.Generator().manual_seed(99)
        nb = per * n_seqs + 5
        self.tables = torch.randperm(nb, generator=g)[:per * n_seqs].view(
            n_seqs, per).to(torch.int32)
        kind, heads, d = mx.cache_shape()
        rows = torch.randn(nb, heads, bs, d, generator=g).to(dtype).to(device)
        self.cache = rows
        if kind == "keyval":
            self.cache = (rows, torch.rand(nb, heads, bs,
                                           generator=g).to(device))

    def run(self, parts, more=()):
        """parts: [(sequence, first position, inputs [n, width])], longer
        portions before single tokens; returns one output per part (for each
        of `more`, mixers on the same cache, as well)."""
        bs, dev = self.bs, self.device
        h = torch.cat([p for _, _, p in parts]).to(dev)
        pos, tseq, slots, rows, r0 = [], [], [], [], 0
        for i, (s, p0, p) in enumerate(parts):
            for pp in range(p0, p0 + p.shape[0]):
                pos.append(pp)
                tseq.append(i)
                slots.append(int(self.tables[s][pp // bs]) * bs + pp % bs)
            rows.append([r0, p.shape[0], p0, s])
            r0 += p.shape[0]
        rows = torch.tensor(rows, dtype=torch.int32)
        meta = BatchMeta(
            positions=torch.tensor(pos, dtype=torch.int32, device=dev),
            slot_mapping=torch.tensor(slots, dtype=torch.long, device=dev),
            num_prefill_tokens=sum(
                p.shape[0] for _, _, p in parts if p.shape[0] > 1),
            prefill_token_seq=None, prefill_token_pos=None,
            prefill_block_tables=None, num_decode_seqs=0,
            decode_seq_lens=None, decode_block_tables=None,
            block_tables=torch.stack(
                [self.tables[s] for s, _, _ in parts]).to(dev),
            token_seq=torch.tensor(tseq, dtype=torch.int32, device=dev),
            seq_rows=rows.to(dev), seq_rows_host=rows.tolist())
        shared: dict = {}
        sizes = [p.shape[0] for _, _, p in parts]
        outs = [list(mx(h, meta, self.cache, shared).split(sizes))
                for mx in (self.mixer, *more)]
        return outs if more else outs[0]


# ---------------------------------------------------------------------------
# attention over keys that are their values
# ---------------------------------------------------------------------------
def test_slopes_follow_the_head_count():
    for H in (1, 3, 6, 8):
        cfg = make_cfg([(attn(H, 1, 8), None)])
        mx = load_model(cfg, make_weights(cfg), "float32",
                        "cpu").layers[0].mixer
        assert relerr(mx.slopes(torch.device("cpu")), O.slopes(H)) < 1e-7


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(5, 4, 2, 24), (3, 6, 6, 7), (1, 1, 1, 1),
                                   (9, 8, 1, 256), (40, 33, 3, 128),
                                   (2, 3, 1, 600)])
def test_keyval_prep(device, dtype, shape):
    """Queries over their root mean square; keys untouched in the cache, one
    over their root mean square beside them; padding rows (slot -1 on a GPU)
    store nothing."""
    T, H, G, D = shape
    bs, nb = 5, 12
    proj = rnd((T, (H + G) * D + 8), 1, 2.0).to(TD[dtype])
    slots = torch.randperm(nb * bs, generator=torch.Generator(
        ).manual_seed(3))[:T]
    on = torch.ones(T, dtype=torch.bool)
    if device == "cuda" and T > 2:
        slots[1], on[1] = -1, False
    rows = torch.full((nb, G, bs, D), 7.0).to(TD[dtype]).to(device)
    scale = torch.full((nb, G, bs), 9.0, device=device)
    p = proj.clone().to(device)
    ops.keyval_prep(p[:, :H * D], p[:, H * D:(H + G) * D], 1e-3, rows, scale,
                    slots.to(device), H)
    q = O.unit_rms(proj[:, :H * D].to(F64).view(T, H, D), 1e-3)
    assert relerr(p[:, :H * D].cpu().view(T, H, D), q) < (
        1e-6 if dtype == "float32" else 4e-3)
    assert torch.equal(p[:, H * D:].cpu(), proj[:, H * D:])
    k = proj[:, H * D:(H + G) * D].view(T, G, D)
    inv = 1.0 / torch.sqrt(k.to(F64).pow(2).mean(-1) + 1e-3)
    kept = torch.full((nb * bs,), True)
    for t in range(T):
        if not on[t]:
            continue
        b, o = int(slots[t]) // bs, int(slots[t]) % bs
        kept[int(slots[t])] = False
        assert torch.equal(rows[b, :, o].cpu(), k[t])
        assert relerr(scale[b, :, o], inv[t]) < 1e-6
    flat = rows.cpu().transpose(1, 2).reshape(nb * bs, G, D)
    assert bool((flat[kept] == 7.0).all())
    assert bool((scale.cpu().transpose(1, 2).reshape(nb * bs, G)[kept]
                 == 9.0).all())


SHAPES = [
    # heads, kv heads, dim, window, scale
    (4, 2, 24, 20, 0.3),
    (6, 2, 16, 7, 0.4),        # three heads on one key
    (3, 3, 20, 33, 0.3),       # rows of no whole vectors
    (1, 1, 8, 1, 1.0),         # a window of the token itself
    (5, 1, 40, 500, 0.2),      # longer than the sequence
    (18, 1, 136, 0, 0.1),      # no window; more heads than a narrow tile
]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("sizes", [[70], [1] * 70, [2] * 35,
                                   [31, 2, 1, 1, 16, 19], [64, 6]])
def test_attention_in_portions(device, dtype, shape, sizes):
    layer, width = attn(*shape), 48
    cfg = make_cfg([(layer, None)], width=width)
    W = make_weights(cfg, seed=31)
    h = rnd((70, width), 32, 1.0, torch.bfloat16)
    want = O.attention(W, "l0.mix.", layer["mixer"], h.to(F64), 1e-5)
    mx = load_model(cfg, W, dtype, device).layers[0].mixer
    hs = Harness(mx, device, TD[dtype])
    outs, at = [], 0
    for n in sizes:
        outs += hs.run([(1, at, h[at:at + n].to(TD[dtype]))])
        at += n
    assert rel_err(mx.project(torch.cat(outs)), want) < TOL[dtype]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_ragged_batch(device, dtype):
    """Three sequences of unequal length in shared steps, portions beside
    single tokens, against each alone."""
    layer, width = attn(6, 2, 32, 40, 0.25), 48
    cfg = make_cfg([(layer, None)], width=width)
    W = make_weights(cfg, seed=16)
    mx = load_model(cfg, W, dtype, device).layers[0].mixer
    hs = Harness(mx, device, TD[dtype])
    hh = [rnd((n, width), 20 + i, 1.0, torch.bfloat16)
          for i, n in enumerate((300, 9, 151))]
    steps = [[(0, 200), (2, 80)], [(0, 60), (2, 70), (1, 1)],
             [(1, 2), (0, 1), (2, 1)], [(0, 39), (1, 5)], [(1, 1)]]
    at, outs = [0, 0, 0], [[], [], []]
    for step in steps:
        res = hs.run([(s, at[s], hh[s][at[s]:at[s] + n].to(TD[dtype]))
                      for s, n in step])
        for (s, n), o in zip(step, res):
            outs[s].append(o)
            at[s] += n
    assert at == [300, 9, 151]
    for s in range(3):
        want = O.attention(W, "l0.mix.", layer["mixer"], hh[s].to(F64), 1e-5)
        assert rel_err(mx.project(torch.cat(outs[s])), want) < TOL[dtype], s


def test_every_term_of_the_attention_shows():
    """The oracle itself: norms, distance penalty, sink, biases and window
    each move the result (so none of them can be left out unnoticed)."""
    layer = attn(4, 2, 24, 20, 0.3)
    W = make_weights(make_cfg([(layer, None)], width=48), seed=31)
    h = rnd((70, 48), 32).to(F64)
    m = layer["mixer"]
    base = O.attention(W, "l0.mix.", m, h, 1e-5)

    def moved(W2=None, m2=None, eps=1e-5):
        got = O.attention(W2 or W, "l0.mix.", m2 or m, h, eps)
        return rel_err(got, base)

    for name in ("q.b", "k.b", "o.b", "sink"):
        W2 = dict(W)
        W2["l0.mix." + name] = torch.zeros_like(W["l0.mix." + name])
        assert moved(W2) > 1e-2, name
    for size in (19, 21):
        assert moved(m2=dict(m, mask={"size": size})) > 1e-2
    assert moved(eps=1.0) > 1e-2
    keep, O.slopes = O.slopes, lambda H: torch.zeros(H, dtype=F64)
    try:
        assert moved() > 1e-2
    finally:
        O.slopes = keep


# ---------------------------------------------------------------------------
# latent attention
# ---------------------------------------------------------------------------
LATENT = [
    # heads, dim, rot_dim, vdim, kv_rank, scale, base
    (3, 12, 8, 20, 24, 0.25, 1000.0),
    (1, 8, 2, 8, 16, 0.5, 10.0),
    (5, 6, 10, 7, 18, 0.3, 1e4),
    (2, 24, 8, 40, 136, 0.2, 5e5),
    (8, 32, 16, 32, 64, 0.15, 20.0),
]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", LATENT)
@pytest.mark.parametrize("sizes", [[70], [1] * 70, [2] * 35,
                                   [31, 2, 1, 1, 16, 19]])
def test_latent_attention_on_shared_rows(device, dtype, shape, sizes):
    """A layer with a cache and two layers that read it (other head counts
    and widths, other up-projections), each against the oracle."""
    width = 48
    H, D, Rd, DV, L, sc, base = shape
    a = latent(*shape)
    b = latent(H + 1, D + 4, Rd, DV, L, sc, base, src=0)
    c = latent(H, D, Rd, DV + 8, L, sc * 0.5, base, src=0)
    cfg = make_cfg([(a, None), (b, None), (c, None)], width=width)
    W = make_weights(cfg, seed=31)
    h = rnd((70, width), 32, 1.0, torch.bfloat16)
    model = load_model(cfg, W, dtype, device)
    mxs = [layer.mixer for layer in model.layers]
    assert mxs[1].cache_shape() == ("layer", 0)
    hs = Harness(mxs[0], device, TD[dtype])
    outs, at = [[], [], []], 0
    for n in sizes:
        res = hs.run([(1, at, h[at:at + n].to(TD[dtype]))], mxs[1:])
        for o, r in zip(outs, res):
            o += r
        at += n
    rows = O.latent_rows(W, "l0.mix.", a["mixer"], h.to(F64), 1e-5)
    for i, layer in enumerate((a, b, c)):
        want = O.latent_attention(W, f"l{i}.mix.", layer["mixer"], h.to(F64),
                                  rows)
        got = torch.nn.functional.linear(torch.cat(outs[i]),
                                         mxs[i].out_weight)
        assert rel_err(got, want) < TOL[dtype], i


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_both_forms_of_latent_attention_agree(device, dtype):
    """The same ragged steps through the folded and the unfolded form, the
    sharing layer gathering its rows itself or taking the first layer's."""
    width = 48
    cfg = make_cfg([(latent(4, 16, 8, 24, 32, 0.25, 20.0), None),
                    (latent(5, 16, 8, 16, 32, 0.3, 20.0, src=0), None)],
                   width=width)
    W = make_weights(cfg, seed=17)
    mxs = [y.mixer for y in load_model(cfg, W, dtype, device).layers]
    h = rnd((150, width), 3, 1.0).to(TD[dtype])
    outs = []
    for ratios in ((0, 0), (1 << 20, 1 << 20), (0, 1 << 20)):
        for mx, r in zip(mxs, ratios):
            mx.EXPAND_RATIO = r
        hs = Harness(mxs[0], device, TD[dtype])
        got = [[], []]
        for parts in ([(0, 0, h[:60])],
                      [(0, 60, h[60:62]), (1, 0, h[:50])],
                      [(0, 62, h[62:])]):
            res = hs.run(parts, mxs[1:])
            for o, r in zip(got, res):
                o.append(r[0])
        outs.append([torch.cat(o) for o in got])
    for other in outs[1:]:
        for a, b in zip(outs[0], other):
            assert rel_err(a, b) < TOL[dtype]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rot,dims", [(8, 8), (12, 6), (10, 4), (4, 2)])
@pytest.mark.parametrize("fold", [True, False])
def test_half_split_pairs(device, dtype, rot, dims, fold):
    """Queries and cached rows turn by halves, at far positions too; entries
    past the turned ones pass."""
    T, H, D, L, bs = 6, 5, 7, 16, 4
    dt = TD[dtype]
    pos = torch.tensor([0, 1, 2, 77, 500, 999], dtype=torch.int32)
    q = rnd((T, H * (D + rot)), 1).to(dt)
    dkv = rnd((T, L + rot), 2).to(dt)
    w = rnd((L,), 3) + 1.0
    q_lat = rnd((H, T, L), 4).to(dt) if fold else None
    cache = torch.zeros((4, 1, bs, L + rot), dtype=dt, device=device)
    slots = torch.tensor([3, 0, 9, 15, 6, 1])
    cs = ops.rope_table(1000, dims, 100.0)
    rotspec = {"base": 100.0, "dims": dims}
    # the oracle turns row t by position t: a long sequence, then the picks
    wide = torch.zeros(1000, H + 1, rot, dtype=F64)
    wide[pos.long(), :H] = q.to(F64).view(T, H, D + rot)[..., D:]
    wide[pos.long(), H] = dkv.to(F64)[:, L:]
    turned = O.turn_halves(wide, rotspec)[pos.long()]
    qg = q.clone().to(device)
    got = ops.latent_prep(
        q_lat.to(device) if fold else None, qg, dkv.to(device),
        w.to(device), 1e-5, cs.to(device), pos.to(device), cache,
        slots.to(device), H, D, rot, dims, True)
    tol = 2e-6 if dtype == "float32" else 5e-3
    g = got.cpu().view(T, H, -1)
    assert relerr(g[..., -rot:], turned[:, :H]) < tol
    lead = q_lat.transpose(0, 1) if fold else q.view(T, H, D + rot)[..., :D]
    assert torch.equal(g[..., :-rot], lead)
    rows = cache.cpu().view(-1, L + rot)[slots]
    assert relerr(rows[:, L:], turned[:, H]) < tol
    assert relerr(rows[:, :L], O.rms_norm(dkv.to(F64)[:, :L], w, 1e-5)) < tol
    # without a latent the same queries come out and no row is written
    before = cache.clone()
    again = ops.latent_prep(
        q_lat.to(device) if fold else None, q.clone().to(device), None, None,
        1e-5, cs.to(device), pos.to(device), cache, slots.to(device), H, D,
        rot, dims, True)
    assert torch.equal(again.cpu(), got.cpu())
    assert torch.equal(cache, before)


# ---------------------------------------------------------------------------
# boundary, router, feed-forwards
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(3, 64), (5, 61), (300, 1100), (2, 8192),
                                   (2, 8200), (260, 2052), (1, 4)])
def test_boundary_with_and_without_a_next_norm(device, dtype, shape):
    """Rows of no whole vectors, wider than the registers hold, few and many
    rows; serving-dtype and fp32 sublayer outputs, row-strided."""
    T, W_ = shape
    dt = TD[dtype]
    x, wp, wn = rnd((T, W_), 1, 3.0), rnd((W_,), 2), rnd((W_,), 3)
    for ddt in {dt, torch.float32}:
        for pad in (0, 8):
            d = rnd((T, W_ + pad), 4, 2.0).to(ddt)[:, pad:]
            for nxt in (None, wn):
                xg = x.clone().to(device)
                h = ops.post_norm_add_norm32(
                    xg, d.to(device) if pad == 0 else torch.nn.functional.pad(
                        d.to(device), (pad, 0))[:, pad:], wp.to(device),
                    nxt.to(device) if nxt is not None else None, 1e-3, dt)
                want = x.to(F64) + O.rms_norm(d.to(F64), wp, 1e-3)
                assert relerr(xg, want) < 1e-6
                assert h.dtype == dt and h.data_ptr() != xg.data_ptr()
                if nxt is not None:
                    want = O.rms_norm(want, nxt, 1e-3)
                assert relerr(h, want) < (1e-6 if dtype == "float32"
                                          else 4e-3)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(7, 64, 5, 2), (1, 60, 3, 3), (40, 72, 1, 1),
                                   (9, 256, 70, 6), (3, 64, 300, 1)])
def test_biased_router(device, dtype, shape):
    """Choice and weights both see the bias; fp32 logits of the inputs as
    they are; logits so far apart that the plain softmax underflows still
    rank right."""
    T, W_, n, top = shape
    dt = TD[dtype]
    for gain in (1.0, 60.0):
        x = rnd((T, W_), 1, 1.0, torch.bfloat16)
        rw = rnd((n, W_), 2, gain * W_ ** -0.5, torch.bfloat16)
        b = rnd((n,), 3, 2.0 * gain)
        W = {"router": rw, "router.b": b}
        m = {"router": {"top": top}}
        want_w, want_e = O.route(W, "", m, x.to(F64))
        wts, sel, wm = ops.moe_route(
            x.to(dt).to(device), rw.to(dt).to(device), top, "softmax", True,
            bias=b.to(device))
        assert torch.equal(sel.cpu(), want_e)
        assert relerr(wts, want_w) < 1e-4
        assert relerr(wm.cpu().gather(1, want_e), want_w) < 1e-4
        if n > top:
            _, plain = O.route({"router": rw}, "", m, x.to(F64))
            assert not torch.equal(plain, want_e)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("small", [True, False])
@pytest.mark.parametrize("shape", [(24, 5, 2, 40), (8, 1, 1, 0),
                                   (20, 3, 3, 12), (16, 40, 1, 24),
                                   (40, 6, 4, 0)])
def test_routed_experts(device, dtype, small, shape):
    """Both dispatch forms, with and without a shared expert, experts nobody
    chose. A row whose choice is a close call is left out."""
    cfg = make_cfg([(attn(), moe(*shape))])
    W = make_weights(cfg, seed=8)
    layer = load_model(cfg, W, dtype, device).layers[0]
    m = cfg["layers"][0]["mlp"]
    for n in (1, 7, 150):
        h = rnd((n, 64), 40 + n, 1.0, torch.bfloat16)
        want = O.moe_ff(W, "l0.mlp.", m, h.to(F64))
        y = layer.feed_forward(h.to(TD[dtype]).to(device), small)
        assert y.dtype == torch.float32
        z = O.lin(W, "l0.mlp.router", h.to(F64)).sort(-1).values
        top, E = m["router"]["top"], m["router"]["experts"]
        sure = (z[:, E - top] - z[:, E - top - 1] > 1e-4 if top < E
                else torch.ones(n, dtype=torch.bool))
        assert int(sure.sum()) > n // 2
        assert rel_err(y.cpu()[sure], want[sure]) < TOL[dtype], n


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_dense_feed_forward(device, dtype):
    cfg = make_cfg([(attn(), dense(56))])
    W = make_weights(cfg, seed=3)
    layer = load_model(cfg, W, dtype, device).layers[0]
    h = rnd((23, 64), 5, 1.0, torch.bfloat16)
    y = layer.feed_forward(h.to(TD[dtype]).to(device), True)
    assert rel_err(y.float(), O.gated_ff(W, "l0.mlp.", h.to(F64))) \
        < TOL[dtype]


# ---------------------------------------------------------------------------
# kernels against the reference ops
# ---------------------------------------------------------------------------
def page_setup(lens, G, D, BS, seed):
    """Scattered pages of sequences of the given lengths, random rows and
    row factors."""
    S, per = len(lens), max(lens) // BS + 1
    g = torch.Generator().manual_seed(seed)
    tables = torch.randperm(S * per + 3, generator=g)[:S * per].view(
        S, per).int()
    rows = rnd((S * per + 3, G, BS, D), seed + 1, 1.0, torch.bfloat16)
    fac = torch.rand(S * per + 3, G, BS, generator=g) + 0.5
    return tables, rows, fac


def key_like(rows, tables, s, j, BS, q):
    """Makes row j of sequence s match q [H, D] (per KV head the mean of its
    query heads) strongly."""
    G, D = rows.shape[1], rows.shape[3]
    rows[tables[s, j // BS], :, j % BS] = (
        q.float().view(G, -1, D).mean(1) * 6).to(rows.dtype)


KERNEL_SHAPES = [
    # heads, kv heads, dim, window, sink, page, slopes, factors
    (8, 2, 128, 0, None, 16, True, True),
    (6, 2, 24, 50, "learned", 16, True, True),
    (3, 3, 64, 1, "zero", 16, True, True),
    (16, 1, 96, 129, "learned", 7, True, True),
    (20, 1, 40, 64, "learned", 32, True, False),
    (4, 4, 256, 200, None, 16, False, True),
    (32, 4, 8, 70, "learned", 16, True, True),
    (10, 2, 136, 65, "learned", 5, True, True),
    (64, 8, 72, 100, "learned", 16, True, True),
]


@pytest.mark.gpu
@pytest.mark.parametrize("shape", KERNEL_SHAPES)
@pytest.mark.parametrize("splits", [0, 1, 3, 16])
def test_keyval_token_kernel(shape, splits):
    """Single tokens: lengths around tile borders, shares with and without
    rows, a key that stands out just inside and outside the window, on a page
    border and at the start."""
    H, G, D, win, sink, BS, sl, fa = shape
    lens = [1, 2, 31, 32, 33, 200, 129, 5, 300]
    S = len(lens)
    tables, rows, fac = page_setup(lens, G, D, BS, H + D)
    q = rnd((S, H * D + 8), 2, 1.0, torch.bfloat16)[:, 8:]
    sv = rnd((H,), 5) if sink == "learned" else None
    slopes = O.slopes(H).float() * 0.2 if sl else None
    pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32)
    seq = torch.arange(S, dtype=torch.int32)
    for back in [None, 0, BS, max(win, 1) - 1, max(win, 1), 299]:
        c = rows.clone()
        if back is not None:
            for s, n in enumerate(lens):
                if n - 1 - back >= 0:
                    key_like(c, tables, s, n - 1 - back, BS, q[s])
        f = fac if fa else None
        want = R.talk_attention(
            q.reshape(S, H, D), c, c, tables, seq, pos, D ** -0.5, 0, win,
            bool(sink), None, 0, 0.0, sv, D, None, f, slopes).reshape(S, -1)
        cc = c.cuda()
        got = ops.talk_attention(
            q.cuda(), cc, cc, tables.cuda(), seq.cuda(), pos.cuda(),
            D ** -0.5, H, variant=9, splits=splits, window=win,
            sink=bool(sink), vdim=D,
            sink_vals=sv.cuda() if sv is not None else None,
            key_scale=f.cuda() if fa else None,
            slopes=slopes.cuda() if sl else None)
        err = (got.cpu().float() - want.float()).norm(dim=-1) / \
            want.float().norm(dim=-1)
        assert float(err.max()) < 1e-2, back


@pytest.mark.gpu
@pytest.mark.parametrize("shape", KERNEL_SHAPES + [
    (130, 1, 16, 40, "learned", 16, True, True)])
def test_keyval_prompt_kernel(shape):
    """Portions of 1 to 300 rows with and without history in one batch
    (workgroups whose rows belong to several sequences), a key that stands
    out around the window's edge of one row."""
    H, G, D, win, sink, BS, sl, fa = shape
    segs = [(0, 150), (130, 67), (5, 2), (64, 64), (0, 1), (99, 1), (0, 3)]
    lens = [a + n for a, n in segs]
    tables, rows, fac = page_setup(lens, G, D, BS, H + D)
    pos = torch.cat([torch.arange(a, a + n) for a, n in segs]).int()
    seq = torch.cat([torch.full((n,), i) for i, (_, n) in enumerate(segs)]
                    ).int()
    T = len(pos)
    q = rnd((T, H * D + 8), 2, 1.0, torch.bfloat16)[:, 8:]
    sv = rnd((H,), 5) if sink == "learned" else None
    slopes = O.slopes(H).float() * 0.2 if sl else None
    f = fac if fa else None
    probe = 140                 # row and position of the first sequence
    spots = [probe - max(win, 60) + 1, probe - max(win, 60), probe,
             probe - probe % BS, 0]
    for spot in [None] + [s for s in spots if s >= 0]:
        c = rows.clone()
        if spot is not None:
            key_like(c, tables, 0, spot, BS, q[probe])
        want = R.talk_attention(
            q.reshape(T, H, D), c, c, tables, seq, pos, D ** -0.5, 0, win,
            bool(sink), None, 0, 0.0, sv, D, None, f, slopes).reshape(T, -1)
        cc = c.cuda()
        kw = dict(window=win, sink=bool(sink), vdim=D,
                  sink_vals=sv.cuda() if sv is not None else None,
                  key_scale=f.cuda() if fa else None,
                  slopes=slopes.cuda() if sl else None)
        for variant in (8, 1):      # matrix cores, and the vector kernel
            got = ops.talk_attention(
                q.cuda(), cc, cc, tables.cuda(), seq.cuda(), pos.cuda(),
                D ** -0.5, H, variant=variant, **kw)
            err = (got.cpu().float() - want.float()).norm(dim=-1) / \
                want.float().norm(dim=-1)
            assert float(err.max()) < 1e-2, (spot, variant)


@pytest.mark.gpu
@pytest.mark.parametrize("shape", [(2, 1, 8, 0), (8, 4, 128, 500),
                                   (3, 3, 64, 0), (6, 2, 24, 40)])
def test_known_score_bound_changes_nothing(shape):
    """Unit queries and keys: with the bound given, keys beyond the reach of
    every slope of a group are passed over; the result is the same, with and
    without a window, at short and long distances."""
    H, G, D, win = shape
    lens, BS = [900, 1, 70, 333], 16
    S = len(lens)
    tables, rows, _ = page_setup(lens, G, D, BS, 7)
    fac = 1.0 / rows.float().pow(2).mean(-1).sqrt()
    slopes, sv = O.slopes(H).float(), rnd((H,), 3)
    scale = D ** -0.5
    for token in (True, False):
        if token:
            pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32)
            seq = torch.arange(S, dtype=torch.int32)
        else:
            pos = torch.cat([torch.arange(max(0, n - 150), n)
                             for n in lens]).int()
            seq = torch.cat([torch.full((min(n, 150),), i)
                             for i, n in enumerate(lens)]).int()
        T = len(pos)
        q = rnd((T, H, D), 2)
        q = (q / q.pow(2).mean(-1, keepdim=True).sqrt()).to(torch.bfloat16)
        want = R.talk_attention(
            q, rows, rows, tables, seq, pos, scale, 0, win, True, None, 0,
            0.0, sv, D, None, fac, slopes).reshape(T, -1)
        c = rows.cuda()
        outs = [ops.talk_attention(
            q.reshape(T, H * D).cuda(), c, c, tables.cuda(), seq.cuda(),
            pos.cuda(), scale, H, window=win, sink=True, sink_vals=sv.cuda(),
            vdim=D, variant=9 if token else 8, key_scale=fac.cuda(),
            slopes=slopes.cuda(), score_bound=b)
            for b in (0.0, 1.01 * scale * D)]
        for o in outs:
            err = (o.cpu().float() - want.float()).norm(dim=-1) / \
                want.float().norm(dim=-1)
            assert float(err.max()) < 1e-2, token
        # the rounding of a result may fall either way, no more than that
        assert relerr(*outs) < 1e-3


@pytest.mark.gpu
@pytest.mark.parametrize("variant", [1, 2, 4])
@pytest.mark.parametrize("shape", [(6, 2, 24, 20), (4, 1, 64, 0),
                                   (3, 3, 100, 33)])
def test_vector_kernels_take_factors_and_slopes(variant, shape):
    """float32: the plain, tiled and split-key kernels."""
    H, G, D, win = shape
    lens, BS = [1, 40, 33, 90], 16
    S = len(lens)
    tables, rows, fac = page_setup(lens, G, D, BS, 7)
    rows = rows.float()
    if variant == 4:
        pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32)
        seq = torch.arange(S, dtype=torch.int32)
    else:
        pos = torch.cat([torch.arange(n) for n in lens]).int()
        seq = torch.cat([torch.full((n,), i) for i, n in enumerate(lens)]
                        ).int()
    T = len(pos)
    q, sv = rnd((T, H * D), 2), rnd((H,), 3)
    slopes = O.slopes(H).float()
    want = R.talk_attention(
        q.view(T, H, D), rows, rows, tables, seq, pos, 0.3, 0, win, True,
        None, 0, 0.0, sv, D, None, fac, slopes).reshape(T, -1)
    c = rows.cuda()
    for splits in ((1, 4) if variant == 4 else (1,)):
        got = ops.talk_attention(
            q.cuda(), c, c, tables.cuda(), seq.cuda(), pos.cuda(), 0.3, H,
            window=win, sink=True, sink_vals=sv.cuda(), vdim=D,
            variant=variant, splits=splits, key_scale=fac.cuda(),
            slopes=slopes.cuda())
        assert relerr(got, want) < 1e-5
