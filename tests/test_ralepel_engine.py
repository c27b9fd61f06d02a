"""Ralepel through the engine: checkpoint folder -> registry -> runner ->
scheduler / block manager, against the float64 oracle in
tests/oracle_ralepel.py. Every test builds its own small configuration and
random weights. CPU runs the reference ops; gpu-marked variants run the HIP
kernels."""

import json
import os

import pytest
import torch

import oracle_ralepel as O
from production_stack_amd.engine.models import registry
from production_stack_amd.engine.sampling import SamplingParams
from ralepel_util import (TOL, attn, close, dense, latent, make_cfg,
                          make_engine, make_weights, moe, rel_err,
                          save_checkpoint)

pytestmark = pytest.mark.filterwarnings("ignore::UserWarning")

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = ["float32", "bfloat16"]

# windows of 20 / 13 / 33 positions, three query heads on a key among them,
# two latent caches, each read by a later layer too, every feed-forward kind
STACK = [
    (attn(4, 2, 24, 20, 0.3), dense(80)),
    (latent(3, 12, 8, 20, 24, 0.25, 1000.0), moe(24, 5, 2, 40)),
    (attn(6, 2, 16, 13, 0.4), moe(16, 7, 3, 0)),
    (latent(2, 16, 4, 8, 40, 0.3, 50.0), None),
    (latent(5, 8, 8, 12, 24, 0.3, 1000.0, src=1), dense(48)),
    (attn(3, 3, 32, 33, 0.2), moe(24, 6, 2, 16)),
    (latent(4, 8, 4, 16, 40, 0.35, 50.0, src=3), None),
]
VOCAB = 97


@pytest.fixture(scope="module")
def ckpt(tmp_path_factory):
    cfg = make_cfg(STACK, width=64, vocab=VOCAB)
    W = make_weights(cfg, seed=6)
    path = save_checkpoint(tmp_path_factory.mktemp("rl") / "m", cfg, W)
    return path, cfg, W


def tokens(n, seed, vocab=VOCAB):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def cuts(n, sizes):
    out, at = [], 0
    for s in sizes:
        s = n - at if s is None else min(s, n - at)
        if s > 0:
            out.append((at, at + s))
            at += s
    assert at == n
    return out


def replay(eng, rid, toks, sizes):
    """Feed toks in portions of the given sizes (None = the rest); returns
    logits at every position."""
    out = []
    for a, b in cuts(len(toks), sizes):
        out.append(eng.replay_step(
            [(rid, toks[a:b], list(range(b - a)))],
            end=[rid] if b == len(toks) else []))
    return torch.cat(out)


def replay_many(eng, toks, plan):
    """toks: id -> tokens; plan: steps of [(id, count)]. Returns id ->
    logits at every position; ids end with their last token."""
    at = {k: 0 for k in toks}
    got = {k: [] for k in toks}
    for step in plan:
        entries, end = [], []
        for rid, n in step:
            lo = at[rid]
            entries.append((rid, toks[rid][lo:lo + n], list(range(n))))
            at[rid] += n
            if at[rid] == len(toks[rid]):
                end.append(rid)
        out = eng.replay_step(entries, end=end)
        r0 = 0
        for rid, n in step:
            got[rid].append(out[r0:r0 + n])
            r0 += n
    assert at == {k: len(v) for k, v in toks.items()}
    return {k: torch.cat(v) for k, v in got.items()}


# ---------------------------------------------------------------------------
def test_registry_reads_checkpoint_folder(ckpt):
    path, cfg, W = ckpt
    mc = registry.config_from_dir(path)
    assert mc.family == "ralepel" and mc.vocab_size == VOCAB
    assert mc.hidden_size == 64 and len(mc.layer_specs) == len(STACK)
    assert not mc.has_recurrent_state and not mc.tie_word_embeddings
    s0, s1, s2, s3, s4, s5, s6 = mc.layer_specs
    assert (s0.post_norm, s0.pre_norm, s0.parallel) == (True, False, False)
    m = s0.mixer
    assert (m.kind, m.heads, m.kv_heads, m.dim, m.window, m.scale, m.bias,
            m.out_bias, m.learned_sink, m.key_values, m.unit_qk,
            m.distance_bias, m.rope) == (
        "attention", 4, 2, 24, 20, 0.3, True, True, True, True, True, True,
        False)
    m = s1.mixer
    assert (m.kind, m.heads, m.dim, m.rot_dim, m.rot_dims, m.vdim,
            m.kv_rank, m.scale, m.rot_base, m.rot_layout, m.window,
            m.kv_from) == (
        "latent_attention", 3, 12, 8, 8, 20, 24, 0.25, 1000.0, "half", 0,
        None)
    assert s4.mixer.kv_from == 1 and s6.mixer.kv_from == 3
    f = s1.mlp
    assert (f.kind, f.ff, f.experts, f.top, f.score, f.renormalize, f.act,
            f.router_bias, f.shared_ff, f.shared_gate) == (
        "moe", 24, 5, 2, "softmax", True, "silu", True, 40, True)
    assert s2.mlp.shared_ff == 0 and s3.mlp is None
    assert (s0.mlp.kind, s0.mlp.ff, s0.mlp.act, s0.mlp.gated) == (
        "dense", 80, "silu", True)
    assert "ralepel" in registry.FP32_FAMILIES


@pytest.mark.parametrize("bad", [
    [(latent(src=1), None), (latent(), None)],           # a later layer
    [(attn(), None), (latent(src=0), None)],             # no latent layer
    [(latent(), None), (latent(src=0), None), (latent(src=1), None)],
    [(latent(kv_rank=16), None), (latent(src=0), None)],
    [(latent(base=10.0), None), (latent(src=0), None)],
])
def test_bad_cache_sources_are_refused(tmp_path, bad):
    cfg = make_cfg(bad)
    path = save_checkpoint(tmp_path / "b", cfg, make_weights(cfg))
    with pytest.raises(ValueError, match="kv_from"):
        registry.config_from_dir(path)


def test_shared_layers_hold_no_cache_of_their_own(ckpt):
    """Layers 4 and 6 read the caches of 1 and 3; the pool's size counts
    every cache once, keys without values."""
    path, _, _ = ckpt
    for dtype, esz in (("float32", 4), ("bfloat16", 2)):
        eng = make_engine(path, dtype, "cpu")
        kv = eng.runner.kv_caches
        assert kv[4] is kv[1] and kv[6] is kv[3]
        assert kv[0][0].shape[1:] == (2, 16, 24)
        assert kv[0][1].shape[1:] == (2, 16)
        assert kv[0][1].dtype == torch.float32
        per = 16 * (2 * (24 * esz + 4) + (24 + 8) * esz + 2 * (16 * esz + 4)
                    + (40 + 4) * esz + 3 * (32 * esz + 4))
        assert eng.runner.model.kv_bytes_per_block(16) == per
        seen = {}
        for c in kv:
            for t in (c if isinstance(c, tuple) else (c,)):
                seen[t.data_ptr()] = t.numel() * t.element_size()
        assert sum(seen.values()) == per * eng.runner.num_blocks


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_prompt_and_every_layer(ckpt, device, dtype):
    path, cfg, W = ckpt
    toks = tokens(70, 1)
    layers = []
    want = O.forward(cfg, W, toks, layers)
    eng = make_engine(path, dtype, device)
    seen = {}
    eng.runner.model.residual_hook = lambda i, x: seen.__setitem__(
        i, x.detach().clone())
    got = replay(eng, "a", toks, [None])
    assert close(got, want, dtype)
    assert sorted(seen) == list(range(len(STACK)))
    for i, s in enumerate(layers):
        assert seen[i].dtype == torch.float32     # fp32 residual stream
        assert close(seen[i], s, dtype), i


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_and_single_token_prompt(ckpt, device, dtype):
    path, cfg, W = ckpt
    eng = make_engine(path, dtype, device)
    for n in (1, 2, 3, 9):
        toks = tokens(n, 10 + n)
        want = O.forward(cfg, W, toks)
        assert close(replay(eng, f"p{n}", toks, [None]), want, dtype)
        assert close(replay(eng, f"q{n}", toks, [1] * n), want, dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [
    [1] * 90, [2] * 45, [3, 2, 17, 2, 31, 2, None], [19, 1, 1, 1, None],
    [20, 20, 13, None], [33, 1, 33, None], [16, 16, 16, 16, 16, None],
    [64, 2, 2, None]])
def test_portions_match_whole_prompt(ckpt, device, dtype, sizes):
    """Prefill against token-by-token decoding, and portions of several
    sizes down to two tokens, cut inside pages and windows and exactly on
    their edges."""
    path, cfg, W = ckpt
    toks = tokens(90, 2)
    want = O.forward(cfg, W, toks)
    eng = make_engine(path, dtype, device)
    assert close(replay(eng, "a", toks, sizes), want, dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decode_past_many_windows(ckpt, device, dtype):
    path, cfg, W = ckpt
    toks = tokens(290, 3)
    want = O.forward(cfg, W, toks)
    eng = make_engine(path, dtype, device)
    # a first portion of more than 128 rows runs one GEMM pair per expert,
    # the short one and the single tokens the grouped kernels
    got = replay(eng, "a", toks, [150, 20] + [1] * 120)
    assert close(got, want, dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_reuse_pages(ckpt, device, dtype):
    """Up to three live requests of unequal length per step, portions
    beside single tokens; the pool (12 pages) is smaller than the sum of all
    requests, so pages with stale rows pass from finished requests to new
    ones. Every request must equal itself alone."""
    path, cfg, W = ckpt
    lens = {"a": 61, "b": 7, "c": 40, "d": 1, "e": 47, "f": 22}
    toks = {k: tokens(n, 30 + i) for i, (k, n) in enumerate(lens.items())}
    eng = make_engine(path, dtype, device, blocks=12, max_seqs=3)
    got = replay_many(eng, toks, [
        [("a", 17), ("b", 2), ("c", 3)],
        [("a", 1), ("b", 5), ("c", 16)],          # b ends
        [("a", 2), ("d", 1), ("c", 1)],           # d: one-token request
        [("c", 20), ("e", 31)],                   # a sits out; c ends
        [("a", 41), ("e", 1), ("f", 2)],          # a ends
        [("e", 15), ("f", 20)],                   # both end
    ])
    assert eng.block_manager.num_free == 12       # all given back
    for k in toks:
        assert close(got[k], O.forward(cfg, W, toks[k]), dtype), k


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_large_mixed_step(ckpt, device, dtype):
    """A step whose portions add up to several hundred rows beside single
    tokens, over sequences with and without history."""
    path, cfg, W = ckpt
    lens = {"a": 300, "b": 180, "c": 50, "d": 30}
    toks = {k: tokens(n, 60 + i) for i, (k, n) in enumerate(lens.items())}
    eng = make_engine(path, dtype, device, blocks=60)
    got = replay_many(eng, toks, [
        [("a", 40), ("c", 49), ("d", 2)],
        [("a", 200), ("b", 150), ("c", 1), ("d", 1)],
        [("a", 59), ("b", 2), ("d", 27)],
        [("a", 1), ("b", 28)],
    ])
    for k in toks:
        assert close(got[k], O.forward(cfg, W, toks[k]), dtype), k


def oracle_greedy(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(O.forward(cfg, W, toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("budget,blocks", [(1 << 20, 64), (7, 64), (24, 9)])
def test_greedy_generation_through_the_scheduler(ckpt, device, budget,
                                                 blocks):
    """LLMEngine.generate: the scheduler's own chunking (token budgets of
    7 and 24 cut the prompts into portions), continuous batching of three
    unequal requests, and with 9 pages preemption with recomputation, must
    all give the oracle's greedy continuation."""
    path, cfg, W = ckpt
    prompts = [tokens(45, 50), tokens(3, 51), tokens(28, 52)]
    n_new = 10
    want = [oracle_greedy(cfg, W, p, n_new) for p in prompts]
    eng = make_engine(path, "float32", device, blocks=blocks, max_seqs=3,
                      budget=budget)
    out = eng.generate(prompts, SamplingParams(
        max_tokens=n_new, temperature=0.0, ignore_eos=True))
    for i in range(3):
        assert out[f"offline-{i}"] == want[i], i
    assert eng.block_manager.num_free == blocks


@pytest.mark.parametrize("device", DEVICES)
def test_prefix_pages_are_shared(ckpt, device):
    """A second prompt with the same beginning takes the first one's pages
    (rows, their factors and latent rows alike)."""
    path, cfg, W = ckpt
    eng = make_engine(path, "float32", device)
    head = tokens(48, 70)
    one = SamplingParams(max_tokens=4, temperature=0.0, ignore_eos=True)
    for tail in (tokens(9, 71), tokens(5, 72)):
        p = head + tail
        got = eng.generate([p], one)
        assert list(got.values())[0] == oracle_greedy(cfg, W, p, 4)


OTHER_STACKS = [
    # (stack, width, vocab, eps)
    # one head of everything, window of one position, one expert
    ([(attn(1, 1, 8, 1, 1.0), moe(8, 1, 1, 8)),
      (latent(1, 4, 2, 4, 8, 1.0, 10.0), None)], 32, 41, 1e-6),
    # widths that are no multiple of 8, top = experts, odd head groups
    ([(latent(5, 6, 10, 7, 18, 0.4, 1e4), moe(20, 3, 3, 12)),
      (attn(9, 3, 20, 11, 0.3), dense(52)),
      (latent(7, 10, 10, 9, 18, 0.3, 1e4, src=0), None)], 60, 53, 3e-4),
    # no feed-forward at all; window longer than the sequence; three layers
    # on one cache
    ([(latent(6, 16, 16, 16, 48, 0.2, 1e5), None),
      (latent(8, 24, 16, 24, 48, 0.2, 1e5, src=0), None),
      (attn(8, 2, 40, 500, 0.2), None),
      (latent(2, 8, 16, 8, 48, 0.3, 1e5, src=0), None)], 72, 71, 1e-5),
    # heads wider than 128 entries, a group of 18 heads, many small experts,
    # latent wider than 128 entries
    ([(attn(18, 1, 136, 24, 0.08), moe(16, 40, 1, 24)),
      (latent(2, 32, 16, 32, 136, 0.15, 5e5), dense(24)),
      (attn(2, 2, 256, 17, 0.06), moe(8, 6, 4, 0))], 64, 37, 1e-5),
]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", range(len(OTHER_STACKS)))
def test_other_orders_and_sizes(tmp_path, device, dtype, which):
    stack, width, vocab, eps = OTHER_STACKS[which]
    cfg = make_cfg(stack, width=width, vocab=vocab, eps=eps)
    W = make_weights(cfg, seed=40 + which)
    path = save_checkpoint(tmp_path / f"o{which}", cfg, W)
    toks = tokens(80, 70 + which, vocab=vocab)
    want = O.forward(cfg, W, toks)
    eng = make_engine(path, dtype, device)
    assert close(replay(eng, "a", toks, [None]), want, dtype)
    assert close(replay(eng, "b", toks, [6, 1, 2, 30, 1, 1, None]), want,
                 dtype)
    # two requests side by side, cut differently
    got = replay_many(eng, {"x": toks, "y": toks}, [
        [("x", 9), ("y", 33)], [("x", 40), ("y", 2)],
        [("x", 31), ("y", 45)]])
    assert close(got["x"], want, dtype) and close(got["y"], want, dtype)


# ---------------------------------------------------------------------------
# a key made to stand out: at the window's edges, on a page border, far away
# ---------------------------------------------------------------------------
NEEDLE, PROBE = 3, 4


def needle_embedding(W, cfg):
    """The NEEDLE token is channel 0 alone, the PROBE token channel 1 alone,
    no other token reaches either channel."""
    emb = W["embed"].float()
    emb[:, :2] = 0.0
    emb[NEEDLE], emb[PROBE] = 0.0, 0.0
    emb[NEEDLE, 0] = emb[PROBE, 1] = 4.0
    W["embed"] = emb.to(torch.bfloat16)


def needle_attention(size, heads, kv_heads, dim=16, width=32, vocab=23):
    """One attention layer whose PROBE query lies along a direction u that
    only the NEEDLE's key has; that key, which is its own value, is large.
    Whether the needle is visible decides the probe's logits."""
    cfg = make_cfg([(attn(heads, kv_heads, dim, size, 1.0), None)],
                   width=width, vocab=vocab)
    W = make_weights(cfg, seed=9)
    needle_embedding(W, cfg)
    u = torch.ones(dim)
    u[::2] = -1.0                             # unit root mean square
    p = "l0.mix."
    for name, n, chan, gain in (("q", heads, 1, 1.0), ("k", kv_heads, 0, 2.0)):
        w = W[p + name].float().view(n, dim, width)
        b = W[p + name + ".b"].float().view(n, dim)
        # everything else keeps off the direction
        w -= u[:, None] * (w * u[:, None]).sum(1, keepdim=True) / dim
        b -= u * (b * u).sum(1, keepdim=True) / dim
        w[:, :, chan] = gain * u
        W[p + name] = w.reshape(n * dim, width).to(torch.bfloat16)
        W[p + name + ".b"] = (0.2 * b).reshape(-1).to(torch.bfloat16)
    return cfg, W


def needle_latent(heads=2, width=32, vocab=23, L=16):
    """Two latent layers on the first one's rows. The first adds nothing (a
    zero norm weight), so the second reads embeddings: its PROBE query
    matches the NEEDLE's key far above every other pair, through a latent
    entry that no other token reaches."""
    shape = (heads, 8, 4, 8, L, 1.0, 100.0)
    cfg = make_cfg([(latent(*shape), None), (latent(*shape, src=0), None)],
                   width=width, vocab=vocab)
    W = make_weights(cfg, seed=9)
    needle_embedding(W, cfg)
    W["l0.norm1"] = torch.zeros(width, dtype=torch.bfloat16)
    d = W["l0.mix.dkv"].float()
    d[:, :2], d[0] = 0.0, 0.0
    d[0, 0] = 6.0
    W["l0.mix.dkv"] = d.to(torch.bfloat16)
    W["l0.mix.dkv.norm"] = torch.ones(L, dtype=torch.bfloat16)
    q = W["l1.mix.q"].float() * 0.3
    q[:, :2] = 0.0
    q[::12] = 0.0
    q[::12, 1] = 1.5
    W["l1.mix.q"] = q.to(torch.bfloat16)
    k = W["l1.mix.uk"].float() * 0.3
    k[:, 0] = 0.0
    k[::8] = 0.0
    k[::8, 0] = 1.5
    W["l1.mix.uk"] = k.to(torch.bfloat16)
    v = W["l1.mix.uv"].float()
    v[:, 0] = 2.0
    W["l1.mix.uv"] = v.to(torch.bfloat16)
    return cfg, W


def needle_tokens(n, needle_at, probe_at, seed, vocab=23):
    g = torch.Generator().manual_seed(seed)
    t = torch.randint(5, vocab, (n,), generator=g).tolist()
    t[needle_at] = NEEDLE
    t[probe_at] = PROBE
    return t


CUTS = ([None], [90] + [1] * 14, [77, 2, 2, None], [64, 35, 1, None],
        [98, 2, None])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads", [(2, 2), (6, 2), (4, 1)])
def test_window_edges_with_a_stand_out_key(tmp_path, device, dtype, heads,
                                           kv_heads):
    """The probe sits at position 99, the window holds 24 positions
    (76..99). The needle is put just inside (76), just outside (75), on a
    page border inside (80) and outside (64), beside the probe (98) and far
    back (2): in prompt portions and in single decoded tokens."""
    cfg, W = needle_attention(24, heads, kv_heads)
    path = save_checkpoint(tmp_path / "n", cfg, W)
    eng = make_engine(path, dtype, device)
    seen = {}
    for spot in (76, 75, 80, 64, 98, 2):
        toks = needle_tokens(104, spot, 99, 60)
        want = O.forward(cfg, W, toks)
        seen[spot] = want[99]
        for sizes in CUTS:
            got = replay(eng, f"r{spot}", toks, sizes)
            assert close(got, want, dtype, routed=False), (spot, sizes)
    # the test has teeth: the probe's logits tell the cases apart
    for a in (76, 80, 98):
        assert rel_err(seen[a], seen[75]) > 0.3, a
        assert rel_err(seen[a], seen[2]) > 0.3, a


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys_in_a_shared_latent_cache(tmp_path, device, dtype):
    """No window: the needle at the start, far back, at page borders and
    beside the probe, seen by a layer that reads another layer's cache."""
    cfg, W = needle_latent()
    path = save_checkpoint(tmp_path / "l", cfg, W)
    eng = make_engine(path, dtype, device)
    base = O.forward(cfg, W, needle_tokens(104, 103, 99, 60))[99]
    for spot in (0, 2, 63, 64, 98):
        toks = needle_tokens(104, spot, 99, 60)
        want = O.forward(cfg, W, toks)
        assert rel_err(want[99], base) > 0.3, spot
        for sizes in CUTS:
            got = replay(eng, f"r{spot}", toks, sizes)
            assert close(got, want, dtype, routed=False), (spot, sizes)


@pytest.mark.parametrize("device", DEVICES)
def test_distance_penalty_and_sink_hold_the_weights(tmp_path, device):
    """Equal keys everywhere: weights follow slope and sink alone, so the
    attended value is the closed form of a geometric sum over the window."""
    H, D, size, sc = 3, 8, 12, 0.5
    cfg = make_cfg([(attn(H, 1, D, size, sc), None)], width=16, vocab=11)
    W = make_weights(cfg, seed=5)
    toks = [7] * 40
    eng = make_engine(save_checkpoint(tmp_path / "g", cfg, W), "float32",
                      device)
    got = replay(eng, "a", toks, [25, 2, 1, 1, None])
    x = W["embed"][7].double()
    q = O.lin(W, "l0.mix.q", x).view(H, D)
    v = O.lin(W, "l0.mix.k", x)
    s = sc * (O.unit_rms(q, 1e-5) @ O.unit_rms(v, 1e-5))
    rows = []
    for t in range(40):
        o = []
        for h in range(H):
            a = torch.arange(min(t + 1, size), dtype=torch.float64)
            e = torch.exp(s[h] - 2.0 ** (-8.0 * (h + 1) / H) * a).sum()
            w = e / (e + torch.exp(W["l0.mix.sink"][h].double()))
            o.append(w * v)
        y = O.lin(W, "l0.mix.o", torch.cat(o))
        rows.append(x + O.rms_norm(y, W["l0.norm1"], 1e-5))
    want = O.rms_norm(torch.stack(rows), W["final.norm"], 1e-5) \
        @ W["head"].double().t()
    assert rel_err(got, want) < 2e-4


def test_router_bias_and_shared_gate_show():
    """Guards the oracle: the bias moves choice and weights, the shared
    expert is gated."""
    cfg = make_cfg([(attn(), moe(8, 4, 2, 8))])
    W = make_weights(cfg, seed=4)
    toks = tokens(24, 7)
    base = O.forward(cfg, W, toks)
    for name in ("router.b", "shared.sg", "shared.down"):
        W2 = dict(W)
        W2["l0.mlp." + name] = torch.zeros_like(W["l0.mlp." + name])
        assert rel_err(O.forward(cfg, W2, toks), base) > 1e-2, name


def test_named_config_generates_deterministically():
    """The named tiny stack: random init, engine entry point, greedy."""
    from production_stack_amd.engine.config import (CacheConfig,
                                                    EngineConfig,
                                                    SchedulerConfig)
    from production_stack_amd.engine.engine import LLMEngine

    def run(budget):
        eng = LLMEngine(EngineConfig(
            model="tiny-ralepel", dtype="float32", max_model_len=256,
            enforce_eager=True,
            cache=CacheConfig(num_gpu_blocks=32, block_size=16),
            scheduler=SchedulerConfig(max_num_seqs=2,
                                      max_num_batched_tokens=budget,
                                      max_prefill_chunk=budget)),
            device="cpu")
        return eng.generate(
            [tokens(70, 1, 300), tokens(4, 2, 300)],
            SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True))

    a, b = run(256), run(11)
    assert a == b and all(len(v) == 6 for v in a.values())


def test_trace_run_command(ckpt, tmp_path):
    """bin/trace_run end to end: JSON lines in, 'done' lines and logit
    files out, requests ended and replaced, one request filling the whole
    pool."""
    import subprocess
    import sys

    import numpy as np

    path, cfg, W = ckpt
    root = os.path.join(os.path.dirname(__file__), "..")
    ta, tb, tc = tokens(40, 80), tokens(7, 81), tokens(128, 82)
    steps = [
        {"step": 0, "entries": [
            {"id": "a", "tokens": ta[:33], "want": [0, 32]},
            {"id": "b", "tokens": tb, "want": [6]}], "end": ["b"]},
        {"step": 1, "entries": [
            {"id": "a", "tokens": ta[33:34], "want": []}], "end": []},
        {"step": 2, "entries": [
            {"id": "a", "tokens": ta[34:], "want": [5]}], "end": ["a"]},
        {"step": 3, "entries": [
            {"id": "c", "tokens": tc, "want": [127]}], "end": ["c"]},
    ]
    out = tmp_path / "out"
    r = subprocess.run(
        [sys.executable, os.path.join(root, "bin", "trace_run"), "--model",
         path, "--dtype", "float32", "--out", str(out), "--max-tokens", "128",
         "--max-seqs", "2", "--device", "cpu"],
        input="\n".join(json.dumps(s) for s in steps) + "\n",
        capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    done = [ln for ln in r.stdout.splitlines() if ln.startswith("done ")]
    assert done == [f"done {i}" for i in range(4)]
    assert not (out / "1.f32").exists()
    wa, wb, wc = (O.forward(cfg, W, t) for t in (ta, tb, tc))

    def read(i, n):
        return torch.from_numpy(np.fromfile(
            out / f"{i}.f32", dtype="<f4").reshape(n, -1).copy())

    assert rel_err(read(0, 3), torch.stack([wa[0], wa[32], wb[6]])) < 2e-4
    assert rel_err(read(2, 1), wa[39:40]) < 2e-4
    assert rel_err(read(3, 1), wc[127:]) < 2e-4


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
def test_decode_graph_replays_match_eager(ckpt, dtype):
    """Single-token steps replay a captured hipGraph (padded to a batch
    bucket, experts planned on the device). Three requests of unequal length
    join and leave, so bucket sizes and padding rows change between replays;
    eager prompt portions run in between. Every step's logits must match the
    eager engine's."""
    from production_stack_amd.engine.config import (CacheConfig,
                                                    EngineConfig,
                                                    SchedulerConfig)
    from production_stack_amd.engine.engine import LLMEngine

    path, cfg, W = ckpt

    def make(eager):
        return LLMEngine(EngineConfig(
            model=path, dtype=dtype, max_model_len=256, enforce_eager=eager,
            cache=CacheConfig(num_gpu_blocks=48, block_size=16,
                              enable_prefix_caching=False),
            scheduler=SchedulerConfig(max_num_seqs=4,
                                      max_num_batched_tokens=64)),
            device="cuda")

    graph, eager = make(False), make(True)
    assert graph.runner.graphs is not None and eager.runner.graphs is None
    prompts = [tokens(37, 90), tokens(5, 91), tokens(70, 92)]
    lens = [9, 14, 6]
    outs = []
    for eng in (graph, eager):
        got, seen = {}, []
        orig = eng.runner.sample

        def spy(logits, seqs, _orig=orig, _seen=seen):
            _seen.append(logits.detach().float().cpu().clone())
            return _orig(logits, seqs)

        eng.runner.sample = spy
        for i, (p, n) in enumerate(zip(prompts, lens)):
            eng.add_request(f"r{i}", p, SamplingParams(
                max_tokens=n, temperature=0.0, ignore_eos=True))
        while eng.has_unfinished():
            for o in eng.step():
                got.setdefault(o.request_id, []).extend(o.new_token_ids)
        outs.append((got, seen))
    (g_tok, g_log), (e_tok, e_log) = outs
    assert len(g_log) == len(e_log) and len(g_log) >= max(lens)
    for a, b in zip(g_log, e_log):
        assert a.shape == b.shape
        if dtype == "float32":
            assert rel_err(a, b) < TOL["float32"]
    if dtype == "float32":
        assert g_tok == e_tok
        want = [oracle_greedy(cfg, W, p, n) for p, n in zip(prompts, lens)]
        assert [g_tok[f"r{i}"] for i in range(3)] == want
