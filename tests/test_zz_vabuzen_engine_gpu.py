"""GPU tier: the Vabuzen family on the layer-list engine against the plain float64 restatement in tests/layer_list_oracle.py, on
small made-up configurations with random (or crafted) weights: Dynamic Tanh norms on both sides of every sublayer, loop passes that add the
embedding output back, short convolutions on q, k and v ahead of sliding windows that keep the first tokens (with a one in the softmax
denominator), latent attention with direct queries and half-split rotation pairs, feed-forwards with biases, experts chosen by groups,
capped logits.

float32 runs are held to a relative RMS error of 2e-4 per logits row, bfloat16 runs to 4e-2 (layer_list_engine_helpers.TOL).
"""

import json

import numpy as np
import pytest
import torch

import layer_list_oracle as O
from layer_list_engine_helpers import TOL, in_portions, make_engine, rel_err, tokens_for, whole

pytestmark = pytest.mark.gpu

# five layers, the middle three run twice: windows of 20 + 3 and 13 + 5 first tokens, convolutions of 4 and 6 taps, every kind of feed-forward and none
MIXED = O.vabuzen_config([O.vabuzen_attention_layer(),
                          O.vabuzen_latent_layer(mlp=None),
                          O.vabuzen_attention_layer(heads=6, kv_heads=3, dim=24, vdim=8, conv=6, rot_dims=24, window=13, keep_first=5, mlp=O.vabuzen_moe()),
                          O.vabuzen_latent_layer(heads=3, dim=24, vdim=16, rot_dim=12, kv_rank=24, mlp={"kind": "dense", "ff": 50}),
                          O.vabuzen_attention_layer(heads=2, kv_heads=2, dim=20, vdim=12, conv=2, rot_dims=0, window=29, keep_first=0, mlp=None)], loop=(1, 4, 2))
RUNS = 5 + 3

A_ = O.vabuzen_attention_layer
L_ = O.vabuzen_latent_layer
M_ = O.vabuzen_moe
LAYERS = {
    "attention": A_(),
    "attention_no_feed_forward": A_(mlp=None),
    "attention_window_of_one": A_(window=1, keep_first=0),
    "attention_window_of_one_and_the_first": A_(window=1, keep_first=1),
    "attention_keeps_none": A_(keep_first=0),
    "attention_keeps_more_than_the_window": A_(window=5, keep_first=18),
    "attention_keeps_every_token": A_(window=2, keep_first=100),
    "attention_window_beyond_the_sequence": A_(window=400, keep_first=7),
    "attention_window_of_a_page": A_(window=16, keep_first=16),
    "attention_one_tap": A_(conv=1),
    "attention_two_taps": A_(conv=2),
    "attention_many_taps": A_(conv=30),
    "attention_no_rotation": A_(rot_dims=0),
    "attention_full_rotation": A_(dim=24, rot_dims=24),
    "attention_as_many_kv_heads": A_(heads=3, kv_heads=3, dim=8, vdim=8, rot_dims=8),
    "attention_one_kv_head": A_(heads=6, kv_heads=1),
    "attention_one_head": A_(heads=1, kv_heads=1, dim=32, vdim=40),
    "attention_large_group": A_(heads=20, kv_heads=1, dim=8, vdim=8, rot_dims=4),
    "attention_wide_heads": A_(heads=2, kv_heads=1, dim=128, vdim=96, rot_dims=64),
    "attention_widest_heads": A_(heads=2, kv_heads=2, dim=136, vdim=72),
    "attention_keys_of_80": A_(heads=6, kv_heads=2, dim=80, vdim=56, rot_dims=80),
    "attention_values_of_112": A_(heads=4, kv_heads=4, dim=40, vdim=112, rot_dims=20),
    "attention_group_of_eight": A_(heads=8, kv_heads=1, dim=96, vdim=64, rot_dims=32, window=9, keep_first=8),
    "attention_group_of_three": A_(heads=9, kv_heads=3, dim=56, vdim=48, rot_dims=56, conv=8),
    "attention_nine_taps": A_(conv=9, dim=18, vdim=14),
    "attention_odd_sizes": A_(heads=6, kv_heads=2, dim=10, vdim=13, conv=3, rot_dims=6, window=11, mlp={"kind": "dense", "ff": 13}),
    "latent": L_(),
    "latent_no_feed_forward": L_(mlp=None),
    "latent_one_head": L_(heads=1, dim=24, vdim=8, rot_dim=4, kv_rank=12),
    "latent_many_heads": L_(heads=20, dim=8, vdim=8, rot_dim=4, kv_rank=16),
    "latent_odd_sizes": L_(heads=5, dim=10, vdim=9, rot_dim=6, kv_rank=21, mlp={"kind": "dense", "ff": 13}),
    "latent_rotation_of_two": L_(rot_dim=2),
    "latent_row_of_160": L_(heads=6, dim=24, vdim=40, rot_dim=32, kv_rank=128),
    "latent_rotation_wider_than_the_rest": L_(heads=4, dim=8, vdim=32, rot_dim=48, kv_rank=56),
    "latent_rank_of_the_middle_tile": L_(heads=3, dim=16, vdim=16, rot_dim=16, kv_rank=104),
    "latent_wide": L_(heads=2, dim=72, vdim=40, rot_dim=64, kv_rank=192),
    "latent_wider": L_(heads=3, dim=16, vdim=16, rot_dim=16, kv_rank=240),
    "latent_wide_odd": L_(heads=2, dim=16, vdim=16, rot_dim=10, kv_rank=150),
    "latent_widest": L_(heads=2, dim=16, vdim=16, rot_dim=8, kv_rank=264),
    "experts_one_of_one": L_(mlp=M_(experts=1, top=1, ff=16, shared=0, groups=(1, 1))),
    "experts_all_taken": L_(mlp=M_(experts=4, top=4, ff=16, groups=(2, 2))),
    "experts_groups_of_one": L_(mlp=M_(experts=7, top=2, ff=16, groups=(7, 4))),
    "experts_one_group_kept": L_(mlp=M_(experts=12, top=3, ff=16, groups=(3, 1))),
    "experts_whole_groups_taken": L_(mlp=M_(experts=8, top=4, ff=16, groups=(4, 2))),
    "experts_no_shared": L_(mlp=M_(experts=6, top=2, ff=32, shared=0)),
    "experts_many": L_(mlp=M_(experts=72, top=5, ff=8, shared=16, groups=(8, 3))),
    "experts_scale_of_one": L_(mlp=M_(scale=1.0)),
    "experts_large_scale": L_(mlp=M_(scale=16.0)),
    "experts_odd_sizes": L_(mlp=M_(experts=9, top=2, ff=9, shared=13)),
}


class Reference(np.ndarray):
    """Logits of the restatement; ``sure`` marks the rows whose experts no rounding of the router's input can exchange."""


def reference(config, W, toks, streams=None):
    margins = []
    out = O.vabuzen_forward(config, W, toks, streams, margins).view(Reference)
    out.sure = np.all(np.stack(margins) > 0.01, 0) if margins else np.ones(len(toks), dtype=bool)
    return out


def close(got, want, dtype):
    """Every row in float32; in bfloat16 the rows without a close call of a router (at least half of them)."""
    if dtype == torch.float32 or not hasattr(want, "sure") or len(want.sure) != len(want):
        return rel_err(got, want) < TOL[dtype]
    assert len(want) < 4 or want.sure.mean() > 0.5
    return np.isfinite(got).all() and (not want.sure.any() or rel_err(np.asarray(got)[want.sure], np.asarray(want)[want.sure]) < TOL[dtype])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("layer", sorted(LAYERS))
def test_each_mechanism_alone(layer, dtype):
    config = O.vabuzen_config([LAYERS[layer]])
    W = O.make_vabuzen_weights(config, seed=3)
    toks = tokens_for(config, 53, seed=4)
    want = reference(config, W, toks)
    engine = make_engine(config, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [19, 1, 1, 6, 1]), want, dtype)
    finally:
        engine.close()


@pytest.mark.parametrize("loop", [None, (0, 3, 1), (0, 1, 4), (2, 3, 3), (1, 3, 2), (0, 3, 2)])
@pytest.mark.parametrize("mult,cap", [(1.0, 0), (0.4, 2.0)])
def test_loops_of_every_placement(loop, mult, cap):
    """A loop over the first, the last, the middle and all layers, one pass (its vector is added all the same); residual factors; logits with and without a cap.
    The pass entry leaves with the sum before it or is a launch of its own (at the first layer; with tracing on): the logits are the same bits."""
    config = O.vabuzen_config([A_(), L_(mlp={"kind": "dense", "ff": 24}), A_(conv=3, window=9, mlp=None)], loop=loop, residual_mult=mult, logit_softcap=cap)
    W = O.make_vabuzen_weights(config, seed=40)
    toks = tokens_for(config, 38, seed=41)
    want = reference(config, W, toks)
    engine = make_engine(config, W)
    try:
        got = whole(engine, toks)
        assert close(got, want, torch.float32)
        assert close(in_portions(engine, toks, [7, 1, 2]), want, torch.float32)
        engine.set_trace(True)
        assert np.array_equal(whole(engine, toks), got)
        assert close(in_portions(engine, toks, [1]), want, torch.float32)
    finally:
        engine.close()


@pytest.mark.parametrize("taps", [2, 3, 9])
def test_the_inputs_before_a_portion_are_the_sequences_own(taps):
    """Convolutions whose earlier taps outweigh the last: the first tokens of every portion need the sequence's own inputs before it -- beside another
    sequence in the same steps, in a slot that held a third one, after device-side decode steps (which move the inputs on inside the preparation), and
    after the sequence changed its slot."""
    config = O.vabuzen_config([A_(conv=taps, window=12, keep_first=2, mlp=None), A_(heads=2, kv_heads=1, conv=taps + 1, mlp=None)], loop=(0, 2, 2))
    W = O.make_vabuzen_weights(config, seed=42)
    for i in range(2):
        for n in "qkv":
            W[f"l{i}.mix.{n}.conv"][:, :-1] *= 2.0
    a, b, c = (tokens_for(config, n, seed=43 + n) for n in (21, 20, 16))
    wa, wb, wc = (O.vabuzen_forward(config, W, t) for t in (a, b, c))
    engine = make_engine(config, W)
    try:
        engine.begin(0)
        engine.begin(1)
        got_a, got_b = [], []
        for lo in range(0, 20, 4):
            rows = engine.logits_host(engine.step([(1, b[lo:lo + 4], range(4)), (0, a[lo:lo + 4], range(4))]))
            got_b.append(rows[:4])
            got_a.append(rows[4:])
        assert close(np.concatenate(got_a), wa[:20], torch.float32) and close(np.concatenate(got_b), wb[:20], torch.float32)
        engine.release(1)
        engine.begin(1)
        got_c = [engine.logits_host(engine.step([(1, c[:1], [0])])), engine.logits_host(engine.step([(1, c[1:], range(15)), (0, a[20:], [0])]))]
        assert close(got_c[0], wc[:1], torch.float32) and close(got_c[1][:15], wc[1:], torch.float32) and close(got_c[1][15:], wa[20:], torch.float32)
        engine.set_token(0, 5)
        engine.decode(1, slots=[0])
        nxt = engine.read_pending_slots([0])[0]
        engine.decode(1, slots=[0], use_graph=False)
        engine.move(0, 3)
        full = a + [5, nxt, 9, 11]
        want = O.vabuzen_forward(config, W, full)
        assert close(engine.logits_host(engine.step([(3, [9, 11], [0, 1])])), want[-2:], torch.float32)
    finally:
        engine.close()


def test_width_and_vocabulary_that_are_no_multiples_of_4():
    config = O.vabuzen_config([A_(), L_(mlp=None), L_(mlp=M_())], width=54, vocab=77, loop=(0, 2, 2))
    W = O.make_vabuzen_weights(config, seed=60)
    toks = tokens_for(config, 30, seed=61)
    want = reference(config, W, toks)
    for dtype in (torch.float32, torch.bfloat16):
        engine = make_engine(config, W, dtype)
        try:
            assert close(whole(engine, toks), want, dtype)
            assert close(in_portions(engine, toks, [1]), want, dtype)
        finally:
            engine.close()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_row_kernel_twin_of_the_tile_kernel(dtype, monkeypatch):
    """TL_HYBRID_ATTN_ROWS=1 sends every attention through the row kernel (a wave per row and head): the twin of the matrix-core kernel,
    with the same window, kept first tokens and sink."""
    monkeypatch.setenv("TL_HYBRID_ATTN_ROWS", "1")
    W = O.make_vabuzen_weights(MIXED, seed=62)
    toks = tokens_for(MIXED, 70, seed=63)
    want = reference(MIXED, W, toks)
    engine = make_engine(MIXED, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [33, 1]), want, dtype)
    finally:
        engine.close()


def test_stream_after_every_layer():
    W = O.make_vabuzen_weights(MIXED, seed=5)
    toks = tokens_for(MIXED, 29, seed=6)
    streams = []
    want = reference(MIXED, W, toks, streams)
    engine = make_engine(MIXED, W)
    try:
        assert engine.stats()["layer_runs"] == len(streams) == RUNS
        engine.set_trace(True)
        engine.begin(0)
        n = engine.step([(0, toks, list(range(len(toks))))])
        for run, ref in enumerate(streams):
            assert rel_err(engine.read_trace(run, len(toks)), ref) < 1e-5, f"layer run {run}"
        assert rel_err(engine.logits_host(n), want) < TOL[torch.float32]
        engine.release(0)
    finally:
        engine.close()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_prefill_against_token_by_token(dtype):
    W = O.make_vabuzen_weights(MIXED, seed=7)
    toks = tokens_for(MIXED, 45, seed=8)
    want = reference(MIXED, W, toks)
    engine = make_engine(MIXED, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [1]), want, dtype)
        assert close(in_portions(engine, toks, [30, 1]), want, dtype)  # a prompt, then decoding
    finally:
        engine.close()


@pytest.mark.parametrize("sizes", [[2], [3, 2, 7], [16], [15, 17, 1], [24, 5, 2, 40], [70, 13], [64, 1, 63, 2]])
def test_portions_of_several_sizes(sizes):
    """Portions end inside pages (16 tokens) and inside windows (20, 13 and 29 positions); the convolutions' inputs are carried across every cut."""
    W = O.make_vabuzen_weights(MIXED, seed=9)
    toks = tokens_for(MIXED, 150, seed=10)
    engine = make_engine(MIXED, W)
    try:
        assert rel_err(in_portions(engine, toks, sizes), reference(MIXED, W, toks)) < TOL[torch.float32]
    finally:
        engine.close()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_unequal_requests_in_one_batch_against_each_alone(dtype):
    """Portions of some requests beside single tokens of others; every request's rows must equal its whole-sequence logits."""
    W = O.make_vabuzen_weights(MIXED, seed=11)
    prompts = [tokens_for(MIXED, n, seed=10 + n) for n in (70, 9, 41, 25)]
    want = [reference(MIXED, W, p) for p in prompts]
    cuts = [[20, 1, 1, 30, 1, 1, 1, 15], [2, 1, 1, 1, 1, 1, 1, 1], [1, 17, 3, 19, 1], [25]]
    engine = make_engine(MIXED, W, dtype)
    try:
        at = [0] * 4
        got = [[] for _ in prompts]
        for s in range(4):
            engine.begin(s)
        turn = 0
        while any(at[i] < len(prompts[i]) for i in range(4)):
            entries, who = [], []
            for i in range(4):
                if at[i] < len(prompts[i]):
                    n = cuts[i][turn] if turn < len(cuts[i]) else 1
                    if (turn + i) % 5 == 4 and entries:
                        continue  # a request may sit out a step
                    part = prompts[i][at[i]:at[i] + n]
                    entries.append((i, part, list(range(len(part)))))
                    who.append((i, len(part)))
                    at[i] += len(part)
            turn += 1
            if not entries:
                continue
            rows = engine.logits_host(engine.step(entries))
            r = 0
            for i, n in who:
                got[i].append(rows[r:r + n])
                r += n
        for i in range(4):
            assert close(np.concatenate(got[i], 0), want[i], dtype), f"request {i}"
    finally:
        engine.close()


def test_pages_and_slots_are_used_again():
    """6 pages of 16 tokens and 2 slots serve 6 requests in pairs: pages that held another request's keys are overwritten before they are
    read, and a slot's convolution inputs start at zero again."""
    W = O.make_vabuzen_weights(MIXED, seed=12)
    engine = make_engine(MIXED, W, page_size=16, num_pages=6, max_batch=2, max_prefill_rows=96)
    try:
        prompts = [tokens_for(MIXED, n, seed=20 + n) for n in (40, 33, 48, 17, 31, 47)]
        want = [reference(MIXED, W, p) for p in prompts]
        for k in range(0, 6, 2):
            a, b = prompts[k], prompts[k + 1]
            engine.begin(0)
            engine.begin(1)
            ra = [engine.logits_host(engine.step([(0, a[:10], list(range(10)))]))]
            both = engine.logits_host(engine.step([(0, a[10:], list(range(len(a) - 10))), (1, b, list(range(len(b))))]))
            ra.append(both[:len(a) - 10])
            assert rel_err(np.concatenate(ra, 0), want[k]) < TOL[torch.float32]
            assert rel_err(both[len(a) - 10:], want[k + 1]) < TOL[torch.float32]
            engine.release(0)
            engine.release(1)
        st = engine.stats()
        assert st["reused_page_allocations"] > 0 and st["reused_slot_begins"] == 4 and st["pages_in_use"] == 0
        engine.begin(0)
        engine.step([(0, tokens_for(MIXED, 90, seed=1), [])])
        engine.begin(1)
        with pytest.raises(RuntimeError, match="exhausted"):
            engine.step([(1, tokens_for(MIXED, 10, seed=2), [])])
    finally:
        engine.close()


# ---- one key that decides the answer ---------------------------------------------------------------------------------------------

def _quiet(W, A, B):
    """Tokens A and B excite a channel of their own each; no other token excites either."""
    W["embed"][:, :2] = 0.0
    W["embed"][A] *= 0.05
    W["embed"][B] *= 0.05
    W["embed"][A, 0] = 8.0
    W["embed"][B, 1] = 8.0
    W["l0.norm1.b"][:2] = 0.0
    W["l0.norm1"][:2] = 1.0


def _bf16(W):
    for k in W:
        W[k] = torch.from_numpy(np.asarray(W[k], dtype=np.float32)).to(torch.bfloat16).float().numpy()


def _needle_attention(window, keep_first, delay=0, heads=4, kv_heads=2, dim=16, vdim=16):
    """B's query reads the channel only B excites, one unrotated key dimension of every head the one only A excites: where A is among the keys B sees, the
    score of (B, A) towers over the others and over the sink, so a lost, shifted or doubled key -- or a window, or a run of first tokens, that is one off --
    changes the logits at B by far more than the tolerance.  delay > 0: the convolutions of k and v pass the input `delay` tokens back and nothing else, so it
    is position p + delay that carries what token p says."""
    config = O.vabuzen_config([O.vabuzen_attention_layer(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=delay + 1, rot_dims=8, scale=0.5, window=window,
                                                         keep_first=keep_first, mlp=None)], vocab=50, logit_softcap=None)
    W = O.make_vabuzen_weights(config, seed=15)
    A, B = 48, 49
    _quiet(W, A, B)
    m = "l0.mix."
    for name in "qkv":
        W[m + name + ".conv"][:] = 0.0
        W[m + name + ".conv"][:, -1 if name == "q" else 0] = 1.0
    for name, n, channel in (("k", kv_heads, 0), ("q", heads, 1)):
        W[m + name] *= 0.3
        W[m + name][:, channel] = 0.0
        for h in range(n):
            W[m + name][h * dim + 12, :] = 0.0
            W[m + name][h * dim + 12, channel] = 6.0
    W[m + "v"][:, 0] += 1.0
    _bf16(W)
    return config, W, A, B


def _needle_latent(kv_rank=24):
    """The same through the latent: latent 0 of the cache is the one only A excites, and one unrotated dimension of every head joins it to B's query."""
    config = O.vabuzen_config([O.vabuzen_latent_layer(heads=2, dim=16, vdim=16, rot_dim=8, kv_rank=kv_rank, scale=0.5, mlp=None)], vocab=50, logit_softcap=None)
    W = O.make_vabuzen_weights(config, seed=16)
    A, B = 48, 49
    _quiet(W, A, B)
    m = "l0.mix."
    W[m + "dkv"][:, 0] = 0.0
    W[m + "dkv"][0, :] = 0.0
    W[m + "dkv"][0, 0] = 6.0
    W[m + "dkv.norm"][:] = 1.0
    W[m + "q"][:, 1] = 0.0
    W[m + "uk"][:, 0] = 0.0
    for h in range(2):
        W[m + "q"][h * 24, :] = 0.0
        W[m + "q"][h * 24, 1] = 6.0
        W[m + "uk"][h * 16, :] = 0.0
        W[m + "uk"][h * 16, 0] = 3.0
    W[m + "uv"][:, 0] += 1.0
    _bf16(W)
    return config, W, A, B


def _needle_prompt(config, A, B, n, needle_at, seed):
    toks = tokens_for(config, n, seed=seed, avoid=(A, B))
    toks[needle_at] = A
    toks[-1] = B
    return toks


def _needle_case(config, W, A, B, n, needle_at, query, seen, **pool):
    toks = _needle_prompt(config, A, B, n, needle_at, 16)
    want = O.vabuzen_forward(config, W, toks)[-1]
    other = list(toks)
    other[needle_at] = toks[needle_at - 1] if needle_at else toks[1]
    moved = rel_err(O.vabuzen_forward(config, W, other)[-1][None], want[None])
    assert (moved > 0.1) if seen else (moved < 1e-9)   # the needle decides the answer exactly where the mask lets B see it
    engine = make_engine(config, W, **pool)
    try:
        engine.begin(0)
        if query == "prompt":
            cut = n - 40
            engine.step([(0, toks[:cut], [])])
            k = engine.step([(0, toks[cut:], [n - cut - 1])])
        else:
            engine.step([(0, toks[:-1], [])])
            k = engine.step([(0, toks[-1:], [0])])
        assert rel_err(engine.logits_host(k), want[None]) < TOL[torch.float32]
        engine.release(0)
    finally:
        engine.close()


@pytest.mark.parametrize("needle_at", [0, 3, 15, 16, 17, 31, 32, 63, 64, 250, 298])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
@pytest.mark.parametrize("mixer", ["attention", "attention_large_group", "latent", "latent_wide"])
def test_far_keys_and_page_borders(mixer, needle_at, query):
    """A window beyond the sequence, or none: the last token sees every key; the needle sits far back, at page borders (16) and key-tile borders (64).  At
    300 tokens a decoded token's key range is split over workgroups."""
    config, W, A, B = {"attention": lambda: _needle_attention(1000, 4), "attention_large_group": lambda: _needle_attention(1000, 0, heads=20, kv_heads=1),
                       "latent": _needle_latent, "latent_wide": lambda: _needle_latent(192)}[mixer]()
    _needle_case(config, W, A, B, 300, needle_at, query, True, page_size=16, num_pages=24, max_batch=1)


@pytest.mark.parametrize("needle_at,seen", [(191, False), (192, True), (193, True), (207, True), (208, True), (254, True), (127, False), (0, True), (4, True), (5, False), (6, False)])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
def test_keys_just_inside_and_just_outside_a_window(needle_at, seen, query):
    """A window of 64 positions over pages of 16, 5 first tokens kept: the query at position 255 sees 0 .. 4 and 192 .. 255 and nothing else."""
    config, W, A, B = _needle_attention(64, 5)
    _needle_case(config, W, A, B, 256, needle_at, query, seen, page_size=16, num_pages=24, max_batch=1)


@pytest.mark.parametrize("n,needle_at,seen", [(101, 0, True), (103, 2, True), (104, 3, False), (150, 49, False), (150, 50, True), (201, 100, False), (201, 101, True),
                                              (450, 349, False), (450, 350, True), (450, 383, True), (450, 384, True), (450, 448, True), (450, 2, True), (450, 3, False),
                                              (100, 0, True), (102, 3, True), (103, 3, True), (60, 0, True)])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
def test_window_edges_that_are_no_page_or_tile_edges(n, needle_at, seen, query):
    """A window of 100 positions, 3 first tokens kept: its edge falls inside pages and inside the kernels' 64-key tiles, moves with every query, and starts to
    leave the first tokens behind at position 103."""
    config, W, A, B = _needle_attention(100, 3)
    _needle_case(config, W, A, B, n, needle_at, query, seen, page_size=16, num_pages=30, max_batch=1)


@pytest.mark.parametrize("keep_first,needle_at,seen", [(16, 15, True), (16, 16, False), (17, 16, True), (17, 17, False), (64, 63, True), (64, 64, False), (70, 69, True),
                                                       (70, 70, False), (70, 64, True), (1, 0, True), (1, 1, False), (200, 199, True), (200, 200, False), (0, 0, False),
                                                       (200, 450 - 31, True), (200, 450 - 30, True), (200, 450 - 32, False), (64, 450 - 30, True), (64, 450 - 31, False)])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
def test_first_tokens_that_end_at_pages_tiles_and_between(keep_first, needle_at, seen, query):
    """Runs of kept first tokens that end at a page (16), at a key tile (64) and inside one, and one that is longer than the window."""
    config, W, A, B = _needle_attention(31 if keep_first == 200 else 30, keep_first)
    _needle_case(config, W, A, B, 450, needle_at, query, seen, page_size=16, num_pages=30, max_batch=1)


@pytest.mark.parametrize("n,needle_at,seen", [(700, 399, False), (700, 400, True), (700, 401, True), (700, 463, True), (700, 464, True), (700, 650, True), (320, 19, True),
                                              (700, 19, True), (700, 20, False), (321, 20, False), (320, 20, True), (280, 0, True), (700, 0, True)])
def test_wide_window_of_a_decoded_token_over_split_key_ranges(n, needle_at, seen):
    """A window of 300 positions and 20 first tokens in a long context: the decoded token's keys are split over workgroups, the kept ones first."""
    config, W, A, B = _needle_attention(300, 20)
    _needle_case(config, W, A, B, n, needle_at, "decoded", seen, page_size=64, num_pages=12, max_batch=1, max_prefill_rows=1024)


@pytest.mark.parametrize("needle_at,seen", [(99, False), (100, True), (19, True), (20, False)])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(1, 1, 16, 16), (6, 2, 80, 96), (2, 1, 128, 128), (2, 1, 136, 40)])
def test_the_same_with_heads_of_every_width(needle_at, seen, query, heads, kv_heads, dim, vdim):
    """Head widths of every tile template and of the row kernel."""
    config, W, A, B = _needle_attention(300, 20, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim)
    _needle_case(config, W, A, B, 400, needle_at, query, seen, page_size=64, num_pages=12, max_batch=1, max_prefill_rows=1024)


@pytest.mark.parametrize("needle_at,seen", [(57, False), (58, False), (60, False), (61, True), (62, True), (0, True), (1, True), (2, False), (3, False), (156, True), (100, True)])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
def test_the_window_counts_positions_behind_the_convolution(needle_at, seen, query):
    """k and v delayed by 3 tokens, a window of 96 positions and 5 first ones: what token p says lies at position p + 3, and is seen at 159 from there."""
    config, W, A, B = _needle_attention(96, 5, delay=3)
    _needle_case(config, W, A, B, 160, needle_at, query, seen, page_size=16, num_pages=12, max_batch=1)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n,window,keep_first", [(40, 12, 4), (400, 1000, 0), (400, 300, 20)])
def test_the_one_in_the_denominator_counts_once(n, window, keep_first, dtype):
    """Scores around minus the logarithm of the number of keys: the one holds about half of the weight, alone in a window of few keys and over split key
    ranges (decoding at 400 tokens); a one that is left out, or counted once per split, moves the logits by far more than the tolerance."""
    config = O.vabuzen_config([A_(heads=4, kv_heads=2, conv=2, rot_dims=0, window=window, keep_first=keep_first, scale=1.0, mlp=None)], logit_softcap=None)
    W = O.make_vabuzen_weights(config, seed=70)
    m = "l0.mix."
    W["embed"][:, 2] = 30.0                # a channel every token excites (the norm saturates at its weight)
    W["l0.norm1"][2], W["l0.norm1.b"][2] = 1.0, 0.0
    for name in "qk":
        W[m + name] *= 0.1
        W[m + name][:, 2] = 0.0
        W[m + name + ".conv"][:] = [0.0, 1.0]
    seen = min(n, window + keep_first)
    W[m + "q"][np.arange(4) * 16, 2] = 1.0
    W[m + "k"][np.arange(2) * 16, 2] = -np.log(seen)
    W[m + "v"][:, 2] = np.where(np.arange(48) % 2, 1.5, -1.5)   # (values with a mean: what the one takes away shows)
    W[m + "v.conv"][:] = [0.0, 1.0]
    _bf16(W)
    toks = tokens_for(config, n, seed=71)
    want = O.vabuzen_forward(config, W, toks)
    plain = O.keep_first_window_attention
    try:
        def without(q, k, v, scale, window, keep):  # no one in the denominator: scores lifted until it vanishes
            c = np.concatenate([q, np.ones_like(q[..., :1])], -1), np.concatenate([k, np.full_like(k[..., :1], 60.0 / scale)], -1)
            return plain(c[0], c[1], v, scale, window, keep)
        O.keep_first_window_attention = without
        assert rel_err(O.vabuzen_forward(config, W, toks)[-1:], want[-1:]) > 2 * TOL[dtype]
        def twice(q, k, v, scale, window, keep):    # a two in the denominator
            c = np.concatenate([q, np.ones_like(q[..., :1])], -1), np.concatenate([k, np.full_like(k[..., :1], -np.log(2.0) / scale)], -1)
            return plain(c[0], c[1], v, scale, window, keep)
        O.keep_first_window_attention = twice
        assert rel_err(O.vabuzen_forward(config, W, toks)[-1:], want[-1:]) > TOL[dtype]
    finally:
        O.keep_first_window_attention = plain
    engine = make_engine(config, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [n - 3, 1])[-3:], want[-3:], dtype)
    finally:
        engine.close()


def test_the_group_score_and_the_weights_of_the_router():
    """Groups by their largest expert, weights that are not divided by their sum, or a missing factor: each planted in the restatement moves the logits of many
    rows; the engine's (prompts, and decode steps that stream only the experts taken) do not move."""
    config = O.vabuzen_config([L_(mlp=M_(experts=12, top=3, ff=16, groups=(4, 2), scale=1.7))], logit_softcap=None)
    W = O.make_vabuzen_weights(config, seed=72)
    toks = tokens_for(config, 40, seed=73)
    want = reference(config, W, toks)
    plain = O.grouped_sigmoid_route

    def by_largest(z, top, count, keep, scale):
        s, per = O.sigmoid(z), len(z) // count
        kept = sorted(range(count), key=lambda g: -s[g * per:(g + 1) * per].max())[:keep]
        taken = sorted((j for j in range(len(z)) if j // per in kept), key=lambda j: -s[j])[:top]
        return {j: s[j] / sum(s[i] for i in taken) * scale for j in taken}, np.inf

    def not_renormalised(z, top, count, keep, scale):
        taken, margin = plain(z, top, count, keep, scale)
        return {j: O.sigmoid(z[j]) * scale for j in taken}, margin

    for wrong, share in ((by_largest, 0.1), (not_renormalised, 0.9), (lambda z, top, count, keep, scale: plain(z, top, count, keep, 1.0), 0.9)):
        O.grouped_sigmoid_route = wrong
        try:
            other = O.vabuzen_forward(config, W, toks)
        finally:
            O.grouped_sigmoid_route = plain
        assert np.mean([rel_err(other[i:i + 1], want[i:i + 1]) > 5 * TOL[torch.float32] for i in range(40)]) > share
    engine = make_engine(config, W)
    try:
        assert close(whole(engine, toks), want, torch.float32)
        assert close(in_portions(engine, toks, [1]), want, torch.float32)
        assert close(in_portions(engine, toks, [5]), want, torch.float32)
    finally:
        engine.close()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_first_tokens(dtype):
    """The first tokens of a sequence have few keys and no inputs before them: single tokens and portions of two from position 0."""
    W = O.make_vabuzen_weights(MIXED, seed=18)
    toks = tokens_for(MIXED, 12, seed=19)
    want = reference(MIXED, W, toks)
    engine = make_engine(MIXED, W, dtype)
    try:
        assert close(in_portions(engine, toks, [1, 1, 1, 2, 2, 5]), want, dtype)
        assert close(in_portions(engine, toks, [2]), want, dtype)
        assert not want.sure[0] or close(whole(engine, toks[:1]), np.asarray(want[:1]), dtype)
    finally:
        engine.close()


ODD = O.vabuzen_config([A_(heads=1, kv_heads=1, dim=12, vdim=20, conv=7, rot_dims=2, window=3, keep_first=1, mlp=M_(experts=3, top=1, ff=5, shared=3, groups=(1, 1), scale=0.3)),
                        L_(heads=3, dim=4, vdim=6, rot_dim=2, kv_rank=15, mlp={"kind": "dense", "ff": 11}),
                        A_(heads=5, kv_heads=5, dim=6, vdim=10, conv=1, rot_dims=6, window=7, keep_first=9, mlp=None)],
                       width=40, vocab=37, eps=1e-3, residual_mult=1.0, loop=(0, 2, 3), logit_softcap=1.5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_other_sizes(dtype):
    """Sizes that are no multiples of 8, one head, heads * vdim != width, a large eps, tiny windows, a convolution longer than they are, a residual factor of 1."""
    W = O.make_vabuzen_weights(ODD, seed=24)
    toks = tokens_for(ODD, 41, seed=25)
    want = reference(ODD, W, toks)
    engine = make_engine(ODD, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [5, 1, 2, 9]), want, dtype)
    finally:
        engine.close()


WIDE = O.vabuzen_config([A_(heads=4, kv_heads=2, dim=32, vdim=32, conv=3, rot_dims=32, window=90, keep_first=10, mlp={"kind": "dense", "ff": 256}),
                         L_(heads=8, dim=32, vdim=32, rot_dim=16, kv_rank=64, mlp=M_(experts=4, top=2, ff=64, shared=128, groups=(2, 1))),
                         A_(heads=8, kv_heads=2, dim=16, vdim=64, conv=4, rot_dims=8, window=128, keep_first=4, mlp=None),
                         L_(heads=4, dim=64, vdim=32, rot_dim=32, kv_rank=96, mlp={"kind": "dense", "ff": 128})],
                        width=128, vocab=200, loop=(1, 4, 2))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_large_chunks_of_rows(dtype):
    """From 192 rows the bfloat16 products run on the 256-wide tile GEMM and a branch's norm, sum, pass entry and next norm are a launch behind it; the same
    prompt in small portions (64-wide tiles, row kernel: the tail rides the product) must give the same logits."""
    W = O.make_vabuzen_weights(WIDE, seed=26)
    toks = tokens_for(WIDE, 300, seed=27)
    want = reference(WIDE, W, toks)
    engine = make_engine(WIDE, W, dtype, page_size=64, num_pages=8, max_batch=2)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [250, 3, 40, 1]), want, dtype)
    finally:
        engine.close()


def test_long_greedy_decoding_on_the_device_and_graph_replays():
    """160 greedy steps through the captured decode step (across window and page borders); the ids are the float64 restatement's greedy
    choices, and replaying the graph gives what eager launches give."""
    W = O.make_vabuzen_weights(MIXED, seed=28)
    prompt = tokens_for(MIXED, 21, seed=29)
    engine = make_engine(MIXED, W, page_size=16, num_pages=16, max_batch=2)
    try:
        ids = engine.generate(prompt, 161, slot=1)
        assert engine.stats()["graph_replays"] >= 160
        full = prompt + ids
        ref = O.vabuzen_forward(MIXED, W, full[:-1])
        for k, tok in enumerate(ids):
            row = ref[len(prompt) - 1 + k]
            assert row[tok] >= row.max() - 1e-3 * np.abs(row).max(), f"generated token {k}"
        engine.begin(0)
        engine.prefill(0, prompt)
        engine.decode(40, slots=[0], use_graph=False)
        assert engine.read_tokens(0, 41) == ids[:41]
        engine.release(0)
    finally:
        engine.close()


@pytest.mark.parametrize("mixed", [True, False])
def test_greedy_generation_through_the_scheduler(mixed):
    """engine.batch_generate_ids (continuous batching: chunked prefill in a staging slot, adoption into decode slots, retirement):
    every request's ids are what the request alone generates."""
    from tiny_llm_hip.engine import batch_generate_ids

    W = O.make_vabuzen_weights(MIXED, seed=30)
    prompts = [tokens_for(MIXED, n, seed=30 + n) for n in (5, 23, 40, 9, 31)]
    limits = [12, 7, 9, 15, 4]
    engine = make_engine(MIXED, W, page_size=16, num_pages=40, max_batch=4, max_prefill_rows=64)
    try:
        alone = [engine.generate(p, n, slot=0) for p, n in zip(prompts, limits)]
        done = dict(batch_generate_ids(engine, prompts, limits, batch_size=3, prefill_step=16, mixed_steps=mixed))
        assert sorted(done) == list(range(5))
        for i in range(5):
            assert done[i] == alone[i], f"request {i}"
        assert engine.stats()["pages_in_use"] == 0
    finally:
        engine.close()


def _save(tmp_path, config, W):
    from safetensors.torch import save_file

    tmp_path.mkdir(exist_ok=True)
    (tmp_path / "config.json").write_text(json.dumps(config))
    save_file({k: torch.from_numpy(np.asarray(v, dtype=np.float32)).to(torch.bfloat16) for k, v in W.items()}, str(tmp_path / "model.safetensors"))


def test_checkpoint_directory_through_loader_registry_and_command_line(tmp_path):
    W = O.make_vabuzen_weights(MIXED, seed=31)
    _save(tmp_path, MIXED, W)
    from tiny_llm_hip import load
    from tiny_llm_hip.models import engine_for

    model, tokenizer = load(str(tmp_path))
    assert tokenizer is None and model.family == "Vabuzen"
    prompt = tokens_for(MIXED, 11, seed=32)
    engine = engine_for(model, dtype=torch.float32, page_size=16, num_pages=8, max_batch=1, max_prefill_rows=32)
    try:
        want = engine.generate(prompt, 6)
    finally:
        engine.close()
    import main as cli

    out = cli.main(["--model", str(tmp_path), "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "6", "--dtype", "float32"])
    assert [int(t) for t in out.split()] == want
    out = cli.main(["--model", str(tmp_path), "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "6", "--dtype", "float32",
                    "--sampler-temp", "1e-4", "--sampler-top-k", "1"])
    assert [int(t) for t in out.split()] == want


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_command_line(tmp_path, dtype):
    """bin/trace_run on a checkpoint directory: two requests share steps, one ends, and its slot and pages serve a third."""
    import subprocess
    import sys
    from pathlib import Path

    W = O.make_vabuzen_weights(MIXED, seed=33)
    model_dir, out_dir = tmp_path / "model", tmp_path / "out"
    _save(model_dir, MIXED, W)
    long, short, third = (tokens_for(MIXED, n, seed=34 + n) for n in (150, 30, 50))
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": long[:100], "want": [0, 99]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": long[100:149], "want": []}, {"id": "y", "tokens": short[:29], "want": [28]}], "end": []},
             {"step": 2, "entries": [{"id": "y", "tokens": short[29:], "want": [0]}, {"id": "x", "tokens": long[149:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [], "end": []},
             {"step": 4, "entries": [{"id": "z", "tokens": third, "want": [49, 3]}, {"id": "y", "tokens": [5], "want": []}], "end": ["y", "z"]}]
    root = Path(__file__).resolve().parent.parent
    run = subprocess.run([sys.executable, str(root / "bin" / "trace_run"), "--model", str(model_dir), "--dtype", dtype, "--out", str(out_dir),
                          "--max-tokens", str(192 + 64), "--slots", "2"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                         capture_output=True, text=True, timeout=110)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    ref_long, ref_short, ref_third = (O.vabuzen_forward(MIXED, W, t) for t in (long, short, third))
    got = {i: np.fromfile(out_dir / f"{i}.f32", dtype="<f4").reshape(-1, MIXED["vocab"]) for i in (0, 1, 2, 4)}
    tol = TOL[torch.float32 if dtype == "float32" else torch.bfloat16]
    assert rel_err(got[0], ref_long[[0, 99]]) < tol
    assert rel_err(got[1], ref_short[[28]]) < tol
    assert rel_err(got[2], np.stack([ref_short[29], ref_long[149]])) < tol
    assert rel_err(got[4], ref_third[[49, 3]]) < tol
