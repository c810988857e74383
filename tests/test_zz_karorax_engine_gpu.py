"""GPU tier: the Karorax family on the layer-list engine against the plain float64 restatement in tests/layer_list_oracle.py, on
small made-up configurations with random (or crafted) weights: a token-pair embedding, sequential blocks with layer scales, latent
attention with direct queries (sliding window, learned sinks, one gate per head, another layer's cache), two mixers side by side
(capped attention with a distance bias and a query temperature; lightning attention), squared-ReLU feed-forwards, experts weighted
by a softmax over the chosen logits beside a shared one, capped logits.

float32 runs are held to a relative RMS error of 2e-4 per logits row, bfloat16 runs to 4e-2 (layer_list_engine_helpers.TOL).
"""

import json

import numpy as np
import pytest
import torch

import layer_list_oracle as O
from layer_list_engine_helpers import TOL, in_portions, make_engine, rel_err, tokens_for, whole

pytestmark = pytest.mark.gpu

# six layers: windows of 20, 20 (the first one's cache) and 37; two parallel layers of different sizes; every kind of feed-forward and none
MIXED = O.karorax_config([O.karorax_parallel_layer(),
                          O.karorax_latent_layer(),
                          O.karorax_latent_layer(heads=6, dim=8, vdim=12, window=29, kv_from=1, mlp=None),
                          O.karorax_parallel_layer(heads=6, kv_heads=3, dim=24, vdim=8, softcap=9.0, coef=0.5, every=7, right_heads=2, right_dim=20, right_vdim=28,
                                                   decay=[0.9, 0.999], mlp=O.karorax_moe(experts=4, top=3, ff=16, shared=0)),
                          O.karorax_latent_layer(heads=2, dim=24, vdim=16, rot_dim=12, kv_rank=24, window=37, mlp={"kind": "dense", "ff": 50}),
                          O.karorax_parallel_layer(mlp=None)])

LAYERS = {
    "latent": O.karorax_latent_layer(),
    "latent_no_feed_forward": O.karorax_latent_layer(mlp=None),
    "latent_no_window": O.karorax_latent_layer(window=0),
    "latent_window_of_one": O.karorax_latent_layer(window=1),
    "latent_window_across_pages": O.karorax_latent_layer(window=23),
    "latent_no_rotation": O.karorax_latent_layer(rot_dim=0),
    "latent_one_head": O.karorax_latent_layer(heads=1, dim=24, vdim=8, rot_dim=4, kv_rank=12),
    "latent_many_heads": O.karorax_latent_layer(heads=20, dim=8, vdim=8, rot_dim=4, kv_rank=16),
    "latent_odd_sizes": O.karorax_latent_layer(heads=5, dim=10, vdim=9, rot_dim=6, kv_rank=21, window=11, mlp={"kind": "dense", "ff": 13}),
    "latent_rank_of_the_middle_tile": O.karorax_latent_layer(heads=3, dim=16, vdim=16, rot_dim=16, kv_rank=104, window=33),
    "latent_wide": O.karorax_latent_layer(heads=2, dim=72, vdim=40, rot_dim=64, kv_rank=192, window=31),
    "latent_wider": O.karorax_latent_layer(heads=3, dim=16, vdim=16, rot_dim=16, kv_rank=240, window=0),
    "latent_wide_odd": O.karorax_latent_layer(heads=2, dim=16, vdim=16, rot_dim=10, kv_rank=150),
    "latent_widest": O.karorax_latent_layer(heads=2, dim=16, vdim=16, rot_dim=8, kv_rank=264),
    "parallel": O.karorax_parallel_layer(),
    "parallel_no_feed_forward": O.karorax_parallel_layer(mlp=None),
    "parallel_as_many_kv_heads": O.karorax_parallel_layer(heads=3, kv_heads=3, dim=8, vdim=8),
    "parallel_one_kv_head": O.karorax_parallel_layer(heads=6, kv_heads=1),
    "parallel_one_head": O.karorax_parallel_layer(heads=1, kv_heads=1, dim=32, vdim=40, right_heads=1, right_dim=8, right_vdim=8, decay=[1.0]),
    "parallel_large_group": O.karorax_parallel_layer(heads=20, kv_heads=1, dim=8, vdim=8),
    "parallel_wide_heads": O.karorax_parallel_layer(heads=2, kv_heads=1, dim=128, vdim=96, right_heads=1, right_dim=96, right_vdim=128, decay=[0.98]),
    "parallel_widest_heads": O.karorax_parallel_layer(heads=2, kv_heads=2, dim=136, vdim=72, right_heads=2, right_dim=160, right_vdim=40),
    "parallel_odd_sizes": O.karorax_parallel_layer(heads=6, kv_heads=2, dim=10, vdim=13, right_heads=5, right_dim=9, right_vdim=7, mlp={"kind": "dense", "ff": 9}),
    "parallel_no_cap": O.karorax_parallel_layer(softcap=None),
    "parallel_tight_cap": O.karorax_parallel_layer(softcap=0.5, scale=1.0),
    "parallel_temperature_every_token": O.karorax_parallel_layer(coef=0.8, every=1),
    "parallel_no_temperature": O.karorax_parallel_layer(coef=0.0),
    "parallel_temperature_of_a_long_period": O.karorax_parallel_layer(every=1000),
    "parallel_factors_of_one": O.karorax_parallel_layer(left_scale=1.0, right_scale=1.0),
    "parallel_left_only": O.karorax_parallel_layer(right_scale=0.0),
    "parallel_right_only": O.karorax_parallel_layer(left_scale=0.0),
    "parallel_negative_factor": O.karorax_parallel_layer(left_scale=-0.7),
    "lightning_fast_decay": O.karorax_parallel_layer(decay=[0.5, 0.2, 0.01]),
    "lightning_many_heads": O.karorax_parallel_layer(right_heads=24, right_dim=8, right_vdim=8),
    "lightning_wide": O.karorax_parallel_layer(right_heads=2, right_dim=128, right_vdim=136),
    "experts_one_of_one": O.karorax_parallel_layer(mlp=O.karorax_moe(experts=1, top=1, ff=16, shared=0)),
    "experts_all_taken": O.karorax_parallel_layer(mlp=O.karorax_moe(experts=4, top=4, ff=16)),
    "experts_one_taken": O.karorax_latent_layer(mlp=O.karorax_moe(experts=7, top=1, ff=16)),
    "experts_no_shared": O.karorax_latent_layer(mlp=O.karorax_moe(experts=5, top=2, ff=32, shared=0)),
    "experts_many": O.karorax_latent_layer(mlp=O.karorax_moe(experts=70, top=3, ff=8, shared=16)),
    "experts_odd_sizes": O.karorax_latent_layer(mlp=O.karorax_moe(experts=3, top=2, ff=9, shared=13)),
}


class Reference(np.ndarray):
    """Logits of the restatement; ``sure`` marks the rows whose experts no rounding of the router's input can exchange."""


def reference(config, W, toks, streams=None):
    margins = []
    out = O.karorax_forward(config, W, toks, streams, margins).view(Reference)
    out.sure = np.all(np.stack(margins) > 0.05, 0) if margins else np.ones(len(toks), dtype=bool)
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
    config = O.karorax_config([LAYERS[layer]])
    W = O.make_karorax_weights(config, seed=3)
    toks = tokens_for(config, 53, seed=4)
    want = reference(config, W, toks)
    engine = make_engine(config, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [19, 1, 1, 6, 1]), want, dtype)
    finally:
        engine.close()


@pytest.mark.parametrize("bigram,cap", [(None, 0), ((1, 1, 1), 2.0), ((7, 0, 3), 0), ((211, 104729, 1299709), 30.0)])
def test_token_pairs_and_capped_logits(bigram, cap):
    """No pair table, one bucket, a hash that ignores the token before, large factors; logits with and without a cap."""
    config = O.karorax_config([O.karorax_latent_layer(), O.karorax_parallel_layer()], bigram=bigram, logit_softcap=cap)
    W = O.make_karorax_weights(config, seed=40)
    toks = tokens_for(config, 38, seed=41)
    want = reference(config, W, toks)
    engine = make_engine(config, W)
    try:
        assert close(whole(engine, toks), want, torch.float32)
        assert close(in_portions(engine, toks, [7, 1, 2]), want, torch.float32)
        assert close(in_portions(engine, toks, [1]), want, torch.float32)
    finally:
        engine.close()


def test_the_token_before_a_portion_is_the_sequences_own():
    """A pair table whose rows stand far apart: the first token of every portion needs the last token of the portion before, of the same
    sequence -- beside another sequence in the same steps, in a slot that held a third one, and across device-side decode steps."""
    config = O.karorax_config([O.karorax_parallel_layer(mlp=None)], bigram=(29, 7, 4))
    W = O.make_karorax_weights(config, seed=42)
    W["bigram"] *= 6.0
    a, b, c = (tokens_for(config, n, seed=43 + n) for n in (21, 20, 16))
    wa, wb, wc = (O.karorax_forward(config, W, t) for t in (a, b, c))
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
        # decode steps on the device between packed steps; the sequence then changes its slot
        engine.set_token(0, 5)
        engine.decode(1, slots=[0])
        nxt = engine.read_pending_slots([0])[0]
        engine.decode(1, slots=[0], use_graph=False)
        engine.move(0, 3)
        full = a + [5, nxt, 9]
        want = O.karorax_forward(config, W, full)
        assert close(engine.logits_host(engine.step([(3, [9], [0])])), want[-1:], torch.float32)
    finally:
        engine.close()


def test_width_and_vocabulary_that_are_no_multiples_of_8():
    config = O.karorax_config([O.karorax_parallel_layer(), O.karorax_latent_layer(mlp=None)], width=52, vocab=77)
    W = O.make_karorax_weights(config, seed=60)
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
    with the same window, sinks, cap and distance bias."""
    monkeypatch.setenv("TL_HYBRID_ATTN_ROWS", "1")
    W = O.make_karorax_weights(MIXED, seed=62)
    toks = tokens_for(MIXED, 70, seed=63)
    want = reference(MIXED, W, toks)
    engine = make_engine(MIXED, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [33, 1]), want, dtype)
    finally:
        engine.close()


def test_stream_after_every_layer():
    W = O.make_karorax_weights(MIXED, seed=5)
    toks = tokens_for(MIXED, 29, seed=6)
    streams = []
    want = reference(MIXED, W, toks, streams)
    engine = make_engine(MIXED, W)
    try:
        assert engine.stats()["layer_runs"] == len(streams) == 6
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
    W = O.make_karorax_weights(MIXED, seed=7)
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
    """Portions end inside pages (16 tokens) and inside windows (20, 29 and 37 positions); the recurrent state is carried across every cut."""
    W = O.make_karorax_weights(MIXED, seed=9)
    toks = tokens_for(MIXED, 150, seed=10)
    engine = make_engine(MIXED, W)
    try:
        assert rel_err(in_portions(engine, toks, sizes), reference(MIXED, W, toks)) < TOL[torch.float32]
    finally:
        engine.close()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_unequal_requests_in_one_batch_against_each_alone(dtype):
    """Portions of some requests beside single tokens of others; every request's rows must equal its whole-sequence logits."""
    W = O.make_karorax_weights(MIXED, seed=11)
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
    read, and a slot's recurrent state starts at zero again."""
    W = O.make_karorax_weights(MIXED, seed=12)
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


def _bf16(W):
    for k in W:
        W[k] = torch.from_numpy(np.asarray(W[k], dtype=np.float32)).to(torch.bfloat16).float().numpy()


def _needle_latent(window, kv_rank=24, shared=False):
    """B's query reads the channel only B excites, latent 0 of the cache the one only A excites, and one unrotated dimension of every head joins
    them: where A is among the keys B sees, the score of (B, A) towers over the others and over the sinks, so a lost, shifted or doubled key -- or
    a window that is one position off -- changes the logits at B by far more than the tolerance.  shared: the layer that answers reads the cache
    of a layer before it, whose own result is scaled away."""
    layer = lambda kv_from: O.karorax_latent_layer(heads=2, dim=16, vdim=16, rot_dim=8, kv_rank=kv_rank, scale=0.5, window=window, kv_from=kv_from, mlp=None)
    config = O.karorax_config([layer(None), layer(0)] if shared else [layer(None)], width=64, vocab=50, bigram=None, logit_softcap=None)
    W = O.make_karorax_weights(config, seed=16)
    A, B = 48, 49
    _quiet(W, A, B)
    W["l0.mix.dkv"][:, 0] = 0.0
    W["l0.mix.dkv"][0, :] = 0.0
    W["l0.mix.dkv"][0, 0] = 6.0
    W["l0.mix.dkv.norm"][:] = 1.0
    for m in ("l0.mix.", "l1.mix.") if shared else ("l0.mix.",):
        W[m + "q"][:, 1] = 0.0
        W[m + "uk"][:, 0] = 0.0
        for h in range(2):
            W[m + "q"][h * 24, :] = 0.0
            W[m + "q"][h * 24, 1] = 6.0
            W[m + "uk"][h * 16, :] = 0.0
            W[m + "uk"][h * 16, 0] = 3.0
        W[m + "uv"][:, 0] += 1.0
    if shared:
        W["l0.ls1"][:] = 0.0
    _bf16(W)
    return config, W, A, B


def _needle_left():
    """Capped attention without a window: the score of (B, A) reaches the cap, every other stays small; 8 heads whose distance slopes reach down to
    2^-8, so that the key still wins from a few hundred positions back.  The other mixer is scaled away."""
    config = O.karorax_config([O.karorax_parallel_layer(heads=8, kv_heads=4, dim=16, vdim=16, scale=0.5, softcap=30.0, coef=0.1, every=50, right_scale=0.0, mlp=None)],
                              width=64, vocab=50, bigram=None, logit_softcap=None)
    W = O.make_karorax_weights(config, seed=15)
    A, B = 48, 49
    _quiet(W, A, B)
    m = "l0.mix.left."
    for name, heads, channel in (("k", 4, 0), ("q", 8, 1)):
        W[m + name] *= 0.3
        W[m + name][:, channel] = 0.0
        for h in range(heads):
            W[m + name][h * 16 + 8, :] = 0.0
            W[m + name][h * 16 + 8, channel] = 6.0
    W[m + "v"][:, 0] += 1.0
    _bf16(W)
    return config, W, A, B


def _needle_right():
    """Lightning attention keeps no history but its state: with decays of 1 and 0.999 the outer product that A left long ago answers B's query, so a
    state that was lost, reset, or carried over from another sequence shows at B.  The other mixer is scaled away."""
    config = O.karorax_config([O.karorax_parallel_layer(right_heads=2, right_dim=16, right_vdim=16, decay=[1.0, 0.999], left_scale=0.0, mlp=None)],
                              width=64, vocab=50, bigram=None, logit_softcap=None)
    W = O.make_karorax_weights(config, seed=17)
    A, B = 48, 49
    _quiet(W, A, B)
    m = "l0.mix.right."
    for name, channel in (("k", 0), ("q", 1)):
        W[m + name] *= 0.1
        W[m + name][:, channel] = 0.0
        for h in range(2):
            W[m + name][h * 16 + 12, :] = 0.0
            W[m + name][h * 16 + 12, channel] = 6.0
    W[m + "v"][:, 0] += 1.0
    _bf16(W)
    return config, W, A, B


def _needle_prompt(config, A, B, n, needle_at, seed):
    toks = tokens_for(config, n, seed=seed, avoid=(A, B))
    toks[needle_at] = A
    toks[-1] = B
    return toks


def _needle_case(config, W, A, B, n, needle_at, query, seen, **pool):
    toks = _needle_prompt(config, A, B, n, needle_at, 16)
    want = O.karorax_forward(config, W, toks)[-1]
    other = list(toks)
    other[needle_at] = toks[needle_at - 1] if needle_at else toks[1]
    moved = rel_err(O.karorax_forward(config, W, other)[-1][None], want[None])
    assert (moved > 0.2) if seen else (moved < 1e-9)   # the needle decides the answer exactly where the mask lets B see it
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
@pytest.mark.parametrize("mixer", ["latent", "latent_shared_cache", "latent_wide", "left", "right"])
def test_far_keys_and_page_borders(mixer, needle_at, query):
    """No window: the last token sees every key; the needle sits far back, at page borders (16) and key-tile borders (64).  At 300 tokens
    a decoded token's key range is split over workgroups."""
    config, W, A, B = {"latent": lambda: _needle_latent(0), "latent_shared_cache": lambda: _needle_latent(0, shared=True),
                       "latent_wide": lambda: _needle_latent(0, kv_rank=192), "left": _needle_left, "right": _needle_right}[mixer]()
    _needle_case(config, W, A, B, 300, needle_at, query, True, page_size=16, num_pages=24, max_batch=1)


@pytest.mark.parametrize("needle_at,seen", [(191, False), (192, True), (193, True), (207, True), (208, True), (254, True), (127, False), (0, False)])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
@pytest.mark.parametrize("kv_rank,shared", [(24, False), (24, True), (192, False)])
def test_keys_just_inside_and_just_outside_a_window(needle_at, seen, query, kv_rank, shared):
    """A window of 64 positions over pages of 16: the query at position 255 sees 192 .. 255 and nothing before."""
    config, W, A, B = _needle_latent(64, kv_rank, shared)
    _needle_case(config, W, A, B, 256, needle_at, query, seen, page_size=16, num_pages=24, max_batch=1)


@pytest.mark.parametrize("n,needle_at,seen", [(101, 0, False), (101, 1, True), (150, 49, False), (150, 50, True), (201, 100, False), (201, 101, True),
                                              (450, 349, False), (450, 350, True), (450, 383, True), (450, 384, True), (450, 448, True), (100, 0, True), (60, 0, True)])
@pytest.mark.parametrize("query", ["prompt", "decoded"])
@pytest.mark.parametrize("kv_rank", [24, 136])
def test_window_edges_that_are_no_page_or_tile_edges(n, needle_at, seen, query, kv_rank):
    """A window of 100 positions: its edge falls inside pages and inside the kernels' 64-key tiles, and moves with every query."""
    config, W, A, B = _needle_latent(100, kv_rank)
    _needle_case(config, W, A, B, n, needle_at, query, seen, page_size=16, num_pages=30, max_batch=1)


@pytest.mark.parametrize("n,needle_at,seen", [(700, 399, False), (700, 400, True), (700, 401, True), (700, 463, True), (700, 464, True), (700, 650, True), (320, 19, False),
                                              (320, 20, True), (280, 0, True)])
@pytest.mark.parametrize("kv_rank", [24, 192])
def test_wide_window_of_a_decoded_token_over_split_key_ranges(n, needle_at, seen, kv_rank):
    """A window of 300 positions in a long context: the decoded token's keys are split over workgroups, counted from the window's first key."""
    config, W, A, B = _needle_latent(300, kv_rank)
    _needle_case(config, W, A, B, n, needle_at, "decoded", seen, page_size=64, num_pages=12, max_batch=1, max_prefill_rows=1024)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [40, 400])
def test_a_sink_counts_once(n, dtype):
    """Sinks that hold half of the weight and more, alone in a window of few keys and over split key ranges (decoding at 400 tokens): a sink that is
    left out, scaled with the scores or counted once per split moves the logits by far more than the tolerance."""
    config = O.karorax_config([O.karorax_latent_layer(heads=4, window=0, mlp=None, scale=0.05)], bigram=None, logit_softcap=None)
    W = O.make_karorax_weights(config, seed=70)
    W["l0.mix.sink"] = np.log(n) + np.array([0.0, 1.0, 2.0, -1.0], dtype=np.float32)
    W["embed"][:, 2] = 3.0                 # a channel every token excites: latent 0 is common to all keys, and so are the values' means
    W["l0.mix.dkv"][0] = 0.0
    W["l0.mix.dkv"][0, 2] = 2.0
    W["l0.mix.uv"][:, 0] = np.where(np.arange(96) % 2, 0.5, -0.5)
    W["l0.mix.g"][:] = 0.0
    W["l0.ls1"][:] = 2.0
    _bf16(W)
    toks = tokens_for(config, n, seed=71)
    want = O.karorax_forward(config, W, toks)
    for shift in (-50.0, np.log(2.0)):
        other = dict(W)
        other["l0.mix.sink"] = W["l0.mix.sink"] + shift
        assert rel_err(O.karorax_forward(config, other, toks)[-1:], want[-1:]) > 2 * TOL[dtype]
    engine = make_engine(config, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [n - 3, 1])[-3:], want[-3:], dtype)
    finally:
        engine.close()


@pytest.mark.parametrize("n", [70, 300])
def test_distance_bias_and_query_temperature_by_position(n):
    """One head with a slope of 2^-8 among eight, temperatures that step at every 16th position: a bias on the key's position alone (not the distance),
    a temperature one position late, or one read from the portion instead of the sequence shows against the restatement with that mistake planted in it."""
    config = O.karorax_config([O.karorax_parallel_layer(heads=8, kv_heads=2, softcap=2.0, coef=2.0, every=16, scale=0.6, right_scale=0.0, mlp=None)], bigram=None, logit_softcap=None)
    W = O.make_karorax_weights(config, seed=72)
    toks = tokens_for(config, n, seed=73)
    want = O.karorax_forward(config, W, toks)
    late = O.query_temperature
    try:
        O.query_temperature = lambda pos, coef, every: late(np.asarray(pos) - 1, coef, every)
        planted = O.karorax_forward(config, W, toks)
        at = [i for i in range(n) if i % 16 == 15]
        assert np.median([rel_err(planted[i:i + 1], want[i:i + 1]) for i in at]) > 5 * TOL[torch.float32]
    finally:
        O.query_temperature = late
    engine = make_engine(config, W)
    try:
        assert close(whole(engine, toks), want, torch.float32)
        assert close(in_portions(engine, toks, [15, 1, 1, 14, 17]), want, torch.float32)
        assert close(in_portions(engine, toks, [n - 12, 1])[-12:], want[-12:], torch.float32)
    finally:
        engine.close()


def test_the_head_norm_gate_and_heads_of_lightning_attention_are_one_row():
    """One head's values stand out: the norm over all heads together shrinks the others (a norm per head would not), and the gate is a sigmoid of
    every channel's own number."""
    config = O.karorax_config([O.karorax_parallel_layer(left_scale=0.0, mlp=None)], bigram=None, logit_softcap=None)
    W = O.make_karorax_weights(config, seed=74)
    W["l0.mix.right.v"][:16] *= 8.0
    W["l0.mix.right.g"] *= 4.0
    _bf16(W)
    toks = tokens_for(config, 40, seed=75)
    want = reference(config, W, toks)
    engine = make_engine(config, W)
    try:
        assert close(whole(engine, toks), want, torch.float32)
        assert close(in_portions(engine, toks, [5, 1]), want, torch.float32)
    finally:
        engine.close()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_first_tokens(dtype):
    """The first tokens of a sequence have few keys and an empty state: single tokens and portions of two from position 0."""
    W = O.make_karorax_weights(MIXED, seed=18)
    toks = tokens_for(MIXED, 12, seed=19)
    want = reference(MIXED, W, toks)
    engine = make_engine(MIXED, W, dtype)
    try:
        assert close(in_portions(engine, toks, [1, 1, 1, 2, 2, 5]), want, dtype)
        assert close(in_portions(engine, toks, [2]), want, dtype)
        assert not want.sure[0] or close(whole(engine, toks[:1]), np.asarray(want[:1]), dtype)
    finally:
        engine.close()


ODD = O.karorax_config([O.karorax_latent_layer(heads=1, dim=12, vdim=20, rot_dim=2, kv_rank=15, window=3, mlp=None),
                        O.karorax_parallel_layer(heads=5, kv_heads=5, dim=6, vdim=10, softcap=0.7, coef=1.5, every=3, right_heads=1, right_dim=24, right_vdim=40, decay=[0.75],
                                                 mlp=O.karorax_moe(experts=2, top=1, ff=5, shared=3)),
                        O.karorax_latent_layer(heads=3, dim=4, vdim=6, rot_dim=2, kv_rank=15, window=7, kv_from=0, mlp={"kind": "dense", "ff": 11})],
                       width=40, vocab=37, eps=1e-3, bigram=(3, 2, 1), logit_softcap=1.5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_other_sizes(dtype):
    """Sizes that are no multiples of 8, one head, heads * vdim != width, a large eps, tiny windows, a tight cap on scores and logits, a table of three buckets."""
    W = O.make_karorax_weights(ODD, seed=24)
    toks = tokens_for(ODD, 41, seed=25)
    want = reference(ODD, W, toks)
    engine = make_engine(ODD, W, dtype)
    try:
        assert close(whole(engine, toks), want, dtype)
        assert close(in_portions(engine, toks, [5, 1, 2, 9]), want, dtype)
    finally:
        engine.close()


WIDE = O.karorax_config([O.karorax_parallel_layer(heads=4, kv_heads=2, dim=32, vdim=32, right_heads=4, right_dim=32, right_vdim=32, mlp={"kind": "dense", "ff": 256}),
                         O.karorax_latent_layer(heads=8, dim=32, vdim=32, rot_dim=16, kv_rank=64, window=128, mlp=O.karorax_moe(experts=4, top=2, ff=64, shared=128)),
                         O.karorax_latent_layer(heads=8, dim=32, vdim=32, rot_dim=16, kv_rank=64, window=70, kv_from=1, mlp={"kind": "dense", "ff": 128}),
                         O.karorax_parallel_layer(heads=8, kv_heads=2, dim=16, vdim=64, right_heads=2, right_dim=16, right_vdim=64, mlp=O.karorax_moe(experts=8, top=2, ff=32, shared=64))],
                        width=128, vocab=200)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_large_chunks_of_rows(dtype):
    """From 192 rows the bfloat16 products run on the 256-wide tile GEMM (layer scales in its epilogue); the same prompt in small
    portions (64-wide tiles, row kernel) must give the same logits."""
    W = O.make_karorax_weights(WIDE, seed=26)
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
    W = O.make_karorax_weights(MIXED, seed=28)
    prompt = tokens_for(MIXED, 21, seed=29)
    engine = make_engine(MIXED, W, page_size=16, num_pages=16, max_batch=2)
    try:
        ids = engine.generate(prompt, 161, slot=1)
        assert engine.stats()["graph_replays"] >= 160
        full = prompt + ids
        ref = O.karorax_forward(MIXED, W, full[:-1])
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

    W = O.make_karorax_weights(MIXED, seed=30)
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
    W = O.make_karorax_weights(MIXED, seed=31)
    _save(tmp_path, MIXED, W)
    from tiny_llm_hip import load
    from tiny_llm_hip.models import engine_for

    model, tokenizer = load(str(tmp_path))
    assert tokenizer is None and model.family == "Karorax"
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

    W = O.make_karorax_weights(MIXED, seed=33)
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
    ref_long, ref_short, ref_third = (O.karorax_forward(MIXED, W, t) for t in (long, short, third))
    got = {i: np.fromfile(out_dir / f"{i}.f32", dtype="<f4").reshape(-1, MIXED["vocab"]) for i in (0, 1, 2, 4)}
    tol = TOL[torch.float32 if dtype == "float32" else torch.bfloat16]
    assert rel_err(got[0], ref_long[[0, 99]]) < tol
    assert rel_err(got[1], ref_short[[28]]) < tol
    assert rel_err(got[2], np.stack([ref_short[29], ref_long[149]])) < tol
    assert rel_err(got[4], ref_third[[49, 3]]) < tol
