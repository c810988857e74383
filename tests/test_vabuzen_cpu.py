"""CPU tier of the Vabuzen family: the config reader, the tensor table, the engine's packed layout, the loader's checks, and the
float64 restatement (tests/layer_list_oracle.py) held against itself -- each mechanism against a second, differently written form."""

import json

import numpy as np
import pytest
import torch

import layer_list_oracle as O
from tiny_llm_hip.layer_list import FAMILIES, pack_layer_list

CONFIG = O.vabuzen_config([
    O.vabuzen_attention_layer(heads=6, kv_heads=3, dim=12, vdim=8, conv=5, rot_dims=4, base=700.0, scale=0.21, window=7, keep_first=2, mlp={"kind": "dense", "ff": 20}),
    O.vabuzen_latent_layer(heads=2, dim=20, vdim=12, rot_dim=6, kv_rank=28, base=900.0, scale=0.11, mlp=O.vabuzen_moe(experts=9, top=4, ff=10, shared=14, groups=(3, 2), scale=2.5)),
    O.vabuzen_attention_layer(heads=2, kv_heads=2, dim=8, vdim=24, conv=1, rot_dims=8, window=1, keep_first=0, mlp=None),
    O.vabuzen_latent_layer(mlp=O.vabuzen_moe(experts=4, top=1, ff=6, shared=0, groups=(4, 1))),
], width=48, vocab=61, eps=2e-5, residual_mult=0.6, loop=(1, 3, 3), logit_softcap=9.0)


def test_config_reader_takes_every_size_and_constant_from_the_file():
    read, table = FAMILIES["Vabuzen"]
    cfg = read(CONFIG)
    assert (cfg.family, cfg.block, cfg.norm_kind, cfg.width, cfg.vocab, cfg.norm_eps, cfg.residual_mult, cfg.loop, cfg.logit_softcap) == \
        ("Vabuzen", "sandwich", "dyt", 48, 61, 2e-5, 0.6, (1, 3, 3), 9.0)
    assert cfg.loop_add_embed and not cfg.loop_projection and not cfg.layer_scale and not cfg.embed_norm and cfg.layer_runs == 4 + 2 * 2
    a, l, b, m = cfg.layers
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.conv_taps, a.rot_dims, a.rot_base, a.rot_half, a.scale, a.window, a.keep_first, a.sink, a.learned_sink) == \
        ("attention", 6, 3, 12, 8, 5, 4, 700.0, False, 0.21, 7, 2, True, False)
    assert not a.gated and not a.bias and not a.qk_head_norm and not a.qk_unit_rms
    assert (a.ff, a.ff_kind, a.ff_act, a.ff_bias) == (20, "plain", "gelu_tanh", True)
    assert (l.kind, l.heads, l.dim, l.vdim, l.q_rank, l.kv_rank, l.rot_dim, l.rot_dims, l.rot_base, l.rot_half, l.scale, l.gated, l.sink, l.window) == \
        ("latent", 2, 20, 12, 0, 28, 6, 6, 900.0, True, 0.11, False, False, 0)
    assert (l.ff, l.ff_kind, l.ff_act, l.experts, l.top, l.groups, l.keep, l.expert_ff, l.shared_ff, l.router, l.moe_gated, l.ff_bias) == \
        (14 + 9 * 10, "moe", "silu", 9, 4, 3, 2, 10, 14, "sigmoid", True, False)
    assert (l.moe_group_score, l.moe_renorm, l.moe_scale, l.moe_shared_sg, l.moe_correction) == ("top2", True, 2.5, False, False)
    assert (b.conv_taps, b.window, b.keep_first, b.ff) == (1, 1, 0, 0) and (m.groups, m.keep, m.shared_ff) == (4, 1, 0)
    names = table(cfg)
    assert names["l0.mix.q"] == (72, 48) and names["l0.mix.k.conv"] == (36, 5) and names["l0.mix.v.conv"] == (24, 5) and names["l0.mix.o"] == (48, 48)
    assert names["l0.norm1b.alpha"] == () and names["l0.norm2b.b"] == (48,) and names["l0.mlp.up.b"] == (20,) and names["l0.mlp.down.b"] == (48,)
    assert names["l1.mix.q"] == (2 * 26, 48) and names["l1.mix.dkv"] == (34, 48) and names["l1.mix.dkv.norm"] == (28,) and names["l1.mlp.router"] == (9, 48)
    assert names["loop.step"] == (3, 48) and "loop.in" not in names and "l2.norm2" not in names and "l3.mlp.shared.up" not in names and names["final.norm.alpha"] == ()
    assert set(names) == set(O.make_vabuzen_weights(CONFIG))
    plain = {k: v for k, v in CONFIG.items() if k not in ("loop", "logit_softcap")}
    cfg2 = read(plain)
    assert cfg2.loop is None and cfg2.logit_softcap == 0.0 and "loop.step" not in table(cfg2)
    moe = lambda **kw: {**CONFIG, "layers": [O.vabuzen_latent_layer(mlp=O.vabuzen_moe(**kw))], "loop": None}
    for bad in ({**CONFIG, "layers": [dict(CONFIG["layers"][0], type="delta")]}, {k: v for k, v in CONFIG.items() if k != "residual_mult"},
                {**CONFIG, "loop": {"start": 2, "stop": 5, "times": 2}}, {**CONFIG, "layers": [O.vabuzen_attention_layer(heads=3, kv_heads=2)], "loop": None},
                {**CONFIG, "layers": [O.vabuzen_attention_layer(conv=0)], "loop": None}, {**CONFIG, "layers": [O.vabuzen_attention_layer(mlp={"kind": "gated", "ff": 4})], "loop": None},
                moe(experts=7, groups=(3, 2)), moe(experts=6, groups=(3, 4)), moe(experts=6, groups=(3, 1), top=3)):
        with pytest.raises(ValueError):
            read(bad)


def test_packed_layout():
    read, _ = FAMILIES["Vabuzen"]
    W = O.make_vabuzen_weights(CONFIG, seed=1)
    packed = pack_layer_list(read(CONFIG), {k: torch.from_numpy(np.asarray(v)) for k, v in W.items()}, torch.float32, "cpu")
    l0, l1, l2, l3 = packed["layers"]
    assert tuple(l0["w_in"].shape) == (72 + 36 + 24, 48) and tuple(l0["w_out"].shape) == (48, 48) and "w_in_bias" not in l0 and "sink" not in l0
    assert tuple(l0["conv"].shape) == (72 + 36 + 24, 5) and tuple(l2["conv"].shape) == (16 + 16 + 48, 1) and "conv" not in l1
    np.testing.assert_array_equal(l0["conv"][72:108].numpy(), W["l0.mix.k.conv"])
    np.testing.assert_array_equal(l0["w_in"][108:].numpy(), W["l0.mix.v"])
    np.testing.assert_array_equal(l0["ff_in_bias"].numpy(), W["l0.mlp.up.b"])
    np.testing.assert_array_equal(l0["ff_out_bias"].numpy(), W["l0.mlp.down.b"])
    for key, name in (("norm", "norm1"), ("norm2", "norm2"), ("post_norm", "norm1b"), ("post_norm2", "norm2b")):
        np.testing.assert_array_equal(l0[key].numpy(), W[f"l0.{name}"])
        np.testing.assert_array_equal(l0[key + "_bias"].numpy(), W[f"l0.{name}.b"])
        assert l0[key + "_alpha"] == pytest.approx(float(W[f"l0.{name}.alpha"]))
    assert "norm2" not in l2 and "post_norm2" not in l2 and "w_in2" not in l2 and "ls1" not in l0
    assert tuple(l1["w_in"].shape) == (52 + 34, 48) and tuple(l1["uk_t"].shape) == (2, 28, 20) and "ff_in_bias" not in l1 and "correction" not in l1
    assert tuple(l1["w_in2"].shape) == ((2 * 104 + 9 + 7) // 8 * 8, 48) and tuple(l1["w_out2"].shape) == (48, 104)
    np.testing.assert_array_equal(l1["w_in2"][14:24].numpy(), W["l1.mlp.e0.gate"])
    np.testing.assert_array_equal(l1["w_in2"][208:217].numpy(), W["l1.mlp.router"])
    np.testing.assert_array_equal(packed["loop_step"].numpy(), W["loop.step"])
    assert "loop_in" not in packed and tuple(l3["w_out2"].shape) == (48, 24)


def test_loader_checks_names_and_shapes(tmp_path):
    from safetensors.torch import save_file

    from tiny_llm_hip.loader import load_weights

    W = O.make_vabuzen_weights(CONFIG, seed=2)
    (tmp_path / "config.json").write_text(json.dumps(CONFIG))

    def save(weights):
        save_file({k: torch.from_numpy(np.asarray(v, dtype=np.float32)).to(torch.bfloat16) for k, v in weights.items()}, str(tmp_path / "model.safetensors"))

    save(W)
    model = load_weights(str(tmp_path), dtype=torch.float32)
    assert model.family == "Vabuzen" and model.config.layers[0].keep_first == 2 and model.tensors["l0.norm1b.alpha"].shape == ()
    save({**W, "l0.mix.q.conv": np.ones((72, 4), dtype=np.float32)})
    with pytest.raises(ValueError, match="l0.mix.q.conv"):
        load_weights(str(tmp_path))
    save({k: v for k, v in W.items() if k != "l1.norm2b.alpha"})
    with pytest.raises(Exception, match="l1.norm2b.alpha"):
        load_weights(str(tmp_path))


# ---- the restatement against second forms -------------------------------------------------------------------------------------

@pytest.mark.parametrize("taps", [1, 2, 5, 30])
def test_short_convolution_against_a_library_convolution(taps):
    rng = np.random.default_rng(3)
    z, w = rng.normal(size=(23, 4)), rng.normal(size=(4, taps))
    want = np.stack([np.convolve(z[:, c], w[c, ::-1])[:23] for c in range(4)], 1)
    np.testing.assert_allclose(O.short_conv(z, w), want, rtol=1e-12, atol=1e-12)
    with_act = O.short_conv_silu(z, w)
    np.testing.assert_allclose(with_act, want / (1 + np.exp(-want)), rtol=1e-12, atol=1e-12)


def test_windows_that_keep_the_first_tokens_against_a_dense_form():
    rng = np.random.default_rng(4)
    L, H, G, D, V, win, keep = 29, 4, 2, 6, 5, 5, 3
    q, k, v = rng.normal(size=(L, H, D)), rng.normal(size=(L, G, D)), rng.normal(size=(L, G, V))
    got = O.keep_first_window_attention(q, k, v, 0.4, win, keep)
    i, j = np.indices((L, L))
    hidden = (j > i) | ((i - j >= win) & (j >= keep))
    for h in range(H):
        e = np.where(hidden, 0.0, np.exp((q[:, h] @ k[:, h // 2].T) * 0.4))
        np.testing.assert_allclose(got[:, h], (e @ v[:, h // 2]) / (1 + e.sum(1, keepdims=True)), rtol=1e-10, atol=1e-12)
    for at, reach in ((keep, keep + win - 1), (10, 10 + win - 1), (keep - 1, L - 1), (0, L - 1)):  # the last query that a key reaches
        v2 = v.copy()
        v2[at] += 1.0
        moved = np.abs(O.keep_first_window_attention(q, k, v2, 0.4, win, keep) - got).max(axis=(1, 2))
        assert moved[at:reach + 1].min() > 1e-4 and (moved[:at] == 0).all() and (moved[reach + 1:] == 0).all()
    np.testing.assert_allclose(O.keep_first_window_attention(q, k, v, 0.4, L, 0), O.sink_attention(q, k, v, 0.4))
    np.testing.assert_allclose(O.keep_first_window_attention(q, k, v, 0.4, 1, L), O.sink_attention(q, k, v, 0.4))
    low = O.keep_first_window_attention(q, k, v, 400.0, win, keep)  # scores of hundreds, of either sign
    assert np.isfinite(low).all()


def test_routing_by_groups():
    # groups (0.9, 0.1), (0.6, 0.55), (0.7, 0.2): by their largest the first and the third stay, by the sum of two the second (1.15) and the first (1.0)
    s = np.array([0.9, 0.1, 0.6, 0.55, 0.7, 0.2])
    z = np.log(s / (1 - s))
    got, margin = O.grouped_sigmoid_route(z, 2, 3, 2, 1.5)
    assert sorted(got) == [0, 2] and margin == pytest.approx(0.05)
    assert got[0] == pytest.approx(1.5 * 0.9 / 1.5) and got[2] == pytest.approx(1.5 * 0.6 / 1.5)
    got, margin = O.grouped_sigmoid_route(z, 3, 3, 2, 1.0)
    assert sorted(got) == [0, 2, 3] and sum(got.values()) == pytest.approx(1.0)
    got, margin = O.grouped_sigmoid_route(z, 1, 6, 6, 2.0)   # groups of one expert, all kept: the sum's second part does not exist
    assert got == {0: pytest.approx(2.0)} and margin == pytest.approx(0.2)
    got, _ = O.grouped_sigmoid_route(z, 6, 1, 1, 1.0)
    assert sorted(got) == list(range(6))


def test_forward_is_causal_and_looped_with_the_embedding_added_back():
    W = O.make_vabuzen_weights(CONFIG, seed=6)
    toks = [int(t) for t in np.random.default_rng(7).integers(0, 61, 30)]
    streams = []
    base = O.vabuzen_forward(CONFIG, W, toks, streams)
    assert len(streams) == 8 and base.shape == (30, 61) and np.abs(base).max() < 9.0
    later = list(toks)
    later[20] = (toks[20] + 1) % 61
    moved = np.abs(O.vabuzen_forward(CONFIG, W, later) - base).max(1)
    assert moved[:20].max() == 0.0 and moved[20:].min() > 0.0
    # the looped layers alone, written out: three passes, the second and third with the embedding output added back
    def one_pass(x, t):
        sub = {**CONFIG, "layers": CONFIG["layers"][1:3], "loop": {"start": 0, "stop": 2, "times": 1}, "vocab": 30}
        V = {k.replace("l1.", "l0.", 1) if k.startswith("l1.") else k.replace("l2.", "l1.", 1): v for k, v in W.items() if k.startswith(("l1.", "l2."))}
        out = []
        O.vabuzen_forward(sub, {**V, **{k: v for k, v in W.items() if k.startswith(("final", "head"))}, "embed": x, "loop.step": W["loop.step"][t:t + 1]}, range(30), out)
        return out[-1]

    x0 = np.asarray(W["embed"], dtype=np.float64)[toks]
    x = one_pass(streams[0], 0)
    np.testing.assert_allclose(x, streams[2], rtol=1e-10, atol=1e-12)
    x = one_pass(x + x0, 1)
    np.testing.assert_allclose(x, streams[4], rtol=1e-10, atol=1e-12)
    np.testing.assert_allclose(one_pass(x + x0, 2), streams[6], rtol=1e-10, atol=1e-12)
