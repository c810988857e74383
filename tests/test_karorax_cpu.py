"""CPU tier of the Karorax family: the config reader, the tensor table, the engine's packed layout, the loader's checks, and the
float64 restatement (tests/layer_list_oracle.py) held against itself -- each mechanism against a second, differently written form."""

import json
import math

import numpy as np
import pytest
import torch

import layer_list_oracle as O
from tiny_llm_hip.layer_list import FAMILIES, pack_layer_list

CONFIG = O.karorax_config([
    O.karorax_latent_layer(heads=3, dim=12, vdim=20, rot_dim=6, kv_rank=28, base=700.0, scale=0.21, window=9, mlp=None),
    O.karorax_parallel_layer(heads=6, kv_heads=3, dim=10, vdim=8, scale=0.17, softcap=3.0, coef=0.4, every=5, right_heads=2, right_dim=14, right_vdim=18,
                             decay=[0.5, 0.97], left_scale=0.8, right_scale=1.4, mlp=O.karorax_moe(experts=5, top=3, ff=12, shared=0)),
    O.karorax_latent_layer(heads=5, dim=8, vdim=4, rot_dim=6, kv_rank=28, base=700.0, window=30, kv_from=0, mlp={"kind": "dense", "ff": 33}),
    O.karorax_parallel_layer(mlp=O.karorax_moe(experts=4, top=1, ff=20, shared=11)),
], width=48, vocab=61, eps=2e-5, bigram=(37, 11, 6), logit_softcap=9.0)


def test_config_reader_takes_every_size_and_constant_from_the_file():
    read, table = FAMILIES["Karorax"]
    cfg = read(CONFIG)
    assert (cfg.family, cfg.block, cfg.width, cfg.vocab, cfg.norm_eps, cfg.norm_offset, cfg.pair_embed, cfg.logit_softcap) == \
        ("Karorax", "sequential", 48, 61, 2e-5, 1.0, (37, 11, 6), 9.0)
    assert cfg.layer_scale and cfg.norm_kind == "rms" and cfg.layer_runs == 4
    a, p, b, p2 = cfg.layers
    assert (a.kind, a.heads, a.dim, a.vdim, a.rot_dim, a.rot_dims, a.rot_base, a.q_rank, a.kv_rank, a.scale, a.window, a.kv_from, a.ff) == \
        ("latent", 3, 12, 20, 6, 6, 700.0, 0, 28, 0.21, 9, -1, 0)
    assert a.sink and a.learned_sink and a.gated and a.head_gate
    assert (b.kv_from, b.window, b.ff, b.ff_kind, b.ff_act) == (0, 30, 33, "plain", "relu2")
    assert (p.kind, p.heads, p.kv_heads, p.dim, p.vdim, p.scale, p.softcap, p.q_temp, p.mix_scale, p.mix_prefix) == \
        ("attention", 6, 3, 10, 8, 0.17, 3.0, (0.4, 5.0), 0.8, "mix.left.")
    assert p.distance_bias and not p.gated and not p.sink and p.rot_dims == 0
    r = p.beside
    assert (r.kind, r.rec_kind, r.heads, r.dim, r.vdim, r.decay, r.mix_scale, r.mix_prefix) == ("linrec", "fixed", 2, 14, 18, (0.5, 0.97), 1.4, "mix.right.")
    assert r.rec_silu and r.rec_plain_k and r.rec_joint_norm and r.rec_sigmoid_gate and r.rot_dims == 0 and r.ff == 0
    assert (p.ff_kind, p.ff, p.experts, p.top, p.expert_ff, p.shared_ff, p.router, p.moe_gated, p.moe_bias) == ("moe", 60, 5, 3, 12, 0, "chosen_softmax", True, True)
    assert (p2.ff, p2.shared_ff, p2.top) == (91, 11, 1) and not p2.moe_shared_sg and not p2.moe_correction
    names = table(cfg)
    assert names["bigram"] == (38, 48) and names["l0.mix.q"] == (54, 48) and names["l0.mix.dkv"] == (34, 48) and names["l0.mix.g"] == (3, 48)
    assert "l2.mix.dkv" not in names and "l2.mix.dkv.norm" not in names and names["l2.mix.uk"] == (40, 28) and names["l2.mix.sink"] == (5,)
    assert names["l1.mix.left.k"] == (30, 48) and names["l1.mix.right.norm"] == (36,) and names["l1.mlp.router.b"] == (5,) and "l1.mlp.shared.up" not in names
    assert "l0.norm2" not in names and "l0.ls2" not in names and names["l2.mlp.down"] == (48, 33)
    assert set(names) == set(O.make_karorax_weights(CONFIG))
    plain = read({k: v for k, v in CONFIG.items() if k not in ("embedding", "logit_softcap")})
    assert plain.pair_embed is None and plain.logit_softcap == 0.0 and "bigram" not in table(plain)
    L0, L1 = CONFIG["layers"][:2]
    for bad in ({**CONFIG, "layers": [dict(L0, type="delta")]}, {k: v for k, v in CONFIG.items() if k != "norm"},
                {**CONFIG, "layers": [O.karorax_latent_layer(kv_from=0)]}, {**CONFIG, "layers": [O.karorax_parallel_layer(right_heads=3, decay=[0.5, 0.6])]},
                {**CONFIG, "layers": [O.karorax_parallel_layer(heads=4, kv_heads=3)]}, {**CONFIG, "layers": [dict(L1, mlp=O.karorax_moe(experts=3, top=4))]},
                {**CONFIG, "layers": [dict(L1, mlp={"kind": "gated", "ff": 8})]}):
        with pytest.raises(ValueError):
            read(bad)


def test_packed_layout():
    read, _ = FAMILIES["Karorax"]
    cfg = read(CONFIG)
    W = O.make_karorax_weights(CONFIG, seed=1)
    packed = pack_layer_list(cfg, {k: torch.from_numpy(np.asarray(v)) for k, v in W.items()}, torch.float32, "cpu")
    l0, l1, l2, l3 = packed["layers"]
    np.testing.assert_array_equal(l0["w_in"].numpy(), np.concatenate([W["l0.mix.q"], W["l0.mix.dkv"], W["l0.mix.g"]]))
    assert "dq_norm" not in l0 and "uq" not in l0 and tuple(l0["uk_t"].shape) == (3, 28, 12) and "w_in2" not in l0 and "ls2" not in l0
    np.testing.assert_array_equal(l2["w_in"].numpy(), np.concatenate([W["l2.mix.q"], W["l2.mix.g"]]))
    np.testing.assert_array_equal(l2["sink"].numpy(), W["l2.mix.sink"])
    # two mixers: the rows of both in one input matrix, the columns of both in one output matrix, vectors of the second in an entry of their own
    np.testing.assert_array_equal(l1["w_in"].numpy(), np.concatenate([W["l1.mix." + n] for n in ("left.q", "left.k", "left.v", "right.q", "right.k", "right.v", "right.g")]))
    np.testing.assert_array_equal(l1["w_out"].numpy(), np.concatenate([W["l1.mix.left.o"], W["l1.mix.right.o"]], 1))
    assert l1["beside"]["decay"].tolist() == pytest.approx([0.5, 0.97]) and tuple(l1["beside"]["out_norm"].shape) == (36,)
    assert l1["bias_slope"].tolist() == pytest.approx([2.0 ** (-8 * (h + 1) / 6) for h in range(6)])
    h = torch.randn(3, 48)
    z = h @ l3["w_in2"].T
    np.testing.assert_allclose(z[:, 11:31].numpy(), (h @ torch.from_numpy(W["l3.mlp.e0.gate"]).T).numpy(), rtol=1e-5, atol=1e-5)
    np.testing.assert_allclose(z[:, 91 + 31:91 + 51].numpy(), (h @ torch.from_numpy(W["l3.mlp.e1.up"]).T).numpy(), rtol=1e-5, atol=1e-5)
    np.testing.assert_allclose(z[:, 182:186].numpy(), (h @ torch.from_numpy(W["l3.mlp.router"]).T).numpy(), rtol=1e-5, atol=1e-5)
    assert l3["w_in2"].shape[0] % 8 == 0 and tuple(l3["w_out2"].shape) == (48, 91)
    np.testing.assert_array_equal(l3["router_bias"].numpy(), W["l3.mlp.router.b"])
    np.testing.assert_array_equal(packed["pair_embed"].numpy(), W["bigram"])


def test_loader_checks_names_and_shapes(tmp_path):
    from safetensors.torch import save_file

    from tiny_llm_hip.loader import load_weights

    W = O.make_karorax_weights(CONFIG, seed=2)
    (tmp_path / "config.json").write_text(json.dumps(CONFIG))

    def save(weights):
        save_file({k: torch.from_numpy(np.asarray(v, dtype=np.float32)).to(torch.bfloat16) for k, v in weights.items()}, str(tmp_path / "model.safetensors"))

    save(W)
    model = load_weights(str(tmp_path), dtype=torch.float32)
    assert model.family == "Karorax" and model.config.layers[1].beside.heads == 2 and model.tensors["l2.mix.g"].shape == (5, 48)
    bad = dict(W)
    bad["l1.mix.right.norm"] = np.ones(18, dtype=np.float32)
    save(bad)
    with pytest.raises(ValueError, match="l1.mix.right.norm"):
        load_weights(str(tmp_path))
    save({k: v for k, v in W.items() if k != "bigram"})
    with pytest.raises(Exception, match="bigram"):
        load_weights(str(tmp_path))


# ---- the restatement against second forms -------------------------------------------------------------------------------------

def test_window_and_sink_against_a_dense_form():
    rng = np.random.default_rng(3)
    L, H, D, V, win = 23, 3, 6, 5, 5
    q, k, v, sinks = rng.normal(size=(L, H, D)), rng.normal(size=(L, H, D)), rng.normal(size=(L, H, V)), np.array([0.3, -1.0, 2.0])
    got = O.window_sink_attention(q, k, v, 0.4, win, sinks)
    i, j = np.indices((L, L))
    for h in range(H):
        e = np.where((j <= i) & (i - j < win), np.exp((q[:, h] @ k[:, h].T) * 0.4), 0.0)
        np.testing.assert_allclose(got[:, h], (e / (e.sum(1, keepdims=True) + math.exp(sinks[h]))) @ v[:, h], rtol=1e-10, atol=1e-12)
    moved = v.copy()
    moved[10] += 1.0
    diff = np.abs(O.window_sink_attention(q, k, moved, 0.4, win, sinks) - got).max(axis=(1, 2))
    assert diff[10 + win - 1] > 1e-3 and diff[10 + win] == 0.0 and diff[9] == 0.0
    np.testing.assert_allclose(O.window_sink_attention(q, k, v, 0.4, None, np.full(H, -1e9)), O.causal_softmax_attention(q, k, v, 0.4))


def test_capped_bias_attention_against_a_dense_form():
    rng = np.random.default_rng(4)
    L, H, G, D, V = 19, 4, 2, 6, 5
    q, k, v, slopes = 3 * rng.normal(size=(L, H, D)), rng.normal(size=(L, G, D)), rng.normal(size=(L, G, V)), O.distance_slopes(4)
    assert slopes.tolist() == pytest.approx([0.25, 0.0625, 0.015625, 0.00390625])
    got = O.capped_bias_attention(q, k, v, 0.5, 2.0, slopes)
    i, j = np.indices((L, L))
    for h in range(H):
        s = 2.0 * np.tanh((q[:, h] @ k[:, h // 2].T) * 0.5 / 2.0) - slopes[h] * (i - j)
        e = np.where(j <= i, np.exp(s), 0.0)
        np.testing.assert_allclose(got[:, h], (e / e.sum(1, keepdims=True)) @ v[:, h // 2], rtol=1e-10, atol=1e-12)
    assert np.abs(O.capped_bias_attention(q, k, v, 0.5, None, slopes) - got).max() > 1e-2 and np.abs(O.capped_bias_attention(q, k, v, 0.5, 2.0) - got).max() > 1e-2
    t = O.query_temperature(np.arange(12), 0.5, 4)
    assert t[:3].tolist() == [1.0] * 3 and t[3:7].tolist() == pytest.approx([1 + 0.5 * math.log(2)] * 4) and t[11] == pytest.approx(1 + 0.5 * math.log(4))


def test_router_takes_the_softmax_over_the_chosen_only():
    w = O.chosen_softmax_route(np.array([0.1, 2.0, -1.0, 1.0, 2.0]), 3)
    assert sorted(w) == [1, 3, 4] and sum(w.values()) == pytest.approx(1.0) and w[1] == w[4] and w[1] / w[3] == pytest.approx(math.e)
    assert O.chosen_softmax_route(np.array([3.0, 3.0]), 1) == {0: 1.0}


def test_pair_rows():
    assert O.bigram_rows([4, 7, 7, 0], 11, 6, 37) == [37, (44 + 42) % 37, (77 + 42) % 37, 77 % 37]


def test_forward_is_causal_and_reads_the_token_before():
    W = O.make_karorax_weights(CONFIG, seed=6)
    toks = [int(t) for t in np.random.default_rng(7).integers(0, 61, 30)]
    streams = []
    base = O.karorax_forward(CONFIG, W, toks, streams)
    assert len(streams) == 4 and base.shape == (30, 61) and np.abs(base).max() < 9.0
    later = list(toks)
    later[20] = (toks[20] + 1) % 61
    moved = np.abs(O.karorax_forward(CONFIG, W, later) - base).max(1)
    assert moved[:20].max() == 0.0 and moved[20:].min() > 0.0
    # the pair table: a row is read by one pair of tokens only; the first token's row stands behind the buckets
    first = dict(W, bigram=W["bigram"].copy())
    first["bigram"][37] += 1.0
    s2 = []
    O.karorax_forward(CONFIG, first, toks, s2)
    assert np.abs(s2[0][0] - streams[0][0]).max() > 0.1
    # the cache another layer filled: its down-projection moves both layers
    W3 = dict(W)
    W3["l0.mix.dkv.norm"] = W["l0.mix.dkv.norm"] * 1.5
    s3 = []
    O.karorax_forward(CONFIG, W3, toks, s3)
    assert np.abs(s3[2] - s3[1] - (streams[2] - streams[1])).max() > 1e-2
