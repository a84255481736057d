"""Host-side parts of the Gasavik design that need no GPU: its config reader (every size and constant from config.json), its tensor names, the registry's
choice, a checkpoint round trip, the scheduler's length limit, and the oracle's own mechanisms against closed forms."""
import json
import os

import numpy as np
import pytest

from krasis_amd import model_registry as R
from krasis_amd import serve_store as S
from tests import oracle_gasavik as O


def small_cfg():
    return O.make_config(width=40, vocab=37, eps=3e-6, residual_mult=0.8, side=7, positions=90, layers=[
        O.layer(O.delta(6, 3, 10, 14, 5), O.dense(20)),
        O.layer(O.wkv(3, 9, 11), None),
        O.layer(O.parallel(8, 2, 12, 6, 17, 4, 3, 5, 7, scale=0.21, left_scale=0.6, right_scale=-1.4, decay=[0.5, 0.75, 0.99]), O.dense(16)),
        O.layer(O.wkv(2, 14, 3), O.dense(24)),
        O.layer(O.parallel(5, 5, 8, 8, 0, 0, 2, 6, 6, left_scale=0.0), None),
    ])


def test_config_reader_takes_every_size_and_constant_from_config():
    cfg = small_cfg()
    W = O.random_weights(cfg, 0)
    spec = R.gasavik_spec({k: v for k, v in cfg.items() if not k.startswith("_")})
    spec.fit(spec, lambda n: W[n].shape)
    assert (spec.vocab, spec.width, spec.norm_kind, spec.norm_eps, spec.residual_mult) == (37, 40, S.NORM_RMS, 3e-6, 0.8)
    assert (spec.block_kind, spec.pre_norm, spec.post_norm, spec.norm_bias, spec.embed_norm, spec.norm_weight_offset) == (S.BLOCK_PARALLEL, 1, 0, 0, 1, 0.0)
    assert (spec.pos_rows, spec.token_side, spec.embed_scale, spec.logit_scale) == (90, 7, 0.0, 0.0)
    a, b, c, d, e = spec.layers
    assert (a.mixer_kind, a.heads, a.kv_heads, a.dim, a.vdim, a.proj_conv, a.lin_norm_weight) == (S.MIX_DELTA, 6, 3, 10, 14, 5, 2)
    assert (a.mlp_kind, a.ff, a.dense_act, a.ff_bias) == (S.MLP_DENSE, 20, S.ACT_SILU, 1)
    assert (b.mixer_kind, b.heads, b.kv_heads, b.dim, b.vdim, b.decay_rank, b.lin_norm_weight, b.mlp_kind, b.ff_bias) == (S.MIX_WKV, 3, 3, 9, 9, 11, 1, S.MLP_NONE, 0)
    assert (d.heads, d.dim, d.decay_rank, d.ff) == (2, 14, 3, 24)
    assert (c.mixer_kind, c.heads, c.kv_heads, c.dim, c.vdim, c.scale, c.window, c.keep_first) == (S.MIX_ATTENTION, 8, 2, 12, 6, 0.21, 17, 4)
    assert (c.qk_unit_norm, c.proj_bias, c.out_gate, c.rot_dims, c.has_sink) == (S.QKNORM_WEIGHTED, 3, S.OGATE_HEAD_SIGMOID, 0, S.SINK_NONE)
    assert (c.side_mixer, c.lt_heads, c.lt_dim, c.lt_vdim, c.mix_scale, c.side_scale) == (S.MIX_LIGHTNING, 3, 5, 7, 0.6, -1.4)
    assert (e.window, e.keep_first, e.side_scale) == (0, 0, 1.3) and 0.0 < e.mix_scale < 1e-20
    assert np.allclose(spec.extra["l2.mix.right.decay"], [0.5, 0.75, 0.99]) and spec.extra["l4.mix.right.decay"].shape == (2,)
    roles = list(spec.tensors(spec))
    assert {n for _, _, _, n in roles} == set(W) | set(spec.extra)              # the store asks for exactly the checkpoint's tensors and the config's decays
    assert len(roles) == len({n for _, _, _, n in roles})
    assert [i for l, r, i, _ in roles if l == 1 and r == "wkv_mu"] == [0, 1, 2, 3, 4]


def test_sizes_that_config_may_leave_out():
    cfg = {k: v for k, v in small_cfg().items() if not k.startswith("_")}
    W = O.random_weights(small_cfg(), 0)
    for k in ("max_positions", "token_side", "residual_mult"):
        cfg.pop(k)
    cfg["layers"] = json.loads(json.dumps(cfg["layers"]))
    for k in ("kv_heads", "vdim", "conv"):
        cfg["layers"][0]["mixer"].pop(k)
    spec = R.gasavik_spec(cfg)
    spec.fit(spec, lambda n: W[n].shape)
    assert (spec.pos_rows, spec.token_side, spec.residual_mult) == (90, 0, 1.0)
    assert (spec.layers[0].kv_heads, spec.layers[0].vdim, spec.layers[0].proj_conv) == (6, 10, 1)
    assert not [n for _, _, _, n in spec.tensors(spec) if "side" in n]


def test_config_reader_refuses_what_the_design_has_not():
    for edit in (lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][0]["mlp"].update(kind="moe"), lambda c: c["layers"][2]["mixer"]["right"].update(decay=[0.5])):
        bad = json.loads(json.dumps(small_cfg())); edit(bad)
        with pytest.raises(ValueError):
            R.gasavik_spec(bad)


def test_registry_and_checkpoint_roundtrip(tmp_path):
    assert {"Gasavik", "Ripupel", "Lufozen", "Midisun", "Pamulix", "Lomutar"} <= set(R.architectures())
    cfg = small_cfg(); W = O.random_weights(cfg, 0)
    assert R.model_family(cfg) == "serve:Gasavik"
    O.write_checkpoint(str(tmp_path), cfg, W)
    f = R.SafetensorsFile(os.path.join(tmp_path, "model.safetensors"))
    assert sorted(f.names()) == sorted(W)
    assert f.shape("l1.mix.w1") == (11, 40) and f.shape("l1.mix.u") == (3, 9) and f.shape("l0.mix.v.conv") == (84, 5) and f.shape("side.embed") == (37, 35)
    got = f.get("pos")
    assert got.dtype == np.uint16 and np.array_equal((got.astype(np.uint32) << 16).view(np.float32), O.bf16_round(W["pos"]))
    spec = R.gasavik_spec(R.read_config(str(tmp_path))); spec.fit(spec, f.shape)
    assert [l.decay_rank for l in spec.layers] == [0, 11, 0, 3, 0]


def test_scheduler_refuses_requests_longer_than_the_position_table():
    from krasis_amd.scheduler import Scheduler

    class Store:
        page_tokens, pool_tokens, max_slots, max_positions = 64, 1024, 4, 100

    class Engine:
        store = Store()
    sch = Scheduler(Engine())
    sch.submit([1] * 91, 10)                                  # the last token sampled is not fed
    with pytest.raises(ValueError):
        sch.submit([1] * 92, 10)


def test_oracle_mechanisms_against_closed_forms():
    rng = np.random.default_rng(0)
    # token shift: weight 0 is the token, weight 1 the one before, nothing before the first
    h = rng.standard_normal((4, 3))
    y = O.token_shift(h, np.array([0.0, 1.0, 0.25]))
    assert np.allclose(y[:, 0], h[:, 0]) and np.allclose(y[1:, 1], h[:-1, 1]) and y[0, 1] == 0.0 and np.allclose(y[2, 2], 0.75 * h[2, 2] + 0.25 * h[1, 2])
    # wkv as a sum over earlier tokens: the read-out at t sees token s < t under the decays of s + 1 .. t - 1, token t under the bonus
    T, d, dv = 6, 3, 2
    r, k, v, dec, u = (rng.standard_normal(s) for s in ((T, 1, d), (T, 1, d), (T, 1, dv), (T, 1, d), (1, d)))
    dec = O.sigmoid(dec)
    got = O.wkv_recurrence(r, k, v, dec, u)
    for t in range(T):
        want = (r[t, 0] * u[0] @ k[t, 0]) * v[t, 0] + sum((r[t, 0] * np.prod(dec[s + 1:t, 0], axis=0) @ k[s, 0]) * v[s, 0] for s in range(t))
        assert np.allclose(got[t, 0], want)
    assert np.allclose(O.wkv_decay(np.ones((1, 2)), np.zeros((1, 2)), np.ones((1, 1)), np.array([np.log(2.0)])), np.exp(-2.0))
    # delta rule: a full-strength write of a unit key makes the state answer that key with that value, whatever it held before
    q = O.unit_vector(rng.standard_normal((4, 1, 5))); v = rng.standard_normal((4, 1, 3))
    got = O.delta_recurrence(q, q, v, np.ones((4, 1)), np.ones((4, 1)))
    assert np.allclose(got, v, atol=1e-5)
    got = O.delta_recurrence(q[:1].repeat(3, 0), q[:1].repeat(3, 0), v[:3], np.full((3, 1), 0.5), np.array([[1.0], [0.0], [0.5]]))
    assert np.allclose(got[1, 0], 0.5 * v[0, 0], atol=1e-5) and np.allclose(got[2, 0], 0.125 * v[0, 0] + 0.5 * v[2, 0], atol=1e-5)
    # convolution: the last column is the current token's
    x = rng.standard_normal((5, 2)); w = rng.standard_normal((2, 3))
    y = O.causal_conv(x, w)
    assert np.allclose(y[0], w[:, 2] * x[0]) and np.allclose(y[4], w[:, 0] * x[2] + w[:, 1] * x[3] + w[:, 2] * x[4])
    # lightning: decay to the power of the distance
    q, k, v = (rng.standard_normal((4, 1, 3)) for _ in range(3))
    got = O.lightning_recurrence(q, k, v, [0.5])
    assert np.allclose(got[3, 0], sum(0.5 ** (3 - s) * (q[3, 0] @ k[s, 0]) * v[s, 0] for s in range(4)))
    # the mask
    assert [j for j in range(12) if O.visible(10, j, 4, 2)] == [0, 1, 7, 8, 9, 10] and [j for j in range(5) if O.visible(2, j, 4, 2)] == [0, 1, 2]
    assert [j for j in range(6) if O.visible(4, j, 0, 0)] == [0, 1, 2, 3, 4]
    # attention weights sum to one: constant values pass
    o = O.softmax_attention(rng.standard_normal((5, 2, 3)), rng.standard_normal((5, 1, 3)), np.ones((5, 1, 2)), 0.7, 1, 2, 1)
    assert np.allclose(o, 1.0)
    assert np.allclose(O.gelu_tanh(np.array([0.0, 100.0, -100.0])), [0.0, 100.0, 0.0]) and np.allclose(O.softplus(np.array([0.0, 800.0, -800.0])), [np.log(2.0), 800.0, 0.0])
