"""The batched serving store (kr_serve_*) with the Gasavik design against the plain float64 restatement in tests/oracle_gasavik.py.

Small random models of several shapes; every comparison is between what the store's step function returns (logits, or the residual stream after each
layer) and the oracle run on the whole sequence.  The f32 store is held to 2e-4 of the stream's scale, the bf16 store to a few percent."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from tests import oracle_gasavik as O

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = 2e-4


def engine(cfg, W, dtype="float32", max_tokens=1024, max_slots=4):
    from krasis_amd import model_registry as R
    from krasis_amd.scheduler import BatchEngine
    spec = R.gasavik_spec(cfg)
    spec.fit(spec, lambda n: W[n].shape)
    eng = BatchEngine(spec, dtype=dtype, max_tokens=max_tokens, max_slots=max_slots)
    eng.load_arrays(W)
    return eng


def rel(got, ref):
    """largest row error, relative to the root mean square of the reference rows"""
    d = np.asarray(got, np.float64) - ref
    return float(np.sqrt((d ** 2).mean(-1)).max() / np.sqrt((ref ** 2).mean()))


def tokens(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


# no two layers alike and no size a multiple of eight by accident: odd head counts, value width unlike key width, 1 : 1, 2 : 1 and 3 : 1 shared keys, 1 - 5 taps,
# windows shorter and longer than the kept first tokens, layers without feed-forward
def cfg_varied():
    return O.make_config(width=94, vocab=101, layers=[
        O.layer(O.delta(6, 2, 10, 14, 4), O.dense(40)),
        O.layer(O.wkv(5, 12, 7), O.dense(33)),
        O.layer(O.parallel(6, 2, 12, 20, 9, 4, 3, 10, 18), None),
        O.layer(O.wkv(3, 20, 2), None),
        O.layer(O.parallel(5, 5, 18, 6, 23, 31, 7, 6, 5, scale=0.4, left_scale=1.6, right_scale=0.3), O.dense(56)),
        O.layer(O.delta(3, 3, 21, 9, 2), O.dense(24)),
        O.layer(O.delta(4, 2, 8, 30, 1), None),
    ])


def cfg_wide():
    """rows that are multiples of 16 bytes (vector loads), heads of 32, 64 and 128 (the matrix-instruction forms of attention and recurrences)"""
    return O.make_config(width=128, vocab=260, eps=1e-6, residual_mult=0.45, side=32, layers=[
        O.layer(O.wkv(2, 64, 32), O.dense(96)),
        O.layer(O.delta(4, 2, 64, 64, 4), O.dense(64)),
        O.layer(O.parallel(8, 2, 64, 64, 48, 5, 2, 64, 128), O.dense(128)),
        O.layer(O.delta(2, 1, 128, 64, 3), None),
        O.layer(O.wkv(1, 128, 16), O.dense(64)),
        O.layer(O.parallel(4, 4, 128, 128, 70, 2, 3, 32, 32, left_scale=0.9), O.dense(64)),
    ])


@pytest.mark.parametrize("make,n", [(cfg_varied, 75), (cfg_wide, 200)])
def test_every_layer_and_logits_f32(make, n):
    cfg = make(); W = O.random_weights(cfg, 1); toks = tokens(cfg, n, 2)
    ref_logits, ref_streams = O.forward(cfg, W, toks)
    eng = engine(cfg, W)
    eng.store.set_capture(True)
    logits, amax = eng.step([("a", toks, list(range(n)))])
    streams = eng.store.read_capture(n)
    for li in range(len(ref_streams)):
        assert rel(streams[li], ref_streams[li]) < TOL, f"layer {li}"
    assert rel(logits, ref_logits) < TOL
    assert np.array_equal(amax, logits.argmax(-1))


@pytest.mark.parametrize("make,n", [(cfg_varied, 75), (cfg_wide, 150)])
def test_bf16_store_close_to_oracle(make, n):
    cfg = make(); W = {k: O.bf16_round(v) for k, v in O.random_weights(cfg, 3).items()}; toks = tokens(cfg, n, 4)
    ref_logits, _ = O.forward(cfg, W, toks)
    eng = engine(cfg, W, "bfloat16")
    logits, _ = eng.step([("a", toks, list(range(n)))])
    e = np.sqrt(((logits - ref_logits) ** 2).mean(-1)) / np.sqrt((ref_logits ** 2).mean())
    assert np.median(e) < 3e-2 and e.max() < 8e-2


@pytest.mark.parametrize("width,side,n", [(384, 200, 130), (256, 17, 65), (128, 256, 97), (640, 128, 66), (192, 40, 90)])
def test_token_rows_of_prompts_in_bf16(width, side, n):
    """prompt-sized steps form gate and activation of the token rows in one launch when the rows are whole fragments (widths that are multiples of 128), else in two"""
    cfg = O.make_config(width=width, vocab=61, side=side, layers=[O.layer(O.wkv(2, 8, 3), None), O.layer(O.delta(2, 1, 8, 8, 2), O.dense(24))])
    W = {k: O.bf16_round(v) for k, v in O.random_weights(cfg, 43).items()}
    W["side.embed"] = O.bf16_round(W["side.embed"] * 3.0); W["l0.side.norm"][:] = 2.0; W["l1.side.norm"][:] = 2.0
    toks = tokens(cfg, n, 44)
    ref, streams = O.forward(cfg, W, toks)
    swapped, _ = O.forward(cfg, {**W, "l1.side.gate": W["l1.side.gate"][::-1]}, toks)
    assert rel(swapped, ref) > 0.3
    eng = engine(cfg, W, "bfloat16")
    eng.store.set_capture(True)
    logits, _ = eng.step([("a", toks, list(range(n)))])
    got = eng.store.read_capture(n)
    for li in range(2):
        assert rel(got[li], streams[li]) < 3e-2, li
    assert rel(logits, ref) < 6e-2


def small_model(layers, **kw):
    kw.setdefault("width", 64); kw.setdefault("vocab", 50)
    return O.make_config(layers=layers, **kw)


def set_to(name, value):
    def patch(W):
        W[name][...] = value
    return patch


def scaled(name, by):
    def patch(W):
        W[name] = W[name] * np.float32(by)
    return patch


def spread(name, lo, hi):
    def patch(W):
        W[name] = np.linspace(lo, hi, W[name].size).reshape(W[name].shape).astype(np.float32)
    return patch


def both(*patches):
    def patch(W):
        for f in patches:
            f(W)
    return patch


def shifts_none_and_all(W):
    for i, n in enumerate("rkvgw"):
        W["l0.mix.mu." + n][:] = i % 2


def one_key_direction(W):
    """all keys nearly the same unit vector, writes near one: every token overwrites the one before"""
    k = W["l0.mix.k"]
    W["l0.mix.k"] = (0.02 * k + np.outer(np.abs(k[:, 0]) + 0.5, np.ones(k.shape[1]) / k.shape[1])).astype(np.float32)
    W["l0.norm1"][:] = 1.0
    W["embed"] = np.abs(W["embed"]) + 0.5
    W["l0.mix.k.conv"][:] = 1.0
    W["l0.mix.b"] = np.full_like(W["l0.mix.b"], 8.0 / W["l0.mix.b"].shape[1])
    W["l0.mix.A_log"][:] = -6.0


WKV = O.wkv(4, 12, 5)
DEL = O.delta(4, 2, 12, 10, 3)
PAR = O.parallel(4, 2, 12, 10, 11, 3, 3, 8, 6)
MECHANISMS = [
    ("wkv_plain", [O.layer(WKV, None)], {}, None),
    ("wkv_one_head_of_five_rank_one", [O.layer(O.wkv(1, 5, 1), None)], {}, None),
    ("wkv_heads_of_64", [O.layer(O.wkv(2, 64, 16), None)], {}, None),
    ("wkv_heads_of_65", [O.layer(O.wkv(1, 65, 48), None)], {}, None),
    ("wkv_heads_of_128_rank_70", [O.layer(O.wkv(1, 128, 70), None)], {}, None),
    ("wkv_heads_of_130", [O.layer(O.wkv(1, 130, 8), None)], {}, None),
    ("wkv_rank_wider_than_the_heads", [O.layer(O.wkv(2, 6, 31), None)], {}, None),
    ("wkv_shifts_of_nothing_and_of_everything", [O.layer(WKV, None)], {}, shifts_none_and_all),
    ("wkv_decays_next_to_one", [O.layer(O.wkv(2, 16, 4), None)], {}, both(set_to("l0.mix.w0", -9.0), scaled("l0.mix.w2", 0.1))),
    ("wkv_decays_over_the_whole_range", [O.layer(O.wkv(2, 32, 4), O.dense(24))], {}, spread("l0.mix.w0", -12.0, 3.0)),
    ("wkv_decays_that_leave_nothing", [O.layer(O.wkv(2, 64, 4), None)], {}, set_to("l0.mix.w0", 5.0)),
    ("wkv_decays_at_the_switch_of_the_two_forms", [O.layer(O.wkv(2, 32, 4), None)], {}, both(spread("l0.mix.w0", 1.2, 1.5), scaled("l0.mix.w2", 0.2))),
    ("wkv_low_rank_saturated", [O.layer(WKV, None)], {}, scaled("l0.mix.w1", 40.0)),
    ("wkv_bonus_large", [O.layer(WKV, None)], {}, scaled("l0.mix.u", 12.0)),
    ("wkv_bonus_none", [O.layer(WKV, None)], {}, set_to("l0.mix.u", 0.0)),
    ("wkv_output_norm_near_eps", [O.layer(WKV, None)], {"eps": 1e-3}, scaled("l0.mix.v", 0.02)),
    ("delta_plain", [O.layer(DEL, None)], {}, None),
    ("delta_one_head_no_past_in_the_convolution", [O.layer(O.delta(1, 1, 5, 3, 1), None)], {}, None),
    ("delta_seven_taps_three_heads_a_key", [O.layer(O.delta(6, 2, 12, 10, 7), None)], {}, None),
    ("delta_taps_longer_than_most_portions", [O.layer(O.delta(2, 1, 16, 16, 33), None)], {}, None),
    ("delta_one_value_column", [O.layer(O.delta(4, 4, 12, 1, 3), None)], {}, None),
    ("delta_64_64", [O.layer(O.delta(4, 2, 64, 64, 4), None)], {}, None),
    ("delta_128_128", [O.layer(O.delta(2, 1, 128, 128, 4), None)], {}, None),
    ("delta_70_100", [O.layer(O.delta(2, 2, 70, 100, 2), None)], {}, None),
    ("delta_130_keys", [O.layer(O.delta(1, 1, 130, 20, 2), None)], {}, None),
    ("delta_130_values", [O.layer(O.delta(2, 1, 20, 130, 2), None)], {}, None),
    ("delta_decays_next_to_one", [O.layer(DEL, None)], {}, set_to("l0.mix.A_log", -9.0)),
    ("delta_decays_that_leave_nothing", [O.layer(DEL, None)], {}, set_to("l0.mix.A_log", 5.0)),
    ("delta_decays_over_the_whole_range", [O.layer(O.delta(8, 4, 12, 10, 3), O.dense(24))], {}, spread("l0.mix.A_log", -9.0, 4.0)),
    ("delta_write_strengths_from_zero_to_one", [O.layer(DEL, None)], {}, scaled("l0.mix.b", 8.0)),
    ("delta_one_key_direction_written_over_and_over", [O.layer(O.delta(2, 1, 32, 16, 2), None)], {}, one_key_direction),
    ("delta_small_keys_near_the_unit_vectors_eps", [O.layer(DEL, None)], {}, both(scaled("l0.mix.k", 1e-3), scaled("l0.mix.q", 1e-3))),
    ("parallel_plain", [O.layer(PAR, None)], {}, None),
    ("parallel_without_a_window", [O.layer(O.parallel(4, 2, 12, 10, 0, 0, 3, 8, 6), None)], {}, None),
    ("parallel_window_of_one_nothing_kept", [O.layer(O.parallel(4, 2, 12, 10, 1, 0, 3, 8, 6), None)], {}, None),
    ("parallel_window_of_one_and_the_first_token", [O.layer(O.parallel(4, 1, 12, 10, 1, 1, 3, 8, 6), None)], {}, None),
    ("parallel_window_longer_than_the_sequence", [O.layer(O.parallel(4, 4, 12, 10, 300, 5, 3, 8, 6), None)], {}, None),
    ("parallel_more_kept_than_the_window_holds", [O.layer(O.parallel(4, 2, 12, 10, 4, 40, 3, 8, 6), None)], {}, None),
    ("parallel_more_kept_than_there_are_tokens", [O.layer(O.parallel(4, 2, 12, 10, 4, 500, 3, 8, 6), None)], {}, None),
    ("parallel_matrix_path_64_32", [O.layer(O.parallel(8, 2, 64, 32, 13, 6, 1, 64, 64), None)], {}, None),
    ("parallel_matrix_path_one_key_head_for_sixteen", [O.layer(O.parallel(16, 1, 32, 32, 20, 3, 2, 16, 40), None)], {}, None),
    ("parallel_value_rows_of_80", [O.layer(O.parallel(6, 3, 64, 80, 21, 5, 2, 16, 16), None)], {}, None),
    ("parallel_scores_of_a_wide_range", [O.layer(O.parallel(4, 2, 12, 10, 11, 3, 3, 8, 6, scale=4.0), None)], {}, None),
    ("parallel_gates_near_zero_and_one", [O.layer(PAR, None)], {}, scaled("l0.mix.left.g", 8.0)),
    ("parallel_biases_that_dominate", [O.layer(PAR, None)], {}, both(scaled("l0.mix.left.q.b", 20.0), scaled("l0.mix.left.k.b", 20.0), scaled("l0.mix.left.v.b", 20.0))),
    ("parallel_norm_near_eps", [O.layer(PAR, None)], {"eps": 1e-3}, both(scaled("l0.mix.left.q", 0.02), scaled("l0.mix.left.k", 0.02), scaled("l0.mix.left.q.b", 0.02), scaled("l0.mix.left.k.b", 0.02))),
    ("parallel_scales_of_one_and_minus_two", [O.layer(O.parallel(4, 2, 12, 10, 11, 3, 3, 8, 6, left_scale=1.0, right_scale=-2.0), None)], {}, None),
    ("parallel_left_weighted_by_zero", [O.layer(O.parallel(4, 2, 12, 10, 11, 3, 3, 8, 6, left_scale=0.0, right_scale=1.0), None)], {}, None),
    ("lightning_decays_of_one_and_nearly_none", [O.layer(O.parallel(2, 1, 8, 8, 5, 1, 4, 16, 12, decay=[1.0, 1e-6, 0.5, 0.999]), None)], {}, None),
    ("lightning_decay_of_zero", [O.layer(O.parallel(2, 1, 8, 8, 5, 1, 2, 16, 12, decay=[0.0, 0.9]), None)], {}, None),
    ("lightning_one_head_128_128", [O.layer(O.parallel(2, 1, 8, 8, 5, 1, 1, 128, 128), None)], {}, None),
    ("lightning_keys_of_140", [O.layer(O.parallel(2, 1, 8, 8, 5, 1, 1, 140, 24), None)], {}, None),
    ("lightning_norm_over_all_heads_near_eps", [O.layer(PAR, None)], {"eps": 1e-3}, scaled("l0.mix.right.v", 0.02)),
    ("feed_forward_biases_that_dominate", [O.layer(WKV, O.dense(24))], {}, both(scaled("l0.mlp.gate.b", 10.0), scaled("l0.mlp.up.b", 10.0), scaled("l0.mlp.down.b", 10.0))),
    ("token_rows_one_wide", [O.layer(WKV, O.dense(24)), O.layer(DEL, None)], {"side": 1}, None),
    ("token_rows_wider_than_the_model", [O.layer(PAR, O.dense(24)), O.layer(WKV, None)], {"side": 72}, None),
    ("token_rows_large", [O.layer(WKV, None), O.layer(WKV, None)], {"side": 8}, scaled("side.embed", 30.0)),
    ("token_rows_norm_near_eps", [O.layer(WKV, None)], {"side": 8, "eps": 1e-2}, scaled("l0.side.proj", 0.05)),
    ("no_token_rows", [O.layer(WKV, O.dense(24)), O.layer(DEL, O.dense(20)), O.layer(WKV, None)], {"side": 0}, None),
    ("residual_multiplier_of_one", [O.layer(DEL, O.dense(24)), O.layer(WKV, O.dense(24))], {"residual_mult": 1.0}, None),
    ("residual_multiplier_small", [O.layer(DEL, O.dense(24)), O.layer(PAR, O.dense(24))], {"residual_mult": 0.03}, None),
    ("positions_that_dominate", [O.layer(WKV, O.dense(24)), O.layer(PAR, None)], {}, scaled("pos", 10.0)),
    ("as_many_positions_as_tokens", [O.layer(WKV, O.dense(24))], {"positions": 70}, None),
]


@pytest.mark.parametrize("name,layers,kw,patch", MECHANISMS, ids=[m[0] for m in MECHANISMS])
def test_each_mechanism_alone(name, layers, kw, patch):
    cfg = small_model(layers, **kw)
    W = O.random_weights(cfg, 5)
    if patch:
        patch(W)
    toks = tokens(cfg, 70, 6)
    ref_logits, ref_streams = O.forward(cfg, W, toks)
    eng = engine(cfg, W)
    eng.store.set_capture(True)
    logits, _ = eng.step([("a", toks, list(range(70)))])
    got = eng.store.read_capture(70)
    for li in range(len(ref_streams)):
        assert rel(got[li], ref_streams[li]) < TOL, (name, li)
    assert rel(logits, ref_logits) < TOL, name
    eng.store.set_capture(False)
    # and the same tokens one by one, through the cache and the state
    rows = [eng.step([("d", [t], [0])])[0][0] for t in toks]
    assert rel(np.stack(rows), ref_logits) < TOL, name


def test_the_oracle_feels_every_mechanism(monkeypatch):
    """the oracle itself: leaving out any part of the design moves its result far beyond the tolerance the store is held to"""
    cfg = small_model([O.layer(O.wkv(3, 10, 4), O.dense(24)), O.layer(O.delta(4, 2, 12, 10, 3), O.dense(20)), O.layer(O.parallel(4, 2, 12, 10, 7, 3, 3, 8, 6, scale=0.5), None),
                       O.layer(O.wkv(2, 8, 3), None)])
    W = O.random_weights(cfg, 5); toks = tokens(cfg, 30, 6)
    base, _ = O.forward(cfg, W, toks)

    def changed(**patch):
        with monkeypatch.context() as m:
            for k, v in patch.items():
                m.setattr(O, k, v)
            return O.forward(cfg, W, toks)[0]

    def weights(**patch):
        W2 = dict(W); W2.update(patch)
        return O.forward(cfg, W2, toks)[0]

    def config(edit):
        c2 = json.loads(json.dumps(cfg)); edit(c2)
        return O.forward(c2, W, toks)[0]
    rec, drec, att, lrec, mleft = O.wkv_recurrence, O.delta_recurrence, O.softmax_attention, O.lightning_recurrence, O.mixer_left

    def write_before_reading(r, k, v, dec, u):
        return rec(r, k, v, dec, np.ones_like(u))

    def no_correction(q, k, v, g, beta):
        T, H, d = q.shape
        o = np.zeros((T, H, v.shape[2]))
        for h in range(H):
            S = np.zeros((d, v.shape[2]))
            for t in range(T):
                S = g[t, h] * S + np.outer(k[t, h], beta[t, h] * v[t, h]); o[t, h] = S.T @ q[t, h]
        return o
    assert rel(changed(token_shift=lambda h, mu: h), base) > 1e-2
    assert rel(changed(wkv_decay=lambda z, w1, w2, w0: np.exp(-np.exp(w0)) * np.ones((len(z), 1))), base) > 1e-3
    assert rel(changed(wkv_recurrence=write_before_reading), base) > 1e-2
    assert rel(changed(wkv_recurrence=lambda r, k, v, dec, u: rec(r, k, v, np.ones_like(dec), u)), base) > 1e-2
    assert rel(changed(delta_recurrence=no_correction), base) > 1e-2
    assert rel(changed(delta_recurrence=lambda q, k, v, g, b: drec(q, k, v, np.ones_like(g), b)), base) > 1e-2
    assert rel(changed(delta_recurrence=lambda q, k, v, g, b: drec(q, k, v, g, np.ones_like(b))), base) > 1e-2
    assert rel(changed(causal_conv=lambda u, w: u * w[:, -1]), base) > 1e-2
    assert rel(changed(unit_vector=lambda x: x), base) > 1e-2
    assert rel(changed(softmax_attention=lambda q, k, v, s, g, size, keep: att(q, k, v, s, g, size, 0)), base) > 1e-3
    assert rel(changed(softmax_attention=lambda q, k, v, s, g, size, keep: att(q, k, v, s, g, size + 1, keep)), base) > 1e-3
    assert rel(changed(softmax_attention=lambda q, k, v, s, g, size, keep: att(q, k, v, s, g, size, keep + 1)), base) > 1e-3
    assert rel(changed(lightning_recurrence=lambda q, k, v, dec: lrec(q, k, v, [1.0] * len(dec))), base) > 1e-2
    assert rel(changed(gelu_tanh=O.silu), base) > 1e-3
    for n in [f"l2.mix.left.{x}.b" for x in "qkv"] + [f"l0.mlp.{x}.b" for x in ("gate", "up", "down")] + ["l0.mix.u", "l1.mix.dt_bias", "l1.mix.A_log", "pos", "side.embed"]:
        assert rel(weights(**{n: np.zeros_like(W[n])}), base) > 1e-3, n
    for n in ("l0.mix.norm", "l1.mix.norm", "l2.mix.left.q.norm", "l2.mix.left.k.norm", "l2.mix.right.norm", "embed.norm", "final.norm", "l0.side.norm", "l3.norm1"):
        assert rel(weights(**{n: np.ones_like(W[n])}), base) > 1e-3, n
    for n in ("l2.mix.left.g", "l2.mix.right.g", "l1.mix.g", "l0.mix.g", "l1.mix.b", "l1.mix.a"):
        assert rel(weights(**{n: np.zeros_like(W[n])}), base) > 1e-3, n
    for side in ("left_scale", "right_scale"):
        assert rel(config(lambda c: c["layers"][2]["mixer"].update({side: 1.0})), base) > 1e-2
    assert rel(config(lambda c: c.update(residual_mult=1.0)), base) > 1e-2
    assert rel(config(lambda c: c["layers"][2]["mixer"]["left"].update(scale=0.2)), base) > 1e-3


# ---------------------------------------------------------------------------------------------------------------- one key that decides
def peaked_model(size, keep, heads=4, kv_heads=2, dim=32, vdim=16, vocab=40):
    """attention that finds ONE key among hundreds: without position rows a token's key depends on the token alone, and the query of token 1 is steered along the key of
    token 0 in every head: normed to the same length it scores about scale * dim, any other key scale * sqrt(dim)"""
    cfg = small_model([O.layer(O.parallel(heads, kv_heads, dim, vdim, size, keep, 2, 8, 8, scale=0.9, left_scale=1.5, right_scale=0.2), None)], vocab=vocab)
    W = O.random_weights(cfg, 11)
    W["pos"][:] = 0.0
    p = "l0.mix.left."
    W[p + "q.norm"][:] = 1.0; W[p + "k.norm"][:] = 1.0; W[p + "q.b"][:] = 0.0
    w = {k: v.astype(np.float64) for k, v in W.items()}
    h = O.rms_unit(O.embed(cfg, w, [0, 1]), cfg["norm"]["eps"]) * w["l0.norm1"]
    k0 = O.rms_unit((h[0] @ w[p + "k"].T + w[p + "k.b"]).reshape(kv_heads, dim), 0.0)
    W[p + "q"] = np.concatenate([np.outer(k0[g // (heads // kv_heads)], h[1]) / (h[1] @ h[1]) for g in range(heads)]).astype(np.float32)
    W[p + "g"] *= 0.2
    return cfg, W


def needle_sequence(vocab, n, needle_at, query_at, seed):
    """random tokens 2.., token 0 (the needle) once, token 1 (the query) once"""
    t = [int(x) for x in np.random.default_rng(seed).integers(2, vocab, n)]
    t[needle_at] = 0; t[query_at] = 1
    return t


CASES = [(40, 6, n, q) for n, q in [(0, 1), (0, 300), (5, 300), (6, 300), (5, 45), (6, 45), (6, 46), (261, 300), (260, 300), (88, 127), (87, 127), (64, 103), (63, 103), (63, 102), (128, 129)]] + \
        [(64, 0, n, q) for n, q in [(1, 64), (0, 64), (0, 63), (64, 127), (63, 127), (200, 263), (199, 263)]] + \
        [(1, 3, n, q) for n, q in [(2, 200), (3, 200), (199, 200), (0, 3)]] + \
        [(10, 130, n, q) for n, q in [(129, 400), (130, 400), (64, 140), (128, 140), (130, 140), (131, 140), (391, 400), (390, 400)]] + \
        [(0, 0, n, q) for n, q in [(3, 700), (0, 128)]] + [(500, 20, n, q) for n, q in [(19, 530), (20, 530), (30, 530), (31, 530)]]


@pytest.mark.parametrize("head", [(4, 2, 32, 16), (6, 2, 30, 14)], ids=["matrix", "vector"])
@pytest.mark.parametrize("size,keep,needle,query", CASES)
def test_one_key_at_every_edge_prompt_and_decode(head, size, keep, needle, query):
    cfg, W = peaked_model(size, keep, *head)
    n = query + 3
    toks = needle_sequence(cfg["vocab"], n, needle, query, 19)
    ref, _ = O.forward(cfg, W, toks)
    moved = list(toks); moved[needle] = 7
    # the oracle without that key at that place, the right-hand mixer's memory of it left alone: the needle decides exactly when it is seen
    zeroed = dict(W); zeroed["l0.mix.right.o"] = np.zeros_like(W["l0.mix.right.o"])
    a, b = O.forward(cfg, zeroed, toks)[0][query], O.forward(cfg, zeroed, moved)[0][query]
    sees = O.visible(query, needle, size, keep)
    assert (rel(b[None], a[None]) > 0.05) == sees
    eng = engine(cfg, W, max_tokens=1024)
    places = [query - 1, query, query + 1]
    whole, _ = eng.step([("w", toks, places)])
    assert rel(whole, ref[places]) < TOL
    eng.finish("w")
    cut = max((query // 64) * 64 if query % 64 else query - 1, 1)      # the prompt cut at the page border before the query, then decoded
    eng.step([("a", toks[:cut], [])])
    got = [eng.step([("a", [toks[p]], [0])])[0][0] for p in range(cut, query + 1)]
    assert rel(np.stack(got), ref[cut:query + 1]) < TOL


def remembering_model(kind):
    """a recurrence that keeps a token for hundreds of positions among a few filler tokens"""
    mixer = {"wkv": O.wkv(2, 48, 4), "delta": O.delta(2, 1, 64, 24, 2), "lightning": O.parallel(2, 1, 8, 8, 5, 1, 2, 48, 24, left_scale=0.3, right_scale=1.5, decay=[0.9999, 1.0])}[kind]
    cfg = small_model([O.layer(mixer, None)], vocab=12)
    W = O.random_weights(cfg, 12)
    W["pos"][:] = 0.0
    w = {k: v.astype(np.float64) for k, v in W.items()}
    h = O.rms_unit(O.embed(cfg, w, list(range(8))), cfg["norm"]["eps"]) * w["l0.norm1"]
    only0 = np.linalg.pinv(h)[:, 0]                              # a direction that token 0's input has and the fillers' have not
    if kind == "wkv":
        W["l0.mix.w0"][:] = -12.0; W["l0.mix.w2"] *= 0.01
        W["l0.mix.mu.k"][:] = 0.0
        W["l0.mix.k"] = (0.02 * W["l0.mix.k"] + np.outer(np.ones(96), 6.0 * only0)).astype(np.float32)
    elif kind == "delta":
        W["l0.mix.A_log"][:] = -12.0
        W["l0.mix.k.conv"][:] = [0.0, 1.0]; W["l0.mix.v.conv"][:] = [0.0, 1.0]; W["l0.mix.q.conv"][:] = [0.0, 1.0]
        W["l0.mix.b"] = (np.outer(np.ones(2), 24.0 * only0) + np.zeros_like(W["l0.mix.b"])).astype(np.float32)
        W["l0.mix.b"] -= np.float32(12.0) * np.linalg.pinv(h).sum(1).astype(np.float32)      # strength sigmoid(12) for token 0, sigmoid(-12) for the fillers
    else:
        W["l0.mix.right.k"] = (0.02 * W["l0.mix.right.k"] + np.outer(np.ones(96), 6.0 * only0)).astype(np.float32)
    return cfg, W


@pytest.mark.parametrize("kind", ["wkv", "delta", "lightning"])
def test_far_token_among_hundreds_through_the_state(kind):
    """a token fed 700 positions earlier, in another step, still decides the answer: only the state can have carried it"""
    cfg, W = remembering_model(kind)
    n = 760
    toks = needle_sequence(8, n, 40, 740, 17)                    # fillers 2 .. 7
    ref, _ = O.forward(cfg, W, toks)
    toks_moved = list(toks); toks_moved[40] = 5
    ref_moved, _ = O.forward(cfg, W, toks_moved)
    assert rel(ref_moved[740:741], ref[740:741]) > 0.03         # far beyond the tolerance below
    eng = engine(cfg, W, max_tokens=1024)
    eng.step([("a", toks[:300], []), ("other", toks_moved[:90], [])])
    eng.step([("a", toks[300:700], [])])
    lg, _ = eng.step([("a", toks[700:], [40]), ("other", toks_moved[90:95], [])])
    assert rel(lg, ref[740:741]) < TOL
    eng.finish("a")
    eng.step([("b", toks[:739], [])])
    eng.step([("b", toks[739:740], [])])
    lg, _ = eng.step([("b", toks[740:741], [0])])
    assert rel(lg, ref[740:741]) < TOL


def test_first_tokens_of_a_sequence():
    cfg = cfg_varied(); W = O.random_weights(cfg, 21); toks = tokens(cfg, 8, 22)
    ref, _ = O.forward(cfg, W, toks)
    eng = engine(cfg, W)
    one, _ = eng.step([("one", toks[:1], [0])])
    assert rel(one, ref[:1]) < TOL
    two, _ = eng.step([("two", toks[:2], [0, 1])])
    assert rel(two, ref[:2]) < TOL
    nxt, _ = eng.step([("one", toks[1:2], [0])])
    assert rel(nxt, ref[1:2]) < TOL
    rest, _ = eng.step([("one", toks[2:4], [0, 1]), ("two", toks[2:3], [0])])       # the convolutions reach back over three separate steps
    assert rel(rest, np.stack([ref[2], ref[3], ref[2]])) < TOL
    last, _ = eng.step([("two", toks[3:8], [0, 1, 2, 3, 4]), ("one", toks[4:5], [0])])
    assert rel(last, np.concatenate([ref[3:8], ref[4:5]])) < TOL


@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
def test_prefill_equals_token_by_token_decode(dtype, tol):
    cfg = cfg_wide(); W = {k: O.bf16_round(v) for k, v in O.random_weights(cfg, 23).items()}; n = 90; toks = tokens(cfg, n, 24)
    ref, _ = O.forward(cfg, W, toks)
    eng = engine(cfg, W, dtype)
    whole, _ = eng.step([("w", toks, list(range(n)))])
    rows = [eng.step([("d", [t], [0])])[0][0] for t in toks]
    assert rel(whole, ref) < tol and rel(np.stack(rows), ref) < tol


@pytest.mark.parametrize("sizes", [[2] * 30, [3, 2, 7, 2, 64, 5, 65, 2, 31, 2, 9], [37, 3, 3, 37, 37, 5, 11, 25, 24, 2], [1, 128, 2, 60], [1, 1, 2, 1, 3, 1, 1, 4], [33, 32, 31, 34, 48, 17, 16]])
@pytest.mark.parametrize("make", [cfg_varied, cfg_wide])
def test_portions_of_several_sizes(make, sizes):
    cfg = make(); W = O.random_weights(cfg, 25); n = sum(sizes); toks = tokens(cfg, n, 26)
    ref, _ = O.forward(cfg, W, toks)
    eng = engine(cfg, W)
    at, rows = 0, []
    for s in sizes:
        lg, _ = eng.step([("c", toks[at:at + s], list(range(s)))])
        rows.append(lg); at += s
    assert rel(np.concatenate(rows), ref) < TOL


@pytest.mark.parametrize("make", [cfg_varied, cfg_wide])
def test_unequal_requests_in_one_batch_equal_each_alone(make):
    cfg = make(); W = O.random_weights(cfg, 27)
    lens = {"a": 70, "b": 9, "c": 131, "d": 33}
    toks = {k: tokens(cfg, n, 30 + i) for i, (k, n) in enumerate(lens.items())}
    refs = {k: O.forward(cfg, W, t)[0] for k, t in toks.items()}
    eng = engine(cfg, W, max_tokens=512)
    # a schedule that mixes portions with single tokens: every request advances by its own stride; 0 = the request sits this step out
    stride = {"a": [17, 1, 0, 30, 1, 20], "b": [2, 1, 1, 0, 0, 4], "c": [64, 1, 65, 0, 1], "d": [1, 1, 31]}
    at = {k: 0 for k in lens}
    got = {k: [] for k in lens}
    step = 0
    while any(at[k] < lens[k] for k in lens):
        entries, owners = [], []
        for k in lens:
            if at[k] >= lens[k]:
                continue
            s = min(stride[k][step] if step < len(stride[k]) else 1, lens[k] - at[k])
            if s == 0:
                continue
            entries.append((k, toks[k][at[k]:at[k] + s], list(range(s)))); owners.append((k, s)); at[k] += s
        lg, _ = eng.step(entries)
        o = 0
        for k, s in owners:
            got[k].append(lg[o:o + s]); o += s
        step += 1
    for k in lens:
        assert rel(np.concatenate(got[k]), refs[k]) < TOL, k


@pytest.mark.parametrize("n_req", [2, 4, 7, 20])
def test_batches_of_single_tokens(n_req):
    """decode steps of several requests at different positions, below and above the size at which a projection reads its weights once for all of them"""
    cfg = cfg_varied(); W = O.random_weights(cfg, 29)
    toks = {r: tokens(cfg, 6 + (5 * r) % 47 + 6, 60 + r) for r in range(n_req)}
    refs = {r: O.forward(cfg, W, t)[0] for r, t in toks.items()}
    eng = engine(cfg, W, max_tokens=2048, max_slots=20)
    eng.step([(r, t[:-6], []) for r, t in toks.items()])
    for i in range(6):
        order = [(r * 3 + i) % n_req for r in range(n_req)] if n_req % 3 else list(range(n_req))      # slots in changing order
        lg, _ = eng.step([(r, [toks[r][len(toks[r]) - 6 + i]], [0]) for r in order])
        assert rel(lg, np.stack([refs[r][len(toks[r]) - 6 + i] for r in order])) < TOL, i


def test_pages_and_slots_are_used_again():
    """a pool of five pages and four slots: requests come and go; the later ones run in pages and slots -- convolution rows, shifted rows, recurrent states -- that the
    earlier ones gave back"""
    cfg = cfg_varied(); W = O.random_weights(cfg, 31)
    eng = engine(cfg, W, max_tokens=320, max_slots=4)
    assert eng.store.free_pages() == 5
    seqs = [tokens(cfg, n, 40 + i) for i, n in enumerate([130, 60, 64, 100, 65, 190, 20, 129])]
    refs = [O.forward(cfg, W, t)[0] for t in seqs]
    a, _ = eng.step([(0, seqs[0], [129]), (1, seqs[1], [59]), (2, seqs[2], [63])])      # 3 + 1 + 1 pages: the pool is full
    assert eng.store.free_pages() == 0
    with pytest.raises(RuntimeError):
        eng.step([(3, seqs[3], [0])])                        # no page left: refused, nothing changed
    assert rel(a, np.stack([refs[0][129], refs[1][59], refs[2][63]])) < TOL
    eng.finish(0); eng.finish(3)                            # request 3 was admitted (slot) but holds no page
    assert eng.store.free_pages() == 3
    b, _ = eng.step([(3, seqs[3], [99]), (4, seqs[4][:40], [39])])          # 2 + 1 pages, out of request 0's
    assert rel(b, np.stack([refs[3][99], refs[4][39]])) < TOL
    eng.finish(1); eng.finish(2)
    c, _ = eng.step([(4, seqs[4][40:], [24]), (3, [seqs[3][0]], [])])      # request 4 crosses into a second page (one that request 1 or 2 held)
    assert rel(c, refs[4][64:65]) < TOL
    eng.finish(3); eng.finish(4)
    assert eng.store.free_pages() == 5
    d, _ = eng.step([(5, seqs[5], [0, 189]), (6, seqs[6], [19])])
    assert rel(d, np.stack([refs[5][0], refs[5][189], refs[6][19]])) < TOL
    eng.finish(5)
    e, _ = eng.step([(7, seqs[7][:1], [0])])                # one token into a slot whose state another request filled
    f, _ = eng.step([(7, seqs[7][1:], [127]), (6, [3], [0])])
    assert rel(np.concatenate([e, f[:1]]), np.stack([refs[7][0], refs[7][128]])) < TOL


def test_long_decoding_through_pages():
    cfg = cfg_wide(); W = O.random_weights(cfg, 33); n = 330; toks = tokens(cfg, n, 34)
    ref, _ = O.forward(cfg, W, toks)
    eng = engine(cfg, W)
    eng.step([("a", toks[:20], [])])
    rows = [eng.step([("a", [toks[p]], [0])])[0][0] for p in range(20, n)]
    assert rel(np.stack(rows), ref[20:]) < TOL


def test_a_prompt_of_many_blocks():
    """more than sixteen blocks of 64 tokens in one portion, slow decays: the serial launches over the blocks take several rounds; then one decoded token"""
    cfg = small_model([O.layer(O.wkv(2, 32, 4), None), O.layer(O.delta(2, 1, 32, 16, 3), O.dense(24)), O.layer(O.parallel(2, 1, 16, 16, 100, 4, 2, 32, 32, decay=[0.999, 0.98]), None)])
    W = O.random_weights(cfg, 36); n = 1300; toks = tokens(cfg, n, 37)
    W["l0.mix.w0"] = np.linspace(-9.0, -1.0, 64).astype(np.float32); W["l1.mix.A_log"][:] = [-6.0, -2.0]
    ref, _ = O.forward(cfg, W, toks)
    eng = engine(cfg, W, max_tokens=2048)
    places = [63, 64, 1023, 1024, 1087, n - 2]
    lg, _ = eng.step([("a", toks[:-1], places)])
    assert rel(lg, ref[places]) < TOL
    lg, _ = eng.step([("a", toks[-1:], [0])])
    assert rel(lg, ref[-1:]) < TOL


def test_positions_end_where_the_table_ends():
    cfg = small_model([O.layer(WKV, None)], positions=70); W = O.random_weights(cfg, 5)
    eng = engine(cfg, W)
    toks = tokens(cfg, 70, 6)
    with pytest.raises(ValueError):
        eng.step([("a", toks + [1], [0])])
    ref, _ = O.forward(cfg, W, toks)
    lg, _ = eng.step([("a", toks, [69])])                    # the refused step changed nothing
    assert rel(lg, ref[69:]) < TOL
    with pytest.raises(ValueError):
        eng.step([("a", [1], [0])])
    with pytest.raises(ValueError):
        eng.generate([toks[:60]], 12)                        # 60 + 11 fed positions
    eng.finish("a")
    assert len(eng.generate([toks[:60]], 11)[0]) == 11


def greedy_oracle(cfg, W, prompt, n_new):
    seq, out, margins = list(prompt), [], []
    for _ in range(n_new):
        lg = O.forward(cfg, W, seq)[0][-1]
        top = np.sort(lg)[-2:]
        margins.append(float(top[1] - top[0]))
        out.append(int(lg.argmax())); seq.append(out[-1])
    return out, min(margins)


def test_greedy_generation_through_the_scheduler():
    """five prompts, four slots, a pool that cannot hold all at once, a step budget that cuts prompts into portions"""
    cfg = cfg_varied(); W = O.random_weights(cfg, 35)
    prompts = [tokens(cfg, n, 50 + i) for i, n in enumerate([45, 3, 70, 18, 29])]
    eng = engine(cfg, W, max_tokens=256, max_slots=4)
    outs = eng.generate(prompts, 6, token_budget=32)
    assert eng.store.free_pages() == 4 and not eng.live()
    for p, o in zip(prompts, outs):
        want, margin = greedy_oracle(cfg, W, p, 6)
        if margin > 1e-3:                                   # a near-tie of the two best logits may fall either way in f32
            assert o == want
        else:
            assert o[0] == want[0] or margin < 1e-3


def test_sampling_uses_the_frameworks_sampler():
    cfg = cfg_varied(); W = O.random_weights(cfg, 37); p = tokens(cfg, 12, 38)
    eng = engine(cfg, W)
    a = eng.generate([p], 8, temperature=0.8, top_k=5, top_p=0.9, seed=7)
    b = eng.generate([p], 8, temperature=0.8, top_k=5, top_p=0.9, seed=7)
    assert a == b and len(a[0]) == 8
    g = eng.generate([p], 8)
    k1 = eng.generate([p], 8, temperature=1.3, top_k=1, seed=3)      # top_k = 1 is greedy whatever the temperature
    assert g == k1


def test_checkpoint_directory_command_line_and_trace_replay(tmp_path):
    cfg = cfg_varied(); W = {k: O.bf16_round(v) for k, v in O.random_weights(cfg, 39).items()}
    model = str(tmp_path / "model"); O.write_checkpoint(model, cfg, W)
    from krasis_amd import model_registry as R
    assert R.model_family(R.read_config(model)) == "serve:Gasavik"
    p1, p2 = tokens(cfg, 20, 60), tokens(cfg, 7, 61)
    env = dict(os.environ, PYTHONPATH=ROOT)
    out = subprocess.run([sys.executable, "-m", "krasis_amd", "generate", "--model", model, "--dtype", "float32", "--max-new-tokens", "4",
                          "--prompt", ",".join(map(str, p1)), "--prompt", ",".join(map(str, p2))], env=env, capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    lines = [json.loads(x) for x in out.stdout.splitlines() if x.startswith("{")]
    for p, line in zip((p1, p2), lines):
        want, margin = greedy_oracle(cfg, W, p, 4)
        assert line["prompt"] == p and (line["tokens"] == want or margin < 1e-3)
    # trace replay: two requests, portions beside single tokens, one ends early and its slot is used again
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": p1[:11], "want": [10]}, {"id": "y", "tokens": p2[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": p1[11:12], "want": [0]}, {"id": "y", "tokens": p2[2:], "want": [0, 4]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": p1[12:], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "z", "tokens": p2, "want": [6]}], "end": ["x", "z"]}]
    outdir = str(tmp_path / "out")
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", model, "--dtype", "float32", "--out", outdir, "--max-tokens", "128"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", env=env, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    r1, r2 = O.forward(cfg, W, p1)[0], O.forward(cfg, W, p2)[0]
    V = cfg["vocab"]
    g0, g1, g3 = (np.fromfile(os.path.join(outdir, f"{i}.f32"), "<f4").reshape(-1, V) for i in (0, 1, 3))
    assert not os.path.exists(os.path.join(outdir, "2.f32"))
    assert rel(g0, r1[10:11]) < TOL and rel(g1, np.stack([r1[11], r2[2], r2[6]])) < TOL and rel(g3, r2[6:7]) < TOL


def test_store_refuses_what_it_cannot_run():
    from krasis_amd import serve_store as S
    par = dict(block_kind=S.BLOCK_PARALLEL, norm_kind=S.NORM_RMS, norm_bias=0)
    wkv = dict(heads=2, kv_heads=2, dim=8, vdim=8, mixer_kind=S.MIX_WKV, lin_norm_weight=1, decay_rank=4)
    dlt = dict(heads=4, kv_heads=2, dim=8, vdim=6, mixer_kind=S.MIX_DELTA, lin_norm_weight=2, proj_conv=3)
    att = dict(heads=4, kv_heads=2, dim=8, vdim=8, window=5, keep_first=2)
    lt = dict(lt_heads=2, lt_dim=8, lt_vdim=6)
    bad = [[S.LayerSpec(**{**wkv, "vdim": 6})], [S.LayerSpec(**{**wkv, "decay_rank": 0})], [S.LayerSpec(**wkv, window=4)], [S.LayerSpec(**{**wkv, "kv_heads": 1})],
           [S.LayerSpec(**wkv, keep_first=2)], [S.LayerSpec(**{**dlt, "proj_conv": 0})], [S.LayerSpec(**{**dlt, "kv_heads": 3})], [S.LayerSpec(**{**dlt, "lin_norm_weight": 1})],
           [S.LayerSpec(**{**att, "window": 0}, chunk=8)], [S.LayerSpec(**att, side_mixer=S.MIX_LIGHTNING)], [S.LayerSpec(**att, **lt)], [S.LayerSpec(**att, ff_bias=1)],
           [S.LayerSpec(**att, side_mixer=S.MIX_WKV)], [S.LayerSpec(**att, side_mixer=S.MIX_LIGHTNING, **{**lt, "lt_dim": 600})]]
    for layers in bad:
        with pytest.raises(ValueError):
            S.ServeStore(50, 32, layers, **par)
    with pytest.raises(ValueError):
        S.ServeStore(50, 32, [S.LayerSpec(**att)], block_kind=S.BLOCK_PARALLEL, norm_kind=S.NORM_LAYER, token_side=4)      # the token input is RMS-normed
    with pytest.raises(ValueError):
        S.ServeStore(50, 32, [S.LayerSpec(**att)], pos_rows=16, bigram=(7, 1, 1), **par)                                  # one second table beside the embedding
    st = S.ServeStore(50, 32, [S.LayerSpec(**wkv), S.LayerSpec(**dlt), S.LayerSpec(**att, side_mixer=S.MIX_LIGHTNING, **lt)], pos_rows=40, token_side=3, **par)
    with pytest.raises(RuntimeError):
        st.finalize()                                         # tensors missing
    for layer, role, shape, index in ((0, "q", (8, 32), 0), (0, "wkv_mu", (32,), 5), (0, "delta_b", (2, 32), 0), (1, "q", (32, 32), 0), (1, "lt_q", (16, 32), 0), (2, "lt_v", (16, 32), 0),
                                      (2, "wkv_u", (2, 8), 0), (0, "gate_b", (8,), 0), (-1, "pos", (39, 32), 0), (-1, "side_embed", (50, 3), 0), (2, "side_gate", (4, 32), 0)):
        with pytest.raises(ValueError):
            st.set_tensor(layer, role, np.zeros(shape, np.float32), index)
    st.set_tensor(0, "wkv_mu", np.zeros(32, np.float32), 4)


@pytest.mark.parametrize("n_req", [2, 3])
def test_graph_replays_equal_eager_steps(n_req):
    """decode steps replay a captured graph from their second visit on; every replay is compared with a store that runs eagerly, with eager steps of
    other shapes (a prompt portion of another request) and host synchronisation between the replays"""
    cfg = cfg_wide(); W = O.random_weights(cfg, 41)
    seqs = {r: tokens(cfg, 150, 42 + r) for r in range(n_req)}
    start = {r: 30 - 9 * r for r in range(n_req)}
    c = tokens(cfg, 60, 49)
    eng_g, eng_e = engine(cfg, W, "bfloat16"), engine(cfg, W, "bfloat16")
    eng_e.store.set_use_graph(False)
    for eng in (eng_g, eng_e):
        eng.step([(r, seqs[r][:start[r]], []) for r in seqs])
    for i in range(100):
        entries = [(r, [seqs[r][start[r] + i]], [0]) for r in seqs]
        lg, am = eng_g.step(entries)
        le, ae = eng_e.step(entries)
        assert np.array_equal(lg, le) and np.array_equal(am, ae), i
        if i % 25 == 10:                                    # an eager step of another shape in between
            part = c[(i // 25) * 15:(i // 25) * 15 + 15]
            lg, _ = eng_g.step([("c", part, [14])]); le, _ = eng_e.step([("c", part, [14])])
            assert np.array_equal(lg, le)
    assert eng_g.store.graph_replays() >= 60 and eng_e.store.graph_replays() == 0
    lg, _ = eng_g.step([(0, [seqs[0][130]], [0])])
    ref = O.forward(cfg, {k: O.bf16_round(v) for k, v in W.items()}, seqs[0][:131])[0]
    e = np.sqrt(((lg[0] - ref[130]) ** 2).mean()) / np.sqrt((ref ** 2).mean())
    assert e < 6e-2


def test_mechanisms_in_sequential_blocks():
    """the same mixers as another design may put them together: sequential blocks, lightning attention as a layer's only mixer, feed-forward biases, the token input after
    the feed-forward's own residual"""
    from krasis_amd import model_registry as R, serve_store as S
    from krasis_amd.scheduler import BatchEngine
    base = small_model([O.layer(O.wkv(3, 10, 4), O.dense(24)), O.layer(O.delta(4, 2, 12, 10, 3), None), O.layer(O.parallel(2, 1, 8, 8, 5, 1, 3, 8, 6), O.dense(20)), O.layer(O.wkv(2, 8, 3), None)])
    W = {k: v for k, v in O.random_weights(base, 9).items() if ".left." not in k}
    rng = np.random.default_rng(10)
    for i in (0, 2):
        W[f"l{i}.norm2"] = (1.0 + 0.2 * rng.standard_normal(base["width"])).astype(np.float32)
    spec = R.gasavik_spec(base)
    spec.fit(spec, lambda n: W[n].shape)
    spec.block_kind = S.BLOCK_SEQUENTIAL
    m = base["layers"][2]["mixer"]["right"]
    spec.layers[2] = S.LayerSpec(heads=1, kv_heads=1, dim=1, vdim=1, mixer_kind=S.MIX_LIGHTNING, lt_heads=m["heads"], lt_dim=m["dim"], lt_vdim=m["vdim"], mlp_kind=S.MLP_DENSE, ff=20,
                                 dense_act=S.ACT_SILU, ff_bias=1)
    names = spec.tensors

    def tensors(sp):
        for layer, role, index, name in names(sp):
            if ".left." not in name:
                yield layer, role, index, name
        for i in (0, 2):
            yield i, "norm2_w", 0, f"l{i}.norm2"
    spec.tensors = tensors
    eng = BatchEngine(spec, dtype="float32", max_tokens=256)
    eng.load_arrays(W)
    toks = tokens(base, 80, 3)
    w = {k: v.astype(np.float64) for k, v in W.items()}
    eps, mult = base["norm"]["eps"], base["residual_mult"]
    x = O.embed(base, w, toks)
    for i, lc in enumerate(base["layers"]):
        h = O.rms_unit(x, eps) * w[f"l{i}.norm1"]
        mix = O.mixer_right(m, w, "l2.mix.right.", h, eps) if i == 2 else O.MIXERS[lc["type"]](lc["mixer"], w, f"l{i}.mix.", h, eps)
        x = x + mult * mix
        if lc["mlp"] is not None:
            x = x + mult * O.feed_forward(w, f"l{i}.mlp.", O.rms_unit(x, eps) * w[f"l{i}.norm2"])
        x = x + mult * O.token_side(base, w, i, toks, x, eps)
    ref = (O.rms_unit(x, eps) * w["final.norm"]) @ w["head"].T
    whole, _ = eng.step([("w", toks, list(range(80)))])
    assert rel(whole, ref) < TOL
    rows = [eng.step([("d", toks[:7], [6])])[0][0]] + [eng.step([("d", [t], [0])])[0][0] for t in toks[7:]]
    assert rel(np.stack(rows), ref[6:]) < TOL
