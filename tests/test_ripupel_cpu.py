"""Host-side parts of the Ripupel design that need no GPU: its config reader (every size and constant from config.json), its tensor names, the registry's
choice, a checkpoint round trip, and the oracle's own mechanisms against closed forms."""
import json
import os

import numpy as np
import pytest

from krasis_amd import model_registry as R
from krasis_amd import serve_store as S
from tests import oracle_ripupel as O


def small_cfg():
    return O.make_config(width=40, vocab=37, eps=3e-6, embed_scale=2.5, layers=[
        O.layer(O.rglru(36, 3, 5), O.dense(20)),
        O.layer(O.latent(6, 8, 4, 10, 14, scale=0.2, base=123.0), O.moe(9, 4, 12)),
        O.layer(O.rglru(28, 7, 1), None),
        O.layer(O.latent(5, 12, 4, 6, 14, scale=0.3, base=123.0, kv_from=1), O.dense(16)),
        O.layer(O.latent(2, 16, 8, 16, 30, scale=0.15, base=77.0), O.moe(4, 1, 24)),
    ])


def test_config_reader_takes_every_size_and_constant_from_config():
    cfg = small_cfg()
    spec = R.ripupel_spec(cfg)
    assert (spec.vocab, spec.width, spec.norm_kind, spec.norm_eps, spec.embed_scale) == (37, 40, S.NORM_LAYER, 3e-6, 2.5)
    assert (spec.block_kind, spec.pre_norm, spec.post_norm, spec.norm_bias, spec.residual_mult) == (S.BLOCK_SEQUENTIAL, 1, 1, 0, 1.0)
    a, b, c, d, e = spec.layers
    assert (a.mixer_kind, a.rg_width, a.rg_blocks, a.rg_conv, a.rg_rate, a.mlp_kind, a.ff, a.dense_act) == (S.MIX_RGLRU, 36, 3, 5, 8.0, S.MLP_DENSE, 20, S.ACT_SILU)
    assert (c.rg_width, c.rg_blocks, c.rg_conv, c.mlp_kind) == (28, 7, 1, S.MLP_NONE)
    assert (b.mixer_kind, b.heads, b.kv_heads, b.dim, b.vdim, b.kv_rank, b.q_rank, b.rot_dims, b.rot_interleaved, b.rot_base, b.scale) == \
        (S.MIX_LATENT, 6, 1, 8, 10, 14, 0, 4, 0, 123.0, 0.2)
    assert (b.has_sink, b.out_gate, b.kv_from, b.window, b.chunk) == (S.SINK_TENSOR, S.OGATE_ELEM_SIGMOID, -1, 0, 0)
    assert (b.mlp_kind, b.experts, b.top, b.groups, b.keep, b.renorm, b.router_score, b.router_bias, b.expert_in_weight, b.expert_ff, b.expert_act, b.shared_ff) == \
        (S.MLP_MOE, 9, 4, 1, 1, 0, S.RSCORE_SIGMOID, 0, 1, 12, S.ACT_SILU, 0)
    assert (d.kv_from, d.heads, d.dim, d.vdim, d.kv_rank, d.scale) == (1, 5, 12, 6, 14, 0.3)
    assert (e.kv_from, e.rot_base, e.rot_dims, e.kv_rank, e.top) == (-1, 77.0, 8, 30, 1)
    W = O.random_weights(cfg, 0)
    roles = list(spec.tensors(spec))
    assert {n for _, _, _, n in roles} == set(W)              # the store asks for exactly the checkpoint's tensors
    assert sorted(n for _, _, _, n in roles if n == "embed") == ["embed", "embed"]      # as table and as vocabulary projection
    assert not [n for _, _, _, n in roles if n in ("l3.mix.dkv", "l3.mix.dkv.norm", "l2.norm2", "l2.norm2b")]


def test_config_reader_refuses_what_the_design_has_not():
    for edit in (lambda c: c["layers"][0].update(type="retention"), lambda c: c["layers"][0]["mlp"].update(kind="gated"), lambda c: c["layers"][1]["mixer"]["rot"].update(dims=2)):
        bad = json.loads(json.dumps(small_cfg())); edit(bad)
        with pytest.raises(ValueError):
            R.ripupel_spec(bad)


def test_registry_and_checkpoint_roundtrip(tmp_path):
    assert {"Ripupel", "Lufozen", "Midisun", "Pamulix", "Lomutar"} <= set(R.architectures())
    cfg = small_cfg(); W = O.random_weights(cfg, 0)
    assert R.model_family(cfg) == "serve:Ripupel"
    O.write_checkpoint(str(tmp_path), cfg, W)
    assert R.read_config(str(tmp_path)) == cfg
    f = R.SafetensorsFile(os.path.join(tmp_path, "model.safetensors"))
    assert sorted(f.names()) == sorted(W)
    assert f.shape("l0.mix.ra") == (3, 12, 12) and f.shape("l0.mix.ri.b") == (3, 12) and f.shape("l2.mix.conv") == (28, 1)
    got = f.get("l0.mix.lam")
    assert got.dtype == np.uint16 and np.array_equal((got.astype(np.uint32) << 16).view(np.float32), O.bf16_round(W["l0.mix.lam"]))


def test_structures_match_the_header():
    """the Python mirror of the store's structures lists the header's fields in the header's order"""
    import re

    from krasis_amd import _lib
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    src = open(os.path.join(root, "include", "krasis_hip.h")).read()
    assert int(re.search(r"#define KR_SERVE_ABI (\d+)", src).group(1)) == _lib.SERVE_ABI
    for cls, name in ((_lib.ServeLayerC, "kr_serve_layer"), (_lib.ServeConfigC, "kr_serve_config")):
        body = src[:src.index("} " + name + ";")]
        body = re.sub(r"/\*.*?\*/", "", body[body.rindex("typedef struct {") + len("typedef struct {"):], flags=re.S)
        fields = [v.strip() for decl in body.split(";") if decl.strip() for v in decl.strip().split(None, 1)[1].split(",")]
        assert fields == [f[0] for f in cls._fields_]
    roles = src[src.index("enum { KR_SV_EMBED"):]
    roles = re.sub(r"/\*.*?\*/", "", roles[:roles.index("};")], flags=re.S)
    assert [r.lower() for r in re.findall(r"KR_SV_(\w+)", roles)][:-1] == list(S.ROLES)


def test_oracle_mechanisms_against_closed_forms():
    rng = np.random.default_rng(0)
    # layer norm: no bias, variance from the mean
    x = rng.standard_normal((3, 10)) + 5.0
    y = O.layer_norm(x, np.full(10, 2.0), 0.0)
    assert np.allclose(y.mean(-1), 0.0) and np.allclose(y.std(-1), 2.0)
    # convolution: the last column is the current token's
    u = rng.standard_normal((5, 2)); w = rng.standard_normal((2, 3)); b = rng.standard_normal(2)
    y = O.causal_conv(u, w, b)
    assert np.allclose(y[0], b + w[:, 2] * u[0]) and np.allclose(y[4], b + w[:, 0] * u[2] + w[:, 1] * u[3] + w[:, 2] * u[4])
    # gates: part b of u meets matrix b only
    g = O.block_gate(np.array([[1.0, 2.0, 3.0, 4.0]]), np.array([[[1.0, 0.5], [0.0, 1.0]], [[0.0, 1.0], [2.0, 0.0]]]), np.array([[0.1, 0.2], [0.3, 0.4]]))
    assert np.allclose(g, O.sigmoid(np.array([[2.1, 2.2, 4.3, 6.4]])))
    # the recurrence as a sum over earlier tokens: S_t = sum_s (prod_{s < q <= t} a_q) sqrt(1 - a_s^2) i_s u_s; the first token is no special case
    T, C = 7, 3
    u, r, i, lam = rng.standard_normal((T, C)), O.sigmoid(rng.standard_normal((T, C))), O.sigmoid(rng.standard_normal((T, C))), rng.standard_normal(C)
    got = O.gated_recurrence(u, r, i, lam)
    a = np.exp(-8.0 * r * np.log1p(np.exp(lam)))
    want = np.zeros((T, C))
    for t in range(T):
        for s in range(t + 1):
            want[t] += np.prod(a[s + 1:t + 1], axis=0) * np.sqrt(1.0 - a[s] ** 2) * i[s] * u[s]
    assert np.allclose(got, want) and np.allclose(got[0], np.sqrt(1.0 - a[0] ** 2) * i[0] * u[0])
    # rotation: pairs (i, i + d / 2), position 0 leaves a vector alone, scores depend on the distance only
    x = rng.standard_normal((6, 2, 4))
    y = O.rotate(x, 50.0)
    assert np.array_equal(y[0], x[0])
    ang = 3 * 50.0 ** -0.5
    assert np.allclose(y[3, 1, 1], x[3, 1, 1] * np.cos(ang) - x[3, 1, 3] * np.sin(ang)) and np.allclose(y[3, 1, 3], x[3, 1, 3] * np.cos(ang) + x[3, 1, 1] * np.sin(ang))
    same = O.rotate(np.tile(x[0, 0], (6, 1)), 50.0)
    assert np.allclose(same[1] @ same[4], same[2] @ same[5])
    # sink: weights sum to less than one, by exactly the sink's share
    p = O.sink_softmax(np.array([[0.0, np.log(2.0), -np.inf]]), np.log(3.0))
    assert np.allclose(p, [[1 / 6, 2 / 6, 0.0]])
    # the router: sigmoid scores as they are, largest first; the weight goes into the expert
    h = rng.standard_normal((4, 6)); wr = rng.standard_normal((5, 6))
    ids, wt = O.route(h, wr, 2)
    s = O.sigmoid(h @ wr.T)
    assert np.array_equal(ids[:, 0], s.argmax(-1)) and np.allclose(wt[:, 0], s.max(-1)) and np.allclose(wt[:, 1], np.sort(s, -1)[:, -2])
    W = {"m.router": wr}
    for e in range(5):
        for n, shape in (("gate", (3, 6)), ("up", (3, 6)), ("down", (6, 3))):
            W[f"m.e{e}.{n}"] = rng.standard_normal(shape)
    got = O.experts_ff(h, W, "m.", 2)
    want = sum(O.gated_ff(h[t:t + 1] * wt[t, k], W, f"m.e{ids[t, k]}.") for t in (1,) for k in range(2))
    assert np.allclose(got[1], want[0])


def test_a_borrowed_latent_is_the_lenders(monkeypatch):
    """the oracle: a layer with kv_from reads the named layer's rows, which that layer formed from ITS input"""
    cfg = O.make_config(width=24, vocab=19, layers=[O.layer(O.latent(2, 6, 4, 5, 9), None), O.layer(O.latent(3, 4, 4, 6, 9), O.dense(10)),
                                                    O.layer(O.latent(2, 8, 4, 7, 9, kv_from=0), None)])
    W = O.random_weights(cfg, 3); toks = [3, 1, 4, 1, 5, 9, 2, 6]
    base, _ = O.forward(cfg, W, toks)
    for src in (1,):
        c2 = json.loads(json.dumps(cfg)); c2["layers"][2]["mixer"]["kv_from"] = src
        assert np.abs(O.forward(c2, W, toks)[0] - base).max() > 1e-2
    seen = []
    real = O.latent_rows
    monkeypatch.setattr(O, "latent_rows", lambda m, w, p, h, eps: seen.append(p) or real(m, w, p, h, eps))
    O.forward(cfg, W, toks)
    assert seen == ["l0.mix.", "l1.mix."]
