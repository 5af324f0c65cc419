"""The plain Nukopel implementation of the tests against closed forms, and what the
library says about model folders without touching a GPU."""
import ctypes
import json

import numpy as np
import pytest

import nukopel_models as M
import nukopel_oracle as N


def test_norm_has_eps_inside_the_root():
    x = np.array([[3e-3, -4e-3]])
    np.testing.assert_allclose(N.scalar_norm(x, 2.0, 1e-5),
                               2 * x / np.sqrt(12.5e-6 + 1e-5), rtol=1e-12)


def test_input_convolution_is_causal_and_adds_its_input():
    rng = np.random.default_rng(0)
    h, w = rng.standard_normal((9, 4)), rng.standard_normal((4, 3))
    got = N.input_conv(h, w)
    for c in range(4):
        full = np.convolve(h[:, c], w[c, ::-1])[:9]
        np.testing.assert_allclose(got[:, c], h[:, c] + full, rtol=1e-12)


def test_rotation_depends_on_the_gap_only():
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((1, 8)), rng.standard_normal((1, 8))
    dots = [float((N.rotate(q, np.array([p]), 100.0) @ N.rotate(k, np.array([p - 5.0]), 100.0).T)[0, 0])
            for p in (5.0, 17.0, 400.0)]
    np.testing.assert_allclose(dots, dots[0], rtol=1e-9)
    np.testing.assert_array_equal(N.rotate(q, np.array([0.0]), 100.0), q)
    a = N.rotate(np.array([[1.0, 0, 0, 0]]), np.array([1.0]), 100.0)   # 0 turns with 2
    np.testing.assert_allclose(a, [[np.cos(1), 0, np.sin(1), 0]], rtol=1e-12, atol=1e-15)


def test_lightning_is_a_decayed_double_sum():
    rng = np.random.default_rng(2)
    c = M.linear(decay=(0.6, 0.95), dim=4, vdim=3)["mixer"]
    W, n = 10, 7
    w = {k: rng.standard_normal(s) for k, s in
         dict(q=(8, W), k=(8, W), v=(6, W), g=(6, W), o=(W, 6), norm=(6,)).items()}
    h = rng.standard_normal((n, W))
    q, k, v = (N.silu(h @ w[x].T) for x in "qkv")
    o = np.zeros((n, 6))
    for hd in range(2):
        for i in range(n):
            for j in range(i + 1):
                s = q[i, hd * 4:hd * 4 + 4] @ k[j, hd * 4:hd * 4 + 4]
                o[i, hd * 3:hd * 3 + 3] += c["decay"][hd] ** (i - j) * s * v[j, hd * 3:hd * 3 + 3]
    o = o / np.sqrt((o * o).mean(-1, keepdims=True) + 1e-5) * w["norm"] * N.sigmoid(h @ w["g"].T)
    np.testing.assert_allclose(N.lightning(h, w, c, 1e-5), o @ w["o"].T, rtol=1e-9)


def test_window_of_one_returns_the_tokens_own_value():
    rng = np.random.default_rng(3)
    c = M.latent(heads=2, dim=4, rot=2, vdim=3, rank=5, window=1)["mixer"]
    W = 6
    w = {k: rng.standard_normal(s) for k, s in
         {"q": (12, W), "dkv": (7, W), "dkv.norm": (5,), "uk": (8, 5), "uv": (6, 5), "g": (2, W),
          "o": (W, 6)}.items()}
    h = rng.standard_normal((4, W))
    lat = N.rms((h @ w["dkv"].T)[:, :5], 1e-5) * w["dkv.norm"]
    v = lat @ w["uv"].T * np.repeat(N.sigmoid(h @ w["g"].T), 3, axis=1)
    np.testing.assert_allclose(N.latent_attention(h, w, c, 1e-5), v @ w["o"].T, rtol=1e-9)


def test_expert_limits_and_routing():
    h = np.array([[1.0]])
    one = np.ones((1, 1))
    # gate cut from above only, up on both sides
    assert N.expert(h, 9 * one, -9 * one, one, 2.0)[0, 0] == pytest.approx(
        2 * (1 / (1 + np.exp(-3.404))) * (-2 + 1))
    assert N.expert(h, -9 * one, 0 * one, one, 2.0)[0, 0] == pytest.approx(
        -9 * (1 / (1 + np.exp(9 * 1.702))))
    idx, w = N.route(np.array([[1.0]]), np.array([[0.5], [2.0], [2.0], [-1.0]]), 2)
    assert idx.tolist() == [[1, 2]] and w.tolist() == [[0.5, 0.5]]


def test_bfloat16_rounding_is_to_nearest_even():
    assert N.bf16(1.00390625) == 1.0 and N.bf16(1.01171875) == 1.015625


def test_file_round_trip(tmp_path):
    folder, t = M.build(tmp_path, M.SIZES["odd"])
    cfg, back = N.read_model(folder)
    assert cfg == M.SIZES["odd"] and set(back) == set(t)
    for k in t:
        np.testing.assert_array_equal(back[k], t[k])


@pytest.mark.parametrize("what", ["window", "taps", "order", "shared", "limit", "decay"])
def test_every_mechanism_shows_in_the_logits(what):
    """The random models are only worth comparing if a mistake is visible in them:
    plant one in the oracle's configuration and look."""
    cfg = json.loads(json.dumps(M.SIZES["mixed"]))
    t = N.random_tensors(cfg, 0)
    tokens = np.random.default_rng(4).integers(0, cfg["vocab"], 40)
    good = N.forward(cfg, t, tokens)
    bad = json.loads(json.dumps(cfg))
    t = dict(t)
    if what == "window":
        bad["layers"][0]["mixer"]["mask"]["size"] -= 1
    elif what == "taps":
        t["l1.canon1"] = np.roll(t["l1.canon1"], 1, axis=1)
    elif what == "order":
        t["l0.mix.uk"] = t["l0.mix.uk"][::-1]
    elif what == "shared":
        bad["layers"][2]["mlp"]["shared"] = None
    elif what == "limit":
        bad["layers"][1]["mlp"]["expert"]["limit"] += 0.1
    elif what == "decay":
        bad["layers"][1]["mixer"]["decay"][2] = 0.99
    assert M.row_errors(N.forward(bad, t, tokens), good).max() > 2e-3


# ---- the library, no GPU ---------------------------------------------------------

def create(bh, folder):
    h = bh.buddy_hip_session_create_from_folder(str(folder).encode(), None)
    if h:
        bh.buddy_hip_session_destroy(h)
    return h, bh.buddy_hip_last_error().decode()


def test_registry_knows_the_architecture():
    from buddy_mlir_amd.session import architectures
    assert "Nukopel" in architectures()


def test_folder_errors_are_reported(bh, tmp_path):
    assert "config.json" in create(bh, tmp_path / "nothing")[1]
    folder, _ = M.build(tmp_path / "m", M.SIZES["odd"])
    cfg = json.loads((folder / "config.json").read_text())
    (folder / "config.json").write_text(json.dumps({**cfg, "architecture": "Somebody"}))
    h, msg = create(bh, folder)
    assert not h and "Somebody" in msg
    (folder / "config.json").write_text('{"architecture": ')
    h, msg = create(bh, folder)
    assert not h and "JSON" in msg
    (folder / "config.json").write_text(json.dumps(cfg))
    raw = (folder / "model.safetensors").read_bytes()
    for broken in (raw[:4], raw[:-7], b"\xff" * 8 + raw[8:], raw[:8] + b"[" + raw[9:]):
        (folder / "model.safetensors").write_bytes(broken)
        h, msg = create(bh, folder)
        assert not h and msg
    assert not bh.buddy_hip_session_create_from_folder(None, None)


def test_options_are_checked(bh, tmp_path):
    from buddy_mlir_amd.session import ModelOptions
    folder, _ = M.build(tmp_path, M.SIZES["odd"])
    for bad in (ModelOptions(7, 0, 0, None), ModelOptions(0, -1, 0, None)):
        assert not bh.buddy_hip_session_create_from_folder(str(folder).encode(), ctypes.byref(bad))
