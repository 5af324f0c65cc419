"""Products with resident bfloat16 matrices: one row and many rows, at shapes that
select every tile of the many-row kernel, against float64 sums of the same operands."""
import numpy as np
import pytest
import torch

import nukopel_oracle as N

pytestmark = pytest.mark.gpu


def make(bh, K, Nout, seed):
    rng = np.random.default_rng(seed)
    w = N.bf16(rng.standard_normal((Nout, K)) / np.sqrt(K))
    dev = torch.from_numpy(N.to_bf16_bits(w).view(np.int16)).cuda()
    tiles = torch.empty(bh.buddy_hip_bf16_tiles_bytes(K, Nout), dtype=torch.uint8, device="cuda")
    torch.cuda.synchronize()
    assert bh.buddy_hip_pack_bf16_tiles(dev.data_ptr(), K, Nout, tiles.data_ptr(), None) == 0
    torch.cuda.synchronize()
    return w, tiles


def test_tiles_hold_what_the_layout_says(bh):
    K, Nout = 70, 21
    w, tiles = make(bh, K, Nout, 1)
    got = tiles.cpu().numpy().view(np.uint16)
    assert got.size == 2 * 4 * 512
    want = np.zeros((32, 128), np.uint16)
    want[:Nout, :K] = N.to_bf16_bits(w)
    lanes = np.arange(64)
    for g in range(2):
        for c in range(4):
            tile = got[(g * 4 + c) * 512:][:512].reshape(64, 8)
            for j in range(8):
                np.testing.assert_array_equal(
                    tile[:, j], want[g * 16 + lanes % 16, c * 32 + lanes // 16 * 8 + j])


# rows <= 16, <= 32, 64-row tiles narrow and wide, 128-row tiles; K that ends inside a
# step, a tile and a run of eight
@pytest.mark.parametrize("dtype", [0, 1])
@pytest.mark.parametrize("M,K,Nout", [
    (1, 64, 16), (3, 100, 40), (16, 7, 5), (16, 96, 16500), (20, 130, 65), (32, 64, 17000),
    (50, 1, 1), (64, 333, 96), (200, 192, 130), (300, 320, 4100), (513, 71, 200),
    (1000, 264, 8200), (2048, 512, 4096), (1300, 40, 12000)])
def test_many_rows(bh, M, K, Nout, dtype):
    w, tiles = make(bh, K, Nout, M + K)
    rng = np.random.default_rng(M)
    a = rng.standard_normal((M, K)).astype(np.float32)
    if dtype == 0:
        a = N.bf16(a)
    lda, ldc = (K + 7) // 8 * 8 + 8, (Nout + 15) // 16 * 16 + 4
    # what lies beside the rows must not get in
    if dtype == 0:
        buf = np.full((M, lda), 0x7FC0, np.uint16)
        buf[:, :K] = N.to_bf16_bits(a)
        A = torch.from_numpy(buf.view(np.int16)).cuda()
    else:
        buf = np.full((M, lda), np.nan, np.float32)
        buf[:, :K] = a
        A = torch.from_numpy(buf).cuda()
    C = torch.full((M, ldc), 7.0, device="cuda")
    torch.cuda.synchronize()
    assert bh.buddy_hip_gemm_bf16(A.data_ptr(), lda, dtype, tiles.data_ptr(), C.data_ptr(), ldc,
                                  M, K, Nout, None) == 0
    torch.cuda.synchronize()
    got = C.cpu().numpy()
    want = np.asarray(a, np.float64) @ w.T
    err = np.abs(got[:, :Nout] - want).max()
    assert err < 3e-6 * max(1.0, np.abs(want).max()), err
    assert (got[:, (Nout + 15) // 16 * 16:] == 7.0).all()      # nothing past the padding


@pytest.mark.parametrize("K,Nout", [(64, 16), (1, 3), (37, 50), (2048, 96), (2052, 70), (4100, 33),
                                    (8200, 17), (9001, 20), (1536, 40000), (300, 4100)])
def test_one_row(bh, K, Nout):
    w, tiles = make(bh, K, Nout, K)
    x = np.random.default_rng(K).standard_normal(K).astype(np.float32)
    X = torch.from_numpy(x).cuda()
    y = torch.empty((Nout + 15) // 16 * 16, device="cuda")
    torch.cuda.synchronize()
    assert bh.buddy_hip_gemv_bf16(X.data_ptr(), tiles.data_ptr(), y.data_ptr(), K, Nout, None) == 0
    torch.cuda.synchronize()
    want = w @ x.astype(np.float64)
    err = np.abs(y.cpu().numpy()[:Nout] - want).max()
    assert err < 3e-6 * max(1.0, np.abs(want).max()), err


def test_refusals(bh):
    t = torch.zeros(4096, device="cuda")
    p = t.data_ptr()
    ok = (p, 64, 1, p, p, 16, 4, 64, 16, None)
    for i, bad in ((1, 60), (1, 32), (2, 5), (5, 8), (5, 18), (0, p + 4), (6, 0)):
        args = list(ok)
        args[i] = bad
        assert bh.buddy_hip_gemm_bf16(*args) != 0
    assert bh.buddy_hip_gemv_bf16(None, p, p, 64, 16, None) != 0
    assert bh.buddy_hip_bf16_tiles_bytes(0, 4) == 0
