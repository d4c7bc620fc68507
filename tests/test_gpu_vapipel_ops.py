"""Vapipel's operators one at a time against fp64 restatements: bf16 products
with their epilogues, the fp32 post-sublayer norm, latent attention over pages
(bf16 MFMA form, bf16 row form, fp32)."""
import ctypes

import numpy as np
import pytest

import flexflow_amd.ffmi as F
from hip_util import Buf
from vapipel_models import bf16, bf16_bits

pytestmark = pytest.mark.gpu


def to_f32(bits):
    return (bits.astype(np.uint32) << 16).view(np.float32)


@pytest.mark.parametrize("T,N,K", [(1, 32, 32), (5, 96, 64), (16, 1056, 320), (17, 544, 4096),
                                   (40, 2048, 96), (8, 17408, 512), (24, 16384, 1024), (64, 160, 2080),
                                   (65, 416, 352), (168, 1024, 2048), (300, 96, 4128), (520, 4096, 512),
                                   (1024, 4096, 1088)])
def test_linear_bf16_epilogues(T, N, K):
    rng = np.random.default_rng(T + N + K)
    X, W = bf16(rng.uniform(-1, 1, (T, K))), bf16(rng.uniform(-1, 1, (N, K)))
    ref = X.astype(np.float64) @ W.astype(np.float64).T
    mag = np.abs(X).astype(np.float64) @ np.abs(W).astype(np.float64).T
    bx, bw = Buf(bf16_bits(X)), Buf(bf16_bits(W))
    L = F.lib()
    out = {}
    for epi, dt in ((F.BF16_PLAIN, np.uint16), (F.BF16_RELU2, np.uint16), (F.BF16_SUM, np.float32)):
        y = Buf.empty((T, N), dt)
        assert L.ffmi_linear_bf16(bx.ptr, bw.ptr, y.ptr, T, N, K, epi, None) == 0
        out[epi] = y.get()
    s = out[F.BF16_SUM]
    assert (np.abs(s - ref) <= 2e-6 * mag + 1e-6).all()
    # the 16-bit epilogues: the sums rounded once (another split of K may move a sum by an ulp)
    p = to_f32(out[F.BF16_PLAIN]).astype(np.float64)
    assert (np.abs(p - ref) <= 2.0 ** -8 * np.abs(ref) + 3e-6 * mag).all()
    r = np.maximum(ref, 0.0)
    q = to_f32(out[F.BF16_RELU2]).astype(np.float64)
    assert (np.abs(q - r * r) <= 2.0 ** -8 * r * r + 2 * (r + 3e-6 * mag) * 3e-6 * mag).all()


def test_linear_bf16_rows_do_not_depend_on_the_batch():
    rng = np.random.default_rng(5)
    X, W = bf16(rng.standard_normal((64, 512))), bf16(rng.standard_normal((288, 512)))
    bw = Buf(bf16_bits(W))
    L = F.lib()
    rows = []
    for T in (1, 7, 33):
        y = Buf.empty((T, 288), np.float32)
        assert L.ffmi_linear_bf16(Buf(bf16_bits(X[:T])).ptr, bw.ptr, y.ptr, T, 288, 512, F.BF16_SUM,
                                  None) == 0
        rows.append(y.get()[0])
    assert (rows[0] == rows[1]).all() and (rows[0] == rows[2]).all()


@pytest.mark.parametrize("T,H,n,slabs", [(1, 32, 32, 1), (3, 96, 70, 2), (5, 1024, 1000, 3),
                                         (2, 2048, 2048, 8), (7, 4096, 4096, 4), (2, 8192, 8192, 1),
                                         (1, 16384, 16370, 1)])
def test_post_norm(T, H, n, slabs):
    rng = np.random.default_rng(H + slabs)
    y = rng.standard_normal((slabs, T, H)).astype(np.float32)
    y[:, :, n:] = 0
    w, x = rng.standard_normal(H).astype(np.float32), rng.standard_normal((T, H)).astype(np.float32)
    eps = 1e-3
    by, bw, bx = Buf(y), Buf(w), Buf(x)
    assert F.lib().ffmi_post_rmsnorm(by.ptr, slabs, bw.ptr, bx.ptr, T, H, n, eps, None) == 0
    s = y.astype(np.float64).sum(0)
    ref = x + s / np.sqrt((s * s).sum(1, keepdims=True) / n + eps) * w
    assert np.abs(bx.get() - ref).max() < 2e-5


def attention(q, cache, heads, scale, seqs, full):
    """seqs: (tokens, first position, pages).  fp64 rows of the same."""
    rank = q.shape[-1]
    arr = (F.PagedSeq * len(seqs))()
    keep = []
    for a, (n, p0, pages) in zip(arr, seqs):
        t = np.ascontiguousarray(pages, np.int32)
        keep.append(t)
        a.num_tokens, a.pos0 = n, p0
        a.pages = t.ctypes.data_as(ctypes.POINTER(ctypes.c_int32))
    enc = (lambda v: np.ascontiguousarray(v, np.float32)) if full else bf16_bits
    bq, bc = Buf(enc(q)), Buf(enc(cache))
    bo = Buf.empty(q.shape, np.float32 if full else np.uint16)
    print("latent attention", q.shape, heads, rank, scale, seqs, full, flush=True)
    assert F.lib().ffmi_latent_attention(bq.ptr, bc.ptr, len(cache), bo.ptr, heads, rank, scale, arr,
                                         len(seqs), int(full)) == 0
    got = bo.get() if full else to_f32(bo.get())
    ref = np.empty(q.shape)
    t0 = 0
    for n, p0, pages in seqs:
        flat = cache[np.asarray(pages)].reshape(-1, rank).astype(np.float64)
        for i in range(n):
            rows = slice((t0 + i) * heads, (t0 + i + 1) * heads)
            c = flat[:p0 + i + 1]
            s = q[rows].astype(np.float64) @ c.T * scale
            e = np.exp(s - s.max(1, keepdims=True))
            ref[rows] = e / e.sum(1, keepdims=True) @ c
        t0 += n
    return got.astype(np.float64), ref


def paged(rng, lens, spare=3):
    """distinct shuffled pages for requests of the given total lengths"""
    need = [(n + 63) // 64 for n in lens]
    order = rng.permutation(sum(need) + spare)
    out, at = [], 0
    for k in need:
        out.append(order[at:at + k])
        at += k
    return out, len(order)


CASES = [(1, 64), (3, 64), (5, 128), (16, 192), (20, 256), (2, 384), (32, 512), (40, 512), (7, 512),
         (3, 576), (130, 64)]


@pytest.mark.parametrize("heads,rank", CASES)
@pytest.mark.parametrize("full", [False, True])
def test_latent_attention_batches(heads, rank, full):
    """Decoding rows of several requests, one portion of a prompt and a whole
    prompt, on shuffled pages; positions at and around page edges."""
    rng = np.random.default_rng(heads * 1000 + rank)
    spans = [(1, 0), (1, 63), (1, 64), (1, 200), (2, 126), (9, 60), (70, 0)]
    if heads <= 8:
        spans += [(1, 1300), (3, 700)]
    pages, total = paged(rng, [n + p for n, p in spans])
    cache = bf16(rng.standard_normal((total, 64, rank)))
    T = sum(n for n, _ in spans)
    q = bf16(rng.standard_normal((T * heads, rank)))
    got, ref = attention(q, cache, heads, 1.5 / np.sqrt(rank), [(n, p, g) for (n, p), g in zip(spans, pages)], full)
    tol = 2e-5 if full else 2.5e-2
    assert np.abs(got - ref).max() < tol * np.abs(ref).max()


@pytest.mark.parametrize("full", [False, True])
@pytest.mark.parametrize("heads,rank", [(2, 64), (20, 512), (33, 128), (4, 576)])
def test_latent_attention_finds_each_key(heads, rank, full):
    """One key stands out: at the first position, either side of every page
    edge, the query's own position -- and just past it, where it must not be
    seen.  The output is that key's latent, or the others' mean."""
    rng = np.random.default_rng(rank + heads)
    pos, scale = 131, 1.0
    pages, total = paged(rng, [pos + 1 + 60])
    unit = rng.standard_normal(rank)
    unit = bf16(unit / np.linalg.norm(unit))
    for n_tok in (1, 3):  # decoded alone / inside a portion
        for key in (0, 1, 63, 64, 127, 128, pos - 1, pos, pos + 1):
            base = bf16(rng.standard_normal((total, 64, rank)) * 0.01)
            cache = base.copy()
            g = pages[0]
            cache[g[key // 64], key % 64] = unit
            q = np.repeat(bf16(40.0 * unit)[None], n_tok * heads, 0)
            got, ref = attention(q, cache, heads, scale, [(n_tok, pos - n_tok + 1, g)], full)
            assert np.abs(got - ref).max() < (1e-4 if full else 1e-2), (n_tok, key)
            last = got[-heads:]  # the rows at `pos`
            seen = np.abs(last @ unit - 1.0).max() < 0.05
            assert seen == (key <= pos), (n_tok, key)


def test_latent_attention_rejects_bad_tables():
    q = Buf.empty((2, 64), np.uint16)
    c = Buf.empty((2, 64, 64), np.uint16)
    t = np.array([0, 2], np.int32)
    s = F.PagedSeq(1, 64, t.ctypes.data_as(ctypes.POINTER(ctypes.c_int32)))
    L = F.lib()
    assert L.ffmi_latent_attention(q.ptr, c.ptr, 2, q.ptr, 2, 64, 1.0, ctypes.byref(s), 1, 0) == 1
    assert L.ffmi_latent_attention(q.ptr, c.ptr, 2, q.ptr, 2, 72, 1.0, ctypes.byref(s), 1, 0) == 5
