"""Every mechanism of the Sopulorn decoder alone: the kernel against the plain function of
``tests/plain/sopulorn.py``, at sizes of the tests' own, whole and in steps, beside other requests
and padding, with inputs made so that a lost token, a far key or the sink shows."""

from __future__ import annotations

import pytest
import torch

from tests.darovik_helpers import batch_tensors
from tests.plain import sopulorn as plain

pytestmark = pytest.mark.gpu

DEV = "cuda"
F64 = torch.float64
DTYPES = [torch.float32, torch.bfloat16]
IDS = ["f32", "bf16"]


def gpu(t, dtype=torch.float32):
    return t.to(device=DEV, dtype=dtype).contiguous()


def rel(got, want):
    return float((got.double().cpu() - want).pow(2).mean().sqrt() / (want.pow(2).mean().sqrt() + 1e-30))


def rnd(*shape, gen, std=1.0, dtype=F64):
    """Random values that ``dtype`` holds exactly, in float64."""
    t = torch.randn(*shape, generator=gen, dtype=F64) * std
    return t if dtype == F64 else t.to(dtype).double()


# ------------------------------------------------------------------- the pair embedding
@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("V,H,bucket", [(211, 96, (101, 7, 29)), (70001, 40, (60013, 8191, 131)),
                                        (97, 300, (1, 5, 0)), (50, 8, (7, 0, 3)), (65000, 16, (997, 100003, 65537))])
def test_pair_embedding_in_steps_beside_others_and_padding(dtype, V, H, bucket):
    """Three requests cut into steps of one to many tokens, one that pauses, a slot that is used
    again, padding; the state starts as leftovers that must not be read.  Products beyond 32 bits."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(V + H)
    buckets, mul_prev, mul_cur = bucket
    w = {"embed": rnd(V, H, gen=gen, dtype=torch.bfloat16), "bigram": rnd(buckets + 1, H, gen=gen, dtype=torch.bfloat16)}
    cfg = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}
    seqs = {k: torch.randint(V - min(V, 60), V, (n,), generator=gen).tolist() for k, n in
            (("a", 40), ("b", 9), ("c", 17), ("d", 5))}
    want = {k: plain.embedding(cfg, w, v) for k, v in seqs.items()}
    slot = {"a": 3, "b": 0, "c": 1, "d": 0}  # d follows b in its slot
    last = torch.full((4, 1), -1, dtype=torch.int32, device=DEV)
    at = dict.fromkeys(seqs, 0)
    table, pairs = gpu(w["embed"], dtype), gpu(w["bigram"], dtype)
    plan = [[("a", 7), ("b", 1)], [("b", 2), None, ("c", 1), ("a", 1)], [("c", 1), ("b", 6), None], [("a", 31), ("d", 4)],
            [("c", 15), ("d", 1), ("a", 1)]]
    for group in plan:
        reqs, ids = [], []
        for item in group:
            if item is None:
                reqs.append(None)
                ids.append(0)
            else:
                k, n = item
                reqs.append((slot[k], at[k], n))
                ids += seqs[k][at[k]: at[k] + n]
        batch, T = batch_tensors(reqs)
        batch.pop("num_reqs")
        out = torch.full((T, H), float("nan"), device=DEV)
        ops.embed_pairs(out, table, pairs, torch.tensor(ids, dtype=torch.int32, device=DEV), last,
                        mul_prev=mul_prev, mul_cur=mul_cur, **batch)
        row = 0
        for item in group:
            if item is None:
                assert float(out[row].abs().max()) == 0.0
                row += 1
                continue
            k, n = item
            assert torch.equal(out[row: row + n].double().cpu(), want[k][at[k]: at[k] + n].float().double()), (k, at[k])
            at[k] += n
            row += n
    assert all(at[k] == len(v) for k, v in seqs.items())
    # a later token whose slot holds no token shows as NaN instead of some row
    last.fill_(-1)
    batch, T = batch_tensors([(2, 5, 2)])
    batch.pop("num_reqs")
    out = torch.empty((T, H), device=DEV)
    ops.embed_pairs(out, table, pairs, torch.tensor([V - 1, V - 2], dtype=torch.int32, device=DEV), last,
                    mul_prev=mul_prev, mul_cur=mul_cur, **batch)
    assert torch.isnan(out[0]).all() and torch.isfinite(out[1]).all() and int(last[2]) == V - 2


# --------------------------------------------------------------------------- attention
def pages_of(k, v, page, dtype):
    """Keys and values ``[S, G, d / dv]`` in pages of a shuffled order: caches and a table whose row 1
    names them (places nobody wrote hold NaN)."""
    S, G, d = k.shape
    dv = v.shape[2]
    n_pages = -(-S // page)
    order = torch.randperm(n_pages, generator=torch.Generator().manual_seed(1))
    k_cache = torch.full((n_pages + 1, G, page, d), float("nan"), dtype=dtype, device=DEV)
    v_cache = torch.full((n_pages + 1, G, dv, page), float("nan"), dtype=dtype, device=DEV)
    table = torch.zeros((2, n_pages), dtype=torch.int32, device=DEV)
    for p in range(n_pages):
        pid = int(order[p]) + 1
        table[1, p] = pid
        n = min(page, S - p * page)
        k_cache[pid, :, :n] = gpu(k[p * page:p * page + n].transpose(0, 1), dtype)
        v_cache[pid, :, :, :n] = gpu(v[p * page:p * page + n].permute(1, 2, 0), dtype)
        k_cache[pid, :, n:] = 0  # the rest of the last page: beyond every query, never seen
        v_cache[pid, :, :, n:] = 0
    return k_cache, v_cache, table


def attend(q, k, v, page, *, scale, dtype, sink=True, positions=None, kernel="general", nsplit=1):
    from kvcore_amd.ops import library as ops

    T, H, d = q.shape
    G, dv = v.shape[1:]
    k_cache, v_cache, table = pages_of(k, v, page, dtype)
    pos = list(range(T)) if positions is None else positions
    ints = dict(dtype=torch.int32, device=DEV)
    out = torch.full((T, H * dv), float("nan"), dtype=dtype, device=DEV)
    common = dict(table=table, slots=torch.tensor([1], **ints), nh=H, nkv=G, d=d, dv=dv, scale=scale,
                  sinks=torch.zeros(H, device=DEV) if sink else None)
    rows = gpu(q.reshape(T, -1), dtype)
    parts = {}
    if nsplit > 1:
        parts = dict(nsplit=nsplit, part_o=torch.full((T * H * nsplit, dv), float("nan"), device=DEV),
                     part_ml=torch.full((T * H * nsplit, 2), float("nan"), device=DEV))
    if kernel == "portion":
        ops.prefill_attention(out, rows, k_cache, v_cache, positions=torch.tensor(pos, **ints),
                              q_start=torch.tensor([0, T], **ints), num_reqs=1, **common, **parts)
    elif kernel == "single":
        for i in range(T):
            ops.decode_attention(out[i:i + 1], rows[i:i + 1], k_cache, v_cache, positions=torch.tensor(pos[i:i + 1], **ints),
                                 token_req=torch.zeros(1, **ints), **common, **parts)
    else:
        ops.paged_attention(out, rows, k_cache, v_cache, positions=torch.tensor(pos, **ints),
                            token_req=torch.zeros(T, **ints), **common)
    return out.double().cpu().view(T, H, dv)


def plain_heads(q, k, v, scale):
    T, H, _ = q.shape
    g = H // k.shape[1]
    return torch.stack([plain.softmax_with_one((q[:, h] @ k[:, h // g].T) * scale) @ v[:, h // g] for h in range(H)], 1)


@pytest.mark.parametrize("H,G,d,dv,page", [(4, 2, 24, 40, 8), (1, 1, 8, 1, 4), (6, 2, 16, 24, 16), (3, 1, 280, 72, 16)])
def test_the_denominator_s_one_in_the_general_kernel(H, G, d, dv, page):
    gen = torch.Generator().manual_seed(d)
    T = 90
    q, k, v = (rnd(T, n, s, gen=gen, dtype=torch.bfloat16) for n, s in ((H, d), (G, d), (G, dv)))
    want = plain_heads(q, k, v, 0.3 * d ** -0.5)
    kw = dict(scale=0.3 * d ** -0.5)
    assert rel(attend(q, k, v, page, dtype=torch.float32, **kw), want) < 2e-6
    assert rel(attend(q, k, v, page, dtype=torch.float32, sink=False, **kw), want) > 1e-2
    assert rel(attend(q, k, v, page, dtype=torch.bfloat16, **kw), want) < 1e-2


@pytest.mark.parametrize("kernel,nsplit", [("portion", 1), ("portion", 3), ("single", 1), ("single", 4)])
@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 64, 32), (16, 4, 128, 64), (8, 1, 64, 32), (3, 3, 128, 64), (16, 1, 32, 16),
                                      (4, 2, 96, 48), (2, 1, 256, 128), (4, 4, 64, 64), (2, 2, 160, 80), (6, 3, 224, 112)])
def test_matrix_core_kernels_with_values_half_as_wide(kernel, nsplit, H, G, d, dv):
    """Every position of a prompt of 300 tokens, the key range in one part and in several (the
    denominator's one counts once); then a key that outscores all others, on either side of a page's
    edge, at the start and 299 tokens back."""
    from kvcore_amd.ops import library as ops

    if kernel == "portion" and not ops.prefill_attention_supported(H, G, d, 16, torch.bfloat16, dv):
        pytest.skip("the kernel for portions serves keys of 64 and 128")
    assert ops.decode_attention_supported(H, G, d, 16, torch.bfloat16, dv)
    assert not ops.decode_attention_supported(H, G, d, 16, torch.bfloat16, dv + 8)
    gen = torch.Generator().manual_seed(H + d)
    T, page = 300, 16
    q, k, v = (rnd(T, n, s, gen=gen, dtype=torch.bfloat16) for n, s in ((H, d), (G, d), (G, dv)))
    scale = 0.5 * d ** -0.5
    want = plain_heads(q, k, v, scale)
    rows = list(range(T)) if kernel == "portion" else [0, 1, 15, 16, 47, 63, 64, 127, 128, 255, 256, 299]
    got = attend(q[rows] if kernel == "single" else q, k, v, page, scale=scale, dtype=torch.bfloat16, positions=rows,
                 kernel=kernel, nsplit=nsplit)
    assert rel(got, want[rows]) < 1e-2
    none = attend(q[rows] if kernel == "single" else q, k, v, page, scale=scale, dtype=torch.bfloat16, positions=rows,
                  kernel=kernel, nsplit=nsplit, sink=False)
    assert rel(none, want[rows]) > 1e-2
    for marked, query in ((0, 299), (15, 299), (16, 299), (16, 15), (31, 31), (32, 31), (298, 299), (63, 64), (64, 63)):
        k2, q2 = rnd(T, G, d, gen=gen, std=0.3), rnd(T, H, d, gen=gen, std=0.3)
        k2[:, :, 0] = 0.0
        k2[marked] = 0.0
        k2[marked, :, 0] = 1.0
        q2[:, :, 0] = 40.0
        rows = [query - 2, query - 1, query] if kernel == "portion" else [query]
        got = attend(q2[rows], k2, v, page, scale=1.0, dtype=torch.bfloat16, positions=rows, kernel=kernel, nsplit=nsplit)
        assert torch.allclose(got[-1, H - 1], v[marked, G - 1], atol=2e-2) == (marked <= query), (marked, query)


@pytest.mark.parametrize("nsplit", [1, 5])
@pytest.mark.parametrize("own", [True, False], ids=["own keys", "borrowed"])
@pytest.mark.parametrize("H,G,d,dv,rot,inter", [(4, 2, 64, 32, 64, False), (3, 1, 128, 128, 32, False),
                                                (16, 1, 32, 16, 2, False), (8, 4, 96, 48, 96, True), (4, 4, 64, 64, 0, False),
                                                (2, 1, 256, 128, 200, False)])
def test_norm_rotation_write_and_attention_of_single_tokens_in_one_kernel(H, G, d, dv, rot, inter, own, nsplit):
    """The decode kernel with the norm of the heads against norm, rotation and attention one after
    the other: three requests of 1, 37 and 150 tokens and a padding token; the written key and value,
    and a layer that writes nothing and finds its keys in the cache."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(d + rot + own)
    page, eps, scale, base = 16, 1e-4, 0.6 * d ** -0.5, 5000.0
    lens, width = [1, 37, 150], H * d + (G * (d + dv) if own else 0)
    q_gain, k_gain = rnd(d, gen=gen, std=0.3) + 1, rnd(d, gen=gen, std=0.3) + 1
    q_gain, k_gain = q_gain.float().double(), k_gain.float().double()
    n_pages = sum(-(-n // page) for n in lens)
    k_cache = torch.full((n_pages + 1, G, page, d), float("nan"), dtype=torch.bfloat16, device=DEV)
    v_cache = torch.full((n_pages + 1, G, dv, page), float("nan"), dtype=torch.bfloat16, device=DEV)
    table = torch.zeros((4, 10), dtype=torch.int32, device=DEV)
    rows = rnd(4, width, gen=gen, dtype=torch.bfloat16)

    def turn(x, pos):  # x [heads, d]
        if not rot:
            return x
        full = torch.zeros(pos + 1, x.shape[0], d, dtype=F64)
        if inter:  # neighbouring pairs: the same turn on reordered elements
            order = list(range(0, rot, 2)) + list(range(1, rot, 2)) + list(range(rot, d))
            full[pos] = x[:, order]
            back = torch.empty_like(x)
            back[:, order] = plain.rotate(full, rot, base)[pos]
            return back
        full[pos] = x
        return plain.rotate(full, rot, base)[pos]

    want, next_page, keys, values = [], 1, [], []
    for r, n in enumerate(lens):
        k, v = rnd(n, G, d, gen=gen, dtype=torch.bfloat16), rnd(n, G, dv, gen=gen, dtype=torch.bfloat16)
        if own:
            raw = rows[r, H * d:]
            k[n - 1] = turn(plain.over_rms(raw[: G * d].view(G, d), eps) * k_gain, n - 1).to(torch.bfloat16).double()
            v[n - 1] = raw[G * d:].view(G, dv)
        for p in range(-(-n // page)):
            table[r + 1, p] = next_page
            m = min(page, n - p * page) - (1 if own and p == (n - 1) // page else 0)
            k_cache[next_page, :, :m] = gpu(k[p * page:p * page + m].transpose(0, 1), torch.bfloat16)
            v_cache[next_page, :, :, :m] = gpu(v[p * page:p * page + m].permute(1, 2, 0), torch.bfloat16)
            next_page += 1
        q = turn(plain.over_rms(rows[r, : H * d].view(H, d), eps) * q_gain, n - 1).to(torch.bfloat16).double()
        s = torch.stack([k[:, h // (H // G)] @ q[h] for h in range(H)]) * scale
        e = torch.exp(s)
        p_ = e / (1 + e.sum(-1, keepdim=True))
        want.append(torch.stack([p_[h] @ v[:, h // (H // G)] for h in range(H)]).reshape(-1))
        keys.append(k[n - 1])
        values.append(v[n - 1])
    ints = dict(dtype=torch.int32, device=DEV)
    pos = torch.tensor([n - 1 for n in lens] + [0], **ints)
    half = rot // 2
    cos, sin = torch.empty(4, half, device=DEV), torch.empty(4, half, device=DEV)
    if rot:
        ops.rope_table(cos, sin, pos, gpu(base ** (-2.0 * torch.arange(half, dtype=F64) / rot)))
    out = torch.full((4, H * dv), float("nan"), dtype=torch.bfloat16, device=DEV)
    parts = {} if nsplit == 1 else dict(part_o=torch.full((4 * H * nsplit, dv), float("nan"), device=DEV),
                                        part_ml=torch.full((4 * H * nsplit, 2), float("nan"), device=DEV))
    x = gpu(rows, torch.bfloat16)
    before = x.clone()
    ops.decode_attention(out, x, k_cache, v_cache, table=table, positions=pos, token_req=torch.tensor([0, 1, 2, -1], **ints),
                         slots=torch.tensor([1, 2, 3, 0], **ints), nh=H, nkv=G, d=d, dv=dv, scale=scale,
                         sinks=torch.zeros(H, device=DEV), cos=cos, sin=sin, rot_dim=rot, interleaved=inter, write_kv=own,
                         q_gain=gpu(q_gain), k_gain=gpu(k_gain) if own else None, eps=eps, nsplit=nsplit, **parts)
    assert torch.equal(x, before)
    for r, n in enumerate(lens):
        assert rel(out[r], want[r]) < 1e-2, r
        page_id = int(table[r + 1, (n - 1) // page])
        assert rel(k_cache[page_id, :, (n - 1) % page], keys[r]) < 4e-3
        assert torch.equal(v_cache[page_id, :, :, (n - 1) % page].double().cpu(), values[r])
    assert float(out[3].float().abs().max()) == 0.0


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("queries_only", [False, True], ids=["q, k, v", "queries alone"])
@pytest.mark.parametrize("H,G,d,dv,rot,T,page", [
    (4, 2, 64, 32, 64, 75, 16), (4, 2, 64, 32, 64, 3, 16), (5, 3, 128, 64, 128, 40, 16), (3, 1, 32, 48, 16, 33, 8),
    (2, 2, 256, 128, 64, 21, 16), (4, 2, 24, 40, 16, 75, 8), (3, 1, 280, 72, 30, 20, 16), (6, 2, 128, 128, 20, 50, 16),
    (4, 1, 64, 64, 0, 30, 4), (16, 4, 128, 64, 128, 300, 16), (7, 7, 96, 48, 32, 50, 16), (1, 1, 8, 1, 2, 17, 4)])
def test_norm_rotation_and_cache_write_of_portions(H, G, d, dv, rot, T, page, queries_only, dtype):
    """Two requests' tokens, one from the middle of a page on, with a padding token between them: q
    and k in place, keys and values at their places, nothing else touched; rows of queries alone."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(H * d + T)
    eps, base = 1e-4, 5000.0
    starts = [(1, 5, T - T // 3), (2, 0, T // 3)]
    batch, total = batch_tensors([starts[0], None, starts[1]])
    width = H * d + (0 if queries_only else G * (d + dv))
    rows = rnd(total, width, gen=gen, dtype=torch.bfloat16)
    q_gain, k_gain = (rnd(d, gen=gen, std=0.3) + 1).float().double(), (rnd(d, gen=gen, std=0.3) + 1).float().double()
    n_pages = -(-(T + 5) // page)
    table = torch.zeros((3, n_pages), dtype=torch.int32, device=DEV)
    table[1:] = torch.randperm(2 * n_pages, generator=gen).view(2, -1).int().to(DEV) + 1
    k_cache = torch.full((2 * n_pages + 1, G, page, d), 7.0, dtype=dtype, device=DEV)
    v_cache = torch.full((2 * n_pages + 1, G, dv, page), 7.0, dtype=dtype, device=DEV)
    kv_slot = torch.empty(total, dtype=torch.int32, device=DEV)
    ops.kv_slots(kv_slot, positions=batch["positions"], token_req=batch["token_req"], slots=batch["slots"], table=table,
                 page_size=page, num_pages=2 * n_pages + 1)
    half = rot // 2
    cos, sin = torch.empty(total, half, device=DEV), torch.empty(total, half, device=DEV)
    if rot:
        ops.rope_table(cos, sin, batch["positions"], gpu(base ** (-2.0 * torch.arange(half, dtype=F64) / rot)))
    x = gpu(rows, dtype)
    ops.qk_norm_rope_kv_write(x, k_cache, v_cache, cos, sin, rot_dim=rot, interleaved=False, kv_slot=kv_slot, nh=H,
                              nkv=G, d=d, dv=dv, q_gain=gpu(q_gain), k_gain=gpu(q_gain if queries_only else k_gain), eps=eps,
                              write_kv=not queries_only, queries_only=queries_only)
    tol = 2e-6 if dtype == torch.float32 else 4e-3
    x, kc, vc = x.double().cpu(), k_cache.double().cpu(), v_cache.double().cpu()
    pad = starts[0][2]
    assert torch.equal(x[pad], rows[pad])
    written = torch.zeros(2 * n_pages + 1, page, dtype=torch.bool)
    at = 0
    for slot, start, n in starts:
        def heads(lo, count, gain):
            full = torch.zeros(start + n, count, d, dtype=F64)
            full[start:] = plain.over_rms(rows[at: at + n, lo: lo + count * d].reshape(n, count, d), eps) * gain
            return (plain.rotate(full, rot, base) if rot else full)[start:]

        want_q = heads(0, H, q_gain).reshape(n, -1)
        assert rel(x[at: at + n, : H * d], want_q) < tol
        if not queries_only:
            want_k = heads(H * d, G, k_gain)
            assert rel(x[at: at + n, H * d: (H + G) * d], want_k.reshape(n, -1)) < tol
            values = rows[at: at + n, (H + G) * d:].view(n, G, dv)
            assert torch.equal(x[at: at + n, (H + G) * d:], rows[at: at + n, (H + G) * d:])
            for i in range(n):
                p, off = int(table[slot, (start + i) // page]), (start + i) % page
                written[p, off] = True
                assert rel(kc[p, :, off], want_k[i]) < 2 * tol, (slot, i)
                assert torch.equal(vc[p, :, :, off], values[i]), (slot, i)
        at += n + 1
    untouched = ~written
    assert (kc.transpose(1, 2)[untouched] == 7.0).all() and (vc.permute(0, 3, 1, 2)[untouched] == 7.0).all()


# ----------------------------------------------------------------------- feed-forward
@pytest.mark.parametrize("limit", [0.4, 1.0, 7.0])
@pytest.mark.parametrize("M,I,K", [(1, 80, 96), (8, 512, 1024), (16, 96, 128), (40, 256, 512), (100, 128, 1024),
                                   (300, 192, 128), (5, 20, 36)])
def test_the_clamped_gate_in_every_product(M, I, K, limit):
    """Few rows, a few dozen, many: the product that joins its branches on the way out against its
    steps (the branches rounded as if stored), and float32 against the plain rule."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(M + I)
    x = rnd(M, K, gen=gen, dtype=torch.bfloat16)
    w = {"gate": rnd(I, K, gen=gen, std=1.5 * K ** -0.5, dtype=torch.bfloat16),
         "up": rnd(I, K, gen=gen, std=1.5 * K ** -0.5, dtype=torch.bfloat16), "down": torch.eye(I, dtype=F64)}
    want = plain.dense_ff(x, w, {"limit": limit})
    off = plain.dense_ff(x, w, {"limit": limit * 1.5})
    assert limit > 5 or rel(off, want) > 1e-2
    act = ops.GateAct("clamped", limit, 1.702, 1.0)
    both = torch.cat([w["gate"], w["up"]])
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 1e-2)):
        for packed in (False, True):
            wt = gpu(both, dtype)
            if packed and not (dtype == torch.bfloat16 and ops.can_pack_weight(wt)):
                continue
            if packed:
                ops.pack_weight(wt)
            out = torch.full((M, I), float("nan"), dtype=dtype, device=DEV)
            ops.linear_silu_mul(out, gpu(x, dtype), wt, None, lambda: torch.empty(M, 2 * I, dtype=dtype, device=DEV), act=act)
            assert rel(out, want) < tol, (dtype, packed)
    gu = torch.cat([x @ w["gate"].T, x @ w["up"].T], 1).to(torch.bfloat16)
    out = torch.empty(M, I, dtype=torch.bfloat16, device=DEV)
    ops.silu_mul(out, gu.to(DEV), act)
    g, u = gu.double()[:, :I].clamp(max=limit), gu.double()[:, I:].clamp(-limit, limit)
    assert rel(out, g * torch.sigmoid(1.702 * g) * (u + 1)) < 4e-3


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("gated", [False, True], ids=["no gate row", "gate row"])
@pytest.mark.parametrize("E,top,H,T", [(12, 3, 96, 75), (32, 4, 256, 1100), (1, 1, 40, 1), (3, 3, 36, 9), (33, 5, 130, 20),
                                       (64, 8, 128, 33), (130, 3, 64, 20), (16, 4, 72, 9000), (8, 2, 1024, 3)])
def test_router_with_bias_weights_over_the_chosen_and_a_gate_row(dtype, gated, E, top, H, T):
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(E + T)
    x = rnd(T, H, gen=gen, dtype=dtype)
    w = {"router": rnd(E, H, gen=gen, std=2 * H ** -0.5, dtype=torch.float32),
         "router.b": rnd(E, gen=gen, dtype=torch.float32), "sg": rnd(1, H, gen=gen, std=H ** -0.5, dtype=torch.float32)}
    rows = torch.cat([w["router"], w["sg"]]) if gated else w["router"]

    def run(n):
        choice = torch.full((n, top), -1, dtype=torch.int32, device=DEV)
        weight = torch.full((n, top), float("nan"), device=DEV)
        gate = torch.full((n, 1), float("nan"), device=DEV) if gated else None
        ops.moe_router(choice, weight, gpu(x[:n], dtype), gpu(rows), top=top, score="logit", bias=gpu(w["router.b"]), gate=gate)
        return choice, weight, gate

    choice, weight, gate = run(T)
    want_e, want_w = plain.route(x, w, {"top": top})
    z = (x @ w["router"].T + w["router.b"]).sort(-1, descending=True).values
    close = (z[:, :top] - z[:, 1:top + 1]).min(-1).values < 1e-4 if E > top else torch.zeros(T, dtype=torch.bool)
    if E <= top and E > 1:
        close = (z[:, :-1] - z[:, 1:]).min(-1).values < 1e-4
    ok = ~close
    assert float(ok.double().mean()) > 0.9
    assert torch.equal(choice.cpu().long()[ok], want_e[ok])
    assert torch.allclose(weight.double().cpu()[ok], want_w[ok], atol=1e-5)
    assert torch.allclose(weight.sum(1), torch.ones(T, device=DEV), atol=1e-5)
    if gated:
        assert torch.allclose(gate.double().cpu(), torch.sigmoid(x @ w["sg"].T), atol=1e-5)
    # a token's result does not depend on the batch: the first rows alone give the same bits
    n = min(T, 3)
    for a, b in zip(run(n), (choice, weight, gate)):
        assert (a is None and b is None) or torch.equal(a, b[:n])
    # the same rule from given logits, and far logits whose exponentials over all experts vanish
    logits = (x @ w["router"].T).float()
    logits[0] = torch.arange(E) * -200.0
    c2, w2 = torch.empty_like(choice), torch.empty_like(weight)
    ops.moe_route(c2, w2, gpu(logits), top=top, score="logit")
    assert c2[0].tolist() == list(range(top)) and float(w2[0, 0]) == pytest.approx(1.0)
    best = logits.double().topk(top, dim=-1)
    assert torch.allclose(w2.double().cpu(), torch.softmax(best.values, -1), atol=1e-6)


@pytest.mark.parametrize("H", [96, 40, 36, 2048, 100])
@pytest.mark.parametrize("top,with_add,with_gate", [(1, False, False), (3, True, True), (4, True, False), (7, True, True)])
def test_experts_added_up_by_the_norm_behind_them(H, top, with_add, with_gate):
    """The norm behind the experts on their weighted rows against the sum made first, in both forms
    of the kernel (rows of a multiple of 8 values, any rows)."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(H + top)
    T, eps = 11, 1e-5
    y, weight = rnd(T * top, H, gen=gen, dtype=torch.float32), rnd(T, top, gen=gen, dtype=torch.float32)
    add = rnd(T, H, gen=gen, dtype=torch.float32) if with_add else None
    gate = rnd(T, 1, gen=gen, dtype=torch.float32) if with_gate else None
    post, nxt, res = (rnd(n, gen=gen, dtype=torch.float32) for n in (H, H, T * H))
    res = res.view(T, H)
    summed = (weight[:, :, None] * y.view(T, top, H)).sum(1)
    if with_add:
        summed = summed + add * (gate if with_gate else 1.0)
    want_res = res + plain.over_rms(summed, eps) * post
    want_out = plain.over_rms(want_res, 2 * eps) * nxt
    rows = ops.WeightedRows(gpu(y), gpu(weight), None if add is None else gpu(add), None if gate is None else gpu(gate))
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 4e-3)):
        residual, out = gpu(res), torch.empty(T, H, dtype=dtype, device=DEV)
        ops.norm_add_norm(out, residual, rows, gpu(post), eps, gpu(nxt), 2 * eps)
        assert rel(residual, want_res) < 2e-6 and rel(out, want_out) < tol
    residual = gpu(res)
    ops.norm_add_norm(None, residual, rows, gpu(post), eps)
    assert rel(residual, want_res) < 2e-6
    total = torch.empty(T, H, device=DEV)
    ops.moe_combine(total, rows.data, rows.weight, None, rows.add, add1_gate=rows.add_gate)
    assert rel(total, summed) < 2e-6


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("E,top,H,I,shared,T", [(12, 3, 96, 40, 56, 75), (8, 2, 128, 64, 96, 300), (1, 1, 40, 8, 8, 1),
                                                (5, 5, 36, 20, 12, 19), (3, 1, 96, 64, 0, 800), (16, 4, 64, 32, 32, 33),
                                                (4, 2, 512, 64, 512, 40), (2, 2, 64, 32, 0, 300)])
def test_the_routed_feed_forward_with_a_gated_shared_expert(dtype, E, top, H, I, shared, T):
    """The part on rows of its own: both of its results (rows added up, weighted rows) against the
    plain function."""
    from kvcore_amd.engine.context import StepBuffers, StepContext
    from kvcore_amd.ops import library as ops
    from kvcore_amd.parts.base import FEED_FORWARDS, PartSpec, Runtime

    gen = torch.Generator().manual_seed(E + H + T)
    names = {"router": "router", "router_bias": "router.b", "expert": "e{e}", "shared": "shared",
             "shared_gate": "shared.sg", "gate": "gate", "up": "up", "down": "down"}
    part = FEED_FORWARDS.build(PartSpec("routed_experts", dict(
        hidden_size=H, experts=E, top=top, expert_size=I, limit=None, alpha=1.0, up_shift=0.0, score="logit",
        router_bias=True, shared_size=shared, shared_gate=shared > 0, tensor_names=names)))
    part.setup(Runtime(dtype, torch.device(DEV)))
    w, params = {}, {}
    for ps in part.param_specs():
        rows = []
        for src in ps.resolved_sources():
            std = 1.0 if src.name == "router.b" else 1.5 * ps.shape[-1] ** -0.5
            w[src.name] = rnd(src.rows, *ps.shape[1:], gen=gen, std=std, dtype=torch.bfloat16)
            rows.append(w[src.name])
        params[ps.name] = gpu(torch.cat(rows), torch.float32 if ps.kind == "vector" else dtype)
    part.bind(params)
    x = rnd(T, H, gen=gen, dtype=torch.bfloat16)
    mlp = {"router": {"experts": E, "top": top}, "shared": {"ff": shared} if shared else None}
    want = plain.routed_ff(x, w, mlp)
    ctx = StepContext(num_tokens=T, num_reqs=1, token_ids=None, positions=None, token_req=None, q_start=None, seq_lens=None,
                      slots=None, groups=[], states=[], buffers=StepBuffers(torch.device(DEV), token_capacity=T),
                      dtype=dtype, device=torch.device(DEV))
    z = (x @ w["router"].T + w["router.b"]).sort(-1, descending=True).values
    far = torch.ones(T, dtype=torch.bool) if top == E else (z[:, top - 1] - z[:, top]) > 1e-4
    tol = 3e-6 if dtype == torch.float32 else 1e-2
    got = part.forward(gpu(x, dtype), ctx, None)
    assert rel(got[far.to(DEV)], want[far]) < tol
    rows = part.forward_weighted(gpu(x, dtype), ctx, None)
    residual = torch.zeros(T, H, device=DEV)
    ops.norm_add_norm(None, residual, rows, torch.ones(H, device=DEV), 1e-6)
    assert rel(residual[far.to(DEV)], plain.over_rms(want, 1e-6)[far]) < tol
    if shared:
        part.params["router.weight"][E].zero_()  # without its row the gate is a half for every token
        got = part.forward(gpu(x, dtype), ctx, None)
        assert rel(got[far.to(DEV)], want[far]) > 1e-2
