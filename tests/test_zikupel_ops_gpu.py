"""Every mechanism of the Zikupel decoder alone: the kernel against the plain function of
``tests/plain/zikupel.py``, at sizes of the tests' own, whole and in steps, beside other requests
and padding, with inputs made so that a far key, a lost state or a missing cap shows."""

from __future__ import annotations

import pytest
import torch

from tests.darovik_helpers import batch_tensors
from tests.plain import zikupel as plain

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


# ------------------------------------------------------------- scores, caps, output gates
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


def attend(q, k, v, page, *, scale, dtype, cap=0.0, gate=None, positions=None, kernel="general", nsplit=1, sinks=None):
    """``gate [T, H * dv]`` stands inside wider rows, as the input product leaves it."""
    from kvcore_amd.ops import library as ops

    T, H, d = q.shape
    G, dv = v.shape[1:]
    k_cache, v_cache, table = pages_of(k, v, page, dtype)
    pos = list(range(T)) if positions is None else positions
    ints = dict(dtype=torch.int32, device=DEV)
    out = torch.full((T, H * dv), float("nan"), dtype=dtype, device=DEV)
    g = None if gate is None else gpu(torch.cat([gate * 0 + 9.0, gate], 1), dtype)[:, H * dv:]
    common = dict(table=table, slots=torch.tensor([1], **ints), nh=H, nkv=G, d=d, dv=dv, scale=scale, softcap=cap,
                  sinks=sinks)
    rows = gpu(q.reshape(T, -1), dtype)
    parts = {}
    if nsplit > 1:
        parts = dict(nsplit=nsplit, part_o=torch.full((T * H * nsplit, dv), float("nan"), device=DEV),
                     part_ml=torch.full((T * H * nsplit, 2), float("nan"), device=DEV))
    if kernel == "portion":
        ops.prefill_attention(out, rows, k_cache, v_cache, positions=torch.tensor(pos, **ints),
                              q_start=torch.tensor([0, T], **ints), num_reqs=1, gate=g, **common, **parts)
    elif kernel == "single":
        for i in range(T):
            ops.decode_attention(out[i:i + 1], rows[i:i + 1], k_cache, v_cache, positions=torch.tensor(pos[i:i + 1], **ints),
                                 token_req=torch.zeros(1, **ints), gate=None if g is None else g[i:i + 1], **common, **parts)
    else:
        ops.paged_attention(out, rows, k_cache, v_cache, positions=torch.tensor(pos, **ints),
                            token_req=torch.zeros(T, **ints), gate=g, **common)
    return out.double().cpu().view(T, H, dv)


def plain_heads(q, k, v, scale, cap):
    T, H, _ = q.shape
    g = H // k.shape[1]

    def scores(h):
        s = (q[:, h] @ k[:, h // g].T) * scale
        return plain.capped(s, cap) if cap else s

    return torch.stack([plain.causal_softmax(scores(h)) @ v[:, h // g] for h in range(H)], 1)


@pytest.mark.parametrize("cap", [2.0, 30.0, 70.0])
@pytest.mark.parametrize("H,G,d,dv,page", [(4, 2, 24, 40, 8), (1, 1, 8, 1, 4), (6, 2, 16, 16, 16), (3, 1, 280, 72, 16)])
def test_capped_scores_and_output_gate_in_the_general_kernel(H, G, d, dv, page, cap):
    gen = torch.Generator().manual_seed(d)
    T = 90
    q, k, v = (rnd(T, n, s, gen=gen, dtype=torch.bfloat16) for n, s in ((H, d), (G, d), (G, dv)))
    gate = rnd(T, H * dv, gen=gen, dtype=torch.bfloat16)
    kw = dict(scale=cap * d ** -0.5)  # scaled scores as large as the cap
    want = plain_heads(q, k, v, kw["scale"], cap)
    gated = want * torch.sigmoid(gate).view(T, H, dv)
    assert rel(attend(q, k, v, page, dtype=torch.float32, cap=cap, **kw), want) < 5e-6
    assert rel(attend(q, k, v, page, dtype=torch.float32, cap=cap, gate=gate, **kw), gated) < 5e-6
    assert rel(attend(q, k, v, page, dtype=torch.float32, **kw), want) > 1e-2
    assert rel(attend(q, k, v, page, dtype=torch.bfloat16, cap=cap, gate=gate, **kw), gated) < 1e-2


@pytest.mark.parametrize("cap", [2.0, 20.0, 44.0, 70.0])
@pytest.mark.parametrize("kernel,nsplit", [("portion", 1), ("portion", 3), ("single", 1), ("single", 4)])
@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 64, 64), (16, 4, 128, 128), (8, 1, 64, 32), (3, 3, 128, 64), (16, 1, 32, 32),
                                      (4, 2, 96, 96), (2, 1, 256, 256)])
def test_capped_scores_and_output_gate_in_the_matrix_core_kernels(kernel, nsplit, H, G, d, dv, cap):
    """Every position of a prompt of 300 tokens, the key range in one part and in several; caps that are
    taken relative to a score of zero and one that needs the running maximum."""
    from kvcore_amd.ops import library as ops

    if kernel == "portion" and not ops.prefill_attention_supported(H, G, d, 16, torch.bfloat16, dv):
        pytest.skip("the kernel for portions serves keys of 64 and 128")
    gen = torch.Generator().manual_seed(H + d)
    T, page = 300, 16
    q, k, v = (rnd(T, n, s, gen=gen, dtype=torch.bfloat16) for n, s in ((H, d), (G, d), (G, dv)))
    gate = rnd(T, H * dv, gen=gen, dtype=torch.bfloat16)
    scale = 0.7 * cap * d ** -0.5
    want = plain_heads(q, k, v, scale, cap)
    gated = want * torch.sigmoid(gate).view(T, H, dv)
    rows = list(range(T)) if kernel == "portion" else [0, 1, 15, 16, 47, 63, 64, 127, 128, 255, 256, 299]
    kw = dict(scale=scale, dtype=torch.bfloat16, positions=rows, kernel=kernel, nsplit=nsplit)
    got = attend(q[rows], k, v, page, cap=cap, gate=gate[rows], **kw)
    assert rel(got, gated[rows]) < 1e-2
    assert rel(attend(q[rows], k, v, page, cap=cap, **kw), want[rows]) < 1e-2
    assert rel(attend(q[rows], k, v, page, gate=gate[rows], **kw), gated[rows]) > 3e-2
    sinks = torch.full((H,), 1.5, device=DEV)  # one more score, which is not capped
    got = attend(q[rows], k, v, page, cap=cap, sinks=sinks, **kw)
    last = plain.capped((q[299, 0] @ k[:, 0].T) * scale, cap)
    e = torch.exp(last - last.max())
    assert rel(got[-1, 0], (e @ v[:, 0]) / (e.sum() + torch.exp(1.5 - last.max()))) < 1e-2


@pytest.mark.parametrize("kernel,nsplit", [("portion", 1), ("portion", 4), ("single", 1), ("single", 4), ("general", 1)])
@pytest.mark.parametrize("H,G,d", [(4, 2, 64), (6, 3, 128)])
def test_a_key_that_stands_out_under_the_cap(kernel, nsplit, H, G, d):
    """A key whose score reaches the cap, on either side of a page's edge, at the start and 299 tokens back,
    while all others lie far below it: all attention is on it iff it lies at or before the query.  And scores
    far beyond the cap on both sides: the weights stay finite, those at the cap share alike."""
    gen = torch.Generator().manual_seed(H + d)
    T, page = 300, 16
    v = rnd(T, G, d, gen=gen, dtype=torch.bfloat16)
    for marked, query in ((0, 299), (15, 299), (16, 299), (16, 15), (31, 31), (32, 31), (298, 299), (63, 64), (64, 63)):
        k2, q2 = rnd(T, G, d, gen=gen, std=0.3), rnd(T, H, d, gen=gen, std=0.3)
        k2[:, :, 0] = 0.0
        k2[marked] = 0.0
        k2[marked, :, 0] = 1.0
        q2[:, :, 0] = 40.0
        rows = [query - 2, query - 1, query] if kernel == "portion" else [query]
        got = attend(q2[rows], k2, v, page, scale=1.0, cap=25.0, dtype=torch.bfloat16, positions=rows, kernel=kernel,
                     nsplit=nsplit)
        assert torch.allclose(got[-1, H - 1], v[marked, G - 1], atol=2e-2) == (marked <= query), (marked, query)
    for cap in (20.0, 44.0, 80.0):
        k2, q2 = torch.zeros(T, G, d, dtype=F64), torch.zeros(T, H, d, dtype=F64)
        q2[:, :, 0] = 100.0
        k2[:, :, 0] = -100.0
        rows = [297, 298, 299]
        got = attend(q2[rows], k2, v, page, scale=1.0, cap=cap, dtype=torch.bfloat16, positions=rows, kernel=kernel, nsplit=nsplit)
        assert torch.allclose(got[-1, 0], v[:, 0].mean(0), atol=1e-2)  # every score at minus the cap
        k2[[3, 170], :, 0] = 100.0
        got = attend(q2[rows], k2, v, page, scale=1.0, cap=cap, dtype=torch.bfloat16, positions=rows, kernel=kernel, nsplit=nsplit)
        assert torch.allclose(got[-1, 0], (v[3, 0] + v[170, 0]) / 2, atol=2e-2)


# ----------------------------------------------------- values that are the keys as projected
@pytest.mark.parametrize("nsplit", [1, 5])
@pytest.mark.parametrize("H,G,d,rot", [(4, 2, 64, 32), (3, 1, 128, 128), (16, 1, 32, 2), (8, 4, 96, 96), (2, 1, 256, 200)])
def test_single_tokens_whose_values_are_their_keys(H, G, d, rot, nsplit):
    """The decode kernel on rows [q | k | gate]: norm, YaRN rotation, the written key (normed and turned) and
    value (the key as projected), capped scores, gate; three requests and a padding token."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(d + rot)
    page, eps, scale, cap = 16, 1e-4, 2.0 * d ** -0.5, 6.0
    rot_cfg = {"dims": rot, "base": 5000.0, "scaling": {"factor": 4.0, "original": 60, "fast": 8.0, "slow": 1.0}}
    lens, width = [1, 37, 150], (H + G + H) * d
    q_gain, k_gain = ((rnd(d, gen=gen, std=0.3) + 1).float().double() for _ in range(2))
    n_pages = sum(-(-n // page) for n in lens)
    k_cache = torch.full((n_pages + 1, G, page, d), float("nan"), dtype=torch.bfloat16, device=DEV)
    v_cache = torch.full((n_pages + 1, G, d, page), float("nan"), dtype=torch.bfloat16, device=DEV)
    table = torch.zeros((4, 10), dtype=torch.int32, device=DEV)
    rows = rnd(4, width, gen=gen, dtype=torch.bfloat16)

    def turn(x, pos):
        full = torch.zeros(pos + 1, x.shape[0], d, dtype=F64)
        full[pos] = x
        return plain.rotate(full, rot_cfg)[pos]

    want, next_page, keys = [], 1, []
    for r, n in enumerate(lens):
        raw = rnd(n, G, d, gen=gen, dtype=torch.bfloat16)
        raw[n - 1] = rows[r, H * d: (H + G) * d].view(G, d)
        k = rnd(n, G, d, gen=gen, dtype=torch.bfloat16)  # any keys of the tokens before, already normed and turned
        k[n - 1] = turn(plain.over_rms(raw[n - 1], eps) * k_gain, n - 1).to(torch.bfloat16).double()
        for p in range(-(-n // page)):
            table[r + 1, p] = next_page
            m = min(page, n - p * page) - (1 if p == (n - 1) // page else 0)
            k_cache[next_page, :, :m] = gpu(k[p * page:p * page + m].transpose(0, 1), torch.bfloat16)
            v_cache[next_page, :, :, :m] = gpu(raw[p * page:p * page + m].permute(1, 2, 0), torch.bfloat16)
            next_page += 1
        q = turn(plain.over_rms(rows[r, : H * d].view(H, d), eps) * q_gain, n - 1).to(torch.bfloat16).double()
        s = plain.capped(torch.stack([k[:, h // (H // G)] @ q[h] for h in range(H)]) * scale, cap)
        p_ = torch.softmax(s, -1)
        heads = torch.stack([p_[h] @ raw[:, h // (H // G)] for h in range(H)]).reshape(-1)
        want.append(heads * torch.sigmoid(rows[r, (H + G) * d:]))
        keys.append((k[n - 1], raw[n - 1]))
    ints = dict(dtype=torch.int32, device=DEV)
    pos = torch.tensor([n - 1 for n in lens] + [0], **ints)
    half = rot // 2
    cos, sin = torch.empty(4, half, device=DEV), torch.empty(4, half, device=DEV)
    freqs, factor = plain.frequencies(rot_cfg)
    ops.rope_table(cos, sin, pos, gpu(torch.tensor(freqs, dtype=F64)), factor)
    out = torch.full((4, H * d), float("nan"), dtype=torch.bfloat16, device=DEV)
    parts = {} if nsplit == 1 else dict(part_o=torch.full((4 * H * nsplit, d), float("nan"), device=DEV),
                                        part_ml=torch.full((4 * H * nsplit, 2), float("nan"), device=DEV))
    x = gpu(rows, torch.bfloat16)
    before = x.clone()
    ops.decode_attention(out, x, k_cache, v_cache, table=table, positions=pos, token_req=torch.tensor([0, 1, 2, -1], **ints),
                         slots=torch.tensor([1, 2, 3, 0], **ints), nh=H, nkv=G, d=d, scale=scale, softcap=cap, cos=cos,
                         sin=sin, rot_dim=rot, write_kv=True, values_are_keys=True, gate=x[:, (H + G) * d:],
                         q_gain=gpu(q_gain), k_gain=gpu(k_gain), eps=eps, nsplit=nsplit, **parts)
    assert torch.equal(x, before)
    for r, n in enumerate(lens):
        assert rel(out[r], want[r]) < 1e-2, r
        page_id = int(table[r + 1, (n - 1) // page])
        assert rel(k_cache[page_id, :, (n - 1) % page], keys[r][0]) < 4e-3
        assert torch.equal(v_cache[page_id, :, :, (n - 1) % page].double().cpu(), keys[r][1])
    assert float(out[3].float().abs().max()) == 0.0


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("H,G,d,rot,T,page", [
    (4, 2, 64, 32, 75, 16), (4, 2, 64, 64, 3, 16), (5, 3, 128, 128, 40, 16), (3, 1, 32, 16, 33, 8), (2, 2, 256, 64, 21, 16),
    (4, 2, 24, 16, 75, 8), (3, 1, 280, 30, 20, 16), (4, 1, 64, 0, 30, 4), (7, 7, 96, 32, 50, 16), (1, 1, 8, 2, 17, 4)])
def test_portions_whose_values_are_their_keys(H, G, d, rot, T, page, dtype):
    """Two requests' tokens, one from the middle of a page on, with a padding token between them: queries
    normed and turned in place, the keys' and the gate's columns left as they are, normed and turned keys and
    raw keys as values at their places, nothing else touched."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(H * d + T)
    eps = 1e-4
    rot_cfg = {"dims": rot, "base": 5000.0, "scaling": {"factor": 3.0, "original": 40, "fast": 4.0, "slow": 0.5}} if rot else None
    starts = [(1, 5, T - T // 3), (2, 0, T // 3)]
    batch, total = batch_tensors([starts[0], None, starts[1]])
    width = (H + G + H) * d
    rows = rnd(total, width, gen=gen, dtype=torch.bfloat16)
    q_gain, k_gain = ((rnd(d, gen=gen, std=0.3) + 1).float().double() for _ in range(2))
    n_pages = -(-(T + 5) // page)
    table = torch.zeros((3, n_pages), dtype=torch.int32, device=DEV)
    table[1:] = torch.randperm(2 * n_pages, generator=gen).view(2, -1).int().to(DEV) + 1
    k_cache = torch.full((2 * n_pages + 1, G, page, d), 7.0, dtype=dtype, device=DEV)
    v_cache = torch.full((2 * n_pages + 1, G, d, page), 7.0, dtype=dtype, device=DEV)
    kv_slot = torch.empty(total, dtype=torch.int32, device=DEV)
    ops.kv_slots(kv_slot, positions=batch["positions"], token_req=batch["token_req"], slots=batch["slots"], table=table,
                 page_size=page, num_pages=2 * n_pages + 1)
    half = rot // 2
    cos, sin = torch.empty(total, half, device=DEV), torch.empty(total, half, device=DEV)
    if rot:
        freqs, factor = plain.frequencies(rot_cfg)
        ops.rope_table(cos, sin, batch["positions"], gpu(torch.tensor(freqs, dtype=F64)), factor)
    x = gpu(rows, dtype)
    ops.qk_norm_rope_kv_write(x, k_cache, v_cache, cos, sin, rot_dim=rot, interleaved=False, kv_slot=kv_slot, nh=H,
                              nkv=G, d=d, dv=d, q_gain=gpu(q_gain), k_gain=gpu(k_gain), eps=eps, values_are_keys=True)
    tol = 2e-6 if dtype == torch.float32 else 4e-3
    x, kc, vc = x.double().cpu(), k_cache.double().cpu(), v_cache.double().cpu()
    pad = starts[0][2]
    assert torch.equal(x[pad], rows[pad]) and torch.equal(x[:, H * d:], rows[:, H * d:])
    written = torch.zeros(2 * n_pages + 1, page, dtype=torch.bool)
    at = 0
    for slot, start, n in starts:
        def heads(lo, count, gain):
            full = torch.zeros(start + n, count, d, dtype=F64)
            full[start:] = plain.over_rms(rows[at: at + n, lo: lo + count * d].reshape(n, count, d), eps) * gain
            return plain.rotate(full, rot_cfg)[start:]

        assert rel(x[at: at + n, : H * d], heads(0, H, q_gain).reshape(n, -1)) < tol
        want_k, raw = heads(H * d, G, k_gain), rows[at: at + n, H * d: (H + G) * d].view(n, G, d)
        for i in range(n):
            p, off = int(table[slot, (start + i) // page]), (start + i) % page
            written[p, off] = True
            assert rel(kc[p, :, off], want_k[i]) < 2 * tol, (slot, i)
            assert torch.equal(vc[p, :, :, off], raw[i]), (slot, i)
        at += n + 1
    untouched = ~written
    assert (kc.transpose(1, 2)[untouched] == 7.0).all() and (vc.permute(0, 3, 1, 2)[untouched] == 7.0).all()


# ------------------------------------------------------------ the matrix with a fixed decay
SCANS = ["token by token", "in chunks"]


def run_fixed_decay(how, rows, decay, state, reqs, *, heads, dim, vdim, silu_in=True, qk_heads=None, q_scale=1.0):
    from kvcore_amd.ops import library as ops

    batch, T = batch_tensors(reqs)
    out = torch.full((T, heads * vdim), float("nan"), device=DEV)
    nqk = heads if qk_heads is None else qk_heads
    proj = gpu(rows)
    qk = nqk * dim
    parts = (proj[:, :qk], proj[:, qk:2 * qk], proj[:, 2 * qk:2 * qk + heads * vdim])
    kw = dict(heads=heads, qk_heads=nqk, dim=dim, vdim=vdim, silu_in=silu_in, q_scale=q_scale, **batch)
    lam = torch.tensor([decay], dtype=torch.float32, device=DEV)
    if how == "in chunks":
        each = heads * ops.linear_state_rows(dim) * vdim
        work = torch.full((ops.fixed_decay_chunk_count(T, len(reqs)), each), float("nan"), device=DEV)
        ops.fixed_decay_chunks(out, *parts, lam, state, work, **kw)
    else:
        ops.linear_state_scan(out, *parts, lam, None, state, scalar_gates=True, **kw)
    return out


def new_state(slots, heads, dim, vdim, fill=float("nan")):
    from kvcore_amd.ops import library as ops

    return torch.full((slots, heads, ops.linear_state_rows(dim), vdim), fill, device=DEV)


def plain_state(rows, decay, heads, dim, vdim, silu_in=True, qk_heads=None, q_scale=1.0):
    T, nqk = rows.shape[0], heads if qk_heads is None else qk_heads
    act = plain.silu if silu_in else (lambda z: z)
    qk = nqk * dim
    q, k = act(rows[:, :qk]).view(T, nqk, dim) * q_scale, act(rows[:, qk:2 * qk]).view(T, nqk, dim)
    spread = [h // (heads // nqk) for h in range(heads)]
    v = act(rows[:, 2 * qk:2 * qk + heads * vdim]).view(T, heads, vdim)
    lam = torch.tensor(decay, dtype=torch.float32).double()
    return plain.lightning_state(q[:, spread], k[:, spread], v, lam).reshape(T, -1)


@pytest.mark.parametrize("how", SCANS)
@pytest.mark.parametrize("dim,vdim,decay", [(24, 40, (0.97, 0.5, 0.999)), (8, 5, (0.9,)), (200, 72, (0.95, 0.3)),
                                            (64, 64, (0.999, 0.0, 1.0, 0.8)), (32, 130, (0.7, 0.99)), (1, 1, (0.9,)),
                                            (128, 128, (0.99, 0.4)), (256, 20, (0.9,)), (30, 64, (0.98, 0.2, 0.9))])
def test_a_fixed_decay_whole_in_steps_and_beside_others(dim, vdim, decay, how):
    """A request of 203 tokens from a slot that holds another's leftovers (NaN): whole; in steps of every size
    down to one token, cut inside stages and chunks, alternating with the other way to compute; beside a
    padded row and another request that is further on."""
    heads = len(decay)
    gen = torch.Generator().manual_seed(dim + vdim)
    T, width = 203, heads * (2 * dim + vdim) + (4 if dim % 4 == 0 else 3)  # rows wider than what is read
    rows = rnd(T, width, gen=gen, dtype=torch.float32)
    want = plain_state(rows, decay, heads, dim, vdim)
    kw = dict(heads=heads, dim=dim, vdim=vdim)
    state = new_state(3, heads, dim, vdim)
    assert rel(run_fixed_decay(how, rows, decay, state, [(1, 0, T)], **kw), want) < 3e-6
    state = new_state(3, heads, dim, vdim)
    at, got = 0, []
    for i, n in enumerate((2, 1, 17, 64, 1, 16, 65, 2, 35)):
        ways = (how, SCANS[1 - SCANS.index(how)])
        got.append(run_fixed_decay(ways[i % 2], rows[at:at + n], decay, state, [(2, at, n)], **kw))
        at += n
    assert at == T and rel(torch.cat(got), want) < 3e-6
    other = new_state(3, heads, dim, vdim, 0.0)
    run_fixed_decay(how, rows[:140], decay, other, [(0, 0, 140)], **kw)
    other[1].fill_(float("nan"))
    mixed = torch.cat([rows[140:203], rows[:1], rows[:90], rows[:1]])
    out = run_fixed_decay(how, mixed, decay, other, [(0, 140, 63), None, (1, 0, 90), (2, 0, 1)], **kw)
    assert rel(out[:63], want[140:]) < 3e-6 and rel(out[64:154], want[:90]) < 3e-6 and rel(out[154:], want[:1]) < 3e-6
    assert float(out[63].abs().max()) == 0.0


@pytest.mark.parametrize("how", SCANS)
def test_shared_queries_a_scale_and_no_activation(how):
    gen = torch.Generator().manual_seed(8)
    heads, nqk, dim, vdim, T = 6, 2, 20, 36, 130
    rows = rnd(T, 2 * nqk * dim + heads * vdim, gen=gen, dtype=torch.float32)
    decay = (0.9, 0.99, 0.5, 0.999, 0.8, 0.7)
    kw = dict(heads=heads, dim=dim, vdim=vdim, qk_heads=nqk, q_scale=0.3, silu_in=False)
    got = run_fixed_decay(how, rows, decay, new_state(1, heads, dim, vdim), [(0, 0, T)], **kw)
    assert rel(got, plain_state(rows, decay, **kw)) < 3e-6


@pytest.mark.parametrize("how", SCANS)
def test_a_token_written_a_thousand_tokens_ago_is_still_read(how):
    """One token alone has a key and a value; every later query reads it, weaker by the decay to the power
    of the distance, whether or not a step or a chunk ends in between."""
    dim, vdim, T = 16, 24, 1200
    decay = (0.999, 0.97)
    rows = torch.zeros(T, 2 * (2 * dim + vdim), dtype=F64)
    rows[:, : 2 * dim] = 3.0
    marked = 63
    rows[marked, 2 * dim:] = 2.0
    one = float(plain.silu(torch.tensor(3.0, dtype=F64)) * plain.silu(torch.tensor(2.0, dtype=F64)) ** 2) * dim
    state, at = new_state(1, 2, dim, vdim), 0
    for n in (63, 1, 700, 2, 434):
        out = run_fixed_decay(how, rows[at:at + n], decay, state, [(0, at, n)], heads=2, dim=dim, vdim=vdim).double().cpu()
        for i in {0, n // 2, n - 1}:
            for h in range(2):
                back = at + i - marked
                want = one * float(torch.tensor(decay[h])) ** back if back >= 0 else 0.0
                assert torch.allclose(out[i, h * vdim:(h + 1) * vdim], torch.full((vdim,), want, dtype=F64),
                                      rtol=2e-4, atol=1e-12), (at + i, h)
        at += n


@pytest.mark.parametrize("act", ["sigmoid", "silu"])
@pytest.mark.parametrize("T,heads,vdim,norm_heads", [(5, 4, 64, 1), (33, 3, 40, 1), (2, 16, 128, 1), (7, 5, 13, 1), (9, 2, 300, 2),
                                                     (4, 2, 5, 1), (300, 4, 32, 4)])
def test_the_norm_over_all_heads_and_its_gate(T, heads, vdim, norm_heads, act):
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(T + vdim)
    inner = heads * vdim
    o, wide = rnd(T, inner, gen=gen, dtype=torch.float32), rnd(T, inner + 4, gen=gen, dtype=torch.bfloat16)
    gain = rnd(inner // norm_heads, gen=gen, dtype=torch.float32)
    z = wide[:, 4:]
    g = torch.sigmoid(z) if act == "sigmoid" else plain.silu(z)
    want = (plain.over_rms(o.view(T, norm_heads, -1), 1e-5) * gain).reshape(T, -1) * g
    for gate_dtype in DTYPES:
        for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 4e-3)):
            out = torch.empty(T, inner, dtype=dtype, device=DEV)
            ops.head_rmsnorm_gate(out, gpu(o), gpu(wide, gate_dtype)[:, 4:], gpu(gain), 1e-5, norm_heads, inner // norm_heads,
                                  act=act)
            assert rel(out, want) < tol, (gate_dtype, dtype)


# -------------------------------------------------------------------------- routed experts
@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("E,top,H,T", [(12, 1, 96, 75), (32, 4, 256, 1100), (1, 1, 40, 1), (3, 3, 36, 9), (33, 5, 130, 20),
                                       (8, 2, 1024, 3)])
def test_router_weights_that_are_the_sigmoids_themselves(dtype, E, top, H, T):
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(E + T)
    x = rnd(T, H, gen=gen, dtype=dtype)
    w = {"router": rnd(E, H, gen=gen, std=2 * H ** -0.5, dtype=torch.float32)}
    choice = torch.full((T, top), -1, dtype=torch.int32, device=DEV)
    weight = torch.full((T, top), float("nan"), device=DEV)
    ops.moe_router(choice, weight, gpu(x, dtype), gpu(w["router"]), top=top, score="sigmoid", renormalize=False)
    want_e, want_w = plain.route(x, w, top)
    z = torch.sigmoid(x @ w["router"].T).sort(-1, descending=True).values
    ok = torch.ones(T, dtype=torch.bool) if E == 1 else (z[:, :-1] - z[:, 1:])[:, :top].min(-1).values > 1e-5
    assert float(ok.double().mean()) > 0.9
    assert torch.equal(choice.cpu().long()[ok], want_e[ok])
    assert torch.allclose(weight.double().cpu()[ok], want_w[ok], atol=1e-6)
    again = torch.empty_like(weight)
    ops.moe_route(choice, again, gpu((x @ w["router"].T).float()), top=top, score="sigmoid", renormalize=False, weight_scale=2.0)
    assert torch.allclose(again.double().cpu()[ok], 2 * want_w[ok], atol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("packed", [False, True], ids=["rows", "packed"])
@pytest.mark.parametrize("E,top,H,I,shared,T", [(12, 3, 96, 40, 56, 75), (8, 2, 128, 64, 96, 300), (1, 1, 40, 8, 8, 1),
                                                (5, 5, 36, 20, 12, 19), (3, 1, 96, 64, 0, 800), (16, 1, 64, 32, 32, 33),
                                                (4, 2, 512, 64, 512, 40), (2, 2, 64, 128, 0, 300), (6, 1, 256, 64, 64, 8)])
def test_experts_without_a_gate_weighted_on_their_input(dtype, packed, E, top, H, I, shared, T):
    """The part on rows of its own: both of its results (rows added up; rows for the norm behind, which also
    hands on the stream itself) against the plain function, which really multiplies the inputs; the same
    weights on the outputs give something else."""
    from kvcore_amd.engine.context import StepBuffers, StepContext
    from kvcore_amd.ops import library as ops
    from kvcore_amd.parts.base import FEED_FORWARDS, PartSpec, Runtime

    gen = torch.Generator().manual_seed(E + H + T)
    names = {"router": "router", "expert": "e{e}", "shared": "shared", "up": "up", "down": "down"}

    def build(**kw):
        return FEED_FORWARDS.build(PartSpec("routed_experts", dict(
            hidden_size=H, experts=E, top=top, expert_size=I, limit=None, score="sigmoid", renormalize=False,
            activation="relu_squared", shared_size=shared, tensor_names=names, **kw)))

    part = build(weight_on_input=True)
    part.setup(Runtime(dtype, torch.device(DEV)))
    w, params = {}, {}
    for ps in part.param_specs():
        rows = []
        for src in ps.resolved_sources():
            w[src.name] = rnd(src.rows, *ps.shape[1:], gen=gen, std=1.5 * ps.shape[-1] ** -0.5, dtype=torch.bfloat16)
            rows.append(w[src.name])
        params[ps.name] = gpu(torch.cat(rows), torch.float32 if ps.kind == "vector" else dtype)
    if packed:
        able = [n for n in part.product_weights() if ops.can_pack_weight(params[n])]
        if not able:
            pytest.skip("nothing here has a packed form")
        for n in able:
            ops.pack_weight(params[n])
    part.bind(params)
    x = rnd(T, H, gen=gen, dtype=torch.bfloat16)
    mlp = {"router": {"experts": E, "top": top}, "shared": {"ff": shared} if shared else None}
    want = plain.routed_ff(x, w, mlp)
    ctx = StepContext(num_tokens=T, num_reqs=1, token_ids=None, positions=None, token_req=None, q_start=None, seq_lens=None,
                      slots=None, groups=[], states=[], buffers=StepBuffers(torch.device(DEV), token_capacity=T),
                      dtype=dtype, device=torch.device(DEV))
    z = (x @ w["router"].T).sort(-1, descending=True).values
    far = torch.ones(T, dtype=torch.bool) if top == E else (z[:, top - 1] - z[:, top]) > 1e-4
    tol = 3e-6 if dtype == torch.float32 else 1.2e-2
    assert rel(part.forward(gpu(x, dtype), ctx, None)[far.to(DEV)], want[far]) < tol
    rows = part.forward_weighted(gpu(x, dtype), ctx, None)
    assert rows.weight is None and rows.count == top
    res, gain = rnd(T, H, gen=gen, dtype=torch.float32), rnd(H, gen=gen, dtype=torch.float32)
    residual, out = gpu(res), torch.empty(T, H, dtype=dtype, device=DEV)
    ops.norm_add_norm(out, residual, rows, gpu(gain), 1e-6)
    stream = res + plain.over_rms(want, 1e-6) * gain
    assert rel(residual[far.to(DEV)], stream[far]) < tol
    assert torch.equal(out, residual.to(dtype))
    onto = torch.ones(T, H, device=DEV)
    part.forward_into(onto, gpu(x, dtype), ctx, None)
    assert rel((onto - 1)[far.to(DEV)], want[far]) < max(tol, 1e-5)
    other = build(weight_on_input=False)
    other.setup(Runtime(dtype, torch.device(DEV)))
    other.bind(params)
    assert rel(other.forward(gpu(x, dtype), ctx, None), want) > 2e-2


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("H", [96, 40, 36, 2048, 100, 5000])
def test_the_norm_behind_a_sublayer_hands_on_the_stream(H, dtype):
    """``x += gain * y / rms(y)`` and the new x rounded, from plain rows of either dtype and from partial sums."""
    from kvcore_amd.ops import library as ops

    gen = torch.Generator().manual_seed(H)
    T, eps = 9, 1e-5
    res, y = rnd(T, H, gen=gen, dtype=torch.float32), rnd(T, H, gen=gen, dtype=torch.bfloat16)
    gain = rnd(H, gen=gen, dtype=torch.float32)
    want = res + plain.over_rms(y, eps) * gain
    for delta_dtype in DTYPES:
        residual, out = gpu(res), torch.empty(T, H, dtype=dtype, device=DEV)
        ops.norm_add_norm(out, residual, gpu(y, delta_dtype), gpu(gain), eps)
        assert rel(residual, want) < 2e-6 and torch.equal(out, residual.to(dtype))
    parts = rnd(3, T, H, gen=gen, dtype=torch.float32)
    want = res + plain.over_rms(parts.sum(0), eps) * gain
    residual, out = gpu(res), torch.empty(T, H, dtype=dtype, device=DEV)
    ops.norm_add_norm(out, residual, ops.SlicedRows(gpu(parts.reshape(3 * T, H)), 3, T, H), gpu(gain), eps)
    assert rel(residual, want) < 2e-6 and torch.equal(out, residual.to(dtype))


@pytest.mark.parametrize("T", [1, 40])
def test_rotation_tables_carry_the_yarn_factor(T):
    from kvcore_amd.ops import library as ops
    from kvcore_amd.parts.rotary import rotary_inv_freq, rotary_table_scale

    rot = {"dims": 24, "base": 10000.0, "scaling": {"factor": 8.0, "original": 300, "fast": 16.0, "slow": 1.0}}
    scaling = {"rope_type": "yarn", **rot["scaling"]}
    pos = torch.arange(T, dtype=torch.int32, device=DEV) * 37
    cos, sin = torch.empty(T, 12, device=DEV), torch.empty(T, 12, device=DEV)
    ops.rope_table(cos, sin, pos, rotary_inv_freq(24, 10000.0, scaling).to(DEV), rotary_table_scale(scaling))
    freqs, factor = plain.frequencies(rot)
    angle = pos.double().cpu()[:, None] * torch.tensor(freqs, dtype=F64)
    assert torch.allclose(cos.double().cpu(), torch.cos(angle) * factor, atol=2e-4)
    assert torch.allclose(sin.double().cpu(), torch.sin(angle) * factor, atol=2e-4)
