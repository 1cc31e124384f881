"""Koduzen on the engine against the plain float64 oracle (tests/koduzen_oracle.py): every mechanism
alone, whole prompts against token-by-token decoding and portions down to two tokens, mixed batches of
unequal requests over pages and state slots that are freed and reused, keys far away, on either side of
page borders, just inside and just outside the window, chunk edges of the retention, the first tokens of
a sequence, long decoding, other sizes, greedy generation through the scheduler. Each case runs on the
CPU reference ops and, marked gpu, on the HIP kernels."""
import json
import math
import os

import pytest
import torch
from safetensors.torch import save_file

import koduzen_oracle as oracle
from llmd_amd.engine.attn_meta import SeqMeta
from llmd_amd.engine.config import EngineConfig, ModelConfig
from llmd_amd.engine.engine import LLMEngine
from llmd_amd.engine.request import SamplingParams
from llmd_amd.models.mixers import GatedMLP, GroupedAttention, RetentionMixer, ScoreMoE, rope_table
from llmd_amd.ops import seqmix as sm

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
OP_DTYPES = [("cpu", torch.float32), pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
             pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)]
F64 = torch.float64
RAMP = {"factor": 3.0, "original": 96, "fast": 6.0, "slow": 1.0}


def att(heads, kv, dim, vdim, size, rot_dims=None, base=10000.0, scaling=RAMP, scale=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or 1.0 / math.sqrt(dim),
         "mask": {"size": size}, "rot": {"dims": rot_dims or dim, "base": base}}
    if scaling:
        m["rot"]["scaling"] = scaling
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def att2(heads, kv, dim, vdim, size, coef=0.4, every=16, scale=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or 1.0 / math.sqrt(dim),
         "mask": {"size": size}, "q_temp": {"coef": coef, "every": every}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention_2", "mixer": m}


def ret(heads, dim, vdim, rot_dims=None, base=10000.0, decay=None):
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"dims": rot_dims or dim, "base": base},
                                           "decay": decay or [1.0 - 2.0 ** (-3 - i) for i in range(heads)]}}


def ff(n, limit=1.5):
    return {"kind": "dense", "ff": n, "limit": limit}


def moe(experts, top, n, shared, identity=0, groups=1, keep=1, scale=1.3, limit=1.0, shared_limit=2.0):
    return {"kind": "moe", "expert": {"ff": n, "limit": limit}, "shared": {"ff": shared, "limit": shared_limit},
            "router": {"experts": experts, "identity": identity, "top": top, "groups": {"count": groups, "keep": keep},
                       "scale": scale}}


def config(layers, width=48, vocab=70, eps=1e-5, streams=2):
    return {"architecture": "Koduzen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "streams": streams,
            "layers": [dict(l, mlp=f) for l, f in layers]}


# sizes that differ wherever the design lets them: windows that are no multiple of a page or a key tile and differ
# from layer to layer (also between layers that share keys), partial and full rotation, three streams, groups of
# experts that mix real and identity ones, layers without a feed-forward
MIXED = config([(att2(6, 3, 24, 16, 20, coef=0.4, every=12), moe(7, 3, 24, 40, identity=5, groups=4, keep=2)),
                (ret(3, 16, 24, rot_dims=8), ff(40)),
                (att2(3, 3, 24, 16, 33, coef=-0.1, every=7, kv_from=0), None),
                (att(4, 2, 16, 40, 90, rot_dims=12, base=500.0), ff(56, limit=0.7)),
                (ret(5, 8, 12, decay=[0.5, 0.8, 0.9, 0.99, 0.999]), moe(10, 4, 16, 8, identity=2, groups=3, keep=2)),
                (att(2, 2, 16, 40, 12, rot_dims=12, base=500.0, kv_from=3), None),
                (att2(9, 3, 8, 24, 50), ff(24))], streams=3)
# values the first configuration keeps apart, made equal or 1 here: one head, one stream, one expert, all experts
# chosen, one group, a window of the token alone, a window of exactly a page, temperature off
PLAIN = config([(att2(1, 1, 16, 16, 1, coef=0.0, every=1, scale=1.0), ff(16, limit=1.0)),
                (att(1, 1, 16, 16, 64, scale=1.0, scaling=None), moe(1, 1, 16, 16, scale=1.0, limit=1.0, shared_limit=1.0)),
                (ret(1, 16, 16, decay=[0.9]), moe(4, 4, 32, 32, scale=1.0)),
                (att2(2, 2, 16, 16, 64, kv_from=None), None),
                (att2(2, 2, 16, 16, 64, kv_from=3), moe(2, 2, 16, 16, identity=2, groups=2, keep=2))],
               width=32, vocab=64, streams=1)
# multiples of nothing: vector loads, matrix-core padding and lane groups all take their slow paths
ODD = config([(att(9, 3, 10, 14, 13, rot_dims=6, scale=0.7), ff(22)),
              (ret(7, 6, 14, rot_dims=2), moe(3, 2, 10, 14, identity=2, groups=5, keep=3)),
              (att2(5, 5, 18, 6, 37, every=5, coef=1.1), None),
              (ret(3, 10, 34, rot_dims=10, base=77.0), ff(26)),
              (att2(10, 5, 18, 6, 100, scale=0.2, kv_from=2), moe(5, 3, 6, 10, identity=1))], width=34, vocab=51, eps=1e-3,
             streams=5)
ONLY_RETENTION = config([(ret(2, 32, 64), ff(16)), (ret(4, 64, 32, rot_dims=16), moe(6, 3, 8, 24, groups=2, keep=1))], width=32,
                        vocab=40, streams=4)
ONLY_ATTENTION = config([(att(8, 2, 64, 32, 40, rot_dims=32), moe(8, 3, 48, 48, groups=2, keep=1)),
                         (att2(4, 4, 128, 64, 300), ff(96)), (att2(8, 4, 128, 64, 70, kv_from=1), ff(64))], width=64, vocab=96)


def model_dir(tmp_path, cfg, seed=0, W=None):
    W = W or oracle.random_weights(cfg, seed)
    d = tmp_path / f"m{seed}"
    d.mkdir(exist_ok=True)
    (d / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in W.items()}, str(d / "model.safetensors"))
    return str(d), W


def engine(path, device, dtype="float32", pages=16, seqs=4, **kw):
    mc = ModelConfig.from_hf(path)
    kw.setdefault("enable_prefix_caching", False)
    cfg = EngineConfig.create(path, model_config=mc, device=device, dtype=dtype, load_format="safetensors",
                              weights_path=path, block_size=64, num_gpu_blocks=pages, max_num_seqs=seqs,
                              max_model_len=pages * 64 + 1, max_num_batched_tokens=pages * 64,
                              enforce_eager=True, prefill_token_align=0, **kw)
    return LLMEngine(cfg, capture_graphs=False)


def row_errs(got, want):
    d = got.double().cpu() - want
    return torch.sqrt((d * d).mean(-1)) / torch.sqrt((want * want).mean())


def rel_err(got, want):
    return float(row_errs(got, want).max())


def close(got, want, dtype):
    """float32: every row within rounding of the oracle. bfloat16: a router's close call can go the other
    way for a token, so the bound is held by nine rows in ten and by the median."""
    e = row_errs(got, want)
    if dtype == "float32":
        return float(e.max()) < 1e-4
    return float(e.quantile(0.9)) < 0.15 and float(e.median()) < 5e-2


def replay(eng, prompts, steps):
    """steps: list of lists of (name, count). Returns name -> logits [len, vocab] (all positions)."""
    at = {n: 0 for n in prompts}
    out = {n: [] for n in prompts}
    for step in steps:
        entries, end = [], []
        for n, c in step:
            toks = prompts[n][at[n]:at[n] + c]
            entries.append((n, toks, list(range(len(toks)))))
            at[n] += c
            if at[n] == len(prompts[n]):
                end.append(n)
        lg = eng.forced_step(entries, end)
        o = 0
        for n, c in step:
            out[n].append(lg[o:o + c].cpu())
            o += c
    return {n: torch.cat(v) for n, v in out.items() if v}


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _ti(v, device):
    return torch.tensor(v, dtype=torch.int32, device=device)


def _seq(device, q_lens, slots, init, lens=None, tables=None):
    """SeqMeta of a step: sequence i brings q_lens[i] tokens (ending at context length lens[i])."""
    n = len(q_lens)
    start = [0]
    for c in q_lens:
        start.append(start[-1] + c)
    lens = lens or q_lens
    row_seq = [i for i, c in enumerate(q_lens) for _ in range(c)]
    row_len = [lens[i] - c + j + 1 for i, c in enumerate(q_lens) for j in range(c)]
    tab = torch.zeros(n, 1, dtype=torch.int32)
    if tables is not None:
        tab = torch.zeros(n, max(len(t) for t in tables), dtype=torch.int32)
        for i, t in enumerate(tables):
            tab[i, :len(t)] = t
    return SeqMeta(n, _ti(start, device), _ti(slots, device), _ti(init, device), _ti(row_seq, device),
                   _ti(row_len, device), tab.to(device), max_len=max(lens), max_q=max(q_lens), q_lens=list(q_lens),
                   ctx_lens=list(lens))


def _tol(dtype, f32=1e-5, bf16=1e-2):
    return f32 if dtype == torch.float32 else bf16


def _shuffled_tables(lens, bs, g):
    total = sum(-(-n // bs) for n in lens) + 2
    perm = torch.randperm(total, generator=g).int()
    tables, off = [], 0
    for n in lens:
        tables.append(perm[off:off + -(-n // bs)])
        off += -(-n // bs)
    return total, tables


# ------------------------------------------------------------------ mechanisms alone (ops)
@pytest.mark.parametrize("device,dtype", OP_DTYPES)
@pytest.mark.parametrize("S,d", [(1, 40), (2, 33), (3, 64), (3, 2052), (4, 300), (5, 300), (16, 24)])
def test_streams_and_rms_norm(device, dtype, S, d):
    """One sublayer's end: streams remixed and fed, and the next input's RMS norm - the mean stays (it is far from zero)."""
    g = torch.Generator().manual_seed(S * d)
    T = 7
    X0 = torch.randn(S, T, d, generator=g) + 2.0
    w_in, w_out, nxt = (torch.randn(S, generator=g) for _ in range(3))
    mix = torch.randn(S, S, generator=g)
    nw, nw2 = ((1 + 0.3 * torch.randn(d, generator=g)).to(dtype) for _ in range(2))
    y = torch.randn(T, d, generator=g).to(dtype)
    X = X0.clone().to(device)
    h = sm.hyper_norm(X, w_in.to(device), nw.to(device), 1e-5, dtype, rms=True)
    u = sum(w_in[s].double() * X0[s].double() for s in range(S))
    assert h.dtype == dtype and rel_err(h.float(), oracle.rms_norm(u, 1e-5, nw)) < _tol(dtype)
    h2 = sm.hyper_update_norm(X, y.to(device), mix.to(device), w_out.to(device), nxt.to(device), nw2.to(device), 1e-5, dtype,
                              rms=True)
    W = {"in": w_in, "out": w_out, "mix": mix}
    new = oracle.hyper([s.double() for s in X0], W, "", lambda u: y.double())
    assert rel_err(X, torch.stack(new)) < 1e-5
    assert rel_err(h2.float(), oracle.rms_norm(sum(nxt[s].double() * new[s] for s in range(S)), 1e-5, nw2)) < _tol(dtype)


def test_ramp_scaled_frequencies():
    for dims, base, sc in [(12, 500.0, RAMP), (16, 300.0, dict(RAMP, original=512, fast=8.0)), (8, 1e4, None),
                           (64, 5e5, {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}),
                           (4, 10.0, {"factor": 2.0, "original": 7, "fast": 1.0, "slow": 1.0})]:
        f, mag = oracle.frequencies(dims, base, sc)
        if sc is RAMP:  # the ramp is entered: kept, blended and divided frequencies
            ratio = [a / b for a, b in zip(f, oracle.frequencies(dims, base)[0])]
            assert ratio[0] == 1.0 and abs(ratio[-1] - 1 / 3) < 1e-9 and any(0.34 < r < 0.99 for r in ratio)
        tab = rope_table(dims, base, 200, "cpu", sc)
        want = torch.tensor([[mag * math.cos(p * x) for x in f] + [mag * math.sin(p * x) for x in f] for p in (0, 1, 57, 199)],
                            dtype=F64)
        assert torch.allclose(tab[[0, 1, 57, 199]].double(), want, atol=1e-6)


def _page_rows(cache, dim, vdim, tab, n):
    """Rows [n, Hkv, dim + vdim] of a sequence out of the grouped-attention pages (keys row-major, values
    transposed)."""
    nb, Hkv, bs, Dr = cache.shape
    flat = cache.float().cpu().view(nb, Hkv, bs * Dr)
    k = flat[:, :, :bs * dim].view(nb, Hkv, bs, dim)
    v = flat[:, :, bs * dim:].view(nb, Hkv, vdim, bs)
    return torch.stack([torch.cat([k[int(tab[i // bs]), :, i % bs], v[int(tab[i // bs]), :, :, i % bs]], -1)
                        for i in range(n)])


@pytest.mark.parametrize("device,dtype", OP_DTYPES)
@pytest.mark.parametrize("wide,temp", [(True, False), (False, True), (True, True)], ids=["norms", "temperature", "both"])
@pytest.mark.parametrize("Hq,Hkv,dim,vdim,rot", [(6, 3, 24, 16, 12), (4, 2, 64, 40, 32), (2, 1, 128, 24, 128), (5, 5, 10, 6, 6),
                                                  (8, 8, 16, 8, 0), (32, 8, 128, 16, 64), (1, 1, 512, 16, 512),
                                                  (70, 2, 128, 8, 16), (34, 2, 512, 8, 32)])
def test_norms_of_whole_projections_temperature_and_cache(device, dtype, wide, temp, Hq, Hkv, dim, vdim, rot):
    """Norms over all of q and all of k (one head's columns far larger than the others', so that a norm per head
    would show), rotation, position factor and cache writes; then the same queries alone, without keys or a cache."""
    g = torch.Generator().manual_seed(Hq * dim)
    nq, nk, nv = Hq * dim, Hkv * dim, Hkv * vdim
    big = Hq * dim > 2048
    T, first = (20, 50) if big else (300, 50)          # positions 50 ..: over page borders and multiples of ``every``
    p = torch.randn(T, -(-(nq + nk + nv) // 8) * 8, generator=g)
    p[:, :dim] *= 5.0
    p[:, nq:nq + dim] *= 0.2
    p = p.to(dtype)
    w = 1 + 0.3 * torch.randn(nq + nk, generator=g)
    q_temp = {"coef": 0.6, "every": 17}
    m = GroupedAttention(8, Hq, Hkv, dim, vdim, 1.0, None, 1e-5, 512, device, dtype, bias=False, unit_norm=False, gate=False,
                         q_temp=q_temp)
    total, (tab,) = _shuffled_tables([first + T], 64, g)
    cache = torch.randn(total, Hkv, 64, dim + vdim, generator=g).to(dtype).to(device)
    cs = rope_table(rot, 300.0, 512, device, RAMP) if rot else None
    pos = torch.arange(first, first + T)
    slots = torch.tensor([int(tab[i // 64]) * 64 + i % 64 for i in pos.tolist()])
    x = p.double()
    q, k, v = x[:, :nq], x[:, nq:nq + nk], x[:, nq + nk:nq + nk + nv]
    if wide:
        q, k = oracle.rms_norm(q, 1e-5, w[:nq]), oracle.rms_norm(k, 1e-5, w[nq:])

    def turned(t, heads):
        full = torch.cat([torch.zeros(first, heads, dim, dtype=F64), t.reshape(T, heads, dim)])
        return oracle.rotate(full, rot, 300.0, RAMP)[first:] if rot else full[first:]

    q, k = turned(q, Hq), turned(k, Hkv)
    if temp:
        q = q * torch.tensor([oracle.temperature(i, q_temp) for i in pos.tolist()], dtype=F64)[:, None, None]
    args = (pos, cs.to(device) if rot else None)
    kw = dict(wide_norm=wide, q_scale=m.q_scale if temp else None)
    out = torch.empty(T, Hq, dim, dtype=dtype, device=device)
    sm.qkv_rope_cache(p.to(device), None, args[0].to(device), args[1], Hq, Hkv, dim, vdim, rot, False, 1e-5 if wide else None,
                      None, 0, 0.0, slots.to(device), cache, out, w.to(device) if wide else None, **kw)
    rows = _page_rows(cache, dim, vdim, tab, first + T)[first:]
    assert rel_err(out.float().view(T, -1), q.reshape(T, -1)) < _tol(dtype)
    assert rel_err(rows[..., :dim].reshape(T, -1), k.reshape(T, -1)) < _tol(dtype)
    assert rel_err(rows[..., dim:].reshape(T, -1), v) < _tol(dtype)
    alone = torch.empty(T, Hq, dim, dtype=dtype, device=device)
    sm.qkv_rope_cache(p[:, :nq].contiguous().to(device), None, args[0].to(device), args[1], Hq, 0, dim, vdim, rot, False,
                      1e-5 if wide else None, None, 0, 0.0, slots.to(device), None, alone,
                      w[:nq].contiguous().to(device) if wide else None, **kw)
    assert rel_err(alone.float().view(T, -1), q.reshape(T, -1)) < _tol(dtype)


def test_temperature_steps_at_multiples():
    """The factor is the same inside a stretch of ``every`` positions and rises where p + 1 is a multiple of it."""
    m = GroupedAttention(8, 1, 1, 8, 8, 1.0, None, 1e-5, 300, "cpu", torch.float32, unit_norm=False, gate=False,
                         q_temp={"coef": 0.5, "every": 49})
    f = m.q_scale
    assert float(f[0]) == 1.0 and float(f[47]) == 1.0 and abs(float(f[48]) - (1 + 0.5 * math.log(2))) < 1e-6
    assert float(f[96]) == float(f[48]) and float(f[97]) > float(f[96])
    assert torch.allclose(f.double(), torch.tensor([oracle.temperature(p, {"coef": 0.5, "every": 49}) for p in range(300)],
                                                   dtype=F64), atol=1e-6)


def _write_pages(rows, bs, dim, device, dtype, seed=1):
    n, Hkv, Dr = rows.shape
    nb = -(-n // bs)
    perm = torch.randperm(nb + 3, generator=torch.Generator().manual_seed(seed))[:nb]
    cache = torch.randn(nb + 3, Hkv, bs, Dr, generator=torch.Generator().manual_seed(seed + 1)).to(dtype)
    for i in range(n):
        cache[perm[i // bs], :, i % bs] = rows[i].to(dtype)
    k = cache[..., :dim].reshape(nb + 3, Hkv, bs * dim)
    v = cache[..., dim:].transpose(2, 3).reshape(nb + 3, Hkv, (Dr - dim) * bs)
    return torch.cat([k, v], -1).reshape(nb + 3, Hkv, bs, Dr).contiguous().to(device), perm.int()


WHERE = ["window-first", "before-window", "page-end", "page-start", "very-first", "last-seen", "first-unseen"]


@pytest.mark.parametrize("device,dtype", OP_DTYPES)
@pytest.mark.parametrize("decode", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("size", [90, 300, 697])
@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("biased", [False, True], ids=["plain", "bias+sink"])
def test_one_key_stands_out(device, dtype, where, decode, size, biased):
    """One key among 700 has a score far above the rest: the output is its value if and only if the row may
    see it, as the last row of a 5-token portion and as a single decoded token; without and with the distance
    bias and a sink."""
    Hq, Hkv, dim, vdim, n, seen = 6, 3, 24, 16, 700, 697
    i = seen - 1
    j = max(0, {"window-first": i - size + 1, "before-window": i - size, "page-end": 639, "page-start": 640, "very-first": 0,
                "last-seen": i, "first-unseen": seen}[where])
    sees = oracle.visible(seen - 1, j, size)
    g = torch.Generator().manual_seed(7)
    rows = torch.randn(n, Hkv, dim + vdim, generator=g) * 0.3
    nq = 1 if decode else 5
    q = torch.randn(nq, Hq, dim, generator=g) * 0.3
    h = 5                                                  # the head with the smallest slope reads kv head 2
    rows[j, 2, :dim] = q[-1, h] / q[-1, h].norm() * 16.0   # and looks straight at key j
    q[-1, h] *= 6.0
    rows, q = rows.to(dtype).float(), q.to(dtype).float()
    cache, table = _write_pages(rows, 64, dim, device, dtype)
    seq = _seq(device, [nq], [0], [0], lens=[seen], tables=[table])
    sinks = torch.tensor([0.5, -1.0, 2.0, 0.0, 1.0, -3.0])
    slopes = torch.tensor([oracle.slope(a, Hq) for a in range(Hq)])
    out = sm.grouped_attention(q.to(dtype).to(device), cache, dim, vdim, 1.0, seq, None, slopes.to(device) if biased else None,
                               0, sinks.to(device) if biased else None, size).float().cpu().view(nq, Hq, vdim)
    assert torch.allclose(out[-1, h], rows[j, 2, dim:], atol=3e-2) == sees
    for t in range(nq):
        at = seen - nq + t
        js = torch.tensor([k for k in range(n) if oracle.visible(at, k, size)])
        for a in range(Hq):
            s = rows[js, a // 2, :dim].double() @ q[t, a].double()
            if biased:
                s = torch.cat([s - oracle.slope(a, Hq) * (at - js).double(), sinks[a:a + 1].double()])
            want = torch.softmax(s, 0)[:js.numel()] @ rows[js, a // 2, dim:].double()
            assert rel_err(out[t, a][None], want[None]) < _tol(dtype, 1e-4, 3e-2)


@pytest.mark.parametrize("device,dtype", OP_DTYPES)
@pytest.mark.parametrize("Hq,Hkv,dim,vdim,size,bs", [(40, 1, 64, 32, 300, 64), (12, 4, 48, 40, 75, 64), (34, 2, 32, 48, 650, 32),
                                                     (6, 2, 192, 136, 500, 64), (4, 4, 128, 80, 90, 96), (8, 2, 64, 64, 200, 16),
                                                     (6, 3, 20, 12, 300, 64), (3, 1, 256, 256, 90, 64)])
def test_steps_of_single_tokens(device, dtype, Hq, Hkv, dim, vdim, size, bs):
    """Decoded tokens of four sequences at once - hundreds of keys, less than a tile, exactly a page, one key -
    with a distance bias, a window and sinks, page sizes that are and are not multiples of a key tile, sizes
    outside the direct form; the pages' unwritten rest holds NaN."""
    g = torch.Generator().manual_seed(Hq * dim)
    lens = [701, 21, 64, 1]
    total, tables = _shuffled_tables(lens, bs, g)
    cache = torch.full((total, Hkv, bs * (dim + vdim)), float("nan"))
    k, v = cache[:, :, :bs * dim].view(total, Hkv, bs, dim), cache[:, :, bs * dim:].view(total, Hkv, vdim, bs)
    rows = [(torch.randn(n, Hkv, dim + vdim, generator=g) * 0.5).to(dtype).float() for n in lens]
    for r, tab in zip(rows, tables):
        for i in range(r.shape[0]):
            k[int(tab[i // bs]), :, i % bs] = r[i, :, :dim]
            v[int(tab[i // bs]), :, :, i % bs] = r[i, :, dim:]
    q = (torch.randn(4, Hq, dim, generator=g) * 0.5).to(dtype).float()
    sinks = torch.randn(Hq, generator=g)
    slopes = torch.tensor([oracle.slope(a, Hq) for a in range(Hq)])
    seq = _seq(device, [1] * 4, [0] * 4, [0] * 4, lens=lens, tables=tables)
    pages = cache.to(dtype).view(total, Hkv, bs, dim + vdim).to(device)
    out = sm.grouped_attention(q.to(dtype).to(device), pages, dim, vdim, 0.4, seq, None, slopes.to(device), 0,
                               sinks.to(device), size)
    for t, n in enumerate(lens):
        js = torch.tensor([j for j in range(n) if oracle.visible(n - 1, j, size)])
        want = []
        for h in range(Hq):
            kv = rows[t][js, h // (Hq // Hkv)].double()
            s = kv[:, :dim] @ q[t, h].double() * 0.4 - oracle.slope(h, Hq) * (n - 1 - js).double()
            want.append(torch.softmax(torch.cat([s, sinks[h:h + 1].double()]), 0)[:-1] @ kv[:, dim:])
        assert rel_err(out[t].float().view(Hq, vdim), torch.stack(want)) < _tol(dtype, 1e-4, 3e-2), n


def _retention_rows(p, H, dk, dv, gate, rot, decay, eps):
    """One sequence's projected rows [T, q | k | v (| g)] through the oracle's equations."""
    T = p.shape[0]
    x = p.double()
    q, k = x[:, :H * dk].view(T, H, dk), x[:, H * dk:2 * H * dk].view(T, H, dk)
    if rot:
        q, k = oracle.rotate(q, rot, 300.0), oracle.rotate(k, rot, 300.0)
    k = k / math.sqrt(dk)
    v = x[:, 2 * H * dk:2 * H * dk + H * dv].view(T, H, dv)
    o = torch.cat([oracle.rms_norm(oracle.retention_rows(q[:, n], k[:, n], v[:, n], decay[n]), eps) for n in range(H)], -1)
    return o * oracle.silu(x[:, 2 * H * dk + H * dv:2 * H * dk + 2 * H * dv]) if gate else o


@pytest.mark.parametrize("device,dtype", OP_DTYPES)
@pytest.mark.parametrize("H,dk,dv,rot,gate", [(3, 16, 24, 8, True), (2, 64, 64, 64, True), (2, 64, 128, 32, True),
                                              (1, 32, 256, 32, True), (2, 6, 14, 2, True), (1, 10, 34, 10, False),
                                              (1, 72, 320, 48, True), (2, 130, 70, 0, True), (3, 1, 1, 0, False),
                                              (1, 260, 1030, 4, True)])
def test_retention_steps(device, dtype, H, dk, dv, rot, gate):
    """Sequences in portions over several steps: single tokens ahead of portions, a single token behind a portion,
    steps of single tokens only, two tokens, portions of exactly a chunk, one less and one more, of several chunks;
    slots swapped against the step's order and holding something old; a later sequence takes over a used slot."""
    g = torch.Generator().manual_seed(H * dk + dv)
    n = 2 * H * dk + (2 if gate else 1) * H * dv
    lens = {"a": 330, "b": 137, "c": 66, "d": 2}
    p = {k: torch.randn(m, -(-n // 8) * 8, generator=g).to(dtype) for k, m in lens.items()}
    decay = [0.999, 0.7, 0.96][:H]
    powers = (torch.tensor(decay, dtype=F64)[:, None] ** torch.arange(sm.RETENTION_CHUNK + 1)).float().to(device)
    cs = rope_table(rot, 300.0, 512, device) if rot else None
    state = torch.randn(3, H, dk, dv, generator=g).to(device)
    slot = {"a": 2, "b": 0, "c": 0, "d": 1}
    at, got = dict.fromkeys(lens, 0), {k: [] for k in lens}
    for step in ([("b", 1), ("a", 2)], [("b", 1), ("a", 1)], [("a", 1), ("b", 64)], [("a", 63), ("d", 1), ("b", 65)],
                 [("d", 1), ("a", 1)], [("b", 1), ("a", 130)], [("a", 2), ("b", 4)], [("b", 1), ("a", 5)],
                 [("a", 1), ("c", 3)], [("a", 1), ("c", 63)], [("a", 123)]):
        names = [k for k, _ in step]
        seq = _seq(device, [c for _, c in step], [slot[k] for k in names], [int(at[k] > 0) for k in names],
                   lens=[at[k] + c for k, c in step])
        pos = torch.tensor([i for k, c in step for i in range(at[k], at[k] + c)], device=device)
        out = sm.retention(torch.cat([p[k][at[k]:at[k] + c] for k, c in step]).to(device), H, dk, dv, gate, pos, cs, rot,
                           powers, 1e-5, state, seq)
        assert out.dtype == dtype
        o = 0
        for k, c in step:
            got[k].append(out[o:o + c].float().cpu())
            at[k] += c
            o += c
    for k, m in lens.items():
        assert at[k] == m
        want = _retention_rows(p[k][:, :n], H, dk, dv, gate, rot, decay, 1e-5)
        assert rel_err(torch.cat(got[k]), want) < _tol(dtype), k


@pytest.mark.parametrize("device,dtype", OP_DTYPES)
def test_retention_of_a_far_token(device, dtype):
    """A head that hardly forgets: the query looks straight at a key hundreds of tokens back, over many chunks."""
    H, dk, dv, T, at = 1, 16, 16, 700, 3
    g = torch.Generator().manual_seed(2)
    p = torch.randn(T, 2 * dk + dv, generator=g) * 0.05
    p[at, dk:2 * dk] = 3.0
    p[T - 1, :dk] = 3.0
    p[at, 2 * dk:] = torch.arange(1.0, dv + 1)
    p = p.to(dtype)
    powers = (torch.tensor([[0.9999]], dtype=F64) ** torch.arange(sm.RETENTION_CHUNK + 1)).float().to(device)
    for cuts in ([700], [699, 1], [350, 350], [64] * 10 + [58, 2], [5] * 140):
        state = torch.ones(1, H, dk, dv, device=device)
        done, out = 0, None
        for c in cuts:
            seq = _seq(device, [c], [0], [int(done > 0)], lens=[done + c])
            out = sm.retention(p[done:done + c].to(device), H, dk, dv, False, torch.arange(done, done + c, device=device), None, 0,
                               powers, 1e-6, state, seq)
            done += c
        v = p[at, 2 * dk:].double()
        assert rel_err(out[-1:].float(), oracle.rms_norm(v, 0.0)[None]) < 0.05, cuts
        assert rel_err(out[-1:].float(), _retention_rows(p, H, dk, dv, False, 0, [0.9999], 1e-6)[-1:]) < _tol(dtype), cuts


@pytest.mark.parametrize("device,dtype", OP_DTYPES)
@pytest.mark.parametrize("n", [1, 24, 37, 2048])
@pytest.mark.parametrize("limit", [0.5, 1.0, 7.0])
def test_clamped_units(device, dtype, n, limit):
    """Gates far above the limit and far below zero, ups beyond both limits."""
    g = torch.Generator().manual_seed(n)
    gu = (torch.randn(5, 2 * n + 8, generator=g) * 3.0 * limit).to(dtype)
    gu[0, :n] = -20.0
    gu[1, n:2 * n] = -30.0
    x = gu.double()
    a, u = x[:, :n].clamp(max=limit), x[:, n:2 * n].clamp(-limit, limit)
    want = a / (1 + torch.exp(-1.702 * a)) * (u + 1)
    got = sm.gated_act(gu.to(device)[:, :2 * n], n, "swish_limit", limit)
    assert got.dtype == dtype and rel_err(got.float(), want) < _tol(dtype)
    assert bool((gu[:, :n].float() > limit).any()) or n == 1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n,top,groups,keep", [(22, 4, 2, 1), (12, 4, 4, 2), (9, 9, 3, 3), (132, 8, 4, 2), (64, 1, 64, 1),
                                               (500, 6, 50, 3), (130, 5, 65, 4), (600, 7, 6, 2), (16, 2, 1, 1)])
def test_routing_inside_the_best_groups(device, n, top, groups, keep):
    """Choices, weights and scale against the oracle, choice scores of both signs (an excluded expert that counted as
    zero instead of minus infinity would win), a group kept for one large expert while its others are small."""
    g = torch.Generator().manual_seed(n + top)
    z = torch.randn(40, n, generator=g) * 2.0
    corr = torch.randn(n, generator=g) * 0.3 - 1.5
    router = {"top": top, "groups": {"count": groups, "keep": keep}, "scale": 1.7}
    ids, w = sm.moe_route_scores(z.to(device), corr.to(device), top, groups, keep, 1.7)
    ids, w = ids.cpu(), w.cpu()
    negative = 0
    for t in range(40):
        want = dict(oracle.route(z[t].double(), corr.double(), router))
        got = {int(i): float(x) for i, x in zip(ids[t], w[t])}
        assert set(got) == set(want), t
        assert all(abs(got[i] - want[i]) < 1e-5 for i in want), t
        negative += any(float(torch.softmax(z[t].double(), 0)[i] + corr[i]) < 0 for i in want)
    assert negative > 0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n,groups", [(12, 4), (600, 6)])
def test_routing_ties_go_to_the_lower_index(device, n, groups):
    ids, w = sm.moe_route_scores(torch.zeros(2, n).to(device), torch.zeros(n).to(device), 3, groups, 2, 1.0)
    per = n // groups
    if device == "cpu":   # top-k of equal numbers: some members of the first two groups
        assert bool((ids < 2 * per).all())
    else:
        assert ids.cpu().tolist() == [[0, 1, 2]] * 2
    assert torch.allclose(w.cpu(), torch.full((2, 3), 1 / 3))


@pytest.mark.parametrize("device,dtype", OP_DTYPES)
@pytest.mark.parametrize("E,identity,top,groups,keep,d,n,shared", [(7, 5, 3, 4, 2, 40, 24, 40), (64, 2, 6, 3, 2, 128, 96, 200),
                                                                   (3, 0, 3, 1, 1, 34, 10, 14), (1, 1, 2, 1, 1, 16, 16, 0),
                                                                   (12, 4, 4, 2, 1, 64, 32, 0)])
@pytest.mark.parametrize("T", [1, 70])
def test_experts_with_a_shared_one(device, dtype, E, identity, top, groups, keep, d, n, shared, T):
    """Router, clamped experts, identity experts and the shared expert with a limit of its own, the router's rows scaled
    so that no call is close."""
    spec = moe(E, top, n, shared, identity, groups, keep, scale=1.6, limit=0.8, shared_limit=2.5)
    if not shared:
        spec["shared"] = None
    cfg = config([(ret(1, 8, 8), spec)], width=d, vocab=8)
    W = {k: v.to(dtype) for k, v in oracle.random_weights(cfg, 3).items()}
    W["l0.mlp.router"] = W["l0.mlp.router"] * 4.0
    sh = GatedMLP(d, shared, "swish_limit", device, dtype, limit=2.5) if shared else None
    m = ScoreMoE(d, n, E, identity, top, "swish_limit", device, dtype, limit=0.8, groups=groups, keep=keep, scale=1.6, shared=sh)
    m.router.copy_(W["l0.mlp.router"])
    m.correction.copy_(W["l0.mlp.correction"])
    for e in range(E):
        m.w1[e, :n].copy_(W[f"l0.mlp.e{e}.gate"])
        m.w1[e, n:].copy_(W[f"l0.mlp.e{e}.up"])
        m.w2[e].copy_(W[f"l0.mlp.e{e}.down"])
    if shared:
        sh.gate_up.weight[:shared].copy_(W["l0.mlp.shared.gate"])
        sh.gate_up.weight[shared:].copy_(W["l0.mlp.shared.up"])
        sh.down.weight.copy_(W["l0.mlp.shared.down"])
    m.finalize()
    h = torch.randn(T, d, generator=torch.Generator().manual_seed(T)).to(dtype)
    want = oracle.experts(h.double(), W, "l0.mlp.", spec)
    assert rel_err(m(h.to(device)).float(), want) < _tol(dtype, 1e-5, 3e-2)


def test_groups_must_fit():
    for bad in (dict(groups=5, keep=1), dict(groups=4, keep=5), dict(groups=4, keep=0), dict(groups=4, keep=1)):
        with pytest.raises(ValueError):
            ScoreMoE(8, 8, 10, 2, 4, "silu", "cpu", torch.float32, **bad)
    with pytest.raises(ValueError):
        RetentionMixer(8, 2, 4, 4, [0.5], None, 1e-5, 8, "cpu", torch.float32)


# ------------------------------------------------------------------ the model on the engine
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("layers", [[(att(6, 3, 24, 16, 20, rot_dims=12), ff(40))], [(att2(4, 2, 16, 24, 50), None)],
                                    [(ret(3, 16, 24), None)], [(ret(2, 16, 8, rot_dims=4), moe(6, 2, 24, 16))],
                                    [(att2(2, 1, 32, 32, 30), moe(4, 1, 16, 32, identity=2, groups=3, keep=1))],
                                    [(att2(4, 2, 16, 24, 20), None), (att2(2, 2, 16, 24, 45, kv_from=0), None)],
                                    [(att(4, 2, 16, 24, 20), None), (att(6, 2, 16, 24, 45, kv_from=0), None)]],
                         ids=["attention+ff", "attention_2-only", "retention-only", "retention+experts", "attention_2+experts",
                              "shared-keys", "shared-rotated-keys"])
def test_each_layer_kind_alone(tmp_path, device, layers):
    cfg = config(layers)
    path, W = model_dir(tmp_path, cfg)
    toks = tokens(70, cfg["vocab"], 1)
    got = replay(engine(path, device), {"a": toks}, [[("a", 70)]])["a"]
    assert rel_err(got, oracle.forward(cfg, W, toks)) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
def test_residual_after_every_layer(tmp_path, device):
    import numpy as np

    path, W = model_dir(tmp_path, MIXED)
    toks = tokens(40, MIXED["vocab"], 2)
    per_layer = []
    oracle.forward(MIXED, W, toks, per_layer)
    r = engine(path, device).runner
    pl = {"graph": False, "nd": 0, "ids": toks, "pos": list(range(40)), "slots": list(range(40)),
          "d_bt": np.zeros((0, r.width), "int32"), "d_len": np.zeros(0, "int32"), "p_ql": [40], "p_ctx": [40],
          "p_bt": np.zeros((1, r.width), "int32"), "rows": [], "seq": ([0], [0])}
    ids, meta = r._eager_meta(pl)
    got = []
    r.model(ids, meta, layer_out=got)
    assert len(got) == len(MIXED["layers"])
    for i, (a, b) in enumerate(zip(got, per_layer)):
        assert rel_err(a, b) < 1e-4, i


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_decode_and_portions_agree(tmp_path, device, dtype):
    path, W = model_dir(tmp_path, MIXED)
    toks = tokens(150, MIXED["vocab"], 3)
    want = oracle.forward(MIXED, W, toks)
    whole = replay(engine(path, device, dtype), {"a": toks}, [[("a", 150)]])["a"]
    assert close(whole, want, dtype)
    # a short prompt, then 140 tokens one by one over two page borders; every window passes over decoded tokens
    dec = replay(engine(path, device, dtype), {"a": toks}, [[("a", 10)]] + [[("a", 1)]] * 140)["a"]
    assert close(dec, want, dtype)
    # portions that end just before, at and just after page, chunk and window edges, down to two and one tokens
    cuts = [2, 17, 1, 1, 40, 3, 2, 58, 1, 1, 2, 14, 8]
    assert sum(cuts) == 150
    por = replay(engine(path, device, dtype), {"a": toks}, [[("a", c)] for c in cuts])["a"]
    assert close(por, want, dtype)
    two = replay(engine(path, device, dtype), {"a": toks}, [[("a", 2)]] * 75)["a"]
    assert close(two, want, dtype)
    if dtype == "float32":  # the ways differ by rounding only
        for other in (dec, por, two):
            assert rel_err(other, whole.double()) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_batches_reuse_pages_and_slots(tmp_path, device):
    """Five unequal requests through three live places and seven pages: portions beside single
    tokens, requests that pause, end and hand their pages and state slots to the next one."""
    path, W = model_dir(tmp_path, MIXED)
    lens = {"a": 130, "b": 1, "c": 67, "d": 90, "e": 64}
    prompts = {n: tokens(k, MIXED["vocab"], 10 + i) for i, (n, k) in enumerate(lens.items())}
    steps = [[("a", 60), ("b", 1), ("c", 2)],
             [("c", 1), ("a", 4)],
             [("a", 1), ("c", 62), ("d", 30)],           # b's page and slot reused by d
             [("d", 1), ("a", 63)],                      # a reaches 128: exactly two pages
             [("c", 1), ("d", 34), ("a", 1)],
             [("c", 1), ("a", 1), ("d", 25)],            # all three end: every page and slot is free again
             [("e", 3)],
             [("e", 61)]]
    eng = engine(path, device, pages=7, seqs=3)
    got = replay(eng, prompts, steps)
    for n in prompts:
        assert got[n].shape[0] == lens[n], n
        assert rel_err(got[n], oracle.forward(MIXED, W, prompts[n])) < 1e-4, n
    eng.bm.check_invariants()
    assert eng.bm.num_free() == 7 and eng.bm.slots.num_free() == 3
    alone = replay(engine(path, device, pages=6, seqs=3), {"d": prompts["d"]}, [[("d", 90)]])["d"]
    assert rel_err(got["d"], alone.double()) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cfg", [PLAIN, ODD, ONLY_RETENTION, ONLY_ATTENTION],
                         ids=["equal-or-one", "odd", "retention-only", "attention-only"])
def test_other_sizes(tmp_path, device, cfg, dtype):
    path, W = model_dir(tmp_path, cfg, seed=5)
    toks = tokens(80, cfg["vocab"], 6)
    want = oracle.forward(cfg, W, toks)
    got = replay(engine(path, device, dtype), {"a": toks},
                 [[("a", 5)], [("a", 60)], [("a", 2)]] + [[("a", 1)]] * 13)["a"]
    assert close(got, want, dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_of_a_sequence(tmp_path, device):
    """One-, two- and three-token sequences and a prompt cut after its first and third token: the retention starts
    from zeros whatever its slot holds, then continues its state."""
    path, W = model_dir(tmp_path, ODD, seed=9)
    eng = engine(path, device)
    for n, cuts in ((1, [1]), (2, [2]), (3, [1, 2]), (9, [1, 2, 1, 5]), (9, [2, 7]), (12, [1] * 12)):
        toks = tokens(n, ODD["vocab"], n)
        got = replay(eng, {"a": toks}, [[("a", c)] for c in cuts])["a"]
        assert rel_err(got, oracle.forward(ODD, W, toks)) < 1e-4, (n, cuts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["attention", "attention_2", "shared"])
def test_the_windows_edge_decides(tmp_path, device, kind):
    """Queries that look straight at one token, hundreds of decoded tokens: the last logits follow that token while
    it is the window's first key and no longer once it has left. "shared": the second of two layers over the same
    keys has the wider window and decides."""
    size, at, n = 40, 190, 235
    if kind == "attention":
        cfg = config([(att(2, 1, 16, 16, size, rot_dims=4, scaling=None, scale=1.0), None)], width=16, vocab=30)
    elif kind == "attention_2":
        cfg = config([(att2(2, 1, 16, 16, size, scale=6.0, coef=0.05, every=64), None)], width=16, vocab=30)
    else:
        cfg = config([(att2(2, 1, 16, 16, 11, scale=6.0), None), (att2(2, 1, 16, 16, size, scale=6.0, kv_from=0), None)],
                     width=16, vocab=30)
    W = oracle.random_weights(cfg, 4)
    for q in range(len(cfg["layers"])):
        W[f"l{q}.hc1.in"], W[f"l{q}.hc1.out"] = torch.full((2,), 0.5), torch.full((2,), 0.1)
        W[f"l{q}.hc1.mix"] = torch.eye(2)
        if kind != "attention":
            W[f"l{q}.mix.sink"] = torch.full((2,), -20.0)
    # the other tokens are alike, so one rank-one query matrix points all of them at token 0's key
    W["embed"] = torch.randn(30, 16, generator=torch.Generator().manual_seed(8)) * 0.2 + W["embed"][3]
    W["embed"][0] = oracle.rms_norm(torch.ones(16, dtype=F64), 0.0).float() * 3.0
    if kind == "attention":
        W["l0.mix.k"][:4] = 0.0                              # the rotated dimensions take no part
    e0 = oracle.rms_norm(W["embed"][0].double(), cfg["norm"]["eps"], W["l0.norm1"])
    k0 = W["l0.mix.k"].double() @ e0
    for q in range(len(cfg["layers"])):
        a0 = oracle.rms_norm(W["embed"][1:].double(), cfg["norm"]["eps"], W[f"l{q}.norm1"]).mean(0)
        W[f"l{q}.mix.q"] = torch.outer(k0.repeat(2), a0 / (a0 @ a0)).float()
    path, _ = model_dir(tmp_path, cfg, W=W)
    base = [1 + t for t in tokens(n + 1, 29, 5)]
    runs = {}
    for name, tok in (("zero", 0), ("other", base[at])):
        toks = base[:at] + [tok] + base[at + 1:]
        got = replay(engine(path, device), {"a": toks}, [[("a", 180)]] + [[("a", 1)]] * (n - 179))["a"]
        assert rel_err(got, oracle.forward(cfg, W, toks)) < 1e-4, name
        runs[name] = got
    inside, outside = at + size - 1, at + size
    diff = lambda i: rel_err(runs["zero"][i][None], runs["other"][i][None].double())   # noqa: E731
    assert diff(inside) > 1e-3
    assert diff(outside) < (1e-2 * diff(inside) if kind == "shared" else 1e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_a_far_token_stays_in_the_retention(tmp_path, device):
    """A retention layer that hardly forgets, a token 300 places back: the logits still follow it, in a prompt, over
    portions and after long decoding, and every run agrees with the oracle."""
    cfg = config([(ret(2, 16, 16, rot_dims=4, decay=[0.9999, 0.9995]), None), (att2(2, 1, 16, 16, 20), ff(24))], width=32, vocab=30)
    W = oracle.random_weights(cfg, 6)
    path, _ = model_dir(tmp_path, cfg, W=W)
    base = tokens(300, 30, 7)
    other = [(base[0] + 1) % 30] + base[1:]
    last = {}
    for name, toks in (("base", base), ("other", other)):
        want = oracle.forward(cfg, W, toks)
        for cuts in ([300], [100] + [1] * 200, [2, 63, 1, 64, 65, 100, 5]):
            got = replay(engine(path, device), {"a": toks}, [[("a", c)] for c in cuts])["a"]
            assert rel_err(got, want) < 1e-4, (name, cuts)
        last[name] = want[-1]
    assert rel_err(last["base"][None], last["other"][None]) > 1e-3


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(tmp_path, device):
    path, W = model_dir(tmp_path, MIXED, seed=8)
    shared = tokens(70, MIXED["vocab"], 21)
    prompts = [tokens(9, MIXED["vocab"], 20), shared, tokens(1, MIXED["vocab"], 22), shared[:66] + [1, 2, 3]]
    eng = engine(path, device, pages=10, seqs=2, async_scheduling=False)   # 4 requests over 2 places
    reqs = eng.generate(prompts, SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True))
    for p, r in zip(prompts, reqs):
        seq = list(p)
        for _ in range(6):
            seq.append(int(oracle.forward(MIXED, W, seq)[-1].argmax()))
        assert r.output_token_ids == seq[len(p):]
    eng.bm.check_invariants()


@pytest.mark.parametrize("device", DEVICES)
def test_a_stack_without_retention_reuses_cached_prefixes(tmp_path, device):
    """No recurrent state: no slots, and a prompt that begins like an earlier one starts from its cached pages - the
    layer that shares keys reads them there too."""
    path, W = model_dir(tmp_path, ONLY_ATTENTION, seed=2)
    shared = tokens(140, ONLY_ATTENTION["vocab"], 30)
    eng = engine(path, device, enable_prefix_caching=True, async_scheduling=False)
    assert not eng.runner.stateful and eng.runner.state_pool is None
    for tail in ([5, 6], [7, 8, 9]):
        r = eng.generate([shared + tail], SamplingParams(max_tokens=3, temperature=0.0, ignore_eos=True))[0]
        seq = shared + tail
        for _ in range(3):
            seq.append(int(oracle.forward(ONLY_ATTENTION, W, seq)[-1].argmax()))
        assert r.output_token_ids == seq[len(shared + tail):]
    assert r.num_cached_tokens == 128


@pytest.mark.parametrize("device", DEVICES)
def test_preset_serves_with_random_weights(device):
    """``--model tiny-koduzen`` without a checkpoint: the engine's ordinary generate path, sampled
    and greedy requests together, decoding past page borders and the windows."""
    from llmd_amd.engine.config import get_model_config

    mc = get_model_config("tiny-koduzen")
    assert mc.model_type == "koduzen" and mc.hyper_streams == 2 and len(mc.layer_specs) == 4 and mc.tie_word_embeddings
    cfg = EngineConfig.create("tiny-koduzen", device=device, block_size=16, num_gpu_blocks=40, max_num_seqs=3,
                              max_model_len=200, max_num_batched_tokens=64, enforce_eager=True)
    eng = LLMEngine(cfg, capture_graphs=False)
    prompts = [tokens(30, 512, 1), tokens(5, 512, 2), tokens(61, 512, 3), tokens(30, 512, 1)]
    params = [SamplingParams(max_tokens=20, temperature=0.0, ignore_eos=True),
              SamplingParams(max_tokens=8, temperature=0.8, top_p=0.9, seed=4, ignore_eos=True),
              SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True),
              SamplingParams(max_tokens=20, temperature=0.0, ignore_eos=True)]
    reqs = [eng.add_request(f"r{i}", p, sp) for i, (p, sp) in enumerate(zip(prompts, params))]
    while eng.has_unfinished():
        eng.step()
    assert [len(r.output_token_ids) for r in reqs] == [20, 8, 12, 20]
    assert all(0 <= t < 512 for r in reqs for t in r.output_token_ids)
    eng.bm.check_invariants()


def test_config_reads_every_size_from_the_file(tmp_path):
    path, _ = model_dir(tmp_path, ODD)
    mc = ModelConfig.from_hf(path)
    assert mc.model_type == "koduzen" and mc.hidden_size == 34 and mc.vocab_size == 51 and mc.hyper_streams == 5
    assert mc.rms_norm_eps == 1e-3 and mc.num_hidden_layers == 5
    assert [l["type"] for l in mc.layer_specs] == ["attention", "retention", "attention_2", "retention", "attention_2"]
    assert mc.layer_specs[2]["mixer"]["mask"] == {"size": 37} and mc.layer_specs[4]["mixer"]["kv_from"] == 2
    assert mc.num_local_experts == 5 and mc.num_experts_per_tok == 3 and mc.moe_intermediate_size == 10
    for change in (lambda c: c["layers"][1].update(type="something else"),
                   lambda c: c["layers"][0]["mlp"].update(kind="something else"),
                   lambda c: c["layers"][4]["mixer"].update(kv_from=0),           # another kind of layer
                   lambda c: c["layers"][2]["mixer"].update(kv_from=4),           # a later layer
                   lambda c: c["layers"][4]["mixer"].update(kv_heads=10),         # other heads than its source
                   lambda c: c["layers"][1]["mixer"]["decay"].pop(),
                   lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4),
                   lambda c: c["layers"][1]["mlp"]["router"].update(top=4)):
        bad = json.loads(json.dumps(ODD))
        change(bad)
        with pytest.raises(ValueError):
            ModelConfig.from_hf(bad)


def test_a_missing_tensor_is_an_error(tmp_path):
    for name in ("l3.mix.k.norm", "l1.mix.g", "l0.mix.sink", "l4.mlp.correction", "l6.hc2.mix"):
        W = oracle.random_weights(MIXED, 0)
        W.pop(name)
        path, _ = model_dir(tmp_path, MIXED, W=W)
        with pytest.raises(KeyError):
            engine(path, "cpu")


def test_trace_runner_program(tmp_path):
    """bin/trace_run as a program on this design: a request that skips a step, ends, and a later one
    that takes over its pages and its state slot."""
    import subprocess
    import sys

    import numpy as np

    path, W = model_dir(tmp_path, ODD, seed=3)
    V = ODD["vocab"]
    a, b, c = (tokens(n, V, 40 + i) for i, n in enumerate((70, 3, 5)))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:62], "want": [0, 61]}, {"id": "b", "tokens": b[:2], "want": []}],
              "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[62:63], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[2:], "want": [0]}, {"id": "a", "tokens": a[63:], "want": [1, 6]}],
              "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": c, "want": [4]}], "end": ["c"]}]
    out = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "192", "--max-seqs", "2", "--device", "cpu"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    la, lb, lc = (oracle.forward(ODD, W, t) for t in (a, b, c))
    want = {0: torch.stack([la[0], la[61]]), 1: la[62:63], 2: torch.stack([lb[2], la[64], la[69]]), 3: lc[4:5]}
    for i, w in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, V).copy())
        assert got.shape == w.shape and rel_err(got, w) < 1e-4, i
