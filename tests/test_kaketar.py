"""Kaketar decoder: the engine (scheduler, paged latent pool, state pool,
batch builder, ops) against the plain float64 oracle in kaketar_oracle.py.

Every test builds its own small configuration and random bf16 weights,
replays token schedules through the product's trace-replay entry point
(or LLM.generate) and compares logits with the oracle run on each whole
sequence alone. CPU runs exercise the engine with the torch reference
ops; the same tests marked ``gpu`` exercise the HIP kernels in fp32
(tight tolerance) and bf16.
"""

import json
import os
import tempfile

import numpy as np
import pytest
import torch

import kaketar_oracle as oracle

DEVICES = [pytest.param("cpu", "float32", id="cpu-f32"),
           pytest.param("cuda", "float32", id="gpu-f32",
                        marks=pytest.mark.gpu),
           pytest.param("cuda", "bfloat16", id="gpu-bf16",
                        marks=pytest.mark.gpu)]
TOL = {"float32": 3e-4, "bfloat16": 8e-2}
F64 = torch.float64


# ------------------------------------------------------------------ models
def latent(heads=3, dim=12, rot_dim=8, vdim=10, q_rank=20, kv_rank=24,
           window=9, base=300.0, scaling=(3.0, 40, 6.0, 1.5), scale=0.21,
           ff=44):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": {"dims": rot_dim, "base": base}}
    if window:
        m["mask"] = {"size": window}
    if scaling:
        m["rot"]["scaling"] = dict(zip(
            ("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mixer": m,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads=4, kv_heads=2, dim=12, vdim=10, conv=3, ranks=(5, 7),
          ff=None):
    return {"type": "channel_delta",
            "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "_ranks": ranks,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "conv": conv}}


def make_config(layers, width=40, vocab=70, eps=1e-5, embed_scale=3.0,
                side=12, cap=9.0, max_positions=1280):
    cfg = {"architecture": "Kaketar", "embedding": {"scale": embed_scale},
           "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
           "width": width, "max_positions": max_positions,
           "token_side": {"dim": side}}
    if cap:
        cfg["logit_softcap"] = cap
    return cfg


def make_weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def lin(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain / inp ** 0.5

    def vec(name, n, gain=0.2, mean=0.0):
        w[name] = mean + gain * torch.randn(n, generator=g)

    w["embed"] = torch.randn(cfg["vocab"], W, generator=g) / 3.0
    w["pos"] = torch.randn(cfg["max_positions"], W, generator=g)
    w["side.embed"] = torch.randn(
        cfg["vocab"], len(cfg["layers"]) * cfg["token_side"]["dim"],
        generator=g)
    for n in ("embed.norm", "final.norm"):
        vec(n, W)
    lin("head", cfg["vocab"], W, 3.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        x = p + "mix."
        vec(p + "norm1", W)
        if layer["type"] == "latent_attention":
            H, D, Dr, Dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
            lin(x + "dq", m["q_rank"], W)
            vec(x + "dq.norm", m["q_rank"], 0.2, 1.0)
            lin(x + "uq", H * (D + Dr), m["q_rank"], 2.0)
            lin(x + "dkv", m["kv_rank"] + Dr, W, 1.5)
            vec(x + "dkv.norm", m["kv_rank"], 0.2, 1.0)
            lin(x + "uk", H * D, m["kv_rank"], 2.0)
            lin(x + "uv", H * Dv, m["kv_rank"])
            vec(x + "sink", H, 1.0)
            lin(x + "g", H * Dv, W, 2.0)
            lin(x + "o", W, H * Dv)
        else:
            H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            ra, rg = layer["_ranks"]
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                lin(x + n, rows, W, 2.0)
                w[x + n + ".conv"] = torch.randn(
                    rows, m["conv"], generator=g) / m["conv"] ** 0.5
            lin(x + "b", H, W, 2.0)
            vec(x + "A_log", H, 0.7, -1.0)
            vec(x + "norm", Dv, 0.3, 1.0)
            lin(x + "a1", ra, W)
            lin(x + "a2", H * D, ra, 2.0)
            vec(x + "dt_bias", H * D, 1.0, -1.0)
            lin(x + "g1", rg, W)
            lin(x + "g2", H * Dv, rg, 2.0)
            lin(x + "o", W, H * Dv)
        if layer["mlp"]:
            vec(p + "norm2", W)
            lin(p + "mlp.up", layer["mlp"]["ff"], W, 2.0)
            lin(p + "mlp.down", W, layer["mlp"]["ff"])
        n = cfg["token_side"]["dim"]
        lin(p + "side.gate", n, W, 2.0)
        lin(p + "side.proj", W, n)
        vec(p + "side.norm", W, 0.2, 0.8)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}


def clean(cfg):
    """config.json as a checkpoint would carry it (the low ranks are the
    row counts of a1 and g1, not config keys)."""
    c = json.loads(json.dumps(cfg))
    for lay in c["layers"]:
        lay.pop("_ranks", None)
    return c


def save_model(cfg, weights):
    from safetensors.torch import save_file
    d = tempfile.mkdtemp(prefix="kaketar_test_")
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(clean(cfg), f)
    save_file(weights, os.path.join(d, "model.safetensors"))
    return d


def f64(weights):
    return {k: v.to(F64) for k, v in weights.items()}


# both mixers with and without feed-forward, grouped and ungrouped q/k
# heads, windows of different sizes, dim != vdim
STACK = [delta(), latent(),
         delta(heads=3, kv_heads=3, dim=8, vdim=16, conv=4, ranks=(3, 3),
               ff=20),
         latent(heads=2, dim=8, rot_dim=4, vdim=16, kv_rank=16, q_rank=12,
                window=17, scaling=None, ff=None)]


# ------------------------------------------------------------------ harness
def engine(model_dir, device, dtype, max_tokens=256, slots=4, page=16):
    from gllm_amd.entrypoints.trace_replay import build_engine
    return build_engine(model_dir, dtype, max_tokens, slots, device, page)


def run_steps(llm, steps, vocab):
    """steps: [{"entries": [(rid, tokens, want)], "end": [rid]}] ->
    {rid: {position: logits}} through trace_replay.replay."""
    from gllm_amd.entrypoints.trace_replay import replay
    out = tempfile.mkdtemp(prefix="kaketar_out_")
    lines, where, at = [], [], {}
    for n, st in enumerate(steps):
        ents, rows = [], []
        for rid, toks, want in st["entries"]:
            lo = at.get(rid, 0)
            ents.append({"id": rid, "tokens": toks, "want": want})
            rows += [(rid, lo + k) for k in want]
            at[rid] = lo + len(toks)
        for rid in st.get("end", []):
            at.pop(rid, None)
        lines.append(json.dumps({"step": n, "entries": ents,
                                 "end": st.get("end", [])}))
        where.append(rows)
    replay(llm, lines, out, emit=lambda t: None)
    got = {}
    for n, rows in enumerate(where):
        if not rows:
            continue
        arr = np.fromfile(os.path.join(out, "%d.f32" % n),
                          dtype="<f4").reshape(len(rows), vocab)
        for j, (rid, pos) in enumerate(rows):
            got.setdefault(rid, {})[pos] = arr[j]
    return got


def rel_err(got, want):
    d = got.astype(np.float64) - want
    d = d - d.mean()
    c = want - want.mean()
    return float(np.sqrt((d ** 2).mean()) / np.sqrt((c ** 2).mean()))


def check_against_oracle(cfg, weights, got, prompts, tol):
    """Every position within tol. bf16: one in sixteen may lie over it,
    up to four times: where a sublayer's result happens to be small, the
    norm that follows magnifies its 16-bit rounding (the reference ops in
    bf16 show the same places)."""
    refs, W = {}, f64(weights)
    for rid, rows in got.items():
        key = tuple(prompts[rid.split("#")[0]])
        if key not in refs:
            refs[key] = oracle.forward(clean(cfg), W, list(key)).numpy()
        errs = {pos: rel_err(lg, refs[key][pos]) for pos, lg in rows.items()}
        over = {p: e for p, e in errs.items() if not e < tol}
        allowed = 0 if tol < 1e-2 else max(1, len(errs) // 16)
        assert len(over) <= allowed, (rid, over)
        assert all(e < 4 * tol for e in over.values()), (rid, over)


def cut(rid, tokens, sizes, want=None):
    """One request alone, cut into portions of the given sizes; ``want``
    (positions) None = all."""
    steps, lo = [], 0
    for n in sizes:
        steps.append({"entries": [(rid, tokens[lo:lo + n], [
            k for k in range(n) if want is None or lo + k in want])]})
        lo += n
    assert lo == len(tokens)
    steps[-1]["end"] = [rid]
    return steps


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


# ------------------------------------------------------------------ tests
MECHANISMS = {
    "attention": [latent()],
    "attention-no-ff": [latent(ff=None)],
    "one-head-plain-rotary": [latent(heads=1, scaling=None, window=4)],
    "window1": [latent(window=1)],
    "no-window": [latent(window=None, dim=4, rot_dim=12)],
    "wide-window-small-value": [latent(window=300, vdim=4, heads=5)],
    "yarn-narrow-ramp": [latent(rot_dim=16, base=50.0,
                                scaling=(8.0, 64, 2.0, 1.9))],
    "yarn-lo-clamped": [latent(rot_dim=4, scaling=(2.0, 16, 30.0, 1.0))],
    "delta": [delta()],
    "delta-ff": [delta(ff=24)],
    "delta-one-head-odd": [delta(heads=1, kv_heads=1, dim=7, vdim=9,
                                 ranks=(1, 2))],
    "delta-group4-taps5": [delta(heads=8, kv_heads=2, conv=5)],
    "delta-one-tap": [delta(conv=1)],
    "delta-two-taps-dim40": [delta(conv=2, dim=40, vdim=8)],
    # head sizes of the one-token kernel (vdim 64, 128) and of every
    # register tiling of the recurrence; ranks of the MFMA latent kernel
    "delta-d64-v64": [delta(heads=2, kv_heads=1, dim=64, vdim=64)],
    "delta-d32-v128": [delta(heads=2, kv_heads=2, dim=32, vdim=128)],
    "delta-d128-v64": [delta(heads=2, kv_heads=2, dim=128, vdim=64)],
    "delta-d136-v64": [delta(heads=2, kv_heads=2, dim=136, vdim=64)],
    "delta-d256-v8": [delta(heads=1, kv_heads=1, dim=256, vdim=8)],
    "attention-r128": [latent(heads=4, dim=16, rot_dim=16, vdim=16,
                              kv_rank=128)],
    "attention-r256-h9": [latent(heads=9, dim=16, rot_dim=32, vdim=8,
                                 kv_rank=256, window=33)],
    "attention-r512": [latent(heads=2, dim=24, rot_dim=64, vdim=8,
                              kv_rank=512, window=20)],
}


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", list(MECHANISMS))
@pytest.mark.parametrize("width", [32, 36], ids=["w32", "w36"])
def test_each_mechanism_alone(name, device, dtype, width):
    """Small models around one mechanism each, every position of a whole
    prompt, then the same prompt as a portion and single tokens (other
    pages, the decode kernels). Width 36 and side 6 are not multiples
    of 8: unaligned rows everywhere."""
    cfg = make_config(MECHANISMS[name], width=width,
                      side=16 if width == 32 else 6)
    w = make_weights(cfg, 1)
    llm = engine(save_model(cfg, w), device, dtype)
    toks = tokens_for(cfg, 37, 2)
    got = run_steps(llm, cut("a", toks, [37])
                    + cut("b", toks, [30] + [1] * 7), cfg["vocab"])
    check_against_oracle(cfg, w, got, {"a": toks, "b": toks}, TOL[dtype])


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_without_cap(device, dtype):
    """No logit cap, and an embedding scale of one."""
    cfg = make_config([delta(), latent()], cap=None, embed_scale=1.0)
    w = make_weights(cfg, 5)
    llm = engine(save_model(cfg, w), device, dtype)
    toks = tokens_for(cfg, 25, 6)
    got = run_steps(llm, cut("a", toks, [20] + [1] * 5), cfg["vocab"])
    check_against_oracle(cfg, w, got, {"a": toks}, TOL[dtype])


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_layer_trail_matches(device, dtype):
    """The residual stream after every layer against the oracle's."""
    cfg = make_config(STACK)
    w = make_weights(cfg, 21)
    llm = engine(save_model(cfg, w), device, dtype)
    toks = tokens_for(cfg, 19, 22)
    trail, want = {}, []
    llm.runner.model.layer_probe = \
        lambda r, x: trail.__setitem__(r, x.detach().float().cpu().clone())
    run_steps(llm, cut("a", toks, [19]), cfg["vocab"])
    oracle.forward(clean(cfg), f64(w), toks, probe=want)
    assert len(trail) == len(want) == len(STACK)
    tol = 2e-4 if dtype == "float32" else 6e-2
    for r, b in enumerate(want):
        assert float((trail[r].double() - b).norm() / b.norm()) < tol, r


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_prefill_decode_and_portions(device, dtype):
    """Whole prompt == prompt + token-by-token decoding == portions of
    many sizes (down to two tokens and one), at every position: the
    windows (9 and 17 keys) are crossed inside portions, at their starts
    and by decoded tokens; the convolutions' history (2 and 3 rows) and
    the recurrent states are handed on, also by portions shorter than
    the history."""
    cfg = make_config(STACK, vocab=90)
    w = make_weights(cfg, 3)
    llm = engine(save_model(cfg, w), device, dtype)
    toks = tokens_for(cfg, 61, 4)
    plans = {"whole": [61], "decode": [20] + [1] * 41,
             "parts": [2, 3, 2, 7, 1, 16, 5, 2, 17, 4, 2],
             "pairs": [2] * 30 + [1],
             "ones-first": [1, 1, 1, 2, 1, 55]}
    steps = []
    for rid, sizes in plans.items():
        steps += cut(rid, toks, sizes)
    got = run_steps(llm, steps, cfg["vocab"])
    check_against_oracle(cfg, w, got, {r: toks for r in plans}, TOL[dtype])


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_mixed_batches_recycle_pages_and_slots(device, dtype):
    """Unequal requests batched together (portions beside single decode
    tokens) equal each request alone; the pool holds 10 pages and 3
    state slots, so later requests land on freed pages and on slots that
    still hold another sequence's history and state."""
    cfg = make_config(STACK, vocab=64)
    w = make_weights(cfg, 5)
    llm = engine(save_model(cfg, w), device, dtype, max_tokens=160, slots=3)
    P = {c: tokens_for(cfg, n, 10 + i)
         for i, (c, n) in enumerate([("a", 50), ("b", 9), ("c", 33),
                                     ("d", 21), ("e", 47), ("f", 3)])}
    steps = [
        {"entries": [("a", P["a"][:18], [0, 17]), ("b", P["b"][:2], [1])]},
        {"entries": [("b", P["b"][2:3], [0]), ("a", P["a"][18:33], [14]),
                     ("c", P["c"][:30], [0, 15, 16, 29])]},
        {"entries": [("c", P["c"][30:31], [0]), ("b", P["b"][3:9], [5]),
                     ("a", P["a"][33:34], [0])], "end": ["b"]},
        {"entries": [("a", P["a"][34:35], [0]), ("c", P["c"][31:33], [0, 1]),
                     ("d", P["d"][:21], [0, 15, 20])], "end": ["c", "d"]},
        {"entries": [("e", P["e"][:31], [15, 16, 30]),
                     ("a", P["a"][35:36], [0]),
                     ("f", P["f"][:3], [0, 1, 2])], "end": ["f"]},
        {"entries": [("a", P["a"][36:37], [0]), ("e", P["e"][31:32], [0])]},
        {"entries": [("a", P["a"][37:50], [12])], "end": ["a"]},
        {"entries": [("e", P["e"][32:47], list(range(15)))], "end": ["e"]},
        {"entries": [("a#2", P["a"][:50], [0, 17, 32, 49])], "end": ["a#2"]},
    ]
    pages, slots = [], {}
    alloc, ensure = llm.scheduler.mm._allocate_fresh, \
        llm.runner.ssm_pool.ensure

    def spy_pages(n):
        got = alloc(n)
        pages.extend(got)
        return got

    def spy_slot(seq):
        s = ensure(seq)
        slots.setdefault(s, set()).add(seq.seq_id)
        return s
    llm.scheduler.mm._allocate_fresh = spy_pages
    llm.runner.ssm_pool.ensure = spy_slot
    got = run_steps(llm, steps, cfg["vocab"])
    assert len(set(pages)) < len(pages), "meant to recycle pages"
    assert any(len(v) > 1 for v in slots.values()), "meant to recycle slots"
    check_against_oracle(cfg, w, got, P, TOL[dtype])


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_long_decoding(device, dtype):
    """A short prompt, then 150 tokens decoded one by one: the windows
    slide over decoded tokens only, the state is carried 150 times."""
    cfg = make_config([delta(heads=2, kv_heads=1, dim=16, vdim=64, conv=2,
                             ranks=(4, 4)),
                       latent(heads=4, dim=8, vdim=8, window=33),
                       latent(kv_rank=32, window=64, ff=None)],
                      width=24, vocab=40)
    w = make_weights(cfg, 9)
    llm = engine(save_model(cfg, w), device, dtype)
    toks = tokens_for(cfg, 156, 11)
    got = run_steps(llm, cut("a", toks, [6] + [1] * 150), cfg["vocab"])
    check_against_oracle(cfg, w, got, {"a": toks}, TOL[dtype])


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_long_prompt_and_its_continuation(device, dtype):
    """A 540-token prompt in one step, as 515 tokens + a portion of 2 +
    single tokens, and as two long portions: the ends and places around
    both cuts and the window edges."""
    cfg = make_config([latent(heads=4, dim=16, vdim=8, window=70,
                              kv_rank=64, rot_dim=16),
                       delta(heads=2, kv_heads=1, dim=64, vdim=64, conv=4),
                       latent(heads=2, kv_rank=48, window=300)],
                      width=32, vocab=50)
    w = make_weights(cfg, 17)
    llm = engine(save_model(cfg, w), device, dtype, max_tokens=1200)
    toks = tokens_for(cfg, 540, 18)
    want = {0, 1, 69, 70, 71, 299, 300, 301, 511, 512, 513, 514, 515, 516,
            517, 530, 538, 539}
    got = run_steps(llm, cut("whole", toks, [540], want)
                    + cut("tail", toks, [515, 2] + [1] * 23, want)
                    + cut("halves", toks, [513, 27], want), cfg["vocab"])
    check_against_oracle(cfg, w, got, {r: toks for r in got}, TOL[dtype])


# ------------------------------------------------------------------ latent op
LATENT_DIMS = [(3, 20, 6), (4, 24, 8), (4, 128, 64), (16, 256, 32),
               (5, 512, 64), (20, 40, 16), (7, 64, 0), (2, 520, 8)]


def _latent_call(q_lat, q_rot, rows, perm, page, npages, lens, qsl, scale,
                 window, sinks, device, tdt):
    """ops.latent_attention on per-sequence cache rows scattered over
    shuffled pages. q_lat [T, H, R], q_rot [T, H, Dr]; rows: list of
    [L, R + Dr]; returns [T, H, R] in fp32 on the CPU."""
    from gllm_amd import ops
    D = rows[0].shape[1]
    cache = torch.zeros(npages, page, 1, D)
    most = max(-(-n // page) for n in lens)
    bt = torch.zeros(len(lens), most, dtype=torch.int32)
    at = 0
    for b, n in enumerate(lens):
        k = -(-n // page)
        mine = perm[at:at + k]
        at += k
        bt[b, :k] = mine.to(torch.int32)
        j = torch.arange(n)
        cache[mine[j // page], j % page, 0] = rows[b]
    max_q = max(b - a for a, b in zip(qsl, qsl[1:]))
    o = ops.latent_attention(
        q_lat.transpose(0, 1).contiguous().to(tdt).to(device),
        q_rot.to(tdt).to(device), cache.to(tdt).to(device), bt.to(device),
        torch.tensor(lens, dtype=torch.int32, device=device),
        torch.tensor(qsl, dtype=torch.int32, device=device), scale, window,
        None if sinks is None else sinks.to(device), max_q)
    return o.transpose(0, 1).float().cpu()


@pytest.mark.parametrize("dims", LATENT_DIMS,
                         ids=["h%d-r%d-d%d" % d for d in LATENT_DIMS])
@pytest.mark.parametrize("page", [16, 64], ids=["p16", "p64"])
@pytest.mark.parametrize("device,dtype", DEVICES)
def test_latent_attention_op(device, dtype, dims, page):
    """Ragged batches (portions of several sizes beside single tokens,
    and decode-only ones) over shuffled pages, with sinks, windows below,
    at and above the kernels' 64-key tiles and none, against the
    oracle's attention with the latent as key and value."""
    H, R, Dr = dims
    tdt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(R + Dr)
    lens = [150, 1, 70, 33, 129]
    npages = 64
    perm = torch.randperm(npages, generator=g)
    rows = [torch.randn(n, R + Dr, generator=g).to(tdt).float()
            for n in lens]
    sinks = torch.randn(H, generator=g) * 2
    for new in ([40, 1, 2, 33, 1], [1] * 5):
        T = sum(new)
        qsl = [0]
        for n in new:
            qsl.append(qsl[-1] + n)
        q = (2.0 * torch.randn(T, H, R + Dr, generator=g)).to(tdt).float()
        scale = 1.5 / (R + Dr) ** 0.5
        for window in (0, 5, 63, 64, 65, 128):
            o = _latent_call(q[..., :R], q[..., R:], rows, perm, page,
                             npages, lens, qsl, scale, window, sinks,
                             device, tdt)
            for b, n in enumerate(lens):
                first = n - new[b]
                kv = rows[b].double()[:, None].expand(n, H, R + Dr)
                want = torch.stack([
                    _one_row(q[qsl[b] + i].double(), kv, first + i, scale,
                             window, sinks)
                    for i in range(new[b])])[..., :R]
                got = o[qsl[b]:qsl[b + 1]].double()
                tol = 1e-5 if dtype == "float32" else 2e-2
                err = float((got - want).norm() / want.norm())
                assert err < tol, (new, window, b, err)


def _one_row(q, kv, i, scale, window, sinks):
    """q [H, D], kv [n, H, D]: the oracle's sink softmax for query i."""
    lo = 0 if not window else max(0, i - window + 1)
    return torch.stack([
        oracle.sink_softmax((kv[lo:i + 1, h] @ q[h]) * scale, sinks[h])
        @ kv[lo:i + 1, h] for h in range(q.shape[0])])


@pytest.mark.parametrize("dims", LATENT_DIMS,
                         ids=["h%d-r%d-d%d" % d for d in LATENT_DIMS])
@pytest.mark.parametrize("device,dtype", DEVICES)
def test_planted_key_at_the_window_edges(device, dtype, dims):
    """One cached row whose score towers over all others: the query
    returns it exactly when it lies inside the window — just inside and
    just outside the edge, at page and tile borders, at the query's own
    place, far back — for a query that ends a portion and for a decoded
    token. The score sits in the rotated part when there is one."""
    H, R, Dr = dims
    tdt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(7)
    L, page, npages = 300, 16, 32
    perm = torch.randperm(npages, generator=g)
    hot = R if Dr else 1        # column that carries the score
    base = 0.05 * torch.randn(L, R + Dr, generator=g)
    for q_len in (1, 23):
        for i in (299, 271, 255, 256):
            for window, j, seen in [
                    (0, 0, True), (0, i - 200, True), (48, i, True),
                    (48, i - 47, True), (48, i - 48, False),
                    (64, i - 63, True), (64, i - 64, False),
                    (17, i - 16, True), (17, i - 17, False),
                    (1, i, True), (1, i - 1, False),
                    (250, i - 249, True), (250, i - 250, False)]:
                rows = base[:i + 1].clone()
                rows[j, hot] = 8.0
                rows[j, 0] = 100.0
                q = torch.zeros(q_len, H, R + Dr)
                q[-1, :, hot] = 8.0
                o = _latent_call(q[..., :R], q[..., R:], [rows], perm, page,
                                 npages, [i + 1], [0, q_len], 1.0, window,
                                 torch.zeros(H), device, tdt)[-1, :, 0]
                if seen:
                    assert (o - 100.0).abs().max() < 1.0, (q_len, i, window)
                else:
                    assert o.abs().max() < 1.0, (q_len, i, window, j)


@pytest.mark.parametrize("dims", [(3, 20, 6), (4, 128, 64), (16, 512, 64)],
                         ids=["r20", "r128", "r512"])
@pytest.mark.parametrize("device,dtype", DEVICES)
def test_sink_share(device, dtype, dims):
    """Zero queries: every visible key weighs the same and the sink of
    head h takes exp(sink_h) / (n + exp(sink_h)), counted once whatever
    the number of tiles and key splits; sinks far below and above."""
    H, R, Dr = dims
    tdt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(3)
    perm = torch.randperm(40, generator=g)
    sinks = torch.linspace(-3.0, 6.0, H)
    for L, new, window in ((1, 1, 0), (200, 1, 0), (200, 1, 130),
                           (130, 40, 0), (130, 40, 20)):
        rows = torch.ones(L, R + Dr)
        q = torch.zeros(new, H, R + Dr)
        o = _latent_call(q[..., :R], q[..., R:], [rows], perm, 16, 40, [L],
                         [0, new], 0.5, window, sinks, device, tdt)
        for r in range(new):
            n = L - new + r + 1
            n = min(n, window) if window else n
            want = n / (n + sinks.double().exp())
            err = (o[r].double() - want[:, None]).abs().max()
            assert err < (1e-5 if dtype == "float32" else 1e-2), (L, r)


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_latent_rope_store_op(device, dtype):
    """The latent's norm, the shared rotated key part and the query
    heads' rotated parts at positions far from zero, rows scattered over
    pages in a shuffled order; a long position keeps its angle."""
    from gllm_amd import ops
    from gllm_amd.layers.rotary import PairRotary
    tdt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(13)
    for H, D, R, Dr, scaling in ((3, 12, 24, 8, None), (2, 5, 20, 6, {
            "factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0})):
        T = 11
        rot = PairRotary(Dr, 200.0, scaling)
        ref = {"dims": Dr, "base": 200.0, "scaling": scaling}
        q = torch.randn(T, H * (D + Dr), generator=g).to(tdt)
        wide = torch.randn(T, R + Dr + 16, generator=g).to(tdt)
        w = (1 + 0.3 * torch.randn(R, generator=g)).to(tdt)
        pos = torch.arange(4000, 4000 + T)
        slot = torch.randperm(5 * 16, generator=g)[:T]
        cache = torch.zeros(5, 16, 1, R + Dr, dtype=tdt, device=device)
        qd = q.clone().to(device)
        ops.latent_rope_store(
            qd, wide.to(device)[:, 8:8 + R + Dr], w.to(device), 1e-5,
            pos.to(device), slot.to(device), rot.freqs.to(device), rot.mag,
            cache, H, D, R, Dr)
        ckv = wide[:, 8:8 + R + Dr].double()

        def turned(x):
            full = torch.zeros(4000 + T, *x.shape[1:], dtype=F64)
            full[4000:] = x
            return oracle.rotate_pairs(full, ref)[4000:]

        tol = 2e-5 if dtype == "float32" else 4e-2
        heads = q.double().view(T, H, D + Dr)
        got = qd.cpu().double().view(T, H, D + Dr)
        assert torch.equal(got[..., :D], heads[..., :D])
        assert (got[..., D:] - turned(heads[..., D:])).abs().max() < tol
        row = cache.view(-1, R + Dr)[slot.to(device)].cpu().double()
        want = oracle.over_rms(ckv[:, :R], 1e-5) * w.double()
        assert (row[:, :R] - want).abs().max() < tol
        assert (row[:, R:] - turned(ckv[:, R:])).abs().max() < tol


# ------------------------------------------------------------------ delta op
def _rows(device, slots, init, qsl):
    return (torch.tensor(slots, dtype=torch.long, device=device),
            torch.tensor(init, dtype=torch.int32, device=device),
            torch.tensor(qsl, dtype=torch.int32, device=device))


DELTA_DIMS = [(2, 1, 8, 8), (4, 2, 12, 20), (3, 3, 32, 64), (4, 1, 64, 128),
              (2, 2, 128, 64), (2, 1, 200, 64), (1, 1, 256, 10),
              (96, 3, 40, 16), (520, 520, 36, 8)]


@pytest.mark.parametrize("dims", DELTA_DIMS,
                         ids=["h%d-g%d-k%d-v%d" % d for d in DELTA_DIMS])
@pytest.mark.parametrize("device,dtype", DEVICES)
def test_channel_delta_rule_op(device, dtype, dims):
    """A long portion, short ones, decode-only batches and slots that
    held another sequence, against the oracle's recurrence on the whole
    sequences; few and many heads (both widths of the portion kernel)."""
    from gllm_amd import ops
    tdt = getattr(torch, dtype)
    H, G, D, Dv = dims
    g = torch.Generator().manual_seed(5)
    A = torch.randn(H, generator=g) * 0.5 - 1.0
    dt = torch.randn(H * D, generator=g) - 1.0
    lens = (40, 5, 12) if H < 100 else (9, 4, 5)
    widths = (G * D, G * D, H * Dv, H * D, H)
    seqs = [[torch.randn(n, c, generator=g).to(tdt) for c in widths]
            for n in lens]
    want = []
    for q, k, v, a, b in seqs:
        n = len(q)

        def unit(x):
            x = x.double().view(n, G, D)
            return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)
        dec = torch.exp(-torch.exp(A.double())[:, None] * oracle.softplus(
            a.double() + dt.double()).view(n, H, D))
        if H < 100:
            want.append(oracle.delta_recurrence(
                unit(q) * D ** -0.5, unit(k), v.double().view(n, H, Dv),
                dec, torch.sigmoid(b.double())))
        else:   # first and last head stand for all
            pick = torch.tensor([0, H - 1])
            want.append(oracle.delta_recurrence(
                unit(q)[:, pick] * D ** -0.5, unit(k)[:, pick],
                v.double().view(n, H, Dv)[:, pick], dec[:, pick],
                torch.sigmoid(b.double())[:, pick]))
    state = torch.full((4, H, D, Dv), 3.0, device=device)
    slot = [2, 0, 1]
    got = [torch.zeros(n, H, Dv) for n in lens]
    if H < 100:
        plan = [(29, 1, 0), (1, 1, 2), (2, 1, 1), (1, 1, 1), (7, 1, 8)]
    else:
        plan = [(5, 1, 2), (1, 1, 1), (3, 2, 2)]
    at = [0, 0, 0]
    for sizes in plan:
        parts, sl, init, qsl, where = [], [], [], [0], []
        for b, n in enumerate(sizes):
            if not n:
                continue
            parts.append([x[at[b]:at[b] + n] for x in seqs[b]])
            sl.append(slot[b])
            init.append(int(at[b] > 0))
            qsl.append(qsl[-1] + n)
            where.append((b, at[b], n))
            at[b] += n
        x = [torch.cat([p[i] for p in parts]) for i in range(5)]
        qkv = torch.cat(x[:3], 1).to(device)
        q, k, v = qkv.split(widths[:3], dim=-1)
        s_t, i_t, q_t = _rows(device, sl, init, qsl)
        o = ops.channel_delta_rule(
            q, k, v, x[3].to(device), x[4].to(device), A.to(device),
            dt.to(device), state, s_t, i_t, q_t, D ** -0.5,
            max(sizes)).cpu()
        for (b, lo, n), o0 in zip(where, qsl):
            got[b][lo:lo + n] = o[o0:o0 + n]
    assert at == list(lens)
    tol = 2e-4 if dtype == "float32" else 2e-3
    for a, b in zip(got, want):
        if H >= 100:
            a = a[:, [0, H - 1]]
        assert float((a.double() - b).norm() / b.norm()) < tol


@pytest.mark.parametrize("Dv", [16, 64], ids=["v16", "v64"])
@pytest.mark.parametrize("device,dtype", DEVICES)
def test_state_keeps_a_far_pair(device, dtype, Dv):
    """A pair written at position 0 with decay 1 is read back 400 tokens
    later, through a prompt portion and 40 single steps (nothing in
    between writes); a channel that decays takes its part of the key
    with it; writing zero along the same key erases it."""
    from gllm_amd import ops
    tdt = getattr(torch, dtype)
    H, D, L = 2, 16, 400
    g = torch.Generator().manual_seed(6)
    key = torch.randn(D, generator=g).to(tdt).float()
    unit = key / key.norm()

    def run(erase_at=None, dead=None):
        k = torch.zeros(L, H * D)
        k[0] = key.repeat(H)
        if erase_at is not None:
            k[erase_at] = k[0]
        v = torch.zeros(L, H * Dv)
        v[0] = 3.0
        q = torch.zeros(L, H * D)
        q[-1] = key.repeat(H)
        a = torch.full((L, H * D), -60.0)      # softplus -> 0, decay -> 1
        if dead is not None:
            a[1:, dead::D] = 60.0
        b = torch.full((L, H), 60.0)           # full write strength
        state = torch.zeros(2, H, D, Dv, device=device)
        outs, lo = [], 0
        for n in [L - 40] + [1] * 40:
            s_t, i_t, q_t = _rows(device, [1], [int(lo > 0)], [0, n])
            x = [t[lo:lo + n].to(tdt) for t in (q, k, v)]
            qkv = torch.cat(x, 1).to(device)
            outs.append(ops.channel_delta_rule(
                *qkv.split([H * D, H * D, H * Dv], dim=-1),
                a[lo:lo + n].to(tdt).to(device),
                b[lo:lo + n].to(tdt).to(device),
                torch.zeros(H, device=device),
                torch.zeros(H * D, device=device), state, s_t, i_t, q_t,
                1.0, n).cpu())
            lo += n
        return torch.cat(outs)[-1]

    tol = 1e-3 if dtype == "float32" else 2e-2
    assert (run() - 3.0).abs().max() < tol
    part = 3.0 * (1.0 - float(unit[5]) ** 2)
    assert (run(dead=5) - part).abs().max() < tol
    assert run(erase_at=200).abs().max() < tol


# ------------------------------------------------------------------ small ops
@pytest.mark.parametrize("device,dtype", DEVICES)
def test_embedding_op(device, dtype):
    """embed_rmsnorm against the oracle: scale, position rows (clamped
    for padding), weight around zero, with and without positions."""
    from gllm_amd import ops
    tdt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(2)
    for width in (32, 36, 600):
        table = torch.randn(20, width, generator=g).to(tdt)
        pos = torch.randn(9, width, generator=g).to(tdt)
        w = (0.3 * torch.randn(width, generator=g)).to(tdt)
        ids = torch.tensor([3, 19, 0, 7])
        at = torch.tensor([0, 8, 5, 40])
        for p in (pos, None):
            x, h = ops.embed_rmsnorm(
                ids.to(device), at.to(device), table.to(device),
                None if p is None else p.to(device), w.to(device), 2.5, 1.0,
                1e-5)
            r = table.double()[ids] * 2.5
            if p is not None:
                r = r + p.double()[at.clamp_max(8)]
            want = oracle.centred_norm(r, w.double(), 1e-5)
            assert x.dtype == torch.float32 and h.dtype == tdt
            assert (x.cpu().double() - want).abs().max() < 2e-5
            assert torch.equal(h.cpu(), x.cpu().to(tdt))


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_stream_norm_with_weight_offset(device, dtype):
    """x += RMS(y) (1 + w), then the stream itself in the model dtype or
    another offset norm of it; a weight of 2^-9 must not be lost in
    1 + w."""
    from gllm_amd.layers.layernorm import StreamRMSNorm
    tdt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(8)
    for width in (32, 36, 600):
        T = 5
        post, pre = (StreamRMSNorm(width, 1e-5, tdt, 1.0).to(device)
                     for _ in range(2))
        wp = torch.full((width,), 2.0 ** -9)
        wn = (0.2 * torch.randn(width, generator=g)).to(tdt)
        post.weight.data.copy_(wp)
        pre.weight.data.copy_(wn)
        x0 = torch.randn(T, width, generator=g)
        wide = torch.randn(T, width + 8, generator=g).to(tdt)
        ref = x0.double() + oracle.centred_norm(
            wide[:, :width].double(), wp.double(), 1e-5)
        for nxt in (None, pre):
            x = x0.clone().to(device)
            h = post.add_into(x, wide.to(device)[:, :width], nxt, read=True)
            assert (x.cpu().double() - ref).abs().max() < 2e-5
            want = ref if nxt is None else \
                oracle.centred_norm(ref, wn.double(), 1e-5)
            tol = 2e-5 if dtype == "float32" else 4e-2
            assert h.dtype == tdt and h.data_ptr() != x.data_ptr()
            assert (h.cpu().double() - want).abs().max() < tol


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_activation_gate_ops(device, dtype):
    """Exact gelu, the token-table gate and the head-major sigmoid gate,
    aligned and odd sizes, strided rows."""
    from gllm_amd import ops
    tdt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(9)
    tol = 1e-5 if dtype == "float32" else 4e-2
    for n in (16, 6):
        z = (3 * torch.randn(7, 2 * n + 8, generator=g)).to(tdt)
        zs = z.to(device)[:, :n]
        got = ops.gelu_erf(zs).cpu().double()
        assert (got - oracle.gelu_erf(z[:, :n].double())).abs().max() < tol
        table = torch.randn(12, 3 * n, generator=g).to(tdt)
        ids = torch.tensor([0, 11, 5, 5, 3, 7, 1])
        got = ops.token_gate(zs, table.to(device), ids.to(device),
                             2 * n).cpu().double()
        want = oracle.gelu_tanh(z[:, :n].double()) \
            * table.double()[ids, 2 * n:]
        assert (got - want).abs().max() < tol * 2
        x = torch.randn(3, 7, n, generator=g).to(tdt)
        gate = (2 * torch.randn(7, 3 * n + 8, generator=g)).to(tdt)
        for use in (True, False):
            got = ops.head_gate(x.to(device), gate.to(device)[:, :3 * n]
                                if use else None).cpu().double()
            want = x.double().transpose(0, 1).reshape(7, 3 * n)
            if use:
                want = want * torch.sigmoid(gate[:, :3 * n].double())
            assert (got - want).abs().max() < tol


# ------------------------------------------------------------------ engine
def _check_greedy(cfg, w, seq, tokens, dtype):
    """How many tokens were decided (no near-tie); those must match."""
    margin = 0.05 if dtype == "float32" else 0.5
    seq, W, decided = list(seq), f64(w), 0
    for tok in tokens:
        logits = oracle.forward(clean(cfg), W, seq)[-1]
        top2 = torch.topk(logits, 2).values
        if float(top2[0] - top2[1]) >= margin:
            assert tok == int(logits.argmax()), (len(seq), tok)
            decided += 1
        seq.append(tok)
    return decided


@pytest.mark.parametrize("graph", [False, True], ids=["eager", "graph"])
@pytest.mark.parametrize("device,dtype", DEVICES)
def test_greedy_generation_through_the_scheduler(device, dtype, graph):
    """LLM.generate (scheduler policy, chunked prefill, sampler) picks
    the oracle's greedy tokens; with ``graph`` the decode steps replay
    captured hipGraph buckets, interleaved with eager prefill steps of
    the later prompts."""
    if graph and device == "cpu":
        pytest.skip("decode graphs are captured on the GPU only")
    from gllm_amd.config import EngineConfig
    from gllm_amd.engine.llm import LLM
    from gllm_amd.sequence import SamplingParams
    cfg = make_config(STACK, vocab=48)
    w = make_weights(cfg, 14)
    config = EngineConfig(model=save_model(cfg, w), dtype=dtype,
                          device=device, page_size=16, maxp=16, maxd=8,
                          use_graph=graph, max_graph_bs=8,
                          model_max_length=256, enable_overlap=False)
    llm = LLM(config=config, num_pages_override=64)
    assert (llm.runner.graph_runner is not None) == graph
    prompts = [tokens_for(cfg, n, 20 + n) for n in (5, 37, 18)]
    outs = llm.generate(prompts, SamplingParams(
        temperature=0.0, max_tokens=12, ignore_eos=True))
    decided = sum(_check_greedy(cfg, w, p, o.token_ids, dtype)
                  for p, o in zip(prompts, outs))
    assert all(len(o.token_ids) == 12 for o in outs)
    # (bf16 needs a wide margin to call a token decided; fewer qualify)
    assert decided >= (8 if dtype == "float32" else 3)


@pytest.mark.gpu
def test_graph_replays_equal_eager_steps():
    """Captured decode buckets (sizes whose kernels are the MFMA latent
    kernel with split keys and the one-token recurrence) replayed many
    times, with eager prefills in between, generate what eager steps
    generate."""
    from gllm_amd.config import EngineConfig
    from gllm_amd.engine.llm import LLM
    from gllm_amd.sequence import SamplingParams
    cfg = make_config([latent(heads=4, dim=16, rot_dim=16, vdim=16,
                              kv_rank=64, window=150),
                       delta(heads=2, kv_heads=1, dim=64, vdim=64)],
                      width=64, vocab=48)
    d = save_model(cfg, make_weights(cfg, 24))
    prompts = [tokens_for(cfg, n, 40 + n) for n in (200, 7, 65, 30)]
    runs = []
    for graph in (False, True):
        llm = LLM(config=EngineConfig(
            model=d, dtype="bfloat16", device="cuda", page_size=16,
            maxp=64, maxd=8, use_graph=graph, max_graph_bs=8,
            model_max_length=512, enable_overlap=False,
            enable_prefix_caching=False), num_pages_override=80)
        assert (llm.runner.graph_runner is not None) == graph
        outs = []
        for _ in range(2):   # the second round on used pages and slots
            outs += [o.token_ids for o in llm.generate(
                prompts, SamplingParams(temperature=0.0, max_tokens=24,
                                        ignore_eos=True))]
        assert outs[:4] == outs[4:]
        runs.append(outs)
    assert runs[0] == runs[1]


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_prefix_cache_hit_restores_state(device, dtype):
    """A second prompt that shares two full pages with an earlier one
    re-uses the cached latent pages and the snapshot of convolution
    history and recurrent state taken at that page boundary."""
    from gllm_amd.config import EngineConfig
    from gllm_amd.engine.llm import LLM
    from gllm_amd.sequence import SamplingParams
    cfg = make_config(STACK, vocab=48)
    w = make_weights(cfg, 23)
    config = EngineConfig(model=save_model(cfg, w), dtype=dtype,
                          device=device, page_size=16, maxp=16, maxd=8,
                          use_graph=False, enable_overlap=False,
                          enable_prefix_caching=True)
    llm = LLM(config=config, num_pages_override=64)
    first = tokens_for(cfg, 48, 31)
    second = first[:32] + tokens_for(cfg, 9, 32)
    sp = SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True)
    llm.generate([first], sp)
    before = llm.runner.memory_manager.hit_tokens
    out = llm.generate([second], sp)[0]
    assert llm.runner.memory_manager.hit_tokens - before == 32
    assert _check_greedy(cfg, w, second, out.token_ids, dtype) \
        >= (3 if dtype == "float32" else 1)


def test_positions_end_where_the_table_ends():
    """The position table bounds the context: generation stops when it
    is full, the last position works, nothing past it is admitted."""
    from gllm_amd.config import EngineConfig
    from gllm_amd.engine.llm import LLM
    from gllm_amd.sequence import SamplingParams
    cfg = make_config([latent(), delta()], max_positions=40)
    w = make_weights(cfg, 4)
    d = save_model(cfg, w)
    llm = LLM(config=EngineConfig(model=d, dtype="float32", device="cpu",
                                  page_size=16), num_pages_override=16)
    assert llm.config.model_max_length == 40
    sp = SamplingParams(temperature=0.0, max_tokens=500, ignore_eos=True)
    out = llm.generate([tokens_for(cfg, 35, 1)], sp)[0]
    assert len(out.token_ids) == 5 and out.finish_reason == "length"
    assert sp.max_tokens == 500     # the caller's parameters stay
    assert len(llm.generate([tokens_for(cfg, 40, 1)], sp)[0].token_ids) == 1
    with pytest.raises(ValueError):
        llm.generate([tokens_for(cfg, 41, 1)], sp)
    llm = engine(d, "cpu", "float32")
    toks = tokens_for(cfg, 41, 3)
    got = run_steps(llm, cut("a", toks[:40], [38, 1, 1]), cfg["vocab"])
    check_against_oracle(cfg, w, got, {"a": toks[:40]}, TOL["float32"])
    with pytest.raises(ValueError):
        run_steps(llm, cut("b", toks, [40, 1]), cfg["vocab"])


def test_config_and_registry():
    """The loader picks the class from config.json's architecture key;
    attention layers own one cached row per token, delta layers a state
    entry; the low ranks come with a1 and g1 whatever the order of the
    tensors; unknown tensors and a missing a1 raise."""
    from gllm_amd.config import EngineConfig
    from gllm_amd.models.loader import load_model
    cfg = make_config(STACK, vocab=48)
    wts = make_weights(cfg, 15)

    def load(weights, c=cfg):
        return load_model(EngineConfig(model=save_model(c, weights),
                                       dtype="float32", device="cpu"))[0]
    model = load(wts)
    assert type(model).__name__ == "KaketarForCausalLM"
    assert model.kv_layer_shapes == [(1, 32, 0), (1, 20, 0)]
    assert [(s.conv_dim, s.conv_kernel, s.num_v_heads, s.head_k_dim,
             s.head_v_dim) for s in model.ssm_spec.layers] == \
        [(88, 3, 4, 12, 10), (96, 4, 3, 8, 16)]
    assert [model.layers[i].mix.ranks for i in (0, 2)] == [(5, 7), (3, 3)]
    late = {k: v for k, v in wts.items() if not k.endswith("a1")}
    late.update({k: v for k, v in wts.items() if k.endswith("a1")})
    from gllm_amd.models.loader import create_model, load_hf_config
    ec = EngineConfig(model=save_model(cfg, wts), dtype="float32",
                      device="cpu")
    other = create_model(load_hf_config(ec.model), ec)
    other.load_weights(late.items())
    for (n, a), (_, b) in zip(sorted(model.named_parameters()),
                              sorted(other.named_parameters())):
        assert torch.equal(a, b), n
    with pytest.raises(KeyError):
        load(dict(wts, **{"l0.mix.sink": torch.zeros(
            4, dtype=torch.bfloat16)}))
    with pytest.raises(KeyError):
        load({k: v for k, v in wts.items() if k != "l2.mix.a1"})
    bad = make_config([dict(latent(), type="attention")])
    with pytest.raises(ValueError):
        load({}, bad)


def test_yarn_table():
    """PairRotary's YaRN frequencies against the oracle's, with the ramp
    cut at both ends, inverted to a step, and a factor of one."""
    from gllm_amd.layers.rotary import PairRotary
    for dims, base, sc in ((16, 300.0, (3.0, 40, 6.0, 1.5)),
                           (4, 50.0, (2.0, 16, 30.0, 1.0)),
                           (32, 1e4, (8.0, 4096, 32.0, 1.0)),
                           (16, 100.0, (5.0, 64, 2.0, 1.99)),
                           (8, 100.0, (1.0, 64, 8.0, 1.0)), (8, 70.0, None)):
        s = dict(zip(("factor", "original", "fast", "slow"), sc)) \
            if sc else None
        f, mag = oracle.yarn({"dims": dims, "base": base, "scaling": s})
        r = PairRotary(dims, base, s)
        assert torch.allclose(r.freqs, f, rtol=1e-13, atol=0)
        assert abs(r.mag - mag) < 1e-14
