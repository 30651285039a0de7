"""What the tests of a whole design share: the comparison of logits, the replay of a trace through the framework's own
replayer with an eye on which pages and slots are handed out again, and hand-made batches and paged caches for one
mechanism alone."""

from __future__ import annotations

import random

import torch

DEV = "cuda"


def close(ours, ref, dtype, what, loose=None, caps=(0.15, 0.08)):
    """32-bit: 1e-4 of the row's largest logit.  bfloat16: the root mean square of the difference (means taken off) against
    the root mean square of the row's logits about their mean: at most 15% in a row and, of eight rows or more, 8% in the
    median row (the 32-bit runs are the sharp test; a design that rounds a sublayer's output to bfloat16 and then norms it,
    in every sublayer of every pass, is left a few per cent by rounding alone).  A row between 15% and 100% is counted in
    ``loose`` (a list) if one is given: in bfloat16 a token whose router scores lie within rounding of each other may take
    another expert than the plain implementation, and whoever collects the rows says how few of them may."""
    ours = ours.float().cpu()
    assert ours.shape == ref.shape, (what, ours.shape, ref.shape)
    assert torch.isfinite(ours).all(), what
    if dtype == torch.float32:
        err = ((ours - ref).abs().amax(-1) / ref.abs().amax(-1)).max().item()
        assert err <= 1e-4, f"{what}: {err:.2e} of the row's largest logit"
    else:
        d = ours - ref
        d = d - d.mean(-1, keepdim=True)
        spread = (ref - ref.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()
        err = d.pow(2).mean(-1).sqrt() / spread
        if loose is not None:
            loose.extend([what] * int(((err > caps[0]) & (err <= 1.0)).sum()))
            err = err[(err <= caps[0]) | (err > 1.0)]
            if not len(err):
                return
        assert err.max() <= caps[0] and (len(err) < 8 or err.median() <= caps[1]), f"{what}: {err.max():.3f} of the logits' spread (median {err.median():.3f})"


def replay(model, steps, where, ref, dtype, max_tokens, page, graphs=True, loose_share=10, caps=(0.15, 0.08)):
    from nanospec_amd.engine.replay import Replayer

    rep = Replayer(model, max_tokens, page_size=page, use_graphs=graphs)
    holders, slots = {}, {}
    real_reserve = rep.manager.reserve

    def reserve(req_id, n):
        rc = real_reserve(req_id, n)
        slots.setdefault(rc.slot, set()).add(req_id)
        for g, table in enumerate(rc.tables):
            for p in table:
                if p >= 0:
                    holders.setdefault((g, p), set()).add(req_id)
        return rc

    rep.manager.reserve = reserve
    rep.graph_steps = 0
    loose, rows = [], 0
    for step, w in zip(steps, where):
        out = rep.step(step["entries"], step["end"])
        rep.graph_steps += bool(rep.runner.last_used_graph)
        if w:
            rows += len(w)
            close(out, torch.stack([ref[rid][p] for rid, p in w]), dtype, f"step {step['step']} {[(e['id'], len(e['tokens'])) for e in step['entries']]}", loose, caps)
    # (a model here asks its routers four to eight times a token, each time with a chance of a few per cent that bfloat16 rounding
    # moves a close call; such a row then differs by more than rounding)
    assert len(loose) <= max(2, rows // loose_share), f"{len(loose)} of {rows} rows are off by more than rounding: {loose[:5]}"
    rep.manager.check()
    rep.pages_again = sum(1 for who in holders.values() if len(who) > 1)
    rep.slots_again = sum(1 for who in slots.values() if len({r for r in who if r != "__pad__"}) > 1)
    return rep


def batch(lens, slots):
    """Device arrays of a step's batch for hand-made requests: (token_req, qo_indptr, state_slots)."""
    req = torch.tensor([b for b, n in enumerate(lens) for _ in range(n)], dtype=torch.int32, device=DEV)
    indptr = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), dtype=torch.int32, device=DEV)
    return req, indptr, torch.tensor(slots, dtype=torch.int32, device=DEV)


def paged(keys, values, page, order_seed=0):
    """One request's keys [T, G, hd] and values [T, G, vd] in pages handed out in a scrambled order -> (k pages, v pages, table)."""
    T, G, hd = keys.shape
    vd = values.shape[2]
    n_pages = -(-T // page)
    ids = list(range(1, n_pages + 3))
    random.Random(order_seed).shuffle(ids)
    ids = ids[:n_pages]
    k = torch.zeros(n_pages + 4, G, page, hd, dtype=keys.dtype)
    v = torch.zeros(n_pages + 4, G, vd, page, dtype=keys.dtype)
    for t in range(T):
        k[ids[t // page], :, t % page] = keys[t]
        v[ids[t // page], :, :, t % page] = values[t]
    return k.to(DEV), v.to(DEV), torch.tensor([ids], dtype=torch.int32, device=DEV)


def step_context(lens, starts, tables):
    """The framework's own batch builder for hand-made requests: tables[b] lists the pages of request b."""
    import numpy as np

    from nanospec_amd.engine.arena import Arena
    from nanospec_amd.engine.context import BatchLayout, StepContext, fill_batch
    from nanospec_amd.parts.attention import TILES

    width = max(len(t) for t in tables)
    layout = BatchLayout(sum(lens), len(lens), 0, 1, width, plans=[(TILES, TILES.shape(lens))])
    host = np.zeros(layout.total, dtype=np.int32)
    table = np.full((len(lens), width), -1, dtype=np.int32)
    for b, t in enumerate(tables):
        table[b, : len(t)] = t
    fill_batch(host, layout, [0] * sum(lens), starts, lens, list(range(len(lens))), [], [table])
    max_kv = max(s + n for s, n in zip(starts, lens))
    chunk_kv = max((s + n for s, n in zip(starts, lens) if n != 1), default=0)
    return StepContext(layout, torch.from_numpy(host).to(DEV), Arena(DEV), max_position=max_kv - 1, max_kv_len=max_kv, max_chunk_kv=chunk_kv)


class PartCtx:
    """The little that a part asks of a step's context when it is run alone."""

    captured = False

    def __init__(self):
        from nanospec_amd.engine.arena import Arena

        self.arena, self.plans = Arena(torch.device(DEV)), {}

    def requests(self, lens, slots, positions, plan=None, spare=0):
        """A batch of hand-made requests; ``plan``: a batch plan that describes it, in a region of ``spare`` more entries than it needs."""
        import types

        import numpy as np

        self.token_req, self.qo_indptr, self.state_slots = batch(lens, slots)
        self.positions = torch.tensor(positions, dtype=torch.int32, device=DEV)
        self.max_position = max(positions)
        self.plans = {}
        if plan is not None:
            shape = plan.shape(lens)
            shape = (shape[0] + spare, *shape[1:])
            out = np.full(max(1, plan.ints(shape)), -1, dtype=np.int32)
            plan.fill(out, shape, types.SimpleNamespace(covered=len(lens), lens=np.array(lens), indptr=np.concatenate([[0], np.cumsum(lens)])))
            self.plans = {plan.key: (torch.from_numpy(out).to(DEV), shape)}


def off(got, want):
    """The largest difference over the largest value, and the root mean square of the difference over that of the values."""
    d = got.cpu().double() - want
    return float(d.abs().max() / want.abs().max()), float(d.pow(2).mean().sqrt() / want.pow(2).mean().sqrt())
