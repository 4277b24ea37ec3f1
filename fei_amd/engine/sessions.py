"""Paged multi-session serving: continuous batching over a PagedKVPool.

The reference serves one remote conversation per Assistant; this engine
serves MANY resident agent sessions on one GPU: each session's KV lives in
16-token blocks of a shared pool (`engine/kv_cache.py`), sessions join and
leave the decode batch at any step, and the attention read path is the HIP
block-table kernel (`k_attn_decode_paged`). Admission is explicit — a
session that cannot get blocks raises and the caller can evict.

Control-plane costs stay host-side (per-step RoPE/append scatter is a few
microseconds of torch indexing per layer); the O(context) work — attention
over the pool — is the paged HIP kernel, and all GEMVs take the same
streaming kernels as the single-session path. Greedy decode (serving
agents at temperature 0); graphs are off (batch membership changes).

Models of unlike layers (``model.step_cache``) get ``StepSessionManager``, a
subclass with the same surface whose steps are ragged batches: portions of
prompts run beside the decoding sessions' tokens, so a long prompt does not
stall the others.
"""

from __future__ import annotations

import logging
import math
import os as _os
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Union

logger = logging.getLogger(__name__)

import torch
import torch.nn.functional as F

from fei_amd import ops
from fei_amd.engine.kv_cache import PagedKVPool
from fei_amd.engine.step import StepEntry, StepRunner
from fei_amd.ops import reference as ref


@dataclass
class Session:
    sid: int
    prompt_ids: List[int]
    generated: List[int] = field(default_factory=list)
    pos: int = 0                     # current context length in the pool
    max_new_tokens: int = 256
    done: bool = False


class PagedSessionManager:
    def __new__(cls, engine, *args, **kwargs):
        step = getattr(engine.model, "step_cache", False)
        return object.__new__(StepSessionManager if step else cls)

    def __init__(self, engine, block_size: int = 16,
                 num_blocks: Optional[int] = None,
                 mem_fraction: float = 0.25):
        self.engine = engine
        self.model = engine.model
        m = self.model
        assert m.tp_size == 1, "paged session serving is single-GPU"

        self.pool = PagedKVPool(
            num_layers=m.spec.num_layers, num_kv_heads=m.hkv_l,
            head_dim=m.D, block_size=block_size, num_blocks=num_blocks,
            device=m.device, dtype=m.dtype, mem_fraction=mem_fraction)
        self.sessions: Dict[int, Session] = {}
        self.eos = engine.tokenizer.eos_id
        self._ws: Dict[int, tuple] = {}     # split-K workspace per batch size
        # hipGraph per (B, table_width): one captured decode step (forward
        # + argmax feedback + pos advance) over static buffers. Measured
        # NEUTRAL (836 vs 869 tok/s eager at 8 sessions): the eager chunk
        # loop already queues launches ahead of the GPU, so the step is
        # GPU-time-bound, not host-bound. Opt-in via FEI_SESS_GRAPH=1.
        self._graphs: Dict[tuple, dict] = {}
        self.use_graph = m.device.type == "cuda" and \
            _os.environ.get("FEI_SESS_GRAPH", "0") == "1"

    def _splits(self, B: int) -> int:
        # batch-aware split count (engine ctor note): the B-wide grid
        # already fills the chip at 16 splits once B >= 4 — 32 over-splits
        # (batch-8 plain path measured 6.34 -> 5.85 ms/step at 16)
        return min(self.engine.attn_splits, 16) if B >= 4 \
            else self.engine.attn_splits

    def _workspace(self, B: int):
        if B not in self._ws:
            m = self.model
            sp = self._splits(B)
            self._ws[B] = (
                torch.zeros(B, m.hq_l, sp, m.D, dtype=torch.float32,
                            device=m.device),
                torch.zeros(B, m.hq_l, sp, 2, dtype=torch.float32,
                            device=m.device))
        return self._ws[B]

    def _chunk_graph(self, B: int, max_blocks: int, token, pos, table):
        """Capture (or fetch) the hipGraph of ONE decode step for batch B
        and a table of width >= max_blocks: forward + in-place argmax
        token feedback + pos advance over static buffers. Warm-up runs 2
        real steps whose KV rows are garbage; they are rewritten by the
        first replays before anything attends them (the per-layer append
        at `pos` precedes the attention read of key `pos`, and rows past
        the accepted stream are never attended)."""
        W = 16
        while W < max_blocks:
            W *= 2
        key = (B, W)
        ent = self._graphs.get(key)
        if ent is not None:
            return ent
        dev = self.model.device
        bt = torch.zeros(B, W, dtype=torch.int32, device=dev)
        tk = torch.zeros(B, dtype=torch.int64, device=dev)
        ps = torch.zeros(B, dtype=torch.int32, device=dev)
        bt[:, :max_blocks].copy_(table)
        tk.copy_(token)
        ps.copy_(pos)
        try:
            side = torch.cuda.Stream()
            side.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(side):
                for _ in range(2):
                    lg = self._forward_paged(tk, ps, bt)
                    tk.copy_(lg.argmax(dim=-1))
                    ps.add_(1)
            torch.cuda.current_stream().wait_stream(side)
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                lg = self._forward_paged(tk, ps, bt)
                tk.copy_(lg.argmax(dim=-1))
                ps.add_(1)
            torch.cuda.synchronize()
        except Exception as e:                      # pragma: no cover - GPU
            logger.warning("sessions graph capture failed (%s); "
                           "falling back to eager chunks", e)
            self.use_graph = False
            return None
        ent = {"graph": g, "token": tk, "pos": ps, "table": bt}
        self._graphs[key] = ent
        logger.info("sessions decode step captured (B=%d, W=%d)", B, W)
        return ent

    # -- admission -----------------------------------------------------------

    def open(self, prompt: Union[str, List[int]],
             max_new_tokens: int = 256) -> int:
        """Prefill a new session into the pool; returns its id. Raises
        MemoryError when the pool has no blocks (caller evicts/queues)."""
        ids = (self.engine.tokenizer.encode(prompt)
               if isinstance(prompt, str) else list(prompt))
        m, dev = self.model, self.model.device
        S = len(ids)
        sid = self.pool.new_sequence()
        try:
            self.pool.ensure_capacity(sid, S + 1)
        except MemoryError:
            self.pool.release(sid)
            raise
        # prefill through the normal MFMA path into a contiguous scratch,
        # then scatter each layer's S rows into this session's blocks
        k_tmp = [torch.zeros(1, m.hkv_l, S, m.D, device=dev, dtype=m.dtype)
                 for _ in range(m.spec.num_layers)]
        v_tmp = [torch.zeros_like(k_tmp[0]) for _ in range(m.spec.num_layers)]
        tokens = torch.tensor([ids], dtype=torch.int64, device=dev)
        pos0 = torch.zeros(1, dtype=torch.int32, device=dev)
        logits = m.forward_prefill(tokens, pos0, k_tmp, v_tmp)
        BS = self.pool.block_size
        blocks = self.pool.table(sid).blocks
        for li in range(m.spec.num_layers):
            for j in range(0, S, BS):
                blk = blocks[j // BS]
                n = min(BS, S - j)
                self.pool.k[li][blk, :, :n, :] = k_tmp[li][0, :, j:j + n, :]
                self.pool.v[li][blk, :, :n, :] = v_tmp[li][0, :, j:j + n, :]
        first = int(logits[0].argmax())
        sess = Session(sid=sid, prompt_ids=ids, generated=[first], pos=S,
                       max_new_tokens=max_new_tokens)
        if first == self.eos:
            sess.done = True
        self.sessions[sid] = sess
        return sid

    def close(self, sid: int) -> None:
        self.pool.release(sid)
        self.sessions.pop(sid, None)

    # -- decode --------------------------------------------------------------

    @property
    def active(self) -> List[Session]:
        return [s for s in self.sessions.values() if not s.done]

    def step(self) -> int:
        """One greedy decode step for every active session. Returns the
        number of sessions that advanced."""
        return self.step_chunk(1)

    def step_chunk(self, chunk: int = 8) -> int:
        """Up to ``chunk`` greedy decode steps for the CURRENT active set
        with device-resident token feedback — ONE host sync (the chunk's
        token download) instead of one per step; block capacity for the
        whole chunk is reserved up front and the table tensor is built
        once. Admission/retirement happens between chunks. A session that
        hits EOS mid-chunk keeps decoding garbage rows into its reserved
        blocks until the chunk ends (its `generated`/`pos` stop at the
        EOS, so the extra rows are never attended and the blocks are
        freed on close). Returns sessions advanced (0 = none active)."""
        act = self.active
        if not act:
            return 0
        m, dev = self.model, self.model.device
        # +3 headroom: graph capture warm-up runs 2 extra steps (their
        # garbage KV rows are rewritten by real replays before any
        # attention reads them — append-at-pos precedes the read of pos)
        reserve = max(chunk, 3) if self.use_graph else chunk
        for s in act:
            self.pool.ensure_capacity(s.sid, s.pos + reserve)
        max_blocks = max(len(self.pool.table(s.sid).blocks) for s in act)
        table = torch.full((len(act), max_blocks), -1, dtype=torch.int32)
        for i, s in enumerate(act):
            blocks = self.pool.table(s.sid).blocks
            table[i, :len(blocks)] = torch.tensor(blocks, dtype=torch.int32)
        table = table.to(dev)
        token = torch.tensor([s.generated[-1] for s in act],
                             dtype=torch.int64, device=dev)
        pos = torch.tensor([s.pos for s in act], dtype=torch.int32, device=dev)
        g = self._chunk_graph(len(act), max_blocks, token, pos, table) \
            if self.use_graph else None
        if g is not None:
            g["token"].copy_(token)
            g["pos"].copy_(pos)
            g["table"].zero_()
            g["table"][:, :max_blocks].copy_(table)
            outs = torch.empty(len(act), chunk, dtype=torch.int64,
                               device=dev)
            for j in range(chunk):
                g["graph"].replay()
                outs[:, j].copy_(g["token"])
            allt = outs.tolist()                           # the one sync
        else:
            steps = []
            for _ in range(chunk):
                logits = self._forward_paged(token, pos, table)
                token = logits.argmax(dim=-1)
                steps.append(token)
                pos = pos + 1
            allt = torch.stack(steps, dim=1).tolist()      # the one sync
        for i, s in enumerate(act):
            for t in allt[i]:
                s.generated.append(int(t))
                s.pos += 1
                if int(t) == self.eos or \
                        len(s.generated) >= s.max_new_tokens:
                    s.done = True
                    break
        return len(act)

    def run(self, max_steps: int = 4096, chunk: int = 8) -> None:
        done = 0
        while done < max_steps:
            k = min(chunk, max_steps - done)
            if self.step_chunk(k) == 0:
                break
            done += k

    def result(self, sid: int) -> Dict[str, object]:
        s = self.sessions[sid]
        gen = s.generated
        if self.eos in gen:
            gen = gen[: gen.index(self.eos) + 1]
        return {"token_ids": gen,
                "text": self.engine.tokenizer.decode(gen),
                "done": s.done}

    # -- model forward over the pool ------------------------------------------

    def _forward_paged(self, token: torch.Tensor, pos: torch.Tensor,
                       table: torch.Tensor) -> torch.Tensor:
        """Plain decode forward with block-table attention. Same GEMV /
        norm kernels as LlamaModel.forward_decode (llama.py); RoPE + the
        single-row KV append are torch-side (control plane — O(Hkv*D) per
        session, independent of context length) and fully device-resident:
        the block/offset of the appended row derive from `pos` and `table`
        with gather/advanced indexing, so a whole step chain runs without
        a host sync (step_chunk)."""
        m = self.model
        s = m.spec
        B = token.shape[0]
        BS = self.pool.block_size
        h = F.embedding(token.long(), m.emb)
        scale = 1.0 / math.sqrt(m.D)
        n_layers = len(m.layers)
        x = ops.rmsnorm(h, m.layers[0].norm_attn, s.norm_eps)
        pos_l = pos.long()
        gpu = m.device.type == "cuda"
        if not gpu:
            blk = table.gather(1, (pos_l // BS).unsqueeze(1)) \
                .squeeze(1).long()
            off = pos_l % BS
        for li, lw in enumerate(m.layers):
            qkv = ops.linear_decode(x, lw.wqkv)
            q, k, v = m._qkv_views(qkv, B)
            kp, vp = self.pool.k[li], self.pool.v[li]
            if gpu:
                # fused in-kernel RoPE + paged append (the eager torch
                # rope/append chain was ~15 launches/layer — ~30% of the
                # serving step)
                att = ops.attn_decode_paged(q, kp, vp, table, pos,
                                            splits=self._splits(B),
                                            scale=scale,
                                            workspace=self._workspace(B),
                                            k=k, v=v, table=m.rope)
            else:
                q_r = ref.apply_rope(q, pos_l, m.rope).contiguous()
                k_r = ref.apply_rope(k, pos_l, m.rope)
                kp[blk, :, off, :] = k_r
                vp[blk, :, off, :] = v
                att = ops.attn_decode_paged(q_r, kp, vp, table, pos,
                                            splits=self._splits(B),
                                            scale=scale,
                                            workspace=self._workspace(B))
            o = ops.linear_decode(att.reshape(B, -1), lw.wo)
            x, h = ops.fused_add_rmsnorm(o, h, lw.norm_mlp, s.norm_eps)
            act = ops.gemv_swiglu(x, lw.wgu)
            d = ops.linear_decode(act, lw.wdown)
            next_norm = (m.layers[li + 1].norm_attn if li + 1 < n_layers
                         else m.norm_f)
            x, h = ops.fused_add_rmsnorm(d, h, next_norm, s.norm_eps)
        return ops.linear_decode(x, m.lm_head)


class StepSessionManager(PagedSessionManager):
    """Sessions over a StepRunner: one cache of rows and state slots,
    one ragged batch per step.

    ``open`` admits a session (a state slot, and blocks for its prompt) and
    queues its prompt. While any prompt is queued, a step takes the next token
    of every decoding session and up to ``prefill_budget`` prompt tokens, in
    order of admission; otherwise decoding runs in device-resident chunks.
    """

    def __init__(self, engine, block_size: int = 64,
                 num_blocks: Optional[int] = None,
                 mem_fraction: float = 0.25, max_sessions: int = 64,
                 prefill_budget: int = 2048):
        self.engine = engine
        self.model = m = engine.model
        if num_blocks is None:
            if m.device.type == "cuda":
                budget = int(torch.cuda.mem_get_info(m.device)[0] *
                             mem_fraction)
            else:
                budget = 1 << 26
            num_blocks = max(16, budget // max(
                1, m.cache_bytes_per_token() * block_size))
            # no more than all sessions at full length can use
            num_blocks = min(num_blocks, max_sessions *
                             -(-m.max_seq_len // block_size))
        self.runner = StepRunner(m, num_blocks, max_sessions, block_size)
        self.pool = self.runner.cache
        self.prefill_budget = prefill_budget
        self.sessions: Dict[int, Session] = {}
        self.eos = engine.tokenizer.eos_id

    # -- admission -----------------------------------------------------------

    def open(self, prompt: Union[str, List[int]],
             max_new_tokens: int = 256) -> int:
        """Queue a session; MemoryError when no slot or blocks are free."""
        ids = (self.engine.tokenizer.encode(prompt)
               if isinstance(prompt, str) else list(prompt))
        if not ids:
            raise ValueError("empty prompt")
        if len(ids) + 1 > self.model.max_seq_len:
            raise ValueError(f"prompt of {len(ids)} tokens does not fit "
                             f"{self.model.max_seq_len}")
        sid = self.runner.admit(len(ids) + 1)
        self.sessions[sid] = Session(sid=sid, prompt_ids=ids,
                                     max_new_tokens=max_new_tokens)
        return sid

    def close(self, sid: int) -> None:
        if self.sessions.pop(sid, None) is not None:
            self.runner.release(sid)

    # -- steps ---------------------------------------------------------------

    def _emit(self, s: Session, token: int) -> None:
        s.generated.append(token)
        if token == self.eos or len(s.generated) >= s.max_new_tokens:
            s.done = True

    def _mixed_step(self, act: List[Session]) -> int:
        """One ragged batch; sessions that took part."""
        entries: List[StepEntry] = []
        emits: List[Session] = []
        budget = self.prefill_budget
        for s in act:
            n = len(s.prompt_ids)
            if s.pos >= n:
                entries.append(StepEntry(s.sid, [s.generated[-1]], [0]))
                emits.append(s)
            elif budget > 0:
                part = s.prompt_ids[s.pos:s.pos + budget]
                budget -= len(part)
                last = s.pos + len(part) == n
                entries.append(StepEntry(s.sid, part,
                                         [len(part) - 1] if last else []))
                if last:
                    emits.append(s)
        logits = self.runner.step(entries)
        for e in entries:
            self.sessions[e.seq].pos += len(e.tokens)
        if emits:
            for s, t in zip(emits, logits.argmax(dim=-1).tolist()):
                self._emit(s, int(t))
        return len(entries)

    @torch.no_grad()
    def step_chunk(self, chunk: int = 8) -> int:
        """Up to ``chunk`` steps. Returns sessions advanced (0 = none)."""
        advanced = 0
        left = chunk
        while left > 0:
            for s in self.active:
                if s.pos >= self.model.max_seq_len:
                    s.done = True            # no room for another token
            act = self.active
            if not act:
                break
            if any(s.pos < len(s.prompt_ids) for s in act):
                advanced = max(advanced, self._mixed_step(act))
                left -= 1
                continue
            advanced = max(advanced, len(act))
            left -= self._decode_chunk(act, left)
        return advanced

    def _decode_chunk(self, act: List[Session], chunk: int) -> int:
        """Decode steps with token feedback on the device and one download. A
        session that ends inside the chunk runs on to its end: its blocks and
        slot are its own and go back when it is closed."""
        n = min(chunk, min(self.model.max_seq_len - s.pos for s in act),
                max(s.max_new_tokens - len(s.generated) for s in act))
        batch = self.runner.decode_batch([s.sid for s in act], n,
                                         [s.generated[-1] for s in act])
        steps = []
        for _ in range(n):
            logits = self.model.forward(batch, self.runner.cache)
            batch.tokens = logits.argmax(dim=-1)
            batch.pos += 1
            steps.append(batch.tokens)
        rows = torch.stack(steps, dim=1).tolist()
        for s, row in zip(act, rows):
            self.runner.set_length(s.sid, s.pos + n)
            for t in row:
                if s.done:
                    break
                s.pos += 1
                self._emit(s, int(t))
        return n
