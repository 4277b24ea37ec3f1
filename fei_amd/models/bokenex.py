"""Bokenex: a decoder of parallel layers, sigmoid attention beside a dense
feed-forward or a mixture of experts.

Both sublayers of a layer read one norm of a float32 residual, which gets
their sum times a constant: one stacked product makes everything the layer
reads (projections, router logits, the dense activations), one product over
the concatenated outputs adds to the residual. The norms have a single gain,
so a norm commutes with a product and the decode kernels make it inside.
Positions enter as learned vectors added to the embedding.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Callable, Dict, List, Optional

import torch

from fei_amd import ops
from fei_amd.engine.kv_cache import HybridCache
from fei_amd.models.feedforward import FEED_FORWARDS, FeedForward
from fei_amd.models.mixers import MIXERS, Mixer
from fei_amd.models.step_model import StepModel


@dataclass
class BokenexLayer:
    norm: "ops.GainNorm"
    w_in: torch.Tensor         # [mixer rows + (router or ff) rows, C]
    w_out: torch.Tensor        # [C, mixer cols + dense ff]
    mixer: Mixer
    mlp: Optional[FeedForward]


class BokenexModel(StepModel):

    def mixers(self) -> List[Mixer]:
        return [L.mixer for L in self.layers]

    # -- weights -------------------------------------------------------------

    def _shapes(self) -> Dict[str, tuple]:
        s, C = self.spec, self.spec.hidden_size
        out = {"embed": (s.vocab_size, C), "pos": (s.max_seq_len, C),
               "final.norm": (), "head": (s.vocab_size, C)}
        for i, L in enumerate(s.layers):
            out[f"l{i}.norm1"] = ()
            for name, shape in MIXERS[L.mixer.kind].shapes(L.mixer, C).items():
                out[f"l{i}.mix.{name}"] = shape
            if L.mlp is not None:
                cls = FEED_FORWARDS[L.mlp.kind]
                for name, shape in cls.shapes(L.mlp, C).items():
                    out[f"l{i}.mlp.{name}"] = shape
        return out

    def _random(self, seed: int) -> Callable[[str], torch.Tensor]:
        shapes = self._shapes()
        gen = torch.Generator(device=self.device)
        gen.manual_seed(seed)
        depth = math.sqrt(2 * len(self.spec.layers))

        def get(name: str) -> torch.Tensor:
            shape = shapes[name]
            if name.endswith(("norm", "norm1")):
                return torch.ones(shape, device=self.device)
            t = torch.randn(*shape, generator=gen, device=self.device)
            if name.endswith((".r1", ".r2")):
                return 0.1 + t.abs()
            if name.endswith(".pb"):
                return t - 4.0           # a few keys' worth of weight
            if name in ("embed", "pos"):
                return t
            scale = 1.0 / math.sqrt(shape[-1])
            if name.endswith((".o", ".down")):
                scale /= depth
            return t * scale
        return get

    def _set_weights(self, get: Callable[[str], torch.Tensor]) -> None:
        s, dt = self.spec, self.dtype
        mat = lambda name: get(name).to(dt).contiguous()
        vec = lambda name: get(name).float().contiguous()
        self.emb, self.pos_emb = mat("embed"), mat("pos")
        self.layers: List[BokenexLayer] = []
        for i, L in enumerate(s.layers):
            p = f"l{i}."
            mixer = MIXERS[L.mixer.kind]
            rows = [mat(p + "mix." + n) for n in mixer.IN]
            cols = [mat(p + "mix.o")]
            mlp = None
            if L.mlp is not None:
                mlp = FEED_FORWARDS[L.mlp.kind](
                    L.mlp, lambda n, p=p: mat(p + "mlp." + n))
                rows += [mat(p + "mlp." + n) for n in mlp.IN]
                cols += [mat(p + "mlp." + n) for n in mlp.OUT]
            self.layers.append(BokenexLayer(
                norm=ops.GainNorm(vec(p + "norm1"), s.hidden_size, s.norm_eps),
                w_in=torch.cat(rows, dim=0).contiguous(),
                w_out=torch.cat(cols, dim=1).contiguous(),
                mixer=mixer(L.mixer, s.norm_eps,
                            lambda n, p=p: mat(p + "mix." + n),
                            lambda n, p=p: vec(p + "mix." + n)),
                mlp=mlp))
        self.norm_f = ops.GainNorm(vec("final.norm"), s.hidden_size,
                                   s.norm_eps)
        self.lm_head = mat("head")

    def state_dict_full(self) -> Dict[str, torch.Tensor]:
        s = self.spec
        out = {"embed": self.emb, "pos": self.pos_emb, "head": self.lm_head,
               "final.norm": self.norm_f.gain}
        for i, (L, lw) in enumerate(zip(s.layers, self.layers)):
            p, m = f"l{i}.", L.mixer
            out[p + "norm1"] = lw.norm.gain
            shapes = lw.mixer.shapes(m, s.hidden_size)
            at = 0
            for n in lw.mixer.IN:
                out[p + "mix." + n] = lw.w_in[at:at + shapes[n][0]]
                at += shapes[n][0]
            out[p + "mix.o"] = lw.w_out[:, :m.out_cols]
            for n, t in lw.mixer.own_weights().items():
                out[p + "mix." + n] = t
            if lw.mlp is not None:
                for n in lw.mlp.IN:
                    out[p + "mlp." + n] = lw.w_in[at:]
                for n in lw.mlp.OUT:
                    out[p + "mlp." + n] = lw.w_out[:, m.out_cols:]
                for n, t in lw.mlp.own_weights().items():
                    out[p + "mlp." + n] = t
        return out

    # -- forward -----------------------------------------------------------------

    def forward(self, batch, cache: HybridCache,
                on_run: Optional[Callable[[int, torch.Tensor], None]] = None
                ) -> torch.Tensor:
        """One step -> float32 logits of ``batch.want_rows`` (all rows if
        None). ``on_run(r, residual)`` is called after every layer."""
        s, dt = self.spec, self.dtype
        x = ops.embed_pos(batch.tokens, batch.pos, self.emb, self.pos_emb)
        for r, (lw, L) in enumerate(zip(self.layers, s.layers)):
            n_mix, mlp = L.mixer.out_cols, lw.mlp
            ff = mlp.act_cols if mlp is not None else 0
            cat = torch.empty(x.shape[0], n_mix + ff, dtype=dt,
                              device=x.device)
            h = ops.GainNormed(x, lw.norm, dt)
            proj, router = ops.parallel_in(
                h, lw.w_in, L.mixer.in_rows, ff,
                mlp.router_rows if mlp is not None else 0, cat[:, n_mix:])
            lw.mixer.run(proj, cat[:, :n_mix], batch, cache, r, {})
            if router is None:
                x = ops.residual_linear(x, cat, lw.w_out, s.residual_mult)
            else:
                x = ops.residual_moe(x, h, router, cat, lw.w_out, mlp.up,
                                     mlp.down, mlp.f, s.residual_mult)
            if on_run is not None:
                on_run(r, x)
        if batch.want_rows is not None:
            x = x[batch.want_rows]
        return ops.gain_logits(ops.GainNormed(x, self.norm_f, dt),
                               self.lm_head)
