"""A whole decoder assembled from a plan (reference model.py:102-146)."""
from typing import Dict, List

import torch

from ..config.spec import ModelPlan
from ..ops import kernels as K
from ..ops import linear as L
from ..ops import streams as ST
from .base import (BLOCKS, INPUT_ADDS, NORMS, POSITIONS, STREAM_STEPS, Param, ResidualStream, Runtime,
                   check_bound)
from .block import StreamRead


class DecoderModel:
    """Embedding, the plan's layers in the plan's order, final norm, output head; around
    them the optional steps a plan may state (a factor on the embedded rows, a position
    encoding added to them, a factor and a soft cap on the logits).

    ``forward`` runs the tokens of one step: embeds them, passes the float32 residual
    stream through every run of the order with that run's cache entry, then norms and
    projects only the rows whose logits are wanted (the reference projects every
    position, model.py:144-146)."""

    def __init__(self, plan: ModelPlan, runtime: Runtime):
        plan.validate()
        self.plan = plan
        self.rt = runtime
        self.blocks = [BLOCKS.build(_Arranged(layer), runtime) for layer in plan.layers]
        self.final_norm = NORMS.build(plan.final_norm, runtime)
        # what reads the stream last: the final norm, over the sum of the streams if there are several
        self.final_read = self.final_norm if plan.streams is None else \
            StreamRead(self.final_norm, runtime, streams=plan.streams)
        self.input_position = None
        if plan.input_position is not None:
            self.input_position = POSITIONS.build(plan.input_position, runtime)
            if not hasattr(self.input_position, "add_to_stream"):
                raise TypeError(f"position kind '{plan.input_position.kind}' cannot be a plan's "
                                f"input_position: its part has no add_to_stream(residual, batch)")
        # further parts that add to the embedded rows; each may keep state in a cache entry of
        # its own, which stands behind the runs' entries
        self.input_adds = [INPUT_ADDS.build(spec, runtime) for spec in plan.input_adds]
        # steps on the stream that stand before a run (Run.enter), one part per spec: runs that
        # name the same spec share its parameters
        self.enter_steps = {}
        for run in plan.order:
            spec = getattr(run, "enter", None)
            if spec is not None and spec not in self.enter_steps:
                self.enter_steps[spec] = STREAM_STEPS.build(spec, runtime)
        self.embedding = self.head = None
        # ``tap(n, rows)`` is called with the float32 stream [N, D] (the sum of several) after run n of
        # the order (tracing, tests); None: nothing is called
        self.tap = None

    # ------------------------------------------------------------------ parameters
    def parameters(self) -> Dict[str, Param]:
        p = {self.plan.embedding_name: Param((self.plan.vocab_size, self.plan.dim)),
             self.plan.head_name: Param((self.plan.vocab_size, self.plan.dim))}
        for name, param in self.final_norm.parameters().items():
            p[f"{self.plan.final_norm_name}.{name}"] = param
        if self.input_position is not None:
            for name, param in self.input_position.parameters().items():
                p[f"{self.plan.input_position_name}.{name}"] = param
        for spec, part in zip(self.plan.input_adds, self.input_adds):
            for name, param in part.parameters().items():
                p[f"{spec.name}.{name}"] = param
        for step in self.enter_steps.values():
            p.update(step.parameters())             # under their own full names
        for layer, block in zip(self.plan.layers, self.blocks):
            for name, param in block.parameters().items():
                p[f"{layer.name}.{name}"] = param
        return p

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        declared = self.parameters()
        check_bound("model", declared, tensors)
        extra = sorted(set(tensors) - set(declared))
        if extra:
            raise KeyError(f"model: parameters {extra} belong to no part")
        # (place, elements, bytes per element) of every parameter; the tensors themselves belong to
        # the parts, which may keep them in another form
        self._sizes = {name: (t.data_ptr(), t.numel(), t.element_size()) for name, t in tensors.items()}
        self.embedding = tensors[self.plan.embedding_name]
        self.head = tensors[self.plan.head_name]
        prefix = self.plan.final_norm_name + "."
        self.final_norm.bind({k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)})
        if self.input_position is not None:
            prefix = self.plan.input_position_name + "."
            self.input_position.bind({k[len(prefix):]: v for k, v in tensors.items()
                                      if k.startswith(prefix)})
        for spec, part in zip(self.plan.input_adds, self.input_adds):
            prefix = spec.name + "."
            part.bind({k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)})
        for step in self.enter_steps.values():
            step.bind({k: tensors[k] for k in step.parameters()})
        for layer, block in zip(self.plan.layers, self.blocks):
            prefix = layer.name + "."
            block.bind({k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)})

    def parameter_bytes(self, exclude_embedding: bool = True, rows: int = None) -> int:
        """Bytes of the parameters one decode step reads (the embedding table is a
        gather of a few rows, as in the reference's accounting, generate.py:251-268).  With
        ``rows``, the step's tokens, parts that read only some of their parameters in a step
        of so many rows (a table of which each token takes one row, a mixture of experts)
        take off what such a step leaves unread (``unread_bytes(rows)``)."""
        if rows is not None:
            parts = list(self.blocks) + list(self.input_adds) + [self.input_position]
            unread = sum(getattr(p, "unread_bytes", lambda r: 0)(rows) for p in parts if p is not None)
            return self.parameter_bytes(exclude_embedding) - unread
        total = 0
        for n, size in self._read_once(exclude_embedding):
            total += n * size
        return total

    @property
    def replayable(self) -> bool:
        """Every part issues the same kernels whatever a batch holds: a recorded step can be
        replayed."""
        return (all(getattr(b, "replayable", False) for b in self.blocks)
                and all(getattr(s, "replayable", False) for s in self.enter_steps.values())
                and all(getattr(a, "replayable", False) for a in self.input_adds)
                and getattr(self.final_norm, "replayable", False)
                and (self.input_position is None
                     or getattr(self.input_position, "replayable", False)))

    def parameter_count(self, exclude_embedding: bool = True) -> int:
        """Elements of the same parameters (the reference's ``params`` of
        generate.py:251-268, which feeds its FLOPS line)."""
        return sum(n for n, _ in self._read_once(exclude_embedding))

    def _read_once(self, exclude_embedding: bool):
        """(elements, bytes per element) of every parameter a step reads, shared ones once."""
        head = self._sizes[self.plan.head_name][0]
        seen = set()
        for name, (place, n, size) in self._sizes.items():
            if exclude_embedding and name == self.plan.embedding_name and place != head:
                continue
            if place not in seen:
                seen.add(place)
                yield n, size

    # ------------------------------------------------------------------ cache
    def cache_needs(self) -> List[object]:
        """One need per run of the order, then one per input add."""
        return [self.blocks[run.layer].cache_need() for run in self.plan.order] \
            + [a.cache_need() for a in self.input_adds]

    def cache_borrow(self) -> List[object]:
        return [run.cache_from for run in self.plan.order] + [None] * len(self.input_adds)

    def step_flops(self, q_lens, starts, n_want: int) -> float:
        """Matrix-product work (multiply-adds times two) of one step that brings
        ``q_lens[b]`` tokens to sequences holding ``starts[b]`` and wants ``n_want`` rows of
        logits: every run of the order, as its parts count themselves, and the head."""
        flops = 2.0 * n_want * self.plan.dim * self.plan.vocab_size
        for run in self.plan.order:
            block = self.blocks[run.layer]
            flops += getattr(block, "step_flops", lambda q, s: 0.0)(q_lens, starts)
            if getattr(run, "enter", None) is not None:
                flops += getattr(self.enter_steps[run.enter], "step_flops",
                                 lambda q, s: 0.0)(q_lens, starts)
        return flops

    def kernel_libraries(self):
        """Names of the compiled libraries (csrc/<name>.hip) that a step of this model calls:
        the ones every model uses, by the engine's type, and those its parts name in
        ``libraries`` (a tuple, or a function of the runtime)."""
        names = ["core"]
        if not self.rt.is_float32:
            names += ["gemm_bf16", "gemm_wide_bf16", "gemm_tiled_bf16"]

        def visit(part):
            libs = getattr(part, "libraries", ())
            for n in (libs(self.rt) if callable(libs) else libs):
                if n not in names:
                    names.append(n)
            for child in getattr(part, "children", lambda: {})().values():
                visit(child)
        for part in list(self.blocks) + list(self.enter_steps.values()) + list(self.input_adds) \
                + [self.final_norm, self.input_position]:
            if part is not None:
                visit(part)
        return names

    def step_fields(self):
        """The further fields of a step's description that the parts ask for, each once (by
        name: layers of one kind ask for the same field)."""
        seen = {}
        parts = list(self.blocks) + list(self.input_adds) + [self.final_norm, self.input_position]
        for part in parts:
            for f in (getattr(part, "step_fields", lambda: ())() if part is not None else ()):
                seen.setdefault(f.name, f)
        return list(seen.values())

    # ------------------------------------------------------------------ step
    def forward(self, batch, cache) -> torch.Tensor:
        """float32 logits [n_wanted, vocab] of the step described by ``batch``."""
        plan = self.plan
        residual = K.embed(self.embedding, batch.tokens)                  # model.py:140
        if plan.embedding_scale is not None:
            K.scale_cap(residual, plan.embedding_scale)
        for i, part in enumerate(self.input_adds):
            part.add_to_stream(residual, batch, cache.entries[len(plan.order) + i])
        if self.input_position is not None:
            self.input_position.add_to_stream(residual, batch)
        if plan.streams is not None:
            residual = ST.spread(residual, plan.streams)
        stream = ResidualStream(residual)
        # the embedded rows, for steps that mix them into the stream again; a copy where a
        # block may have changed the stream (in place) before the first such step
        embedded = None
        if self.enter_steps:
            embedded = residual if getattr(plan.order[0], "enter", None) is not None \
                else residual.clone()
        for n, run in enumerate(plan.order):                              # model.py:142-143
            if getattr(run, "enter", None) is not None:
                stream = ResidualStream(self.enter_steps[run.enter].forward(
                    stream.tensor, embedded, batch))
            block = self.blocks[run.layer]
            block.forward(stream if getattr(block, "takes_stream", False) else stream.tensor,
                          batch, cache.entries[n])
            if self.tap is not None:
                self.tap(n, stream.tensor if plan.streams is None else stream.tensor.sum(1))
        if batch.n_want == 0:
            stream.tensor
            return torch.empty((0, self.plan.vocab_size), dtype=torch.float32,
                               device=residual.device)
        # the head takes plain rows (no reader named): with its many columns the halves of a
        # norm cost more than the norm kernel they save
        every = getattr(batch, "every_row_wanted", False)
        x = stream.normed(self.final_read, rows=None if every else batch.want_rows)   # model.py:144
        logits = L.linear(x, self.head, out_dtype=torch.float32)          # model.py:145
        if plan.logit_scale is not None or plan.logit_softcap is not None:
            K.scale_cap(logits, 1.0 if plan.logit_scale is None else plan.logit_scale,
                        plan.logit_softcap or 0.0)
        return logits


class _Arranged:
    """Gives a LayerSpec the ``kind`` its arrangement is registered under."""

    def __init__(self, layer):
        self._layer = layer
        self.kind = layer.arrangement

    def __getattr__(self, name):
        return getattr(self._layer, name)
