"""Serving engine: paged cache and state slots (cache), batch layout (batch), scheduling (scheduler), sampling (sampling) and the
engine that ties them to a model of omniserve_amd.models (engine)."""
from .engine import Engine, SequenceInput          # noqa: F401
from .sampling import SamplingParams               # noqa: F401
