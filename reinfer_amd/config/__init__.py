from .schema import (BlockSpec, ConfigError, DecayMemorySpec, DeltaRuleSpec, FeedForwardSpec,
                     GatedLinearSpec, HyperSpec, InputSpec, LatentAttentionSpec,
                     MatrixMemorySpec, MixerSpec, ModelSpec, MoESpec, NormSpec, PairHashSpec, PositionSpec, RunEntry,
                     ParallelSpec, SideBySideSpec, StreamAdd, UnknownArchitecture, WKVSpec, YarnSpec)
from .registry import (architecture_name, config_from_dict, load_config, register_architecture,
                       registered_architectures)
from .qwen3 import Qwen3Config
from .puresun import PuresunConfig
from .kobolix import KobolixConfig
from .detatar import DetatarConfig
from .gibavik import GibavikConfig
from .sagalorn import SagalornConfig
from .dokanex import DokanexConfig

register_architecture("Qwen3ForCausalLM", Qwen3Config, "qwen3")
register_architecture("Puresun", PuresunConfig, "puresun")
register_architecture("Kobolix", KobolixConfig, "kobolix")
register_architecture("Detatar", DetatarConfig, "detatar")
register_architecture("Gibavik", GibavikConfig, "gibavik")
register_architecture("Sagalorn", SagalornConfig, "sagalorn")
register_architecture("Dokanex", DokanexConfig, "dokanex")

__all__ = [
    "BlockSpec", "ConfigError", "FeedForwardSpec", "MixerSpec", "ModelSpec", "NormSpec",
    "PositionSpec", "RunEntry", "UnknownArchitecture", "architecture_name", "config_from_dict",
    "load_config", "register_architecture", "registered_architectures", "Qwen3Config", "PuresunConfig", "KobolixConfig", "DetatarConfig", "GibavikConfig", "SagalornConfig", "DokanexConfig", "YarnSpec", "DecayMemorySpec", "GatedLinearSpec", "HyperSpec", "ParallelSpec", "WKVSpec",
    "InputSpec", "LatentAttentionSpec", "DeltaRuleSpec", "MatrixMemorySpec", "SideBySideSpec", "MoESpec", "PairHashSpec", "StreamAdd",
]
