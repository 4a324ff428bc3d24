from .spec import (SILU_GLU, AttentionSpec, ClampedGLUSpec, ConfigError, GatedLinearAttentionSpec, GeneralDeltaSpec, HashedBigramSpec,
                   InterleavedRopeSpec,
                   LatentAttentionSpec, LayerNormSpec, LayerSpec, LightningAttentionSpec, LinearDistanceBiasSpec, LogDistanceBiasSpec, Mamba2Spec,
                   MixerSlot, ModelSpec, NoPositionSpec, PolyNormFFNSpec, PowerReluSpec, RampScalingSpec, RetentionSpec, RmsNormSpec, RopeSpec,
                   RoutedExpertsSpec, ScheduleEntry, StreamInjection, SwiGLUSpec, TanhNormSpec, WavelengthScalingSpec)
from .registry import (config_from_dict, load_config, register_architecture,
                       registered_architectures)
from .falcon_h1 import FalconH1Config
from .mukutar import MukutarConfig
from .lutosun import LutosunConfig
from .motolix import MotolixConfig
from .pemarax import PemaraxConfig
from .pipizen import PipizenConfig
from .sazavik import SazavikConfig

register_architecture(FalconH1Config)
register_architecture(MukutarConfig)
register_architecture(LutosunConfig)
register_architecture(MotolixConfig)
register_architecture(PemaraxConfig)
register_architecture(PipizenConfig)
register_architecture(SazavikConfig)

__all__ = ["AttentionSpec", "ClampedGLUSpec", "ConfigError", "FalconH1Config", "GatedLinearAttentionSpec", "GeneralDeltaSpec", "HashedBigramSpec",
           "InterleavedRopeSpec", "LatentAttentionSpec", "LayerNormSpec", "LayerSpec", "LightningAttentionSpec", "LinearDistanceBiasSpec", "LogDistanceBiasSpec", "LutosunConfig",
           "Mamba2Spec", "MixerSlot", "ModelSpec", "MotolixConfig", "MukutarConfig", "NoPositionSpec", "PemaraxConfig", "PipizenConfig", "PolyNormFFNSpec", "PowerReluSpec", "RampScalingSpec", "RetentionSpec",
           "RmsNormSpec", "RopeSpec", "RoutedExpertsSpec", "SILU_GLU", "SazavikConfig", "ScheduleEntry", "StreamInjection", "SwiGLUSpec", "TanhNormSpec", "WavelengthScalingSpec",
           "config_from_dict", "load_config", "register_architecture", "registered_architectures"]
