"""Typed configurations, the architecture registry and the neutral model description."""
from .spec import (AddRowsSpec, AttentionSpec, DenseMlpSpec, GatedDeltaSpec, InterleavedRotarySpec, LatentAttentionSpec, LayerNormSpec, LayerSpec, LearnedPositionsSpec, LightningSpec, MlstmSpec,
                   ModelSpec, NoNormSpec, PartialRotarySpec, RejoinSpec, RmsNormSpec, RotarySpec, RoutedExpertsSpec, RunEntry, ScaleSpec, SelectiveScanSpec, SideBySideSpec, SoftCapSpec,
                   StreamAccessSpec, SwiGluSpec, TokenPairSpec, TokenShiftSpec, TokenSideInputSpec)
from .errors import ConfigError
from .registry import (config_class_for, parse_config, read_config, register_architecture,
                       registered_architectures)
from .llama import Llama3Scaling, LlamaConfig          # registers itself
from .fekorax import FekoraxConfig                     # registers itself
from .rigalorn import RigalornConfig                   # registers itself
from .zidevik import ZidevikConfig                     # registers itself
from .mimitar import MimitarConfig                     # registers itself
from .vubenex import VubenexConfig                     # registers itself
from .puzorax import PuzoraxConfig                     # registers itself
