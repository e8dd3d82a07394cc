// A decoder described as a list of layers (see layered.hip): which mixer and feed-forward each layer
// has, with their sizes and constants.  A model design is a function that turns its configuration
// into this description (registry.hip).
#pragma once

#include "checkpoint.hpp"
#include "decoder.hpp"
#include "layers.hpp"

#include <functional>

namespace litenn_hip
{
	enum class MixerKind { LatentAttention, GatedLinearAttention, GroupedAttention, StateSpace };

	struct MixerDesc
	{
		MixerKind kind = MixerKind::LatentAttention;
		std::string name;    // its tensors are '<layer>.mix.<name>...'
		float weight = 1.0f; // of its output in the layer's sum
		int heads = 0, dim = 0, vdim = 0;
		// attention of either kind
		int window = 0; // 0: every earlier position
		float scale = 1.0f;
		// latent attention
		int q_rank = 0, kv_rank = 0;
		// gated linear attention
		int decay_rank = 0;
		float tau = 1.0f;
		// grouped attention
		int kv_heads = 0;
		bool projection_norm = false;  // queries and keys are normalised as whole projections ('q.norm', 'k.norm')
		bool values_are_keys = false;  // no value projection: the values are the keys as projected
		int rot_dims = 0;              // 0: no rotation
		double rot_base = 10000.0;
		// state space
		int state = 0, groups = 0, taps = 0, norm_groups = 0;
	};

	struct LayerDesc
	{
		// one, or several side by side whose weighted outputs are added (grouped attention and state space only)
		std::vector<MixerDesc> mixers;
		int ff = 0; // 0: no feed-forward
		ClampedGlu act;
		int weights_of = -1; // >= 0: the layer that owns this layer's tensors (and has none of another's)
	};

	enum class NormPlacement
	{
		Around, // x += norm_b(f(norm(x))): 'norm1', 'norm1b', 'norm2', 'norm2b'
		Output, // x += norm(f(x)): 'norm1', 'norm2'
	};

	struct LayeredDesc
	{
		std::string architecture;
		int vocab = 0, width = 0;
		float eps = 0.0f;
		double sinusoid_base = 0.0; // > 0: sinusoidal position vectors are added to the embeddings
		NormPlacement norms = NormPlacement::Around;
		bool tied_head = true;      // otherwise 'head'
		float logit_softcap = 0.0f; // > 0: logits become softcap tanh(logits / softcap)
		std::vector<LayerDesc> layers;
	};

	// The shape of a named tensor of the checkpoint; throws when there is none
	using ShapeOf = std::function<const std::vector<size_t>&(const std::string&)>;

	struct Architecture
	{
		const char* name; // config.json's "architecture"
		LayeredDesc (*describe)(const Json& config, const ShapeOf& shape_of);
	};
	const Architecture* find_architecture(const std::string& name);

	// Builds a resident model from host tensors; 0 or a status with a message.
	int layered_create(int dev, const LayeredDesc& desc, const litenn_hip_model_tensor* tensors, size_t count, int dtype,
	                   int context_length, litenn_hip_model** out);
} // namespace litenn_hip
