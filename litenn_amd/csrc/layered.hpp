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
	enum class MixerKind { LatentAttention, GatedLinearAttention };

	struct MixerDesc
	{
		MixerKind kind = MixerKind::LatentAttention;
		int heads = 0, dim = 0, vdim = 0;
		// latent attention
		int q_rank = 0, kv_rank = 0;
		int window = 0; // 0: every earlier position
		float scale = 1.0f;
		// gated linear attention
		int decay_rank = 0;
		float tau = 1.0f;
	};

	struct LayerDesc
	{
		MixerDesc mixer;
		int ff = 0; // 0: no feed-forward
		ClampedGlu act;
	};

	struct LayeredDesc
	{
		std::string architecture;
		int vocab = 0, width = 0;
		float eps = 0.0f;
		double sinusoid_base = 0.0; // > 0: sinusoidal position vectors are added to the embeddings
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
