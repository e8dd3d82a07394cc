// Model registry: which designs a folder with config.json and model.safetensors may hold, how their
// configurations are read, and the loader that picks the model class from what it finds.
#include "layered.hpp"

#include <cmath>
#include <sys/stat.h>

namespace litenn_hip
{
	namespace
	{
		const char* kAction = "HIP model";
		constexpr int kMaxSize = 1 << 24;
		constexpr int kDefaultContext = 32768;

		// the layer's feed-forward, if it has one; its constants are the design's
		const Json* dense_feed_forward(const Json& layer, LayerDesc& L)
		{
			const Json* mlp = layer.find("mlp");
			if (!mlp || mlp->is_null())
			{
				return nullptr;
			}
			const std::string& kind = mlp->string("kind");
			if (kind != "dense")
			{
				throw std::runtime_error("configuration: unknown feed-forward kind '" + kind + "'");
			}
			L.ff = mlp->integer("ff", 1, kMaxSize);
			return mlp;
		}

		// ---- Kulurax -------------------------------------------------------------------------
		// Sinusoidal positions; layers of latent attention or gated linear attention, each optionally
		// followed by a clamped gated feed-forward; norms on both sides of every sublayer; tied head.
		LayeredDesc describe_kulurax(const Json& c, const ShapeOf& shape_of)
		{
			LayeredDesc d;
			d.vocab = c.integer("vocab", 1, kMaxSize);
			d.width = c.integer("width", 1, kMaxSize);
			d.eps = static_cast<float>(c.at("norm").real("eps"));
			d.sinusoid_base = 10000.0;
			const Json& layers = c.at("layers");
			if (layers.kind != Json::Array || layers.items.empty())
			{
				throw std::runtime_error("configuration: 'layers' is not a list of layers");
			}
			for (size_t i = 0; i < layers.items.size(); ++i)
			{
				const Json& in = layers.items[i];
				const Json& mix = in.at("mixer");
				const std::string& type = in.string("type");
				LayerDesc L;
				MixerDesc m;
				m.heads = mix.integer("heads", 1, 32768);
				if (type == "latent_attention")
				{
					m.kind = MixerKind::LatentAttention;
					m.dim = mix.integer("dim", 1, 1024);
					m.vdim = mix.integer("vdim", 1, 1024);
					m.q_rank = mix.integer("q_rank", 1, kMaxSize);
					m.kv_rank = mix.integer("kv_rank", 1, latent_step_max_rank());
					m.scale = static_cast<float>(mix.real("scale"));
					const Json* mask = mix.find("mask");
					m.window = mask && !mask->is_null() ? mask->integer("size", 1, 1 << 30) : 0;
				}
				else if (type == "gla")
				{
					m.kind = MixerKind::GatedLinearAttention;
					m.dim = mix.integer("dim", 1, gla_max_dim());
					m.vdim = mix.integer("vdim", 1, gla_max_vdim());
					m.tau = static_cast<float>(mix.real("tau"));
					if (!(m.tau > 0.0f))
					{
						throw std::runtime_error("configuration: 'tau' must be greater than zero");
					}
					const std::vector<size_t>& low = shape_of("l" + std::to_string(i) + ".mix.a1");
					if (low.size() != 2 || low[0] < 1 || low[0] > 512)
					{
						throw std::runtime_error("the decay's low-rank projection must have 1 to 512 rows");
					}
					m.decay_rank = static_cast<int>(low[0]);
				}
				else
				{
					throw std::runtime_error("configuration: unknown layer type '" + type + "'");
				}
				L.mixers.push_back(m);
				if (const Json* mlp = dense_feed_forward(in, L))
				{
					L.act.limit = static_cast<float>(mlp->real("limit"));
					L.act.alpha = 1.702f;
					L.act.shift = 1.0f;
				}
				d.layers.push_back(L);
			}
			return d;
		}

		// ---- Degedra -------------------------------------------------------------------------
		// Layers of windowed attention and a state-space recurrence side by side, each optionally followed by a
		// gated feed-forward; only what a sublayer returns is normalised; soft-capped logits.  A layer may use
		// an earlier or later layer's weights.
		MixerDesc degedra_attention(const Json& c)
		{
			MixerDesc m;
			m.kind = MixerKind::GroupedAttention;
			m.name = "left.";
			m.heads = c.integer("heads", 1, 32768);
			m.kv_heads = c.integer("kv_heads", 1, m.heads);
			m.dim = c.integer("dim", 1, grouped_max_dim());
			m.vdim = c.integer("vdim", 1, grouped_max_dim());
			m.scale = static_cast<float>(c.real("scale"));
			const Json* mask = c.find("mask");
			m.window = mask && !mask->is_null() ? mask->integer("size", 1, 1 << 30) : 0;
			const Json* rot = c.find("rot");
			if (rot && !rot->is_null())
			{
				m.rot_dims = rot->integer("dims", 0, m.dim);
				m.rot_base = rot->real("base");
			}
			m.projection_norm = true;
			m.values_are_keys = true;
			if (m.heads % m.kv_heads != 0)
			{
				throw std::runtime_error("configuration: 'heads' is not a multiple of 'kv_heads'");
			}
			if (m.vdim != m.dim)
			{
				throw std::runtime_error("configuration: the values are the keys, but 'vdim' is not 'dim'");
			}
			if (m.rot_dims % 2 != 0 || (m.rot_dims > 0 && !(m.rot_base > 0.0)))
			{
				throw std::runtime_error("configuration: the rotation takes an even number of dimensions and a base greater than zero");
			}
			return m;
		}

		MixerDesc degedra_state_space(const Json& c)
		{
			MixerDesc m;
			m.kind = MixerKind::StateSpace;
			m.name = "right.";
			m.heads = c.integer("heads", 1, 32768);
			m.vdim = c.integer("vdim", 1, 32768);
			m.state = c.integer("state", 1, ssm_max_state());
			m.groups = c.integer("groups", 1, m.heads);
			m.norm_groups = c.integer("norm_groups", 1, kMaxSize);
			m.taps = c.integer("conv", 1, 1024);
			if (m.heads % m.groups != 0)
			{
				throw std::runtime_error("configuration: 'heads' is not a multiple of 'groups'");
			}
			if (static_cast<long long>(m.heads) * m.vdim > kMaxSize || m.heads * m.vdim % m.norm_groups != 0)
			{
				throw std::runtime_error("configuration: 'norm_groups' does not divide heads times 'vdim'");
			}
			return m;
		}

		LayeredDesc describe_degedra(const Json& c, const ShapeOf&)
		{
			LayeredDesc d;
			d.vocab = c.integer("vocab", 1, kMaxSize);
			d.width = c.integer("width", 1, kMaxSize);
			d.eps = static_cast<float>(c.at("norm").real("eps"));
			d.norms = NormPlacement::Output;
			d.tied_head = false;
			const Json* cap = c.find("logit_softcap");
			if (cap && !cap->is_null())
			{
				d.logit_softcap = static_cast<float>(c.real("logit_softcap"));
				if (!(d.logit_softcap > 0.0f))
				{
					throw std::runtime_error("configuration: 'logit_softcap' must be greater than zero");
				}
			}
			const Json& layers = c.at("layers");
			if (layers.kind != Json::Array || layers.items.empty())
			{
				throw std::runtime_error("configuration: 'layers' is not a list of layers");
			}
			const int count = static_cast<int>(layers.items.size());
			for (int i = 0; i < count; ++i)
			{
				// the owner of the layer's weights describes the layer
				int owner = i;
				for (int hops = 0; const Json* of = layers.items[owner].find("weights_of"); ++hops)
				{
					if (of->is_null())
					{
						break;
					}
					owner = layers.items[owner].integer("weights_of", 0, count - 1);
					if (hops == count)
					{
						throw std::runtime_error("configuration: 'weights_of' leads round in a circle");
					}
				}
				const Json& in = layers.items[owner];
				const std::string& type = in.string("type");
				if (type != "parallel" || layers.items[i].string("type") != type)
				{
					throw std::runtime_error("configuration: unknown layer type '" + layers.items[i].string("type") + "'");
				}
				const Json& mix = in.at("mixer");
				LayerDesc L;
				L.weights_of = owner == i ? -1 : owner;
				L.mixers = { degedra_attention(mix.at("left")), degedra_state_space(mix.at("right")) };
				L.mixers[0].weight = static_cast<float>(mix.real("left_scale"));
				L.mixers[1].weight = static_cast<float>(mix.real("right_scale"));
				if (dense_feed_forward(in, L))
				{
					L.act.limit = INFINITY;
					L.act.alpha = 1.0f;
				}
				d.layers.push_back(L);
			}
			return d;
		}

		constexpr Architecture kArchitectures[] = {
			{ "Kulurax", describe_kulurax },
			{ "Degedra", describe_degedra },
		};

		int dtype_of(const std::string& name)
		{
			return name == "BF16" ? LITENN_BF16 : name == "F32" ? LITENN_F32 : name == "F16" ? LITENN_F16 : name == "I32" ? LITENN_I32 : -1;
		}

		int create(int dev, const std::string& config_text, const litenn_hip_model_tensor* tensors, size_t count, int dtype,
		           int context_length, litenn_hip_model** out)
		{
			const Json config = Json::parse(config_text.data(), config_text.size(), "config.json");
			const std::string& name = config.string("architecture");
			const Architecture* arch = find_architecture(name);
			if (!arch)
			{
				throw std::runtime_error("unknown architecture '" + name + "'");
			}
			std::map<std::string, std::vector<size_t>> shapes;
			for (size_t i = 0; i < count; ++i)
			{
				if (!tensors[i].name || tensors[i].rank > 4)
				{
					throw std::runtime_error("a tensor without a name or of more than four dimensions");
				}
				shapes[tensors[i].name].assign(tensors[i].shape, tensors[i].shape + tensors[i].rank);
			}
			const ShapeOf shape_of = [&](const std::string& tensor) -> const std::vector<size_t>& {
				const auto it = shapes.find(tensor);
				if (it == shapes.end())
				{
					throw std::runtime_error("Missing tensor '" + tensor + "'");
				}
				return it->second;
			};
			LayeredDesc desc = arch->describe(config, shape_of);
			desc.architecture = name;
			return layered_create(dev, desc, tensors, count, dtype, context_length > 0 ? context_length : kDefaultContext, out);
		}
	} // namespace

	const Architecture* find_architecture(const std::string& name)
	{
		for (const Architecture& a : kArchitectures)
		{
			if (name == a.name)
			{
				return &a;
			}
		}
		return nullptr;
	}
} // namespace litenn_hip

using namespace litenn_hip;

extern "C" int litenn_hip_model_create(int dev, const char* config_json, const litenn_hip_model_tensor* tensors,
                                       size_t count, int dtype, int32_t context_length, litenn_hip_model** out)
{
	if (!config_json || !out || (count && !tensors))
	{
		return fail(kAction, "null argument");
	}
	*out = nullptr;
	try
	{
		return create(dev, config_json, tensors, count, dtype, context_length, out);
	}
	catch (const std::exception& ex)
	{
		return fail(kAction, ex.what());
	}
}

extern "C" int litenn_hip_model_load(int dev, const char* path, int dtype, int32_t context_length,
                                     litenn_hip_model** out)
{
	if (!path || !out)
	{
		return fail(kAction, "null argument");
	}
	*out = nullptr;
	struct stat st{};
	if (stat(path, &st) != 0)
	{
		return fail(kAction, std::string("cannot open '") + path + "'");
	}
	if (!S_ISDIR(st.st_mode))
	{
		// a GGUF file or a LiteNN archive
		litenn_hip_llama* llama = nullptr;
		if (litenn_hip_llama_load_gguf(dev, path, dtype == LITENN_F32 ? LITENN_F32 : LITENN_F16, context_length, &llama) != 0)
		{
			return 1;
		}
		*out = litenn_hip_llama_model(llama);
		if (dtype == LITENN_F32)
		{
			(*out)->base_flags = LITENN_HIP_MATMUL_PRECISE;
		}
		return 0;
	}
	try
	{
		const std::string dir(path);
		const std::string config = read_text_file(dir + "/config.json");
		const Safetensors file(dir + "/model.safetensors");
		std::vector<litenn_hip_model_tensor> tensors;
		for (const auto& t : file.tensors())
		{
			litenn_hip_model_tensor d{};
			d.name = t.first.c_str();
			d.dtype = dtype_of(t.second.dtype);
			d.rank = t.second.shape.size();
			if (d.dtype < 0 || d.rank > 4)
			{
				throw std::runtime_error("tensor '" + t.first + "' has an unsupported type or shape");
			}
			std::copy(t.second.shape.begin(), t.second.shape.end(), d.shape);
			d.data = t.second.data;
			tensors.push_back(d);
		}
		return create(dev, config, tensors.data(), tensors.size(), dtype, context_length, out);
	}
	catch (const std::exception& ex)
	{
		return fail(kAction, ex.what());
	}
}
