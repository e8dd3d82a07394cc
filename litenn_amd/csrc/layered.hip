// The layered decoder: any sequence of layers out of the mechanisms of layers.hip over one sequence.
//
// Memory: weights stay in bfloat16; projections that read the same input are one matrix (their rows
// concatenated, so a layer's first product is one launch), gate and up rows of a feed-forward are
// interleaved so that the launch forms their product.  Mixers that run side by side share the input
// projection and, with their weights folded into what it reads, the output projection.  An attention layer
// keeps a ring of normalised latents, or of keys and values, long enough for its window plus one pass of tokens, a
// recurrent layer its Float32 state: what a sequence holds does not grow with its length beyond the window.
// Layers that use another's weights hold a cache and state of their own.
//
// A pass of kRowsMin tokens and more runs on the matrix cores, fewer tokens go one by one through the
// single-row form, whose launches read their position from device memory (so that one can be
// captured and replayed).  The residual stream is Float32; the step behind every sublayer, norm of its
// output, addition, norm for the next sublayer, runs in the prologue of the next product (single row)
// or as one kernel (many rows).
#include "layered.hpp"

#include <algorithm>
#include <climits>
#include <cmath>
#include <cstring>

namespace litenn_hip
{
	void launch_zero_ints(int* p, size_t n, hipStream_t s);

	namespace
	{
		const char* kAction = "HIP model";

		constexpr int kRowsMin = 4;        // from here on a pass runs on the matrix cores
		constexpr int kExpandMin = 16;     // from here on attention expands the cached latents
		constexpr int kPassRows = 4096;    // most tokens of a pass (LITENN_HIP_PASS_ROWS)
		constexpr int kSplitRows = 1024;   // up to here a sublayer's last product may walk K in several ranges at once
		constexpr int kAlignRows = 8;      // first row of every part of a concatenated matrix

		struct MixerState
		{
			MixerDesc desc;
			// first columns of the parts of the input projections' product, and of its share of the output projection's input
			int at_q = 0, at_k = 0, at_v = 0, at_gate = 0, at_low = 0, at_latent = 0, at_in = 0, at_mid = 0;
			// latent attention
			DenseMatrix uq, uk, uv, ukv; // uk and uv are rows of ukv
			int v_first = 0;
			const float *q_norm = nullptr, *latent_norm = nullptr, *sink = nullptr;
			LatentCache cache;
			int splits = 1;
			// gated linear attention
			DenseMatrix a2;
			const float *a2_bias = nullptr, *head_norm = nullptr;
			float* state = nullptr;
			// grouped attention
			const float* k_norm = nullptr; // beside q_norm
			const double* turns = nullptr;
			HeadCache heads;
			// state space
			const float *conv_w = nullptr, *conv_b = nullptr, *dt_bias = nullptr, *a_log = nullptr, *skip = nullptr,
			            *group_norm = nullptr;
			float* ring = nullptr; // the convolution's last inputs
		};

		struct LayerState
		{
			LayerDesc desc;
			// norms ahead of the sublayers (null where there are none) and behind them
			const float *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr;
			DenseMatrix in, out; // concatenated input projections, output projection
			std::vector<MixerState> mixers;
			// feed-forward
			DenseMatrix gate_up, down;
		};

		// where a tensor of the checkpoint goes
		struct Slot
		{
			uint16_t* matrix = nullptr; // bfloat16 rows, `stride` elements apart
			float* vector = nullptr;    // Float32 [rows], or [cols, rows] of a tensor [rows, cols]
			size_t rows = 0, cols = 0, stride = 0;
			bool filled = false;
		};
	} // namespace

	struct LayeredModel : litenn_hip_model
	{
		LayeredDesc desc;
		bool f32 = false;
		DenseMatrix embed, head;
		const float* final_norm = nullptr;
		const double* turns = nullptr;
		std::vector<LayerState> layers;
		std::map<std::string, Slot> slots;
		int max_pass = kPassRows;

		// scratch for cap_rows tokens
		size_t cap_rows = 0;
		float *x = nullptr, *proj = nullptr, *y = nullptr, *q = nullptr, *absorbed = nullptr, *partial = nullptr,
		      *log_decay = nullptr, *chunk_states = nullptr, *xbc = nullptr;
		void *h = nullptr, *mid = nullptr, *kv = nullptr;
		int ld_proj = 0, ld_y = 0, ld_q = 0, ld_h = 0, ld_mid = 0, ld_kv = 0;
		// single-row form
		float *xt[2] = { nullptr, nullptr }, *row_mid = nullptr, *row_ssm = nullptr;

		~LayeredModel() override { free_scratch(); }

		void free_scratch()
		{
			void** bufs[] = { reinterpret_cast<void**>(&x),       reinterpret_cast<void**>(&proj), reinterpret_cast<void**>(&y),
				              reinterpret_cast<void**>(&q),       reinterpret_cast<void**>(&absorbed), reinterpret_cast<void**>(&partial),
				              reinterpret_cast<void**>(&log_decay), reinterpret_cast<void**>(&chunk_states),
				              reinterpret_cast<void**>(&xbc), &h, &mid, &kv };
			for (void** b : bufs)
			{
				if (*b)
				{
					(void)hipFree(*b);
					*b = nullptr;
				}
			}
			cap_rows = 0;
		}

		// ---- construction -------------------------------------------------------------------
		void* allocate(size_t bytes)
		{
			void* p = nullptr;
			bytes = std::max<size_t>(bytes, 256);
			hipError_t e = hipMalloc(&p, bytes);
			if (e == hipSuccess)
			{
				owned.push_back(p);
				e = hipMemset(p, 0, bytes);
			}
			if (e != hipSuccess)
			{
				throw std::runtime_error(std::string("device memory: ") + hipGetErrorString(e));
			}
			return p;
		}

		struct Part
		{
			std::string name;
			int rows;
			int* at; // receives the part's first row, may be null
		};

		DenseMatrix matrix(const std::vector<Part>& parts, int cols)
		{
			if (static_cast<size_t>(dense_pitch(cols)) > dense_row_max_k())
			{
				throw std::runtime_error("'" + parts[0].name + "' has rows longer than " + std::to_string(dense_row_max_k()));
			}
			int total = 0;
			for (const Part& p : parts)
			{
				total = (total + kAlignRows - 1) / kAlignRows * kAlignRows;
				if (p.at)
				{
					*p.at = total;
				}
				total += p.rows;
			}
			DenseMatrix m;
			m.n = total;
			m.k = cols;
			m.pitch = dense_pitch(cols);
			uint16_t* w = static_cast<uint16_t*>(allocate(sizeof(uint16_t) * static_cast<size_t>(total) * m.pitch));
			m.w = w;
			int at = 0;
			for (const Part& p : parts)
			{
				at = (at + kAlignRows - 1) / kAlignRows * kAlignRows;
				Slot s;
				s.matrix = w + static_cast<size_t>(at) * m.pitch;
				s.rows = static_cast<size_t>(p.rows);
				s.cols = static_cast<size_t>(cols);
				s.stride = static_cast<size_t>(m.pitch);
				slots[p.name] = s;
				at += p.rows;
			}
			return m;
		}

		// rows of the two tensors alternate
		DenseMatrix interleaved(const std::string& even, const std::string& odd, int rows, int cols)
		{
			DenseMatrix m = matrix({ { even, rows, nullptr }, { odd, rows, nullptr } }, cols);
			m.n = 2 * rows; // rows need not be a multiple of the parts' alignment here
			Slot& a = slots[even];
			Slot& b = slots[odd];
			b.matrix = a.matrix + m.pitch;
			a.stride = b.stride = 2 * static_cast<size_t>(m.pitch);
			return m;
		}

		// the tensors' columns one behind the other: their products, added
		DenseMatrix side_by_side(const std::vector<std::pair<std::string, int>>& parts, int rows)
		{
			int cols = 0;
			for (const auto& p : parts)
			{
				cols += p.second;
			}
			DenseMatrix m = matrix({ { parts[0].first, rows, nullptr } }, cols);
			const Slot whole = slots[parts[0].first];
			int at = 0;
			for (const auto& p : parts)
			{
				Slot s = whole;
				s.matrix = whole.matrix + at;
				s.cols = static_cast<size_t>(p.second);
				slots[p.first] = s;
				at += p.second;
			}
			return m;
		}

		const double* turns_per_position(double base, int dims)
		{
			std::vector<double> f((static_cast<size_t>(dims) + 1) / 2);
			for (size_t i = 0; i < f.size(); ++i)
			{
				f[i] = std::pow(base, -2.0 * static_cast<double>(i) / dims) / (2.0 * M_PI);
			}
			double* p = static_cast<double*>(allocate(sizeof(double) * f.size()));
			copy_in(p, f.data(), sizeof(double) * f.size());
			return p;
		}

		// a tensor [rows, cols], kept column by column
		const float* columns(const std::string& name, int rows, int cols)
		{
			Slot s;
			s.vector = static_cast<float*>(allocate(sizeof(float) * static_cast<size_t>(rows) * cols));
			s.rows = static_cast<size_t>(rows);
			s.cols = static_cast<size_t>(cols);
			slots[name] = s;
			return s.vector;
		}

		const float* vector(const std::string& name, int n)
		{
			Slot s;
			s.vector = static_cast<float*>(allocate(sizeof(float) * ((static_cast<size_t>(n) + 3) & ~size_t{ 3 }))); // whole pieces
			s.rows = static_cast<size_t>(n);
			slots[name] = s;
			return s.vector;
		}

		// weights of one mixer: its input projections join `parts`, its output projection `outs`
		void build_mixer(const std::string& mix, MixerState& M, std::vector<Part>& parts, std::vector<std::pair<std::string, int>>& outs)
		{
			const MixerDesc& m = M.desc;
			const int values = m.heads * m.vdim, keys = m.heads * m.dim;
			switch (m.kind)
			{
			case MixerKind::LatentAttention: {
				parts.insert(parts.end(), { { mix + "dq", m.q_rank, &M.at_q }, { mix + "dkv", m.kv_rank, &M.at_latent }, { mix + "g", values, &M.at_gate } });
				M.q_norm = vector(mix + "dq.norm", m.q_rank);
				M.latent_norm = vector(mix + "dkv.norm", m.kv_rank);
				M.sink = vector(mix + "sink", m.heads);
				M.uq = matrix({ { mix + "uq", keys, nullptr } }, m.q_rank);
				int uv_at = 0;
				M.ukv = matrix({ { mix + "uk", keys, nullptr }, { mix + "uv", values, &uv_at } }, m.kv_rank);
				M.v_first = uv_at;
				M.uk = M.uv = M.ukv;
				M.uk.n = keys;
				M.uv.n = values;
				M.uv.w = M.ukv.w + static_cast<size_t>(uv_at) * M.ukv.pitch;
				break;
			}
			case MixerKind::GatedLinearAttention:
				parts.insert(parts.end(), { { mix + "q", keys, &M.at_q }, { mix + "k", keys, &M.at_k }, { mix + "v", values, &M.at_v },
				                            { mix + "g", values, &M.at_gate }, { mix + "a1", m.decay_rank, &M.at_low } });
				M.a2 = matrix({ { mix + "a2", keys, nullptr } }, m.decay_rank);
				M.a2_bias = vector(mix + "a2.b", keys);
				M.head_norm = vector(mix + "norm", m.vdim);
				break;
			case MixerKind::GroupedAttention:
				parts.insert(parts.end(), { { mix + "q", keys, &M.at_q }, { mix + "k", m.kv_heads * m.dim, &M.at_k } });
				if (!m.values_are_keys)
				{
					parts.push_back({ mix + "v", m.kv_heads * m.vdim, &M.at_v });
				}
				if (m.projection_norm)
				{
					M.q_norm = vector(mix + "q.norm", keys);
					M.k_norm = vector(mix + "k.norm", m.kv_heads * m.dim);
				}
				if (m.rot_dims > 0)
				{
					M.turns = turns_per_position(m.rot_base, m.rot_dims);
				}
				break;
			case MixerKind::StateSpace: {
				const int channels = values + 2 * m.groups * m.state;
				parts.push_back({ mix + "in", values + channels + m.heads, &M.at_in });
				M.conv_w = columns(mix + "conv", channels, m.taps);
				M.conv_b = vector(mix + "conv.b", channels);
				M.dt_bias = vector(mix + "dt_bias", m.heads);
				M.a_log = vector(mix + "A_log", m.heads);
				M.skip = vector(mix + "D", m.heads);
				M.group_norm = vector(mix + "norm", values);
				break;
			}
			}
			outs.emplace_back(mix + "o", values);
		}

		void build_weights(const std::string& p, LayerState& L)
		{
			const int width = desc.width;
			const bool around = desc.norms == NormPlacement::Around;
			(around ? L.norm1 : L.norm1b) = vector(p + "norm1", width);
			if (around)
			{
				L.norm1b = vector(p + "norm1b", width);
			}
			std::vector<Part> parts;
			std::vector<std::pair<std::string, int>> outs;
			L.mixers.resize(L.desc.mixers.size()); // before their members' addresses go into `parts`
			for (size_t i = 0; i < L.mixers.size(); ++i)
			{
				MixerState& M = L.mixers[i];
				M.desc = L.desc.mixers[i];
				for (const auto& before : outs)
				{
					M.at_mid += before.second;
				}
				build_mixer(p + "mix." + M.desc.name, M, parts, outs);
			}
			L.in = matrix(parts, width);
			for (MixerState& M : L.mixers)
			{
				if (M.desc.kind == MixerKind::GroupedAttention && M.desc.values_are_keys)
				{
					M.at_v = M.at_k;
				}
			}
			L.out = side_by_side(outs, width);
			if (L.desc.ff > 0)
			{
				const int ff = L.desc.ff;
				(around ? L.norm2 : L.norm2b) = vector(p + "norm2", width);
				if (around)
				{
					L.norm2b = vector(p + "norm2b", width);
				}
				L.gate_up = interleaved(p + "mlp.gate", p + "mlp.up", ff, width);
				L.down = matrix({ { p + "mlp.down", width, nullptr } }, ff);
			}
		}

		// what a sequence holds in one mixer
		void build_state(MixerState& M)
		{
			MixerDesc& m = M.desc;
			m.window = m.window > 0 ? std::min(m.window, context_length) : context_length;
			// a pass appends before it reads: the window behind its first token must survive
			const int ring = static_cast<int>(std::min<long long>(context_length, static_cast<long long>(m.window) - 1 + max_pass));
			switch (m.kind)
			{
			case MixerKind::LatentAttention:
				M.cache.ring = ring;
				M.cache.rank = m.kv_rank;
				M.cache.pitch = M.ukv.pitch;
				M.cache.f32 = f32;
				M.cache.rows = allocate((f32 ? 4 : 2) * static_cast<size_t>(ring) * M.cache.pitch);
				M.splits = latent_step_splits(m.heads, 1, m.window);
				break;
			case MixerKind::GatedLinearAttention:
				M.state = static_cast<float*>(allocate(sizeof(float) * state_floats(m)));
				break;
			case MixerKind::GroupedAttention:
				M.heads.ring = ring;
				M.heads.heads = m.kv_heads;
				M.heads.dim = m.dim;
				M.heads.vdim = m.vdim;
				M.heads.f32 = f32;
				M.heads.rows = allocate((f32 ? 4 : 2) * M.heads.elements());
				M.splits = grouped_step_splits(m.heads, m.kv_heads, m.dim, m.vdim, m.window);
				break;
			case MixerKind::StateSpace:
				M.state = static_cast<float*>(allocate(sizeof(float) * state_floats(m)));
				M.ring = static_cast<float*>(allocate(sizeof(float) * m.taps * static_cast<size_t>(ssm_args(M).channels())));
				break;
			}
		}

		void build()
		{
			const int width = desc.width;
			embed = matrix({ { "embed", desc.vocab, nullptr } }, width);
			head = desc.tied_head ? embed : matrix({ { "head", desc.vocab, nullptr } }, width);
			final_norm = vector("final.norm", width);
			layers.resize(desc.layers.size());
			for (size_t i = 0; i < layers.size(); ++i)
			{
				layers[i].desc = desc.layers[i];
				if (layers[i].desc.weights_of < 0)
				{
					build_weights("l" + std::to_string(i) + ".", layers[i]);
				}
			}
			int widest_mid = std::max(width, 64), proj_cols = 0, q_cols = 4, kv_cols = 0, ssm_cols = 4;
			for (LayerState& L : layers)
			{
				if (L.desc.weights_of >= 0)
				{
					L = LayerState(layers[static_cast<size_t>(L.desc.weights_of)]);
				}
			}
			for (LayerState& L : layers)
			{
				int mid_cols = 0;
				for (MixerState& M : L.mixers)
				{
					build_state(M);
					const MixerDesc& m = M.desc;
					mid_cols += m.heads * m.vdim;
					if (m.kind == MixerKind::LatentAttention)
					{
						kv_cols = std::max(kv_cols, M.ukv.n);
						widest_mid = std::max(widest_mid, m.q_rank);
					}
					if (m.kind == MixerKind::StateSpace)
					{
						ssm_cols = std::max(ssm_cols, m.heads * m.vdim);
					}
					else
					{
						q_cols = std::max(q_cols, m.heads * m.dim);
					}
				}
				widest_mid = std::max({ widest_mid, mid_cols, L.desc.ff });
				proj_cols = std::max(proj_cols, L.in.n);
			}
			const auto up4 = [](int n) { return (n + 3) & ~3; };
			ld_proj = up4(proj_cols);
			ld_y = up4(width);
			ld_q = up4(q_cols);
			ld_h = dense_pitch(width);
			ld_mid = dense_pitch(widest_mid);
			ld_kv = (std::max(kv_cols, 8) + 7) & ~7;
			if (desc.sinusoid_base > 0.0)
			{
				turns = turns_per_position(desc.sinusoid_base, width);
			}
			xt[0] = static_cast<float*>(allocate(sizeof(float) * static_cast<size_t>(width)));
			xt[1] = static_cast<float*>(allocate(sizeof(float) * static_cast<size_t>(width)));
			row_mid = static_cast<float*>(allocate(sizeof(float) * static_cast<size_t>(ld_mid)));
			row_ssm = static_cast<float*>(allocate(sizeof(float) * static_cast<size_t>(ssm_cols)));
		}

		static size_t state_floats(const MixerDesc& m)
		{
			return m.kind == MixerKind::StateSpace ? static_cast<size_t>(m.heads) * m.state * ssm_state_pitch(m.vdim)
			                                       : static_cast<size_t>(m.heads) * m.dim * gla_state_pitch(m.vdim);
		}

		static void copy_in(void* dst, const void* src, size_t bytes)
		{
			const hipError_t e = hipMemcpy(dst, src, bytes, hipMemcpyHostToDevice);
			if (e != hipSuccess)
			{
				throw std::runtime_error(std::string("weight upload: ") + hipGetErrorString(e));
			}
		}

		void upload(const litenn_hip_model_tensor& t)
		{
			const auto it = slots.find(t.name);
			if (it == slots.end())
			{
				throw std::runtime_error(std::string("the configuration has no place for tensor '") + t.name + "'");
			}
			Slot& s = it->second;
			const bool shaped = s.cols ? t.rank == 2 && t.shape[0] == s.rows && t.shape[1] == s.cols
			                           : t.rank == 1 && t.shape[0] == s.rows;
			if (!shaped || !t.data)
			{
				throw std::runtime_error(std::string("tensor '") + t.name + "' has another shape than the configuration gives it");
			}
			if (s.matrix)
			{
				if (t.dtype != LITENN_BF16)
				{
					throw std::runtime_error(std::string("tensor '") + t.name + "' is not BFloat16");
				}
				const hipError_t e = hipMemcpy2D(s.matrix, s.stride * 2, t.data, s.cols * 2, s.cols * 2, s.rows, hipMemcpyHostToDevice);
				if (e != hipSuccess)
				{
					throw std::runtime_error(std::string("weight upload: ") + hipGetErrorString(e));
				}
			}
			else
			{
				const size_t cols = std::max<size_t>(s.cols, 1);
				std::vector<float> v(s.rows * cols);
				for (size_t i = 0; i < v.size(); ++i)
				{
					float& to = v[i % cols * s.rows + i / cols];
					if (t.dtype == LITENN_BF16)
					{
						uint16_t b;
						memcpy(&b, static_cast<const uint8_t*>(t.data) + 2 * i, 2);
						const uint32_t w = static_cast<uint32_t>(b) << 16;
						memcpy(&to, &w, 4);
					}
					else if (t.dtype == LITENN_F32)
					{
						memcpy(&to, static_cast<const uint8_t*>(t.data) + 4 * i, 4);
					}
					else
					{
						throw std::runtime_error(std::string("tensor '") + t.name + "' is neither BFloat16 nor Float32");
					}
				}
				copy_in(s.vector, v.data(), sizeof(float) * v.size());
			}
			s.filled = true;
		}

		// ---- litenn_hip_model ---------------------------------------------------------------
		int check_complete() override
		{
			for (const auto& s : slots)
			{
				if (!s.second.filled)
				{
					return fail(action, "Missing tensor '" + s.first + "'");
				}
			}
			return 0;
		}

		size_t pass_rows() const override { return static_cast<size_t>(max_pass); }
		bool stateful() const override { return true; }

		int ensure_rows(size_t rows) override
		{
			if (rows <= cap_rows)
			{
				return 0;
			}
			decoder_drop_graph(this); // the captured step references the old buffers
			LITENN_HIP_TRY(action, hipStreamSynchronize(stream));
			free_scratch();
			const int n = static_cast<int>(rows);
			size_t absorbed_floats = 0, partial_floats = 0, decay_floats = 0, chunk_floats = 0, kv_rows = 0, xbc_floats = 0;
			for (const LayerState& L : layers)
			{
				for (const MixerState& M : L.mixers)
				{
					const MixerDesc& m = M.desc;
					switch (m.kind)
					{
					case MixerKind::LatentAttention:
						for (int r = 1; r < kExpandMin; ++r)
						{
							absorbed_floats = std::max(absorbed_floats, static_cast<size_t>(r) * m.heads * M.cache.pitch);
							partial_floats = std::max(partial_floats, latent_step_partial_floats(m.heads, r, M.cache.pitch,
							                                                                     latent_step_splits(m.heads, r, m.window)));
						}
						kv_rows = std::max(kv_rows, std::min<size_t>(static_cast<size_t>(context_length), static_cast<size_t>(m.window) - 1 + rows));
						break;
					case MixerKind::GatedLinearAttention:
						decay_floats = std::max(decay_floats, rows * m.heads * m.dim);
						chunk_floats = std::max(chunk_floats, gla_chunk_floats(n, m.heads, m.dim, m.vdim));
						break;
					case MixerKind::GroupedAttention:
						partial_floats = std::max(partial_floats, grouped_step_partial_floats(m.heads, m.vdim, M.splits));
						break;
					case MixerKind::StateSpace: {
						const Ssm shape = ssm_args(M);
						decay_floats = std::max(decay_floats, 2 * rows * m.heads);
						xbc_floats = std::max(xbc_floats, rows * shape.ldx());
						chunk_floats = std::max(chunk_floats, ssm_chunk_floats(n, shape));
						break;
					}
					}
				}
			}
			const size_t operand = f32 ? 4 : 2;
			struct { void** p; size_t bytes; } bufs[] = {
				{ reinterpret_cast<void**>(&x), 4 * rows * desc.width },
				{ reinterpret_cast<void**>(&proj), 4 * rows * ld_proj },
				{ reinterpret_cast<void**>(&y), 4 * rows * ld_y * (rows <= kSplitRows ? kDenseMaxSplits : 1) },
				{ reinterpret_cast<void**>(&q), 4 * rows * ld_q },
				{ reinterpret_cast<void**>(&absorbed), 4 * absorbed_floats },
				{ reinterpret_cast<void**>(&partial), 4 * partial_floats },
				{ reinterpret_cast<void**>(&log_decay), 4 * decay_floats },
				{ reinterpret_cast<void**>(&chunk_states), 4 * chunk_floats },
				{ reinterpret_cast<void**>(&xbc), 4 * xbc_floats },
				{ &h, operand * rows * ld_h },
				{ &mid, operand * rows * ld_mid },
				{ &kv, operand * kv_rows * ld_kv },
			};
			for (auto& b : bufs)
			{
				LITENN_HIP_TRY(action, hipMalloc(b.p, std::max<size_t>(b.bytes, 256)));
			}
			cap_rows = rows;
			return 0;
		}

		int reset_state() override
		{
			for (const LayerState& L : layers)
			{
				for (const MixerState& M : L.mixers)
				{
					if (M.state)
					{
						launch_zero_ints(reinterpret_cast<int*>(M.state), state_floats(M.desc), stream);
					}
				}
			}
			LITENN_HIP_TRY(action, hipGetLastError());
			return 0;
		}

		void forward(const int32_t* ids, size_t rows, size_t logit_rows, unsigned, int past) override
		{
			if (rows < static_cast<size_t>(kRowsMin))
			{
				for (size_t r = 0; r < rows; ++r)
				{
					const bool head = r + logit_rows >= rows;
					forward_token(ids + r, static_cast<int>(r), head ? logits + (r + logit_rows - rows) * vocab : nullptr);
				}
				return;
			}
			forward_rows(ids, static_cast<int>(rows), static_cast<int>(logit_rows), past);
		}

		// ---- single row ---------------------------------------------------------------------
		LatentShape latent_shape(const MixerState& M) const
		{
			const MixerDesc& m = M.desc;
			LatentShape s;
			s.heads = m.heads;
			s.dim = m.dim;
			s.vdim = m.vdim;
			s.window = m.window;
			s.scale = m.scale;
			s.sink = M.sink;
			return s;
		}

		Gla gla_args(const MixerState& M) const
		{
			const MixerDesc& m = M.desc;
			Gla g;
			g.shape.heads = m.heads;
			g.shape.dim = m.dim;
			g.shape.vdim = m.vdim;
			g.shape.q_scale = static_cast<float>(1.0 / std::sqrt(static_cast<double>(m.dim)));
			g.shape.inv_tau = static_cast<float>(1.0 / static_cast<double>(m.tau));
			g.q = proj + M.at_q;
			g.k = proj + M.at_k;
			g.v = proj + M.at_v;
			g.gate = proj + M.at_gate;
			g.a1 = proj + M.at_low;
			g.ld = ld_proj;
			g.a2 = M.a2;
			g.a2_bias = M.a2_bias;
			g.state = M.state;
			g.norm_w = M.head_norm;
			g.eps = desc.eps;
			return g;
		}

		GroupedAttn grouped_args(const MixerState& M) const
		{
			const MixerDesc& m = M.desc;
			GroupedAttn a;
			a.heads = m.heads;
			a.window = m.window;
			a.scale = m.scale;
			a.rot.dims = m.rot_dims;
			a.rot.turns = M.turns;
			a.q_norm = M.q_norm;
			a.k_norm = M.k_norm;
			a.eps = desc.eps;
			a.cache = M.heads;
			a.q = proj + M.at_q;
			a.k = proj + M.at_k;
			a.v = proj + M.at_v;
			a.ld = ld_proj;
			a.q_out = q;
			a.ldq = ld_q;
			a.partial = partial;
			a.splits = M.splits;
			return a;
		}

		Ssm ssm_args(const MixerState& M) const
		{
			const MixerDesc& m = M.desc;
			Ssm a;
			a.heads = m.heads;
			a.vdim = m.vdim;
			a.state = m.state;
			a.groups = m.groups;
			a.taps = m.taps;
			a.conv_w = M.conv_w;
			a.conv_b = M.conv_b;
			a.dt_bias = M.dt_bias;
			a.a_log = M.a_log;
			a.d = M.skip;
			a.in = proj + M.at_in;
			a.ld = ld_proj;
			a.states = M.state;
			a.ring = M.ring;
			a.y = row_ssm;
			a.xbc = xbc;
			a.steps = log_decay;
			a.chunk_states = chunk_states;
			return a;
		}

		// the recurrence's output on its way to the output projection
		GatedNorm gated_norm_args(const MixerState& M) const
		{
			GatedNorm g;
			g.width = M.desc.heads * M.desc.vdim;
			g.parts = M.desc.norm_groups;
			g.norm_w = M.group_norm;
			g.eps = desc.eps;
			g.scale = M.desc.weight;
			return g;
		}

		// grouped attention and state space, alone or side by side, on one token: from proj to row_mid
		void mix_token(const LayerState& L, const Position& pos)
		{
			GroupedAttn attn;
			Ssm ssm;
			GatedNorm norm;
			const MixerState *a = nullptr, *b = nullptr;
			for (const MixerState& M : L.mixers)
			{
				if (M.desc.kind == MixerKind::GroupedAttention)
				{
					a = &M;
					attn = grouped_args(M);
					attn.pos = pos;
				}
				else
				{
					b = &M;
					ssm = ssm_args(M);
					ssm.pos = pos;
					norm = gated_norm_args(M);
					norm.y = row_ssm;
					norm.z = ssm.in;
					norm.out = row_mid + M.at_mid;
				}
			}
			launch_mixer_step(a ? &attn : nullptr, b ? &ssm : nullptr, stream);
			launch_mixer_finish(a ? &attn : nullptr, a ? a->desc.weight : 1.0f, a ? row_mid + a->at_mid : nullptr, b ? &norm : nullptr, stream);
		}

		// the same for a prompt's rows: from proj to mid
		void mix_rows(const LayerState& L, int rows, int past, const Position& pos)
		{
			for (const MixerState& M : L.mixers)
			{
				void* out = static_cast<uint8_t*>(mid) + (f32 ? 4 : 2) * static_cast<size_t>(M.at_mid);
				if (M.desc.kind == MixerKind::GroupedAttention)
				{
					GroupedAttn a = grouped_args(M);
					a.rows = rows;
					a.pos = pos;
					launch_grouped_append(a, stream);
					WindowAttn w = grouped_window(a, past);
					w.out_scale = M.desc.weight;
					w.out = out;
					w.ldo = ld_mid;
					launch_window_attn(w, stream);
				}
				else
				{
					Ssm a = ssm_args(M);
					a.rows = rows;
					a.pos = pos;
					launch_ssm_rows(a, stream);
					GatedNorm g = gated_norm_args(M);
					g.y = a.in;
					g.ldy = ld_proj;
					g.out = out;
					g.ldo = ld_mid;
					g.rows = rows;
					g.f32 = f32;
					launch_gated_norm(g, stream);
				}
			}
		}

		// the token at position counters[0] + offset; logits to `out` unless null
		void forward_token(const int32_t* id, int offset, float* out)
		{
			const Position pos{ d_counters, offset };
			launch_embed_rows(embed, id, 1, turns, pos, xt[0], d_err, stream);
			int at = 0;                // xt[at] is the residual stream, `pending` still to be added
			const float* pending = nullptr; // norm weight of the sublayer output in y
			// norm(x + norm(y)) norm_w through `w`
			const auto enter = [&](const DenseMatrix& w, const float* norm_w, float* dst, bool glu, const ClampedGlu& act, float softcap = 0.0f) {
				DenseRow r;
				r.w = w;
				r.x = xt[at];
				r.y = dst;
				r.softcap = softcap;
				r.prologue = pending || norm_w ? kRowAddNorm : kRowPlain;
				r.norm_w = norm_w;
				r.eps = desc.eps;
				r.glu = glu;
				r.act = act;
				if (pending)
				{
					r.sub = y;
					r.sub_w = pending;
					r.x_out = xt[at ^ 1];
				}
				launch_dense_row(r, stream);
				at ^= pending ? 1 : 0;
				pending = nullptr;
			};
			const auto leave = [&](const DenseMatrix& w, const float* src, const float* after) {
				DenseRow r;
				r.w = w;
				r.x = src;
				r.y = y;
				launch_dense_row(r, stream);
				pending = after;
			};
			for (LayerState& L : layers)
			{
				const MixerState& M = L.mixers[0];
				const MixerDesc& m = M.desc;
				enter(L.in, L.norm1, proj, false, ClampedGlu{});
				if (m.kind == MixerKind::LatentAttention)
				{
					DenseRow r;
					r.w = M.uq;
					r.x = proj + M.at_q;
					r.y = q;
					r.prologue = kRowAddNorm;
					r.norm_w = M.q_norm;
					r.eps = desc.eps;
					launch_dense_row(r, stream);
					LatentStep a;
					a.shape = latent_shape(M);
					a.cache = M.cache;
					a.uk = M.uk;
					a.uv = M.uv;
					a.q = q;
					a.ldq = ld_q;
					a.latent = proj + M.at_latent;
					a.ldl = ld_proj;
					a.latent_w = M.latent_norm;
					a.eps = desc.eps;
					a.gate = proj + M.at_gate;
					a.ldg = ld_proj;
					a.out = row_mid;
					a.ldo = ld_mid;
					a.out_f32 = true;
					a.rows = 1;
					a.pos = pos;
					a.absorbed = absorbed;
					a.partial = partial;
					a.splits = M.splits;
					launch_latent_step(a, stream);
					leave(L.out, row_mid, L.norm1b);
				}
				else if (m.kind == MixerKind::GatedLinearAttention)
				{
					Gla g = gla_args(M);
					g.o = row_mid;
					launch_gla_step(g, stream);
					DenseRow r;
					r.w = L.out;
					r.x = row_mid;
					r.y = y;
					r.prologue = kRowHeadGate;
					r.norm_w = M.head_norm;
					r.gate = proj + M.at_gate;
					r.vdim = m.vdim;
					r.eps = desc.eps;
					launch_dense_row(r, stream);
					pending = L.norm1b;
				}
				else
				{
					mix_token(L, pos);
					leave(L.out, row_mid, L.norm1b);
				}
				if (L.desc.ff > 0)
				{
					enter(L.gate_up, L.norm2, row_mid, true, L.desc.act);
					leave(L.down, row_mid, L.norm2b);
				}
			}
			if (out)
			{
				enter(head, final_norm, out, false, ClampedGlu{}, desc.logit_softcap);
			}
		}

		// ---- many rows ----------------------------------------------------------------------
		void product(const DenseMatrix& w, const void* a, int lda, int rows, void* c, int ldc, int out,
		             const ClampedGlu& act = ClampedGlu{})
		{
			DenseRows d;
			d.w = w;
			d.a = a;
			d.lda = lda;
			d.m = rows;
			d.c = c;
			d.ldc = ldc;
			d.out = out;
			d.f32 = f32;
			d.act = act;
			launch_dense_rows(d, stream);
		}

		void forward_rows(const int32_t* ids, int rows, int logit_rows, int past)
		{
			const Position pos{ d_counters, 0 };
			launch_embed_rows(embed, ids, rows, turns, pos, x, d_err, stream);
			const float* pending = nullptr;
			int parts = 1; // y is the sum of so many buffers
			const size_t part_stride = static_cast<size_t>(rows) * ld_y;
			// x += norm(y) if a sublayer's output is pending, then h = norm(x) norm_w, of rows first ..
			const auto enter = [&](const float* norm_w, int first, int count) {
				AddNorm a;
				a.x = x + static_cast<size_t>(first) * desc.width;
				a.ldx = desc.width;
				if (pending)
				{
					a.sub = y + static_cast<size_t>(first) * ld_y;
					a.ldsub = ld_y;
					a.sub_parts = parts;
					a.sub_stride = part_stride;
					a.sub_w = pending;
					a.x_out = x + static_cast<size_t>(first) * desc.width;
				}
				a.norm_w = norm_w;
				a.out = h;
				a.ldo = ld_h;
				a.rows = count;
				a.width = desc.width;
				a.eps = desc.eps;
				a.f32 = f32;
				launch_add_norm(a, stream);
				pending = nullptr;
			};
			const auto leave = [&](const DenseMatrix& w, const float* after) {
				DenseRows d;
				d.w = w;
				d.a = mid;
				d.lda = ld_mid;
				d.m = rows;
				d.c = y;
				d.ldc = ld_y;
				d.f32 = f32;
				d.splits = parts = !f32 && rows <= kSplitRows ? dense_rows_splits(w, rows) : 1;
				d.split_stride = part_stride;
				launch_dense_rows(d, stream);
				pending = after;
			};
			for (LayerState& L : layers)
			{
				const MixerState& M = L.mixers[0];
				enter(L.norm1, 0, rows);
				product(L.in, h, ld_h, rows, proj, ld_proj, kOutF32);
				if (M.desc.kind == MixerKind::LatentAttention)
				{
					attend(M, rows, past, pos);
				}
				else if (M.desc.kind == MixerKind::GatedLinearAttention)
				{
					Gla g = gla_args(M);
					g.rows = rows;
					g.out = mid;
					g.ldo = ld_mid;
					g.f32 = f32;
					g.log_decay = log_decay;
					g.chunk_states = chunk_states;
					launch_gla_rows(g, stream);
				}
				else
				{
					mix_rows(L, rows, past, pos);
				}
				leave(L.out, L.norm1b);
				if (L.desc.ff > 0)
				{
					enter(L.norm2, 0, rows);
					product(L.gate_up, h, ld_h, rows, mid, ld_mid, kOutGlu, L.desc.act);
					leave(L.down, L.norm2b);
				}
			}
			enter(final_norm, rows - logit_rows, logit_rows);
			DenseRows d;
			d.w = head;
			d.a = h;
			d.lda = ld_h;
			d.m = logit_rows;
			d.c = logits;
			d.ldc = vocab;
			d.f32 = f32;
			d.softcap = desc.logit_softcap;
			launch_dense_rows(d, stream);
		}

		void attend(const MixerState& M, int rows, int past, const Position& pos)
		{
			const MixerDesc& m = M.desc;
			AddNorm n; // queries' latent
			n.x = proj + M.at_q;
			n.ldx = ld_proj;
			n.norm_w = M.q_norm;
			n.out = mid;
			n.ldo = ld_mid;
			n.rows = rows;
			n.width = m.q_rank;
			n.eps = desc.eps;
			n.f32 = f32;
			launch_add_norm(n, stream);
			product(M.uq, mid, ld_mid, rows, q, ld_q, kOutF32);
			launch_latent_append(proj + M.at_latent, ld_proj, M.latent_norm, desc.eps, rows, pos, M.cache, stream);
			if (rows < kExpandMin)
			{
				LatentStep a;
				a.shape = latent_shape(M);
				a.cache = M.cache;
				a.uk = M.uk;
				a.uv = M.uv;
				a.q = q;
				a.ldq = ld_q;
				a.gate = proj + M.at_gate;
				a.ldg = ld_proj;
				a.out = mid;
				a.ldo = ld_mid;
				a.out_f32 = f32;
				a.rows = rows;
				a.pos = pos;
				a.absorbed = absorbed;
				a.partial = partial;
				a.splits = latent_step_splits(m.heads, rows, m.window);
				launch_latent_step(a, stream);
				return;
			}
			const int base = std::max(0, past - m.window + 1);
			const int keys = past + rows - base;
			DenseRows d;
			d.w = M.ukv;
			d.a = M.cache.rows;
			d.lda = M.cache.pitch;
			d.a_first = base % M.cache.ring;
			d.a_ring = M.cache.ring;
			d.m = keys;
			d.c = kv;
			d.ldc = ld_kv;
			d.out = kOutOperand;
			d.f32 = f32;
			launch_dense_rows(d, stream);
			WindowAttn w;
			w.shape = latent_shape(M);
			w.q = q;
			w.ldq = ld_q;
			w.kv = kv;
			w.ldkv = ld_kv;
			w.v_first = M.v_first;
			w.k_head = static_cast<size_t>(m.dim);
			w.v_head = static_cast<size_t>(m.vdim);
			w.keys = keys;
			w.key_base = base;
			w.rows = rows;
			w.q_base = past;
			w.gate = proj + M.at_gate;
			w.ldg = ld_proj;
			w.out = mid;
			w.ldo = ld_mid;
			w.f32 = f32;
			launch_window_attn(w, stream);
		}
	};

	int layered_create(int dev, const LayeredDesc& desc, const litenn_hip_model_tensor* tensors, size_t count, int dtype,
	                   int context_length, litenn_hip_model** out)
	{
		if (dtype != LITENN_BF16 && dtype != LITENN_F32)
		{
			return fail(kAction, "dtype must be BFloat16 or Float32");
		}
		if (context_length <= 0 || context_length > (1 << 30))
		{
			return fail(kAction, "context length must lie in [1, 2^30]");
		}
		DeviceGuard guard(dev);
		if (!guard.ok())
		{
			return fail_hip(kAction, guard.error());
		}
		LayeredModel* m = new LayeredModel();
		try
		{
			m->dev = dev;
			m->action = kAction;
			m->architecture = desc.architecture;
			m->vocab = desc.vocab;
			m->context_length = context_length;
			m->dtype = dtype;
			m->desc = desc;
			m->f32 = dtype == LITENN_F32;
			m->max_pass = std::max(1, env_int("LITENN_HIP_PASS_ROWS", kPassRows));
			const hipError_t e = decoder_init(m);
			if (e != hipSuccess)
			{
				throw std::runtime_error(hipGetErrorString(e));
			}
			m->build();
			for (size_t i = 0; i < count; ++i)
			{
				m->upload(tensors[i]);
			}
			if (m->check_complete() != 0)
			{
				const std::string keep = litenn_hip_last_error();
				decoder_free(m);
				set_error(keep);
				return 1;
			}
			// the uploads and fills ran on the null stream; the model's own stream does not wait for it
			const hipError_t sync = hipDeviceSynchronize();
			if (sync != hipSuccess)
			{
				throw std::runtime_error(hipGetErrorString(sync));
			}
		}
		catch (const std::exception& ex)
		{
			const std::string why = ex.what();
			decoder_free(m);
			return fail(kAction, why);
		}
		*out = m;
		return 0;
	}
} // namespace litenn_hip
