// Mechanisms of the layered decoder for gfx950: token embedding with sinusoidal positions, the
// residual-with-two-norms step, sliding-window attention with a sink over a latent cache (absorbed
// form for few rows, expanded form on the matrix cores for a prompt), and gated linear attention
// (recurrent step, and a chunked form whose contractions run on the Float32 matrix instructions).
// Norms, positions, scores, softmax and everything inside a recurrence are Float32.  The reference
// has no counterpart of these layers.
#include "layer_device.hpp"

#include <algorithm>
#include <cmath>

namespace litenn_hip
{
	namespace
	{
		// ---------------- embedding ----------------------------------------------------------
		__global__ __launch_bounds__(256) void embed_rows_kernel(DenseMatrix table, const int32_t* __restrict__ ids,
		                                                         const double* __restrict__ turns, Position pos,
		                                                         float* __restrict__ x, int* __restrict__ err)
		{
			const int row = blockIdx.x;
			const int id = ids[row];
			if (id < 0 || id >= table.n)
			{
				if (threadIdx.x == 0)
				{
					*err = 1;
				}
				return;
			}
			const uint16_t* t = table.w + static_cast<size_t>(id) * table.pitch;
			float* xr = x + static_cast<size_t>(row) * table.k;
			const double p = static_cast<double>(row_position(pos, row));
			const int i = static_cast<int>(blockIdx.y) * 256 + static_cast<int>(threadIdx.x);
			if (2 * i < table.k)
			{
				float sn = 0.0f, cs = 0.0f;
				if (turns)
				{
					// the angle in turns, reduced in double: what reaches the Float32 sine is below half a turn
					const double t0 = p * turns[i];
					sincosf(static_cast<float>((t0 - rint(t0)) * 6.283185307179586476925), &sn, &cs);
				}
				xr[2 * i] = bf16_to_f32(t[2 * i]) + sn;
				if (2 * i + 1 < table.k)
				{
					xr[2 * i + 1] = bf16_to_f32(t[2 * i + 1]) + cs;
				}
			}
		}

		// ---------------- residual and norms -------------------------------------------------
		// PARTS: how many buffers `sub` may be the sum of (with fewer the last one is loaded again and dropped:
		// the loads must not hang on branches)
		template <typename T, int PARTS>
		__global__ __launch_bounds__(256) void add_norm_kernel(const AddNorm a)
		{
			__shared__ float red[4];
			constexpr int kKept = 16; // values a thread keeps in registers (wider rows are read again)
			const int row = blockIdx.x;
			const float* x = a.x + static_cast<size_t>(row) * a.ldx;
			float kept[kKept], added[kKept], sub_w[kKept], norm_w[kKept];
			float scale_sub = 0.0f;
			const float* sub = a.sub ? a.sub + static_cast<size_t>(row) * a.ldsub : nullptr;
			const auto summed = [&](int i) {
				float v = sub[i];
#pragma unroll
				for (int p = 1; p < PARTS; ++p)
				{
					const float t = sub[min(p, a.sub_parts - 1) * a.sub_stride + i];
					v += p < a.sub_parts ? t : 0.0f;
				}
				return v;
			};
			// every load of the kept part is on its way before the first one is needed
#pragma unroll
			for (int e = 0; e < kKept; ++e)
			{
				const int i = threadIdx.x + 256 * e;
				kept[e] = i < a.width ? x[i] : 0.0f;
				added[e] = sub && i < a.width ? summed(i) : 0.0f;
				sub_w[e] = sub && i < a.width ? a.sub_w[i] : 0.0f;
				norm_w[e] = i < a.width ? (a.norm_w ? a.norm_w[i] : 1.0f) : 0.0f;
			}
			if (sub)
			{
				float ss = 0.0f;
#pragma unroll
				for (int e = 0; e < kKept; ++e)
				{
					ss = fmaf(added[e], added[e], ss);
				}
				for (int i = threadIdx.x + 256 * kKept; i < a.width; i += 256)
				{
					const float v = summed(i);
					ss = fmaf(v, v, ss);
				}
				scale_sub = 1.0f / sqrtf(block_sum256(ss, red) / static_cast<float>(a.width) + a.eps);
			}
			const auto value = [&](int i) { return sub ? x[i] + summed(i) * scale_sub * a.sub_w[i] : x[i]; };
			float ss = 0.0f;
#pragma unroll
			for (int e = 0; e < kKept; ++e)
			{
				kept[e] += added[e] * scale_sub * sub_w[e];
				ss = fmaf(kept[e], kept[e], ss);
			}
			for (int i = threadIdx.x + 256 * kKept; i < a.width; i += 256)
			{
				const float v = value(i);
				ss = fmaf(v, v, ss);
			}
			const float scale = a.norm_w ? 1.0f / sqrtf(block_sum256(ss, red) / static_cast<float>(a.width) + a.eps) : 1.0f;
			float* x_out = a.x_out ? a.x_out + static_cast<size_t>(row) * a.ldx : nullptr;
			T* out = static_cast<T*>(a.out) + static_cast<size_t>(row) * a.ldo;
			const auto put = [&](int i, float v, float w) {
				if (x_out)
				{
					x_out[i] = v;
				}
				operand_store(out + i, v * scale * w);
			};
#pragma unroll
			for (int e = 0; e < kKept; ++e)
			{
				const int i = threadIdx.x + 256 * e;
				if (i < a.width)
				{
					put(i, kept[e], norm_w[e]);
				}
			}
			for (int i = threadIdx.x + 256 * kKept; i < a.width; i += 256)
			{
				put(i, value(i), a.norm_w ? a.norm_w[i] : 1.0f);
			}
		}

		// ---------------- latent cache -------------------------------------------------------
		// norm(src) w -> one cache row, by 256 threads
		template <typename T>
		__device__ __forceinline__ void append_latent(const float* src, const float* w, float eps, const LatentCache& c,
		                                              int position, float* red)
		{
			float ss = 0.0f;
			for (int i = threadIdx.x; i < c.rank; i += 256)
			{
				ss = fmaf(src[i], src[i], ss);
			}
			const float scale = 1.0f / sqrtf(block_sum256(ss, red) / static_cast<float>(c.rank) + eps);
			T* dst = static_cast<T*>(c.rows) + static_cast<size_t>(position % c.ring) * c.pitch;
			for (int i = threadIdx.x; i < c.rank; i += 256)
			{
				operand_store(dst + i, src[i] * scale * w[i]);
			}
		}

		template <typename T>
		__global__ __launch_bounds__(256) void latent_append_kernel(const float* __restrict__ src, int ld,
		                                                            const float* __restrict__ w, float eps, Position pos,
		                                                            LatentCache cache)
		{
			__shared__ float red[4];
			append_latent<T>(src + static_cast<size_t>(blockIdx.x) * ld, w, eps, cache,
			                 row_position(pos, static_cast<int>(blockIdx.x)), red);
		}

		// ---------------- attention in the latent space (few rows) -----------------------------
		constexpr int kAbsorbSlice = 128; // latent columns of a workgroup

		// absorbed[row, h, :] = scale W_uk[h]^T q[row, h]; the last workgroup of a row appends its latent
		template <typename T>
		__global__ __launch_bounds__(256) void latent_absorb_kernel(const LatentStep a)
		{
			__shared__ float qs[256];
			__shared__ float sums[16][kAbsorbSlice + 4];
			__shared__ float red[4];
			const int row = blockIdx.y;
			const int slices = (a.cache.pitch + kAbsorbSlice - 1) / kAbsorbSlice;
			const int h = static_cast<int>(blockIdx.x) / slices;
			if (h == a.shape.heads)
			{
				if (a.latent)
				{
					append_latent<T>(a.latent + static_cast<size_t>(row) * a.ldl, a.latent_w, a.eps, a.cache,
					                 row_position(a.pos, row), red);
				}
				return;
			}
			const int slice = static_cast<int>(blockIdx.x) % slices;
			const int piece = threadIdx.x & 15, group = threadIdx.x >> 4;
			const int r0 = slice * kAbsorbSlice + piece * 8;
			const bool inside = r0 < a.cache.pitch;
			const float* q = a.q + static_cast<size_t>(row) * a.ldq + static_cast<size_t>(h) * a.shape.dim;
			float acc[8];
#pragma unroll
			for (int e = 0; e < 8; ++e)
			{
				acc[e] = 0.0f;
			}
			for (int first = 0; first < a.shape.dim; first += 256)
			{
				const int count = min(256, a.shape.dim - first);
				__syncthreads();
				if (static_cast<int>(threadIdx.x) < count)
				{
					qs[threadIdx.x] = q[first + threadIdx.x];
				}
				__syncthreads();
				if (inside)
				{
					const uint16_t* w = a.uk.w + static_cast<size_t>(h * a.shape.dim + first) * a.uk.pitch + r0;
#pragma unroll 4
					for (int d = group; d < count; d += 16)
					{
						const u32x4 v = *reinterpret_cast<const u32x4*>(w + static_cast<size_t>(d) * a.uk.pitch);
						const float qd = qs[d];
#pragma unroll
						for (int e = 0; e < 4; ++e)
						{
							acc[2 * e] = fmaf(qd, __uint_as_float(v[e] << 16), acc[2 * e]);
							acc[2 * e + 1] = fmaf(qd, __uint_as_float(v[e] & 0xffff0000u), acc[2 * e + 1]);
						}
					}
				}
			}
#pragma unroll
			for (int e = 0; e < 8; ++e)
			{
				sums[group][piece * 8 + e] = acc[e];
			}
			__syncthreads();
			const int r = slice * kAbsorbSlice + static_cast<int>(threadIdx.x);
			if (threadIdx.x < kAbsorbSlice && r < a.cache.pitch)
			{
				float t = 0.0f;
#pragma unroll
				for (int g = 0; g < 16; ++g)
				{
					t += sums[g][threadIdx.x];
				}
				a.absorbed[(static_cast<size_t>(row) * a.shape.heads + h) * a.cache.pitch + r] = t * a.shape.scale;
			}
		}

		// A workgroup takes four heads (one per wavefront) over one split of the visible positions, in tiles
		// of kLatentTile cached rows staged in LDS as Float32; per split and head it leaves the running
		// maximum, the sum of weights and the weighted sum of latents.
		constexpr int kLatentTile = 16, kLatentHeads = 4, kLatentMaxRank = 1024, kLatentMaxSplits = 64;

		template <typename T>
		__global__ __launch_bounds__(256) void latent_step_kernel(const LatentStep a)
		{
			extern __shared__ __attribute__((aligned(16))) float latent_lds[];
			const int pitch = a.cache.pitch, stride = pitch + 4;
			float* const tile = latent_lds;                       // [kLatentTile][stride]
			float* const qa = tile + kLatentTile * stride;        // [kLatentHeads][pitch]
			float* const weights = qa + kLatentHeads * pitch;     // [kLatentHeads][kLatentTile]
			const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
			const int row = blockIdx.z, split = blockIdx.y;
			const int h = static_cast<int>(blockIdx.x) * kLatentHeads + wave;
			const int hc = min(h, a.shape.heads - 1);
			const int last = row_position(a.pos, row);
			const int first = max(0, last - a.shape.window + 1);
			const int tiles = (last - first) / kLatentTile + 1;
			const int per = (tiles + a.splits - 1) / a.splits;
			const int t0 = split * per, t1 = min(tiles, t0 + per);
			const T* const cache = static_cast<const T*>(a.cache.rows);
			// kPer threads per row of a tile, 16 bytes each at a time; a row's first kAhead pieces per thread are
			// requested before anything waits
			constexpr int E = 16 / sizeof(T), kAhead = 4, kPer = 256 / kLatentTile, kStep = kPer * E;
			const int my_key = threadIdx.x / kPer, c0 = (threadIdx.x % kPer) * E;
			const auto row_of = [&](int base) {
				const int count = min(kLatentTile, last - base + 1);
				return cache + static_cast<size_t>((base + min(my_key, count - 1)) % a.cache.ring) * pitch + c0;
			};
			u32x4 ahead[kAhead];
			const auto request = [&](int base) {
				const T* p = row_of(base);
#pragma unroll
				for (int i = 0; i < kAhead; ++i)
				{
					ahead[i] = *reinterpret_cast<const u32x4*>(p + (c0 + kStep * i < pitch ? kStep * i : -c0));
				}
			};
			if (t0 < t1)
			{
				request(first + t0 * kLatentTile);
			}
			const float* src = a.absorbed + (static_cast<size_t>(row) * a.shape.heads + hc) * pitch;
#pragma unroll 8
			for (int i = lane; i < pitch; i += 64)
			{
				qa[wave * pitch + i] = i < a.cache.rank ? src[i] : 0.0f;
			}

			constexpr int kCols = kLatentMaxRank / 256;
			floatx4 o[kCols];
#pragma unroll
			for (int c = 0; c < kCols; ++c)
			{
				o[c] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
			}
			float run_m = -INFINITY, run_l = 0.0f;
			for (int t = t0; t < t1; ++t)
			{
				const int base = first + t * kLatentTile;
				const int count = min(kLatentTile, last - base + 1);
				__syncthreads();
				{
					float* dst = &tile[my_key * stride + c0];
					const auto store = [&](int c, u32x4 w) {
						if constexpr (sizeof(T) == 2)
						{
							*reinterpret_cast<floatx4*>(dst + c) = floatx4{ __uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u),
								                                            __uint_as_float(w.y << 16), __uint_as_float(w.y & 0xffff0000u) };
							*reinterpret_cast<floatx4*>(dst + c + 4) = floatx4{ __uint_as_float(w.z << 16), __uint_as_float(w.z & 0xffff0000u),
								                                                __uint_as_float(w.w << 16), __uint_as_float(w.w & 0xffff0000u) };
						}
						else
						{
							*reinterpret_cast<u32x4*>(dst + c) = w;
						}
					};
#pragma unroll
					for (int i = 0; i < kAhead; ++i)
					{
						if (c0 + kStep * i < pitch)
						{
							store(kStep * i, ahead[i]);
						}
					}
					const T* p = row_of(base);
					for (int c = kStep * kAhead; c0 + c < pitch; c += kStep)
					{
						store(c, *reinterpret_cast<const u32x4*>(p + c));
					}
					if (t + 1 < t1)
					{
						request(base + kLatentTile);
					}
				}
				__syncthreads();
				// scores: kParts lanes per key, each a share of the latent
				constexpr int kParts = 64 / kLatentTile;
				const int key = lane % kLatentTile, part = lane / kLatentTile;
				float acc = 0.0f;
				{
					const float* kr = &tile[key * stride];
					const float* qr = &qa[wave * pitch];
					const int share = pitch / kParts; // the pitch is a multiple of 64
#pragma unroll 8
					for (int c = part * share; c < (part + 1) * share; c += 4)
					{
						const floatx4 kv = *reinterpret_cast<const floatx4*>(kr + c);
						const floatx4 qv = *reinterpret_cast<const floatx4*>(qr + c);
						acc = fmaf(kv.x, qv.x, acc);
						acc = fmaf(kv.y, qv.y, acc);
						acc = fmaf(kv.z, qv.z, acc);
						acc = fmaf(kv.w, qv.w, acc);
					}
				}
#pragma unroll
				for (int off = kLatentTile; off < 64; off *= 2)
				{
					acc += __shfl_xor(acc, off, 64);
				}
				const float score = key < count ? acc : -INFINITY;
				const float new_m = fmaxf(run_m, wave_max(score));
				const float corr = run_m == -INFINITY ? 0.0f : expf(run_m - new_m);
				const float p = expf(score - new_m);
				run_l = run_l * corr + wave_sum(part == 0 ? p : 0.0f);
				run_m = new_m;
				if (part == 0)
				{
					weights[wave * kLatentTile + key] = p;
				}
				// written and read by this wavefront only, in order
				__builtin_amdgcn_wave_barrier();
#pragma unroll
				for (int c = 0; c < kCols; ++c)
				{
					o[c] *= corr;
				}
#pragma unroll 4
				for (int kk = 0; kk < kLatentTile; ++kk) // the tile's unused rows repeat its last one, with weight zero
				{
					const float w = weights[wave * kLatentTile + kk];
#pragma unroll
					for (int c = 0; c < kCols; ++c)
					{
						const int col = c * 256 + lane * 4;
						if (col < pitch)
						{
							o[c] += w * *reinterpret_cast<const floatx4*>(&tile[kk * stride + col]);
						}
					}
				}
			}
			if (h >= a.shape.heads)
			{
				return;
			}
			const size_t slot = (static_cast<size_t>(row) * a.splits + split) * a.shape.heads + h;
			float* dst = a.partial + slot * (pitch + 4);
#pragma unroll
			for (int c = 0; c < kCols; ++c)
			{
				const int col = c * 256 + lane * 4;
				if (col < pitch)
				{
					*reinterpret_cast<floatx4*>(dst + col) = o[c];
				}
			}
			if (lane == 0)
			{
				dst[pitch] = run_m;
				dst[pitch + 1] = run_l;
			}
		}

		// Merges the splits (and the sink), takes the result through W_uv, applies the gate.  A workgroup
		// makes kValueSlice outputs of one head.
		constexpr int kValueSlice = 32, kValueThreads = 512;

		template <typename T>
		__global__ __launch_bounds__(kValueThreads) void latent_value_kernel(const LatentStep a)
		{
			__shared__ __attribute__((aligned(16))) float o[kLatentMaxRank];
			__shared__ float weight[kLatentMaxSplits], sum;
			__shared__ __attribute__((aligned(16))) float shares[4 * kValueThreads];
			const int pitch = a.cache.pitch;
			const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
			const int slices = (a.shape.vdim + kValueSlice - 1) / kValueSlice;
			const int h = static_cast<int>(blockIdx.x) / slices, slice = static_cast<int>(blockIdx.x) % slices;
			const int row = blockIdx.y;
			const size_t step = static_cast<size_t>(a.shape.heads) * (pitch + 4);
			const float* part = a.partial + (static_cast<size_t>(row) * a.splits * a.shape.heads + h) * (pitch + 4);
			// Everything this workgroup reads is requested before anything waits: the splits' maxima and sums, its
			// first latents (four columns per thread; the threads left over by one row of columns share out the
			// splits), this wavefront's rows of W_uv (a rank of up to 512 is one piece per lane) and its gates.
			static_assert(kLatentMaxSplits == 64, "one lane per split");
			const float split_m = lane < a.splits ? part[lane * step + pitch] : -INFINITY;
			const float split_l = lane < a.splits ? part[lane * step + pitch + 1] : 0.0f;
			const int quads = pitch >> 2, groups = kValueThreads / quads;
			const int quad = static_cast<int>(threadIdx.x) % quads, group = static_cast<int>(threadIdx.x) / quads;
			constexpr int kAhead = 16;
			floatx4 ahead[kAhead];
#pragma unroll
			for (int i = 0; i < kAhead; ++i)
			{
				ahead[i] = *reinterpret_cast<const floatx4*>(part + min(group + i * groups, a.splits - 1) * step + 4 * quad);
			}
			constexpr int kWaves = kValueThreads / 64, kRows = kValueSlice / kWaves;
			u32x4 first[kRows];
#pragma unroll
			for (int i = 0; i < kRows; ++i)
			{
				const int e = min(slice * kValueSlice + wave + kWaves * i, a.shape.vdim - 1);
				first[i] = *reinterpret_cast<const u32x4*>(a.uv.w + static_cast<size_t>(h * a.shape.vdim + e) * a.uv.pitch +
				                                           (lane * 8 < pitch ? lane * 8 : 0));
			}
			float gates = 0.0f; // lane i: row i
			if (a.gate && lane < kRows)
			{
				const int e = min(slice * kValueSlice + wave + kWaves * lane, a.shape.vdim - 1);
				gates = a.gate[static_cast<size_t>(row) * a.ldg + h * a.shape.vdim + e];
			}
			// weights of the splits (one without a visible position has maximum -inf and weight 0)
			if (wave == 0)
			{
				const float sink = a.shape.sink ? a.shape.sink[h] : -INFINITY;
				const float top = fmaxf(wave_max(split_m), sink);
				const float w = expf(split_m - top);
				const float all = wave_sum(w * split_l);
				weight[lane] = w;
				if (lane == 0)
				{
					sum = all + expf(sink - top);
				}
			}
			__syncthreads();
			if (group < groups)
			{
				floatx4 v = { 0.0f, 0.0f, 0.0f, 0.0f };
#pragma unroll
				for (int i = 0; i < kAhead; ++i)
				{
					const int s = group + i * groups;
					v += (s < a.splits ? weight[min(s, kLatentMaxSplits - 1)] : 0.0f) * ahead[i];
				}
				for (int s = group + kAhead * groups; s < a.splits; s += groups)
				{
					v += weight[s] * *reinterpret_cast<const floatx4*>(part + s * step + 4 * quad);
				}
				*reinterpret_cast<floatx4*>(&shares[(group * quads + quad) * 4]) = v;
			}
			__syncthreads();
			const float inv = 1.0f / sum;
			for (int c = threadIdx.x; c < pitch; c += kValueThreads)
			{
				float t = 0.0f;
				for (int i = 0; i < groups; ++i)
				{
					t += shares[i * pitch + c];
				}
				o[c] = c < a.cache.rank ? t * inv : 0.0f;
			}
			__syncthreads();
#pragma unroll
			for (int i = 0; i < kRows; ++i)
			{
				const int e = slice * kValueSlice + wave + kWaves * i;
				if (e >= a.shape.vdim)
				{
					break;
				}
				const uint16_t* w = a.uv.w + static_cast<size_t>(h * a.shape.vdim + e) * a.uv.pitch;
				float acc = 0.0f;
				for (int r = lane * 8; r < pitch; r += 512)
				{
					const u32x4 x = r < 512 ? first[i] : *reinterpret_cast<const u32x4*>(w + r);
					const floatx4 o0 = *reinterpret_cast<const floatx4*>(o + r);
					const floatx4 o1 = *reinterpret_cast<const floatx4*>(o + r + 4);
					acc = fmaf(__uint_as_float(x.x << 16), o0.x, acc);
					acc = fmaf(__uint_as_float(x.x & 0xffff0000u), o0.y, acc);
					acc = fmaf(__uint_as_float(x.y << 16), o0.z, acc);
					acc = fmaf(__uint_as_float(x.y & 0xffff0000u), o0.w, acc);
					acc = fmaf(__uint_as_float(x.z << 16), o1.x, acc);
					acc = fmaf(__uint_as_float(x.z & 0xffff0000u), o1.y, acc);
					acc = fmaf(__uint_as_float(x.w << 16), o1.z, acc);
					acc = fmaf(__uint_as_float(x.w & 0xffff0000u), o1.w, acc);
				}
				acc = wave_sum(acc);
				const float gate = __shfl(gates, i, 64);
				if (lane == 0)
				{
					if (a.gate)
					{
						acc *= sigmoid_f32(gate);
					}
					operand_store(static_cast<T*>(a.out) + static_cast<size_t>(row) * a.ldo + h * a.shape.vdim + e, acc);
				}
			}
		}

		// ---------------- windowed attention over expanded keys and values -----------------------
		// the row of the buffer that holds key row r
		__device__ __forceinline__ int window_row(const WindowAttn& a, int r)
		{
			r += a.kv_first;
			return a.kv_ring > 0 && r >= a.kv_ring ? r - a.kv_ring : r;
		}

		// One wavefront per (query row, head), any head size up to 1024; Float32 arithmetic.
		constexpr int kRowAttnMaxDim = 1024;

		template <typename T>
		__global__ __launch_bounds__(64) void window_attn_row_kernel(const WindowAttn a)
		{
			__shared__ float qs[kRowAttnMaxDim];
			__shared__ float ws[64];
			const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
			const int dim = a.shape.dim, vdim = a.shape.vdim;
			const size_t k_at = h / a.shape.share * a.k_head, v_at = a.v_first + h / a.shape.share * a.v_head;
			for (int d = lane; d < dim; d += 64)
			{
				qs[d] = a.q[static_cast<size_t>(row) * a.ldq + h * dim + d];
			}
			__syncthreads();
			const int pos = a.q_base + row;
			const int first = max(a.key_base, pos - a.shape.window + 1), last = min(pos, a.key_base + a.keys - 1);
			const T* kv = static_cast<const T*>(a.kv);
			constexpr int kCols = kRowAttnMaxDim / 64;
			float o[kCols];
#pragma unroll
			for (int c = 0; c < kCols; ++c)
			{
				o[c] = 0.0f;
			}
			float run_m = -INFINITY, run_l = 0.0f;
			for (int base = first; base <= last; base += 64)
			{
				const int key = base + lane;
				float score = -INFINITY;
				if (key <= last)
				{
					const T* k = kv + static_cast<size_t>(window_row(a, key - a.key_base)) * a.ldkv + k_at;
					float acc = 0.0f;
					for (int d = 0; d < dim; ++d)
					{
						acc = fmaf(qs[d], operand_load(k + d), acc);
					}
					score = acc * a.shape.scale;
				}
				const float new_m = fmaxf(run_m, wave_max(score));
				const float corr = run_m == -INFINITY ? 0.0f : expf(run_m - new_m);
				const float p = key <= last ? expf(score - new_m) : 0.0f;
				run_l = run_l * corr + wave_sum(p);
				run_m = new_m;
				__syncthreads();
				ws[lane] = p;
				__syncthreads();
				const int count = min(64, last - base + 1);
#pragma unroll
				for (int c = 0; c < kCols; ++c)
				{
					const int e = c * 64 + lane;
					if (e < vdim)
					{
						float t = o[c] * corr;
						const T* v = kv + v_at + e;
						for (int i = 0; i < count; ++i)
						{
							t = fmaf(ws[i], operand_load(v + static_cast<size_t>(window_row(a, base - a.key_base + i)) * a.ldkv), t);
						}
						o[c] = t;
					}
				}
			}
			float top = run_m, total = run_l, weight = 1.0f;
			if (a.shape.sink)
			{
				const float sink = a.shape.sink[h];
				top = fmaxf(run_m, sink);
				weight = expf(run_m - top);
				total = run_l * weight + expf(sink - top);
			}
#pragma unroll
			for (int c = 0; c < kCols; ++c)
			{
				const int e = c * 64 + lane;
				if (e < vdim)
				{
					float v = o[c] * weight / total * a.out_scale;
					if (a.gate)
					{
						v *= sigmoid_f32(a.gate[static_cast<size_t>(row) * a.ldg + h * vdim + e]);
					}
					operand_store(static_cast<T*>(a.out) + static_cast<size_t>(row) * a.ldo + h * vdim + e, v);
				}
			}
		}

		// Matrix-core form: a workgroup takes 64 query rows of one head (16 per wavefront) and walks the
		// keys any of them sees in tiles of 64, staged in LDS (keys row-major, values transposed).  Both
		// products are formed transposed (keys x queries, value dimensions x queries), so that a query
		// stays in one lane column: the softmax weights leave the first product in the register layout
		// the second one takes, and the running maximum and sum live beside the outputs.  DK and DV are the
		// head sizes rounded up; what lies beyond the true sizes is zero in LDS and in the queries.
		constexpr int kWinQ = 64, kWinKeys = 64, kWinVStride = 72;

		template <int DK, int DV>
		__global__ __launch_bounds__(256) void window_attn_tile_kernel(const WindowAttn a)
		{
			constexpr int KS = DK + 8;
			extern __shared__ __attribute__((aligned(16))) uint16_t win_lds[];
			uint16_t* const k_lds = win_lds;                 // [kWinKeys][KS]
			uint16_t* const v_lds = win_lds + kWinKeys * KS; // [DV][kWinVStride]
			const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
			const int j = lane & 15, g = lane >> 4;
			const int h = blockIdx.x;
			const int tile = static_cast<int>(gridDim.y) - 1 - static_cast<int>(blockIdx.y);
			const int dim = a.shape.dim, vdim = a.shape.vdim;
			const int q_first = tile * kWinQ;
			const int my_q = q_first + 16 * wave + j;
			const int my_row = min(my_q, a.rows - 1);
			const int my_pos = a.q_base + my_row;
			// key rows (relative to key_base) any query of the tile sees
			const int lo = max(0, a.q_base + q_first - a.shape.window + 1 - a.key_base);
			const int hi = min(a.keys, a.q_base + min(q_first + kWinQ, a.rows) - a.key_base);
			const uint16_t* const keys = static_cast<const uint16_t*>(a.kv) + h / a.shape.share * a.k_head;
			const uint16_t* const values = static_cast<const uint16_t*>(a.kv) + a.v_first + h / a.shape.share * a.v_head;
			const float scale2 = a.shape.scale * kLog2e; // scores in units of log 2

			bf16x8 q_frag[DK / 32];
			{
				const float* q = a.q + static_cast<size_t>(my_row) * a.ldq + static_cast<size_t>(h) * dim;
#pragma unroll
				for (int st = 0; st < DK / 32; ++st)
				{
					uint32_t w[4];
#pragma unroll
					for (int e = 0; e < 4; ++e)
					{
						const int d = 32 * st + 8 * g + 2 * e;
						w[e] = d < dim ? pack_bf16(q[d], d + 1 < dim ? q[d + 1] : 0.0f) : 0u;
					}
					q_frag[st] = __builtin_bit_cast(bf16x8, u32x4{ w[0], w[1], w[2], w[3] });
				}
			}
			floatx4 o[DV / 16];
#pragma unroll
			for (int b = 0; b < DV / 16; ++b)
			{
				o[b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
			}
			float run_m = -INFINITY, run_l = 0.0f;
			constexpr int KP = DK / 8, VP = DV / 8;              // 16-byte pieces of a row
			constexpr int KN = kWinKeys * KP / 256, VN = VP / 4; // pieces a thread stages
			u32x4 kr[KN], vr[VN];
			const int v_key = tid & 63, v_piece = (tid >> 6) * VN;
			const auto request = [&](int base) {
#pragma unroll
				for (int i = 0; i < KN; ++i)
				{
					const int c = tid + 256 * i, key = min(base + c / KP, hi - 1), d = (c % KP) * 8;
					kr[i] = d < dim ? *reinterpret_cast<const u32x4*>(keys + static_cast<size_t>(window_row(a, key)) * a.ldkv + d)
					                : u32x4{ 0u, 0u, 0u, 0u };
				}
				const uint16_t* v = values + static_cast<size_t>(window_row(a, min(base + v_key, hi - 1))) * a.ldkv;
#pragma unroll
				for (int i = 0; i < VN; ++i)
				{
					const int e = (v_piece + i) * 8;
					vr[i] = e < vdim ? *reinterpret_cast<const u32x4*>(v + e) : u32x4{ 0u, 0u, 0u, 0u };
				}
			};
			request(lo);
			for (int base = lo; base < hi; base += kWinKeys)
			{
				__syncthreads(); // the previous tile has been consumed
#pragma unroll
				for (int i = 0; i < KN; ++i)
				{
					const int c = tid + 256 * i;
					*reinterpret_cast<u32x4*>(&k_lds[(c / KP) * KS + (c % KP) * 8]) = kr[i];
				}
#pragma unroll
				for (int i = 0; i < VN; ++i)
				{
#pragma unroll
					for (int e = 0; e < 4; ++e)
					{
						const int d = (v_piece + i) * 8 + 2 * e;
						v_lds[d * kWinVStride + v_key] = static_cast<uint16_t>(vr[i][e] & 0xffffu);
						v_lds[(d + 1) * kWinVStride + v_key] = static_cast<uint16_t>(vr[i][e] >> 16);
					}
				}
				if (base + kWinKeys < hi)
				{
					request(base + kWinKeys);
				}
				__syncthreads();
				// lane (j, g) gets keys base + 16 b + 4 g + 0..3 of query j
				floatx4 s[4];
#pragma unroll
				for (int b = 0; b < 4; ++b)
				{
					s[b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
#pragma unroll
					for (int st = 0; st < DK / 32; ++st)
					{
						const bf16x8 kf = *reinterpret_cast<const bf16x8*>(&k_lds[(16 * b + j) * KS + 32 * st + 8 * g]);
						s[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, q_frag[st], s[b], 0, 0, 0);
					}
				}
				const int pos0 = a.key_base + base + 4 * g;
				float sv[4][4];
				float top = -INFINITY;
#pragma unroll
				for (int b = 0; b < 4; ++b)
				{
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
						const int back = my_pos - (pos0 + 16 * b + r);
						sv[b][r] = back >= 0 && back < a.shape.window ? s[b][r] * scale2 : -INFINITY;
						top = fmaxf(top, sv[b][r]);
					}
				}
				top = fmaxf(top, __shfl_xor(top, 16, 64));
				top = fmaxf(top, __shfl_xor(top, 32, 64));
				// a tile may hold no visible key of this query: exponents then take 0 as the maximum
				const float new_m = fmaxf(run_m, top);
				const float ref_m = new_m == -INFINITY ? 0.0f : new_m;
				const float corr = exp2_f32(run_m - ref_m);
				run_m = new_m;
				float sum = 0.0f;
				bf16x8 p_frag[2];
#pragma unroll
				for (int ks = 0; ks < 2; ++ks)
				{
					float p[8];
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
						p[r] = exp2_f32(sv[2 * ks][r] - ref_m);
						p[4 + r] = exp2_f32(sv[2 * ks + 1][r] - ref_m);
					}
#pragma unroll
					for (int e = 0; e < 8; ++e)
					{
						sum += p[e];
					}
					p_frag[ks] = __builtin_bit_cast(bf16x8, u32x4{ pack_bf16(p[0], p[1]), pack_bf16(p[2], p[3]),
					                                               pack_bf16(p[4], p[5]), pack_bf16(p[6], p[7]) });
				}
				run_l = fmaf(run_l, corr, sum);
				// contraction index 8 g + e of step ks stands for key 16 (2 ks) + 4 g + e (e < 4) and key
				// 16 (2 ks + 1) + 4 g + e - 4 (e >= 4)
#pragma unroll
				for (int b = 0; b < DV / 16; ++b)
				{
					o[b] *= corr;
#pragma unroll
					for (int ks = 0; ks < 2; ++ks)
					{
						const uint16_t* col = &v_lds[(16 * b + j) * kWinVStride + 32 * ks + 4 * g];
						const uint2 x = *reinterpret_cast<const uint2*>(col), y = *reinterpret_cast<const uint2*>(col + 16);
						const bf16x8 vf = __builtin_bit_cast(bf16x8, u32x4{ x.x, x.y, y.x, y.y });
						o[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p_frag[ks], o[b], 0, 0, 0);
					}
				}
			}
			run_l += __shfl_xor(run_l, 16, 64);
			run_l += __shfl_xor(run_l, 32, 64);
			if (my_q >= a.rows)
			{
				return;
			}
			float weight = 1.0f, total = run_l;
			if (a.shape.sink)
			{
				const float sink = a.shape.sink[h] * kLog2e;
				const float all_m = fmaxf(run_m, sink);
				weight = exp2_f32(run_m - all_m);
				total = run_l * weight + exp2_f32(sink - all_m);
			}
			const float inv = weight / total * a.out_scale;
			uint16_t* out = static_cast<uint16_t*>(a.out) + static_cast<size_t>(my_q) * a.ldo + static_cast<size_t>(h) * vdim;
			const float* gate = a.gate ? a.gate + static_cast<size_t>(my_q) * a.ldg + static_cast<size_t>(h) * vdim : nullptr;
#pragma unroll
			for (int b = 0; b < DV / 16; ++b)
			{
				const int e = 16 * b + 4 * g;
				if (e < vdim)
				{
					floatx4 v = o[b] * inv;
					if (gate)
					{
#pragma unroll
						for (int r = 0; r < 4; ++r)
						{
							v[r] *= e + r < vdim ? sigmoid_f32(gate[e + r]) : 0.0f;
						}
					}
					if ((vdim & 3) == 0 && (reinterpret_cast<size_t>(a.out) & 7) == 0)
					{
						*reinterpret_cast<uint2*>(out + e) = make_uint2(pack_bf16(v.x, v.y), pack_bf16(v.z, v.w));
					}
					else
					{
#pragma unroll
						for (int r = 0; r < 4; ++r)
						{
							if (e + r < vdim)
							{
								out[e + r] = to_bf16(v[r]);
							}
						}
					}
				}
			}
		}

		// ---------------- gated linear attention ---------------------------------------------------
		__device__ __forceinline__ float log_sigmoid_f32(float z)
		{
			return fminf(z, 0.0f) - log1pf(expf(-fabsf(z)));
		}

		// one row of W_a2 times the rank-wide vector `a1`
		__device__ __forceinline__ float low_rank_dot(const DenseMatrix& a2, int channel, const float* a1)
		{
			const uint16_t* w = a2.w + static_cast<size_t>(channel) * a2.pitch;
			float z = 0.0f;
			for (int r = 0; r < a2.k; ++r)
			{
				z = fmaf(bf16_to_f32(w[r]), a1[r], z);
			}
			return z;
		}

		// log_decay[t, c] = log2 sigmoid(W_a2 a1[t] + bias)[c] / tau
		constexpr int kDecayRows = 16, kDecayMaxRank = 512;

		__global__ __launch_bounds__(256) void gla_decay_kernel(const Gla a)
		{
			__shared__ float a1[kDecayRows][kDecayMaxRank];
			const int channels = a.shape.heads * a.shape.dim, rank = a.a2.k;
			const int row0 = blockIdx.y * kDecayRows;
			const int count = min(kDecayRows, a.rows - row0);
			for (int i = threadIdx.x; i < count * rank; i += 256)
			{
				a1[i / rank][i % rank] = a.a1[static_cast<size_t>(row0 + i / rank) * a.ld + i % rank];
			}
			__syncthreads();
			const int c = blockIdx.x * 256 + threadIdx.x;
			if (c >= channels)
			{
				return;
			}
			const uint16_t* w = a.a2.w + static_cast<size_t>(c) * a.a2.pitch;
			float z[kDecayRows];
			const float bias = a.a2_bias[c];
#pragma unroll
			for (int t = 0; t < kDecayRows; ++t)
			{
				z[t] = bias;
			}
			for (int r = 0; r < rank; ++r)
			{
				const float wr = bf16_to_f32(w[r]);
#pragma unroll
				for (int t = 0; t < kDecayRows; ++t)
				{
					z[t] = fmaf(wr, a1[t][r], z[t]);
				}
			}
#pragma unroll
			for (int t = 0; t < kDecayRows; ++t)
			{
				if (t < count)
				{
					a.log_decay[static_cast<size_t>(row0 + t) * channels + c] = log_sigmoid_f32(z[t]) * (a.shape.inv_tau * kLog2e);
				}
			}
		}

		// One token: S <- diag(alpha) S + k v^T, o = S^T q.  A workgroup takes kStepCols value columns of one
		// head; a thread holds RPT rows (32 apart) of four columns.
		constexpr int kStepCols = 32, kGlaMaxDim = 512;

		template <int RPT>
		__global__ __launch_bounds__(256) void gla_step_kernel(const Gla a)
		{
			__shared__ float alpha[32 * RPT], ks[32 * RPT], qs[32 * RPT];
			__shared__ __attribute__((aligned(16))) float sums[32][kStepCols + 4];
			const int dim = a.shape.dim, vdim = a.shape.vdim, pitch = gla_state_pitch(vdim);
			const int h = blockIdx.x, tid = threadIdx.x;
			const int e = static_cast<int>(blockIdx.y) * kStepCols + (tid & 7) * 4;
			const int d0 = tid >> 3;
			const bool inside = e < pitch;
			float* const state = a.state + static_cast<size_t>(h) * dim * pitch + e;
			floatx4 st[RPT];
#pragma unroll
			for (int i = 0; i < RPT; ++i)
			{
				const int d = d0 + 32 * i;
				st[i] = inside && d < dim ? *reinterpret_cast<const floatx4*>(state + static_cast<size_t>(d) * pitch)
				                          : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
			}
			floatx4 v = { 0.0f, 0.0f, 0.0f, 0.0f };
#pragma unroll
			for (int i = 0; i < 4; ++i)
			{
				v[i] = e + i < vdim ? a.v[h * vdim + e + i] : 0.0f;
			}
			for (int d = tid; d < dim; d += 256)
			{
				const int c = h * dim + d;
				alpha[d] = expf(log_sigmoid_f32(low_rank_dot(a.a2, c, a.a1) + a.a2_bias[c]) * a.shape.inv_tau);
				ks[d] = a.k[c];
				qs[d] = a.q[c] * a.shape.q_scale;
			}
			__syncthreads();
			floatx4 acc = { 0.0f, 0.0f, 0.0f, 0.0f };
#pragma unroll
			for (int i = 0; i < RPT; ++i)
			{
				const int d = d0 + 32 * i;
				if (d < dim)
				{
					st[i] = st[i] * alpha[d] + v * ks[d];
					acc += st[i] * qs[d];
					if (inside)
					{
						*reinterpret_cast<floatx4*>(state + static_cast<size_t>(d) * pitch) = st[i];
					}
				}
			}
			*reinterpret_cast<floatx4*>(&sums[d0][(tid & 7) * 4]) = acc;
			__syncthreads();
			const int col = static_cast<int>(blockIdx.y) * kStepCols + tid;
			if (tid < kStepCols && col < vdim)
			{
				float t = 0.0f;
#pragma unroll
				for (int i = 0; i < 32; ++i)
				{
					t += sums[i][tid];
				}
				a.o[h * vdim + col] = t;
			}
		}

		// ---- chunked form -------------------------------------------------------------------------
		// Tokens in chunks of 64, a chunk in four blocks of 16.  With L_t the sum of a channel's log decays
		// up to and including token t, every factor below is exp of a sum of log decays over some run of
		// tokens, so none exceeds one whatever the decays are (they are kept in units of log 2):
		//   contribution of a chunk to the state:  sum_s (k_s exp(L_end - L_s)) v_s^T
		//   o_t = (q_t exp(L_t - L_begin)) S_begin
		//         + sum over earlier blocks of ((q_t exp(L_t - L_block)) . (k_s exp(L_block - L_s))) v_s
		//         + inside t's own block  sum_s (sum_d q_td k_sd exp(L_td - L_sd)) v_s,
		// L_block being L before the first token of t's block.  The own-block term is split once more the same
		// way into quarters of four tokens; only the pairs inside a quarter are formed one by one.  The
		// contractions run on v_mfma_f32_16x16x4_f32.  Value columns are dealt out to the 16-wide tiles so that
		// a lane's four consecutive columns (one 16-byte access) belong to four tiles.
		constexpr int kChunk = 64, kSlab = 64, kSlabStride = 68;

		// chunk_states: [chunk][head][dim][pitch] floats, then [chunk][head][dim] decays over the chunk
		__device__ __forceinline__ float* chunk_decays(const Gla& a, int chunks)
		{
			return a.chunk_states +
			       static_cast<size_t>(chunks) * a.shape.heads * a.shape.dim * gla_state_pitch(a.shape.vdim);
		}

		// NC: groups of 64 value columns, each the work of four wavefronts (which share out the channels or the
		// tokens); tile b of group c holds columns 64 c + 4 i + b, i = 0 .. 15
		template <int NC>
		__global__ __launch_bounds__(256 * NC) void gla_state_kernel(const Gla a)
		{
			__shared__ float ks[kChunk][kSlabStride];
			__shared__ float totals[4][kSlab];
			const int dim = a.shape.dim, vdim = a.shape.vdim, pitch = gla_state_pitch(vdim), heads = a.shape.heads;
			const int slabs = (dim + kSlab - 1) / kSlab;
			const int h = static_cast<int>(blockIdx.x) / slabs, d0 = static_cast<int>(blockIdx.x) % slabs * kSlab;
			const int chunk = blockIdx.y, row0 = chunk * kChunk, count = min(kChunk, a.rows - row0);
			const int lane = threadIdx.x & 63;
			const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
			const int part = wave & 3, col = wave >> 2;
			const int j = lane & 15, g = lane >> 4;
			const int e = 64 * col + 4 * j;
			// the values are requested first: half of them travel while the keys are decayed
			constexpr int kSteps = kChunk / 4, kAhead = 8;
			const auto value = [&](int step) {
				return load_columns(a.v + static_cast<size_t>(row0 + min(4 * step + g, count - 1)) * a.ld + h * vdim, e, vdim);
			};
			floatx4 ahead[kAhead];
#pragma unroll
			for (int i = 0; i < kAhead; ++i)
			{
				ahead[i] = value(i);
			}
			float la[16], kv[16];
			const bool live = d0 + lane < dim;
			if (col == 0)
			{
				// thread: one channel, 16 tokens
				const size_t channel = static_cast<size_t>(h) * dim + d0 + (live ? lane : 0);
				float total = 0.0f;
#pragma unroll
				for (int t = 0; t < 16; ++t)
				{
					const int row = 16 * part + t;
					const bool in = live && row < count;
					la[t] = in ? a.log_decay[static_cast<size_t>(row0 + row) * heads * dim + channel] : 0.0f;
					kv[t] = in ? a.k[static_cast<size_t>(row0 + row) * a.ld + channel] : 0.0f;
				}
#pragma unroll
				for (int t = 0; t < 16; ++t)
				{
					total += la[t];
				}
				totals[part][lane] = total;
			}
			__syncthreads();
			if (col == 0)
			{
				float after = 0.0f;
				for (int p = part + 1; p < 4; ++p)
				{
					after += totals[p][lane];
				}
#pragma unroll
				for (int t = 15; t >= 0; --t)
				{
					ks[16 * part + t][lane] = kv[t] * exp2_f32(after);
					after += la[t];
				}
				if (part == 0 && live)
				{
					chunk_decays(a, gridDim.y)[(static_cast<size_t>(chunk) * heads + h) * dim + d0 + lane] = exp2_f32(after);
				}
			}
			__syncthreads();
			floatx4 acc[4];
#pragma unroll
			for (int b = 0; b < 4; ++b)
			{
				acc[b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
			}
#pragma unroll
			for (int step = 0; step < kSteps; ++step)
			{
				const float kf = ks[4 * step + g][16 * part + j];
				const floatx4 vv = ahead[step % kAhead];
				if (step + kAhead < kSteps)
				{
					ahead[step % kAhead] = value(step + kAhead);
				}
#pragma unroll
				for (int b = 0; b < 4; ++b)
				{
					acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf, vv[b], acc[b], 0, 0, 0);
				}
			}
			float* dst = a.chunk_states + (static_cast<size_t>(chunk) * heads + h) * dim * pitch;
#pragma unroll
			for (int r = 0; r < 4; ++r)
			{
				const int d = d0 + 16 * part + 4 * g + r;
				if (d < dim && e < pitch)
				{
					*reinterpret_cast<floatx4*>(dst + static_cast<size_t>(d) * pitch + e) =
					    floatx4{ acc[0][r], acc[1][r], acc[2][r], acc[3][r] };
				}
			}
		}

		// replaces every chunk's contribution by the state the chunk begins with; ends with the new state
		__global__ __launch_bounds__(256) void gla_scan_kernel(const Gla a, int chunks)
		{
			const int pitch = gla_state_pitch(a.shape.vdim), quads = pitch >> 2;
			const int rows = a.shape.heads * a.shape.dim;
			const int i = static_cast<int>(blockIdx.x) * 256 + static_cast<int>(threadIdx.x);
			if (i >= rows * quads)
			{
				return;
			}
			const int row = i / quads;
			const size_t at = static_cast<size_t>(row) * pitch + static_cast<size_t>(i % quads) * 4;
			const size_t step = static_cast<size_t>(rows) * pitch;
			const float* decay = chunk_decays(a, chunks) + row;
			floatx4 s = *reinterpret_cast<floatx4*>(a.state + at);
			constexpr int kAhead = 4;
			for (int c0 = 0; c0 < chunks; c0 += kAhead)
			{
				floatx4 in[kAhead];
				float dec[kAhead];
#pragma unroll
				for (int u = 0; u < kAhead; ++u)
				{
					const int c = min(c0 + u, chunks - 1);
					in[u] = *reinterpret_cast<floatx4*>(a.chunk_states + c * step + at);
					dec[u] = decay[static_cast<size_t>(c) * rows];
				}
#pragma unroll
				for (int u = 0; u < kAhead; ++u)
				{
					if (c0 + u < chunks)
					{
						*reinterpret_cast<floatx4*>(a.chunk_states + (c0 + u) * step + at) = s;
						s = s * dec[u] + in[u];
					}
				}
			}
			*reinterpret_cast<floatx4*>(a.state + at) = s;
		}

		// A wavefront makes 64 value columns of a block of 16 tokens.  The NC wavefronts of a block share out the
		// channels for the scores, whose shares meet in LDS, and each takes the state and the values of its
		// own columns.
		template <int NC, typename T>
		__global__ __launch_bounds__(256 * NC) void gla_out_kernel(const Gla a)
		{
			constexpr int kTiles = 10; // score tiles of a chunk: block b against blocks b, b - 1 .. 0
			__shared__ __attribute__((aligned(16))) float lds[3 * kChunk * kSlabStride + 4 * kSlab];
			static_assert(NC * kTiles * 256 <= 3 * kChunk * kSlabStride + 4 * kSlab, "the shares fit over the slab");
			__shared__ float squares[4][NC][16];
			float(*const qs)[kSlabStride] = reinterpret_cast<float(*)[kSlabStride]>(lds);
			float(*const ks)[kSlabStride] = qs + kChunk;
			float(*const ls)[kSlabStride] = ks + kChunk; // log decays summed from the block's first token
			float(*const totals)[kSlab] = reinterpret_cast<float(*)[kSlab]>(lds + 3 * kChunk * kSlabStride); // a block's whole sum
			const int dim = a.shape.dim, vdim = a.shape.vdim, pitch = gla_state_pitch(vdim), heads = a.shape.heads;
			const int h = blockIdx.x, chunk = blockIdx.y;
			const int row0 = chunk * kChunk, count = min(kChunk, a.rows - row0);
			const int lane = threadIdx.x & 63;
			const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
			const int block = wave & 3, col = wave >> 2;
			const int j = lane & 15, g = lane >> 4;
			const int quarter = j >> 2; // of token j in its block
			const int e0 = 64 * col + 4 * j;
			const float* state = a.chunk_states + (static_cast<size_t>(chunk) * heads + h) * dim * pitch;

			floatx4 o[4];      // o[b][r]: value column 64 col + 16 g + 4 r + b of token j of the block
			floatx4 scores[4]; // scores[back][r]: token 4 g + r of `block - back` against token j
			float near[4] = { 0.0f, 0.0f, 0.0f, 0.0f }; // token j against the tokens of its quarter, a share of the channels
#pragma unroll
			for (int b = 0; b < 4; ++b)
			{
				o[b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
				scores[b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
			}
			for (int d0 = 0; d0 < dim; d0 += kSlab)
			{
				__syncthreads();
				{
					// thread: one channel, 16 tokens, of one or more of the three arrays
					const bool live = d0 + lane < dim;
					const size_t channel = static_cast<size_t>(h) * dim + d0 + (live ? lane : 0);
					const auto fetch = [&](const float* src, size_t ld, float (&v)[16]) {
#pragma unroll
						for (int t = 0; t < 16; ++t)
						{
							const int row = 16 * block + t;
							v[t] = live && row < count ? src[static_cast<size_t>(row0 + row) * ld + channel] : 0.0f;
						}
					};
					if (col == 0)
					{
						float la[16], sum = 0.0f;
						fetch(a.log_decay, static_cast<size_t>(heads) * dim, la);
#pragma unroll
						for (int t = 0; t < 16; ++t)
						{
							sum += la[t];
							ls[16 * block + t][lane] = sum;
						}
						totals[block][lane] = sum;
					}
					if (col == (NC > 1 ? 1 : 0))
					{
						float v[16];
						fetch(a.q, static_cast<size_t>(a.ld), v);
#pragma unroll
						for (int t = 0; t < 16; ++t)
						{
							qs[16 * block + t][lane] = v[t] * a.shape.q_scale;
						}
					}
					if (col == (NC > 2 ? 2 : NC - 1))
					{
						float v[16];
						fetch(a.k, static_cast<size_t>(a.ld), v);
#pragma unroll
						for (int t = 0; t < 16; ++t)
						{
							ks[16 * block + t][lane] = v[t];
						}
					}
				}
				__syncthreads();
#pragma unroll
				for (int quad = 0; quad < kSlab / 16; ++quad)
				{
					const int c = 16 * quad + 4 * g; // this lane's four channels of the slab
					if (d0 + 16 * quad >= dim)
					{
						break; // uniform
					}
					floatx4 sv[4];
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
						const int d = min(d0 + c + r, dim - 1); // the query is zero beyond
						sv[r] = e0 < pitch ? *reinterpret_cast<const floatx4*>(state + static_cast<size_t>(d) * pitch + e0)
						                   : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
					}
					const floatx4 qv = *reinterpret_cast<const floatx4*>(&qs[16 * block + j][c]);
					const floatx4 lq = *reinterpret_cast<const floatx4*>(&ls[16 * block + j][c]);
					floatx4 qb; // decayed from the block's first token
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
						qb[r] = qv[r] * exp2_f32(lq[r]);
					}
					const bool mine = quad % NC == col; // this wavefront's share of the scores
					// earlier blocks, the nearest first: `between` is the decay over the blocks in between
					floatx4 between = { 0.0f, 0.0f, 0.0f, 0.0f };
#pragma unroll
					for (int back = 1; back < 4; ++back)
					{
						const int b = block - back; // uniform
						if (b >= 0)
						{
							const floatx4 tot = *reinterpret_cast<const floatx4*>(&totals[b][c]);
							if (mine)
							{
								const floatx4 kv = *reinterpret_cast<const floatx4*>(&ks[16 * b + j][c]);
								const floatx4 lk = *reinterpret_cast<const floatx4*>(&ls[16 * b + j][c]);
								floatx4 sc = scores[back];
#pragma unroll
								for (int r = 0; r < 4; ++r)
								{
									sc = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[r] * exp2_f32(tot[r] - lk[r] + between[r]), qb[r], sc, 0, 0, 0);
								}
								scores[back] = sc;
							}
							between += tot;
						}
					}
					if (mine)
					{
						// own block, earlier quarters: pass u pairs the tokens of quarter u with all tokens before it
						const floatx4 kv = *reinterpret_cast<const floatx4*>(&ks[16 * block + j][c]);
						const floatx4 lk = *reinterpret_cast<const floatx4*>(&ls[16 * block + j][c]);
						floatx4 sc = scores[0];
#pragma unroll
						for (int u = 1; u < 4; ++u)
						{
							const floatx4 lu = *reinterpret_cast<const floatx4*>(&ls[16 * block + 4 * u - 1][c]);
#pragma unroll
							for (int r = 0; r < 4; ++r)
							{
								const float kf = quarter < u ? kv[r] * exp2_f32(lu[r] - lk[r]) : 0.0f;
								const float qf = quarter == u ? qv[r] * exp2_f32(lq[r] - lu[r]) : 0.0f;
								sc = __builtin_amdgcn_mfma_f32_16x16x4f32(kf, qf, sc, 0, 0, 0);
							}
						}
						scores[0] = sc;
						// inside the quarter, pair by pair
#pragma unroll
						for (int s = 0; s < 4; ++s)
						{
							const floatx4 kn = *reinterpret_cast<const floatx4*>(&ks[16 * block + 4 * quarter + s][c]);
							const floatx4 ln = *reinterpret_cast<const floatx4*>(&ls[16 * block + 4 * quarter + s][c]);
#pragma unroll
							for (int r = 0; r < 4; ++r)
							{
								near[s] = fmaf(qv[r] * kn[r], exp2_f32(fminf(lq[r] - ln[r], 0.0f)), near[s]);
							}
						}
					}
					// the state the chunk begins with (`between` now spans all earlier blocks of the chunk)
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
						const float qi = qb[r] * exp2_f32(between[r]);
#pragma unroll
						for (int b = 0; b < 4; ++b)
						{
							o[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[r][b], qi, o[b], 0, 0, 0);
						}
					}
				}
			}
#pragma unroll
			for (int s = 0; s < 4; ++s)
			{
				near[s] += __shfl_xor(near[s], 16, 64);
				near[s] += __shfl_xor(near[s], 32, 64);
				scores[0][s] += g == quarter && s <= (j & 3) ? near[s] : 0.0f;
			}
			if constexpr (NC > 1)
			{
				// the shares, added in a fixed order
				const int first = block * (block + 1) / 2;
				__syncthreads();
#pragma unroll
				for (int back = 0; back < 4; ++back)
				{
					if (back <= block)
					{
						*reinterpret_cast<floatx4*>(lds + ((col * kTiles + first + back) * 64 + lane) * 4) = scores[back];
					}
				}
				__syncthreads();
#pragma unroll
				for (int back = 0; back < 4; ++back)
				{
					if (back <= block)
					{
						floatx4 t = { 0.0f, 0.0f, 0.0f, 0.0f };
#pragma unroll
						for (int n = 0; n < NC; ++n)
						{
							t += *reinterpret_cast<const floatx4*>(lds + ((n * kTiles + first + back) * 64 + lane) * 4);
						}
						scores[back] = t;
					}
				}
			}
			// o += scores . v
#pragma unroll
			for (int back = 0; back < 4; ++back)
			{
				const int b = block - back;
				if (b >= 0)
				{
					floatx4 vv[4];
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
						const int s = min(16 * b + 4 * g + r, count - 1); // scores are zero beyond
						vv[r] = load_columns(a.v + static_cast<size_t>(row0 + s) * a.ld + h * vdim, e0, vdim);
					}
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
#pragma unroll
						for (int x = 0; x < 4; ++x)
						{
							o[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(vv[r][x], scores[back][r], o[x], 0, 0, 0);
						}
					}
				}
			}
			// head norm and gate (columns past vdim are zero)
			float ss = 0.0f;
#pragma unroll
			for (int b = 0; b < 4; ++b)
			{
#pragma unroll
				for (int r = 0; r < 4; ++r)
				{
					ss = fmaf(o[b][r], o[b][r], ss);
				}
			}
			ss += __shfl_xor(ss, 16, 64);
			ss += __shfl_xor(ss, 32, 64);
			if constexpr (NC > 1)
			{
				if (g == 0)
				{
					squares[block][col][j] = ss;
				}
				__syncthreads();
				ss = 0.0f;
#pragma unroll
				for (int n = 0; n < NC; ++n)
				{
					ss += squares[block][n][j];
				}
			}
			const int row = 16 * block + j;
			if (row >= count)
			{
				return;
			}
			const float scale = 1.0f / sqrtf(ss / static_cast<float>(vdim) + a.eps);
			const float* gate = a.gate + static_cast<size_t>(row0 + row) * a.ld + h * vdim;
			T* out = static_cast<T*>(a.out) + static_cast<size_t>(row0 + row) * a.ldo + h * vdim;
#pragma unroll
			for (int r = 0; r < 4; ++r)
			{
				const int e = 64 * col + 16 * g + 4 * r;
				if (e < vdim)
				{
					const floatx4 z = load_columns(gate, e, vdim), w = load_columns(a.norm_w, e, vdim);
					floatx4 y;
#pragma unroll
					for (int b = 0; b < 4; ++b)
					{
						y[b] = o[b][r] * scale * w[b] * (z[b] * sigmoid_f32(z[b]));
					}
					if (sizeof(T) == 2 && (vdim & 3) == 0 && (a.ldo & 3) == 0)
					{
						*reinterpret_cast<uint2*>(out + e) = make_uint2(pack_bf16(y[0], y[1]), pack_bf16(y[2], y[3]));
					}
					else
					{
#pragma unroll
						for (int b = 0; b < 4; ++b)
						{
							if (e + b < vdim)
							{
								operand_store(out + e + b, y[b]);
							}
						}
					}
				}
			}
		}

		template <int DK, int DV>
		void launch_window_tile(const WindowAttn& a, hipStream_t s)
		{
			constexpr size_t lds = sizeof(uint16_t) * (kWinKeys * (DK + 8) + DV * kWinVStride);
			allow_dynamic_lds(reinterpret_cast<const void*>(&window_attn_tile_kernel<DK, DV>), lds);
			window_attn_tile_kernel<DK, DV>
			    <<<dim3(a.shape.heads, (a.rows + kWinQ - 1) / kWinQ), dim3(256), lds, s>>>(a);
		}

		template <int DK>
		void launch_window_tile(const WindowAttn& a, hipStream_t s)
		{
			if (a.shape.vdim <= 64)
			{
				launch_window_tile<DK, 64>(a, s);
			}
			else if (a.shape.vdim <= 128)
			{
				launch_window_tile<DK, 128>(a, s);
			}
			else
			{
				launch_window_tile<DK, 256>(a, s);
			}
		}

		template <int NC>
		void launch_gla_chunks(const Gla& a, int chunks, hipStream_t s)
		{
			const int slabs = (a.shape.dim + kSlab - 1) / kSlab;
			gla_state_kernel<NC><<<dim3(a.shape.heads * slabs, chunks), dim3(256 * NC), 0, s>>>(a);
			const int quads = a.shape.heads * a.shape.dim * (gla_state_pitch(a.shape.vdim) >> 2);
			gla_scan_kernel<<<dim3((quads + 255) / 256), dim3(256), 0, s>>>(a, chunks);
			if (a.f32)
			{
				gla_out_kernel<NC, float><<<dim3(a.shape.heads, chunks), dim3(256 * NC), 0, s>>>(a);
			}
			else
			{
				gla_out_kernel<NC, uint16_t><<<dim3(a.shape.heads, chunks), dim3(256 * NC), 0, s>>>(a);
			}
		}

		size_t latent_step_lds(int pitch)
		{
			return sizeof(float) * (static_cast<size_t>(kLatentTile) * (pitch + 4) + static_cast<size_t>(kLatentHeads) * pitch +
			                        kLatentHeads * kLatentTile);
		}
	} // namespace

	void launch_embed_rows(const DenseMatrix& table, const int32_t* ids, int rows, const double* turns, Position pos,
	                       float* x, int* err, hipStream_t s)
	{
		if (rows > 0)
		{
			embed_rows_kernel<<<dim3(rows, (table.k + 511) / 512), dim3(256), 0, s>>>(table, ids, turns, pos, x, err);
		}
	}

	void launch_add_norm(const AddNorm& a, hipStream_t s)
	{
		if (a.rows <= 0)
		{
			return;
		}
		const dim3 grid(a.rows), threads(256);
		if (a.f32)
		{
			add_norm_kernel<float, 1><<<grid, threads, 0, s>>>(a);
		}
		else if (!a.sub || a.sub_parts == 1)
		{
			add_norm_kernel<uint16_t, 1><<<grid, threads, 0, s>>>(a);
		}
		else
		{
			add_norm_kernel<uint16_t, kDenseMaxSplits><<<grid, threads, 0, s>>>(a);
		}
	}

	void launch_latent_append(const float* src, int ld, const float* norm_w, float eps, int rows, Position pos,
	                          const LatentCache& cache, hipStream_t s)
	{
		if (rows <= 0)
		{
			return;
		}
		if (cache.f32)
		{
			latent_append_kernel<float><<<dim3(rows), dim3(256), 0, s>>>(src, ld, norm_w, eps, pos, cache);
		}
		else
		{
			latent_append_kernel<uint16_t><<<dim3(rows), dim3(256), 0, s>>>(src, ld, norm_w, eps, pos, cache);
		}
	}

	int latent_step_max_rank() { return kLatentMaxRank; }

	// about two workgroups per CU, and no split shorter than a tile
	int latent_step_splits(int heads, int rows, int window)
	{
		const int groups = (heads + kLatentHeads - 1) / kLatentHeads * rows;
		const int tiles = (window + kLatentTile - 1) / kLatentTile;
		return std::max(1, std::min({ tiles, 512 / std::max(1, groups), kLatentMaxSplits }));
	}

	size_t latent_step_partial_floats(int heads, int rows, int pitch, int splits)
	{
		return static_cast<size_t>(heads) * rows * splits * (pitch + 4);
	}

	void launch_latent_step(const LatentStep& a, hipStream_t s)
	{
		const int slices = (a.cache.pitch + kAbsorbSlice - 1) / kAbsorbSlice;
		const dim3 absorb(a.shape.heads * slices + 1, a.rows);
		const dim3 attend((a.shape.heads + kLatentHeads - 1) / kLatentHeads, a.splits, a.rows);
		const size_t lds = latent_step_lds(a.cache.pitch);
		if (a.cache.f32)
		{
			latent_absorb_kernel<float><<<absorb, dim3(256), 0, s>>>(a);
			allow_dynamic_lds(reinterpret_cast<const void*>(&latent_step_kernel<float>), latent_step_lds(kLatentMaxRank));
			latent_step_kernel<float><<<attend, dim3(256), lds, s>>>(a);
		}
		else
		{
			latent_absorb_kernel<uint16_t><<<absorb, dim3(256), 0, s>>>(a);
			allow_dynamic_lds(reinterpret_cast<const void*>(&latent_step_kernel<uint16_t>), latent_step_lds(kLatentMaxRank));
			latent_step_kernel<uint16_t><<<attend, dim3(256), lds, s>>>(a);
		}
		const dim3 value(a.shape.heads * ((a.shape.vdim + kValueSlice - 1) / kValueSlice), a.rows);
		if (a.out_f32)
		{
			latent_value_kernel<float><<<value, dim3(kValueThreads), 0, s>>>(a);
		}
		else
		{
			latent_value_kernel<uint16_t><<<value, dim3(kValueThreads), 0, s>>>(a);
		}
	}

	void launch_window_attn(const WindowAttn& a, hipStream_t s)
	{
		if (a.rows <= 0)
		{
			return;
		}
		const dim3 rows(a.rows, a.shape.heads);
		if (a.f32)
		{
			window_attn_row_kernel<float><<<rows, dim3(64), 0, s>>>(a);
			return;
		}
		// whole 16-byte pieces of a head's keys and values
		const bool pieces = a.k_head % 8 == 0 && a.v_head % 8 == 0 && a.ldkv % 8 == 0 && a.v_first % 8 == 0 &&
		                    (a.ldo % 4 == 0 || a.shape.vdim % 4 != 0) && a.shape.dim <= 256 && a.shape.vdim <= 256;
		if (!pieces)
		{
			window_attn_row_kernel<uint16_t><<<rows, dim3(64), 0, s>>>(a);
		}
		else if (a.shape.dim <= 64)
		{
			launch_window_tile<64>(a, s);
		}
		else if (a.shape.dim <= 128)
		{
			launch_window_tile<128>(a, s);
		}
		else
		{
			launch_window_tile<256>(a, s);
		}
	}

	int gla_max_dim() { return kGlaMaxDim; }
	int gla_max_vdim() { return 256; }

	size_t gla_chunk_floats(int rows, int heads, int dim, int vdim)
	{
		const size_t chunks = (static_cast<size_t>(rows) + kChunk - 1) / kChunk;
		return chunks * heads * dim * (static_cast<size_t>(gla_state_pitch(vdim)) + 1);
	}

	void launch_gla_step(const Gla& a, hipStream_t s)
	{
		const dim3 grid(a.shape.heads, (a.shape.vdim + kStepCols - 1) / kStepCols);
		const int rpt = (a.shape.dim + 31) / 32;
		if (rpt <= 2)
		{
			gla_step_kernel<2><<<grid, dim3(256), 0, s>>>(a);
		}
		else if (rpt <= 4)
		{
			gla_step_kernel<4><<<grid, dim3(256), 0, s>>>(a);
		}
		else if (rpt <= 8)
		{
			gla_step_kernel<8><<<grid, dim3(256), 0, s>>>(a);
		}
		else
		{
			gla_step_kernel<16><<<grid, dim3(256), 0, s>>>(a);
		}
	}

	void launch_gla_rows(const Gla& a, hipStream_t s)
	{
		if (a.rows <= 0)
		{
			return;
		}
		const int channels = a.shape.heads * a.shape.dim;
		gla_decay_kernel<<<dim3((channels + 255) / 256, (a.rows + kDecayRows - 1) / kDecayRows), dim3(256), 0, s>>>(a);
		const int chunks = (a.rows + kChunk - 1) / kChunk;
		if (a.shape.vdim <= 64)
		{
			launch_gla_chunks<1>(a, chunks, s);
		}
		else if (a.shape.vdim <= 128)
		{
			launch_gla_chunks<2>(a, chunks, s);
		}
		else
		{
			launch_gla_chunks<4>(a, chunks, s);
		}
	}
} // namespace litenn_hip
