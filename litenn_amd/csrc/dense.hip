// Linear layers over bfloat16 weights for gfx950: y[m, n] = sum_k x[m, k] W[n, k].
//
// One row (decode) streams the weights once through registers with Float32 activations in LDS; many
// rows (prompt) run on the matrix cores, either with bfloat16 operands or, where Float32 operands are
// asked for, with v_mfma_f32_16x16x4_f32 and the weights widened exactly.  Every accumulation is
// Float32.  The reference has no counterpart (its linears are f32 MatMul nodes,
// src/LiteNN/Layer/Linear.h:67-95).
#include "dense.hpp"

#include <algorithm>

namespace litenn_hip
{
	namespace
	{
		typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
		typedef float floatx4 __attribute__((ext_vector_type(4)));
		typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

		// ------------------------------------------------------------------
		// One activation row.  A wavefront owns R consecutive rows at a time and walks K in blocks of 512
		// (64 lanes x 8 weights, one 16-byte load each); kFlight blocks of every row are requested ahead,
		// the first ones before the activations are even looked at, so that the weights travel while the
		// prologue runs, and the next rows' first blocks while the current rows finish.
		// LDS: the activations as two planes (elements 0..3 and 4..7 of every group of eight), so that
		// consecutive lanes read consecutive 16-byte pieces.
		// ------------------------------------------------------------------
		constexpr int kRowThreads = 512, kRowWaves = kRowThreads / 64, kFlight = 4, kRowBlock = 512;

		struct RowArgs
		{
			DenseRow d;
			int groups; // steps of kFlight blocks that cover a row
		};

		__device__ __forceinline__ int row_slot(int k, int half)
		{
			return ((k >> 2) & 1) * half + (k >> 3) * 4 + (k & 3);
		}

		// elements i .. i + 3 of a vector of k, zero beyond (global loads take any 4-byte address)
		__device__ __forceinline__ floatx4 load_piece(const float* x, int i, int k)
		{
			typedef floatx4 floatx4_a4 __attribute__((aligned(4)));
			floatx4 v = { 0.0f, 0.0f, 0.0f, 0.0f };
			if (i + 3 < k)
			{
				v = *reinterpret_cast<const floatx4_a4*>(x + i);
			}
			else
			{
#pragma unroll
				for (int e = 0; e < 3; ++e)
				{
					v[e] = i + e < k ? x[i + e] : 0.0f;
				}
			}
			return v;
		}

		__device__ __forceinline__ float square_sum(const floatx4& v, float acc)
		{
			acc = fmaf(v.x, v.x, acc);
			acc = fmaf(v.y, v.y, acc);
			acc = fmaf(v.z, v.z, acc);
			return fmaf(v.w, v.w, acc);
		}

		// sum over the workgroup; `red` holds one float per wavefront
		__device__ __forceinline__ float block_sum(float v, float* red)
		{
			v = wave_sum(v);
			__syncthreads();
			if ((threadIdx.x & 63) == 0)
			{
				red[threadIdx.x >> 6] = v;
			}
			__syncthreads();
			float t = 0.0f;
			for (int i = 0; i < static_cast<int>(blockDim.x >> 6); ++i)
			{
				t += red[i];
			}
			return t;
		}

		template <int R>
		__global__ __launch_bounds__(kRowThreads) void dense_row_kernel(const RowArgs args)
		{
			extern __shared__ __attribute__((aligned(16))) float row_lds[];
			__shared__ float red[kRowWaves];
			const DenseRow& d = args.d;
			const int lane = threadIdx.x & 63;
			const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
			const int n = d.w.n, k = d.w.k, pitch = d.w.pitch, groups = args.groups;
			const int row_groups = (n + R - 1) / R;
			const int stride = static_cast<int>(gridDim.x) * kRowWaves;
			int rg = static_cast<int>(blockIdx.x) * kRowWaves + wave;
			const bool busy = rg < row_groups;
			const int half = groups * kFlight * kRowBlock / 2;

			u32x4 cur[R][kFlight], nxt[R][kFlight];
			const auto request = [&](u32x4 (&dst)[R][kFlight], int group_of_rows, int step) {
#pragma unroll
				for (int r = 0; r < R; ++r)
				{
					const uint16_t* row = d.w.w + static_cast<size_t>(min(group_of_rows * R + r, n - 1)) * pitch;
#pragma unroll
					for (int p = 0; p < kFlight; ++p)
					{
						// past the row's end any of its weights will do: the activations there are zero
						const int at = (step * kFlight + p) * kRowBlock + lane * 8;
						dst[r][p] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(row + (at < pitch ? at : 0)));
					}
				}
			};
			if (busy)
			{
				request(cur, rg, 0);
			}

			// activations, four at a time where k allows; a thread's first kKept pieces stay in registers
			const int pieces = half >> 1; // of four floats, zeros behind the k-th
			const auto put = [&](int piece, floatx4 v) {
				*reinterpret_cast<floatx4*>(row_lds + (piece & 1) * half + (piece >> 1) * 4) = v;
			};
			if (d.prologue == kRowAddNorm)
			{
				constexpr int kKept = 2;
				floatx4 x[kKept], sub[kKept], subw[kKept], nw[kKept];
#pragma unroll
				for (int e = 0; e < kKept; ++e)
				{
					const int i = 4 * (static_cast<int>(threadIdx.x) + kRowThreads * e);
					x[e] = load_piece(d.x, i, k);
					sub[e] = d.sub ? load_piece(d.sub, i, k) : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
					subw[e] = d.sub ? load_piece(d.sub_w, i, k) : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
					nw[e] = d.norm_w ? load_piece(d.norm_w, i, k) : floatx4{ 1.0f, 1.0f, 1.0f, 1.0f };
				}
				float scale_sub = 0.0f;
				if (d.sub)
				{
					float ss = 0.0f;
#pragma unroll
					for (int e = 0; e < kKept; ++e)
					{
						ss = square_sum(sub[e], ss);
					}
					for (int p = threadIdx.x + kRowThreads * kKept; p < pieces; p += kRowThreads)
					{
						ss = square_sum(load_piece(d.sub, 4 * p, k), ss);
					}
					scale_sub = 1.0f / sqrtf(block_sum(ss, red) / static_cast<float>(k) + d.eps);
				}
				float ss = 0.0f;
				const auto enter = [&](int p, floatx4 v, floatx4 s, floatx4 sw, floatx4 w) {
					if (d.sub)
					{
						v += s * scale_sub * sw;
					}
					if (d.x_out && blockIdx.x == 0)
					{
#pragma unroll
						for (int i = 0; i < 4; ++i)
						{
							if (4 * p + i < k)
							{
								d.x_out[4 * p + i] = v[i];
							}
						}
					}
					ss = square_sum(v, ss);
					return v * w;
				};
#pragma unroll
				for (int e = 0; e < kKept; ++e)
				{
					x[e] = enter(static_cast<int>(threadIdx.x) + kRowThreads * e, x[e], sub[e], subw[e], nw[e]);
				}
				for (int p = threadIdx.x + kRowThreads * kKept; p < pieces; p += kRowThreads)
				{
					put(p, enter(p, load_piece(d.x, 4 * p, k), d.sub ? load_piece(d.sub, 4 * p, k) : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f },
					             d.sub ? load_piece(d.sub_w, 4 * p, k) : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f },
					             d.norm_w ? load_piece(d.norm_w, 4 * p, k) : floatx4{ 1.0f, 1.0f, 1.0f, 1.0f }));
				}
				const float scale = d.norm_w ? 1.0f / sqrtf(block_sum(ss, red) / static_cast<float>(k) + d.eps) : 1.0f;
#pragma unroll
				for (int e = 0; e < kKept; ++e)
				{
					const int p = static_cast<int>(threadIdx.x) + kRowThreads * e;
					if (p < pieces)
					{
						put(p, x[e] * scale);
					}
				}
				for (int p = threadIdx.x + kRowThreads * kKept; p < pieces; p += kRowThreads)
				{
					floatx4* slot = reinterpret_cast<floatx4*>(row_lds + (p & 1) * half + (p >> 1) * 4);
					*slot = *slot * scale; // this thread's own
				}
			}
			else if (d.prologue == kRowHeadGate)
			{
				const int heads = k / d.vdim;
				for (int h = wave; h < heads; h += kRowWaves)
				{
					const float* o = d.x + static_cast<size_t>(h) * d.vdim;
					float ss = 0.0f;
					for (int e = lane; e < d.vdim; e += 64)
					{
						ss = fmaf(o[e], o[e], ss);
					}
					const float scale = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(d.vdim) + d.eps);
					for (int e = lane; e < d.vdim; e += 64)
					{
						const float g = d.gate[h * d.vdim + e];
						row_lds[row_slot(h * d.vdim + e, half)] = o[e] * scale * d.norm_w[e] * (g * sigmoid_f32(g));
					}
				}
				for (int i = k + threadIdx.x; i < 2 * half; i += kRowThreads)
				{
					row_lds[row_slot(i, half)] = 0.0f;
				}
			}
			else
			{
#pragma unroll 4
				for (int p = threadIdx.x; p < pieces; p += kRowThreads)
				{
					put(p, load_piece(d.x, 4 * p, k));
				}
			}
			__syncthreads();
			if (!busy)
			{
				return;
			}

			float acc[R];
#pragma unroll
			for (int r = 0; r < R; ++r)
			{
				acc[r] = 0.0f;
			}
			int step = 0;
			while (true)
			{
				// the step after this one, possibly of the next rows
				int next_rg = rg, next_step = step + 1;
				if (next_step == groups)
				{
					next_step = 0;
					next_rg = rg + stride;
				}
				const bool more = next_rg < row_groups;
				if (more)
				{
					request(nxt, next_rg, next_step);
				}
#pragma unroll
				for (int p = 0; p < kFlight; ++p)
				{
					const int piece = (step * kFlight + p) * (kRowBlock / 8) + lane;
					const floatx4 x0 = *reinterpret_cast<const floatx4*>(row_lds + piece * 4);
					const floatx4 x1 = *reinterpret_cast<const floatx4*>(row_lds + half + piece * 4);
#pragma unroll
					for (int r = 0; r < R; ++r)
					{
						const u32x4 w = cur[r][p];
						float a = acc[r];
						a = fmaf(__uint_as_float(w.x << 16), x0.x, a);
						a = fmaf(__uint_as_float(w.x & 0xffff0000u), x0.y, a);
						a = fmaf(__uint_as_float(w.y << 16), x0.z, a);
						a = fmaf(__uint_as_float(w.y & 0xffff0000u), x0.w, a);
						a = fmaf(__uint_as_float(w.z << 16), x1.x, a);
						a = fmaf(__uint_as_float(w.z & 0xffff0000u), x1.y, a);
						a = fmaf(__uint_as_float(w.w << 16), x1.z, a);
						a = fmaf(__uint_as_float(w.w & 0xffff0000u), x1.w, a);
						acc[r] = a;
					}
				}
				if (next_step == 0)
				{
#pragma unroll
					for (int r = 0; r < R; ++r)
					{
						acc[r] = wave_sum(acc[r]);
					}
					if (lane == 0)
					{
						if constexpr (R >= 2)
						{
							if (d.glu)
							{
#pragma unroll
								for (int r = 0; r < R; r += 2)
								{
									if (rg * R + r < n)
									{
										d.y[(rg * R + r) >> 1] = clamped_glu(acc[r], acc[r + 1], d.act);
									}
								}
							}
						}
						if (R < 2 || !d.glu)
						{
#pragma unroll
							for (int r = 0; r < R; ++r)
							{
								if (rg * R + r < n)
								{
									d.y[rg * R + r] = soft_cap(acc[r], d.softcap);
								}
							}
						}
					}
#pragma unroll
					for (int r = 0; r < R; ++r)
					{
						acc[r] = 0.0f;
					}
				}
				if (!more)
				{
					return;
				}
				rg = next_rg;
				step = next_step;
#pragma unroll
				for (int r = 0; r < R; ++r)
				{
#pragma unroll
					for (int p = 0; p < kFlight; ++p)
					{
						cur[r][p] = nxt[r][p];
					}
				}
			}
		}

		// ------------------------------------------------------------------
		// Many rows, bfloat16 operands: BM activation rows x BN weight rows per workgroup of four
		// wavefronts, K in tiles of 64 double-buffered in LDS (global -> registers two tiles ahead -> LDS
		// while the previous tile is multiplied), v_mfma_f32_16x16x32_bf16 with the weights as the A operand, so that a lane
		// ends up with four consecutive outputs of one activation row.  The 16-byte pieces of a 128-byte
		// LDS row are permuted by the row's low three bits: the 16 rows a fragment read touches then fall
		// on different banks.
		// ------------------------------------------------------------------
		constexpr int kTileK = 64;

		struct TileArgs
		{
			DenseRows d;
			int m_tiles, n_tiles;
		};

		// Tile of this workgroup: the eight XCDs (workgroups are dealt to them round-robin) walk eight
		// consecutive ranges of tiles, and inside a range eight row tiles share a weight tile's L2 lines.
		__device__ __forceinline__ bool tile_of(const TileArgs& a, int& tm, int& tn)
		{
			const int total = a.m_tiles * a.n_tiles;
			const int per = static_cast<int>(gridDim.x) >> 3;
			const int t = static_cast<int>(blockIdx.x & 7) * per + static_cast<int>(blockIdx.x >> 3);
			if (t >= total)
			{
				return false;
			}
			constexpr int kGroup = 8;
			const int width = kGroup * a.n_tiles;
			const int first = t / width * kGroup, in = t % width;
			const int rows = min(kGroup, a.m_tiles - first);
			tm = first + in % rows;
			tn = in / rows;
			return true;
		}

		__device__ __forceinline__ int operand_row(const DenseRows& d, int m)
		{
			int r = min(m, d.m - 1);
			if (d.a_ring > 0)
			{
				r += d.a_first;
				r -= r >= d.a_ring ? d.a_ring : 0;
			}
			return r;
		}

		// four consecutive outputs n .. n + 3 of activation row m
		template <typename T>
		__device__ __forceinline__ void store_outputs(const DenseRows& d, int m, int n, const floatx4& v)
		{
			if (m >= d.m || n >= d.w.n)
			{
				return;
			}
			float f[4] = { v.x, v.y, v.z, v.w };
			if (d.out == kOutGlu)
			{
				T* c = static_cast<T*>(d.c) + static_cast<size_t>(m) * d.ldc + (n >> 1);
#pragma unroll
				for (int i = 0; i < 2; ++i)
				{
					if (n + 2 * i < d.w.n)
					{
						operand_store(c + i, clamped_glu(f[2 * i], f[2 * i + 1], d.act));
					}
				}
				return;
			}
			if (d.out == kOutOperand && sizeof(T) == 2)
			{
				uint16_t* c = static_cast<uint16_t*>(d.c) + static_cast<size_t>(m) * d.ldc + n;
				if (n + 3 < d.w.n)
				{
					*reinterpret_cast<uint2*>(c) = make_uint2(pack_bf16(f[0], f[1]), pack_bf16(f[2], f[3]));
				}
				else
				{
					for (int i = 0; i < 4 && n + i < d.w.n; ++i)
					{
						c[i] = to_bf16(f[i]);
					}
				}
				return;
			}
			if (d.softcap > 0.0f)
			{
#pragma unroll
				for (int i = 0; i < 4; ++i)
				{
					f[i] = soft_cap(f[i], d.softcap);
				}
			}
			float* c = static_cast<float*>(d.c) + blockIdx.y * d.split_stride + static_cast<size_t>(m) * d.ldc + n;
			if (n + 3 < d.w.n && (d.ldc & 3) == 0)
			{
				*reinterpret_cast<float4*>(c) = make_float4(f[0], f[1], f[2], f[3]);
			}
			else
			{
				for (int i = 0; i < 4 && n + i < d.w.n; ++i)
				{
					c[i] = f[i];
				}
			}
		}

		// WM x WN wavefronts share the tile
		template <int BM, int BN, int WM, int WN>
		__global__ __launch_bounds__(256) void dense_tile_kernel(const TileArgs args)
		{
			static_assert(WM * WN == 4, "four wavefronts");
			constexpr int TM = BM / WM / 16, TN = BN / WN / 16;
			constexpr int LA = BM / 32, LW = BN / 32; // 16-byte pieces a thread stages per K tile
			__shared__ __attribute__((aligned(16))) uint16_t xs[2][BM * kTileK];
			__shared__ __attribute__((aligned(16))) uint16_t ws[2][BN * kTileK];
			const DenseRows& d = args.d;
			int tm, tn;
			if (!tile_of(args, tm, tn))
			{
				return;
			}
			const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
			const int j = lane & 15, g = lane >> 4;
			const int wm = wave / WN, wn = wave % WN;
			const int m0 = tm * BM, n0 = tn * BN;
			const int k = d.w.k;
			// this workgroup's share of K
			const int all_steps = d.w.pitch / kTileK, part = static_cast<int>(blockIdx.y);
			const int first_step = all_steps * part / d.splits;
			const int steps = all_steps * (part + 1) / d.splits - first_step;

			const int ch = tid & 7, row = tid >> 3; // this thread's piece column and first row
			const uint16_t* xp[LA];
			const uint16_t* wp[LW];
#pragma unroll
			for (int i = 0; i < LA; ++i)
			{
				xp[i] = static_cast<const uint16_t*>(d.a) + static_cast<size_t>(operand_row(d, m0 + row + 32 * i)) * d.lda + ch * 8;
			}
#pragma unroll
			for (int i = 0; i < LW; ++i)
			{
				wp[i] = d.w.w + static_cast<size_t>(min(n0 + row + 32 * i, d.w.n - 1)) * d.w.pitch + ch * 8;
			}
			// two K tiles travel at any time: tile t in register set t & 1 until it is staged
			u32x4 rx[2][LA], rw[2][LW];
			const auto request = [&](int step, int set) {
#pragma unroll
				for (int i = 0; i < LA; ++i)
				{
					rx[set][i] = *reinterpret_cast<const u32x4*>(xp[i] + step * kTileK);
				}
#pragma unroll
				for (int i = 0; i < LW; ++i)
				{
					rw[set][i] = *reinterpret_cast<const u32x4*>(wp[i] + step * kTileK);
				}
			};
			const auto stage = [&](int step, int set) {
				const int left = k - step * kTileK - ch * 8; // valid elements of this thread's pieces
				if (left < 8)
				{
					// behind the k-th activation there may be anything: zero it
#pragma unroll
					for (int i = 0; i < LA; ++i)
					{
#pragma unroll
						for (int e = 0; e < 4; ++e)
						{
							const uint32_t keep = left >= 2 * e + 2 ? 0xffffffffu : left == 2 * e + 1 ? 0xffffu : 0u;
							rx[set][i][e] &= keep;
						}
					}
				}
				const int slot = (ch ^ (row & 7)) * 8;
#pragma unroll
				for (int i = 0; i < LA; ++i)
				{
					*reinterpret_cast<u32x4*>(&xs[set][(row + 32 * i) * kTileK + slot]) = rx[set][i];
				}
#pragma unroll
				for (int i = 0; i < LW; ++i)
				{
					*reinterpret_cast<u32x4*>(&ws[set][(row + 32 * i) * kTileK + slot]) = rw[set][i];
				}
			};

			floatx4 acc[TN][TM];
#pragma unroll
			for (int a = 0; a < TN; ++a)
			{
#pragma unroll
				for (int b = 0; b < TM; ++b)
				{
					acc[a][b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
				}
			}
			const auto multiply = [&](int buf) {
#pragma unroll
				for (int ks = 0; ks < 2; ++ks)
				{
					bf16x8 wf[TN], xf[TM];
#pragma unroll
					for (int a = 0; a < TN; ++a)
					{
						const int r = wn * (BN / WN) + 16 * a + j;
						wf[a] = *reinterpret_cast<const bf16x8*>(&ws[buf][r * kTileK + (((4 * ks + g) ^ (r & 7)) * 8)]);
					}
#pragma unroll
					for (int b = 0; b < TM; ++b)
					{
						const int r = wm * (BM / WM) + 16 * b + j;
						xf[b] = *reinterpret_cast<const bf16x8*>(&xs[buf][r * kTileK + (((4 * ks + g) ^ (r & 7)) * 8)]);
					}
#pragma unroll
					for (int a = 0; a < TN; ++a)
					{
#pragma unroll
						for (int b = 0; b < TM; ++b)
						{
							acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[a], xf[b], acc[a][b], 0, 0, 0);
						}
					}
				}
			};
			// past the last tile it is requested and staged again: a branch around the loads would make every
			// wait behind it a wait for all of them
			request(first_step, 0);
			request(first_step + min(1, steps - 1), 1);
			stage(first_step, 0);
			__syncthreads();
			// tile `step` is in LDS buffer `set`, tile step + 1 in the other register set
			const auto advance = [&](int step, int set) {
				request(first_step + min(step + 2, steps - 1), set);
				if constexpr (BM * BN < 128 * 128)
				{
					// on their way before the products, not behind them (the largest tile, whose products take
					// longer than the loads, runs better scheduled freely)
					__builtin_amdgcn_sched_barrier(0);
				}
				multiply(set);
				stage(first_step + min(step + 1, steps - 1), set ^ 1);
				__syncthreads();
			};
			int step = 0;
			for (; step + 1 < steps; step += 2)
			{
				advance(step, 0);
				advance(step + 1, 1);
			}
			if (step < steps)
			{
				advance(step, 0);
			}
#pragma unroll
			for (int b = 0; b < TM; ++b)
			{
				const int m = m0 + wm * (BM / WM) + 16 * b + j;
#pragma unroll
				for (int a = 0; a < TN; ++a)
				{
					store_outputs<uint16_t>(d, m, n0 + wn * (BN / WN) + 16 * a + 4 * g, acc[a][b]);
				}
			}
		}

		// ------------------------------------------------------------------
		// Many rows, Float32 operands: 64 x 64 per workgroup, K in tiles of 32, v_mfma_f32_16x16x4_f32.  The
		// contraction index is dealt out so that a lane's four consecutive elements of a row (one 16-byte
		// LDS read) serve four instructions: step r of a 16-wide block takes element 4 g + r from lane
		// group g, for both operands.
		// ------------------------------------------------------------------
		constexpr int kF32Tile = 64, kF32K = 32, kF32Stride = 36;

		__global__ __launch_bounds__(256) void dense_tile_f32_kernel(const TileArgs args)
		{
			__shared__ __attribute__((aligned(16))) float xs[kF32Tile * kF32Stride];
			__shared__ __attribute__((aligned(16))) float ws[kF32Tile * kF32Stride];
			const DenseRows& d = args.d;
			int tm, tn;
			if (!tile_of(args, tm, tn))
			{
				return;
			}
			const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
			const int j = lane & 15, g = lane >> 4;
			const int wm = wave >> 1, wn = wave & 1;
			const int m0 = tm * kF32Tile, n0 = tn * kF32Tile;
			const int k = d.w.k;
			const int steps = d.w.pitch / kF32K;
			const int xrow = tid >> 3, xc = (tid & 7) * 4;  // two rows (xrow, xrow + 32), four floats
			const int wrow = tid >> 2, wc = (tid & 3) * 8;  // one row, eight weights
			const float* xp[2];
#pragma unroll
			for (int i = 0; i < 2; ++i)
			{
				xp[i] = static_cast<const float*>(d.a) + static_cast<size_t>(operand_row(d, m0 + xrow + 32 * i)) * d.lda + xc;
			}
			const uint16_t* wp = d.w.w + static_cast<size_t>(min(n0 + wrow, d.w.n - 1)) * d.w.pitch + wc;
			floatx4 rx[2];
			u32x4 rw;
			const auto request = [&](int step) {
#pragma unroll
				for (int i = 0; i < 2; ++i)
				{
					rx[i] = *reinterpret_cast<const floatx4*>(xp[i] + step * kF32K);
				}
				rw = *reinterpret_cast<const u32x4*>(wp + step * kF32K);
			};
			floatx4 acc[2][2];
#pragma unroll
			for (int a = 0; a < 2; ++a)
			{
#pragma unroll
				for (int b = 0; b < 2; ++b)
				{
					acc[a][b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
				}
			}
			request(0);
			for (int step = 0; step < steps; ++step)
			{
				const int left = k - step * kF32K - xc;
#pragma unroll
				for (int i = 0; i < 2; ++i)
				{
					floatx4 v = rx[i];
#pragma unroll
					for (int e = 0; e < 4; ++e)
					{
						v[e] = e < left ? v[e] : 0.0f;
					}
					*reinterpret_cast<floatx4*>(&xs[(xrow + 32 * i) * kF32Stride + xc]) = v;
				}
#pragma unroll
				for (int e = 0; e < 2; ++e)
				{
					*reinterpret_cast<floatx4*>(&ws[wrow * kF32Stride + wc + 4 * e]) =
					    floatx4{ __uint_as_float(rw[2 * e] << 16), __uint_as_float(rw[2 * e] & 0xffff0000u),
						         __uint_as_float(rw[2 * e + 1] << 16), __uint_as_float(rw[2 * e + 1] & 0xffff0000u) };
				}
				__syncthreads();
				if (step + 1 < steps)
				{
					request(step + 1);
				}
#pragma unroll
				for (int kb = 0; kb < kF32K; kb += 16)
				{
					floatx4 wf[2], xf[2];
#pragma unroll
					for (int t = 0; t < 2; ++t)
					{
						wf[t] = *reinterpret_cast<const floatx4*>(&ws[(wn * 32 + 16 * t + j) * kF32Stride + kb + 4 * g]);
						xf[t] = *reinterpret_cast<const floatx4*>(&xs[(wm * 32 + 16 * t + j) * kF32Stride + kb + 4 * g]);
					}
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
#pragma unroll
						for (int a = 0; a < 2; ++a)
						{
#pragma unroll
							for (int b = 0; b < 2; ++b)
							{
								acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(wf[a][r], xf[b][r], acc[a][b], 0, 0, 0);
							}
						}
					}
				}
				__syncthreads();
			}
#pragma unroll
			for (int b = 0; b < 2; ++b)
			{
#pragma unroll
				for (int a = 0; a < 2; ++a)
				{
					store_outputs<float>(d, m0 + wm * 32 + 16 * b + j, n0 + wn * 32 + 16 * a + 4 * g, acc[a][b]);
				}
			}
		}

		constexpr size_t kRowLdsLimit = 152 * 1024;

		size_t row_lds_bytes(int pitch, int& groups)
		{
			groups = (pitch + kFlight * kRowBlock - 1) / (kFlight * kRowBlock);
			return sizeof(float) * static_cast<size_t>(groups) * kFlight * kRowBlock;
		}

		template <int R>
		void launch_row(const RowArgs& args, size_t lds, hipStream_t s)
		{
			const int waves = (args.d.w.n + R - 1) / R;
			const int cap = lds > 72 * 1024 ? 256 : 512;
			const int rounds = (waves + cap * kRowWaves - 1) / (cap * kRowWaves);
			const int blocks = (waves + rounds * kRowWaves - 1) / (rounds * kRowWaves);
			allow_dynamic_lds(reinterpret_cast<const void*>(&dense_row_kernel<R>), kRowLdsLimit);
			dense_row_kernel<R><<<dim3(blocks), dim3(kRowThreads), lds, s>>>(args);
		}

		template <int BM, int BN, int WM, int WN>
		void launch_tile(TileArgs& args, hipStream_t s)
		{
			args.m_tiles = (args.d.m + BM - 1) / BM;
			args.n_tiles = (args.d.w.n + BN - 1) / BN;
			const int per = (args.m_tiles * args.n_tiles + 7) / 8;
			dense_tile_kernel<BM, BN, WM, WN><<<dim3(8 * per, args.d.splits), dim3(256), 0, s>>>(args);
		}

		int tiles(const DenseRows& d, int bm, int bn) { return ((d.m + bm - 1) / bm) * ((d.w.n + bn - 1) / bn); }
	} // namespace

	// Few tiles: K is walked in up to four ranges at once, enough for about two workgroups per CU and none
	// shorter than 16 tiles of K.
	int dense_rows_splits(const DenseMatrix& w, int m)
	{
		DenseRows d;
		d.w = w;
		d.m = m;
		const int t = m <= 32 ? tiles(d, 32, 64) : tiles(d, 64, 64);
		return std::max(1, std::min({ kDenseMaxSplits, (512 + t / 2) / t, w.pitch / kTileK / 16 }));
	}

	size_t dense_row_max_k() { return kRowLdsLimit / sizeof(float) / (kFlight * kRowBlock) * (kFlight * kRowBlock); }

	bool launch_dense_row(const DenseRow& a, hipStream_t s)
	{
		if (a.w.n <= 0)
		{
			return true;
		}
		RowArgs args{ a, 0 };
		const size_t lds = row_lds_bytes(a.w.pitch, args.groups);
		if (lds > kRowLdsLimit)
		{
			return false;
		}
		// enough wavefronts to cover the card matters more than rows per wavefront
		if (a.glu || a.w.n >= 2048)
		{
			launch_row<2>(args, lds, s);
		}
		else
		{
			launch_row<1>(args, lds, s);
		}
		return true;
	}

	void launch_dense_rows(const DenseRows& a, hipStream_t s)
	{
		if (a.m <= 0 || a.w.n <= 0)
		{
			return;
		}
		TileArgs args{ a, 0, 0 };
		if (a.f32)
		{
			args.m_tiles = (a.m + kF32Tile - 1) / kF32Tile;
			args.n_tiles = (a.w.n + kF32Tile - 1) / kF32Tile;
			const int per = (args.m_tiles * args.n_tiles + 7) / 8;
			dense_tile_f32_kernel<<<dim3(8 * per), dim3(256), 0, s>>>(args);
			return;
		}
		if (a.m <= 32)
		{
			launch_tile<32, 64, 1, 4>(args, s);
		}
		else if (tiles(a, 128, 128) >= 384)
		{
			launch_tile<128, 128, 2, 2>(args, s);
		}
		else if (a.m > 64 && tiles(a, 128, 64) >= 192)
		{
			launch_tile<128, 64, 2, 2>(args, s);
		}
		else
		{
			launch_tile<64, 64, 2, 2>(args, s);
		}
	}
} // namespace litenn_hip
