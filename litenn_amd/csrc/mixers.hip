// Two more mechanisms of the layered decoder for gfx950, and the launches that run them side by side on one
// token: attention whose query heads share key/value heads (queries and keys normalised as whole projections,
// rotary positions, sliding window over a ring of cached keys and values), and a state-space recurrence with one
// decay per head behind a short causal convolution (recurrent step, and a chunked form whose contractions
// run on the Float32 matrix instructions).  Norms, angles, scores, softmax and everything inside the recurrence
// are Float32.  The reference has no counterpart of these layers.
#include "layer_device.hpp"

#include <algorithm>
#include <cmath>

namespace litenn_hip
{
	namespace
	{
		// ---------------- queries and keys on their way in -------------------------------------------
		constexpr int kGroupedMaxDim = 512;

		// cosines and sines of one position's angles, by 256 threads; the angle in turns, reduced in double
		__device__ __forceinline__ void rotary_angles(const Rotary& rot, int position, float* cs, float* sn)
		{
			for (int i = threadIdx.x; i < rot.dims / 2; i += 256)
			{
				const double t = static_cast<double>(position) * rot.turns[i];
				sincospif(static_cast<float>(2.0 * (t - rint(t))), sn + i, cs + i);
			}
		}

		// element d of the head whose elements start at `first` of a projection x: normalised, then rotated
		__device__ __forceinline__ float rotated(const float* x, const float* w, float scale, int first, int d, const Rotary& rot,
		                                         const float* cs, const float* sn)
		{
			const float own = x[first + d] * scale * (w ? w[first + d] : 1.0f);
			const int half = rot.dims >> 1;
			if (d >= 2 * half)
			{
				return own;
			}
			const bool lower = d < half;
			const int i = lower ? d : d - half, other_d = lower ? d + half : i;
			const float other = x[first + other_d] * scale * (w ? w[first + other_d] : 1.0f);
			return lower ? own * cs[i] - other * sn[i] : own * cs[i] + other * sn[i];
		}

		// one over the root mean square of a whole projection (1 where it has no norm)
		__device__ __forceinline__ float projection_scale(const float* x, const float* w, int n, float eps, float* red)
		{
			if (!w)
			{
				return 1.0f;
			}
			float ss = 0.0f;
#pragma unroll 8
			for (int i = threadIdx.x; i < n; i += 256)
			{
				ss = fmaf(x[i], x[i], ss);
			}
			return 1.0f / sqrtf(block_sum256(ss, red) / static_cast<float>(n) + eps);
		}

		// four elements from element e (a multiple of 4) of n, zero beyond; the row must be readable up to a whole piece
		__device__ __forceinline__ floatx4 load_whole(const float* row, int e, int n)
		{
			floatx4 v = *reinterpret_cast<const floatx4*>(row + min(e, (n - 1) & ~3));
#pragma unroll
			for (int i = 0; i < 4; ++i)
			{
				v[i] = e + i < n ? v[i] : 0.0f;
			}
			return v;
		}

		// the same over two rows, one behind the other, the second one from element up4(n0)
		__device__ __forceinline__ floatx4 load_either(const float* a, int n0, const float* b, int n1, int e)
		{
			const int first = (n0 + 3) & ~3;
			return e < first ? load_whole(a, e, n0) : load_whole(b, e - first, n1);
		}

		// both sums over a workgroup of 256
		__device__ __forceinline__ float2 block_sums256(float2 v, float* red)
		{
			v.x = wave_sum(v.x);
			v.y = wave_sum(v.y);
			__syncthreads();
			if ((threadIdx.x & 63) == 0)
			{
				red[threadIdx.x >> 6] = v.x;
				red[4 + (threadIdx.x >> 6)] = v.y;
			}
			__syncthreads();
			return make_float2((red[0] + red[1]) + (red[2] + red[3]), (red[4] + red[5]) + (red[6] + red[7]));
		}

		__device__ __forceinline__ float sum_squares(const floatx4& v) { return (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }

		__device__ __forceinline__ void store_piece(uint16_t* p, const floatx4& v)
		{
			*reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
		}
		__device__ __forceinline__ void store_piece(float* p, const floatx4& v) { *reinterpret_cast<floatx4*>(p) = v; }

		// KEPT > 0: queries and keys of up to 1024 KEPT elements pass through LDS, read once; 0: any number
		template <typename T, int KEPT>
		__global__ __launch_bounds__(256) void grouped_append_kernel(const GroupedAttn a)
		{
			__shared__ float red[8];
			__shared__ __attribute__((aligned(16))) float cs[kGroupedMaxDim / 2], sn[kGroupedMaxDim / 2];
			__shared__ __attribute__((aligned(16))) float lds[KEPT > 0 ? 1024 * KEPT : 4];
			const int row = blockIdx.x, position = row_position(a.pos, row), tid = threadIdx.x;
			const HeadCache& c = a.cache;
			const float* q = a.q + static_cast<size_t>(row) * a.ld;
			const float* k = a.k + static_cast<size_t>(row) * a.ld;
			const float* v = a.v + static_cast<size_t>(row) * a.ld;
			const int q_cols = a.heads * c.dim, k_cols = c.heads * c.dim, v_cols = c.heads * c.vdim;
			const int k_at = (q_cols + 3) & ~3, half = a.rot.dims >> 1;
			float* q_out = a.q_out + static_cast<size_t>(row) * a.ldq;
			T* rows = static_cast<T*>(c.rows) + static_cast<size_t>(position % c.ring) * c.row_pitch();
			if constexpr (KEPT > 0)
			{
				floatx4 x[KEPT], w[KEPT];
#pragma unroll
				for (int i = 0; i < KEPT; ++i)
				{
					x[i] = load_either(q, q_cols, k, k_cols, 4 * (tid + 256 * i));
				}
#pragma unroll
				for (int i = 0; i < KEPT; ++i)
				{
					w[i] = a.q_norm ? load_either(a.q_norm, q_cols, a.k_norm, k_cols, 4 * (tid + 256 * i)) : floatx4{ 1.0f, 1.0f, 1.0f, 1.0f };
				}
				rotary_angles(a.rot, position, cs, sn);
				float2 ss = make_float2(0.0f, 0.0f);
#pragma unroll
				for (int i = 0; i < KEPT; ++i)
				{
					const int e = 4 * (tid + 256 * i);
					(e < k_at ? ss.x : ss.y) += sum_squares(x[i]);
					*reinterpret_cast<floatx4*>(lds + e) = x[i] * w[i];
				}
				ss = block_sums256(ss, red);
				const float q_scale = a.q_norm ? 1.0f / sqrtf(ss.x / static_cast<float>(q_cols) + a.eps) : 1.0f;
				const float k_scale = a.q_norm ? 1.0f / sqrtf(ss.y / static_cast<float>(k_cols) + a.eps) : 1.0f;
				if (c.dim % 4 == 0 && half % 4 == 0)
				{
					// four elements lie in one head and in one half of its pairs
					const auto turned = [&](int at, int d, float scale) {
						floatx4 x0 = *reinterpret_cast<const floatx4*>(lds + at + d);
						if (d < 2 * half)
						{
							const bool lower = d < half;
							const int i = lower ? d : d - half;
							const floatx4 x1 = *reinterpret_cast<const floatx4*>(lds + at + (lower ? d + half : i));
							const floatx4 co = *reinterpret_cast<const floatx4*>(cs + i), si = *reinterpret_cast<const floatx4*>(sn + i);
							x0 = lower ? x0 * co - x1 * si : x0 * co + x1 * si;
						}
						return x0 * scale;
					};
					for (int e = 4 * tid; e < q_cols; e += 1024)
					{
						const int d = e % c.dim;
						*reinterpret_cast<floatx4*>(q_out + e) = turned(e - d, d, q_scale);
					}
					for (int e = 4 * tid; e < k_cols; e += 1024)
					{
						const int d = e % c.dim;
						store_piece(rows + e / c.dim * c.head_stride() + d, turned(k_at + e - d, d, k_scale));
					}
				}
				else
				{
					for (int e = tid; e < q_cols; e += 256)
					{
						const int d = e % c.dim;
						q_out[e] = rotated(lds, nullptr, q_scale, e - d, d, a.rot, cs, sn);
					}
					for (int e = tid; e < k_cols; e += 256)
					{
						const int d = e % c.dim;
						operand_store(rows + e / c.dim * c.head_stride() + d, rotated(lds + k_at, nullptr, k_scale, e - d, d, a.rot, cs, sn));
					}
				}
			}
			else
			{
				rotary_angles(a.rot, position, cs, sn);
				const float q_scale = projection_scale(q, a.q_norm, q_cols, a.eps, red);
				const float k_scale = projection_scale(k, a.k_norm, k_cols, a.eps, red);
				__syncthreads();
				for (int e = tid; e < q_cols; e += 256)
				{
					const int d = e % c.dim;
					q_out[e] = rotated(q, a.q_norm, q_scale, e - d, d, a.rot, cs, sn);
				}
				for (int e = tid; e < k_cols; e += 256)
				{
					const int d = e % c.dim;
					operand_store(rows + e / c.dim * c.head_stride() + d, rotated(k, a.k_norm, k_scale, e - d, d, a.rot, cs, sn));
				}
			}
			if (c.vdim % 4 == 0)
			{
				for (int e = 4 * tid; e < v_cols; e += 1024)
				{
					store_piece(rows + e / c.vdim * c.head_stride() + c.key_pitch() + e % c.vdim, *reinterpret_cast<const floatx4*>(v + e));
				}
			}
			else
			{
				for (int e = tid; e < v_cols; e += 256)
				{
					operand_store(rows + e / c.vdim * c.head_stride() + c.key_pitch() + e % c.vdim, v[e]);
				}
			}
		}

		// ---------------- one token's attention --------------------------------------------------------
		// A workgroup takes up to kStepHeads query heads of one key/value head over one split of the visible
		// positions, in tiles of KT cached rows staged in LDS (one lane per key, or a quarter of one); per split and
		// head it leaves the running maximum (in units of log 2), the sum of weights and the weighted sum of values.
		// The token's own key and value go into the tile from the projections, and from there into the cache.
		constexpr int kStepHeads = 8, kStepMaxSplits = 64;

		// elements between the key rows of a tile: an odd number of 16-byte pieces
		template <typename T>
		__host__ __device__ constexpr int key_stride(int pitch)
		{
			return ((pitch * static_cast<int>(sizeof(T)) / 16) | 1) * (16 / static_cast<int>(sizeof(T)));
		}

		template <typename T, int KT>
		size_t grouped_step_lds(const GroupedAttn& a)
		{
			const HeadCache& c = a.cache;
			const size_t floats = ((a.rot.dims + 3) & ~3) + (kStepHeads + 1) * c.key_pitch() + c.value_pitch() + kStepHeads * KT;
			return sizeof(float) * floats + sizeof(T) * KT * static_cast<size_t>(key_stride<T>(c.key_pitch()) + c.value_pitch());
		}

		__device__ __forceinline__ void unpack8(const uint16_t* p, floatx4& lo, floatx4& hi)
		{
			const u32x4 w = *reinterpret_cast<const u32x4*>(p);
			lo = floatx4{ __uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
				          __uint_as_float(w.y & 0xffff0000u) };
			hi = floatx4{ __uint_as_float(w.z << 16), __uint_as_float(w.z & 0xffff0000u), __uint_as_float(w.w << 16),
				          __uint_as_float(w.w & 0xffff0000u) };
		}
		__device__ __forceinline__ void unpack8(const float* p, floatx4& lo, floatx4& hi)
		{
			lo = *reinterpret_cast<const floatx4*>(p);
			hi = *reinterpret_cast<const floatx4*>(p + 4);
		}
		__device__ __forceinline__ float2 unpack2(const uint16_t* p)
		{
			const uint32_t w = *reinterpret_cast<const uint32_t*>(p);
			return make_float2(__uint_as_float(w << 16), __uint_as_float(w & 0xffff0000u));
		}
		__device__ __forceinline__ float2 unpack2(const float* p) { return *reinterpret_cast<const float2*>(p); }

		__device__ __forceinline__ float dot8(const floatx4& a, const floatx4& b, const floatx4& x, const floatx4& y, float acc)
		{
#pragma unroll
			for (int i = 0; i < 4; ++i)
			{
				acc = fmaf(a[i], x[i], acc);
			}
#pragma unroll
			for (int i = 0; i < 4; ++i)
			{
				acc = fmaf(b[i], y[i], acc);
			}
			return acc;
		}

		// the least shift, up to 8, whose power of two is n or more
		__device__ __forceinline__ int shift_over(int n) { return min(8, 32 - __clz(n - 1)); }

		__host__ __device__ inline int grouped_chunks(int heads, int kv_heads)
		{
			return (heads / kv_heads + kStepHeads - 1) / kStepHeads;
		}
		__host__ __device__ inline int partial_pitch(int vdim) { return ((vdim + 3) & ~3) + 4; }

		template <typename T, int KT>
		__device__ void grouped_step_block(const GroupedAttn& a, int block, float* lds, float* red)
		{
			const HeadCache& c = a.cache;
			const int share = a.heads / c.heads, chunks = grouped_chunks(a.heads, c.heads);
			const int kvh = block % c.heads, chunk = block / c.heads % chunks, split = block / c.heads / chunks;
			const int head0 = kvh * share + chunk * kStepHeads;
			const int heads = min(kStepHeads, share - chunk * kStepHeads);
			const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
			const int kp = c.key_pitch(), vp = c.value_pitch(), rp = c.row_pitch(), ks = key_stride<T>(kp);
			float* const cs = lds;
			float* const sn = cs + a.rot.dims / 2;
			float* const qs = lds + ((a.rot.dims + 3) & ~3); // [kStepHeads][kp], and the token's own key behind them
			float* const own_key = qs + kStepHeads * kp;
			float* const own_value = own_key + kp;     // [vp]
			float* const weights = own_value + vp;     // [kStepHeads][KT]
			T* const k_tile = reinterpret_cast<T*>(weights + kStepHeads * KT); // [KT][ks]
			T* const v_tile = k_tile + KT * ks;                                // [KT][vp]

			const int last = row_position(a.pos, 0);
			const int first = max(0, last - a.window + 1);
			const int tiles = (last - first) / KT + 1;
			const int per = (tiles + a.splits - 1) / a.splits;
			const int t0 = split * per, t1 = min(tiles, t0 + per);
			float* const partial = a.partial + static_cast<size_t>(split) * a.heads * partial_pitch(c.vdim);
			if (t0 >= t1)
			{
				for (int i = tid; i < heads * partial_pitch(c.vdim); i += 256)
				{
					const int at = i % partial_pitch(c.vdim);
					partial[static_cast<size_t>(head0) * partial_pitch(c.vdim) + i] = at == partial_pitch(c.vdim) - 4 ? -INFINITY : 0.0f;
				}
				return;
			}
			// Threads are dealt to rows by shifts (a kernel this short is bound by the instructions it fetches): a tile's
			// rows in 16-byte pieces, one piece column per thread; its first kAhead pieces are requested before anything waits
			constexpr int E = 16 / static_cast<int>(sizeof(T)), kAhead = 8;
			const int row_pieces = rp / E, piece_shift = shift_over(row_pieces);
			const int piece_row = tid >> piece_shift, piece_step = 256 >> piece_shift, piece = tid & ((1 << piece_shift) - 1);
			const int piece_col = min(piece, row_pieces - 1) * E;
			const T* const cache = static_cast<const T*>(c.rows) + kvh * c.head_stride() + piece_col;
			T* const piece_to = piece_col < kp ? k_tile + piece_col : v_tile + piece_col - kp;
			const int piece_stride = piece_col < kp ? ks : vp;
			int ring_at = (first + t0 * KT) % c.ring; // ring row of the tile's first position
			const auto piece_of = [&](int count, int row) {
				int r = ring_at + min(row, count - 1);
				r -= r >= c.ring ? c.ring : 0;
				return *reinterpret_cast<const u32x4*>(cache + static_cast<size_t>(r) * rp);
			};
			u32x4 ahead[kAhead];
			const auto request = [&](int base) {
				const int count = min(KT, last - base + 1);
#pragma unroll
				for (int i = 0; i < kAhead; ++i)
				{
					ahead[i] = piece_of(count, piece_row + i * piece_step);
				}
			};
			request(first + t0 * KT);

			// this workgroup's queries and key as projected, times the norm's weights, and the value; what lies behind a
			// head is zero.  All of it is requested before anything waits.
			const int q_cols = a.heads * c.dim, k_cols = c.heads * c.dim;
			constexpr int kQuads = 4;
			float2 ss = make_float2(0.0f, 0.0f);
			floatx4 all_q[kQuads], all_k;
#pragma unroll
			for (int i = 0; i < kQuads; ++i)
			{
				all_q[i] = load_whole(a.q, 4 * (tid + 256 * i), q_cols);
			}
			all_k = load_whole(a.k, 4 * tid, k_cols);
			const int own_shift = shift_over(kp), own_d = tid & ((1 << own_shift) - 1);
			const int own_row = tid >> own_shift, own_step = 256 >> own_shift; // a row longer than 256 takes all threads twice
			for (int d = own_d; d < kp; d += 256)
			{
				constexpr int kRows = 3;
				for (int row = own_row; row <= heads; row += kRows * own_step)
				{
					float x[kRows], w[kRows];
#pragma unroll
					for (int u = 0; u < kRows; ++u)
					{
						const int hq = min(row + u * own_step, heads);
						const int at = (hq < heads ? head0 + hq : kvh) * c.dim + min(d, c.dim - 1);
						x[u] = (hq < heads ? a.q : a.k)[at];
						w[u] = a.q_norm ? (hq < heads ? a.q_norm : a.k_norm)[at] : 1.0f;
					}
#pragma unroll
					for (int u = 0; u < kRows; ++u)
					{
						const int hq = min(row + u * own_step, heads);
						(hq < heads ? qs + hq * kp : own_key)[d] = d < c.dim ? x[u] * w[u] : 0.0f;
					}
				}
			}
			for (int i = tid; i < vp; i += 256)
			{
				own_value[i] = i < c.vdim ? a.v[kvh * c.vdim + i] : 0.0f;
			}
			rotary_angles(a.rot, last, cs, sn);
#pragma unroll
			for (int i = 0; i < kQuads; ++i)
			{
				ss.x += sum_squares(all_q[i]);
			}
			ss.y = sum_squares(all_k);
			for (int i = 4 * (tid + 256 * kQuads); i < q_cols; i += 1024)
			{
				ss.x += sum_squares(load_whole(a.q, i, q_cols));
			}
			for (int i = 4 * (tid + 256); i < k_cols; i += 1024)
			{
				ss.y += sum_squares(load_whole(a.k, i, k_cols));
			}
			ss = block_sums256(ss, red);
			const float q_scale = (a.q_norm ? 1.0f / sqrtf(ss.x / static_cast<float>(q_cols) + a.eps) : 1.0f) * (a.scale * kLog2e);
			const float k_scale = a.q_norm ? 1.0f / sqrtf(ss.y / static_cast<float>(k_cols) + a.eps) : 1.0f;
			// scaled and rotated where they are: a thread owns a pair, or an element that passes unchanged
			{
				const int half = a.rot.dims >> 1;
				for (int m = own_d; m < kp - half; m += 256)
				{
					for (int row = own_row; row <= heads; row += own_step)
					{
						const float by = row < heads ? q_scale : k_scale;
						float* const x = row < heads ? qs + row * kp : own_key;
						if (m < half)
						{
							const float u = x[m] * by, v = x[m + half] * by;
							x[m] = u * cs[m] - v * sn[m];
							x[m + half] = v * cs[m] + u * sn[m];
						}
						else
						{
							x[m + half] *= by;
						}
					}
				}
			}

			// wavefront w works on heads w and w + 4 of the workgroup's
			static_assert(kStepHeads == 8, "two heads per wavefront");
			constexpr int kCols = KT == 64 ? 2 : kGroupedMaxDim / 128;
			float2 o[2][kCols];
			float run_m[2] = { -INFINITY, -INFINITY }, run_l[2] = { 0.0f, 0.0f };
#pragma unroll
			for (int u = 0; u < 2; ++u)
			{
#pragma unroll
				for (int i = 0; i < kCols; ++i)
				{
					o[u][i] = make_float2(0.0f, 0.0f);
				}
			}
			for (int t = t0; t < t1; ++t)
			{
				const int base = first + t * KT;
				const int count = min(KT, last - base + 1);
				__syncthreads(); // the previous tile has been consumed
				const auto stage = [&](int row, u32x4 w) {
					if (row < KT && piece < row_pieces && base + row != last)
					{
						if (row >= count)
						{
							w = u32x4{ 0u, 0u, 0u, 0u };
						}
						*reinterpret_cast<u32x4*>(piece_to + row * piece_stride) = w;
					}
				};
#pragma unroll
				for (int i = 0; i < kAhead; ++i)
				{
					stage(piece_row + i * piece_step, ahead[i]);
				}
				for (int row = piece_row + kAhead * piece_step; row < KT; row += piece_step)
				{
					stage(row, piece_of(count, row));
				}
				if (base + count - 1 == last)
				{
					T* const row = static_cast<T*>(c.rows) + kvh * c.head_stride() + static_cast<size_t>(last % c.ring) * rp;
					for (int i = tid; i < rp; i += 256)
					{
						const int e = i < kp ? i : i - kp;
						const float x = own_key[i]; // the value follows the key
						operand_store(i < kp ? k_tile + (count - 1) * ks + e : v_tile + (count - 1) * vp + e, x);
						if (e < (i < kp ? c.dim : c.vdim) && chunk == 0)
						{
							operand_store(row + i, x);
						}
					}
				}
				if (t + 1 < t1)
				{
					ring_at += KT; // there is another tile: the ring is longer than this one
					ring_at -= ring_at >= c.ring ? c.ring : 0;
					request(base + KT);
				}
				__syncthreads();
				// scores: kParts lanes per key, each a share of the key
				constexpr int kParts = 64 / KT;
				const int key = lane % KT, part = lane / KT;
				float acc[2] = { 0.0f, 0.0f };
				{
					const int all = kp / 8, c0 = all * part / kParts, c1 = all * (part + 1) / kParts;
					const T* kr = k_tile + key * ks;
					const float* q0 = qs + wave * kp;
					const float* q1 = qs + (wave + 4) * kp;
#pragma unroll 4
					for (int i = c0; i < c1; ++i)
					{
						floatx4 lo, hi;
						unpack8(kr + 8 * i, lo, hi);
						acc[0] = dot8(lo, hi, *reinterpret_cast<const floatx4*>(q0 + 8 * i), *reinterpret_cast<const floatx4*>(q0 + 8 * i + 4), acc[0]);
						acc[1] = dot8(lo, hi, *reinterpret_cast<const floatx4*>(q1 + 8 * i), *reinterpret_cast<const floatx4*>(q1 + 8 * i + 4), acc[1]);
					}
				}
#pragma unroll
				for (int u = 0; u < 2; ++u)
				{
#pragma unroll
					for (int off = KT; off < 64; off *= 2)
					{
						acc[u] += __shfl_xor(acc[u], off, 64);
					}
					const float score = key < count ? acc[u] : -INFINITY;
					const float new_m = fmaxf(run_m[u], wave_max(score));
					const float corr = exp2_f32(run_m[u] - new_m);
					const float p = exp2_f32(score - new_m);
					run_l[u] = run_l[u] * corr + wave_sum(part == 0 ? p : 0.0f);
					run_m[u] = new_m;
					if (part == 0)
					{
						weights[(wave + 4 * u) * KT + key] = p;
					}
#pragma unroll
					for (int i = 0; i < kCols; ++i)
					{
						o[u][i].x *= corr;
						o[u][i].y *= corr;
					}
				}
				// written and read by this wavefront only, in order
				__builtin_amdgcn_wave_barrier();
				const float* w0 = weights + wave * KT;
				const float* w1 = weights + (wave + 4) * KT;
#pragma unroll 2
				for (int kk = 0; kk < KT; kk += 4) // rows beyond the last position are zero, and so are their weights
				{
					const floatx4 p0 = *reinterpret_cast<const floatx4*>(w0 + kk), p1 = *reinterpret_cast<const floatx4*>(w1 + kk);
#pragma unroll
					for (int e = 0; e < 4; ++e)
					{
#pragma unroll
						for (int i = 0; i < kCols; ++i)
						{
							if (128 * i < vp) // uniform; what lies behind the last column is not stored
							{
								const float2 x = unpack2(v_tile + (kk + e) * vp + min(2 * lane + 128 * i, vp - 2));
								o[0][i].x = fmaf(p0[e], x.x, o[0][i].x);
								o[0][i].y = fmaf(p0[e], x.y, o[0][i].y);
								o[1][i].x = fmaf(p1[e], x.x, o[1][i].x);
								o[1][i].y = fmaf(p1[e], x.y, o[1][i].y);
							}
						}
					}
				}
			}
#pragma unroll
			for (int u = 0; u < 2; ++u)
			{
				const int hq = wave + 4 * u;
				if (hq >= heads)
				{
					break;
				}
				float* dst = partial + static_cast<size_t>(head0 + hq) * partial_pitch(c.vdim);
#pragma unroll
				for (int i = 0; i < kCols; ++i)
				{
					const int col = 2 * lane + 128 * i;
					if (col < ((c.vdim + 3) & ~3))
					{
						*reinterpret_cast<float2*>(dst + col) = o[u][i];
					}
				}
				if (lane == 0)
				{
					dst[(c.vdim + 3) & ~3] = run_m[u];
					dst[((c.vdim + 3) & ~3) + 1] = run_l[u];
				}
			}
		}

		// out[e] = out_scale (sum over splits of weight times value sum) / (sum of weight times weight sum), one output
		// per thread
		__device__ __forceinline__ void grouped_merge(const GroupedAttn& a, int e, float out_scale, float* out)
		{
			const int vdim = a.cache.vdim, pitch = partial_pitch(vdim);
			if (e >= a.heads * vdim)
			{
				return;
			}
			const float* part = a.partial + static_cast<size_t>(e / vdim) * pitch;
			const size_t step = static_cast<size_t>(a.heads) * pitch;
			const int col = e % vdim, at = pitch - 4;
			constexpr int kAhead = 16;
			float run_m = -INFINITY, sum = 0.0f, acc = 0.0f;
			for (int s0 = 0; s0 < a.splits; s0 += kAhead)
			{
				float m[kAhead], l[kAhead], v[kAhead];
#pragma unroll
				for (int i = 0; i < kAhead; ++i)
				{
					const float* p = part + min(s0 + i, a.splits - 1) * step;
					m[i] = p[at];
					l[i] = p[at + 1];
					v[i] = p[col];
				}
				float top = run_m;
#pragma unroll
				for (int i = 0; i < kAhead; ++i)
				{
					m[i] = s0 + i < a.splits ? m[i] : -INFINITY;
					top = fmaxf(top, m[i]);
				}
				// split 0 always holds a position: top is finite
				const float corr = exp2_f32(run_m - top);
				sum *= corr;
				acc *= corr;
				run_m = top;
#pragma unroll
				for (int i = 0; i < kAhead; ++i)
				{
					const float w = exp2_f32(m[i] - top);
					sum = fmaf(w, l[i], sum);
					acc = fmaf(w, v[i], acc);
				}
			}
			out[e] = acc / sum * out_scale;
		}

		// ---------------- state-space recurrence --------------------------------------------------------
		constexpr int kSsmMaxState = 512, kSsmCols = 32;
		constexpr size_t kSsmStepFloats = 2 * kSsmMaxState + 32 * (kSsmCols + 4) + kSsmCols;

		__device__ __forceinline__ float silu_f32(float v) { return v * sigmoid_f32(v); }

		__device__ __forceinline__ float softplus_f32(float v) { return fmaxf(v, 0.0f) + log1pf(expf(-fabsf(v))); }

		// One token: a workgroup takes kSsmCols value columns of one head; a thread holds state rows 32 apart of
		// four columns.
		__device__ void ssm_step_block(const Ssm& a, int block, float* lds)
		{
			float* const bs = lds;                    // dt B
			float* const cs = bs + kSsmMaxState;      // C
			float* const sums = cs + kSsmMaxState;    // [32][kSsmCols + 4]
			float* const xs = sums + 32 * (kSsmCols + 4);
			const int h = block % a.heads, slice = block / a.heads, tid = threadIdx.x;
			const int inner = a.inner(), channels = a.channels(), pitch = ssm_state_pitch(a.vdim);
			const int group = h / (a.heads / a.groups);
			const int e = slice * kSsmCols + (tid & 7) * 4;
			const int r0 = tid >> 3;
			const bool inside = e < pitch;
			float* const state = a.states + static_cast<size_t>(h) * a.state * pitch + e;
			constexpr int kRows = 4; // state rows of a thread that travel together
			floatx4 st[kRows];
			const auto load_rows = [&](int first) {
#pragma unroll
				for (int i = 0; i < kRows; ++i)
				{
					const int r = first + r0 + 32 * i;
					st[i] = inside && r < a.state ? *reinterpret_cast<const floatx4*>(state + static_cast<size_t>(r) * pitch)
					                              : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
				}
			};
			load_rows(0);
			const int p = row_position(a.pos, 0);
			const float* const raw = a.in + inner; // x | B | C
			const float dt_raw = a.in[inner + channels + h] + a.dt_bias[h], rate = a.a_log[h];
			// the last kNear taps of a channel and its input travel together
			constexpr int kNear = 4;
			struct Window
			{
				float w[kNear], x[kNear], bias;
			};
			const int slot0 = p % a.taps; // ring row of the token's own input
			const auto slot = [&](int back) { return slot0 - back + (slot0 < back ? a.taps : 0); };
			const auto request = [&](int ch) {
				Window t;
#pragma unroll
				for (int back = 0; back < kNear; ++back)
				{
					t.w[back] = a.conv_w[static_cast<size_t>(a.taps - 1 - min(back, a.taps - 1)) * channels + ch];
					t.x[back] = back ? a.ring[static_cast<size_t>(slot(min(back, a.taps - 1))) * channels + ch] : raw[ch];
				}
				t.bias = a.conv_b[ch];
				return t;
			};
			const auto convolved = [&](const Window& t, int ch, bool keep) {
				float acc = fmaf(t.w[0], t.x[0], t.bias);
#pragma unroll
				for (int back = 1; back < kNear; ++back)
				{
					acc = back < a.taps && p >= back ? fmaf(t.w[back], t.x[back], acc) : acc;
				}
				for (int back = kNear; back < a.taps && back <= p; ++back)
				{
					acc = fmaf(a.conv_w[static_cast<size_t>(a.taps - 1 - back) * channels + ch],
					           a.ring[static_cast<size_t>(slot(back)) * channels + ch], acc);
				}
				if (keep)
				{
					a.ring[static_cast<size_t>(slot0) * channels + ch] = t.x[0];
				}
				return silu_f32(acc);
			};
			// B and C of the group (one workgroup of a group stores their inputs), then this workgroup's columns of x
			const bool keep = slice == 0 && h % (a.heads / a.groups) == 0;
			const int total = 2 * a.state + kSsmCols;
			const auto channel = [&](int i) {
				i = min(i, total - 1);
				return i < a.state       ? inner + group * a.state + i
				       : i < 2 * a.state ? inner + (a.groups - 1 + group) * a.state + i
				                         : h * a.vdim + min(slice * kSsmCols + i - 2 * a.state, a.vdim - 1);
			};
			const int col = slice * kSsmCols + tid;
			float dt = 0.0f, decay = 0.0f;
			for (int first = 0; first < total; first += 512)
			{
				const int i0 = first + tid, i1 = i0 + 256;
				const Window w0 = request(channel(i0)), w1 = request(channel(i1));
				if (first == 0)
				{
					dt = softplus_f32(dt_raw);
					decay = expf(-expf(rate) * dt);
				}
				const auto put = [&](int i, const Window& w) {
					if (i >= total)
					{
						return;
					}
					const bool is_x = i >= 2 * a.state, inside_head = slice * kSsmCols + i - 2 * a.state < a.vdim;
					const float v = convolved(w, channel(i), is_x ? inside_head : keep);
					float* const to = is_x ? xs + i - 2 * a.state : i < a.state ? bs + i : cs + i - a.state;
					*to = is_x && !inside_head ? 0.0f : i < a.state ? v * dt : v;
				};
				put(i0, w0);
				put(i1, w1);
			}
			__syncthreads();
			const floatx4 x = *reinterpret_cast<const floatx4*>(xs + (tid & 7) * 4);
			floatx4 acc = { 0.0f, 0.0f, 0.0f, 0.0f };
			for (int first = 0; first < a.state; first += 32 * kRows)
			{
				if (first)
				{
					load_rows(first);
				}
#pragma unroll
				for (int i = 0; i < kRows; ++i)
				{
					const int r = first + r0 + 32 * i;
					if (r < a.state)
					{
						st[i] = st[i] * decay + x * bs[r];
						acc += st[i] * cs[r];
						if (inside)
						{
							*reinterpret_cast<floatx4*>(state + static_cast<size_t>(r) * pitch) = st[i];
						}
					}
				}
			}
			*reinterpret_cast<floatx4*>(sums + r0 * (kSsmCols + 4) + (tid & 7) * 4) = acc;
			__syncthreads();
			if (tid < kSsmCols && col < a.vdim)
			{
				float t = a.d[h] * xs[tid];
#pragma unroll
				for (int i = 0; i < 32; ++i)
				{
					t += sums[i * (kSsmCols + 4) + tid];
				}
				a.y[h * a.vdim + col] = t;
			}
		}

		template <typename T, int KT>
		__global__ __launch_bounds__(256) void mixer_step_kernel(const GroupedAttn attn, int attn_blocks, const Ssm ssm)
		{
			extern __shared__ __attribute__((aligned(16))) float step_lds[];
			__shared__ float red[8];
			if (static_cast<int>(blockIdx.x) < attn_blocks)
			{
				grouped_step_block<T, KT>(attn, static_cast<int>(blockIdx.x), step_lds, red);
			}
			else
			{
				ssm_step_block(ssm, static_cast<int>(blockIdx.x) - attn_blocks, step_lds);
			}
		}

		// one part of one row, by 256 threads
		template <typename T>
		__device__ void gated_norm_block(const GatedNorm& a, int row, int part, float* red)
		{
			constexpr int kKept = 16; // values a thread keeps in registers (wider parts are read again)
			const int n = a.width / a.parts, first = part * n;
			const float* y = a.y + static_cast<size_t>(row) * a.ldy + first;
			const float* z = a.z ? a.z + static_cast<size_t>(row) * a.ldz + first : nullptr;
			const float* w = a.norm_w + first;
			float kept[kKept], gate[kKept], weight[kKept];
#pragma unroll
			for (int e = 0; e < kKept; ++e)
			{
				const int i = threadIdx.x + 256 * e;
				kept[e] = i < n ? y[i] : 0.0f;
				gate[e] = z && i < n ? z[i] : 0.0f;
				weight[e] = i < n ? w[i] : 0.0f;
			}
			const auto value = [&](float v, float g) { return z ? v * silu_f32(g) : v; };
			float ss = 0.0f;
#pragma unroll
			for (int e = 0; e < kKept; ++e)
			{
				kept[e] = value(kept[e], gate[e]);
				ss = fmaf(kept[e], kept[e], ss);
			}
			for (int i = threadIdx.x + 256 * kKept; i < n; i += 256)
			{
				const float v = value(y[i], z ? z[i] : 0.0f);
				ss = fmaf(v, v, ss);
			}
			const float scale = a.scale / sqrtf(block_sum256(ss, red) / static_cast<float>(n) + a.eps);
			T* out = static_cast<T*>(a.out) + static_cast<size_t>(row) * a.ldo + first;
#pragma unroll
			for (int e = 0; e < kKept; ++e)
			{
				const int i = threadIdx.x + 256 * e;
				if (i < n)
				{
					operand_store(out + i, kept[e] * scale * weight[e]);
				}
			}
			for (int i = threadIdx.x + 256 * kKept; i < n; i += 256)
			{
				operand_store(out + i, value(y[i], z ? z[i] : 0.0f) * scale * w[i]);
			}
		}

		template <typename T>
		__global__ __launch_bounds__(256) void gated_norm_kernel(const GatedNorm a)
		{
			__shared__ float red[4];
			gated_norm_block<T>(a, blockIdx.x, blockIdx.y, red);
		}

		__global__ __launch_bounds__(256) void mixer_finish_kernel(const GroupedAttn attn, int attn_blocks, float out_scale,
		                                                           float* __restrict__ out, const GatedNorm norm)
		{
			__shared__ float red[4];
			if (static_cast<int>(blockIdx.x) < attn_blocks)
			{
				grouped_merge(attn, static_cast<int>(blockIdx.x) * 256 + static_cast<int>(threadIdx.x), out_scale, out);
			}
			else
			{
				gated_norm_block<float>(norm, 0, static_cast<int>(blockIdx.x) - attn_blocks, red);
			}
		}

		// ---- chunked form ------------------------------------------------------------------------------
		// Tokens in chunks of 64.  With L_t the sum of a head's log decays from the chunk's first token up to and
		// including token t (summed in double, so that differences of large sums keep the small decays):
		//   contribution of a chunk to the state:  sum_s (exp(L_end - L_s) dt_s B_s) x_s^T
		//   y_t = exp(L_t) S_begin^T C_t + sum_(s <= t) (C_t . B_s) exp(L_t - L_s) dt_s x_s + d x_t
		// No factor exceeds one whatever the decays are (they are kept in units of log 2).  The contractions run on
		// v_mfma_f32_16x16x4_f32.  Value columns are dealt out to the 16-wide tiles so that a lane's four consecutive
		// columns (one 16-byte access) belong to four tiles.
		constexpr int kChunk = 64, kSlab = 64, kSlabStride = 68, kSlice = 64;

		// chunk_states: [chunk][head][state][pitch] floats, then [chunk][head] decays over the chunk
		__device__ __forceinline__ float* chunk_decays(const Ssm& a, int chunks)
		{
			return a.chunk_states + static_cast<size_t>(chunks) * a.heads * a.state * ssm_state_pitch(a.vdim);
		}

		constexpr int kConvRows = 8; // rows of a thread

		// x | B | C behind convolution and silu, four channels per thread; the last column of workgroups makes the
		// step sizes and log decays.  TAPS > 0: that many taps, channels a multiple of 4, every input read once; 0: any.
		template <int TAPS>
		__global__ __launch_bounds__(256) void ssm_conv_kernel(const Ssm a)
		{
			const int inner = a.inner(), channels = a.channels(), ldx = a.ldx();
			const int block_row = static_cast<int>(blockIdx.y) * 4 * kConvRows;
			if (blockIdx.x + 1 == gridDim.x)
			{
				const int count = min(4 * kConvRows, a.rows - block_row);
				for (int i = threadIdx.x; i < count * a.heads; i += 256)
				{
					const int row = block_row + i / a.heads, h = i % a.heads;
					const float dt = softplus_f32(a.in[static_cast<size_t>(row) * a.ld + inner + channels + h] + a.dt_bias[h]);
					const size_t at = static_cast<size_t>(row) * a.heads + h;
					a.steps[at] = dt;
					a.steps[static_cast<size_t>(a.rows) * a.heads + at] = -expf(a.a_log[h]) * dt * kLog2e;
				}
				return;
			}
			const int ch = (static_cast<int>(blockIdx.x) * 64 + static_cast<int>(threadIdx.x & 63)) * 4;
			const int row0 = block_row + static_cast<int>(threadIdx.x >> 6) * kConvRows;
			if (ch >= channels || row0 >= a.rows)
			{
				return;
			}
			const int p0 = row_position(a.pos, 0);
			const auto input = [&](int row) {
				row = min(row, a.rows - 1);
				if (row >= 0)
				{
					return load_columns(a.in + static_cast<size_t>(row) * a.ld + inner, ch, channels);
				}
				return p0 + row >= 0 ? load_columns(a.ring + static_cast<size_t>((p0 + row) % a.taps) * channels, ch, channels)
				                     : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
			};
			const floatx4 bias = load_columns(a.conv_b, ch, channels);
			floatx4 acc[kConvRows];
#pragma unroll
			for (int t = 0; t < kConvRows; ++t)
			{
				acc[t] = bias;
			}
			if constexpr (TAPS > 0)
			{
				floatx4 in[kConvRows + TAPS - 1], w[TAPS];
				const float* const column = a.in + inner + ch;
#pragma unroll
				for (int i = 0; i < kConvRows + TAPS - 1; ++i)
				{
					const int row = min(max(row0 + i - (TAPS - 1), 0), a.rows - 1);
					in[i] = *reinterpret_cast<const floatx4_a4*>(column + static_cast<size_t>(row) * a.ld);
				}
#pragma unroll
				for (int tap = 0; tap < TAPS; ++tap)
				{
					w[tap] = *reinterpret_cast<const floatx4*>(a.conv_w + static_cast<size_t>(tap) * channels + ch);
				}
				if (row0 < TAPS - 1) // inputs from ahead of these rows
				{
#pragma unroll
					for (int i = 0; i < TAPS - 1; ++i)
					{
						if (row0 + i < TAPS - 1)
						{
							in[i] = input(row0 + i - (TAPS - 1));
						}
					}
				}
#pragma unroll
				for (int t = 0; t < kConvRows; ++t)
				{
#pragma unroll
					for (int tap = 0; tap < TAPS; ++tap)
					{
						acc[t] += w[tap] * in[t + tap];
					}
				}
			}
			else
			{
				for (int tap = 0; tap < a.taps; ++tap)
				{
					const floatx4 w = load_columns(a.conv_w + static_cast<size_t>(tap) * channels, ch, channels);
#pragma unroll
					for (int t = 0; t < kConvRows; ++t)
					{
						acc[t] += w * input(row0 + t - (a.taps - 1) + tap);
					}
				}
			}
#pragma unroll
			for (int t = 0; t < kConvRows; ++t)
			{
				if (row0 + t < a.rows)
				{
					floatx4 v;
#pragma unroll
					for (int i = 0; i < 4; ++i)
					{
						v[i] = silu_f32(acc[t][i]); // zero behind the last channel
					}
					*reinterpret_cast<floatx4*>(a.xbc + static_cast<size_t>(row0 + t) * ldx + ch) = v;
				}
			}
		}

		// Sums of a chunk's log decays up to and including every token, and its step sizes (zero behind the last
		// token), by the first wavefront.
		__device__ __forceinline__ void chunk_sums(const Ssm& a, int h, int row0, int count, double* sums, float* dts)
		{
			if (threadIdx.x < kChunk)
			{
				const int t = threadIdx.x;
				const size_t at = static_cast<size_t>(row0 + min(t, count - 1)) * a.heads + h;
				double l = t < count ? static_cast<double>(a.steps[static_cast<size_t>(a.rows) * a.heads + at]) : 0.0;
				dts[t] = t < count ? a.steps[at] : 0.0f;
#pragma unroll
				for (int off = 1; off < 64; off *= 2)
				{
					const double before = __shfl_up(l, off, 64);
					l += t >= off ? before : 0.0;
				}
				sums[t] = l;
			}
		}

		// a chunk's contribution: 64 state rows x 64 value columns of one head per workgroup
		__global__ __launch_bounds__(256) void ssm_state_kernel(const Ssm a)
		{
			__shared__ float ks[kChunk][kSlabStride];
			__shared__ double sums[kChunk];
			__shared__ float dts[kChunk];
			const int pitch = ssm_state_pitch(a.vdim), ldx = a.ldx();
			const int slabs = (a.state + kSlab - 1) / kSlab;
			const int h = static_cast<int>(blockIdx.x) % a.heads, rest = static_cast<int>(blockIdx.x) / a.heads;
			const int n0 = rest % slabs * kSlab, v0 = rest / slabs * kSlice;
			const int chunk = blockIdx.y, row0 = chunk * kChunk, count = min(kChunk, a.rows - row0);
			const int lane = threadIdx.x & 63, part = threadIdx.x >> 6;
			const int j = lane & 15, g = lane >> 4;
			const int e = v0 + 4 * j;
			const float* const xs = a.xbc + h * a.vdim;
			const float* const bs = a.xbc + a.inner() + h / (a.heads / a.groups) * a.state;
			// the values are requested first: half of them travel while the keys are decayed
			constexpr int kSteps = kChunk / 4, kAhead = 8;
			const auto value = [&](int step) {
				return load_columns(xs + static_cast<size_t>(row0 + min(4 * step + g, count - 1)) * ldx, e, a.vdim);
			};
			floatx4 ahead[kAhead];
#pragma unroll
			for (int i = 0; i < kAhead; ++i)
			{
				ahead[i] = value(i);
			}
			// thread: one state row, 16 tokens
			const bool live = n0 + lane < a.state;
			float b[16];
#pragma unroll
			for (int t = 0; t < 16; ++t)
			{
				const int row = 16 * part + t;
				b[t] = live && row < count ? bs[static_cast<size_t>(row0 + row) * ldx + n0 + lane] : 0.0f;
			}
			chunk_sums(a, h, row0, count, sums, dts);
			__syncthreads();
			const double end = sums[kChunk - 1];
			if (rest == 0 && threadIdx.x == 0)
			{
				chunk_decays(a, gridDim.y)[static_cast<size_t>(chunk) * a.heads + h] = exp2_f32(static_cast<float>(end));
			}
#pragma unroll
			for (int t = 0; t < 16; ++t)
			{
				const int row = 16 * part + t;
				ks[row][lane] = b[t] * (exp2_f32(static_cast<float>(end - sums[row])) * dts[row]);
			}
			__syncthreads();
			floatx4 acc[4];
#pragma unroll
			for (int i = 0; i < 4; ++i)
			{
				acc[i] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
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
				for (int i = 0; i < 4; ++i)
				{
					acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf, vv[i], acc[i], 0, 0, 0);
				}
			}
			float* dst = a.chunk_states + (static_cast<size_t>(chunk) * a.heads + h) * a.state * pitch;
#pragma unroll
			for (int r = 0; r < 4; ++r)
			{
				const int n = n0 + 16 * part + 4 * g + r;
				if (n < a.state && e < pitch)
				{
					*reinterpret_cast<floatx4*>(dst + static_cast<size_t>(n) * pitch + e) =
					    floatx4{ acc[0][r], acc[1][r], acc[2][r], acc[3][r] };
				}
			}
		}

		// Replaces every chunk's contribution by the state the chunk begins with; ends with the new state.  The
		// workgroups behind those store the convolution's last inputs.
		__global__ __launch_bounds__(256) void ssm_scan_kernel(const Ssm a, int chunks, int scan_blocks)
		{
			if (static_cast<int>(blockIdx.x) >= scan_blocks)
			{
				const int kept = min(a.rows, a.taps), channels = a.channels();
				const int i = (static_cast<int>(blockIdx.x) - scan_blocks) * 256 + static_cast<int>(threadIdx.x);
				if (i < kept * channels)
				{
					const int row = a.rows - kept + i / channels, ch = i % channels;
					a.ring[static_cast<size_t>(row_position(a.pos, row) % a.taps) * channels + ch] =
					    a.in[static_cast<size_t>(row) * a.ld + a.inner() + ch];
				}
				return;
			}
			const int pitch = ssm_state_pitch(a.vdim), quads = pitch >> 2;
			const int rows = a.heads * a.state;
			const int i = static_cast<int>(blockIdx.x) * 256 + static_cast<int>(threadIdx.x);
			if (i >= rows * quads)
			{
				return;
			}
			const size_t at = static_cast<size_t>(i) * 4, step = static_cast<size_t>(rows) * pitch;
			const float* decay = chunk_decays(a, chunks) + i / quads / a.state;
			floatx4 s = *reinterpret_cast<floatx4*>(a.states + at);
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
					dec[u] = decay[static_cast<size_t>(c) * a.heads];
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
			*reinterpret_cast<floatx4*>(a.states + at) = s;
		}

		// A wavefront makes 64 value columns of a block of 16 tokens of one head; y silu(z) goes where z was.
		__global__ __launch_bounds__(256) void ssm_out_kernel(const Ssm a)
		{
			__shared__ __attribute__((aligned(16))) float cs[kChunk][kSlabStride];
			__shared__ __attribute__((aligned(16))) float bs[kChunk][kSlabStride];
			__shared__ double sums[kChunk];
			__shared__ float dts[kChunk];
			const int pitch = ssm_state_pitch(a.vdim), ldx = a.ldx(), vdim = a.vdim;
			const int h = static_cast<int>(blockIdx.x) % a.heads, v0 = static_cast<int>(blockIdx.x) / a.heads * kSlice;
			const int chunk = blockIdx.y, row0 = chunk * kChunk, count = min(kChunk, a.rows - row0);
			const int lane = threadIdx.x & 63;
			const int block = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
			const int j = lane & 15, g = lane >> 4;
			const int e0 = v0 + 4 * j;
			const float* const state = a.chunk_states + (static_cast<size_t>(chunk) * a.heads + h) * a.state * pitch;
			const float* const xs = a.xbc + h * vdim;
			const float* const b_in = a.xbc + a.inner() + h / (a.heads / a.groups) * a.state;
			const float* const c_in = b_in + a.groups * a.state;
			chunk_sums(a, h, row0, count, sums, dts);

			floatx4 o[4];      // o[b][r]: value column v0 + 16 g + 4 r + b of token j of the block
			floatx4 scores[4]; // scores[back][r]: token 4 g + r of `block - back` against token j
#pragma unroll
			for (int b = 0; b < 4; ++b)
			{
				o[b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
				scores[b] = floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
			}
			for (int n0 = 0; n0 < a.state; n0 += kSlab)
			{
				// thread: one state row, 16 tokens
				const bool live = n0 + lane < a.state;
				float cv[16], bv[16];
#pragma unroll
				for (int t = 0; t < 16; ++t)
				{
					const int row = 16 * block + t;
					const size_t at = static_cast<size_t>(row0 + row) * ldx + n0 + lane;
					cv[t] = live && row < count ? c_in[at] : 0.0f;
					bv[t] = live && row < count ? b_in[at] : 0.0f;
				}
				__syncthreads();
#pragma unroll
				for (int t = 0; t < 16; ++t)
				{
					cs[16 * block + t][lane] = cv[t];
					bs[16 * block + t][lane] = bv[t];
				}
				__syncthreads();
#pragma unroll
				for (int quad = 0; quad < kSlab / 16; ++quad)
				{
					const int c = 16 * quad + 4 * g; // this lane's four state rows of the slab
					if (n0 + 16 * quad >= a.state)
					{
						break; // uniform
					}
					floatx4 sv[4];
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
						const int n = min(n0 + c + r, a.state - 1); // C is zero beyond
						sv[r] = e0 < pitch ? *reinterpret_cast<const floatx4*>(state + static_cast<size_t>(n) * pitch + e0)
						                   : floatx4{ 0.0f, 0.0f, 0.0f, 0.0f };
					}
					const floatx4 cq = *reinterpret_cast<const floatx4*>(&cs[16 * block + j][c]);
#pragma unroll
					for (int back = 0; back < 4; ++back)
					{
						if (back <= block) // uniform
						{
							const floatx4 bk = *reinterpret_cast<const floatx4*>(&bs[16 * (block - back) + j][c]);
#pragma unroll
							for (int r = 0; r < 4; ++r)
							{
								scores[back] = __builtin_amdgcn_mfma_f32_16x16x4f32(bk[r], cq[r], scores[back], 0, 0, 0);
							}
						}
					}
#pragma unroll
					for (int r = 0; r < 4; ++r)
					{
#pragma unroll
						for (int b = 0; b < 4; ++b)
						{
							o[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[r][b], cq[r], o[b], 0, 0, 0);
						}
					}
				}
			}
			const int row = 16 * block + j;
			const double mine = sums[row];
			const float from_begin = exp2_f32(static_cast<float>(mine));
#pragma unroll
			for (int b = 0; b < 4; ++b)
			{
				o[b] *= from_begin;
			}
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
						const int s = 16 * b + 4 * g + r;
						vv[r] = load_columns(xs + static_cast<size_t>(row0 + min(s, count - 1)) * ldx, e0, vdim);
						const float w = exp2_f32(static_cast<float>(fmin(mine - sums[s], 0.0))) * dts[s];
						scores[back][r] *= s <= row ? w : 0.0f;
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
			if (row >= count)
			{
				return;
			}
			const float skip = a.d[h];
			float* z = a.in + static_cast<size_t>(row0 + row) * a.ld + h * vdim;
			const float* x = xs + static_cast<size_t>(row0 + row) * ldx;
#pragma unroll
			for (int r = 0; r < 4; ++r)
			{
				const int e = v0 + 16 * g + 4 * r;
				if (e < vdim)
				{
					const floatx4 gate = load_columns(z, e, vdim), xv = load_columns(x, e, vdim);
					floatx4 y;
#pragma unroll
					for (int b = 0; b < 4; ++b)
					{
						y[b] = (o[b][r] + skip * xv[b]) * silu_f32(gate[b]);
					}
					if (e + 3 < vdim)
					{
						*reinterpret_cast<floatx4_a4*>(z + e) = y;
					}
					else
					{
#pragma unroll
						for (int b = 0; b < 3; ++b)
						{
							if (e + b < vdim)
							{
								z[e + b] = y[b];
							}
						}
					}
				}
			}
		}

		bool narrow_heads(const HeadCache& c) { return c.key_pitch() <= 256 && c.value_pitch() <= 256; }

		template <typename T>
		void launch_append(const GroupedAttn& a, hipStream_t s)
		{
			const size_t cols = ((static_cast<size_t>(a.heads) * a.cache.dim + 3) & ~size_t{ 3 }) + static_cast<size_t>(a.cache.heads) * a.cache.dim;
			if (cols <= 2048)
			{
				grouped_append_kernel<T, 2><<<dim3(a.rows), dim3(256), 0, s>>>(a);
			}
			else if (cols <= 5120)
			{
				grouped_append_kernel<T, 5><<<dim3(a.rows), dim3(256), 0, s>>>(a);
			}
			else if (cols <= 10240)
			{
				grouped_append_kernel<T, 10><<<dim3(a.rows), dim3(256), 0, s>>>(a);
			}
			else
			{
				grouped_append_kernel<T, 0><<<dim3(a.rows), dim3(256), 0, s>>>(a);
			}
		}

		template <typename T, int KT>
		void launch_step(const GroupedAttn& attn, int attn_blocks, const Ssm& ssm, int ssm_blocks, hipStream_t s)
		{
			const size_t lds = std::max(attn_blocks ? grouped_step_lds<T, KT>(attn) : size_t{ 0 }, sizeof(float) * kSsmStepFloats);
			allow_dynamic_lds(reinterpret_cast<const void*>(&mixer_step_kernel<T, KT>), 156 * 1024);
			mixer_step_kernel<T, KT><<<dim3(attn_blocks + ssm_blocks), dim3(256), lds, s>>>(attn, attn_blocks, ssm);
		}
	} // namespace

	int grouped_max_dim() { return kGroupedMaxDim; }
	int ssm_max_state() { return kSsmMaxState; }

	void launch_grouped_append(const GroupedAttn& a, hipStream_t s)
	{
		if (a.rows <= 0)
		{
			return;
		}
		if (a.cache.f32)
		{
			launch_append<float>(a, s);
		}
		else
		{
			launch_append<uint16_t>(a, s);
		}
	}

	WindowAttn grouped_window(const GroupedAttn& a, int past)
	{
		const HeadCache& c = a.cache;
		WindowAttn w;
		w.shape.heads = a.heads;
		w.shape.dim = c.dim;
		w.shape.vdim = c.vdim;
		w.shape.share = a.heads / c.heads;
		w.shape.window = a.window;
		w.shape.scale = a.scale;
		w.q = a.q_out;
		w.ldq = a.ldq;
		w.kv = c.rows;
		w.ldkv = c.row_pitch();
		w.v_first = c.key_pitch();
		w.k_head = w.v_head = c.head_stride();
		w.key_base = std::max(0, past - a.window + 1);
		w.keys = past + a.rows - w.key_base;
		w.kv_first = w.key_base % c.ring;
		w.kv_ring = c.ring;
		w.rows = a.rows;
		w.q_base = past;
		w.f32 = c.f32;
		return w;
	}

	// about two workgroups per CU, and no split shorter than a tile
	int grouped_step_splits(int heads, int kv_heads, int dim, int vdim, int window)
	{
		const int tile = dim <= 256 && vdim <= 256 ? 64 : 16;
		const int groups = kv_heads * grouped_chunks(heads, kv_heads), tiles = (window + tile - 1) / tile;
		return std::max(1, std::min({ tiles, 512 / std::max(1, groups), kStepMaxSplits }));
	}

	size_t grouped_step_partial_floats(int heads, int vdim, int splits)
	{
		return static_cast<size_t>(heads) * splits * partial_pitch(vdim);
	}

	size_t ssm_chunk_floats(int rows, const Ssm& a)
	{
		const size_t chunks = (static_cast<size_t>(rows) + kChunk - 1) / kChunk;
		return chunks * a.heads * (static_cast<size_t>(a.state) * ssm_state_pitch(a.vdim) + 1);
	}

	void launch_ssm_rows(const Ssm& a, hipStream_t s)
	{
		if (a.rows <= 0)
		{
			return;
		}
		const int conv_blocks = (a.ldx() / 4 + 63) / 64;
		const dim3 conv_grid(conv_blocks + 1, (a.rows + 4 * kConvRows - 1) / (4 * kConvRows));
		switch (a.channels() % 4 == 0 ? a.taps : 0)
		{
		case 2: ssm_conv_kernel<2><<<conv_grid, dim3(256), 0, s>>>(a); break;
		case 3: ssm_conv_kernel<3><<<conv_grid, dim3(256), 0, s>>>(a); break;
		case 4: ssm_conv_kernel<4><<<conv_grid, dim3(256), 0, s>>>(a); break;
		default: ssm_conv_kernel<0><<<conv_grid, dim3(256), 0, s>>>(a); break;
		}
		const int chunks = (a.rows + kChunk - 1) / kChunk;
		const int slabs = (a.state + kSlab - 1) / kSlab, slices = (a.vdim + kSlice - 1) / kSlice;
		ssm_state_kernel<<<dim3(a.heads * slabs * slices, chunks), dim3(256), 0, s>>>(a);
		const int scan_blocks = (a.heads * a.state * (ssm_state_pitch(a.vdim) >> 2) + 255) / 256;
		const int ring_blocks = (std::min(a.rows, a.taps) * a.channels() + 255) / 256;
		ssm_scan_kernel<<<dim3(scan_blocks + ring_blocks), dim3(256), 0, s>>>(a, chunks, scan_blocks);
		ssm_out_kernel<<<dim3(a.heads * slices, chunks), dim3(256), 0, s>>>(a);
	}

	void launch_gated_norm(const GatedNorm& a, hipStream_t s)
	{
		if (a.rows <= 0)
		{
			return;
		}
		if (a.f32)
		{
			gated_norm_kernel<float><<<dim3(a.rows, a.parts), dim3(256), 0, s>>>(a);
		}
		else
		{
			gated_norm_kernel<uint16_t><<<dim3(a.rows, a.parts), dim3(256), 0, s>>>(a);
		}
	}

	void launch_mixer_step(const GroupedAttn* attn, const Ssm* ssm, hipStream_t s)
	{
		const GroupedAttn a = attn ? *attn : GroupedAttn{};
		const Ssm b = ssm ? *ssm : Ssm{};
		const int attn_blocks = attn ? a.cache.heads * grouped_chunks(a.heads, a.cache.heads) * a.splits : 0;
		const int ssm_blocks = ssm ? b.heads * ((b.vdim + kSsmCols - 1) / kSsmCols) : 0;
		if (attn_blocks + ssm_blocks == 0)
		{
			return;
		}
		const bool narrow = !attn || narrow_heads(a.cache);
		if (attn && a.cache.f32)
		{
			narrow ? launch_step<float, 64>(a, attn_blocks, b, ssm_blocks, s) : launch_step<float, 16>(a, attn_blocks, b, ssm_blocks, s);
		}
		else
		{
			narrow ? launch_step<uint16_t, 64>(a, attn_blocks, b, ssm_blocks, s)
			       : launch_step<uint16_t, 16>(a, attn_blocks, b, ssm_blocks, s);
		}
	}

	void launch_mixer_finish(const GroupedAttn* attn, float out_scale, float* out, const GatedNorm* norm, hipStream_t s)
	{
		const GroupedAttn a = attn ? *attn : GroupedAttn{};
		const GatedNorm n = norm ? *norm : GatedNorm{};
		const int attn_blocks = attn ? (a.heads * a.cache.vdim + 255) / 256 : 0, norm_blocks = norm ? n.parts : 0;
		if (attn_blocks + norm_blocks > 0)
		{
			mixer_finish_kernel<<<dim3(attn_blocks + norm_blocks), dim3(256), 0, s>>>(a, attn_blocks, out_scale, out, n);
		}
	}
} // namespace litenn_hip
