// Linear layers whose weights stay in bfloat16 (see dense.hip): the matrix layout in HBM and the
// launchers used by the C ABI and by the layered decoder.
#pragma once

#include "common.hpp"

namespace litenn_hip
{
	// Rows of weights start on 128-byte boundaries: a row of k weights occupies dense_pitch(k)
	// elements, zeros behind the k-th.  Activation buffers that feed the matrix cores have the same
	// pitch (what lies behind the k-th element there is never used).
	inline int dense_pitch(int k) { return (k + 63) & ~63; }

	struct DenseMatrix
	{
		const uint16_t* w = nullptr; // [n, pitch] bfloat16
		int n = 0, k = 0, pitch = 0;
	};

	// y = g sigmoid(alpha g) (u + shift) with g = min(g, limit), u = clamp(u, -limit, limit); an infinite limit,
	// alpha 1 and shift 0 make it silu(g) u
	struct ClampedGlu
	{
		float limit = 0.0f, alpha = 0.0f, shift = 0.0f;
	};

	// ---- one activation row (decode): Float32 activations, weights streamed once ----------------
	enum DensePrologue
	{
		kRowPlain = 0,    // x as it is
		kRowAddNorm = 1,  // x' = x + norm(sub) sub_w (sub may be null); x' -> x_out if given; norm(x') norm_w, or x' without norm_w
		kRowHeadGate = 2, // per head of `vdim`: norm(x) norm_w, then times silu(gate)
	};
	struct DenseRow
	{
		DenseMatrix w;
		const float* x = nullptr; // [k]
		float* y = nullptr;       // [n], or [n / 2] with glu
		int prologue = kRowPlain;
		const float* sub = nullptr;
		const float* sub_w = nullptr;
		const float* norm_w = nullptr;
		float* x_out = nullptr;
		const float* gate = nullptr;
		int vdim = 0;
		float eps = 0.0f;
		bool glu = false; // rows 2i and 2i + 1 are gate and up of output i
		ClampedGlu act;
		float softcap = 0.0f; // > 0: y becomes softcap tanh(y / softcap)
	};
	// false, with nothing launched, when k does not fit the workgroup's LDS
	bool launch_dense_row(const DenseRow& a, hipStream_t s);
	size_t dense_row_max_k();

	// ---- many activation rows (prompt): matrix cores ---------------------------------------------
	enum DenseOut
	{
		kOutF32 = 0,     // c is Float32
		kOutOperand = 1, // c has the operand type (bfloat16, or Float32 with f32 set)
		kOutGlu = 2,     // operand type, n / 2 columns from interleaved gate / up rows
	};
	struct DenseRows
	{
		DenseMatrix w;
		const void* a = nullptr; // [m, lda] bfloat16, or Float32 with f32 set; readable up to column pitch of w
		int lda = 0;
		int a_first = 0, a_ring = 0; // a_ring > 0: row r lives at (a_first + r) modulo a_ring, m <= a_ring
		int m = 0;
		void* c = nullptr;
		int ldc = 0; // a multiple of 4 for the operand types
		int out = kOutF32;
		// kOutF32 with bfloat16 operands: the products of `splits` ranges of K, split_stride floats apart, to be
		// added by the reader (see dense_rows_splits)
		int splits = 1;
		size_t split_stride = 0;
		bool f32 = false; // Float32 operands (the bfloat16 weights widened exactly), f32 matrix instructions
		ClampedGlu act;
		float softcap = 0.0f; // kOutF32: > 0: c becomes softcap tanh(c / softcap)
	};
	constexpr int kDenseMaxSplits = 4;
	int dense_rows_splits(const DenseMatrix& w, int m);
	void launch_dense_rows(const DenseRows& a, hipStream_t s);
} // namespace litenn_hip

#if defined(__HIPCC__)
namespace litenn_hip
{
	__device__ __forceinline__ float bf16_to_f32(uint32_t bits) { return __uint_as_float(bits << 16); }

	// two floats to a pair of bfloat16, nearest-even
	__device__ __forceinline__ uint32_t pack_bf16(float a, float b)
	{
		typedef float f2 __attribute__((ext_vector_type(2)));
		typedef __bf16 b2 __attribute__((ext_vector_type(2)));
		const f2 v = { a, b };
		return __builtin_bit_cast(uint32_t, __builtin_convertvector(v, b2));
	}
	__device__ __forceinline__ uint16_t to_bf16(float a) { return static_cast<uint16_t>(pack_bf16(a, 0.0f)); }

	// an operand buffer's element types: bfloat16 as raw bits, or float
	__device__ __forceinline__ float operand_load(const uint16_t* p) { return bf16_to_f32(*p); }
	__device__ __forceinline__ float operand_load(const float* p) { return *p; }
	__device__ __forceinline__ void operand_store(uint16_t* p, float v) { *p = to_bf16(v); }
	__device__ __forceinline__ void operand_store(float* p, float v) { *p = v; }

	__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }

	__device__ __forceinline__ float soft_cap(float v, float cap) { return cap > 0.0f ? cap * tanhf(v / cap) : v; }

	__device__ __forceinline__ float clamped_glu(float g, float u, const ClampedGlu& c)
	{
		g = fminf(g, c.limit);
		u = fminf(fmaxf(u, -c.limit), c.limit);
		return g * sigmoid_f32(c.alpha * g) * (u + c.shift);
	}
} // namespace litenn_hip
#endif
