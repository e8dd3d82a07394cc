// Device helpers shared by the kernels of the layer mechanisms.
#pragma once

#include "layers.hpp"

namespace litenn_hip
{
	typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
	typedef float floatx4 __attribute__((ext_vector_type(4)));
	typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
	typedef floatx4 floatx4_a4 __attribute__((aligned(4))); // global loads and stores take any 4-byte address

	constexpr float kLog2e = 1.44269504088896340736f;

	__device__ __forceinline__ float exp2_f32(float x) { return __builtin_amdgcn_exp2f(x); }

	__device__ __forceinline__ int row_position(const Position& p, int row)
	{
		return (p.dev ? *p.dev : 0) + p.add + row;
	}

	// sum over a workgroup of 256
	__device__ __forceinline__ float block_sum256(float v, float* red)
	{
		v = wave_sum(v);
		__syncthreads();
		if ((threadIdx.x & 63) == 0)
		{
			red[threadIdx.x >> 6] = v;
		}
		__syncthreads();
		return (red[0] + red[1]) + (red[2] + red[3]);
	}

	// four columns from column e of a row of `n`, zero beyond
	__device__ __forceinline__ floatx4 load_columns(const float* row, int e, int n)
	{
		floatx4 v = { 0.0f, 0.0f, 0.0f, 0.0f };
		if (e + 3 < n)
		{
			v = *reinterpret_cast<const floatx4_a4*>(row + e);
		}
		else
		{
#pragma unroll
			for (int i = 0; i < 3; ++i)
			{
				v[i] = e + i < n ? row[e + i] : 0.0f;
			}
		}
		return v;
	}
} // namespace litenn_hip
