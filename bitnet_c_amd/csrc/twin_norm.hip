// The residual sum of a block whose two halves read the same stream, and both halves' norms, in one pass over the row:
//     x <- x + y + sum_p z_p          y: one half's output (a tensor of the activations' type), z: slabs of float32 rows
//     f = 1 / sqrt(mean(x^2) + eps);   out_k = x f w_k    (k = 1, 2, an eps for each)
// y, z, and either output may be absent.  The slabs are added in slab order behind y; everything in float32; the order of
// the sums is a function of the row's width alone.
#include "common.h"

struct TwinArgs {
    float* x;                 // [n_rows, dim], rewritten when there is something to add
    const void* y;            // [n_rows, dim] of the outputs' type, or null
    const float* parts;       // n_parts slabs [n_rows, dim], or null
    int n_parts;
    size_t part_stride;
    const float* w[2];        // [dim]; null: no such output
    void* out[2];             // [n_rows, dim]
    float eps[2];
    int dim;
};

__device__ __forceinline__ float4 twin_load4(const bf16* p) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    return make_float4(bf16lo_to_f32(t.x), bf16hi_to_f32(t.x), bf16lo_to_f32(t.y), bf16hi_to_f32(t.y));
}
__device__ __forceinline__ float4 twin_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ void twin_store4(bf16* p, const float4& v) {
    bf16 t[4] = {from_f32<bf16>(v.x), from_f32<bf16>(v.y), from_f32<bf16>(v.z), from_f32<bf16>(v.w)};
    *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(t);
}
__device__ __forceinline__ void twin_store4(float* p, const float4& v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void twin_add4(float4& a, const float4& b) { a.x += b.x; a.y += b.y; a.z += b.z; a.w += b.w; }

// rows of up to 1024 NV elements (a multiple of 4): every load of the row and of the weights is issued before anything
// waits, the row stays in registers, one block reduction
template <typename T, int NV>
__global__ __launch_bounds__(256) void twin_norm_row_kernel(TwinArgs a) {
    __shared__ float scratch[16];
    const int dim = a.dim;
    const size_t row = (size_t)blockIdx.x * dim;
    float4 v[NV], w1[NV], w2[NV];
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = (k * 256 + threadIdx.x) * 4;
        v[k] = w1[k] = w2[k] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (i < dim) {
            v[k] = *reinterpret_cast<const float4*>(a.x + row + i);
            if (a.w[0]) w1[k] = *reinterpret_cast<const float4*>(a.w[0] + i);
            if (a.w[1]) w2[k] = *reinterpret_cast<const float4*>(a.w[1] + i);
        }
    }
    if (a.y) {
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < dim) twin_add4(v[k], twin_load4(reinterpret_cast<const T*>(a.y) + row + i));
        }
    }
    const float* pr = a.parts + row;
#pragma unroll 4
    for (int p = 0; p < a.n_parts; ++p, pr += a.part_stride) {           // several slabs' loads in flight at once
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < dim) twin_add4(v[k], twin_load4(pr + i));
        }
    }
    const bool store = a.y || a.n_parts > 0;
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = (k * 256 + threadIdx.x) * 4;
        if (i < dim && store) *reinterpret_cast<float4*>(a.x + row + i) = v[k];
        ss = fmaf(v[k].x, v[k].x, ss); ss = fmaf(v[k].y, v[k].y, ss);
        ss = fmaf(v[k].z, v[k].z, ss); ss = fmaf(v[k].w, v[k].w, ss);
    }
    if (!a.w[0] && !a.w[1]) return;                      // the sum alone
    ss = block_sum(ss, scratch);
#pragma unroll
    for (int o = 0; o < 2; ++o) {
        if (!a.w[o]) continue;
        const float f = 1.0f / sqrtf(ss / (float)dim + a.eps[o]);
        T* out = reinterpret_cast<T*>(a.out[o]) + row;
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            const float4& w = o ? w2[k] : w1[k];
            if (i < dim) twin_store4(out + i, make_float4(v[k].x * f * w.x, v[k].y * f * w.y, v[k].z * f * w.z, v[k].w * f * w.w));
        }
    }
}

// any width, element by element; a thread reads back what it wrote itself
template <typename T>
__global__ __launch_bounds__(256) void twin_norm_kernel(TwinArgs a) {
    __shared__ float scratch[16];
    const int dim = a.dim;
    const size_t row = (size_t)blockIdx.x * dim;
    const bool store = a.y || a.n_parts > 0;
    float ss = 0.f;
    for (int i = threadIdx.x; i < dim; i += blockDim.x) {
        float v = a.x[row + i];
        if (a.y) v += to_f32(reinterpret_cast<const T*>(a.y)[row + i]);
        for (int p = 0; p < a.n_parts; ++p) v += a.parts[p * a.part_stride + row + i];
        if (store) a.x[row + i] = v;
        ss = fmaf(v, v, ss);
    }
    if (!a.w[0] && !a.w[1]) return;
    ss = block_sum(ss, scratch);
    for (int o = 0; o < 2; ++o) {
        if (!a.w[o]) continue;
        const float f = 1.0f / sqrtf(ss / (float)dim + a.eps[o]);
        T* out = reinterpret_cast<T*>(a.out[o]) + row;
        for (int i = threadIdx.x; i < dim; i += blockDim.x) out[i] = from_f32<T>(a.x[row + i] * f * a.w[o][i]);
    }
}

template <typename T>
static int twin_norm_launch(const TwinArgs& a, int n_rows, hipStream_t s) {
    const dim3 grid(n_rows), block(256);
    const bool aligned = a.dim % 4 == 0 && !(((uintptr_t)a.x | (uintptr_t)a.y | (uintptr_t)a.parts | (uintptr_t)a.w[0] | (uintptr_t)a.w[1] |
                                              (uintptr_t)a.out[0] | (uintptr_t)a.out[1]) & 15);
    const int nv = (a.dim + 1023) / 1024;
    if (aligned && nv == 1) hipLaunchKernelGGL((twin_norm_row_kernel<T, 1>), grid, block, 0, s, a);
    else if (aligned && nv == 2) hipLaunchKernelGGL((twin_norm_row_kernel<T, 2>), grid, block, 0, s, a);
    else if (aligned && nv <= 4) hipLaunchKernelGGL((twin_norm_row_kernel<T, 4>), grid, block, 0, s, a);
    else if (aligned && nv <= 8) hipLaunchKernelGGL((twin_norm_row_kernel<T, 8>), grid, block, 0, s, a);
    else hipLaunchKernelGGL(twin_norm_kernel<T>, grid, block, 0, s, a);
    return bn_launch_status();
}

// dtype: the type of y and of the outputs; parts: n_parts float32 slabs [n_parts][n_rows][dim], n_parts 0: none
extern "C" int bn_twin_norm(int dtype, float* x, const void* y, const float* parts, int n_parts, const float* w1, float eps1, void* out1,
                            const float* w2, float eps2, void* out2, int n_rows, int dim, hipStream_t s) {
    if (n_rows <= 0 || dim <= 0 || !x || n_parts < 0 || (n_parts > 0) != (parts != nullptr)) return BN_ERR_ARG;
    if ((w1 == nullptr) != (out1 == nullptr) || (w2 == nullptr) != (out2 == nullptr)) return BN_ERR_ARG;
    TwinArgs a;
    a.x = x; a.y = y; a.parts = parts; a.n_parts = n_parts; a.part_stride = (size_t)n_rows * dim;
    a.w[0] = w1; a.w[1] = w2; a.out[0] = out1; a.out[1] = out2; a.eps[0] = eps1; a.eps[1] = eps2; a.dim = dim;
    if (dtype == BN_DT_F32) return twin_norm_launch<float>(a, n_rows, s);
    if (dtype == BN_DT_BF16) return twin_norm_launch<bf16>(a, n_rows, s);
    return BN_ERR_DTYPE;
}
