// A norm behind the sum: the stream becomes  x <- w * v / sqrt(mean(v^2) + eps),  v = alpha * x + gain * y,  with y a
// sublayer's output (gain: one number per column, null: 1).  One pass over the row hands the new rows on to the next part
// in the activations' type, as they are or (decode steps, where a row is its sequence's one new token) mixed with the
// previous token's row:  out = x + (x' - x) * mu,  x' the sequence's state (zeros at position 0), which then takes x.
// y is the sum of n_parts slabs (part_stride elements apart, added in slab order) of type TD.  Everything in float32; the
// order of the sums is a function of the row's width alone.
#include "common.h"

struct PostNormArgs {
    float* x;                 // [n_rows, dim], rewritten
    const void* y;            // n_parts slabs [n_rows, dim]
    int n_parts;
    size_t part_stride;
    const float* gain;        // [dim] or null
    float alpha;
    const float* w;           // [dim]
    float eps;
    void* out;                // [n_rows, dim] or null: the stream alone
    int dim;
    const float* mu;          // [dim] or null: out is the rows as they are
    float* state;             // rows of state_stride floats, the first dim of each: the previous token's row
    size_t state_stride;
    const int* positions;     // [n_rows]; < 0: a padding row, whose state row belongs to nobody and is left alone
    const int* slot_ids;      // [n_rows]
};

// rows of up to 1024 NV elements (a multiple of 4): every load of the row is issued before anything waits, the row stays
// in registers, one block reduction, one store
template <typename T, typename TD, int NV>
__global__ __launch_bounds__(256) void post_norm_row_kernel(PostNormArgs a) {
    __shared__ float scratch[16];
    const int r = blockIdx.x, dim = a.dim;
    float* xr = a.x + (size_t)r * dim;
    const TD* yr = reinterpret_cast<const TD*>(a.y) + (size_t)r * dim;
    int pos = -1;
    float* st = nullptr;
    if (a.mu) { pos = a.positions[r]; st = a.state + (size_t)a.slot_ids[r] * a.state_stride; }
    float4 xv[NV], yv[NV], gv[NV], wv[NV], mv[NV], sv[NV];
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = (k * 256 + threadIdx.x) * 4;
        xv[k] = yv[k] = wv[k] = mv[k] = sv[k] = make_float4(0.f, 0.f, 0.f, 0.f);
        gv[k] = make_float4(1.f, 1.f, 1.f, 1.f);
        if (i < dim) {
            xv[k] = *reinterpret_cast<const float4*>(xr + i);
            wv[k] = *reinterpret_cast<const float4*>(a.w + i);
            if (a.gain) gv[k] = *reinterpret_cast<const float4*>(a.gain + i);
            if (a.mu) {
                mv[k] = *reinterpret_cast<const float4*>(a.mu + i);
                if (pos > 0) sv[k] = *reinterpret_cast<const float4*>(st + i);
            }
        }
    }
#pragma unroll 4
    for (int p = 0; p < a.n_parts; ++p, yr += a.part_stride) {
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < dim) {
                float d[4];
                if (sizeof(TD) == 2) {
                    const uint2 t = *reinterpret_cast<const uint2*>(yr + i);
                    d[0] = bf16lo_to_f32(t.x); d[1] = bf16hi_to_f32(t.x); d[2] = bf16lo_to_f32(t.y); d[3] = bf16hi_to_f32(t.y);
                } else {
                    const float4 t = *reinterpret_cast<const float4*>(yr + i);
                    d[0] = t.x; d[1] = t.y; d[2] = t.z; d[3] = t.w;
                }
                yv[k].x += d[0]; yv[k].y += d[1]; yv[k].z += d[2]; yv[k].w += d[3];
            }
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        xv[k].x = fmaf(gv[k].x, yv[k].x, a.alpha * xv[k].x); xv[k].y = fmaf(gv[k].y, yv[k].y, a.alpha * xv[k].y);
        xv[k].z = fmaf(gv[k].z, yv[k].z, a.alpha * xv[k].z); xv[k].w = fmaf(gv[k].w, yv[k].w, a.alpha * xv[k].w);
        ss = fmaf(xv[k].x, xv[k].x, ss); ss = fmaf(xv[k].y, xv[k].y, ss);
        ss = fmaf(xv[k].z, xv[k].z, ss); ss = fmaf(xv[k].w, xv[k].w, ss);
    }
    ss = block_sum(ss, scratch);
    const float f = 1.0f / sqrtf(ss / (float)dim + a.eps);
    T* o = a.out ? reinterpret_cast<T*>(a.out) + (size_t)r * dim : nullptr;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = (k * 256 + threadIdx.x) * 4;
        if (i >= dim) continue;
        float4 v = make_float4(xv[k].x * f * wv[k].x, xv[k].y * f * wv[k].y, xv[k].z * f * wv[k].z, xv[k].w * f * wv[k].w);
        *reinterpret_cast<float4*>(xr + i) = v;
        if (!o) continue;
        if (a.mu) {
            if (pos >= 0) *reinterpret_cast<float4*>(st + i) = v;
            v.x = fmaf(sv[k].x - v.x, mv[k].x, v.x); v.y = fmaf(sv[k].y - v.y, mv[k].y, v.y);
            v.z = fmaf(sv[k].z - v.z, mv[k].z, v.z); v.w = fmaf(sv[k].w - v.w, mv[k].w, v.w);
        }
        if (sizeof(T) == 2) {
            bf16 t[4] = {from_f32<bf16>(v.x), from_f32<bf16>(v.y), from_f32<bf16>(v.z), from_f32<bf16>(v.w)};
            *reinterpret_cast<uint2*>(o + i) = *reinterpret_cast<const uint2*>(t);
        } else {
            *reinterpret_cast<float4*>(o + i) = v;
        }
    }
}

// any width, element by element; the sum v waits in the stream's own row between the passes (a thread reads back what it
// wrote itself)
template <typename T, typename TD>
__global__ __launch_bounds__(256) void post_norm_kernel(PostNormArgs a) {
    __shared__ float scratch[16];
    const int r = blockIdx.x, dim = a.dim;
    float* xr = a.x + (size_t)r * dim;
    const TD* yr = reinterpret_cast<const TD*>(a.y) + (size_t)r * dim;
    int pos = -1;
    float* st = nullptr;
    if (a.mu) { pos = a.positions[r]; st = a.state + (size_t)a.slot_ids[r] * a.state_stride; }
    float ss = 0.f;
    for (int i = threadIdx.x; i < dim; i += blockDim.x) {
        float y = 0.f;
        for (int p = 0; p < a.n_parts; ++p) y += to_f32(yr[p * a.part_stride + i]);
        const float v = fmaf(a.gain ? a.gain[i] : 1.f, y, a.alpha * xr[i]);
        xr[i] = v;
        ss = fmaf(v, v, ss);
    }
    ss = block_sum(ss, scratch);
    const float f = 1.0f / sqrtf(ss / (float)dim + a.eps);
    T* o = a.out ? reinterpret_cast<T*>(a.out) + (size_t)r * dim : nullptr;
    for (int i = threadIdx.x; i < dim; i += blockDim.x) {
        float v = xr[i] * f * a.w[i];
        xr[i] = v;
        if (!o) continue;
        if (a.mu) {
            const float before = pos > 0 ? st[i] : 0.f;
            if (pos >= 0) st[i] = v;
            v = fmaf(before - v, a.mu[i], v);
        }
        o[i] = from_f32<T>(v);
    }
}

template <typename T, typename TD>
static int post_norm_launch(const PostNormArgs& a, int n_rows, hipStream_t s) {
    const dim3 grid(n_rows), block(256);
    const bool aligned = a.dim % 4 == 0 && a.part_stride % 4 == 0 && (!a.mu || a.state_stride % 4 == 0) &&
                         !(((uintptr_t)a.x | (uintptr_t)a.y | (uintptr_t)a.gain | (uintptr_t)a.w | (uintptr_t)a.out |
                            (uintptr_t)a.mu | (uintptr_t)a.state) & 15);
    const int nv = (a.dim + 1023) / 1024;
    if (aligned && nv == 1) hipLaunchKernelGGL((post_norm_row_kernel<T, TD, 1>), grid, block, 0, s, a);
    else if (aligned && nv == 2) hipLaunchKernelGGL((post_norm_row_kernel<T, TD, 2>), grid, block, 0, s, a);
    else if (aligned && nv <= 4) hipLaunchKernelGGL((post_norm_row_kernel<T, TD, 4>), grid, block, 0, s, a);
    else if (aligned && nv <= 8) hipLaunchKernelGGL((post_norm_row_kernel<T, TD, 8>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((post_norm_kernel<T, TD>), grid, block, 0, s, a);
    return bn_launch_status();
}

// dtype: the type of out (and of y when parts_f32 is 0); parts_f32: y is n_parts float32 slabs [n_parts][n_rows][dim].
// mu, state, positions, slot_ids: all or none (with out).
extern "C" int bn_post_norm(int dtype, float* x, const void* y, int n_parts, int parts_f32, const float* gain, float alpha,
                            const float* w, float eps, void* out, int n_rows, int dim, const float* mu, float* state,
                            long long state_stride, const int* positions, const int* slot_ids, hipStream_t s) {
    if (n_rows <= 0 || dim <= 0 || n_parts < 1 || !x || !y || !w) return BN_ERR_ARG;
    if (mu && (!out || !state || !positions || !slot_ids || state_stride < dim)) return BN_ERR_ARG;
    PostNormArgs a;
    a.x = x; a.y = y; a.n_parts = n_parts; a.part_stride = (size_t)n_rows * dim; a.gain = gain; a.alpha = alpha; a.w = w; a.eps = eps;
    a.out = out; a.dim = dim; a.mu = mu; a.state = mu ? state : nullptr; a.state_stride = (size_t)state_stride;
    a.positions = positions; a.slot_ids = slot_ids;
    if (dtype == BN_DT_F32) return post_norm_launch<float, float>(a, n_rows, s);
    if (dtype == BN_DT_BF16) return parts_f32 ? post_norm_launch<bf16, float>(a, n_rows, s) : post_norm_launch<bf16, bf16>(a, n_rows, s);
    return BN_ERR_DTYPE;
}
