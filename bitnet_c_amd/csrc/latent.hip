// Kernels of the latent attention mixer: keys and values are both projections of one normed vector c per token (the
// latent), which is all that the cache keeps.  Because k_h = U_h c and v_h = V_h c are linear in c, the mixer attends in
// the latent's space: the query of head h becomes q'_h = U_h^T q_h, all heads share the one cached vector as key and as
// value (score = q'_h . c, o'_h = sum_j p_j c_j), and the value projection runs once on the result, o_h = V_h o'_h.
//
//   bn_latent_store   c = x / sqrt(mean(x^2) + eps) * w over the latent's columns of a projected row -> the page of the
//                     row's position, once as a key row and once into the transposed value page; beside it, optionally, the
//                     same kind of norm over another run of the row's columns (the queries' own latent), to a tensor
//   bn_head_linear    y[t, h, :] = x[t, h, :] . M_h for every head (M_h [in, out]), optionally times sigmoid(gate[t, h, :]),
//                     or with a run of every head's output columns rotated by the row's position
//   bn_sigmoid_gate   y *= sigmoid(gate), element by element
// All arithmetic in float32; results are stored once in the activations' type.
#include "common.h"
#include <math.h>

// A rotation by the position: pair i of `rot` dimensions (neighbours 2i, 2i + 1, or i with i + rot / 2) turns by
// position * inv_freq[i]; cosine and sine times `mult`
struct Rotation {
    const float* inv_freq;    // [rot / 2] or null (rot 0)
    int rot, interleaved;
    float mult;
};
__device__ __forceinline__ int rot_first(const Rotation& r, int i) { return r.interleaved ? 2 * i : i; }
__device__ __forceinline__ int rot_second(const Rotation& r, int i) { return r.interleaved ? 2 * i + 1 : i + r.rot / 2; }
__device__ __forceinline__ void rot_turn(const Rotation& r, int i, int pos, float& u, float& v) {
    float sn, cs;
    sincosf((float)pos * r.inv_freq[i], &sn, &cs);
    sn *= r.mult; cs *= r.mult;
    const float a = u * cs - v * sn, b = v * cs + u * sn;
    u = a; v = b;
}

struct LatentStoreArgs {
    const void* x;            // [T, ld]; the latent's columns start at column `col`, the rotated key part follows them
    const int* positions;     // [T]; < 0: a padding row, nothing is written
    const int* seq_index;     // [T] row of the block table
    const int* block_table;   // [n_seqs, bt_stride]
    void* k_pages;            // [pages, 1, BN_PAGE, kw]: the latent, then the rotated part, then zeros
    void* v_pages;            // [pages, 1, vw, BN_PAGE]: the latent, then zeros
    const float* w;           // [rank]
    Rotation r;
    int ld, col, rank, bt_stride, kw, vw;
    float eps;
    const float* q_w;         // [q_rank] or null: columns q_col .. q_col + q_rank of a row under a norm of the same kind
    void* q_out;              // [T, q_rank]
    int q_col, q_rank;
};

// the factor of an RMSNorm over n columns of a row; all threads of the workgroup
template <typename T>
__device__ __forceinline__ float latent_rms_factor(const T* x, int n, float eps, float* scratch) {
    float ss = 0.f;
    for (int d = threadIdx.x; d < n; d += blockDim.x) { const float v = to_f32(x[d]); ss = fmaf(v, v, ss); }
    ss = block_sum(ss, scratch);
    return 1.0f / sqrtf(ss / (float)n + eps);
}

template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(LatentStoreArgs a) {
    __shared__ float scratch[16];
    const int t = blockIdx.x;
    if (blockIdx.y == 1) {                               // the queries' latent
        const T* x = reinterpret_cast<const T*>(a.x) + (size_t)t * a.ld + a.q_col;
        const float f = latent_rms_factor(x, a.q_rank, a.eps, scratch);
        T* o = reinterpret_cast<T*>(a.q_out) + (size_t)t * a.q_rank;
        for (int d = threadIdx.x; d < a.q_rank; d += blockDim.x) o[d] = from_f32<T>(to_f32(x[d]) * f * a.q_w[d]);
        return;
    }
    const int pos = a.positions[t];
    if (pos < 0) return;
    const T* x = reinterpret_cast<const T*>(a.x) + (size_t)t * a.ld + a.col;
    const float f = latent_rms_factor(x, a.rank, a.eps, scratch);
    const int page = a.block_table[(size_t)a.seq_index[t] * a.bt_stride + pos / BN_PAGE], slot = pos % BN_PAGE;
    T* kd = reinterpret_cast<T*>(a.k_pages) + ((size_t)page * BN_PAGE + slot) * a.kw;
    T* vd = reinterpret_cast<T*>(a.v_pages) + (size_t)page * a.vw * BN_PAGE + slot;
    for (int d = threadIdx.x; d < a.rank; d += blockDim.x) {
        const T c = from_f32<T>(to_f32(x[d]) * f * a.w[d]);
        kd[d] = c;
        vd[(size_t)d * BN_PAGE] = c;
    }
    for (int d = a.rank + a.r.rot + threadIdx.x; d < a.kw; d += blockDim.x) kd[d] = from_f32<T>(0.f);
    for (int d = a.rank + threadIdx.x; d < a.vw; d += blockDim.x) vd[(size_t)d * BN_PAGE] = from_f32<T>(0.f);
    // the key part that all heads share: not normed, rotated
    for (int i = threadIdx.x; i < a.r.rot / 2; i += blockDim.x) {
        const int d0 = a.rank + rot_first(a.r, i), d1 = a.rank + rot_second(a.r, i);
        float u = to_f32(x[d0]), v = to_f32(x[d1]);
        rot_turn(a.r, i, pos, u, v);
        kd[d0] = from_f32<T>(u);
        kd[d1] = from_f32<T>(v);
    }
}

extern "C" int bn_latent_store(int dtype, const void* x, int ld, int col, const int* positions, const int* seq_index,
                               const int* block_table, int bt_stride, void* k_pages, void* v_pages, const float* w, int n_tokens,
                               int rank, float eps, int rot, const float* inv_freq, float rot_mult, int interleaved, int kw, int vw,
                               int q_col, int q_rank, const float* q_w, void* q_out, hipStream_t s) {
    if (kw < rank + rot || vw < rank || q_rank < 0 || (q_rank > 0 && (!q_w || !q_out || q_col < 0 || ld < q_col + q_rank))) return BN_ERR_ARG;
    if (n_tokens <= 0 || rank <= 0 || col < 0 || rot < 0 || rot % 2 || ld < col + rank + rot || (rot > 0 && !inv_freq)) return BN_ERR_ARG;
    if (!x || !positions || !seq_index || !block_table || !k_pages || !v_pages || !w) return BN_ERR_ARG;
    LatentStoreArgs a;
    a.x = x; a.positions = positions; a.seq_index = seq_index; a.block_table = block_table; a.k_pages = k_pages;
    a.v_pages = v_pages; a.w = w; a.ld = ld; a.col = col; a.rank = rank; a.bt_stride = bt_stride; a.eps = eps;
    a.r.rot = rot; a.r.inv_freq = inv_freq; a.r.mult = rot_mult; a.r.interleaved = interleaved ? 1 : 0;
    a.kw = kw; a.vw = vw; a.q_col = q_col; a.q_rank = q_rank; a.q_w = q_w; a.q_out = q_out;
    const dim3 grid(n_tokens, q_rank > 0 ? 2 : 1), block((rank > q_rank ? rank : q_rank) > 128 ? 256 : 64);
    if (dtype == BN_DT_F32) hipLaunchKernelGGL(latent_store_kernel<float>, grid, block, 0, s, a);
    else if (dtype == BN_DT_BF16) hipLaunchKernelGGL(latent_store_kernel<bf16>, grid, block, 0, s, a);
    else return BN_ERR_DTYPE;
    return bn_launch_status();
}

// ---- a product per head ---------------------------------------------------------------------------------------------
#define HL_ROWS 8             // rows of x that a workgroup takes
#define HL_COLS 64            // output columns of a workgroup
#define HL_SLICES 4           // parts of the input dimension, a wave each; their sums meet in shared memory

struct HeadLinearArgs {
    const void* x;            // [T, ldx]: head h at h * I
    const void* w;            // [H, I, O]
    void* y;                  // [T, ldy]: head h at h * O
    const void* gate;         // [T, ldg]: the gate of output column n is entry n / gate_group (1: one a column; O: one a head); null: none
    int ldx, ldy, ldg, T, H, I, O, gate_group;
    Rotation r;               // rot > 0: columns rot_off .. rot_off + rot of every head's output turn by the row's position
    int rot_off, OC;          // OC: output columns of a workgroup of the wide kernel
    const int* positions;     // [T]; < 0: a padding row, whose columns stay as they are
};

// The rows of x are staged in shared memory as float32 and read by every lane of a wave at the same address; a lane owns
// an output column and walks its wave's part of the input dimension with one coalesced load of the weights a step, eight
// steps' loads in flight.
template <typename T>
__global__ __launch_bounds__(HL_COLS * HL_SLICES) void head_linear_kernel(HeadLinearArgs a) {
    extern __shared__ float xs[];                        // [HL_ROWS][I], then the slices' sums [HL_SLICES][HL_ROWS][HL_COLS]
    float* red = xs + HL_ROWS * a.I;
    const int h = blockIdx.y, t0 = blockIdx.z * HL_ROWS, c = threadIdx.x & (HL_COLS - 1), slice = threadIdx.x / HL_COLS;
    const int o = blockIdx.x * HL_COLS + c;
    const int rows = min(HL_ROWS, a.T - t0);
    const T* x = reinterpret_cast<const T*>(a.x);
    for (int idx = threadIdx.x; idx < HL_ROWS * a.I; idx += HL_COLS * HL_SLICES) {
        const int r = idx / a.I, i = idx - r * a.I;
        xs[idx] = r < rows ? to_f32(x[(size_t)(t0 + r) * a.ldx + (size_t)h * a.I + i]) : 0.f;
    }
    __syncthreads();
    float acc[HL_ROWS];
#pragma unroll
    for (int r = 0; r < HL_ROWS; ++r) acc[r] = 0.f;
    const int per = (a.I + HL_SLICES - 1) / HL_SLICES, i0 = slice * per, i1 = min(a.I, i0 + per);
    if (o < a.O) {
        const T* w = reinterpret_cast<const T*>(a.w) + (size_t)h * a.I * a.O + o;
#pragma unroll 8
        for (int i = i0; i < i1; ++i) {
            const float wv = to_f32(w[(size_t)i * a.O]);
#pragma unroll
            for (int r = 0; r < HL_ROWS; ++r) acc[r] = fmaf(xs[r * a.I + i], wv, acc[r]);
        }
    }
#pragma unroll
    for (int r = 0; r < HL_ROWS; ++r) red[(slice * HL_ROWS + r) * HL_COLS + c] = acc[r];
    __syncthreads();
    if (slice != 0 || o >= a.O) return;
    T* y = reinterpret_cast<T*>(a.y);
    const T* g = reinterpret_cast<const T*>(a.gate);
#pragma unroll
    for (int r = 0; r < HL_ROWS; ++r) {
        if (r >= rows) break;
        float v = 0.f;
#pragma unroll
        for (int k = 0; k < HL_SLICES; ++k) v += red[(k * HL_ROWS + r) * HL_COLS + c];
        if (g) v *= 1.0f / (1.0f + expf(-to_f32(g[(size_t)(t0 + r) * a.ldg + ((size_t)h * a.O + o) / a.gate_group])));
        y[(size_t)(t0 + r) * a.ldy + (size_t)h * a.O + o] = from_f32<T>(v);
    }
}

// The same product with 16-byte loads of the weights: a lane owns HLW_VEC consecutive output columns (8 bf16 or 4 float32),
// O / HLW_VEC lanes cover a row of the head's matrix, and the 256 / (O / HLW_VEC) groups of lanes take the input dimension
// in turn; their sums meet in shared memory.  One workgroup a (head, four rows of x, run of OC output columns): at few rows
// the columns are cut into runs until the launch has workgroups enough for the chip.
#define HLW_ROWS 4
#define HLW_THREADS 256

template <typename T> struct HlwVec;
template <> struct HlwVec<bf16> {
    static constexpr int N = 8;
    static __device__ __forceinline__ void load(const bf16* p, float (&v)[8]) {
        const uint4 w = *reinterpret_cast<const uint4*>(p);
        v[0] = bf16lo_to_f32(w.x); v[1] = bf16hi_to_f32(w.x); v[2] = bf16lo_to_f32(w.y); v[3] = bf16hi_to_f32(w.y);
        v[4] = bf16lo_to_f32(w.z); v[5] = bf16hi_to_f32(w.z); v[6] = bf16lo_to_f32(w.w); v[7] = bf16hi_to_f32(w.w);
    }
};
template <> struct HlwVec<float> {
    static constexpr int N = 4;
    static __device__ __forceinline__ void load(const float* p, float (&v)[4]) {
        const float4 w = *reinterpret_cast<const float4*>(p);
        v[0] = w.x; v[1] = w.y; v[2] = w.z; v[3] = w.w;
    }
};

template <typename T>
__global__ __launch_bounds__(HLW_THREADS) void head_linear_wide_kernel(HeadLinearArgs a) {
    constexpr int V = HlwVec<T>::N;
    extern __shared__ float xs[];                        // [HLW_ROWS][I], then the groups' sums [groups][HLW_ROWS][OC]
    float* red = xs + HLW_ROWS * a.I;
    const int h = blockIdx.x, t0 = blockIdx.y * HLW_ROWS, o0 = blockIdx.z * a.OC, OC = min(a.OC, a.O - o0);
    const int lanes = OC / V, groups = HLW_THREADS / lanes;          // lanes <= 256
    const int grp = threadIdx.x / lanes, cg = threadIdx.x - grp * lanes;
    const int rows = min(HLW_ROWS, a.T - t0);
    const T* x = reinterpret_cast<const T*>(a.x);
    for (int idx = threadIdx.x; idx < HLW_ROWS * a.I; idx += HLW_THREADS) {
        const int r = idx / a.I, i = idx - r * a.I;
        xs[idx] = r < rows ? to_f32(x[(size_t)(t0 + r) * a.ldx + (size_t)h * a.I + i]) : 0.f;
    }
    __syncthreads();
    float acc[HLW_ROWS][V];
#pragma unroll
    for (int r = 0; r < HLW_ROWS; ++r)
#pragma unroll
        for (int k = 0; k < V; ++k) acc[r][k] = 0.f;
    if (grp < groups) {
        const T* w = reinterpret_cast<const T*>(a.w) + (size_t)h * a.I * a.O + o0 + (size_t)cg * V;
#pragma unroll 4
        for (int i = grp; i < a.I; i += groups) {
            float wv[V];
            HlwVec<T>::load(w + (size_t)i * a.O, wv);
#pragma unroll
            for (int r = 0; r < HLW_ROWS; ++r) {
                const float xv = xs[r * a.I + i];
#pragma unroll
                for (int k = 0; k < V; ++k) acc[r][k] = fmaf(xv, wv[k], acc[r][k]);
            }
        }
#pragma unroll
        for (int r = 0; r < HLW_ROWS; ++r)
#pragma unroll
            for (int k = 0; k < V; ++k) red[((size_t)grp * HLW_ROWS + r) * OC + cg * V + k] = acc[r][k];
    }
    __syncthreads();
    T* y = reinterpret_cast<T*>(a.y);
    const T* g = reinterpret_cast<const T*>(a.gate);
    for (int idx = threadIdx.x; idx < rows * OC; idx += HLW_THREADS) {
        const int r = idx / OC, c = idx - r * OC, o = o0 + c;
        float v = 0.f;
        for (int k = 0; k < groups; ++k) v += red[((size_t)k * HLW_ROWS + r) * OC + c];
        if (g) v *= 1.0f / (1.0f + expf(-to_f32(g[(size_t)(t0 + r) * a.ldg + ((size_t)h * a.O + o) / a.gate_group])));
        const int ro = o - a.rot_off, pos = ro >= 0 && ro < a.r.rot ? a.positions[t0 + r] : -1;
        if (pos >= 0) {                                  // this column and its partner, both from this workgroup's sums
            const int i = a.r.interleaved ? ro >> 1 : ro < a.r.rot / 2 ? ro : ro - a.r.rot / 2;
            const bool second = ro != rot_first(a.r, i);
            const int pc = a.rot_off + (second ? rot_first(a.r, i) : rot_second(a.r, i)) - o0;
            float p = 0.f;
            for (int k = 0; k < groups; ++k) p += red[((size_t)k * HLW_ROWS + r) * OC + pc];
            float u = second ? p : v, w = second ? v : p;
            rot_turn(a.r, i, pos, u, w);
            v = second ? w : u;
        }
        y[(size_t)(t0 + r) * a.ldy + (size_t)h * a.O + o] = from_f32<T>(v);
    }
}

// The columns of a workgroup: all of them, or halves of that (down to 32, which leaves a row of the matrix 64 bytes a
// workgroup) while the launch would have fewer than HLW_WORKGROUPS; a run holds both columns of every rotated pair.  The cut
// decides how many groups of lanes share a column's sum: float32 rows are not cut, so that their sums keep one order whatever
// number of rows a step has.
#define HLW_WORKGROUPS 256
static int hlw_columns(const HeadLinearArgs& a, int dtype, int row_tiles) {
    int oc = a.O;
    while (dtype == BN_DT_BF16 && oc % 64 == 0 && (long long)a.H * row_tiles * ((a.O + oc - 1) / oc) < HLW_WORKGROUPS) {
        const int half = oc / 2;
        const bool whole_pairs = a.r.rot == 0 || (a.r.interleaved && a.rot_off % 2 == 0) ||
                                 a.rot_off / half == (a.rot_off + a.r.rot - 1) / half;
        if (!whole_pairs) break;
        oc = half;
    }
    return oc;
}

template <typename T>
static bool hlw_takes(const void* w, int I, int O, int OC) {
    constexpr int V = HlwVec<T>::N;
    if (O % V || OC % V || OC / V > HLW_THREADS || ((uintptr_t)w & 15)) return false;
    const int groups = HLW_THREADS / (OC / V);
    return (size_t)HLW_ROWS * ((size_t)I + (size_t)groups * OC) * sizeof(float) <= 64 * 1024;
}

extern "C" int bn_rope_heads(int dtype, void* x, int ld, const int* positions, const float* inv_freq, int n_rows, int H,
                             int head_stride, int off, int rot, float mult, int interleaved, hipStream_t s);

extern "C" int bn_head_linear(int dtype, const void* x, int ldx, const void* w, void* y, int ldy, const void* gate, int ldg,
                              int gate_group, int n_rows, int H, int I, int O, const int* positions, const float* inv_freq, int rot_off,
                              int rot, float rot_mult, int interleaved, hipStream_t s) {
    if (rot < 0 || rot % 2 || rot_off < 0 || rot_off + rot > O || (rot > 0 && (!positions || !inv_freq || gate))) return BN_ERR_ARG;
    if (n_rows <= 0 || H <= 0 || I <= 0 || O <= 0 || !x || !w || !y) return BN_ERR_ARG;
    if (gate && (gate_group < 1 || (H * O) % gate_group)) return BN_ERR_ARG;
    if (ldx < H * I || ldy < H * O || (gate && ldg < H * O / gate_group) || (size_t)HL_ROWS * (I + HL_SLICES * HL_COLS) * sizeof(float) > 64 * 1024 || H > 65535) return BN_ERR_ARG;
    const int row_tiles = (n_rows + HL_ROWS - 1) / HL_ROWS;
    if (row_tiles > 65535) return BN_ERR_ARG;
    HeadLinearArgs a;
    a.x = x; a.w = w; a.y = y; a.gate = gate; a.ldx = ldx; a.ldy = ldy; a.ldg = ldg; a.T = n_rows; a.H = H; a.I = I; a.O = O; a.gate_group = gate ? gate_group : 1;
    a.r.rot = rot; a.r.inv_freq = inv_freq; a.r.mult = rot_mult; a.r.interleaved = interleaved ? 1 : 0; a.rot_off = rot_off;
    a.positions = positions;
    if (dtype != BN_DT_F32 && dtype != BN_DT_BF16) return BN_ERR_DTYPE;
    const int wide_tiles = (n_rows + HLW_ROWS - 1) / HLW_ROWS;
    a.OC = hlw_columns(a, dtype, wide_tiles);
    const bool wide = dtype == BN_DT_F32 ? hlw_takes<float>(w, I, O, a.OC) : hlw_takes<bf16>(w, I, O, a.OC);
    if (wide && wide_tiles <= 65535) {
        const int vec = dtype == BN_DT_F32 ? 4 : 8, groups = HLW_THREADS / (a.OC / vec);
        const dim3 wgrid(H, wide_tiles, O / a.OC);
        const size_t wshm = (size_t)HLW_ROWS * ((size_t)I + (size_t)groups * a.OC) * sizeof(float);
        if (dtype == BN_DT_F32) hipLaunchKernelGGL(head_linear_wide_kernel<float>, wgrid, dim3(HLW_THREADS), wshm, s, a);
        else hipLaunchKernelGGL(head_linear_wide_kernel<bf16>, wgrid, dim3(HLW_THREADS), wshm, s, a);
        return bn_launch_status();
    }
    const dim3 grid((O + HL_COLS - 1) / HL_COLS, H, row_tiles), block(HL_COLS * HL_SLICES);
    const size_t shm = (size_t)HL_ROWS * (I + HL_SLICES * HL_COLS) * sizeof(float);
    if (dtype == BN_DT_F32) hipLaunchKernelGGL(head_linear_kernel<float>, grid, block, shm, s, a);
    else if (dtype == BN_DT_BF16) hipLaunchKernelGGL(head_linear_kernel<bf16>, grid, block, shm, s, a);
    else return BN_ERR_DTYPE;
    const int rc = bn_launch_status();
    if (rc != 0 || rot == 0) return rc;
    return bn_rope_heads(dtype, y, ldy, positions, inv_freq, n_rows, H, O, rot_off, rot, rot_mult, interleaved, s);
}

// ---- y *= sigmoid(gate) ---------------------------------------------------------------------------------------------
template <typename T>
__global__ void sigmoid_gate_kernel(T* __restrict__ y, int ldy, const T* __restrict__ g, int ldg, int n_rows, int n_cols, int group) {
    const size_t n = (size_t)n_rows * n_cols;
    for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < n; idx += (size_t)gridDim.x * blockDim.x) {
        const size_t r = idx / n_cols, c = idx - r * n_cols;
        const float v = to_f32(y[r * ldy + c]) / (1.0f + expf(-to_f32(g[r * ldg + c / group])));
        y[r * ldy + c] = from_f32<T>(v);
    }
}

extern "C" int bn_sigmoid_gate(int dtype, void* y, int ldy, const void* gate, int ldg, int group, int n_rows, int n_cols, hipStream_t s) {
    if (n_rows <= 0 || n_cols <= 0 || group < 1 || n_cols % group || ldy < n_cols || ldg < n_cols / group || !y || !gate) return BN_ERR_ARG;
    const size_t n = (size_t)n_rows * n_cols;
    const int blocks = (int)((n + 255) / 256 < 4096 ? (n + 255) / 256 : 4096);
    if (dtype == BN_DT_F32) hipLaunchKernelGGL(sigmoid_gate_kernel<float>, dim3(blocks), dim3(256), 0, s, (float*)y, ldy, (const float*)gate, ldg, n_rows, n_cols, group);
    else if (dtype == BN_DT_BF16) hipLaunchKernelGGL(sigmoid_gate_kernel<bf16>, dim3(blocks), dim3(256), 0, s, (bf16*)y, ldy, (const bf16*)gate, ldg, n_rows, n_cols, group);
    else return BN_ERR_DTYPE;
    return bn_launch_status();
}

// ---- a rotation of part of every head, in place ------------------------------------------------------------------------
// x[t, h * head_stride + off + .]: the pairs of a Rotation (see above) turn by the row's position.  Rows with position < 0
// are left alone.  Angles, cosines and sines in float32.
template <typename T>
__global__ void rope_heads_kernel(T* __restrict__ x, int ld, const int* __restrict__ positions, Rotation r, int n_rows, int H,
                                  int head_stride, int off) {
    const int half = r.rot / 2;
    const size_t n = (size_t)n_rows * H * half;
    for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < n; idx += (size_t)gridDim.x * blockDim.x) {
        const int i = (int)(idx % half);
        const size_t th = idx / half;
        const int h = (int)(th % H);
        const size_t t = th / H;
        const int pos = positions[t];
        if (pos < 0) continue;
        T* p = x + t * ld + (size_t)h * head_stride + off;
        const int d0 = rot_first(r, i), d1 = rot_second(r, i);
        float u = to_f32(p[d0]), v = to_f32(p[d1]);
        rot_turn(r, i, pos, u, v);
        p[d0] = from_f32<T>(u);
        p[d1] = from_f32<T>(v);
    }
}

extern "C" int bn_rope_heads(int dtype, void* x, int ld, const int* positions, const float* inv_freq, int n_rows, int H,
                             int head_stride, int off, int rot, float mult, int interleaved, hipStream_t s) {
    if (n_rows <= 0 || H <= 0 || rot <= 0 || rot % 2 || off < 0 || head_stride < off + rot || ld < (H - 1) * head_stride + off + rot
        || !x || !positions || !inv_freq) return BN_ERR_ARG;
    const size_t n = (size_t)n_rows * H * (rot / 2);
    const int blocks = (int)((n + 255) / 256 < 4096 ? (n + 255) / 256 : 4096);
    Rotation r;
    r.inv_freq = inv_freq; r.rot = rot; r.interleaved = interleaved ? 1 : 0; r.mult = mult;
    if (dtype == BN_DT_F32) hipLaunchKernelGGL(rope_heads_kernel<float>, dim3(blocks), dim3(256), 0, s, (float*)x, ld, positions, r, n_rows, H, head_stride, off);
    else if (dtype == BN_DT_BF16) hipLaunchKernelGGL(rope_heads_kernel<bf16>, dim3(blocks), dim3(256), 0, s, (bf16*)x, ld, positions, r, n_rows, H, head_stride, off);
    else return BN_ERR_DTYPE;
    return bn_launch_status();
}
