// State-space (Mamba-2) mixer: short causal convolution, the recurrence, and the gated grouped norm.
//
// The batch is a list of segments, one per sequence: segment i covers rows [cu[i], cu[i + 1]) (cu null: row i) and
// continues state slot slots[i] at absolute position pos0[i]; a segment at position 0 starts from zero, whatever the
// slot holds.  Projections arrive as 16-bit rows or fp32 split-K slabs (common.h ProjSrc).
//
//   conv_silu    xBC columns -> silu(conv) rows of width C; the slot keeps the last taps - 1 inputs
//   ssm_step     S = exp(a dt) S + dt x B^T, y = S C + D x, token by token with S^T in registers (decode; fp32 mode)
//   gated_norm   y silu(z), RMS norm in equal parts, weight, mixer scale -> the output projection's input columns
//
// State S^T is [slots][heads][vdim][N4] fp32 (N4: state size rounded up to 4, zeros past it).
#include "common.h"

// ------------------------------------------------------------------------------------------------ short convolution
template <bool PARTS, typename T>
__device__ __forceinline__ void conv_in8(const ProjSrc& src, int row, int col, float* f) {
    proj8<PARTS>(src, row, col, f);
    if constexpr (PARTS && sizeof(T) == 2) {  // the same 16-bit inputs whichever form the projection took
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] = (float)(T)f[j];
    }
}

// the TAPS - 1 inputs before row t (offset off in its segment): earlier rows, the slot's history, or zeros
template <bool PARTS, typename T, int TAPS>
__device__ __forceinline__ void conv_window(const ProjSrc& src, int t, int off, int col, bool cont, const float* st, int C,
                                            float (*win)[8]) {
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) {
        const int rel = off - (TAPS - 1) + j;
        if (rel >= 0) {
            conv_in8<PARTS, T>(src, t - (TAPS - 1) + j, col, win[j]);
        } else if (cont) {
            load8(st + (size_t)(TAPS - 1 + rel) * C, win[j]);
        } else {
#pragma unroll
            for (int k = 0; k < 8; ++k) win[j][k] = 0.f;
        }
    }
}

// one thread: RUN consecutive rows x 8 channels, the taps slide through registers
template <bool PARTS, typename T, int TAPS, int RUN>
__global__ __launch_bounds__(256) void conv_silu_kernel(ProjSrc src, int at, const float* __restrict__ kernel,
                                                        const float* __restrict__ bias, const float* __restrict__ state,
                                                        SegArgs sg, T* __restrict__ out, int rows, int C) {
    constexpr int W = TAPS > 1 ? TAPS - 1 : 1;
    const int c8 = C >> 3;
    const int idx = blockIdx.x * 256 + threadIdx.x;
    const int c = (idx % c8) * 8, t0 = (idx / c8) * RUN;
    if (t0 >= rows) return;
    float kw[TAPS][8], b[8], win[W][8];
    load8(bias + c, b);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) load8(kernel + (size_t)j * C + c, kw[j]);
    int seg = sg.row_seg[t0], first = sg.cu[seg], end = sg.cu[seg + 1];
    auto window = [&](int t) {
        if constexpr (TAPS > 1)
            conv_window<PARTS, T, TAPS>(src, t, t - first, at + c, sg.pos0[seg] > 0,
                                        state + (size_t)sg.slots[seg] * (TAPS - 1) * C + c, C, win);
    };
    window(t0);
#pragma unroll
    for (int r = 0; r < RUN; ++r) {
        const int t = t0 + r;
        if (t >= rows) break;
        if (t >= end) {  // the next segment starts here
            seg = sg.row_seg[t];
            first = sg.cu[seg];
            end = sg.cu[seg + 1];
            window(t);
        }
        float x[8], acc[8];
        conv_in8<PARTS, T>(src, t, at + c, x);
#pragma unroll
        for (int k = 0; k < 8; ++k) {
            float a = b[k];
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) a += kw[j][k] * win[j][k];
            a += kw[TAPS - 1][k] * x[k];
            acc[k] = a * logistic_for<T>(a);
        }
        store8(out + (size_t)t * C + c, acc);
        if constexpr (TAPS > 1) {
#pragma unroll
            for (int k = 0; k < 8; ++k) {
#pragma unroll
                for (int j = 0; j + 2 < TAPS; ++j) win[j][k] = win[j + 1][k];
                win[TAPS - 2][k] = x[k];
            }
        }
    }
}

// one row per segment (decode): one thread per 4 channels, which advances their history too
template <bool PARTS, typename T, int TAPS>
__global__ __launch_bounds__(64) void conv_step_kernel(ProjSrc src, int at, const float* __restrict__ kernel,
                                                       const float* __restrict__ bias, float* __restrict__ state,
                                                       SegArgs sg, T* __restrict__ out, int C, GeluJob job) {
    const int t = blockIdx.y, c = 4 * (blockIdx.x * 64 + threadIdx.x);
    if constexpr (PARTS) {
        const int own = (C + 255) / 256;
        if ((int)blockIdx.x >= own) {
            gelu_piece<true, T>(src, job, t, 8 * (((int)blockIdx.x - own) * 64 + threadIdx.x));
            return;
        }
    }
    if (c >= C) return;
    const bool cont = sg.pos0[t] > 0;
    float* st = state + (size_t)sg.slots[t] * (TAPS - 1) * C + c;
    float4 win[TAPS], kw[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) kw[j] = *reinterpret_cast<const float4*>(kernel + (size_t)j * C + c);
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) {
        win[j] = *reinterpret_cast<const float4*>(st + (size_t)j * C);
        if (!cont) win[j] = make_float4(0.f, 0.f, 0.f, 0.f);
    }
    float4 x = proj4<PARTS>(src, t, at + c);
    if constexpr (PARTS && sizeof(T) == 2)
        x = make_float4((float)(T)x.x, (float)(T)x.y, (float)(T)x.z, (float)(T)x.w);
    win[TAPS - 1] = x;
    float4 a = *reinterpret_cast<const float4*>(bias + c);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
        a.x += kw[j].x * win[j].x; a.y += kw[j].y * win[j].y; a.z += kw[j].z * win[j].z; a.w += kw[j].w * win[j].w;
    }
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) *reinterpret_cast<float4*>(st + (size_t)j * C) = win[j + 1];
    a.x *= logistic_for<T>(a.x); a.y *= logistic_for<T>(a.y); a.z *= logistic_for<T>(a.z); a.w *= logistic_for<T>(a.w);
    store4(out + (size_t)t * C + c, a);
}

// any number of taps: one thread, one row x 8 channels.  STEP: one row per segment, the state is advanced here.
template <bool PARTS, typename T, bool STEP>
__global__ __launch_bounds__(256) void conv_any_kernel(ProjSrc src, int at, const float* __restrict__ kernel,
                                                       const float* __restrict__ bias, float* __restrict__ state,
                                                       SegArgs sg, T* __restrict__ out, int rows, int C, int taps) {
    const int c8 = C >> 3;
    const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
    const int t = (int)(idx / c8), c = (int)(idx % c8) * 8;
    if (t >= rows) return;
    const int seg = STEP ? t : sg.row_seg[t];
    const int off = STEP ? 0 : t - sg.cu[seg];
    const bool cont = sg.pos0[seg] > 0;
    float* st = state + (size_t)sg.slots[seg] * (taps - 1) * C + c;
    float acc[8], x[8], kw[8];
    load8(bias + c, acc);
    for (int j = 0; j < taps; ++j) {
        const int rel = off - (taps - 1) + j;
        if (rel >= 0) conv_in8<PARTS, T>(src, t - (taps - 1) + j, at + c, x);
        else if (cont) load8(st + (size_t)(taps - 1 + rel) * C, x);
        else continue;
        load8(kernel + (size_t)j * C + c, kw);
#pragma unroll
        for (int k = 0; k < 8; ++k) acc[k] += kw[k] * x[k];
    }
    if (STEP && taps > 1) {
        for (int j = 0; j + 2 < taps; ++j) {
            float h[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (cont) load8(st + (size_t)(j + 1) * C, h);
            store8(st + (size_t)j * C, h);
        }
        store8(st + (size_t)(taps - 2) * C, x);  // x: the current token's input (last tap)
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] *= logistic_for<T>(acc[j]);
    store8(out + (size_t)t * C + c, acc);
}

// the last taps - 1 inputs of every segment into its slot (after conv_silu has read the old ones)
template <bool PARTS, typename T>
__global__ __launch_bounds__(256) void conv_state_kernel(ProjSrc src, int at, float* __restrict__ state, SegArgs sg,
                                                         int C, int taps) {
    const int seg = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 8;
    if (c >= C) return;
    const int b = sg.cu[seg], len = sg.cu[seg + 1] - b;
    const bool cont = sg.pos0[seg] > 0;
    float* st = state + (size_t)sg.slots[seg] * (taps - 1) * C + c;
    for (int k = 0; k < taps - 1; ++k) {  // ascending: old rows are read ahead of where they are overwritten
        const int rel = len - (taps - 1) + k;
        float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (rel >= 0) {
            conv_in8<PARTS, T>(src, b + rel, at + c, x);
        } else if (cont) {
            load8(st + (size_t)(k + len) * C, x);
        }
        store8(st + (size_t)k * C, x);
    }
}

template <bool PARTS, typename T>
static void launch_conv(const ProjSrc& p, int at, const float* kernel, const float* bias, float* state,
                        const SegArgs& sg, void* out, int T_, int nseg, int C, int taps, const GeluJob& job,
                        hipStream_t s) {
    const int blocks = (int)(((long long)T_ * (C / 8) + 255) / 256);
    constexpr int RUN = 8;
    if (!sg.cu) {
        const dim3 g(ceil_div(C / 4, 64) + ceil_div(job.n, 512), T_);
#define STEP_T(TP) conv_step_kernel<PARTS, T, TP><<<g, 64, 0, s>>>(p, at, kernel, bias, state, sg, (T*)out, C, job)
        if (taps == 4) STEP_T(4);
        else if (taps == 3) STEP_T(3);
        else if (taps == 2) STEP_T(2);
        else conv_any_kernel<PARTS, T, true><<<blocks, 256, 0, s>>>(p, at, kernel, bias, state, sg, (T*)out, T_, C, taps);
#undef STEP_T
        return;
    }
    const int run_blocks = (int)(((long long)ceil_div(T_, RUN) * (C / 8) + 255) / 256);
#define CONV_T(TP) \
    conv_silu_kernel<PARTS, T, TP, RUN><<<run_blocks, 256, 0, s>>>(p, at, kernel, bias, state, sg, (T*)out, T_, C)
    if (taps == 4) CONV_T(4);
    else if (taps == 3) CONV_T(3);
    else if (taps == 2) CONV_T(2);
    else conv_any_kernel<PARTS, T, false><<<blocks, 256, 0, s>>>(p, at, kernel, bias, state, sg, (T*)out, T_, C, taps);
#undef CONV_T
    if (taps > 1)
        conv_state_kernel<PARTS, T><<<dim3(ceil_div(C / 8, 256), nseg), 256, 0, s>>>(p, at, state, sg, C, taps);
}

MRSUM_API int mrsum_gelu_cols(const void* src, int S, int ld, int T, int at, int n, void* out, int out32, int ldo,
                              hipStream_t s);

// g_n > 0: columns of the slabs through gelu besides (GeluJob).  src as ProjSrc (S = 0: bf16 rows); kernel [taps][C], bias [C], state [slots][taps - 1][C]; out [T][C] bf16 or fp32
MRSUM_API int mrsum_conv_silu(const void* src, int S, int ld, int T, int at, const float* kernel, const float* bias,
                              float* state, const int* cu, const int* row_seg, const int* slots, const int* pos0,
                              int nseg, void* out, int out32, int C, int taps, int g_at, int g_n, void* g_out, int g_ldo,
                              hipStream_t s) {
    if (T <= 0) return 0;
    if (C % 8 || at % 8 || ld % 8 || taps < 1 || at + C > ld || (cu && !row_seg) || (!cu && (nseg != T || T > 65535)) ||
        (out32 && S < 1) || nseg > 65535)
        return (int)hipErrorInvalidValue;
    const ProjSrc p{src, S, (size_t)T * ld, ld};
    const SegArgs sg{cu, row_seg, slots, pos0};
    GeluJob job{g_at, g_n, g_ldo, g_out};
    if (!gelu_job_ok(job, S, ld)) return (int)hipErrorInvalidValue;
    if (job.n && (cu || taps < 2 || taps > 4)) {  // only the step form takes it along
        const int e = mrsum_gelu_cols(src, S, ld, T, g_at, g_n, g_out, out32, g_ldo, s);
        if (e) return e;
        job.n = 0;
    }
    if (out32) launch_conv<true, float>(p, at, kernel, bias, state, sg, out, T, nseg, C, taps, job, s);
    else if (S) launch_conv<true, bf16>(p, at, kernel, bias, state, sg, out, T, nseg, C, taps, job, s);
    else launch_conv<false, bf16>(p, at, kernel, bias, state, sg, out, T, nseg, C, taps, job, s);
    return (int)hipGetLastError();
}

// ------------------------------------------------------------------------------------------------ recurrence, stepped
struct ScanArgs {
    ProjSrc u;  // dt columns
    int dt_at;
    const float* dt_bias;
    const float* a_neg;   // -exp(A_log) [heads]
    const float* d_skip;  // [heads]
    float* state;         // [slots][heads][P][N4]
    float* y;             // [T][heads * P]
    int ldx;              // row stride of xBC
    int heads, P, N, N4, groups, seg0;
};

constexpr int STEP_RPT = 4;  // state rows (value columns) per thread

// block: (segment, head, STEP_RPT * 256 / LPR value columns); LPR lanes x NV float4 hold one row of S^T
template <bool PARTS, typename T, int LPR, int NV>
__global__ __launch_bounds__(256) void ssm_step_kernel(const T* __restrict__ xbc, ScanArgs a, SegArgs sg) {
    constexpr int RP = 256 / LPR;
    // segments slowest: neighbouring workgroups stream neighbouring state (slots are power-of-two strides apart)
    const int seg = a.seg0 + blockIdx.z, head = blockIdx.y;
    const int r = threadIdx.x / LPR, l = threadIdx.x % LPR;
    const int p0 = blockIdx.x * (RP * STEP_RPT) + r;
    const int b = sg.cu ? sg.cu[seg] : seg, e = sg.cu ? sg.cu[seg + 1] : seg + 1;
    float* st = a.state + ((size_t)sg.slots[seg] * a.heads + head) * a.P * a.N4;
    const bool cont = sg.pos0[seg] > 0;
    const float an = a.a_neg[head], db = a.dt_bias[head], dsk = a.d_skip[head];
    const int inner = a.heads * a.P, g = head / (a.heads / a.groups);
    const int bcol = inner + g * a.N, ccol = inner + (a.groups + g) * a.N;
    float4 S[STEP_RPT][NV];
#pragma unroll
    for (int i = 0; i < STEP_RPT; ++i)
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int p = p0 + RP * i, n = 4 * (l + LPR * v);
            S[i][v] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (cont && p < a.P && n < a.N4) S[i][v] = *reinterpret_cast<const float4*>(st + (size_t)p * a.N4 + n);
        }
    for (int t = b; t < e; ++t) {
        const float dt = softplus(proj_at<PARTS>(a.u, t, a.dt_at + head) + db);
        const float decay = expf(an * dt);
        const T* row = xbc + (size_t)t * a.ldx;
        float B[NV][4], C[NV][4];
#pragma unroll
        for (int v = 0; v < NV; ++v)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int n = 4 * (l + LPR * v) + j;
                B[v][j] = n < a.N ? (float)row[bcol + n] : 0.f;
                C[v][j] = n < a.N ? (float)row[ccol + n] : 0.f;
            }
#pragma unroll
        for (int i = 0; i < STEP_RPT; ++i) {
            const int p = p0 + RP * i;
            const float x = p < a.P ? (float)row[head * a.P + p] : 0.f;
            const float dx = dt * x;
            float y = 0.f;
#pragma unroll
            for (int v = 0; v < NV; ++v) {
                S[i][v].x = decay * S[i][v].x + dx * B[v][0];
                S[i][v].y = decay * S[i][v].y + dx * B[v][1];
                S[i][v].z = decay * S[i][v].z + dx * B[v][2];
                S[i][v].w = decay * S[i][v].w + dx * B[v][3];
                y += S[i][v].x * C[v][0] + S[i][v].y * C[v][1] + S[i][v].z * C[v][2] + S[i][v].w * C[v][3];
            }
#pragma unroll
            for (int o = LPR / 2; o > 0; o >>= 1) y += __shfl_xor(y, o, 64);
            if (l == 0 && p < a.P) a.y[(size_t)t * inner + head * a.P + p] = y + dsk * x;
        }
    }
#pragma unroll
    for (int i = 0; i < STEP_RPT; ++i)
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int p = p0 + RP * i, n = 4 * (l + LPR * v);
            if (p < a.P && n < a.N4) *reinterpret_cast<float4*>(st + (size_t)p * a.N4 + n) = S[i][v];
        }
}

template <bool PARTS, typename T>
static int launch_step(const void* xbc, const ScanArgs& a, const SegArgs& sg, int nseg, hipStream_t s) {
    const int q = a.N4 / 4;  // float4 per state row
#define STEP(L, V)                                                                                             \
    ssm_step_kernel<PARTS, T, L, V>                                                                            \
        <<<dim3(ceil_div(a.P, STEP_RPT * (256 / L)), a.heads, nseg), 256, 0, s>>>((const T*)xbc, a, sg)
    if (q <= 4) STEP(4, 1);
    else if (q <= 8) STEP(8, 1);
    else if (q <= 16) STEP(16, 1);
    else if (q <= 32) STEP(32, 1);
    else if (q <= 64) STEP(64, 1);
    else if (q <= 128) STEP(64, 2);
    else if (q <= 256) STEP(64, 4);
    else return (int)hipErrorInvalidValue;
#undef STEP
    return (int)hipGetLastError();
}

// Segments [seg0, seg0 + nseg) token by token.  xbc [T][ldx] bf16 / fp32 (x32), u: dt columns at dt_at.
MRSUM_API int mrsum_ssm_step(const void* xbc, int ldx, int x32, const void* u, int S, int ld, int T, int dt_at,
                             const float* dt_bias, const float* a_neg, const float* d_skip, float* state,
                             const int* cu, const int* slots, const int* pos0, int seg0, int nseg, float* y, int heads,
                             int P, int N, int groups, hipStream_t s) {
    if (T <= 0 || nseg <= 0) return 0;
    if (heads % groups || heads > 65535 || nseg > 65535 || dt_at + heads > ld || ldx < heads * P + 2 * groups * N || (x32 && S < 1))
        return (int)hipErrorInvalidValue;
    const ScanArgs a{ProjSrc{u, S, (size_t)T * ld, ld}, dt_at, dt_bias, a_neg, d_skip, state, y, ldx,
                     heads, P, N, (N + 3) / 4 * 4, groups, seg0};
    const SegArgs sg{cu, nullptr, slots, pos0};
    if (x32) return launch_step<true, float>(xbc, a, sg, nseg, s);
    if (S) return launch_step<true, bf16>(xbc, a, sg, nseg, s);
    return launch_step<false, bf16>(xbc, a, sg, nseg, s);
}

// ------------------------------------------------------------------------------------------------ gated grouped norm
template <typename T>
__device__ __forceinline__ float4 gated4(const float* y, const float4& z) {
    const float4 v = *reinterpret_cast<const float4*>(y);
    return make_float4(v.x * z.x * logistic_for<T>(z.x), v.y * z.y * logistic_for<T>(z.y),
                       v.z * z.z * logistic_for<T>(z.z), v.w * z.w * logistic_for<T>(z.w));
}

template <int L>
__device__ __forceinline__ float lanes_sum(float v) {
#pragma unroll
    for (int o = L / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}

// L lanes per norm group, VPT float4 each in registers (VPT = 0: any part size, re-read for the second pass).  L <= 64:
// a wave or part of one per group; L = 256 / 1024: one block per group (few rows: all loads in flight).
// POST: the norm first, then the gate, and one weight vector shared by the groups (heads).  Columns from col + n to
// zero_to are zeroed.
template <bool PARTS, typename TO, int L, int VPT, bool POST>
__global__ __launch_bounds__(L <= 64 ? 256 : L) void gated_norm_kernel(const float* __restrict__ y, ProjSrc u, int z_at,
                                                                       const float* __restrict__ w, int n, int groups,
                                                                       float eps, float out_scale, TO* __restrict__ out,
                                                                       int ldo, int col, int zero_to) {
    __shared__ float red[16];
    constexpr int GPB = L <= 64 ? 256 / L : 1;
    const int gb = (groups + GPB - 1) / GPB;
    const int t = blockIdx.x / gb, g0 = (blockIdx.x % gb) * GPB;
    const int l = threadIdx.x % L, g = g0 + threadIdx.x / L;
    const int ng = n / groups;
    const float* yr = y + (size_t)t * n + g * ng;
    const int zc = z_at + g * ng;
    const float* wr = POST ? w : w + g * ng;
    TO* o = out + (size_t)t * ldo + col + g * ng;
    const bool on = g < groups;
    float ss = 0.f;
    if constexpr (VPT > 0) {
        float4 v[VPT], z[POST ? VPT : 1];
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const int c = 4 * (l + L * i);
            v[i] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (on && c < ng) {
                v[i] = POST ? *reinterpret_cast<const float4*>(yr + c) : gated4<TO>(yr + c, proj4<PARTS>(u, t, zc + c));
                if constexpr (POST) z[i] = proj4<PARTS>(u, t, zc + c);
            }
            ss += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
        }
        ss = L <= 64 ? lanes_sum<(L <= 64 ? L : 64)>(ss) : block_sum(ss, red);
        const float inv = out_scale / sqrtf(ss / (float)ng + eps);
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const int c = 4 * (l + L * i);
            if (on && c < ng) {
                float4 k = *reinterpret_cast<const float4*>(wr + c);
                if constexpr (POST) {
                    k.x *= z[i].x * logistic_for<TO>(z[i].x); k.y *= z[i].y * logistic_for<TO>(z[i].y);
                    k.z *= z[i].z * logistic_for<TO>(z[i].z); k.w *= z[i].w * logistic_for<TO>(z[i].w);
                }
                store4(o + c, make_float4(v[i].x * inv * k.x, v[i].y * inv * k.y, v[i].z * inv * k.z, v[i].w * inv * k.w));
            }
        }
    } else {
        for (int c = l; on && c < ng; c += L) {
            const float z = POST ? 0.f : proj_at<PARTS>(u, t, zc + c), v = POST ? yr[c] : yr[c] * z * logistic(z);
            ss += v * v;
        }
        ss = L <= 64 ? lanes_sum<(L <= 64 ? L : 64)>(ss) : block_sum(ss, red);
        const float inv = out_scale / sqrtf(ss / (float)ng + eps);
        for (int c = l; on && c < ng; c += L) {
            const float z = proj_at<PARTS>(u, t, zc + c);
            o[c] = (TO)(yr[c] * z * logistic(z) * inv * wr[c]);
        }
    }
    if (g0 == 0)
        for (int c = col + n + threadIdx.x; c < zero_to; c += blockDim.x) out[(size_t)t * ldo + c] = (TO)0.f;
}

template <bool POST>
static int launch_gated_norm(const float* y, const ProjSrc& p, int T, int z_at, const float* w, int n, int groups, float eps,
                             float out_scale, void* out, int out32, int ldo, int col, int zero_to, hipStream_t s) {
    const int ng = n / groups, q = ng % 4 ? 0 : ng / 4;  // float4 per part (0: unaligned parts)
    const long long gb = groups, gw = (groups + 3) / 4, gn = (groups + 15) / 16, gh = (groups + 7) / 8;
    if ((long long)T * groups > 0x7fffffff) return (int)hipErrorInvalidValue;
#define GN(PT, TO, L_, V, NB_) \
    gated_norm_kernel<PT, TO, L_, V, POST><<<(int)((long long)T * (NB_)), L_ <= 64 ? 256 : L_, 0, s>>>(                  \
        y, p, z_at, w, n, groups, eps, out_scale, (TO*)out, ldo, col, zero_to)
#define GN_L(PT, TO)                                        \
    if (!q || q > 4096) GN(PT, TO, 256, 0, gb);             \
    else if (q <= 16 && T > 512) GN(PT, TO, 16, 1, gn);     \
    else if (q <= 32 && T > 512) GN(PT, TO, 32, 1, gh);     \
    else if (q <= 64 && T > 512) GN(PT, TO, 64, 1, gw);     \
    else if (q <= 256 && T > 512) GN(PT, TO, 64, 4, gw);    \
    else if (q <= 256) GN(PT, TO, 256, 1, gb);              \
    else if (q <= 1024 && T > 512) GN(PT, TO, 256, 4, gb);  \
    else if (q <= 1024) GN(PT, TO, 1024, 1, gb);            \
    else GN(PT, TO, 1024, 4, gb);
    if (out32) { GN_L(true, float) }
    else if (p.S) { GN_L(true, bf16) }
    else { GN_L(false, bf16) }
#undef GN_L
#undef GN
    return (int)hipGetLastError();
}

// out[t, col : col + n] of rows [T][ldo]; columns past it, up to zero_to, are zeroed.  post: norm, then gate; w [n / groups]
MRSUM_API int mrsum_gated_norm(const float* y, const void* u, int S, int ld, int T, int z_at, const float* w, int n,
                               int groups, float eps, float out_scale, void* out, int out32, int ldo, int col, int zero_to,
                               int post, int rows, hipStream_t s) {
    if (T <= 0) return 0;
    if (groups <= 0 || n % groups || z_at % 8 || ld % 8 || z_at + n > ld || col % 8 || col + n > ldo || ldo % 8 ||
        zero_to > ldo || rows < T || (out32 && S < 1))
        return (int)hipErrorInvalidValue;
    const ProjSrc p{u, S, (size_t)rows * ld, ld};  // slabs of ``rows`` rows, of which u points at the first used
    if (post) return launch_gated_norm<true>(y, p, T, z_at, w, n, groups, eps, out_scale, out, out32, ldo, col, zero_to, s);
    return launch_gated_norm<false>(y, p, T, z_at, w, n, groups, eps, out_scale, out, out32, ldo, col, zero_to, s);
}
