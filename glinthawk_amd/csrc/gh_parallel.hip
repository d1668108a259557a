// Input side of a parallel layer: one product of the layer's input with everything that reads it (queries, keys that are also the values,
// a gate per head, gate and up of the feed-forward), and one kernel behind it that brings each part to where it is read.  Where the
// feed-forward is so large that its product fills the chip without a split of K, few rows take the launch that applies the gate itself for
// it, and the product and the kernel serve the heads alone.
//
// work-group  256 threads on one row: first the heads, L lanes a head with V neighbouring elements each, then the feed-forward's columns
// heads       a query is divided by its root mean square and multiplied by its position's temperature; a key goes to the cache as it is,
//             1 / rms of it beside.  Sums, factors and gates are fp32.
#include "gh_product.h"
#include "gh_window.h"

#include <algorithm>
#include <type_traits>

namespace gh {

// gh_gemm.hip: gate, up and SiLU in one launch where the streaming kernel runs without a K split; *done = false: nothing was launched
int gemm_gate_one_launch( void* hb, uint64_t hb_stride, const void* x, const void* w13, uint64_t s, uint64_t hidden, uint64_t b, gh_dtype dt, hipStream_t st, bool* done );

namespace {

struct ParallelCols
{
  uint32_t g;  // first column of the head gates
  uint32_t ff; // first column of the feed-forward's gate
  uint32_t r;  // columns of the product
};

ParallelCols parallel_cols( const gh_window_attn* a, bool gated, uint64_t ff )
{
  ParallelCols c;
  c.g = ( a->heads + a->kv_heads ) * a->dim;
  c.ff = ( c.g + ( gated ? a->heads : 0 ) + 7 ) / 8 * 8;
  c.r = (uint32_t)( ( c.ff + 2 * ff + 7 ) / 8 * 8 );
  return c;
}

template<typename E>
struct ParallelOut
{
  E* q;
  float* head_gates;
  E* hidden;
  uint64_t hidden_stride;
  uint32_t ff;
  int act;
};

template<typename E>
__device__ __forceinline__ float sigmoid( float z )
{
  return 1.0f / ( 1.0f + ( sizeof( E ) == 4 ? expf( -z ) : __expf( -z ) ) );
}

template<int L>
__device__ __forceinline__ float lanes_sum( float v )
{
  v = row16_sum( v );
  if constexpr ( L >= 32 ) {
    v += __shfl_xor( v, 16 );
  }
  if constexpr ( L >= 64 ) {
    v += __shfl_xor( v, 32 );
  }
  return v;
}

// V elements to neighbouring places; V * sizeof(E) is a multiple of 8 bytes, or V is 1
template<typename E, int V>
__device__ __forceinline__ void store_run( E* dst, const float v[V] )
{
  if constexpr ( V == 1 ) {
    *dst = from_f32<E>( v[0] );
  } else {
    union
    {
      E e[V];
      uint2 half[V * sizeof( E ) / 8];
      uint4 full[( V * sizeof( E ) + 15 ) / 16];
    } o;
#pragma unroll
    for ( int i = 0; i < V; i++ ) {
      o.e[i] = from_f32<E>( v[i] );
    }
    if constexpr ( V * sizeof( E ) == 8 ) {
      *reinterpret_cast<uint2*>( dst ) = o.half[0];
    } else {
#pragma unroll
      for ( uint32_t i = 0; i < V * sizeof( E ) / 16; i++ ) {
        reinterpret_cast<uint4*>( dst )[i] = o.full[i];
      }
    }
  }
}

template<int V, typename View>
__device__ __forceinline__ void load_run( float v[V], const View& y, uint64_t row, uint64_t col )
{
  if constexpr ( V == 8 ) {
    y.at8( v, row, col );
  } else if constexpr ( V == 4 ) {
    const float4 a = y.at4( row, col );
    v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w;
  } else {
    v[0] = y.at( row, col );
  }
}

// L lanes a head with NV runs of V elements each (V 8: one run, head size a multiple of 8; V 1: 64 lanes, eight); VF columns of the
// feed-forward a thread
template<typename E, typename View, int V, int L, int VF>
__global__ __launch_bounds__( 256 ) void parallel_rows_kernel( ParallelOut<E> o, View y, WindowRows wr, WindowShape s, gh_unit_heads u, ParallelCols cols, uint32_t head_blocks,
                                                               uint32_t blocks )
{
  constexpr int NV = V == 8 ? 1 : 8;
  const uint64_t row = blockIdx.x / blocks;
  const uint32_t part = blockIdx.x % blocks;
  const uint32_t ctx = (uint32_t)( row / wr.n_tokens ), tok = (uint32_t)( row % wr.n_tokens );
  uint8_t* base = static_cast<uint8_t*>( wr.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  if ( part >= head_blocks ) {
    const uint32_t c = ( ( part - head_blocks ) * 256 + threadIdx.x ) * VF;
    if ( c >= o.ff ) {
      return;
    }
    float g[VF], up[VF];
    load_run<VF>( g, y, row, cols.ff + c );
    load_run<VF>( up, y, row, cols.ff + o.ff + c );
#pragma unroll
    for ( int i = 0; i < VF; i++ ) {
      g[i] = activate<E>( g[i], o.act ) * up[i];
    }
    store_run<E, VF>( o.hidden + row * o.hidden_stride + c, g );
    return;
  }

  const uint32_t unit = ( part * 256 + threadIdx.x ) / L, lane = threadIdx.x % L;
  if ( unit >= s.heads + s.kv_heads ) { // (all lanes of a head leave together)
    return;
  }
  const bool is_q = unit < s.heads;
  const uint32_t pos = wr.start_pos[ctx] + tok;
  float v[NV][V], ss = 0.0f;
#pragma unroll
  for ( int n = 0; n < NV; n++ ) {
    const uint32_t at = ( n * L + lane ) * V;
    const bool live = at < s.dim;
    load_run<V>( v[n], y, row, unit * s.dim + ( live ? at : 0 ) );
#pragma unroll
    for ( int i = 0; i < V; i++ ) {
      v[n][i] = live ? v[n][i] : 0.0f; // also what the padding of a head holds
      ss += v[n][i] * v[n][i];
    }
  }
  const float inv = 1.0f / sqrtf( lanes_sum<L>( ss ) / (float)s.dim + u.eps );
  E* dst;
  float factor = 1.0f;
  if ( is_q ) {
    dst = o.q + ( row * s.heads + unit ) * s.dpad;
    factor = inv;
    if ( u.temp_every != 0 ) {
      factor *= 1.0f + u.temp_coef * logf( (float)( ( pos + 1 ) / u.temp_every ) + 1.0f );
    }
    if ( o.head_gates != nullptr && lane == 0 ) {
      o.head_gates[row * s.heads + unit] = sigmoid<E>( y.at( row, cols.g + unit ) );
    }
  } else {
    const uint32_t g = unit - s.heads;
    dst = reinterpret_cast<E*>( base + wr.offset ) + (uint64_t)pos * s.row_elems() + g * s.dpad;
    if ( lane == 0 ) {
      reinterpret_cast<float*>( base + wr.factors )[factor_index( pos, g, s.kv_heads )] = inv;
    }
  }
#pragma unroll
  for ( int n = 0; n < NV; n++ ) {
    const uint32_t at = ( n * L + lane ) * V;
    if ( at < s.dpad ) {
#pragma unroll
      for ( int i = 0; i < V; i++ ) {
        v[n][i] *= factor;
      }
      store_run<E, V>( dst + at, v[n] );
    }
  }
}

bool aligned16( const void* p ) { return ( reinterpret_cast<uintptr_t>( p ) & 15u ) == 0; }

template<typename E, typename View>
int launch_parallel( const ParallelOut<E>& o, const View& y, const WindowRows& wr, const WindowShape& s, const gh_unit_heads& u, const ParallelCols& cols, uint64_t rows,
                     hipStream_t st )
{
  constexpr int WIDE = std::is_same_v<View, ProductView<__bf16>> ? 8 : 4;
  const bool head_runs = s.dim % 8 == 0 && aligned16( y.data ) && aligned16( o.q );
  const bool ff_runs = o.ff % WIDE == 0 && o.hidden_stride % 8 == 0 && aligned16( y.data ) && aligned16( o.hidden );
  auto launch = [&]( auto v_tag, auto l_tag, auto vf_tag ) -> int {
    constexpr int V = decltype( v_tag )::value, L = decltype( l_tag )::value, VF = decltype( vf_tag )::value;
    const uint32_t head_blocks = ( ( s.heads + s.kv_heads ) * L + 255 ) / 256;
    const uint32_t blocks = head_blocks + ( o.ff + 256 * VF - 1 ) / ( 256 * VF );
    GH_REQUIRE( rows * blocks < ( 1ull << 31 ), "gh_matmul_parallel: grid too large" );
    parallel_rows_kernel<E, View, V, L, VF><<<(unsigned)( rows * blocks ), 256, 0, st>>>( o, y, wr, s, u, cols, head_blocks, blocks );
    GH_LAUNCH_CHECK();
    return GH_OK;
  };
  auto with_ff = [&]( auto v_tag, auto l_tag ) -> int {
    return ff_runs ? launch( v_tag, l_tag, std::integral_constant<int, WIDE> {} ) : launch( v_tag, l_tag, std::integral_constant<int, 1> {} );
  };
  if ( !head_runs ) {
    return with_ff( std::integral_constant<int, 1> {}, std::integral_constant<int, 64> {} );
  }
  const std::integral_constant<int, 8> v8 {};
  if ( s.dim <= 128 ) {
    return with_ff( v8, std::integral_constant<int, 16> {} );
  }
  if ( s.dim <= 256 ) {
    return with_ff( v8, std::integral_constant<int, 32> {} );
  }
  return with_ff( v8, std::integral_constant<int, 64> {} );
}

} // namespace
} // namespace gh

using namespace gh;

extern "C" {

uint64_t gh_parallel_weight_rows( const gh_window_attn* a, int gated, uint64_t ff, uint64_t* ff_row )
{
  const ParallelCols c = parallel_cols( a, gated != 0, ff );
  *ff_row = c.ff;
  return c.r;
}

int gh_matmul_parallel( void* q, float* head_gates, void* hidden, uint64_t hidden_stride, const void* x, const void* w, uint64_t width, const gh_window_attn* a,
                        const gh_unit_heads* u, uint64_t ff, int activation, void* const* context_rows_dev, uint64_t cache_offset, uint64_t factor_offset,
                        const uint32_t* start_pos_dev, uint64_t batch, uint32_t n_tokens, gh_dtype dt, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  const uint64_t rows = batch * n_tokens;
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( q && x && w && a && u && context_rows_dev && start_pos_dev && ( hidden || ff == 0 ), "gh_matmul_parallel: NULL pointer" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_matmul_parallel: unsupported dtype %d", (int)dt );
  GH_REQUIRE( window_shape_ok( a ) && a->values_are_keys && width > 0 && width < ( 1ull << 31 ) && rows < ( 1ull << 31 ) && ff < ( 1ull << 29 ) && hidden_stride >= ff
                && cache_offset % 16 == 0 && factor_offset % 16 == 0,
              "gh_matmul_parallel: bad shape" );
  GH_REQUIRE( activation == GH_ACT_SILU || activation == GH_ACT_GELU_TANH, "gh_matmul_parallel: unknown activation %d", activation );
  const WindowShape s = window_shape( a );
  ParallelCols cols = parallel_cols( a, head_gates != nullptr, ff );
  hipStream_t st = as_stream( stream );
  if ( ff > 0 && dt == GH_BF16 && activation == GH_ACT_SILU ) {
    bool done = false;
    if ( int rc = gemm_gate_one_launch( hidden, hidden_stride, x, static_cast<const __bf16*>( w ) + cols.ff * width, width, ff, rows, dt, st, &done ) ) {
      return rc;
    }
    if ( done ) {
      ff = 0;
      cols.r = cols.ff;
    }
  }
  Product y;
  if ( int rc = make_product( x, w, width, cols.r, rows, dt, false, st, &y ) ) {
    return rc;
  }
  const WindowRows wr { context_rows_dev, cache_offset, factor_offset, start_pos_dev, n_tokens };
  return with_product( dt, y, [&]( auto tag, auto view ) -> int {
    using E = decltype( tag );
    const ParallelOut<E> o { static_cast<E*>( q ), head_gates, static_cast<E*>( hidden ), hidden_stride, (uint32_t)ff, activation };
    return launch_parallel<E>( o, view, wr, s, *u, cols, rows, st );
  } );
}

} // extern "C"
