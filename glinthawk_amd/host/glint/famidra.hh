// Driver of the Famidra design for the hip target: weights, scratch, and the ops of one step.
//
//   embedding        x = embed[token] + pos[position]
//   pass of the loop x = W_in [x; x0] + step[t], in front of the first layer of every pass
//   mixer            h = norm1(x); mLSTM or windowed attention on h; x += norm1b( W_o . )
//   feed-forward     h = norm2(x); x += norm2b( W_down (gelu(W_gate h) * (W_up h)) ), biases on all three
//   output           logits = embed . final_norm(x) * logit_scale (fp32) -> (Gumbel noise if temperature > 0) -> argmax
//
// The residual stream x is fp32.  Every projection is fused with what follows it up to the next product's input (see gh_stream_step), so
// a layer is a handful of launches in either dtype.  The design is hosted whole: a pass needs the embedding output again, so a cut
// between nodes would carry two rows a token.
#pragma once

#include <algorithm>
#include <string>
#include <vector>

#include "glint/design_driver.hh"
#include "glint/famidra_config.hh"

namespace glint {

template<typename DType, typename Context = hip::LayeredContext>
class Famidra : public DesignDriver<configs::Famidra, DType, Context>
{
  using Base = DesignDriver<configs::Famidra, DType, Context>;
  using Base::DT;
  using Base::ops_, Base::x_, Base::h_, Base::final_norm_, Base::settings_, Base::options_, Base::max_start_;
  using Base::tokens_dev, Base::pos_dev, Base::contexts_dev, Base::no_step, Base::lead_to, Base::lead_out;

public:
  Famidra( const FamidraConfig& config, DesignSettings settings, const ModelOptions options = {} )
    : Base( { config.width, config.vocab, config.max_positions, config.eps, 0.0f }, std::move( settings ), options, plan( config ) )
    , config_( config )
    , runs_( config_.runs() )
  {
    describe_layers();
    this->allocate();
  }

  static ContextPlan plan( const FamidraConfig& config )
  {
    ContextPlan p( config.max_positions );
    for ( const auto& run : config.runs() ) {
      const auto& layer = config.layers[run.layer];
      if ( layer.mlstm ) {
        const gh_mlstm m = mlstm_shape( *layer.mlstm, config.eps );
        p.add_state( gh_mlstm_state_bytes( &m ) );
      } else {
        const gh_window_attn a = window_shape( *layer.attention );
        p.add_rows( gh_window_row_bytes( &a, DT ) );
      }
    }
    return p;
  }

  const FamidraConfig& config() const { return config_; }
  size_t n_runs() const override { return runs_.size(); }

private:
  struct Layer
  {
    DType *norm1 {}, *norm1b {}, *norm2 {}, *norm2b {};
    DType *mix_in {}, *mix_bias {}, *mix_out {}; // projections in front of and behind the mixer
    DType *q_norm {}, *k_norm {}, *head_norm {}, *bias_i {}, *bias_f {};
    DType *gate_up {}, *gate_up_bias {}, *down {}, *down_bias {};
    float* distance_bias {};
    uint64_t mixed_cols {};       // columns of the mixer's output
    gh_mlstm mlstm {};
    gh_window_attn attention {};
  };

  static gh_mlstm mlstm_shape( const MlstmConfig& m, const float eps ) { return { m.heads, m.dim, m.vdim, m.gate_cap, eps }; }
  static gh_window_attn window_shape( const WindowAttentionConfig& a )
  {
    // distances beyond the table's last row all have its bias
    const uint32_t n_dist = static_cast<uint32_t>( std::ceil( a.bias_max ) ) + 1;
    return { a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, n_dist, a.scale, 0 };
  }
  static std::string prefix( const size_t layer ) { return "l" + std::to_string( layer ) + "."; }

  void describe_layers()
  {
    layers_.resize( config_.layers.size() );
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      const auto& c = config_.layers[l];
      if ( c.mlstm ) {
        layers_[l].mlstm = mlstm_shape( *c.mlstm, config_.eps );
        layers_[l].mixed_cols = (uint64_t)c.mlstm->heads * c.mlstm->vdim;
        mixed_max_ = std::max( mixed_max_, layers_[l].mixed_cols );
      } else {
        layers_[l].attention = window_shape( *c.attention );
        layers_[l].mixed_cols = (uint64_t)c.attention->heads * c.attention->vdim;
        mixed_max_ = std::max( mixed_max_, layers_[l].mixed_cols );
        query_max_ = std::max( query_max_, gh_window_query_elements( &layers_[l].attention ) );
      }
      ff_max_ = std::max<uint64_t>( ff_max_, c.ff );
    }
  }

  void lay_out( WeightCursor<DType>& cursor ) override
  {
    const uint64_t width = config_.width;
    embed_ = cursor.alone( "embed", { config_.vocab, width } );
    pos_ = cursor.alone( "pos", { config_.max_positions, width } );
    final_norm_ = cursor.alone( "final.norm", { width }, 1.0f );
    if ( config_.looped ) {
      loop_in_ = cursor.alone( "loop.in", { width, 2 * width } );
      loop_step_ = cursor.alone( "loop.step", { config_.loop_times, width } );
    }
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      auto& w = layers_[l];
      const auto& c = config_.layers[l];
      const std::string p = prefix( l );
      w.norm1 = cursor.alone( p + "norm1", { width }, 1.0f );
      w.norm1b = cursor.alone( p + "norm1b", { width }, 1.0f );
      if ( c.mlstm ) {
        const uint64_t hd = (uint64_t)c.mlstm->heads * c.mlstm->dim, hv = (uint64_t)c.mlstm->heads * c.mlstm->vdim, h = c.mlstm->heads;
        uint64_t gate_row = 0;
        const uint64_t rows = gh_mlstm_weight_rows( &w.mlstm, &gate_row );
        w.mix_in = cursor.alone( p + "mix.q", { hd, width } );
        cursor.tensor( p + "mix.k", { hd, width } );
        cursor.tensor( p + "mix.v", { hv, width } );
        cursor.tensor( p + "mix.g", { hv, width } );
        cursor.take( ( gate_row - 2 * hd - 2 * hv ) * width );
        cursor.tensor( p + "mix.i", { h, width } );
        cursor.tensor( p + "mix.f", { h, width } );
        cursor.take( ( rows - gate_row - 2 * h ) * width );
        w.bias_i = cursor.alone( p + "mix.i.b", { h } );
        w.bias_f = cursor.alone( p + "mix.f.b", { h } );
        w.head_norm = cursor.alone( p + "mix.norm", { hv }, 1.0f );
        w.mix_out = cursor.alone( p + "mix.o", { width, hv } );
      } else {
        const auto& a = *c.attention;
        const uint64_t q = (uint64_t)a.heads * a.dim, k = (uint64_t)a.kv_heads * a.dim, v = (uint64_t)a.kv_heads * a.vdim;
        w.mix_in = cursor.alone( p + "mix.q", { q, width } );
        cursor.tensor( p + "mix.k", { k, width } );
        cursor.tensor( p + "mix.v", { v, width } );
        w.mix_bias = cursor.alone( p + "mix.q.b", { q } );
        cursor.tensor( p + "mix.k.b", { k } );
        cursor.tensor( p + "mix.v.b", { v } );
        w.q_norm = cursor.alone( p + "mix.q.norm", { q }, 1.0f );
        w.k_norm = cursor.alone( p + "mix.k.norm", { k }, 1.0f );
        w.mix_out = cursor.alone( p + "mix.o", { width, (uint64_t)a.heads * a.vdim } );
        cursor.align();
        // the bias of every distance up to the table's end, fp32, one row a head
        w.distance_bias = reinterpret_cast<float*>( cursor.take( (uint64_t)w.attention.heads * w.attention.n_dist * sizeof( float ) / sizeof( DType ) ) );
      }
      if ( c.ff > 0 ) {
        w.norm2 = cursor.alone( p + "norm2", { width }, 1.0f );
        w.norm2b = cursor.alone( p + "norm2b", { width }, 1.0f );
        w.gate_up = cursor.alone( p + "mlp.gate", { c.ff, width } );
        cursor.tensor( p + "mlp.up", { c.ff, width } );
        w.gate_up_bias = cursor.alone( p + "mlp.gate.b", { c.ff } );
        cursor.tensor( p + "mlp.up.b", { c.ff } );
        w.down = cursor.alone( p + "mlp.down", { width, c.ff } );
        w.down_bias = cursor.alone( p + "mlp.down.b", { width } );
      }
    }
  }

  std::string load_tables( const SafeTensors& file ) override
  {
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      if ( !config_.layers[l].attention ) {
        continue;
      }
      const std::string name = prefix( l ) + "mix.rel";
      const auto* rel = file.find( name );
      const uint32_t heads = config_.layers[l].attention->heads;
      if ( rel == nullptr || rel->shape.size() != 2 || rel->shape[0] == 0 || rel->shape[1] != heads || rel->dtype == "I32" ) {
        return "tensor " + name + " is missing or does not have a column per head";
      }
      std::vector<float> table( rel->elements() );
      for ( uint64_t i = 0; i < table.size(); i++ ) {
        table[i] = SafeTensors::value( *rel, i );
      }
      set_distance_bias( l, table, static_cast<uint32_t>( rel->shape[0] ) );
    }
    return {};
  }

  void set_distance_bias( const size_t l, const std::vector<float>& table, const uint32_t table_rows )
  {
    const auto& a = layers_[l].attention;
    std::vector<float> by_distance( (uint64_t)a.heads * a.n_dist );
    for ( uint32_t n = 0; n < a.n_dist; n++ ) {
      const uint32_t row = distance_bucket( n, table_rows, config_.layers[l].attention->bias_max );
      for ( uint32_t h = 0; h < a.heads; h++ ) {
        by_distance[(uint64_t)h * a.n_dist + n] = table[(uint64_t)row * a.heads + h];
      }
    }
    GLINT_GH( gh_memcpy( layers_[l].distance_bias, by_distance.data(), by_distance.size() * sizeof( float ), GH_HOST_TO_DEVICE, 0, ops_.stream() ) );
  }

  void randomize_tables( uint64_t seed ) override
  {
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      if ( config_.layers[l].attention ) {
        const auto& a = layers_[l].attention;
        GLINT_GH( gh_fill_normal( layers_[l].distance_bias, (uint64_t)a.heads * a.n_dist, 0.0f, options_.weight_std, seed++, GH_F32, ops_.stream() ) );
      }
    }
  }

  void allocate_layer_scratch( const uint64_t rows ) override
  {
    mixed_ = ops_.device_allocate( rows * mixed_max_ * sizeof( DType ) );
    q_ = ops_.device_allocate( std::max<uint64_t>( rows * query_max_, 8 ) * sizeof( DType ) );
    hidden_ = ops_.device_allocate( std::max<uint64_t>( rows * ff_max_, 8 ) * sizeof( DType ) );
    if ( config_.looped ) {
      cat_ = ops_.device_allocate( rows * 2 * config_.width * sizeof( DType ) );
    }
  }

  // what run k (or the output behind the last run) reads: the next product's input leaves with the residual update in front of it
  void lead_into( gh_stream_step& step, const size_t k, const bool all_rows_classified ) const
  {
    if ( k == runs_.size() ) {
      if ( all_rows_classified ) {
        lead_out( step );
      }
    } else if ( runs_[k].first_of_pass ) {
      step.out = cat_.get();
      step.out_stride = 2ull * config_.width;
    } else {
      lead_to( step, layers_[runs_[k].layer].norm1 );
    }
  }

  void run_layers( const uint64_t batch, const uint32_t n_tokens, const bool all_rows_classified, float* residuals_out ) override
  {
    const uint64_t rows = batch * n_tokens, width = config_.width;
    const gh_stream stream = ops_.stream();
    DType* x0 = config_.looped ? cat_.get() + width : nullptr;
    GLINT_GH( gh_embed_positions( x_.get(), tokens_dev(), pos_dev(), batch, n_tokens, embed_, pos_, width, config_.vocab, config_.max_positions, x0, 2 * width, DT,
                                  stream ) );
    {
      gh_stream_step first = no_step();
      lead_into( first, 0, all_rows_classified );
      GLINT_GH( gh_stream_out( x_.get(), width, rows, &first, DT, stream ) );
    }
    for ( size_t k = 0; k < runs_.size(); k++ ) {
      const auto& run = runs_[k];
      const auto& w = layers_[run.layer];
      const auto& part = settings_.plan->parts[k];
      if ( run.first_of_pass ) {
        gh_stream_step s = no_step();
        s.add = loop_step_ + (uint64_t)run.pass * width;
        lead_to( s, w.norm1 );
        GLINT_GH( gh_matmul_stream( x_.get(), cat_.get(), loop_in_, 2 * width, width, rows, &s, DT, stream ) );
      }
      if ( config_.layers[run.layer].mlstm ) {
        GLINT_GH( gh_mlstm_forward( mixed_.get(), h_.get(), w.mix_in, width, &w.mlstm, w.bias_i, w.bias_f, w.head_norm, contexts_dev(), part.offset, pos_dev(), batch,
                                    n_tokens, DT, stream ) );
      } else {
        GLINT_GH( gh_matmul_window_append( q_.get(), h_.get(), w.mix_in, w.mix_bias, width, &w.attention, w.q_norm, w.k_norm, config_.eps, contexts_dev(),
                                           part.offset, pos_dev(), batch, n_tokens, DT, stream ) );
        GLINT_GH( gh_attn_window( mixed_.get(), w.mixed_cols, nullptr, q_.get(), &w.attention, w.distance_bias, contexts_dev(), part.offset, 0, pos_dev(), batch,
                                  n_tokens, max_start_, DT, stream ) );
      }
      const bool ff = config_.layers[run.layer].ff > 0;
      gh_stream_step s = no_step();
      s.post_norm = w.norm1b;
      s.accumulate = 1;
      if ( ff ) {
        lead_to( s, w.norm2 );
      } else {
        lead_into( s, k + 1, all_rows_classified );
      }
      GLINT_GH( gh_matmul_stream( x_.get(), mixed_.get(), w.mix_out, w.mixed_cols, width, rows, &s, DT, stream ) );
      if ( ff ) {
        const uint64_t hidden = config_.layers[run.layer].ff;
        GLINT_GH( gh_matmul_gate( hidden_.get(), h_.get(), w.gate_up, w.gate_up_bias, width, hidden, rows, GH_ACT_GELU_TANH, DT, stream ) );
        gh_stream_step d = no_step();
        d.bias = w.down_bias;
        d.post_norm = w.norm2b;
        d.accumulate = 1;
        lead_into( d, k + 1, all_rows_classified );
        GLINT_GH( gh_matmul_stream( x_.get(), hidden_.get(), w.down, hidden, width, rows, &d, DT, stream ) );
      }
      this->copy_residuals( residuals_out, k, rows );
    }
  }

  void classify( const uint64_t n ) override
  {
    GLINT_GH( gh_matmul_scaled( this->logits_.get(), h_.get(), embed_, config_.width, config_.vocab, n, config_.logit_scale, DT, ops_.stream() ) );
  }

  FamidraConfig config_;
  std::vector<FamidraConfig::Run> runs_;
  std::vector<Layer> layers_ {};
  uint64_t mixed_max_ { 0 }, query_max_ { 0 }, ff_max_ { 0 };
  DType *embed_ {}, *pos_ {}, *loop_in_ {}, *loop_step_ {};
  typename Base::Operations::DeviceUniquePtr mixed_ {}, q_ {}, hidden_ {}, cat_ {};
};

} // namespace glint
